"""Small Zekazen configurations, helpers and an engine harness shared by the host and GPU tests.  Sizes are deliberately
awkward: key and value sizes that differ, one and several query heads per key head, head sizes that are no multiples of 4
or 8, rotations over all, part and none of a head, one to five taps, windows shorter and longer than a page and none, one
group of experts and many, groups of one output, all groups kept, identity outputs that fill groups of their own, cut one,
and are absent, layers without a feed-forward, one expert per token and all."""

import copy

import torch

import vasonex_cases
from oracle import zekazen as O

row_error, row_errors = vasonex_cases.row_error, vasonex_cases.row_errors


def retention(heads, dim, vdim, decay, rot=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    return "retention", m


def attention(heads, kv_heads, dim, vdim, scale, conv, window=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "conv": conv}
    if window:
        m["mask"] = {"size": window}
    return "attention", m


def moe(experts, top, ff, groups=None, identity=0, scale=1.0):
    r = {"experts": experts, "top": top, "identity": identity, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "router": r, "expert": {"ff": ff}}


def config(vocab, width, layers, eps=1e-5):
    return {"architecture": "Zekazen", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": [{"type": kind, "mixer": copy.deepcopy(m), "mlp": copy.deepcopy(mlp)} for (kind, m), mlp in layers]}


def mixed_config():
    """Attention first; a window of 12 tokens against pages of 16; half of a head rotated; groups cut by the identity
    outputs; two layers without a feed-forward."""
    return config(150, 96, [
        (attention(6, 2, 16, 24, 0.5, 4, 12), moe(7, 3, 24, (3, 2), 2, 1.7)),
        (retention(3, 24, 40, (0.9, 0.97, 0.5), (500.0, 8)), moe(4, 2, 40, (2, 1), 0, 0.6)),
        (attention(3, 3, 24, 8, 0.25, 2, 20), None),
        (retention(2, 16, 16, (0.995, 0.8), (300.0, 16)), None),
        (attention(2, 1, 32, 16, 0.4, 5, 33), moe(3, 2, 24, None, 3, 1.1)),
    ], eps=1e-4)


def odd_config():
    """Nothing is a multiple of 8, some nothing of 4: the general kernels; a single head; one pair rotated and none; one
    tap (no state); every output chosen; one group; no window."""
    return config(77, 100, [
        (retention(1, 10, 12, (0.93,), (50.0, 2)), moe(3, 3, 20, (1, 1), 0, 2.0)),
        (attention(3, 1, 10, 14, 0.7, 3, 7), moe(2, 3, 28, (3, 3), 1, 0.8)),
        (attention(2, 2, 20, 12, 0.35, 1), None),
        (retention(3, 12, 6, (0.6, 0.999, 0.05)), moe(5, 1, 12, (5, 2), 0, 1.3)),
    ], eps=1e-6)


def aligned_config():
    """Sizes in multiples of 16 and 32, where the 16-bit engine takes its matrix-core kernels and prompts their chunks; two
    rotations in one model; windows of one page and of two and a half; groups of identity outputs only."""
    return config(256, 128, [
        (retention(2, 64, 128, (0.98, 0.998), (10000.0, 64)), moe(8, 3, 64, (3, 2), 4, 1.5)),
        (attention(8, 2, 32, 32, 1.0, 4, 16), moe(6, 2, 64, (4, 2), 2, 2.2)),
        (retention(4, 32, 32, (0.5, 0.9, 0.99, 1.0), (2000.0, 16)), None),
        (attention(4, 4, 64, 16, 0.5, 3, 40), moe(8, 2, 32, (8, 3), 0, 1.0)),
    ])


def plain_config():
    """Heads of 128 and more with eight query heads on one key head; a window of one token; a window longer than a request;
    states wider than one slice of columns; one expert per token beside one identity output."""
    return config(90, 64, [
        (attention(8, 1, 128, 40, 0.09, 2, 1), moe(1, 1, 32, (2, 1), 1, 1.0)),
        (retention(1, 136, 72, (0.97,), (20000.0, 136)), None),
        (attention(2, 2, 16, 16, 0.9, 4, 500), moe(2, 1, 24, None, 0, 3.0)),
        (retention(2, 128, 80, (0.85, 0.9921875), (100.0, 32)), moe(4, 2, 16, (2, 2), 4, 0.5)),
    ])


def random_config(seed: int):
    """A configuration drawn from a seed: two to six layers, all sizes, windows and constants independent."""
    import random
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(2, 6)):
        d, dv = rng.choice([16, 20, 24, 32, 48, 64, 88, 104]), rng.choice([8, 12, 16, 24, 40, 64, 72])
        if rng.random() < 0.5:
            H = rng.choice([1, 2, 3, 5])
            rot = rng.choice([0, 2, d // 2, d]) // 2 * 2
            mixer = retention(H, d, dv, [rng.choice([0.3, 0.9, 1.0 - 2.0 ** -rng.randint(3, 12)]) for _ in range(H)],
                              (rng.choice([100.0, 1e4, 3e5]), rot) if rot else None)
        else:
            G = rng.choice([1, 2, 3, 4])
            mixer = attention(G * rng.choice([1, 2, 3, 4]), G, d, dv, rng.choice([d ** -0.5, 0.3, 1.0]), rng.choice([1, 2, 3, 4, 5]),
                              rng.choice([None, 1, 5, 16, 33, 64, 70]))
        mlp = None
        if rng.random() < 0.8:
            count, size = rng.randint(1, 5), rng.randint(1, 4)
            keep = rng.randint(1, count)
            identity = rng.randint(0, count * size - 1)
            mlp = moe(count * size - identity, rng.randint(1, min(4, keep * size)), rng.choice([16, 20, 40, 64]),
                      (count, keep), identity, rng.choice([0.5, 1.0, 2.4]))
        layers.append((mixer, mlp))
    return config(rng.choice([97, 250, 300]), rng.choice([64, 72, 100, 144, 192]), layers, eps=rng.choice([1e-5, 1e-6, 1e-3]))


def random_checkpoint(cfg, seed=0):
    return O.random_weights(cfg, seed)


def engine_config(cfg_json, weights, dtype, blocks=16, slots=4, block_size=16, **kw):
    """The engine's Config for an in-memory checkpoint of one of the configurations above."""
    from byox_vllm_amd.config import Config
    from byox_vllm_amd.models.zekazen import zekazen_config
    hf = zekazen_config(cfg_json, dtype=dtype)
    return Config("synthetic", hf_config=hf, state_dict=weights, kvcache_block_size=block_size, num_kvcache_blocks=blocks,
                  max_num_seqs=slots, num_state_slots=slots, enforce_eager=True, max_num_batched_tokens=1 << 20,
                  max_model_len=1 << 20, **kw)


class Engine(vasonex_cases.Engine):
    """ModelRunner + Scheduler of one configuration, replaying schedules of (request name, token count) steps."""

    def __init__(self, cfg_json, weights, dtype, blocks=16, slots=4, block_size=16):
        from byox_vllm_amd.engine.model_runner import ModelRunner
        from byox_vllm_amd.engine.scheduler import Scheduler
        self.config = engine_config(cfg_json, weights, dtype, blocks=blocks, slots=slots, block_size=block_size)
        self.runner = ModelRunner(self.config, 0, None)
        self.scheduler = Scheduler(self.config)
        self.block_size = block_size
        self.rows, self.moe_calls = [], 0        # (request, position) of the step's rows; mixtures run so far in it
        self.forced = None                       # request -> outputs its tokens are to take (ForcedRoutes)

    def replay(self, requests: dict, schedule: list):
        if self.forced is None:
            return self._replay(requests, schedule)
        with ForcedRoutes(self, self.forced):
            return self._replay(requests, schedule)


class ForcedRoutes:
    """While active, the engine's routers take the outputs the oracle chose, weighed by the engine's own scores: a router
    logit of random weights can lie inside the rounding of its 16-bit input, and a token that takes another expert is off
    by much more than rounding.  ``chosen``: request -> per mixture in order, the outputs of every token."""

    def __init__(self, engine, chosen: dict):
        self.engine, self.chosen = engine, chosen

    def __enter__(self):
        from byox_vllm_amd import kernels
        self.plan = kernels.moe_plan

        def forced(logits, experts, top, mode, *, identity=0, scale=1.0, self_weight=None, **_):
            call = self.engine.moe_calls
            self.engine.moe_calls += 1
            assert mode == kernels.ROUTE_SOFTMAX and logits.size(1) == experts + identity
            idx = torch.stack([self.chosen[name][call][pos] for name, pos in self.engine.rows]).to(logits.device)
            weights = torch.softmax(logits, -1).gather(1, idx) * scale
            if self_weight is not None:
                self_weight.copy_((weights * (idx >= experts)).sum(1))
            flat = idx.flatten()
            order = torch.sort(flat, stable=True).indices                    # identity outputs come last: no rows
            counts = torch.bincount(flat, minlength=experts + identity)[:experts]
            offsets = torch.cat([counts.new_zeros(1), counts.cumsum(0)]).to(torch.int32)
            slot = torch.empty_like(flat)
            slot[order] = torch.arange(flat.numel(), device=flat.device)
            slot[flat >= experts] = -1
            tokens = (order // top).to(torch.int32)
            return offsets, tokens, None, slot.view(-1, top).to(torch.int32).contiguous(), weights.contiguous()
        kernels.moe_plan = forced

    def __exit__(self, *_):
        from byox_vllm_amd import kernels
        kernels.moe_plan = self.plan


def forward_with_routes(tokens, weights, cfg):
    """The oracle's logits and the outputs its routers chose, per mixture [T, top]."""
    chosen, route = [], O.route

    def recording(z, correction, spec):
        idx, w = route(z, correction, spec)
        chosen.append(idx)
        return idx, w
    O.route = recording
    try:
        return O.forward(tokens, weights, cfg), chosen
    finally:
        O.route = route


def rounding_errors(tokens, weights, cfg, chosen, draws=8):
    """Row errors that relative errors of the size of a bfloat16 rounding cause in the oracle itself (same routes), when
    every normed vector has them: the largest of several draws.  A retention head whose result nearly cancels is blown up to
    unit size by its norm, and so are the roundings ahead of it."""
    route, rms, g = O.route, O.rms, torch.Generator().manual_seed(0)

    def noisy(x, eps):
        y = rms(x, eps)
        return y * (1.0 + (2.0 * torch.rand(y.shape, generator=g, dtype=y.dtype) - 1.0) / 256.0)
    want, errors = O.forward(tokens, weights, cfg), []
    O.rms = noisy
    try:
        for _ in range(draws):
            plan = iter(chosen)

            def same_route(z, correction, spec):
                idx = next(plan)
                return idx, torch.softmax(z, -1).gather(1, idx) * float(spec.get("scale", 1.0))
            O.route = same_route
            errors.append(row_errors(O.forward(tokens, weights, cfg), want))
    finally:
        O.route, O.rms = route, rms
    return torch.stack(errors).max(0).values
