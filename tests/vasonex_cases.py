"""Small Vasonex configurations, helpers and an engine harness shared by the host and GPU tests.  Sizes are deliberately
awkward: key and value sizes that differ, one and several query heads per key head, head sizes that are no multiples of 8,
windows shorter and longer than a page, kept tokens fewer and more than a window, none, and more than a request has,
rotations over all, part and none of a head, one expert and several per token, shared experts of the experts' size, of
another size and absent, layers without a feed-forward, weights used by one to three layers, also through a chain."""

import contextlib
import copy

import torch

from oracle import vasonex as O


def attention(heads, kv_heads, dim, vdim, scale, window=None, keep=None, rot=None, scaling=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
        if keep is not None:
            m["mask"]["keep_first"] = keep
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def config(vocab, width, layers, eps=1e-5):
    """layers: (mixer, mlp) pairs, or the number of an earlier layer whose weights are used again."""
    specs = []
    for entry in layers:
        if isinstance(entry, int):
            specs.append(dict(copy.deepcopy(specs[entry]), weights_of=entry))
        else:
            specs.append({"type": "attention", "mixer": copy.deepcopy(entry[0]), "mlp": copy.deepcopy(entry[1])})
    return {"architecture": "Vasonex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": specs}


def mixed_config():
    """Three query heads per key head; a window of 12 tokens beside 3 kept ones against pages of 16; a mixture first, two of
    five experts, a shared expert of another size; the mixture's weights in three layers (one through a chain), the dense
    layer's in two; one layer without a feed-forward."""
    return config(150, 96, [
        (attention(6, 2, 16, 24, 0.3, 12, 3, (500.0, 8), (4.0, 1.0, 4.0, 32)), moe(5, 2, 24, 40)),
        (attention(3, 3, 24, 8, 0.25, 20, 5, (300.0, 24)), dense(56)),
        0,
        (attention(2, 1, 32, 16, 0.2, 33, 40), None),
        1,
        2,
    ], eps=1e-4)


def odd_config():
    """Nothing is a multiple of 8: the general kernels; a single head; one pair rotated; all experts chosen, of sizes that
    leave the vector paths out; no kept tokens."""
    return config(77, 100, [
        (attention(1, 1, 20, 12, 0.4, 9, 0, (50.0, 2)), dense(36)),
        (attention(3, 1, 12, 20, 0.3, 7, 2, (1000.0, 6), (2.0, 0.5, 3.0, 50)), moe(3, 3, 20, 12)),
        (attention(2, 2, 10, 6, 0.35), moe(2, 1, 28)),
        1,
    ], eps=1e-6)


def aligned_config():
    """Sizes in multiples of 16 and 32, where the 16-bit engine takes its matrix-core kernels; a window of one page and
    one of two and a half; four query heads per key head; a shared expert of the experts' size."""
    return config(256, 128, [
        (attention(8, 2, 32, 32, 32 ** -0.5, 16, 4, (10000.0, 16), (8.0, 1.0, 4.0, 256)), moe(8, 2, 64, 64)),
        (attention(4, 4, 64, 16, 0.125, 40, 10, (10000.0, 64), (4.0, 1.0, 2.0, 64)), dense(192)),
        0,
        1,
    ])


def plain_config():
    """One expert per token among two, a shared expert of the same size; heads of 128 with eight query heads on one key
    head; a window of one token beside sixteen kept ones; no window at all; window and kept tokens longer than a request."""
    return config(90, 64, [
        (attention(8, 1, 128, 40, 0.09, 1, 16, (20000.0, 32)), moe(2, 1, 32, 32)),
        (attention(2, 2, 16, 16, 0.25, 500, 600, (100.0, 16)), None),
        (attention(4, 2, 24, 24, 0.2), dense(48)),
    ])


def random_config(seed: int):
    """A configuration drawn from a seed: three to seven layers, some using earlier ones' weights, all sizes, windows and
    constants independent."""
    import random
    rng = random.Random(seed)
    layers = []
    for i in range(rng.randint(3, 7)):
        if i and rng.random() < 0.4:
            layers.append(rng.randrange(i))
            continue
        G = rng.choice([1, 2, 3, 4])
        d = rng.choice([16, 20, 24, 32, 48, 64, 80])
        rot = rng.choice([0, 2, d // 2, d]) // 2 * 2
        mixer = attention(G * rng.choice([1, 2, 3, 4]), G, d, rng.choice([8, 12, 16, 24, 40, 64]),
                          rng.choice([d ** -0.5, 0.1, 0.3]), window=rng.choice([None, 5, 16, 33, 64, 70]),
                          keep=rng.choice([None, 0, 1, 6, 16, 40]), rot=(rng.choice([100.0, 1e4, 1e6]), rot) if rot else None,
                          scaling=rng.choice([None, (2.0, 1.0, 4.0, 64), (8.0, 1.0, 3.0, 200), (4.0, 0.5, 2.0, 20)]))
        kind = rng.random()
        ff = rng.choice([16, 20, 40, 64])
        if kind < 0.45:
            E = rng.choice([2, 3, 7, 12])
            mlp = moe(E, rng.randint(1, min(E, 3)), ff, rng.choice([None, ff, 2 * ff]))
        else:
            mlp = dense(rng.choice([36, 64, 128])) if kind < 0.9 else None
        layers.append((mixer, mlp))
    return config(rng.choice([97, 250, 300]), rng.choice([64, 72, 100, 144, 192]), layers, eps=rng.choice([1e-5, 1e-6, 1e-3]))


def random_checkpoint(cfg, seed=0):
    return O.random_weights(cfg, seed)


def engine_config(cfg_json, weights, dtype, blocks=16, slots=4, block_size=16, **kw):
    """The engine's Config for an in-memory checkpoint of one of the configurations above."""
    from byox_vllm_amd.config import Config
    from byox_vllm_amd.models.vasonex import vasonex_config
    hf = vasonex_config(cfg_json, dtype=dtype)
    return Config("synthetic", hf_config=hf, state_dict=weights, kvcache_block_size=block_size, num_kvcache_blocks=blocks,
                  max_num_seqs=slots, num_state_slots=slots, enforce_eager=True, max_num_batched_tokens=1 << 20,
                  max_model_len=1 << 20, **kw)


class Engine:
    """ModelRunner + Scheduler of one configuration, replaying schedules of (request name, token count) steps."""

    def __init__(self, cfg_json, weights, dtype, blocks=16, slots=4, block_size=16):
        from byox_vllm_amd.engine.model_runner import ModelRunner
        from byox_vllm_amd.engine.scheduler import Scheduler
        self.config = engine_config(cfg_json, weights, dtype, blocks=blocks, slots=slots, block_size=block_size)
        self.runner = ModelRunner(self.config, 0, None)
        self.scheduler = Scheduler(self.config)
        self.block_size = block_size
        self.rows, self.moe_calls = [], 0        # (request, position) of the step's rows; mixtures run so far in it
        self.forced = None                       # request -> experts its tokens are to take (ForcedRoutes)

    def replay(self, requests: dict, schedule: list):
        with ForcedRoutes(self, self.forced) if self.forced is not None else contextlib.nullcontext():
            return self._replay(requests, schedule)

    def _replay(self, requests: dict, schedule: list):
        """requests: name -> token list; schedule: steps of [(name, count)].  Logits of every position, per request.
        A request ends (and gives back pages and slot) with the step that brings its last token."""
        from byox_vllm_amd.engine.sequence import Sequence
        live, at, out = {}, {n: 0 for n in requests}, {n: [] for n in requests}
        for step in schedule:
            plan = []
            for name, count in step:
                piece = requests[name][at[name]: at[name] + count]
                if name not in live:
                    live[name] = Sequence(piece, self.block_size)
                    self.scheduler.add(live[name])
                else:
                    live[name].extend_tokens(piece)
                plan.append((live[name], count))
                at[name] += count
            self.rows = [(name, at[name] - count + i) for name, count in step for i in range(count)]
            self.moe_calls = 0
            self.scheduler.commit(plan)
            logits = self.runner.run_portions(plan, want=[list(range(c)) for _, c in plan]).cpu()
            self.scheduler.advance(plan, [None] * len(plan))
            row = 0
            for name, count in step:
                out[name].append(logits[row: row + count])
                row += count
                if at[name] == len(requests[name]):
                    self.scheduler.finish(live.pop(name))
        return {n: torch.cat(v) for n, v in out.items()}


class ForcedRoutes:
    """While active, the engine's routers choose the experts the oracle chose (their scores stay the engine's own): a
    router logit of random weights can lie inside the rounding of its 16-bit input, and a token that takes another expert
    is off by much more than rounding.  ``chosen``: request -> per mixture run in order, the experts of every token."""

    def __init__(self, engine, chosen: dict):
        self.engine, self.chosen = engine, chosen

    def __enter__(self):
        from byox_vllm_amd import kernels
        plan = self.plan = kernels.moe_plan

        def forced(logits, experts, top, *rest, **kw):
            call = self.engine.moe_calls
            self.engine.moe_calls += 1
            allowed = torch.zeros(logits.size(0), logits.size(1), dtype=torch.bool)
            allowed[:, experts:] = True
            for i, (name, pos) in enumerate(self.engine.rows):
                allowed[i, self.chosen[name][call][pos]] = True
            return plan(torch.where(allowed.to(logits.device), logits, logits - 1000.0), experts, top, *rest, **kw)
        kernels.moe_plan = forced

    def __exit__(self, *_):
        from byox_vllm_amd import kernels
        kernels.moe_plan = self.plan


def forward_with_routes(tokens, weights, cfg):
    """The oracle's logits and the experts its routers chose, per mixture run [T, top]."""
    chosen, route = [], O.route

    def recording(z, top):
        idx, w = route(z, top)
        chosen.append(idx)
        return idx, w
    O.route = recording
    try:
        return O.forward(tokens, weights, cfg), chosen
    finally:
        O.route = route


def row_errors(got: torch.Tensor, want: torch.Tensor) -> torch.Tensor:
    """Per-row error: difference with its mean taken off, root mean square over the vocabulary, relative to the root
    mean square of the expected logits."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    scale = want.double().pow(2).mean().sqrt()
    return d.pow(2).mean(-1).sqrt() / scale


def row_error(got: torch.Tensor, want: torch.Tensor) -> float:
    return float(row_errors(got, want).max())
