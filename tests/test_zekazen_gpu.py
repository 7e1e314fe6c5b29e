"""Zekazen on the GPU: every mechanism's kernel alone against the plain functions of oracle/zekazen.py, then the engine
(scheduler commit, pages, state slots, run_portions) against the oracle run on each request's whole token list."""

import pytest
import torch

from oracle import zekazen as O
from zekazen_cases import (Engine, aligned_config, engine_config, forward_with_routes, mixed_config, odd_config,
                           plain_config, random_checkpoint, random_config, rounding_errors, row_error, row_errors)

pytestmark = pytest.mark.gpu
DEV = "cuda"
F64 = torch.float64
F32_TOL, BF16_TOL = 2e-4, 6e-2          # engine logits against the float64 oracle (row_error)
SAME_TOL = 2e-5                         # fp32 engine against itself under another schedule
DTYPES = [torch.float32, torch.bfloat16]


def _i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def _close(got, want, tol):
    scale = float(want.abs().max()) + 1e-30
    err = float((got.double().cpu() - want.double()).abs().max()) / scale
    assert err <= tol, err


def _round(t, dtype):
    return t.to(dtype).float()


def _dev(t, dtype=None):
    return None if t is None else t.clone().to(DEV) if dtype is None else t.clone().to(DEV).to(dtype)


def _step(pieces):
    """(cu_q, past_lens, seq_of_token) of one step of (past, count) pieces."""
    cu, owner = [0], []
    for r, (_, n) in enumerate(pieces):
        cu.append(cu[-1] + n)
        owner += [r] * n
    return _i32(cu), _i32([p for p, _ in pieces]), _i32(owner)


# ------------------------------------------------------------------------------------------------ routing
def _scores(z, mode):
    return torch.sigmoid(z) if mode == 2 else torch.softmax(z, -1)


def _plain_route(z, mode, correction, groups, keep, top, scale):
    s = _scores(z, mode)
    c = s + correction
    if groups:
        best = c.view(len(c), groups, -1).max(-1).values
        kept = torch.zeros_like(best, dtype=torch.bool).scatter(1, best.topk(keep, -1).indices, True)
        c = c.masked_fill(~kept.repeat_interleave(c.size(1) // groups, 1), -float("inf"))
    idx = c.topk(top, -1).indices
    w = s.gather(1, idx)
    if mode == 1:
        w = w / (w.sum(-1, keepdim=True) + 1e-20)
    return idx, w * scale


@pytest.mark.parametrize("T,E,identity,top,groups,keep", [
    (1, 12, 0, 3, 4, 2), (7, 5, 3, 4, 4, 3), (64, 6, 2, 2, 2, 1), (65, 40, 20, 6, 5, 2), (300, 1, 7, 2, 8, 3), (5, 1, 1, 1, 2, 1),
    (33, 100, 27, 5, 127, 9), (9, 128, 0, 8, 1, 1), (66, 120, 40, 4, 8, 8), (20, 200, 56, 8, 16, 4), (3, 600, 40, 5, 0, 0)])
@pytest.mark.parametrize("mode", [1, 2, 3])
def test_choice_within_groups_by_corrected_scores(T, E, identity, top, groups, keep, mode):
    """Up to 128 outputs are ranked, more are searched; up to 64 tokens go through one launch.  The correction leaves many
    compared numbers negative: what a dropped group holds must stay below them."""
    from byox_vllm_amd import kernels
    g = torch.Generator().manual_seed(T + E)
    n = E + identity
    z = torch.randn(T, n, generator=g) * 1.5
    correction = torch.randn(n, generator=g) * 0.3 - 0.4
    wide = torch.randn(T, n + 5, generator=g)
    wide[:, 3:3 + n] = z
    self_weight = torch.full((T,), float("nan"), device=DEV) if identity else None
    offsets, tokens, row_weight, slot_of, weights = kernels.moe_plan(
        _dev(wide)[:, 3:3 + n], E, top, mode, identity=identity, correction=_dev(correction), groups=groups, keep_groups=keep,
        scale=1.7, self_weight=self_weight)
    want_idx, want_w = _plain_route(z.double(), mode, correction.double(), groups, keep, top, 1.7)
    offsets, tokens, slot_of, weights = (t.cpu() for t in (offsets, tokens, slot_of, weights))
    _close(weights, want_w, 2e-5)
    assert offsets.numel() == E + 1 and offsets[-1] == (want_idx < E).sum()
    assert torch.equal(offsets, torch.cat([torch.zeros(1, dtype=torch.int64), torch.bincount(want_idx.flatten(), minlength=n)[:E].cumsum(0)]).int())
    assert torch.equal(slot_of < 0, want_idx >= E)
    used = slot_of[slot_of >= 0]
    assert torch.equal(used.sort().values, torch.arange(int(offsets[-1]), dtype=torch.int32))
    for t in range(T):
        for j in range(top):
            s, e = int(slot_of[t, j]), int(want_idx[t, j])
            if s >= 0:
                assert offsets[e] <= s < offsets[e + 1] and tokens[s] == t
                assert abs(float(row_weight[s]) - float(weights[t, j])) == 0.0
    if identity:
        _close(self_weight, (want_w * (want_idx >= E)).sum(1), 2e-5)


def test_ties_go_to_the_lower_output_and_no_number_stays_in_range():
    from byox_vllm_amd import kernels
    z = torch.zeros(3, 12)
    z[1, 7] = float("nan")
    z[2] = float("nan")
    for n in (12, 180):
        rows = torch.zeros(3, n)
        rows[:, :12] = z
        sw = torch.zeros(3, device=DEV)
        offsets, tokens, _, slot_of, weights = kernels.moe_plan(_dev(rows), n - 4, 3, kernels.ROUTE_SOFTMAX, identity=4, groups=4,
                                                                keep_groups=2, correction=torch.zeros(n, device=DEV), self_weight=sw)
        assert torch.allclose(weights[0].cpu(), torch.full((3,), 1.0 / n), rtol=1e-5)
        slots = slot_of.cpu()
        off = offsets.cpu()
        assert [int((off <= s).sum()) - 1 for s in slots[0]] == [0, 1, 2]
        assert int(slots.max()) < 9 and 0 <= int(off[-1]) <= 9


def test_bad_groups_are_refused():
    from byox_vllm_amd import kernels
    z = torch.zeros(2, 12, device=DEV)
    for kw in (dict(groups=5, keep_groups=2), dict(groups=4, keep_groups=5), dict(groups=6, keep_groups=1)):
        with pytest.raises(RuntimeError, match="bad groups"):
            kernels.moe_plan(z, 12, 3, kernels.ROUTE_SOFTMAX, **kw)
    with pytest.raises(RuntimeError, match="mode 0"):
        kernels.moe_plan(z, 12, 3, kernels.ROUTE_CHOSEN, groups=4, keep_groups=2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,identity,top,ff,groups,keep", [(7, 2, 3, 24, 3, 2), (3, 0, 3, 20, 1, 1), (8, 4, 2, 32, 6, 3), (1, 3, 2, 12, 0, 0)])
@pytest.mark.parametrize("T", [1, 37, 130])
def test_mixture_layer_joins_the_residual(dtype, E, identity, top, ff, groups, keep, T):
    """The layer's operands through the launch that adds them to the residual and norms the next input."""
    from byox_vllm_amd.layers.moe import GroupedMixtureOfExperts
    from byox_vllm_amd.layers.postnorm import PreNorm
    width, eps = 72, 1e-4
    g = torch.Generator().manual_seed(T + E)
    spec = {"router": {"experts": E, "identity": identity, "top": top, "scale": 1.3}, "expert": {"ff": ff}}
    if groups:
        spec["router"]["groups"] = {"count": groups, "keep": keep}
    W = {"router": _round(torch.randn(E + identity, width, generator=g) * 0.3, dtype), "correction": torch.randn(E + identity, generator=g) * 0.2}
    for e in range(E):
        for name, shape in (("gate", (ff, width)), ("up", (ff, width)), ("down", (width, ff))):
            W[f"e{e}.{name}"] = _round(torch.randn(*shape, generator=g) * shape[1] ** -0.5, dtype)
    default = torch.get_default_dtype()
    torch.set_default_dtype(dtype)
    try:
        layer = GroupedMixtureOfExperts(width, E, top, ff, identity=identity, groups=groups, keep_groups=keep, scale=1.3).to(DEV)
        norm = PreNorm(width, eps).to(DEV)
    finally:
        torch.set_default_dtype(default)
    layer.router.weight.data.copy_(W["router"])
    layer.correction.data.copy_(W["correction"])
    for e in range(E):
        layer.gate_up.data[e].copy_(torch.cat([W[f"e{e}.gate"], W[f"e{e}.up"]]))
        layer.down.data[e].copy_(W[f"e{e}.down"])
    h, x, w = _round(torch.randn(T, width, generator=g), dtype), torch.randn(T, width, generator=g), _round(1 + 0.2 * torch.randn(width, generator=g), dtype)
    norm.pre.data.copy_(w)
    y = O.moe(h.double(), {k: v.double() for k, v in W.items()}, "", spec)
    new = x.double() + y
    xd = _dev(x)
    pending = (layer(_dev(h, dtype)), norm)
    rows = torch.arange(T - 1, -1, -2, dtype=torch.int32)
    some = norm.begin(xd, pending, _dev(rows))                    # only some rows: the residual stays as it is
    assert torch.equal(xd.cpu(), x)
    tol = 1e-5 if dtype == torch.float32 else 1.5e-2
    _close(some.float(), (O.rms(new, eps) * w.double())[rows.long()], tol)
    out = norm.begin(xd, pending)
    _close(xd, new, tol)
    _close(out.float(), O.rms(new, eps) * w.double(), tol)
    xd = _dev(x)
    PreNorm.settle(xd, pending)
    _close(xd, new, tol)


@pytest.mark.parametrize("n", [98, 1028, 4100])              # through LDS, registers, LDS
def test_identity_share_and_absent_rows_in_the_norm_launch(n):
    from byox_vllm_amd import kernels
    g = torch.Generator().manual_seed(n)
    x, y, h = torch.randn(5, n, generator=g), torch.randn(6, n, generator=g), torch.randn(5, n, generator=g)
    slots = torch.tensor([[0, -1], [-1, -1], [3, 5], [-1, 2], [1, 4]], dtype=torch.int32)
    wt, sw, w = torch.rand(5, 2, generator=g), torch.rand(5, generator=g), torch.randn(n, generator=g)
    new = x.double() + sw.double()[:, None] * h.double()
    for t in range(5):
        for j in range(2):
            if slots[t, j] >= 0:
                new[t] += wt[t, j].double() * y[slots[t, j]].double()
    xd = _dev(x)
    out = kernels.sandwich_norm(xd, _dev(y), None, _dev(w), 1e-3, slot_of=_dev(slots), weights=_dev(wt), self_rows=_dev(h), self_weight=_dev(sw))
    _close(xd, new, 1e-6)
    _close(out, O.rms(new, 1e-3) * w.double(), 2e-6)


# ------------------------------------------------------------------------------------------------ retention
def test_rotation_angles_are_formed_in_double():
    from byox_vllm_amd import kernels
    pos = torch.tensor([0, 1, 77, 5000, 1 << 20])
    freq = torch.tensor([10000.0 ** (-i / 7) for i in range(7)], dtype=F64)
    got = kernels.rotation_table(_dev(pos), _dev(freq))
    a = pos.double()[:, None] * freq
    assert float((got.cpu().double() - torch.cat([a.cos(), a.sin()], 1)).abs().max()) < 1e-7


def _memory(proj, offs, schedule, H, d, dv, decay, rot, freq_base, **kw):
    """Requests (one token list of projections each) through nv_matrix_memory in the steps of ``schedule``
    ([(request, count)]); -> outputs per request.  Slots start as NaN."""
    from byox_vllm_amd import kernels
    freq = torch.tensor([freq_base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F64, device=DEV) if rot else None
    state = torch.full((len(proj) + 1, H, d * dv), float("nan"), device=DEV)
    slot = {r: len(proj) - i for i, r in enumerate(proj)}
    at, out = {r: 0 for r in proj}, {r: [] for r in proj}
    dec = torch.tensor(decay, dtype=torch.float32, device=DEV)
    for step in schedule:
        cu, past, _ = _step([(at[r], n) for r, n in step])
        rows = torch.cat([proj[r][at[r]:at[r] + n] for r, n in step])
        pos = torch.cat([torch.arange(at[r], at[r] + n) for r, n in step])
        table = kernels.rotation_table(_dev(pos), freq) if rot else None
        o = kernels.matrix_memory(_dev(rows), offs, state, cu, past, _i32([slot[r] for r, _ in step]), H, d, dv, kernels.MEM_CONST,
                                  decay=dec, rot=table, max_q=max(n for _, n in step), **kw).cpu()
        i = 0
        for r, n in step:
            out[r].append(o[i:i + n])
            i += n
            at[r] += n
    assert torch.isnan(state[0]).all()                         # nobody's slot
    return {r: torch.cat(v) for r, v in out.items()}


MEMORIES = [(2, 16, 24, 8), (1, 24, 8, 24), (3, 8, 80, 0), (2, 64, 64, 64), (1, 72, 20, 16), (2, 128, 130, 128), (2, 128, 132, 96),
            (1, 200, 64, 64), (1, 256, 72, 256), (1, 264, 16, 8), (2, 10, 12, 2), (1, 12, 9, 4), (2, 36, 20, 12)]


@pytest.mark.parametrize("H,d,dv,rot", MEMORIES)
def test_retention_in_pieces(H, d, dv, rot, monkeypatch):
    """Chunks on the matrix cores (sizes that allow them), steps and the general kernel, whole prompts and pieces that end
    inside, at and just behind a chunk, decays from 0.05 to 1."""
    T = 150
    g = torch.Generator().manual_seed(d + dv)
    decay = [0.05, 0.93, 1.0][:H] if H > 1 else [0.97]
    offs = (4, 4 + H * d, 8 + 2 * H * d)
    proj = torch.randn(T, offs[2] + H * dv + 8 - H * dv % 4, generator=g)
    q, k = (O.rotate(proj[:, o:o + H * d].double().view(T, H, d), torch.arange(T), rot, 1000.0) for o in offs[:2])
    want = O.retention(q, k * d ** -0.5, proj[:, offs[2]:offs[2] + H * dv].double().view(T, H, dv),
                       torch.tensor(decay, dtype=torch.float32).double()).reshape(T, H * dv)
    schedules = [[T], [64, 64, 22], [63, 2, 65, 1, 19], [1] * 20 + [130], [16, 17, 33, 2, 32, 31, 3, 16], [129, 21]]
    for sizes in schedules:
        got = _memory({"a": proj}, offs, [[("a", n)] for n in sizes], H, d, dv, decay, rot, 1000.0, k_scale=d ** -0.5)["a"]
        _close(got, want, 3e-6)
    for switch in ("NV_MATRIX_MEMORY_STEPS", "NV_MATRIX_MEMORY_GENERIC"):
        monkeypatch.setenv(switch, "1")
        got = _memory({"a": proj}, offs, [[("a", 100)], [("a", 1)], [("a", 49)]], H, d, dv, decay, rot, 1000.0, k_scale=d ** -0.5)["a"]
        monkeypatch.delenv(switch)
        _close(got, want, 3e-6)


def test_retention_batch_of_unequal_requests():
    """Whole prompts, continued prompts and single tokens in one launch against each request alone; a far token that
    only a slow decay remembers."""
    H, d, dv, rot, decay = 2, 32, 40, 32, [0.998, 0.7]
    g = torch.Generator().manual_seed(3)
    offs = (0, H * d, 2 * H * d)
    lens = {"a": 260, "b": 90, "c": 5, "d": 70}
    proj = {r: torch.randn(n, 2 * H * d + H * dv, generator=g) for r, n in lens.items()}
    proj["a"][3, offs[2]:] = 40.0                              # a value that stands out, 250 tokens ahead of the end
    got = _memory(proj, offs, [[("a", 100), ("b", 1)], [("c", 5), ("a", 1), ("b", 70), ("d", 2)], [("a", 130), ("d", 68), ("b", 1)],
                               [("b", 18), ("a", 28)], [("a", 1)]], H, d, dv, decay, rot, 500.0, k_scale=0.25)
    slow = torch.tensor(decay, dtype=torch.float32).double()
    for r, n in lens.items():
        q, k = (O.rotate(proj[r][:, o:o + H * d].double().view(n, H, d), torch.arange(n), rot, 500.0) for o in offs[:2])
        v = proj[r][:, offs[2]:].double().view(n, H, dv)
        want = O.retention(q, k * 0.25, v, slow)
        _close(got[r], want.reshape(n, -1), 3e-6)
        if r == "a":
            v[3] = 0.0
            assert float((O.retention(q, k * 0.25, v, slow) - want)[-1, 0].abs().max()) > 1.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dv,rot", [(2, 16, 24, 8), (1, 10, 4, 2), (3, 72, 80, 0), (2, 128, 128, 128), (1, 264, 300, 16), (2, 40, 1024, 40)])
@pytest.mark.parametrize("silu", [False, True])
def test_single_token_steps_with_norm_and_gate(dtype, H, d, dv, rot, silu):
    """The one-launch form of decoded tokens: a fresh request and two that continue, token after token."""
    from byox_vllm_amd import kernels
    T, eps = 12, 1e-3
    g = torch.Generator().manual_seed(d + dv)
    decay = torch.tensor([0.05, 0.93, 1.0][:H])
    offs = (1, 2 + H * d, 4 + 2 * H * d + (-2 * H * d) % 4, 8 + 2 * H * d + (-2 * H * d) % 4 + H * dv)
    cols = offs[3] + H * dv + 4 - (offs[3] + H * dv) % 4
    proj = {r: torch.randn(T, cols, generator=g) for r in range(3)}
    freq = torch.tensor([100.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F64, device=DEV) if rot else None
    state = torch.full((4, H, d * dv), float("nan"), device=DEV)
    start, got = [0, 5, 1], {r: [] for r in range(3)}
    table = lambda p: kernels.rotation_table(p.to(DEV), freq) if rot else None     # noqa: E731
    for r in (1, 2):                                       # what these two hold already
        n = start[r]
        kernels.matrix_memory(_dev(proj[r][:n]), offs[:3], state, _i32([0, n]), _i32([0]), _i32([r + 1]), H, d, dv, kernels.MEM_CONST,
                              decay=_dev(decay), k_scale=0.3, rot=table(torch.arange(n)), max_q=n)
    for i in range(T - 5):
        pos = torch.tensor([s + i for s in start])
        rows = torch.stack([proj[r][pos[r]] for r in range(3)])
        y = kernels.retention_step(_dev(rows), offs, _dev(decay), state, _i32([0, 1, 2, 3]), pos.int().to(DEV), _i32([1, 2, 3]), H, d, dv,
                                   eps=eps, out_dtype=dtype, rot=table(pos), k_scale=0.3, gate_silu=silu)
        assert y is not None and y.dtype == dtype
        for r in range(3):
            got[r].append(y[r].float().cpu())
    for r in range(3):
        n = start[r] + T - 5
        x = proj[r][:n].double()
        q, k = (O.rotate(x[:, o:o + H * d].reshape(n, H, d), torch.arange(n), rot, 100.0) for o in offs[:2])
        o = O.retention(q, k * 0.3, x[:, offs[2]:offs[2] + H * dv].reshape(n, H, dv), decay.double())
        z = x[:, offs[3]:offs[3] + H * dv]
        want = O.rms(o, eps).reshape(n, -1) * (O.silu(z) if silu else torch.sigmoid(z))
        _close(torch.stack(got[r]), want[start[r]:], 1e-5 if dtype == torch.float32 else 8e-3)
    assert torch.isnan(state[0]).all()


def test_activated_keys_in_chunks_equal_steps(monkeypatch):
    """Lightning attention's memory (q, k and v through SiLU, no rotation) takes the chunks too."""
    H, d, dv = 2, 64, 72
    g = torch.Generator().manual_seed(5)
    proj = torch.randn(100, 2 * H * d + H * dv, generator=g)
    args = ({"a": proj}, (0, H * d, 2 * H * d), [[("a", 77)], [("a", 23)]], H, d, dv, [0.9, 0.99], 0, 1.0)
    chunks = _memory(*args, silu=True)["a"]
    monkeypatch.setenv("NV_MATRIX_MEMORY_STEPS", "1")
    _close(chunks, _memory(*args, silu=True)["a"].double(), 3e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("groups,n", [(3, 24), (1, 40), (5, 10), (4, 128), (2, 256), (2, 300), (1, 7)])
@pytest.mark.parametrize("silu", [False, True])
def test_head_norm_without_weight_and_gate(dtype, groups, n, silu):
    from byox_vllm_amd import kernels
    g = torch.Generator().manual_seed(n)
    x, gate = torch.randn(9, groups * n, generator=g) * 3, torch.randn(9, groups * n + 8, generator=g)
    x[0] = 0.0
    x[1] *= 1e-3                                              # where eps inside the root counts
    eps = 1e-3
    z = gate[:, 4:4 + groups * n].double()
    want = O.rms(x.double().view(9, groups, n), eps).reshape(9, -1) * (O.silu(z) if silu else torch.sigmoid(z))
    got = kernels.group_rms_norm_f32(_dev(x), None, groups, eps, gate=_dev(gate)[:, 4:4 + groups * n], gate_silu=silu, out_dtype=dtype)
    assert got.dtype == dtype
    _close(got.float(), want, 2e-6 if dtype == torch.float32 else 8e-3)
    w = _round(1 + 0.3 * torch.randn(groups * n, generator=g), dtype)
    got = kernels.group_rms_norm_f32(_dev(x), _dev(w, dtype), groups, eps)
    _close(got.float(), O.rms(x.double().view(9, groups, n), eps).reshape(9, -1) * w.double(), 2e-6 if dtype == torch.float32 else 8e-3)


# ------------------------------------------------------------------------------------------------ convolution, norms, attention
class _Layer:
    """One ConvAttention with its own small cache and slots, stepped by (request, count) pieces of given projections."""

    def __init__(self, H, G, d, dv, taps, window, dtype, block, requests, scale=1.0, eps=1e-4, seed=0):
        from byox_vllm_amd.layers.conv_attention import ConvAttention
        g = torch.Generator().manual_seed(seed)
        default = torch.get_default_dtype()
        torch.set_default_dtype(dtype)
        try:
            self.mix = ConvAttention(8, H, G, d, dv, scale, taps, eps, window).to(DEV)
        finally:
            torch.set_default_dtype(default)
        self.C = (H + G) * d + G * dv
        self.w = _round(torch.randn(self.C, taps, generator=g) * 0.4, dtype)
        self.mix.conv.weight.data.copy_(self.w)
        pages = {r: -(-n // block) for r, n in requests.items()}
        order = torch.randperm(sum(pages.values()), generator=g).tolist()
        self.tables = {r: [order.pop() for _ in range(n)] for r, n in pages.items()}
        self.mix.cache = torch.full((sum(pages.values()) * block, G * (d + dv)), float("nan"), dtype=dtype, device=DEV)
        self.mix.block_size = self.block = block
        self.mix.conv.state = torch.full((len(requests) + 1, max(taps - 1, 0), self.C), float("nan"), device=DEV)
        self.slot = {r: i + 1 for i, r in enumerate(requests)}
        self.at = {r: 0 for r in requests}
        self.dtype = dtype

    def step(self, pieces, proj, gate=None):
        """-> fp32 queries and attention outputs of the step's tokens."""
        from byox_vllm_amd import kernels
        from byox_vllm_amd.utils.context import get_context, reset_context, set_context
        m = self.mix
        cu, past, owner = _step([(self.at[r], n) for r, n in pieces])
        cols = max(len(t) for t in self.tables.values())
        table = torch.full((len(pieces), cols), -1, dtype=torch.int32)
        slots, pos = [], []
        for i, (r, n) in enumerate(pieces):
            table[i, :len(self.tables[r])] = torch.tensor(self.tables[r])
            for p in range(self.at[r], self.at[r] + n):
                slots.append(self.tables[r][p // self.block] * self.block + p % self.block)
                pos.append(p)
        set_context(True, cu_seqlens_q=cu, max_seqlen_q=max(n for _, n in pieces), slot_mapping=_i32(slots), block_tables=table.to(DEV),
                    past_lens=past, state_slots=_i32([self.slot[r] for r, _ in pieces]), seq_of_token=owner)
        try:
            ctx = get_context()
            rows = torch.cat([proj[r][self.at[r]:self.at[r] + n] for r, n in pieces])
            q = m._queries(_dev(rows), torch.tensor(pos, device=DEV), ctx)
            out = torch.empty(rows.size(0), m.heads * m.vdim, dtype=self.dtype, device=DEV)
            z = torch.cat([gate[r][self.at[r]:self.at[r] + n] for r, n in pieces]) if gate else None
            kernels.paged_softmax_attn(q, m.cache, ctx.block_tables, cu, past, owner, ctx.max_seqlen_q, m.heads, m.kv_heads, m.dim, m.vdim,
                                       self.block, out, window=m.window, sink=m.sink, gate=_dev(z))
        finally:
            reset_context()
        for r, n in pieces:
            self.at[r] += n
        return q.cpu(), out.float().cpu()

    def run(self, schedule, proj, gate=None):
        qs, outs = {r: [] for r in proj}, {r: [] for r in proj}
        for pieces in schedule:
            q, o = self.step(pieces, proj, gate)
            i = 0
            for r, n in pieces:
                qs[r].append(q[i:i + n])
                outs[r].append(o[i:i + n])
                i += n
        return {r: torch.cat(v) for r, v in qs.items() if v}, {r: torch.cat(v) for r, v in outs.items() if v}

    def plain(self, rows, gate=None):
        m, T = self.mix, rows.size(0)
        y = O.causal_conv(rows[:, :self.C].double(), self.w.double())
        a, b = m.heads * m.dim, (m.heads + m.kv_heads) * m.dim
        q = O.rms(y[:, :a].view(T, m.heads, m.dim), m.eps)
        k, v = O.rms(y[:, a:b].reshape(T, m.kv_heads, m.dim), m.eps), y[:, b:].reshape(T, m.kv_heads, m.vdim)
        o = O.sink_attention(q, k, v, m.scale, m.window).reshape(T, -1)
        return q.reshape(T, -1) * m.scale, k, v, (o * torch.sigmoid(gate.double()) if gate is not None else o)


HEADS = [(6, 2, 16, 24), (1, 1, 20, 12), (3, 1, 10, 14), (4, 4, 64, 16), (8, 1, 128, 40), (2, 2, 256, 8), (4, 2, 88, 72), (2, 1, 264, 8)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv", HEADS)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
def test_convolution_norm_and_store_in_pieces(dtype, H, G, d, dv, taps):
    """Queries, cached keys and values of whole prompts, of pieces down to one token (shorter than the taps, on both sides of
    a tile of eight) and of batches, in one launch where heads are multiples of 4 (in two otherwise)."""
    lens = {"a": 40, "b": 19, "c": 3}
    g = torch.Generator().manual_seed(d + taps)
    proj = {r: torch.randn(n, (H + G) * d + G * dv + 4, generator=g) for r, n in lens.items()}
    for schedule in ([[(r, n)] for r, n in lens.items()],
                     [[("a", n)] for n in (2, 1, 3, 2, 9, 8, 7, 5, 3)] + [[("b", 1)]] * 19 + [[("c", 1)], [("c", 2)]],
                     [[("c", 1), ("a", 7), ("b", 2)], [("a", 1), ("b", 8), ("c", 2)], [("b", 9), ("a", 32)]]):
        layer = _Layer(H, G, d, dv, taps, 0, dtype, 16, lens, scale=0.7, seed=taps)
        qs, _ = layer.run(schedule, proj)
        for r, n in lens.items():
            q, k, v, _ = layer.plain(proj[r])
            _close(qs[r], q, 3e-6)
            rows = torch.tensor([layer.tables[r][p // 16] * 16 + p % 16 for p in range(n)])
            got = layer.mix.cache.float().cpu()[rows]
            _close(got[:, :G * d], k.reshape(n, -1), 3e-6 if dtype == torch.float32 else 5e-3)
            _close(got[:, G * d:], v.reshape(n, -1), 3e-6 if dtype == torch.float32 else 5e-3)
        if taps > 1:
            assert torch.isnan(layer.mix.conv.state[0]).all()


def test_eps_sits_inside_the_head_norm():
    layer = _Layer(1, 1, 8, 8, 1, 0, torch.float32, 16, {"a": 2}, eps=1e-2)
    layer.mix.conv.weight.data.fill_(1.0)
    layer.w.fill_(1.0)
    rows = torch.full((2, 24), 1e-2)
    rows[1] = 0.0
    q, _ = layer.step([("a", 2)], {"a": rows})
    assert torch.allclose(q[0], torch.full((8,), 1e-2 / (1e-4 + 1e-2) ** 0.5), rtol=1e-5) and torch.equal(q[1], torch.zeros(8))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv", [(6, 2, 16, 24), (3, 1, 10, 14), (8, 2, 32, 32), (8, 1, 128, 40), (4, 4, 64, 16)])
@pytest.mark.parametrize("window", [0, 1, 7, 16, 50])
def test_attention_in_pieces(dtype, H, G, d, dv, window):
    lens = {"a": 77, "b": 35}
    g = torch.Generator().manual_seed(d + window)
    proj = {r: torch.randn(n, (H + G) * d + G * dv, generator=g) for r, n in lens.items()}
    gate = {r: torch.randn(n, H * dv, generator=g) for r, n in lens.items()}
    for schedule in ([[("a", 77)], [("b", 35)]], [[("a", 30)]] + [[("a", 1), ("b", 1)]] * 35 + [[("a", 12)]],
                     [[("a", 2), ("b", 17)], [("b", 1), ("a", 31)], [("a", 44), ("b", 17)]]):
        layer = _Layer(H, G, d, dv, 3, window, dtype, 16, lens, scale=4.0 / d ** 0.5, seed=1)
        _, outs = layer.run(schedule, proj, gate)
        for r in lens:
            want = layer.plain(proj[r], gate[r])[3]
            _close(outs[r], want, 2e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,block", [(48, 16), (64, 64), (16, 16), (7, 16), (0, 16)])
@pytest.mark.parametrize("pieces", [[200], [100, 100], [199, 1], [130] + [1] * 70, [97, 2, 101], [2] * 100])
def test_loud_keys_at_the_edge_of_the_window(dtype, window, block, pieces):
    """Keys at the sequence's start, at page borders and in between answer every query and nobody else does: exactly the
    positions within the window hear them, all others fall to the sink's nothing."""
    H, G, d, dv, T = 2, 1, 16, 8, 200
    loud = [0, 15, 16, 63, 64, 100]
    proj = torch.zeros(T, (H + G) * d + G * dv)
    proj[:, 0], proj[:, d] = 1.0, 1.0                           # queries
    proj[:, 2 * d] = -1.0                                       # quiet keys: score -16
    for n, j in enumerate(loud):
        proj[j, 2 * d] = 1.0                                    # score +16
        proj[j, 3 * d + n] = 1.0                                # each loud key has a value number of its own
    layer = _Layer(H, G, d, dv, 1, window, dtype, block, {"a": T}, scale=1.0, eps=1e-9)
    layer.mix.conv.weight.data.fill_(1.0)
    _, outs = layer.run([[("a", n)] for n in pieces], {"a": proj})
    for i in range(T):
        heard = [n for n, j in enumerate(loud) if O.sees(i, j, window)]
        want = torch.zeros(dv)
        for n in heard:
            want[n] = 1.0 / len(heard)
        assert torch.allclose(outs["a"][i].view(H, dv), want.expand(H, dv), atol=6e-3), (i, heard)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_stands_out_for_a_decoded_token(dtype):
    """One loud key among 1900, at the window's far edge and just outside, through the key split of decoded tokens."""
    H, G, d, dv, block, ctx = 4, 2, 32, 16, 64, 1900
    for window, at, heard in ((0, 0, True), (0, 777, True), (1500, ctx - 1500, True), (1500, ctx - 1501, False)):
        proj = torch.zeros(ctx, (H + G) * d + G * dv)
        proj[:, 0:H * d:d] = 1.0
        proj[:, H * d:(H + G) * d:d] = -1.0
        proj[at, H * d:(H + G) * d:d] = 1.0
        proj[:, (H + G) * d:] = -1.0
        proj[at, (H + G) * d:] = 3.0
        layer = _Layer(H, G, d, dv, 1, window, dtype, block, {"a": ctx}, scale=0.5, eps=1e-9)
        layer.mix.conv.weight.data.fill_(1.0)
        layer.w.fill_(1.0)
        _, outs = layer.run([[("a", ctx - 1)], [("a", 1)]], {"a": proj})
        assert (float(outs["a"][-1].min()) > 2.5) == heard
        want = 3.0 if heard else 0.0                            # otherwise all scores are -16: the sink takes everything
        assert torch.allclose(outs["a"][-1], torch.full((H * dv,), want), atol=2e-2)


# ------------------------------------------------------------------------------------------------ the engine
CASES = {"mixed": mixed_config, "odd": odd_config, "plain": plain_config, "aligned": aligned_config}


@pytest.fixture(scope="module", params=[(n, dt) for n in CASES for dt in DTYPES], ids=lambda p: f"{p[0]}-{str(p[1])[6:]}")
def setup(request):
    name, dtype = request.param
    cfg = CASES[name]()
    weights = random_checkpoint(cfg, seed=11)
    torch.manual_seed(99)
    reqs = {"a": torch.randint(0, cfg["vocab"], (83,)).tolist(), "b": torch.randint(0, cfg["vocab"], (31,)).tolist(),
            "c": torch.randint(0, cfg["vocab"], (2,)).tolist(), "d": torch.randint(0, cfg["vocab"], (50,)).tolist()}
    want, chosen = {}, {}
    for n, t in reqs.items():
        logits, chosen[n] = forward_with_routes(t, weights, cfg)
        want[n] = logits.float()
    engine = Engine(cfg, weights, dtype, blocks=12, slots=3)
    if dtype == torch.bfloat16:
        engine.forced = chosen
    whole = engine.replay(reqs, [[(n, len(t))] for n, t in reqs.items()])
    return cfg, weights, dtype, reqs, want, engine, whole


def _check(setup, got):
    cfg, weights, dtype, reqs, want, engine, whole = setup
    for n in got:
        assert row_error(got[n], want[n]) < (F32_TOL if dtype == torch.float32 else BF16_TOL), (n, row_error(got[n], want[n]))
        if dtype == torch.float32:
            assert row_error(got[n], whole[n]) < SAME_TOL, n


def test_whole_prompts_match_the_oracle(setup):
    _check(setup, setup[6])


def test_every_layer_matches_the_oracle(setup):
    """The residual after every layer, for one request in one step (fp32 only: it is the sharp comparison)."""
    cfg, weights, dtype, reqs, want, engine, whole = setup
    if dtype != torch.float32:
        pytest.skip("layer by layer in fp32 only")
    from byox_vllm_amd.engine.sequence import Sequence
    trace, plain = [], []
    O.forward(reqs["b"], weights, cfg, trace=plain)
    model = engine.runner.model
    forward = model.forward
    model.forward = lambda ids, pos: forward(ids, pos, trace=trace)
    try:
        seq = Sequence(reqs["b"], engine.block_size)
        engine.scheduler.add(seq)
        plan = [(seq, len(reqs["b"]))]
        engine.scheduler.commit(plan)
        engine.runner.run_portions(plan, want=[[0]])
        engine.scheduler.finish(seq)
    finally:
        model.forward = forward
    assert len(trace) == len(plain) == len(cfg["layers"])
    for got, ref in zip(trace, plain):
        _close(got, ref, 2e-5)


def test_prompt_then_token_by_token(setup):
    reqs = setup[3]
    # the decoded stretch crosses page borders, and the windows pass over decoded tokens
    _check(setup, setup[5].replay({"a": reqs["a"]}, [[("a", 20)]] + [[("a", 1)]] * 63))
    _check(setup, setup[5].replay({"b": reqs["b"]}, [[("b", 1)]] * 31))           # from the very first token on


def test_portions_of_many_sizes(setup):
    reqs = setup[3]
    _check(setup, setup[5].replay({"a": reqs["a"]}, [[("a", n)] for n in (2, 2, 3, 9, 16, 1, 17, 2, 15, 14, 2)]))
    _check(setup, setup[5].replay({"d": reqs["d"]}, [[("d", n)] for n in (15, 1, 16, 2, 16)]))
    _check(setup, setup[5].replay({"a": reqs["a"]}, [[("a", 2)]] * 41 + [[("a", 1)]]))


def test_mixed_batches_reuse_pages_and_slots(setup):
    """Three slots, twelve pages of sixteen tokens: four requests only fit because the finished ones give theirs back.
    Prompt pieces run beside single tokens; requests sit out steps."""
    reqs = setup[3]
    schedule = [[("a", 30), ("b", 5)], [("a", 1), ("b", 20), ("c", 2)], [("a", 2), ("b", 1)], [("b", 1), ("d", 7), ("a", 1)],
                [("a", 40), ("d", 1), ("b", 4)], [("d", 30)], [("a", 1), ("d", 1)], [("a", 8), ("d", 11)]]
    _check(setup, setup[5].replay(reqs, schedule))
    # the same requests again, in slots and pages that the first pass has used
    _check(setup, setup[5].replay(reqs, [[("d", 50), ("c", 1)], [("c", 1), ("b", 31)], [("a", 83)]]))


def test_greedy_generation_through_the_engine(setup):
    """LLM.generate (scheduler's own portion policy, sampler at temperature 0) against the oracle's greedy run."""
    cfg, weights, dtype, reqs, want, engine, whole = setup
    if dtype != torch.float32:
        pytest.skip("a close call of a router is no rounding error: token by token in fp32")
    from byox_vllm_amd import LLM, SamplingParams
    conf = engine_config(cfg, weights, dtype, blocks=12, slots=3)
    llm = LLM("synthetic", hf_config=conf.hf_config, state_dict=weights, kvcache_block_size=16, num_kvcache_blocks=12,
              max_num_seqs=3, num_state_slots=3, enforce_eager=True, max_num_batched_tokens=48, max_model_len=1 << 20)
    prompts = [reqs["b"], reqs["c"], reqs["d"][:20], reqs["a"][:40]]
    steps = 10
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=steps, ignore_eos=True), use_tqdm=False)
    llm._exit()
    for prompt, out in zip(prompts, outs):
        tokens = list(prompt) + out["token_ids"]
        logits = O.forward(tokens, weights, cfg)
        spread = float(logits.std())
        for k, tok in enumerate(out["token_ids"]):
            row = logits[len(prompt) + k - 1]
            # the engine's choice is the oracle's argmax, or lies inside the rounding of the engine's dtype
            assert row.max().item() - row[tok].item() <= 1e-3 * spread, (k, tok)
        assert len(out["token_ids"]) == steps


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_captured_decode_steps_equal_eager_ones(dtype):
    """Decode steps replayed from hipGraphs (padded batches, the spare state slot, one staging copy) give the tokens of
    the eager engine, step after step, with prompt portions running eagerly between the replays."""
    from byox_vllm_amd import LLM, SamplingParams
    cfg = mixed_config()
    weights = random_checkpoint(cfg, seed=21)
    torch.manual_seed(5)
    prompts = [torch.randint(0, cfg["vocab"], (n,)).tolist() for n in (37, 3, 18, 25, 9)]
    params = [SamplingParams(temperature=0.0, max_tokens=n, ignore_eos=True) for n in (30, 41, 12, 25, 33)]
    outs = []
    for eager in (True, False):
        conf = engine_config(cfg, weights, dtype, blocks=24, slots=4)
        llm = LLM("synthetic", hf_config=conf.hf_config, state_dict=weights, kvcache_block_size=16, num_kvcache_blocks=24,
                  max_num_seqs=4, num_state_slots=4, enforce_eager=eager, max_num_batched_tokens=32, max_model_len=128)
        assert bool(llm.model_runner.graphs) == (not eager)
        outs.append([o["token_ids"] for o in llm.generate(prompts, params, use_tqdm=False)])
        llm._exit()
    assert outs[0] == outs[1]
    assert [len(t) for t in outs[0]] == [30, 41, 12, 25, 33]


def test_command_line_generation_and_trace_replay_from_a_model_folder(tmp_path):
    """A model folder (config.json + model.safetensors in bf16) through the two command-line entry points, each in a
    process of its own: `python -m byox_vllm_amd generate` against the oracle's greedy continuation, bin/trace_run
    against the oracle's logits for a replayed schedule with pieces, a pause and a request that ends early."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np
    from safetensors.torch import save_file
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = aligned_config()
    weights = random_checkpoint(cfg, seed=31)
    model = tmp_path / "model"
    model.mkdir()
    with open(model / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, str(model / "model.safetensors"))
    torch.manual_seed(3)
    a = torch.randint(0, cfg["vocab"], (70,)).tolist()
    b = torch.randint(0, cfg["vocab"], (9,)).tolist()

    run = subprocess.run([sys.executable, "-m", "byox_vllm_amd", "generate", "--model", str(model), "--dtype", "float32",
                          "--prompt-ids", ",".join(map(str, b)), "--max-tokens", "6", "--block-size", "16", "--eager"],
                         cwd=root, capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr[-3000:]
    line = json.loads([ln for ln in run.stdout.splitlines() if ln.startswith("{")][0])
    logits = O.forward(list(b) + line["token_ids"], weights, cfg)
    for k, tok in enumerate(line["token_ids"]):
        row = logits[len(b) + k - 1]
        assert row.max().item() - row[tok].item() <= 1e-3 * float(logits.std())
    assert len(line["token_ids"]) == 6

    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [0, 39]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:2], "want": []}, {"id": "a", "tokens": a[40:41], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[2:], "want": [6]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[41:], "want": [0, 28]}, {"id": "c", "tokens": b, "want": [8]}], "end": ["a", "c"]}]
    wa, wb = O.forward(a, weights, cfg).float(), O.forward(b, weights, cfg).float()
    for dtype, tol in (("float32", F32_TOL), ("bfloat16", None)):
        out = tmp_path / ("out_" + dtype)
        run = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(model), "--dtype", dtype, "--out", str(out),
                              "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n", cwd=root,
                             capture_output=True, text=True, timeout=100)
        assert run.returncode == 0, run.stderr[-3000:]
        assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
        expect = {0: wa[[0, 39]], 1: wa[[40]], 2: wb[[8]], 3: torch.cat([wa[[41, 69]], wb[[8]]])}
        for i, want in expect.items():
            got = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
            assert got.shape == want.shape and torch.isfinite(got).all()
            if tol is not None:          # in 16 bits a router of random weights may take another expert
                assert row_error(got, want) < tol, (dtype, i)


def test_long_decoding_over_many_windows():
    """170 decoded tokens in a row: every window and every page border passes over decoded keys, the states decay on."""
    cfg = aligned_config()
    weights = random_checkpoint(cfg, seed=41)
    torch.manual_seed(8)
    toks = torch.randint(0, cfg["vocab"], (200,)).tolist()
    want, chosen = forward_with_routes(toks, weights, cfg)
    for dtype, tol in ((torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)):
        engine = Engine(cfg, weights, dtype, blocks=14, slots=1)
        engine.forced = {"a": chosen} if dtype == torch.bfloat16 else None
        got = engine.replay({"a": toks}, [[("a", 30)]] + [[("a", 1)]] * 170)["a"]
        assert row_error(got, want.float()) < tol


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_from_seeds(seed):
    """Layer orders, sizes, windows and constants drawn independently, pages of 64 tokens: whole prompts and a mixed
    schedule."""
    cfg = random_config(seed)
    weights = random_checkpoint(cfg, seed=seed)
    g = torch.Generator().manual_seed(seed)
    reqs = {n: torch.randint(0, cfg["vocab"], (k,), generator=g).tolist() for n, k in (("a", 140), ("b", 67), ("c", 3))}
    mixed = [[("a", 66), ("b", 2)], [("b", 63), ("a", 1), ("c", 2)], [("a", 2), ("b", 1)], [("c", 1), ("a", 60)], [("a", 1), ("b", 1)],
             [("a", 10)]]
    plain = {n: forward_with_routes(t, weights, cfg) for n, t in reqs.items()}
    loose = {n: 2.0 * rounding_errors(t, weights, cfg, plain[n][1]) for n, t in reqs.items()}      # ill-conditioned rows
    for dtype, tol in ((torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)):
        engine = Engine(cfg, weights, dtype, blocks=6, slots=3, block_size=64)
        engine.forced = {n: c for n, (_, c) in plain.items()} if dtype == torch.bfloat16 else None
        for schedule in ([[(n, len(t))] for n, t in reqs.items()], mixed):
            got = engine.replay(reqs, schedule)
            for n, t in reqs.items():
                bound = torch.full((len(t),), tol)
                if dtype == torch.bfloat16:
                    bound = torch.maximum(bound, loose[n])
                errors = row_errors(got[n], plain[n][0].float())
                assert bool((errors < bound).all()), (dtype, n, int((errors / bound).argmax()), float(errors.max()))
        del engine
