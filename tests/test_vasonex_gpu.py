"""Vasonex on the GPU: every mechanism's kernel alone against the plain functions of oracle/vasonex.py, then the engine
(scheduler commit, pages, run_portions) against the oracle run on each request's whole token list."""

import math

import pytest
import torch

from oracle import vasonex as O
from vasonex_cases import (Engine, aligned_config, engine_config, forward_with_routes, mixed_config, odd_config,
                           plain_config, random_checkpoint, random_config, row_error)

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


# ------------------------------------------------------------------------------------------------ norms around a sublayer
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [64, 98, 1028, 2052, 4100])         # one, two and four registers' rows; rows through LDS
@pytest.mark.parametrize("bias", [False, True])
def test_output_norm_residual_and_next_input_norm(dtype, n, bias):
    from byox_vllm_amd import kernels
    g = torch.Generator().manual_seed(n)
    x, y = torch.randn(7, n, generator=g), torch.randn(7, n + 4, generator=g) * 5
    post, pre = (_round(1 + 0.3 * torch.randn(n, generator=g), dtype) for _ in range(2))
    yb = _round(torch.randn(n, generator=g), dtype) if bias else None
    eps = 1e-3
    v = y[:, 4:].double() + (yb.double() if bias else 0.0)
    new = x.double() + O.rms_norm(v, post.double(), eps)
    want = O.rms_norm(new, pre.double(), eps)
    tol = 2e-6 if dtype == torch.float32 else 8e-3
    xd = _dev(x)
    args = dict(y=_dev(y)[:, 4:], w_post=_dev(post, dtype), eps=eps, y_bias=_dev(yb, dtype))
    h = kernels.sandwich_norm(xd, w_pre=_dev(pre, dtype), **args)
    _close(xd, new, 1e-6)                                          # the residual itself stays fp32
    _close(h.float(), want, tol)
    # only some rows, and the residual left as it is
    xd = _dev(x)
    h = kernels.sandwich_norm(xd, w_pre=_dev(pre, dtype), rows_idx=_i32([5, 0, 5]), **args)
    assert torch.equal(xd.cpu(), x)
    _close(h.float(), want[[5, 0, 5]], tol)
    # the residual alone; the input norm alone; a result without an output norm
    assert kernels.sandwich_norm(xd, w_pre=None, **args) is None
    _close(xd, new, 1e-6)
    xd = _dev(x)
    h = kernels.sandwich_norm(xd, None, None, _dev(pre, dtype), eps)
    assert torch.equal(xd.cpu(), x)
    _close(h.float(), O.rms_norm(x.double(), pre.double(), eps), tol)
    h = kernels.sandwich_norm(xd, args["y"], None, _dev(pre, dtype), eps)
    _close(h.float(), O.rms_norm(x.double() + y[:, 4:].double(), pre.double(), eps), tol)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [64, 98])
@pytest.mark.parametrize("weights,last,shared", [(False, False, False), (True, False, True), (False, True, False),
                                                 (False, False, True)])
def test_output_norm_gathers_and_sums_expert_rows(dtype, n, weights, last, shared):
    from byox_vllm_amd import kernels
    g = torch.Generator().manual_seed(n + 1)
    T, C = 9, 3
    x, y = torch.randn(T, n, generator=g), torch.randn(T * C, n, generator=g) * 3
    slots = torch.randperm(T * C, generator=g).view(T, C)
    wt, gates, sh = torch.rand(T, C, generator=g), torch.randn(T, 5, generator=g) * 2, torch.randn(T, n, generator=g)
    post, pre = (_round(1 + 0.3 * torch.randn(n, generator=g), dtype) for _ in range(2))
    f = wt.double() if weights else torch.ones(T, C, dtype=F64)
    if last:
        f[:, -1] = torch.sigmoid(gates[:, 2].double())
    v = (y.double()[slots] * f[:, :, None]).sum(1)
    if shared:
        v = v + torch.sigmoid(gates[:, 3].double())[:, None] * sh.double()
    new = x.double() + O.rms_norm(v, post.double(), 1e-5)
    xd, gd = _dev(x), _dev(gates)
    h = kernels.sandwich_norm(xd, _dev(y), _dev(post, dtype), _dev(pre, dtype), 1e-5, slot_of=slots.to(torch.int32).to(DEV),
                              weights=_dev(wt) if weights else None, last_gate=gd[:, 2] if last else None,
                              shared=_dev(sh) if shared else None, shared_gate=gd[:, 3] if shared else None)
    _close(xd, new, 1e-6)
    _close(h.float(), O.rms_norm(new, pre.double(), 1e-5), 2e-6 if dtype == torch.float32 else 8e-3)


def test_eps_sits_inside_both_roots():
    from byox_vllm_amd import kernels
    ones = torch.ones(64, device=DEV)
    x, y = torch.zeros(2, 64, device=DEV), torch.zeros(2, 64, device=DEV)
    y[1] = 1e-4
    h = kernels.sandwich_norm(x, y, ones, ones, 1e-2)
    new = 1e-4 / (1e-8 + 1e-2) ** 0.5
    assert float(h[0].abs().max()) == 0.0 and abs(float(x[1, 0]) - new) < 1e-9
    assert abs(float(h[1, 0]) - new / (new * new + 1e-2) ** 0.5) < 1e-7


# ------------------------------------------------------------------------------------------------ products
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,N", [(1, 300, 24), (20, 256, 40), (5, 64, 20), (100, 64, 72), (70, 50, 36), (4096, 128, 48)])
def test_gated_unit_with_biases_in_every_route_of_the_product(dtype, M, K, N):
    """Few rows (K split over the wavefronts), general, tiled, and the vendor route with the activation as a pass of its
    own; gate and up have different biases."""
    from byox_vllm_amd import kernels
    g = torch.Generator().manual_seed(M + N)
    x, w = _round(torch.randn(M, K, generator=g), dtype), _round(torch.randn(2 * N, K, generator=g) * K ** -0.5, dtype)
    b = _round(torch.randn(2 * N, generator=g), dtype)
    got = kernels.linear(_dev(x, dtype), _dev(w, dtype), _dev(b, dtype), epilogue=kernels.EPI_GLU, act=kernels.ACT_SILU)
    z = x.double() @ w.double().T + b.double()
    _close(got.float(), O.silu(z[:, :N]) * z[:, N:], 1e-5 if dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,N", [(3, 300, 24), (5, 64, 20), (100, 64, 72), (4096, 128, 48)])
def test_erf_gelu_in_every_route_of_the_product(dtype, M, K, N):
    from byox_vllm_amd import kernels
    g = torch.Generator().manual_seed(M)
    x, w = _round(torch.randn(M, K, generator=g), dtype), _round(torch.randn(N, K, generator=g) * 2 * K ** -0.5, dtype)
    got = kernels.linear(_dev(x, dtype), _dev(w, dtype), epilogue=kernels.EPI_ACT, act=kernels.ACT_GELU_ERF)
    z = x.double() @ w.double().T
    want = O.gelu_erf(z)
    _close(got.float(), want, 1e-6 if dtype == torch.float32 else 5e-3)
    if dtype == torch.float32:       # the tanh form is another function
        tanh = 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))
        assert float((tanh - want).abs().max()) > 20 * float((got.double().cpu() - want).abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [[2, 0, 5], [30, 1, 17], [90, 0, 200]])
def test_row_factors_act_ahead_of_the_activation(dtype, rows):
    """Grouped products over gathered rows: f(s W a), one weight per group, a factor per output row."""
    from byox_vllm_amd import kernels
    K, N, E = 48, 24, len(rows)
    g = torch.Generator().manual_seed(sum(rows))
    R = sum(rows)
    x, w = _round(torch.randn(60, K, generator=g), dtype), _round(torch.randn(E, N, K, generator=g) * 0.4, dtype)
    at, s = torch.randint(0, 60, (R,), generator=g), torch.rand(R, generator=g)
    off = [0]
    for n in rows:
        off.append(off[-1] + n)
    got = kernels.linear(_dev(x, dtype), _dev(w, dtype), rows=R, a_rows=at.to(torch.int32).to(DEV), batch=E, w_batch_stride=N * K,
                         group_offsets=_i32(off), max_group_rows=max(rows), epilogue=kernels.EPI_ACT,
                         act=kernels.ACT_GELU_ERF, row_scale=_dev(s), out_dtype=torch.float32)
    for e in range(E):
        i = slice(off[e], off[e + 1])
        if rows[e]:
            want = O.gelu_erf((s[i, None].double() * x[at[i]].double()) @ w[e].double().T)
            _close(got[i], want, 1e-5)


# ------------------------------------------------------------------------------------------------ mixture
@pytest.mark.parametrize("T,E,top", [(1, 5, 2), (8, 8, 1), (64, 100, 3), (65, 3, 3), (700, 130, 4), (2, 1, 1)])
@pytest.mark.parametrize("shared", [False, True])
def test_plan_of_a_mixture(T, E, top, shared):
    """Choices, weights, groups and the way back, for steps of one launch and of two; more experts than a wavefront has
    lanes; logits far into the sigmoid's saturation still in their order."""
    from byox_vllm_amd import kernels
    z = torch.randn(T, E + 2, generator=torch.Generator().manual_seed(T + E)) * 4
    z[0, :E] = 30.0 + 3.0 * torch.randperm(E, generator=torch.Generator().manual_seed(E))          # sigmoid: 1 in fp32
    offsets, tokens, row_w, slot_of, w = (t.cpu() for t in kernels.moe_plan(_dev(z), E, top, kernels.ROUTE_SIGMOID, shared))
    idx, want = O.route(z[:, :E].double(), top)
    _close(w, want, 1e-6)
    C, groups = top + int(shared), E + int(shared)
    assert offsets.shape == (groups + 1,) and slot_of.shape == (T, C)
    choice = torch.cat([idx, torch.full((T, 1), E)], 1) if shared else idx
    counts = torch.bincount(choice.flatten(), minlength=groups)
    assert torch.equal(offsets.long(), torch.cat([torch.zeros(1, dtype=torch.long), counts.cumsum(0)]))
    assert sorted(slot_of.flatten().tolist()) == list(range(T * C))
    s = slot_of.long()
    assert torch.equal(tokens.long()[s], torch.arange(T)[:, None].expand(T, C))
    group = torch.searchsorted(offsets.long(), s, right=True) - 1
    # (empty groups share their start with the next one; searchsorted lands on the last of them, which owns the row)
    assert torch.equal(group, choice)
    _close(row_w[s[:, :top]], want, 1e-6)
    if shared:
        assert torch.equal(row_w[s[:, top]], torch.ones(T))


def test_equal_logits_go_to_the_lower_expert_and_no_number_stays_in_range():
    from byox_vllm_amd import kernels
    z = torch.zeros(3, 70)
    z[1, 5] = z[1, 69] = 1.0
    z[2] = float("nan")
    offsets, _, _, slot_of, w = kernels.moe_plan(_dev(z), 70, 2, kernels.ROUTE_SIGMOID)
    o = offsets.cpu().tolist()
    assert o[1] - o[0] >= 1 and o[2] - o[1] >= 1 and o[6] - o[5] == 1 and o[70] - o[69] == 1 and o[70] == 6
    assert sorted(slot_of.flatten().tolist()) == list(range(6))
    _close(w[:2].cpu(), torch.sigmoid(torch.tensor([[0.0, 0.0], [1.0, 1.0]])), 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,ff,shared", [(5, 2, 24, 40), (3, 3, 20, None), (8, 1, 32, 32), (1, 1, 12, 12)])
@pytest.mark.parametrize("weigh", ["input", "output"])
@pytest.mark.parametrize("T", [3, 37, 130])
def test_mixture_layer_against_the_plain_mixture(dtype, E, top, ff, shared, weigh, T):
    from byox_vllm_amd import kernels
    from byox_vllm_amd.layers.moe import UnaryMixtureOfExperts
    width = 64
    g = torch.Generator().manual_seed(E + T)
    torch.set_default_device(DEV)
    try:
        layer = UnaryMixtureOfExperts(width, E, top, ff, route="sigmoid", weigh=weigh, shared_ff=shared).to(dtype)
    finally:
        torch.set_default_device(None)
    W = {"router": torch.randn(E, width, generator=g) * 0.3, "shared.sg": torch.randn(1, width, generator=g) * 0.2}
    for name, n in [(f"e{e}", ff) for e in range(E)] + ([("shared", shared)] if shared else []):
        W[name + ".up"] = torch.randn(n, width, generator=g) * 0.3
        W[name + ".down"] = torch.randn(width, n, generator=g) * n ** -0.5
    W = {k: _round(v, dtype) for k, v in W.items()}
    layer.router.weight.data[:E] = _dev(W["router"], dtype)
    if shared:
        layer.router.weight.data[E:] = _dev(W["shared.sg"], dtype)
    for e in range(E):
        layer.up.data[e], layer.down.data[e] = _dev(W[f"e{e}.up"], dtype), _dev(W[f"e{e}.down"], dtype)
    if shared:
        up, down = layer._shared_weights()
        up.copy_(_dev(W["shared.up"], dtype))
        down.copy_(_dev(W["shared.down"], dtype))
    h = _round(torch.randn(T, width, generator=g), dtype)
    W = {k: v.double() for k, v in W.items()}
    spec = {"router": {"experts": E, "top": top}, "expert": {"ff": ff}}
    if shared:
        spec["shared"] = {"ff": shared}
    if weigh == "input":
        want = O.moe(h.double(), W, "", spec)
    else:
        idx, wt = O.route(h.double() @ W["router"].T, top)
        want = torch.zeros(T, width, dtype=F64)
        for t in range(T):
            for j in range(top):
                want[t] += wt[t, j] * O.expert(h[t].double(), W, f"e{int(idx[t, j])}.")
        if shared:
            want = want + torch.sigmoid(h.double() @ W["shared.sg"].T) * O.expert(h.double(), W, "shared.")
    x = torch.zeros(T, width, device=DEV)
    kernels.sandwich_norm(x, w_post=None, w_pre=torch.ones(width, device=DEV, dtype=dtype), eps=1e-5, **layer(_dev(h, dtype)))
    _close(x, want, 1e-5 if dtype == torch.float32 else 1e-2)


# ------------------------------------------------------------------------------------------------ attention
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,rot", [(6, 2, 16, 24, 8), (1, 1, 20, 12, 2), (8, 2, 32, 32, 32), (3, 3, 12, 4, 0),
                                          (4, 1, 64, 8, 30), (2, 2, 18, 8, 6)])
def test_interleaved_rotation_and_store(dtype, H, G, d, dv, rot):
    """What qk_rotate_store leaves as queries and in the cache rows: neighbouring numbers turn together, the rest passes,
    at positions up to 5000; a row without a slot writes nothing."""
    from byox_vllm_amd import kernels
    T = 12
    g = torch.Generator().manual_seed(H + d)
    proj = torch.randn(T, (H + G) * d + G * dv + 4, generator=g)
    offs = (4, 4 + H * d, 4 + (H + G) * d)
    pos = torch.tensor([0, 1, 2, 3, 17, 63, 64, 65, 1000, 4095, 4096, 5000])
    freq = O.frequencies({"base": 700.0, "dims": rot, "scaling": {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 256}})
    cache = torch.full((T + 2, G * (d + dv)), float("nan"), dtype=dtype, device=DEV)
    slots = list(range(T - 1, -1, -1))
    slots[3] = -1
    q = kernels.qk_rotate_store(_dev(proj), offs, _dev(pos), 0.3, _i32(slots), cache, H, G, d, dv,
                                inv_freq=freq.float().to(DEV) if rot else None, rot_dims=rot, interleaved=True)
    p, f32 = proj.double(), freq.float().double()                     # the engine's table is fp32
    wq = O.rotate_pairs(p[:, offs[0]:offs[1]].view(T, H, d), pos, f32) if rot else p[:, offs[0]:offs[1]].view(T, H, d)
    wk = O.rotate_pairs(p[:, offs[1]:offs[2]].view(T, G, d), pos, f32) if rot else p[:, offs[1]:offs[2]].view(T, G, d)
    _close(q.view(T, H, d), wq * 0.3, 5e-4 if rot else 1e-6)          # at position 5000 a float angle is 3e-4 off
    near = pos < 100
    _close(q.view(T, H, d)[near], wq[near] * 0.3, 1e-5)
    rows = cache[:T].float().flip(0).cpu()
    keep = [i for i in range(T) if i != 3]
    tol = (5e-4 if rot else 1e-6) if dtype == torch.float32 else 5e-3
    _close(rows[keep, :G * d].view(-1, G, d), wk[keep], tol)
    _close(rows[keep, G * d:], p[keep][:, offs[2]:offs[2] + G * dv], 1e-6 if dtype == torch.float32 else 5e-3)
    assert torch.isnan(rows[3]).all() and torch.isnan(cache[T:].float()).all()


def _paged(proj, offs, pieces, H, G, d, dv, scale, window, keep, dtype, block, gate=None, seed=0):
    """qk_rotate_store + paged_softmax_attn over one request cut into ``pieces``, on scattered pages."""
    from byox_vllm_amd import kernels
    T = proj.shape[0]
    n_pages = -(-T // block)
    pages = torch.randperm(n_pages + 3, generator=torch.Generator().manual_seed(seed))[:n_pages].tolist()
    cache = torch.full(((n_pages + 3) * block, G * (d + dv)), float("nan"), dtype=dtype, device=DEV)
    table = _i32([pages])
    out = torch.zeros(T, H * dv + 2, dtype=dtype, device=DEV)
    pd, gd = _dev(proj), _dev(gate)
    a = 0
    for n in pieces:
        slots = _i32([pages[p // block] * block + p % block for p in range(a, a + n)])
        q = kernels.qk_rotate_store(pd[a:a + n], offs, torch.arange(a, a + n, device=DEV), scale, slots, cache, H, G, d, dv)
        kernels.paged_softmax_attn(q, cache, table, _i32([0, n]), _i32([a]), _i32([0] * n), n, H, G, d, dv, block,
                                   out[a:a + n, 2:], window=window, keep_first=keep,
                                   gate=gd[a:a + n, 2:] if gd is not None else None, gate_per_head=True)
        a += n
    assert float(out[:, :2].float().abs().max()) == 0.0
    return out[:, 2:].float()


def _inputs(T, H, G, d, dv, dtype, seed):
    g = torch.Generator().manual_seed(seed)
    k_off, v_off = H * d, (H + G) * d
    proj = torch.randn(T, v_off + G * dv, generator=g)
    proj[:, k_off:] = _round(proj[:, k_off:], dtype)
    return proj, torch.randn(T, H + 2, generator=g) * 2, (0, k_off, v_off)


def _plain(proj, offs, H, G, d, dv, scale, mask, gate=None):
    T, p = proj.shape[0], proj.double()
    out = O.softmax_attention(p[:, :offs[1]].view(T, H, d), p[:, offs[1]:offs[2]].view(T, G, d), p[:, offs[2]:].view(T, G, dv),
                              scale, O.visible(T, mask))
    if gate is not None:
        out = out * torch.sigmoid(gate.double())[:, :, None]
    return out.reshape(T, H * dv)


GEOMETRIES = [(6, 2, 16, 24, 16), (1, 1, 20, 12, 16), (8, 1, 128, 40, 64), (4, 4, 72, 16, 16), (3, 1, 10, 6, 32), (4, 2, 136, 200, 16),
              (12, 3, 24, 64, 32), (2, 2, 256, 256, 64)]
MASKS = [(12, 3), (16, 0), (5, 30), (1, 1), (64, 17), (0, 4), (200, 200), (33, 70)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,block", GEOMETRIES)
@pytest.mark.parametrize("window,keep", MASKS)
def test_window_beside_kept_first_tokens_in_pieces(dtype, H, G, d, dv, block, window, keep):
    if (H, d) not in ((6, 16), (4, 72), (1, 20)) and window not in (12, 33):
        pytest.skip("every mask on three geometries")
    T = 110
    proj, gate, offs = _inputs(T, H, G, d, dv, dtype, seed=H * 10 + d)
    want = _plain(proj, offs, H, G, d, dv, d ** -0.5, {"size": window, "keep_first": keep}, gate[:, 2:])
    for pieces in ([T], [1] * T, [2, 2, 3, 9, 16, 1, 17, 2, 15, 3, 40], [T - 1, 1], [33, 77]):
        got = _paged(proj, offs, pieces, H, G, d, dv, d ** -0.5, window, keep, dtype, block, gate)
        _close(got, want, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep,block", [(48, 5, 16), (64, 1, 64), (50, 20, 64), (16, 16, 16), (7, 64, 16), (20, 0, 16)])
@pytest.mark.parametrize("pieces", [[200], [100, 100], [199, 1], [130] + [1] * 70, [97, 2, 101], [2] * 100])
def test_loud_keys_at_the_edges_of_window_and_kept_tokens(dtype, window, keep, block, pieces):
    """Three heads ask for one marked key each, so loudly that a position which sees it hears nothing else: the last kept
    token (head 0: heard for ever), the first token that is not kept (head 1: heard until the window has passed), and a
    token in the middle (head 2: heard by exactly ``window`` positions).  Head 3 has ordinary scores."""
    H, G, d, dv, T = 4, 1, 16, 8, 200
    g = torch.Generator().manual_seed(window)
    k_off, v_off = H * d, (H + G) * d
    proj = torch.randn(T, v_off + G * dv, generator=g) * 0.2
    marks = {0: max(keep - 1, 0), 1: keep, 2: 103}
    proj[:, v_off:v_off + 3] = 0.0
    proj[:, k_off:v_off] *= 0.5
    for h, j in marks.items():
        proj[:, h * d:(h + 1) * d] = 0.0
        proj[:, h * d + h] = 6.0
        proj[:, k_off + h] = 0.0
        proj[j, k_off + h] = 6.0
        proj[j, v_off + h] = 1.0
    proj = _round(proj, dtype)
    want = _plain(proj, (0, k_off, v_off), H, G, d, dv, 1.0, {"size": window, "keep_first": keep})
    got = _paged(proj, (0, k_off, v_off), pieces, H, G, d, dv, 1.0, window, keep, dtype, block)
    i = torch.arange(T)
    for h, j in marks.items():
        hears = (i >= j) & ((i - j < window) | (j < keep))
        for rows in (want, got.cpu()):
            assert torch.equal(rows[:, h * dv + h] > 0.5, hears), (h, j)
            assert float(rows[~hears, h * dv + h].abs().max() if (~hears).any() else 0.0) == 0.0
    _close(got, want, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep", [(0, 0), (1500, 4), (300, 700)])
def test_a_far_key_stands_out_for_a_decoded_token(dtype, window, keep):
    """Long contexts, decoded tokens whose keys several workgroups share; a loud key in the first page, in the window, at
    the last place the window still shows, one beyond it, and among the kept tokens."""
    from byox_vllm_amd import kernels
    H, G, d, dv, block, ctx = 4, 2, 32, 16, 64, [1900, 700, 65]
    g = torch.Generator().manual_seed(7)
    tables, n = [], 0
    order = torch.randperm(64, generator=g).tolist()
    for c in ctx:
        k = -(-c // block)
        tables.append(order[n:n + k])
        n += k
    rows = torch.randn(sum(ctx), G * (d + dv), generator=g) * 0.3
    cache = torch.full((64 * block, G * (d + dv)), float("nan"))
    for trial, places in enumerate(([0, 0, 0], [1, 500, 64], [c - 1 - 299 for c in (1900, 700, 364)], [399, 399, 30],
                                    [400, 100, 1], [699, 650, 3], [700, 3, 20])):
        q = torch.randn(3, H * d, generator=g) * 0.3
        at, k, v = 0, [], []
        for r, c in enumerate(ctx):
            mine = rows[at:at + c].clone()
            j = places[r]
            mine[j, :d] = 0.0
            mine[j, 0] = 8.0
            mine[j, G * d] = 5.0
            q[r, :d] = 0.0
            q[r, 0] = 2.0
            mine = _round(mine, dtype)
            slot = torch.tensor([tables[r][p // block] * block + p % block for p in range(c)])
            cache[slot] = mine
            k.append(mine[:, :G * d].view(c, G, d).double())
            v.append(mine[:, G * d:].view(c, G, dv).double())
            at += c
        table = torch.full((3, 32), -1, dtype=torch.int32)
        for r, t in enumerate(tables):
            table[r, :len(t)] = torch.tensor(t)
        out = torch.zeros(3, H * dv, dtype=dtype, device=DEV)
        kernels.paged_softmax_attn(_dev(q), _dev(cache, dtype), table.to(DEV), _i32([0, 1, 2, 3]), _i32([c - 1 for c in ctx]),
                                   _i32([0, 1, 2]), 1, H, G, d, dv, block, out, window=window, keep_first=keep)
        for r, c in enumerate(ctx):
            seen = O.visible(c, {"size": window, "keep_first": keep})[-1:]
            want = O.softmax_attention(q[r:r + 1].double().view(1, H, d), k[r], v[r], 1.0, seen).reshape(-1)
            heard = bool(seen[0, places[r]])
            assert (float(want[0]) > 4.0) == heard
            _close(out[r].float(), want, 2e-5 if dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_batch_of_unequal_requests(dtype):
    """A piece that continues cached tokens, a decoded token, a whole short prompt and a piece of two tokens in one
    launch, with tables of different lengths, against each request alone."""
    from byox_vllm_amd import kernels
    H, G, d, dv, block, window, keep = 4, 2, 16, 24, 16, 10, 3
    lens, past = [60, 37, 5, 44], [21, 36, 0, 42]
    data = [_inputs(n, H, G, d, dv, dtype, seed=n) for n in lens]
    offs = data[0][2]
    tables = [[7, 2, 9, 13], [4, 1, 8], [5], [0, 3, 6]]
    cache = torch.full((14 * block, G * (d + dv)), float("nan"), dtype=dtype, device=DEV)
    slot = lambda r, p: tables[r][p // block] * block + p % block   # noqa: E731
    for r in range(4):
        if past[r]:
            kernels.qk_rotate_store(_dev(data[r][0][:past[r]]), offs, torch.arange(past[r], device=DEV), 0.25,
                                    _i32([slot(r, p) for p in range(past[r])]), cache, H, G, d, dv)
    proj = torch.cat([data[r][0][past[r]:] for r in range(4)])
    gate = torch.cat([data[r][1][past[r]:] for r in range(4)])
    pos = torch.cat([torch.arange(past[r], lens[r]) for r in range(4)])
    q = kernels.qk_rotate_store(_dev(proj), offs, _dev(pos), 0.25, _i32([slot(r, p) for r in range(4) for p in range(past[r], lens[r])]),
                                cache, H, G, d, dv)
    table = torch.full((4, 4), -1, dtype=torch.int32)
    cu = [0]
    for r, t in enumerate(tables):
        table[r, :len(t)] = torch.tensor(t)
        cu.append(cu[-1] + lens[r] - past[r])
    out = torch.zeros(cu[-1], H * dv, dtype=dtype, device=DEV)
    kernels.paged_softmax_attn(q, cache, table.to(DEV), _i32(cu), _i32(past), _i32([r for r in range(4) for _ in range(lens[r] - past[r])]),
                               39, H, G, d, dv, block, out, window=window, keep_first=keep, gate=_dev(gate)[:, 2:],
                               gate_per_head=True)
    for r in range(4):
        want = _plain(data[r][0], offs, H, G, d, dv, 0.25, {"size": window, "keep_first": keep}, data[r][1][:, 2:])[past[r]:]
        _close(out[cu[r]:cu[r + 1]].float(), want, 2e-5 if dtype == torch.float32 else 2e-2)


def test_chunks_and_kept_tokens_exclude_each_other():
    from byox_vllm_amd import kernels
    with pytest.raises(RuntimeError, match="exclude each other"):
        z = torch.zeros(1, 8, device=DEV)
        kernels.paged_softmax_attn(z, torch.zeros(16, 16, device=DEV), _i32([[0]]), _i32([0, 1]), _i32([0]), _i32([0]), 1, 1, 1, 8,
                                   8, 16, torch.zeros(1, 8, device=DEV), window=4, chunk=4, keep_first=1)


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
    # the decoded stretch crosses page borders, and every window passes over decoded tokens
    _check(setup, setup[5].replay({"a": reqs["a"]}, [[("a", 20)]] + [[("a", 1)]] * 63))
    _check(setup, setup[5].replay({"b": reqs["b"]}, [[("b", 1)]] * 31))           # from the very first token on


def test_portions_of_many_sizes(setup):
    reqs = setup[3]
    _check(setup, setup[5].replay({"a": reqs["a"]}, [[("a", n)] for n in (2, 2, 3, 9, 16, 1, 17, 2, 15, 14, 2)]))
    _check(setup, setup[5].replay({"d": reqs["d"]}, [[("d", n)] for n in (15, 1, 16, 2, 16)]))


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
            assert row.max().item() - row[tok].item() <= (1e-3 if dtype == torch.float32 else 0.1) * spread, (k, tok)
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
                         cwd=root, capture_output=True, text=True, timeout=600)
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
    for dtype, tol in (("float32", F32_TOL), ("bfloat16", BF16_TOL)):
        out = tmp_path / ("out_" + dtype)
        run = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(model), "--dtype", dtype, "--out", str(out),
                              "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n", cwd=root,
                             capture_output=True, text=True, timeout=600)
        assert run.returncode == 0, run.stderr[-3000:]
        assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
        expect = {0: wa[[0, 39]], 1: wa[[40]], 2: wb[[8]], 3: torch.cat([wa[[41, 69]], wb[[8]]])}
        for i, want in expect.items():
            got = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
            assert got.shape == want.shape and row_error(got, want) < tol, (dtype, i)


def test_long_decoding_over_many_windows():
    """170 decoded tokens in a row: every window and every page border passes over decoded keys, the kept ones stay."""
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


@pytest.mark.parametrize("seed", range(8))
def test_configurations_drawn_from_seeds(seed):
    """Layer orders, shared weights, sizes, windows and constants drawn independently, pages of 64 tokens: whole prompts
    and a mixed schedule."""
    cfg = random_config(seed)
    weights = random_checkpoint(cfg, seed=seed)
    g = torch.Generator().manual_seed(seed)
    reqs = {n: torch.randint(0, cfg["vocab"], (k,), generator=g).tolist() for n, k in (("a", 140), ("b", 67), ("c", 3))}
    mixed = [[("a", 66), ("b", 2)], [("b", 63), ("a", 1), ("c", 2)], [("a", 2), ("b", 1)], [("c", 1), ("a", 60)], [("a", 1), ("b", 1)],
             [("a", 10)]]
    plain = {n: forward_with_routes(t, weights, cfg) for n, t in reqs.items()}
    for dtype, tol in ((torch.float32, F32_TOL), (torch.bfloat16, BF16_TOL)):
        engine = Engine(cfg, weights, dtype, blocks=6, slots=3, block_size=64)
        engine.forced = {n: c for n, (_, c) in plain.items()} if dtype == torch.bfloat16 else None
        for schedule in ([[(n, len(t))] for n, t in reqs.items()], mixed):
            got = engine.replay(reqs, schedule)
            for n in reqs:
                assert row_error(got[n], plain[n][0].float()) < tol, (dtype, n, row_error(got[n], plain[n][0].float()))
        del engine
