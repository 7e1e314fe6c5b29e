"""Plain, slow restatement of the Zekazen design in float64 PyTorch on the CPU: one function per mechanism, whole
sequences only, no cache, no batching, nothing shared with byox_vllm_amd.  Tests compare the engine (portions, pages,
state slots, mixed batches) with these functions run on each request's full token list.

Weights are a dict keyed by the checkpoint's tensor names; ``cfg`` is the config.json dict."""

import math

import torch

F = torch.float64


def silu(z):
    return z * torch.sigmoid(z)


def rms(x, eps):
    """Every vector along the last axis over its root mean square, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rotate(x, positions, dims, base):
    """x [T, H, d]: numbers i and i + dims/2 of every head turn together by p * base^(-2i/dims), i < dims/2."""
    half = dims // 2
    if half == 0:
        return x
    freq = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(half)], dtype=F)
    angle = positions.to(F)[:, None] * freq[None, :]
    c, s = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def retention(q, k, v, decay):
    """q, k [T, H, d], v [T, H, dv], decay [H]: S <- decay S + k v^T from zero, o = S^T q.  -> [T, H, dv]"""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=F)
    out = []
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def retention_mixer(h, W, pre, m, eps):
    H, d, dv, T = m["heads"], m["dim"], m["vdim"], h.shape[0]
    rot, p = m.get("rot") or {}, torch.arange(T)
    dims, base = int(rot.get("dims") or 0), float(rot.get("base", 10000.0))
    q = rotate((h @ W[pre + "q"].T).view(T, H, d), p, dims, base)
    k = rotate((h @ W[pre + "k"].T).view(T, H, d), p, dims, base) * d ** -0.5
    v = (h @ W[pre + "v"].T).view(T, H, dv)
    o = rms(retention(q, k, v, torch.tensor(m["decay"], dtype=F)), eps).reshape(T, H * dv)
    return (o * silu(h @ W[pre + "g"].T)) @ W[pre + "o"].T


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros ahead of the first row."""
    T, taps = u.shape[0], w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F), u])
    return sum(w[:, j] * padded[j:j + T] for j in range(taps))


def sees(i, j, window):
    """Does position i see position j?  window 0: every earlier one."""
    return 0 <= i - j and (window == 0 or i - j < window)


def sink_attention(q, k, v, scale, window):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; the softmax's denominator holds one more exp(0).  -> [T, H, dv]"""
    T, H = q.shape[:2]
    per = H // k.shape[1]
    mask = torch.tensor([[sees(i, j, window) for j in range(T)] for i in range(T)])
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T * scale).masked_fill(~mask, -math.inf)
        top = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
        e = torch.exp(s - top)
        out.append(e / (torch.exp(-top) + e.sum(-1, keepdim=True)) @ v[:, h // per])
    return torch.stack(out, 1)


def attention_mixer(h, W, pre, m, eps):
    H, G, d, dv, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    y = {}
    for name in "qkv":
        y[name] = h @ W[pre + name].T
        if pre + name + ".conv" in W:
            y[name] = causal_conv(y[name], W[pre + name + ".conv"])
    q, k = rms(y["q"].view(T, H, d), eps), rms(y["k"].view(T, G, d), eps)
    o = sink_attention(q, k, y["v"].view(T, G, dv), float(m["scale"]), int((m.get("mask") or {}).get("size") or 0))
    return (o.reshape(T, H * dv) * torch.sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


def route(z, correction, spec):
    """Router logits [T, E + I] -> (chosen [T, top], weights [T, top]).  Scores are the softmax over all outputs; they are
    compared after adding ``correction``; only the ``keep`` groups with the largest best member may be chosen from."""
    top, n = spec["top"], z.shape[1]
    s = torch.softmax(z, -1)
    c = s + correction
    groups = spec.get("groups")
    if groups:
        count, keep = groups["count"], groups["keep"]
        best = c.view(-1, count, n // count).max(-1).values
        kept = torch.zeros_like(best, dtype=torch.bool).scatter(1, best.topk(keep, -1).indices, True)
        c = c.masked_fill(~kept.repeat_interleave(n // count, 1), -math.inf)
    idx = c.topk(top, -1).indices
    return idx, s.gather(1, idx) * float(spec.get("scale", 1.0))


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def moe(h, W, pre, spec):
    """Outputs ``experts`` .. ``experts + identity - 1`` of the router return their input."""
    E = spec["router"]["experts"]
    idx, wt = route(h @ W[pre + "router"].T, W[pre + "correction"], spec["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(idx[t].tolist(), wt[t]):
            y = h[t] if e >= E else expert(h[t], W[f"{pre}e{e}.gate"], W[f"{pre}e{e}.up"], W[f"{pre}e{e}.down"])
            out[t] += w * y
    return out


MIXERS = {"retention": retention_mixer, "attention": attention_mixer}


def forward(tokens, W, cfg, trace=None):
    """Token ids -> logits [T, vocab] (float64).  ``trace`` collects the residual after every layer."""
    W = {k: v.to(F) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, spec in enumerate(cfg["layers"]):
        x = x + MIXERS[spec["type"]](rms(x, eps) * W[f"l{i}.norm1"], W, f"l{i}.mix.", spec["mixer"], eps)
        if spec.get("mlp"):
            x = x + moe(rms(x, eps) * W[f"l{i}.norm2"], W, f"l{i}.mlp.", spec["mlp"])
        if trace is not None:
            trace.append(x)
    return (rms(x, eps) * W["final.norm"]) @ W["head"].T


def random_weights(cfg, seed=0):
    """A checkpoint of the design's tensor names for ``cfg``, values representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    width, W = cfg["width"], {}

    def mat(n, k, s=None):
        return (torch.randn(n, k, generator=g) * (k ** -0.5 if s is None else s)).to(torch.bfloat16)

    def vec(n, s=0.1, at=1.0):
        return (at + torch.randn(n, generator=g) * s).to(torch.bfloat16)

    W["embed"], W["head"], W["final.norm"] = mat(cfg["vocab"], width, 1.0), mat(cfg["vocab"], width), vec(width)
    for i, spec in enumerate(cfg["layers"]):
        m, p, mlp = spec["mixer"], f"l{i}.", spec.get("mlp")
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        G = m["kv_heads"] if spec["type"] == "attention" else H
        W[p + "norm1"] = vec(width)
        for name, n in (("q", H * d), ("k", G * d), ("v", G * dv)):
            W[p + "mix." + name] = mat(n, width)
            if spec["type"] == "attention" and m.get("conv"):
                W[p + f"mix.{name}.conv"] = mat(n, m["conv"], 0.3)
                W[p + f"mix.{name}.conv"][:, -1] += 0.7
        W[p + "mix.g"], W[p + "mix.o"] = mat(H * dv, width), mat(width, H * dv)
        if mlp:
            r, ff = mlp["router"], mlp["expert"]["ff"]
            n = r["experts"] + r.get("identity", 0)
            W[p + "norm2"] = vec(width)
            W[p + "mlp.router"], W[p + "mlp.correction"] = mat(n, width, 2.0 * width ** -0.5), vec(n, 0.1, -0.05)
            for e in range(r["experts"]):
                W[f"{p}mlp.e{e}.gate"], W[f"{p}mlp.e{e}.up"] = mat(ff, width), mat(ff, width)
                W[f"{p}mlp.e{e}.down"] = mat(width, ff)
    return W
