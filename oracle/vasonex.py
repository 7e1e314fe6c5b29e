"""Plain, slow restatement of the Vasonex design in float64 PyTorch on the CPU: one function per mechanism, whole
sequences only, no cache, no batching, nothing shared with byox_vllm_amd.  Tests compare the engine (portions, pages,
mixed batches) with these functions run on each request's full token list.

Weights are a dict keyed by the checkpoint's tensor names; ``cfg`` is the config.json dict."""

import math

import torch

F = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def frequencies(rot):
    """rot = {"base", "dims", "scaling": {"factor", "low", "high", "original"} | absent} -> angle per position, one per
    pair.  A pair's wavelength decides: short ones keep their frequency, long ones get it divided by ``factor``, those
    between blend the two linearly in original / wavelength."""
    dims, base = int(rot["dims"]), float(rot["base"])
    sc = rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            factor, low, high, original = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            wavelength = 2.0 * math.pi / f
            if wavelength > original / low:
                f = f / factor
            elif wavelength >= original / high:
                s = (original / wavelength - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=F)


def rotate_pairs(x, positions, freq):
    """x [T, heads, dim]: numbers 2i and 2i + 1 of every head turn by position * freq[i]; the rest pass."""
    n = 2 * freq.numel()
    a = positions.to(F)[:, None, None] * freq
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out = x.clone()
    out[..., 0:n:2] = u * torch.cos(a) - v * torch.sin(a)
    out[..., 1:n:2] = v * torch.cos(a) + u * torch.sin(a)
    return out


def visible(T, mask):
    """bool [query, key]: causal; with a mask only the last ``size`` tokens, and the first ``keep_first`` of the sequence."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if mask and mask.get("size"):
        seen = seen & ((i - j < int(mask["size"])) | (j < int(mask.get("keep_first") or 0)))
    return seen


def softmax_attention(q, k, v, scale, seen):
    """q [T, H, d], k [T, G, d], v [T, G, dv], seen [T, T] -> [T, H, dv]; query head h reads key head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    out = torch.empty(q.shape[0], H, v.shape[2], dtype=F)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        out[:, h] = torch.softmax(s.masked_fill(~seen, float("-inf")), -1) @ v[:, g]
    return out


def attention_mixer(h, W, p, m):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
    q, k = (h @ W[p + "q"].T).view(T, H, d), (h @ W[p + "k"].T).view(T, G, d)
    v = (h @ W[p + "v"].T).view(T, G, dv)
    if m.get("rot"):
        freq, pos = frequencies(m["rot"]), torch.arange(T)
        q, k = rotate_pairs(q, pos, freq), rotate_pairs(k, pos, freq)
    o = softmax_attention(q, k, v, float(m["scale"]), visible(T, m.get("mask")))
    o = o * torch.sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ W[p + "o"].T


def dense_unit(h, W, p):
    gate = h @ W[p + "gate"].T + W[p + "gate.b"]
    up = h @ W[p + "up"].T + W[p + "up.b"]
    return (silu(gate) * up) @ W[p + "down"].T + W[p + "down.b"]


def expert(x, W, p):
    return gelu_erf(x @ W[p + "up"].T) @ W[p + "down"].T


def route(z, top):
    """Router logits [T, E] -> (chosen experts [T, top], their sigmoid scores as they are)."""
    s = torch.sigmoid(z)
    idx = z.topk(top, dim=-1).indices            # the order of the scores, without their saturation
    return idx, s.gather(-1, idx)


def moe(h, W, p, spec):
    """The chosen experts read the input times their weight; a shared expert, gated by one number, reads it as it is."""
    idx, wt = route(h @ W[p + "router"].T, spec["router"]["top"])
    out = torch.zeros(h.shape[0], h.shape[1], dtype=F)
    for e in range(spec["router"]["experts"]):
        for j in range(idx.shape[1]):
            rows = (idx[:, j] == e).nonzero()[:, 0]
            out[rows] += expert(wt[rows, j, None] * h[rows], W, f"{p}e{e}.")
    if spec.get("shared"):
        out = out + torch.sigmoid(h @ W[p + "shared.sg"].T) * expert(h, W, p + "shared.")
    return out


def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(tokens, W, cfg, trace=None):
    """Token ids -> logits [T, vocab] (float64).  ``trace`` collects the residual after every layer."""
    W = {k: v.to(F) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{owner(cfg, i)}."
        y = attention_mixer(rms_norm(x, W[p + "norm1"], eps), W, p + "mix.", spec["mixer"])
        x = x + rms_norm(y, W[p + "norm1b"], eps)
        mlp = spec.get("mlp")
        if mlp:
            h = rms_norm(x, W[p + "norm2"], eps)
            y = dense_unit(h, W, p + "mlp.") if mlp["kind"] == "dense" else moe(h, W, p + "mlp.", mlp)
            x = x + rms_norm(y, W[p + "norm2b"], eps)
        if trace is not None:
            trace.append(x)
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T


def random_weights(cfg, seed=0):
    """A checkpoint of the design's tensor names for ``cfg``, values representable in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    width, W = cfg["width"], {}

    def mat(n, k, s=1.0):
        return (torch.randn(n, k, generator=g) * s * k ** -0.5).to(torch.bfloat16)

    def vec(n, at=0.0, s=0.1):
        return (at + torch.randn(n, generator=g) * s).to(torch.bfloat16)

    W["embed"] = mat(cfg["vocab"], width, width ** 0.5)
    for i, spec in enumerate(cfg["layers"]):
        if spec.get("weights_of") is not None:
            continue
        m, p, mlp = spec["mixer"], f"l{i}.", spec.get("mlp")
        H, G, d, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]
        W[p + "norm1"], W[p + "norm1b"] = vec(width, 1.0), vec(width, 1.0)
        for name, n in (("q", H * d), ("k", G * d), ("v", G * dv), ("g", H)):
            W[p + "mix." + name] = mat(n, width)
        W[p + "mix.o"] = mat(width, H * dv)
        if not mlp:
            continue
        W[p + "norm2"], W[p + "norm2b"] = vec(width, 1.0), vec(width, 1.0)
        if mlp["kind"] == "dense":
            for name, n, k in (("gate", mlp["ff"], width), ("up", mlp["ff"], width), ("down", width, mlp["ff"])):
                W[p + "mlp." + name], W[p + "mlp." + name + ".b"] = mat(n, k), vec(n, 0.0, 0.3)
            continue
        W[p + "mlp.router"] = mat(mlp["router"]["experts"], width, 2.0)
        for e in range(mlp["router"]["experts"]):
            W[f"{p}mlp.e{e}.up"], W[f"{p}mlp.e{e}.down"] = mat(mlp["expert"]["ff"], width, 2.0), mat(width, mlp["expert"]["ff"])
        if mlp.get("shared"):
            ff = mlp["shared"]["ff"]
            W[p + "mlp.shared.up"], W[p + "mlp.shared.down"] = mat(ff, width, 2.0), mat(width, ff)
            W[p + "mlp.shared.sg"] = mat(1, width)
    W["final.norm"], W["head"] = vec(width, 1.0), mat(cfg["vocab"], width)
    return W
