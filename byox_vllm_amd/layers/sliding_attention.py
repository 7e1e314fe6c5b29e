"""Softmax attention with grouped key/value heads over a paged cache, with a sliding window beside which the first tokens
of the sequence stay visible, a partial rotation, and one output gate per head:

    q, k = rotate(W_q h), rotate(W_k h),   v = W_v h      the first rot_dims numbers of every head turn with the position
    s_ij = q_i . k_j * scale   for j <= i and (i - j < window or j < keep_first)      (window 0: every j <= i)
    y    = W_o concat_h(sigmoid(W_g h)[h] * sum_j softmax(s)_ij v_j)

Kept tokens keep their place in the sequence: keys are rotated once, by their own position, when they are cached.  Pairs
are (2i, 2i + 1) when ``interleaved``, else (i, i + rot_dims/2).  Cache rows [k: G * dim | v: G * vdim] live in pages of the
engine's BlockManager in the model dtype; q | k | v | g are one merged projection left in fp32; rotation, scores, softmax
and gate are fp32 (csrc/window_attn.hip: nv_qk_rotate_store, nv_paged_softmax_attn).  A mixer whose weights serve several
layers keeps one cache per layer run (``add_run``)."""

import torch
from torch import nn

from byox_vllm_amd import kernels
from byox_vllm_amd.layers.linear import DenseLinear
from byox_vllm_amd.layers.rotary_embedding import scaled_inv_freq
from byox_vllm_amd.layers.sink_attention import CacheRun
from byox_vllm_amd.utils.context import get_context


class SlidingAttention(nn.Module):
    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, window: int = 0,
                 keep_first: int = 0, rot_dims: int = 0, rot_base: float = 10000.0, rot_scaling: dict | None = None,
                 interleaved: bool = False):
        super().__init__()
        assert heads % kv_heads == 0 and rot_dims % 2 == 0 and rot_dims <= dim
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.scale, self.window, self.keep_first = float(scale), int(window), int(keep_first)
        self.rot_dims, self.interleaved = int(rot_dims), bool(interleaved)
        self.inp = DenseLinear(width, shards={"q": heads * dim, "k": kv_heads * dim, "v": kv_heads * vdim, "g": heads})
        self.o = DenseLinear(heads * vdim, width)
        if rot_dims:
            inv_freq, self.magnitude = scaled_inv_freq(rot_dims, rot_base, rot_scaling)
            self.register_buffer("inv_freq", inv_freq.to(torch.float32), persistent=False)
        else:
            self.inv_freq, self.magnitude = None, 1.0
        self.runs: list[CacheRun] = []

    def add_run(self) -> int:
        """One more layer that uses these weights -> the number of its cache."""
        self.runs.append(CacheRun(self.kv_heads * (self.dim + self.vdim)))
        return len(self.runs) - 1

    def forward(self, h: torch.Tensor, positions: torch.Tensor, run: int = 0) -> torch.Tensor:
        ctx, own = get_context(), self.runs[run]
        H, G, d, dv = self.heads, self.kv_heads, self.dim, self.vdim
        proj = self.inp(h, out_dtype=torch.float32)
        q = kernels.qk_rotate_store(proj, (0, H * d, (H + G) * d), positions, self.scale, ctx.slot_mapping, own.cache, H, G, d,
                                    dv, inv_freq=self.inv_freq, rot_dims=self.rot_dims, interleaved=self.interleaved,
                                    mscale=self.magnitude)
        out = torch.empty(h.size(0), H * dv, dtype=h.dtype, device=h.device)
        g = self.inp.offset("g")
        kernels.paged_softmax_attn(q, own.cache, ctx.block_tables, ctx.cu_seqlens_q, ctx.past_lens, ctx.seq_of_token,
                                   ctx.max_seqlen_q, H, G, d, dv, own.block_size, out, window=self.window,
                                   keep_first=self.keep_first, gate=proj[:, g:g + H], gate_per_head=True)
        return self.o(out, out_dtype=torch.float32)
