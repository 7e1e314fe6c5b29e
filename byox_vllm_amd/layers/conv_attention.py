"""Softmax attention with grouped key/value heads over a paged cache whose queries, keys and values pass through a short
causal convolution over time first:

    q, k, v = conv(W_q h), conv(W_k h), conv(W_v h)       per channel, y_t = sum_j w[:, j] u_(t - taps + 1 + j)
    q, k   <- every head divided by its root mean square (no weight, eps inside the root)
    s_ij   = q_i . k_j * scale   for 0 <= i - j < window (window 0: every j <= i)
    y      = W_o (concat_h(sum_j exp(s_ij) / (1 + sum_j' exp(s_ij')) v_j) * sigmoid(W_g h))

Positions enter through the convolution and the window alone.  The one added to the denominator is a sink: a key whose
score is 0 and which has no value.  A request's state is the last taps - 1 projected rows of q | k | v (fp32, in its state
slot) beside its pages, rows [k: G * dim | v: G * vdim] in the model dtype.  q | k | v | g are one merged projection left in
fp32; convolution, norms, scores, softmax, sink and gate are fp32.  Convolution, norms and page store are one launch
(csrc/window_attn.hip: nv_qk_conv_store) where the head sizes allow it, else two (nv_causal_conv, nv_qk_rotate_store); then
nv_paged_softmax_attn."""

import torch
from torch import nn

from byox_vllm_amd import kernels
from byox_vllm_amd.layers.conv import CausalConv1d
from byox_vllm_amd.layers.linear import DenseLinear
from byox_vllm_amd.utils.context import get_context


class ConvAttention(nn.Module):
    def __init__(self, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, taps: int, eps: float,
                 window: int = 0):
        super().__init__()
        assert heads % kv_heads == 0 and taps >= 1
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.scale, self.window, self.eps = float(scale), int(window), float(eps)
        qkv = {"q": heads * dim, "k": kv_heads * dim, "v": kv_heads * vdim}
        self.inp = DenseLinear(width, shards=dict(qkv, g=heads * vdim))
        self.conv = CausalConv1d(sum(qkv.values()), taps, bias=False, shards=qkv)
        self.o = DenseLinear(heads * vdim, width)
        self.register_buffer("sink", torch.zeros(heads), persistent=False)        # exp(0) = 1 joins the denominator
        self.cache = torch.tensor([])          # [pages * block_size, G * (dim + vdim)], bound by the runner
        self.block_size = 0

    def page_spec(self) -> dict:
        return {"width": self.kv_heads * (self.dim + self.vdim)}

    def state_modules(self):
        return [self.conv] if self.conv.taps > 1 else []

    def _queries(self, proj: torch.Tensor, positions: torch.Tensor, ctx) -> torch.Tensor:
        """Convolution, norms, keys and values to their pages -> fp32 queries [T, heads * dim], scaled."""
        H, G, d, dv = self.heads, self.kv_heads, self.dim, self.vdim
        k_at, v_at = H * d, (H + G) * d
        q = kernels.qk_conv_store(proj, (0, k_at, v_at), self.conv.weight.data, self.conv.state, ctx.cu_seqlens_q, ctx.past_lens,
                                  ctx.state_slots, ctx.seq_of_token, self.scale, ctx.slot_mapping, self.cache, H, G, d, dv,
                                  ctx.max_seqlen_q, unit_heads=True, eps=self.eps)
        if q is not None:
            return q
        rows, _ = self.conv(proj[:, :v_at + G * dv])
        return kernels.qk_rotate_store(rows, (0, k_at, v_at), positions, self.scale, ctx.slot_mapping, self.cache, H, G, d, dv,
                                       unit_heads=True, eps=self.eps)

    def forward(self, h: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        ctx = get_context()
        H, G, d, dv = self.heads, self.kv_heads, self.dim, self.vdim
        proj = self.inp(h, out_dtype=torch.float32)
        q = self._queries(proj, positions, ctx)
        out = torch.empty(h.size(0), H * dv, dtype=h.dtype, device=h.device)
        g = self.inp.offset("g")
        kernels.paged_softmax_attn(q, self.cache, ctx.block_tables, ctx.cu_seqlens_q, ctx.past_lens, ctx.seq_of_token,
                                   ctx.max_seqlen_q, H, G, d, dv, self.block_size, out, window=self.window, sink=self.sink,
                                   gate=proj[:, g:g + H * dv])
        return self.o(out, out_dtype=torch.float32)
