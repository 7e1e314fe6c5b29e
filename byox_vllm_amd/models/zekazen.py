"""Zekazen: a decoder-only language model of pre-norm layers,

    x <- x + mixer(rms_norm(x) * w1),   x <- x + ff(rms_norm(x) * w2),

whose mixers are

* ``retention``: linear attention with a constant decay per head, rotated queries and keys, every head's result divided by
  its root mean square and gated by silu (layers/matrix_memory.py);
* ``attention``: softmax attention over a sliding window behind a short convolution of queries, keys and values, with
  normalised queries and keys, a one in the softmax's denominator and a sigmoid output gate (layers/conv_attention.py);

and whose feed-forward is absent or a mixture of gated SiLU experts, chosen within the best groups by corrected softmax
scores, some of them the identity (layers/moe.py: GroupedMixtureOfExperts).  The head is a matrix of its own behind a final
RMS norm.

config.json: {"architecture": "Zekazen", "vocab", "width", "norm": {"eps"}, "layers": [{"type": "retention", "mixer": {"heads",
"dim", "vdim", "decay", "rot": {"base", "dims"}}} | {"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale",
"conv", "mask": {"size"}}}, each with "mlp": {"kind": "moe", "router": {"experts", "identity", "top", "groups": {"count",
"keep"}, "scale"}, "expert": {"ff"}} | null]}.  Checkpoint tensor names: 'embed', 'head', 'final.norm', 'l<i>.norm1|norm2',
'l<i>.mix.q|k|v|g|o', 'l<i>.mix.q|k|v.conv', 'l<i>.mlp.router|correction', 'l<i>.mlp.e<k>.gate|up|down'.

The residual is fp32 from the embedding to the final norm.  The model steps through portions: any mixture of prompt
pieces and single decoded tokens in one batch, each request continuing from its pages and its state slot
(engine/model_runner.py run_portions)."""

import json
import re
from types import SimpleNamespace

import torch
from torch import nn

from byox_vllm_amd import kernels
from byox_vllm_amd.layers.conv_attention import ConvAttention
from byox_vllm_amd.layers.linear import DenseLinear
from byox_vllm_amd.layers.matrix_memory import Retention
from byox_vllm_amd.layers.moe import GroupedMixtureOfExperts
from byox_vllm_amd.layers.postnorm import PreNorm


def zekazen_config(raw: dict, dtype=torch.bfloat16):
    """config.json contents -> the configuration object the engine and the model read."""
    layers = json.loads(json.dumps(raw["layers"]))           # deep copy
    return SimpleNamespace(
        architecture="Zekazen", vocab_size=raw["vocab"], hidden_size=raw["width"],
        norm_eps=float((raw.get("norm") or {}).get("eps", 1e-6)), layers=layers, num_hidden_layers=len(layers),
        max_position_embeddings=1 << 30, dtype=dtype, tie_word_embeddings=False)


class ZekazenLayer(nn.Module):
    def __init__(self, cfg, spec: dict):
        super().__init__()
        width, eps, m, mlp = cfg.hidden_size, cfg.norm_eps, spec["mixer"], spec.get("mlp")
        self.kind = spec["type"]
        self.norm1 = PreNorm(width, eps)
        self.rot = None           # (dims, base) of the rotation this layer's mixer reads
        if self.kind == "retention":
            rot = m.get("rot") or {}
            if rot.get("dims"):
                self.rot = (int(rot["dims"]), float(rot.get("base", 10000.0)))
            self.mix = Retention(width, m["heads"], m["dim"], m["vdim"], m["decay"], eps)
        elif self.kind == "attention":
            self.mix = ConvAttention(width, m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"], m["scale"],
                                     int(m.get("conv") or 1), eps, int((m.get("mask") or {}).get("size") or 0))
        else:
            raise ValueError(f"unknown mixer type {self.kind!r}")
        self.norm2 = self.mlp = None
        if mlp:
            if mlp["kind"] != "moe":
                raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
            r = mlp["router"]
            groups = r.get("groups") or {}
            self.norm2 = PreNorm(width, eps)
            self.mlp = GroupedMixtureOfExperts(width, r["experts"], r["top"], mlp["expert"]["ff"], "silu",
                                               identity=int(r.get("identity") or 0), groups=int(groups.get("count") or 0),
                                               keep_groups=int(groups.get("keep") or 0), scale=float(r.get("scale", 1.0)))

    def forward(self, x, pending, positions, tables: dict):
        """x: fp32 residual [T, width] (updated in place); pending: what the previous sublayer still owes it; tables: the
        step's cosines and sines by rotation -> what this layer's last sublayer owes it."""
        h = self.norm1.begin(x, pending)
        y = self.mix(h, rot=tables.get(self.rot)) if self.kind == "retention" else self.mix(h, positions)
        pending = ({"y": y}, self.norm1)
        if self.mlp is not None:
            pending = (self.mlp(self.norm2.begin(x, pending)), self.norm2)
        return pending


class ZekazenForCausalLM(nn.Module):
    portioned = True          # steps through ModelRunner.run_portions: prompt pieces and decoded tokens in one batch
    prefix_cache = False      # a recurrent state cannot be rebuilt from cached pages
    kernel_sources = ("linear", "rowops", "streams", "window_attn", "memory", "scan", "moe", "misc", "gemm_lt")

    @staticmethod
    def config_from_json(raw: dict, path: str | None):
        return zekazen_config(raw)

    def __init__(self, cfg):
        super().__init__()
        self.cfg = cfg
        width = cfg.hidden_size
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, width), requires_grad=False)
        self.layers = nn.ModuleList(ZekazenLayer(cfg, spec) for spec in cfg.layers)
        self.final_norm = PreNorm(width, cfg.norm_eps)
        self.head = DenseLinear(width, cfg.vocab_size)
        # frequencies base^(-2i / dims) in float64, once per rotation that occurs: the kernel forms the angles in double
        self.rotations = sorted({layer.rot for layer in self.layers if layer.rot is not None})
        for n, (dims, base) in enumerate(self.rotations):
            freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
            self.register_buffer(f"inv_freq{n}", torch.tensor(freq, dtype=torch.float64), persistent=False)

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, positions, trace: list | None = None):
        """-> (fp32 residual [T, width], what the last sublayer still owes it).  ``trace`` collects the residual after
        every layer (a debugging aid: it adds the pending result in a launch of its own)."""
        x = kernels.embed_scale(input_ids, self.embed.data, 1.0)
        tables = {rot: kernels.rotation_table(positions, getattr(self, f"inv_freq{n}"))
                  for n, rot in enumerate(self.rotations)}
        pending = None
        for layer in self.layers:
            pending = layer(x, pending, positions, tables)
            if trace is not None:
                PreNorm.settle(x, pending)
                pending = None
                trace.append(x.clone())
        return x, pending

    def compute_logits(self, state, rows_idx=None, out_dtype=torch.float32):
        """The last result and the final norm on the wanted rows, then the head -> logits [rows, vocab]."""
        x, pending = state
        if rows_idx is None:
            rows_idx = torch.arange(x.size(0), dtype=torch.int32, device=x.device)
        return self.head(self.final_norm.begin(x, pending, rows_idx), out_dtype=out_dtype)

    def finalize(self, quantization=None) -> None:
        assert quantization is None, "Zekazen runs unquantised"

    # ------------------------------------------------------------------ cache and state
    def page_layers(self):
        """Holders of paged cache rows."""
        return [l.mix for l in self.layers if l.kind == "attention"]

    def state_layers(self):
        """Holders of a piece of a request's state slot: every retention layer's memory, every convolution's last inputs."""
        return [s for l in self.layers for s in l.mix.state_modules()]

    # ------------------------------------------------------------------ checkpoint names
    _LAYER = re.compile(r"^l(\d+)\.(.+)$")
    _EXPERT = re.compile(r"^e(\d+)\.(gate|up|down)$")

    def checkpoint_target(self, name: str):
        """Checkpoint tensor name -> (parameter path, shard id or None); (None, None) for a tensor the configuration
        leaves without a consumer; None for a name this model does not own."""
        if name == "embed":
            return "embed", None
        if name == "head":
            return "head.weight", None
        if name == "final.norm":
            return "final_norm.pre", None
        m = self._LAYER.match(name)
        if not m or int(m.group(1)) >= len(self.layers):
            return None
        i, rest = int(m.group(1)), m.group(2)
        base, layer = f"layers.{i}.", self.layers[i]
        if rest == "norm1":
            return base + "norm1.pre", None
        if rest == "norm2":
            return (base + "norm2.pre", None) if layer.mlp is not None else (None, None)
        part, _, leaf = rest.partition(".")
        if part == "mix":
            if leaf == "o":
                return base + "mix.o.weight", None
            if layer.kind == "attention" and leaf in ("q.conv", "k.conv", "v.conv"):
                return base + "mix.conv.weight", leaf[0]
            return (base + "mix.inp.weight", leaf) if leaf in ("q", "k", "v", "g") else None
        if part != "mlp" or layer.mlp is None:
            return None
        if leaf == "router":
            return base + "mlp.router.weight", None
        if leaf == "correction":
            return base + "mlp.correction", None
        e = self._EXPERT.match(leaf)
        if e and int(e.group(1)) < layer.mlp.experts:
            if e.group(2) == "down":
                return base + "mlp.down", int(e.group(1))
            return base + "mlp.gate_up", (int(e.group(1)), e.group(2))
        return None
