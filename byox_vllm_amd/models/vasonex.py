"""Vasonex: a decoder-only language model whose sublayers are normed before and after (layers/postnorm.py),

    x <- x + rms_norm(f(rms_norm(x) * w)) * w',

first with f = grouped softmax attention over a sliding window beside which the sequence's first tokens stay visible, with a
partial interleaved rotation and one output gate per head (layers/sliding_attention.py), then with f = the layer's
feed-forward (if it has one):

* ``dense``: W_down(silu(W_gate h + b) * (W_up h + b)) + b;
* ``moe``: experts W_down gelu(W_up h) of which each token uses the ``top`` with the largest sigmoid scores; a score
  multiplies its expert's input and the scores are not renormalised; an optional shared expert runs for every token and is
  gated by one sigmoid number per token (layers/moe.py).

Layers may use an earlier layer's weights: an entry with ``weights_of`` owns no tensors, only a cache of its own.  The head
is a matrix of its own behind a final RMS norm.

config.json: {"architecture": "Vasonex", "vocab", "width", "norm": {"eps"}, "layers": [{"type": "attention", "mixer":
{"heads", "kv_heads", "dim", "vdim", "scale", "mask": {"size", "keep_first"}, "rot": {"base", "dims", "scaling"}}, "mlp":
{"kind": "dense", "ff"} | {"kind": "moe", "router": {"experts", "top"}, "expert": {"ff"}, "shared": {"ff"}} | null,
"weights_of"}]}.  Checkpoint tensor names: 'embed', 'head', 'final.norm', 'l<i>.norm1|norm1b|norm2|norm2b',
'l<i>.mix.q|k|v|g|o', 'l<i>.mlp.gate|up|down[.b]', 'l<i>.mlp.router', 'l<i>.mlp.e<k>.up|down',
'l<i>.mlp.shared.up|down|sg'.

The residual is fp32 from the embedding to the final norm.  The model steps through portions: any mixture of prompt
pieces and single decoded tokens in one batch, each request continuing from its pages (engine/model_runner.py
run_portions)."""

import json
import re
from types import SimpleNamespace

import torch
from torch import nn

from byox_vllm_amd import kernels
from byox_vllm_amd.layers.linear import DenseLinear
from byox_vllm_amd.layers.moe import GatedMLP, UnaryMixtureOfExperts
from byox_vllm_amd.layers.postnorm import SandwichNorm
from byox_vllm_amd.layers.sliding_attention import SlidingAttention


def weight_owner(layers: list, i: int) -> int:
    """The layer whose tensors layer ``i`` uses: itself, or the end of its ``weights_of`` chain."""
    seen = {i}
    while layers[i].get("weights_of") is not None:
        i = int(layers[i]["weights_of"])
        assert 0 <= i < len(layers) and i not in seen, f"weights_of names layer {i}"
        seen.add(i)
    return i


def vasonex_config(raw: dict, dtype=torch.bfloat16):
    """config.json contents -> the configuration object the engine and the model read."""
    layers = json.loads(json.dumps(raw["layers"]))           # deep copy
    for i in range(len(layers)):
        own = layers[weight_owner(layers, i)]
        assert layers[i]["type"] == own["type"] and layers[i]["mixer"] == own["mixer"] \
            and layers[i].get("mlp") == own.get("mlp"), f"layer {i} and the layer whose weights it uses differ"
    return SimpleNamespace(
        architecture="Vasonex", vocab_size=raw["vocab"], hidden_size=raw["width"],
        norm_eps=float((raw.get("norm") or {}).get("eps", 1e-6)), layers=layers, num_hidden_layers=len(layers),
        max_position_embeddings=1 << 30, dtype=dtype, tie_word_embeddings=False)


class VasonexLayer(nn.Module):
    def __init__(self, cfg, spec: dict):
        super().__init__()
        width, m, mlp = cfg.hidden_size, spec["mixer"], spec.get("mlp")
        if spec["type"] != "attention":
            raise ValueError(f"unknown mixer type {spec['type']!r}")
        rot, mask = m.get("rot") or {}, m.get("mask") or {}
        self.norm1 = SandwichNorm(width, cfg.norm_eps)
        self.mix = SlidingAttention(width, m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"], m["scale"],
                                    int(mask.get("size") or 0), int(mask.get("keep_first") or 0), int(rot.get("dims") or 0),
                                    float(rot.get("base", 10000.0)), rot.get("scaling"), interleaved=True)
        self.norm2 = self.mlp = None
        self.moe = bool(mlp) and mlp["kind"] == "moe"
        if mlp:
            self.norm2 = SandwichNorm(width, cfg.norm_eps)
            if self.moe:
                self.mlp = UnaryMixtureOfExperts(width, mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"],
                                                 "gelu_erf", route="sigmoid", weigh="input",
                                                 shared_ff=(mlp.get("shared") or {}).get("ff"))
            elif mlp["kind"] == "dense":
                self.mlp = GatedMLP(width, mlp["ff"], "silu", bias=True)
            else:
                raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")

    def forward(self, x, pending, positions, run: int):
        """x: fp32 residual [T, width] (updated in place); pending: what the previous sublayer still owes it
        -> what this layer's last sublayer owes it."""
        y = self.mix(self.norm1.begin(x, pending), positions, run)
        pending = ({"y": y}, self.norm1)
        if self.mlp is not None:
            h = self.norm2.begin(x, pending)
            if self.moe:
                result = self.mlp(h)
            else:
                y, bias = self.mlp(h, defer_bias=True)
                result = {"y": y, "y_bias": bias}
            pending = (result, self.norm2)
        return pending


class VasonexForCausalLM(nn.Module):
    portioned = True          # steps through ModelRunner.run_portions: prompt pieces and decoded tokens in one batch
    prefix_cache = False      # portions extend a request's own pages; they do not look for another request's
    kernel_sources = ("linear", "rowops", "window_attn", "moe", "misc", "gemm_lt")

    @staticmethod
    def config_from_json(raw: dict, path: str | None):
        return vasonex_config(raw)

    def __init__(self, cfg):
        super().__init__()
        self.cfg = cfg
        width = cfg.hidden_size
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, width), requires_grad=False)
        # modules exist for the layers that own tensors; ``order`` = (module, number of its cache) of every layer
        self.layers, self.module_of, self.order = nn.ModuleList(), {}, []
        for i in range(len(cfg.layers)):
            own = weight_owner(cfg.layers, i)
            if own not in self.module_of:
                self.module_of[own] = len(self.layers)
                self.layers.append(VasonexLayer(cfg, cfg.layers[own]))
            at = self.module_of[own]
            self.order.append((at, self.layers[at].mix.add_run()))
        self.final_norm = SandwichNorm(width, cfg.norm_eps, final=True)
        self.head = DenseLinear(width, cfg.vocab_size)

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, positions, trace: list | None = None):
        """-> (fp32 residual [T, width], what the last sublayer still owes it).  ``trace`` collects the residual after
        every layer (a debugging aid: it adds the pending result in a launch of its own)."""
        x = kernels.embed_scale(input_ids, self.embed.data, 1.0)
        pending = None
        for at, run in self.order:
            pending = self.layers[at](x, pending, positions, run)
            if trace is not None:
                SandwichNorm.settle(x, pending)
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
        assert quantization is None, "Vasonex runs unquantised"
        for layer in self.layers:       # frequencies are fp32 whatever dtype the modules were built under
            assert layer.mix.inv_freq is None or layer.mix.inv_freq.dtype == torch.float32

    # ------------------------------------------------------------------ cache and state
    def page_layers(self):
        """Holders of paged cache rows: one per layer, also where layers share their weights."""
        return [self.layers[at].mix.runs[run] for at, run in self.order]

    def state_layers(self):
        """No layer keeps a recurrent state."""
        return []

    # ------------------------------------------------------------------ checkpoint names
    _LAYER = re.compile(r"^l(\d+)\.(.+)$")
    _EXPERT = re.compile(r"^e(\d+)\.(up|down)$")
    _NORMS = {"norm1": "norm1.pre", "norm1b": "norm1.post", "norm2": "norm2.pre", "norm2b": "norm2.post"}
    _DENSE = {"gate": ("gate_up.weight", "gate"), "up": ("gate_up.weight", "up"), "gate.b": ("gate_up.bias", "gate"),
              "up.b": ("gate_up.bias", "up"), "down": ("down.weight", None), "down.b": ("down.bias", None)}

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
        if not m or int(m.group(1)) not in self.module_of:
            return None
        at, rest = self.module_of[int(m.group(1))], m.group(2)
        base, layer = f"layers.{at}.", self.layers[at]
        if rest in self._NORMS:
            if layer.mlp is None and rest.startswith("norm2"):
                return None, None
            return base + self._NORMS[rest], None
        part, _, leaf = rest.partition(".")
        if part == "mix":
            if leaf == "o":
                return base + "mix.o.weight", None
            return (base + "mix.inp.weight", leaf) if leaf in ("q", "k", "v", "g") else None
        if part != "mlp" or layer.mlp is None:
            return None
        base += "mlp."
        if not layer.moe:
            return (base + self._DENSE[leaf][0], self._DENSE[leaf][1]) if leaf in self._DENSE else None
        if leaf == "router":
            return base + "router.weight", "router"
        e = self._EXPERT.match(leaf)
        if e and int(e.group(1)) < layer.mlp.experts:
            return base + e.group(2), int(e.group(1))
        if layer.mlp.shared_ff:
            if leaf == "shared.sg":
                return base + "router.weight", "sg"
            if leaf in ("shared.up", "shared.down"):
                path, shard = layer.mlp.shared_target(leaf[7:])
                return base + path, shard
        return None
