"""Feed-forward blocks on nv_linear: the gated unit W_down(act(W_gate h) * (W_up h)) as two launches (gate and up rows
share one product whose epilogue applies biases, activation and multiplication), a mixture of such units, and a mixture
of units without a gate (``UnaryMixtureOfExperts``).  ``GroupedMixtureOfExperts`` chooses within the best groups of
experts, by corrected scores, and knows experts that return their input.

Mixture: fp32 router logits, the ``top`` largest per token, softmax over the chosen logits only; the (token, choice)
pairs are ordered by expert on the device, the experts' two products run as grouped launches over the gathered rows
(one weight per group, no host synchronisation: the grid covers the worst case and empty tiles leave at once), and the
rows are summed per token in the order of its choices.  An optional shared expert runs for every token and is added
multiplied by sigmoid(w_sg . h), one number per token; its gate row rides in the router's product.

Variants a design may choose: ``route="all"`` takes the softmax over every expert and divides the chosen scores by their
sum (+ 1e-20); the activation ``"clamped"`` is the unit g sigmoid(1.702 g) (u + 1) with g = min(gate, limit) and
u = clamp(up, -limit, limit); ``forward(h, add)`` folds another fp32 result of the same rows (a mixer that runs beside
the feed-forward) into the combining launch; with ``own_router=False`` the layer has no router matrix and takes fp32
logits from the caller, whose own projection of the same rows carries the router's rows (one launch and one read of
the input fewer)."""

import torch
from torch import nn

from byox_vllm_amd import kernels
from byox_vllm_amd.layers.linear import DenseLinear
from byox_vllm_amd.layers.mlp import UNARY

ACTIVATIONS = {"silu": kernels.ACT_SILU, "gelu_tanh": kernels.ACT_GELU_TANH, "clamped": kernels.GLU_CLAMPED}
ROUTES = {"chosen": kernels.ROUTE_CHOSEN, "all": kernels.ROUTE_ALL, "sigmoid": kernels.ROUTE_SIGMOID,
          "softmax": kernels.ROUTE_SOFTMAX}


class GatedMLP(nn.Module):
    def __init__(self, width: int, ff: int, act: str, bias: bool = False):
        super().__init__()
        self.act = ACTIVATIONS[act]
        self.gate_up = DenseLinear(width, bias=bias, shards={"gate": ff, "up": ff})
        self.down = DenseLinear(ff, width, bias=bias)

    def forward(self, h, defer_bias: bool = False):
        """-> fp32 [T, width]; with ``defer_bias`` -> (the down-projection without its bias, that bias or None)."""
        hidden = self.gate_up(h, epilogue=kernels.EPI_GLU, act=self.act)
        if defer_bias:
            return kernels.linear(hidden, self.down.weight.data, out_dtype=torch.float32), \
                (self.down.bias.data if self.down.bias is not None else None)
        return self.down(hidden, out_dtype=torch.float32)


class MixtureOfExperts(nn.Module):
    def __init__(self, width: int, experts: int, top: int, ff: int, act: str = "silu", shared_ff: int | None = None,
                 route: str = "chosen", limit: float = 0.0, own_router: bool = True):
        super().__init__()
        self.experts, self.top, self.ff, self.width, self.act = experts, top, ff, width, ACTIVATIONS[act]
        self.route, self.limit = ROUTES[route], float(limit)
        assert act != "clamped" or self.limit > 0.0
        shards = {"router": experts}
        if shared_ff:
            shards["sg"] = 1
        assert own_router or not shared_ff
        self.router = DenseLinear(width, shards=shards) if own_router else None
        self.gate_up = nn.Parameter(torch.empty(experts, 2 * ff, width), requires_grad=False)
        self.down = nn.Parameter(torch.empty(experts, width, ff), requires_grad=False)
        self.gate_up.weight_loader = self._load_gate_up
        self.down.weight_loader = lambda p, t, e: p.data[e].copy_(t)
        self.shared = GatedMLP(width, shared_ff, act) if shared_ff else None

    def _load_gate_up(self, param, tensor, shard):
        e, part = shard
        at = 0 if part == "gate" else self.ff
        param.data[e, at: at + self.ff].copy_(tensor)

    def expert_rows(self, h, offsets, sorted_token):
        """The experts' outputs for the (token, choice) pairs ordered by expert, fp32 [T * top, width]."""
        T, E, top = h.size(0), self.experts, self.top
        hidden = kernels.linear(h, self.gate_up.data, rows=T * top, a_rows=sorted_token, batch=E,
                                w_batch_stride=2 * self.ff * self.width, group_offsets=offsets, max_group_rows=T,
                                epilogue=kernels.EPI_GLU, act=self.act, cap=self.limit)
        return kernels.linear(hidden, self.down.data, out_dtype=torch.float32, rows=T * top, batch=E,
                              w_batch_stride=self.width * self.ff, group_offsets=offsets, max_group_rows=T)

    def forward(self, h, add=None, logits=None):
        T, E, top = h.size(0), self.experts, self.top
        if logits is None:
            logits = self.router(h, out_dtype=torch.float32)
        assert logits.dtype == torch.float32 and logits.shape == (T, E + (1 if self.shared is not None else 0))
        idx, weights = kernels.moe_route(logits, E, top, self.route)
        offsets, sorted_token, slot_of = kernels.moe_sort(idx, E)
        y = self.expert_rows(h, offsets, sorted_token)
        if self.shared is None:
            return kernels.moe_combine(y, slot_of, weights, add)
        assert add is None, "a shared expert and an addend share one input of the combining launch"
        return kernels.moe_combine(y, slot_of, weights, self.shared(h), logits[:, E:])


class GroupedMixtureOfExperts(MixtureOfExperts):
    """Gated experts of which a token uses the ``top`` best of its ``keep`` best groups: the softmax over all router
    outputs gives scores s; s + correction (one learned number per output) is what is compared, groups of neighbouring
    outputs by their best member first; a chosen output weighs its expert by scale * s.  The last ``identity`` outputs
    have no expert: their output is the layer's input.

    The combining step is left to the consumer, as in UnaryMixtureOfExperts: ``forward`` returns the operands of
    kernels.sandwich_norm, whose launch gathers, weighs and sums the expert rows and adds the identity experts' share."""

    def __init__(self, width: int, experts: int, top: int, ff: int, act: str = "silu", route: str = "softmax",
                 identity: int = 0, groups: int = 0, keep_groups: int = 0, scale: float = 1.0):
        super().__init__(width, experts, top, ff, act, route=route, own_router=False)
        outputs = experts + identity
        assert groups == 0 or (outputs % groups == 0 and 0 < keep_groups <= groups), \
            f"{keep_groups} of {groups} groups of {outputs} router outputs"
        self.identity, self.groups, self.keep_groups, self.scale = identity, groups, keep_groups, float(scale)
        self.router = DenseLinear(width, outputs)
        # fp32 whatever the model dtype (16-bit checkpoint values widen exactly)
        self.correction = nn.Parameter(torch.zeros(outputs, dtype=torch.float32), requires_grad=False)

    def forward(self, h) -> dict:
        T, E, top = h.size(0), self.experts, self.top
        logits = self.router(h, out_dtype=torch.float32)
        self_weight = torch.empty(T, dtype=torch.float32, device=h.device) if self.identity else None
        offsets, tokens, _, slot_of, weights = kernels.moe_plan(
            logits, E, top, self.route, identity=self.identity, correction=self.correction.data, groups=self.groups,
            keep_groups=self.keep_groups, scale=self.scale, self_weight=self_weight, row_weights=False)
        y = self.expert_rows(h, offsets, tokens)
        result = {"y": y, "slot_of": slot_of, "weights": weights}
        if self.identity:
            result.update(self_rows=h, self_weight=self_weight)
        return result


class UnaryMixtureOfExperts(nn.Module):
    """Mixture of units without a gate, W_down act(W_up h), and optionally a shared one that runs for every token, gated by
    sigmoid(w_sg . h).  ``weigh`` says where a choice's weight acts: on the expert's "output" (sum_i w_i E_i(h)) or on its
    "input" (sum_i E_i(w_i h)); the latter is a factor per row of the up-projection's epilogue, since W_up (w h) =
    w (W_up h).

    The combining step is left to the consumer: ``forward`` returns the operands of kernels.sandwich_norm, whose launch
    gathers, weighs and sums the expert rows in front of the output norm.  While the step is short and the shared expert
    has the experts' size it runs as one more group of the same two grouped launches (every token's last choice); the rows
    of longer steps go through products of its own, which the many-row route serves."""

    FOLD_SHARED_UP_TO = 64     # tokens of a step

    def __init__(self, width: int, experts: int, top: int, ff: int, act: str = "gelu_erf", route: str = "chosen",
                 weigh: str = "output", shared_ff: int | None = None):
        super().__init__()
        assert weigh in ("input", "output") and 0 < top <= experts
        self.width, self.experts, self.top, self.ff, self.shared_ff = width, experts, top, ff, shared_ff
        self.act, self.route, self.weigh_input = UNARY[act], ROUTES[route], weigh == "input"
        self.router = DenseLinear(width, shards={"router": experts, **({"sg": 1} if shared_ff else {})})
        self.like_experts = shared_ff == ff        # the shared unit is stored behind the experts' when it has their size
        groups = experts + int(self.like_experts)
        self.up = nn.Parameter(torch.empty(groups, ff, width), requires_grad=False)
        self.down = nn.Parameter(torch.empty(groups, width, ff), requires_grad=False)
        self.up.weight_loader = self.down.weight_loader = self._load_expert
        if shared_ff and not self.like_experts:
            self.shared_up, self.shared_down = DenseLinear(width, shared_ff), DenseLinear(shared_ff, width)

    def _load_expert(self, param, tensor, e):
        assert param.data[e].shape == tensor.shape, f"{tuple(param.data[e].shape)} != {tuple(tensor.shape)}"
        param.data[e].copy_(tensor)

    def shared_target(self, which: str):
        """(parameter path below this module, shard) of the shared expert's matrix ``which`` = "up" | "down"."""
        return (which, self.experts) if self.like_experts else (f"shared_{which}.weight", None)

    def _shared_weights(self):
        if self.like_experts:
            return self.up.data[self.experts], self.down.data[self.experts]
        return self.shared_up.weight.data, self.shared_down.weight.data

    def forward(self, h) -> dict:
        T, E, top = h.size(0), self.experts, self.top
        logits = self.router(h, out_dtype=torch.float32)
        fold = self.like_experts and T <= self.FOLD_SHARED_UP_TO
        groups, rows = E + int(fold), T * (top + int(fold))
        offsets, tokens, row_weight, slot_of, weights = kernels.moe_plan(logits, E, top, self.route, fold)
        hidden = kernels.linear(h, self.up.data, rows=rows, a_rows=tokens, batch=groups, w_batch_stride=self.ff * self.width,
                                group_offsets=offsets, max_group_rows=T, epilogue=kernels.EPI_ACT, act=self.act,
                                row_scale=row_weight if self.weigh_input else None)
        y = kernels.linear(hidden, self.down.data, out_dtype=torch.float32, rows=rows, batch=groups,
                           w_batch_stride=self.width * self.ff, group_offsets=offsets, max_group_rows=T)
        result = {"y": y, "slot_of": slot_of}
        if not self.weigh_input:
            result["weights"] = torch.cat([weights, torch.ones_like(weights[:, :1])], 1) if fold else weights
        if not self.shared_ff:
            return result
        gate = logits[:, E]
        if fold:
            result["last_gate"] = gate
        else:
            up, down = self._shared_weights()
            hidden = kernels.linear(h, up, epilogue=kernels.EPI_ACT, act=self.act)
            result["shared"], result["shared_gate"] = kernels.linear(hidden, down, out_dtype=torch.float32), gate
        return result
