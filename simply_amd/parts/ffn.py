"""Dense gated feed-forward: down(act(gate(x)) * up(x))  (simply/model_lib.py:643-730 with
use_gated_activation_in_ffn=True, ffn_use_bias=False; `act` by its name in the registry, as
simply/model_lib.py:723 looks `ffn_activation` up)."""
from __future__ import annotations

import torch

from ..kernels import ops
from ..registry import ACTIVATIONS, FEED_FORWARDS
from .base import FeedForward, ParamSpec, PendingNorm, as_product_weight, project

# activation name -> its code in the gated product's epilogue (simply/model_lib.py:93-104 registers these three)
ACTIVATIONS.register("gelu_tanh", ops.ACT_GELU_TANH)
ACTIVATIONS.register("silu", ops.ACT_SILU)
ACTIVATIONS.register("squared_relu", ops.ACT_SQUARED_RELU)
ACTIVATIONS.register("gelu_erf", ops.ACT_GELU_ERF)   # the exact GELU, x Phi(x)
# a rule for the two factors of a gated feed-forward (both clamped to a limit), not an activation of one
ACTIVATIONS.register("clamped_glu", ops.ACT_CLAMPED_GLU)


def check_limit(activation: str, limit: float | None) -> float | None:
    """The limit of the clamped gated rule: it comes with that rule and with no other activation."""
    clamped = int(ACTIVATIONS.get(activation)) == ops.ACT_CLAMPED_GLU
    if clamped != (limit is not None) or (limit is not None and not float(limit) > 0):
        raise ValueError(f"activation {activation!r} with limit {limit!r}: a positive limit goes with 'clamped_glu' alone")
    return None if limit is None else float(limit)


@FEED_FORWARDS.register("dense")
class Dense(FeedForward):
    """down(act(up(x))): one factor, no gate (simply/model_lib.py:643-730 with use_gated_activation_in_ffn=False)."""

    defers_sum = True

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "squared_relu"):
        self.hidden_size, self.intermediate_size = int(hidden_size), int(intermediate_size)
        self.activation = activation
        self.activation_code = int(ACTIVATIONS.get(activation))
        if self.activation_code == ops.ACT_CLAMPED_GLU:
            raise ValueError(f"dense: {activation!r} joins two factors, and this feed-forward has one")
        self.up_proj = self.down_proj = None

    def param_specs(self):
        D, F = self.hidden_size, self.intermediate_size
        return {"up_proj": ParamSpec((F, D)), "down_proj": ParamSpec((D, F))}

    def load(self, tensors):
        self.up_proj = as_product_weight(tensors["up_proj"])
        self.down_proj = as_product_weight(tensors["down_proj"])

    def forward(self, x: torch.Tensor, ctx=None, defer_sum=False) -> torch.Tensor:
        z = ops.gemm(x, self.up_proj, activate=self.activation_code)   # (the activation is the product's epilogue)
        return ops.gemm(z, self.down_proj, defer_sum=defer_sum)


@FEED_FORWARDS.register("gated_dense")
class GatedDense(FeedForward):
    """With activation 'clamped_glu' and its `limit` the two factors g = gate(x), u = up(x) are joined as
    g' sigmoid(1.702 g') (u' + 1) with g' = min(g, limit), u' = clamp(u, -limit, limit)."""

    accepts_pending = True
    defers_sum = True

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "gelu_tanh", limit: float | None = None):
        self.hidden_size, self.intermediate_size = int(hidden_size), int(intermediate_size)
        self.activation = activation
        self.activation_code = int(ACTIVATIONS.get(activation))   # an unknown name is refused with the known ones
        self.limit = check_limit(activation, limit)
        self.gate_proj = self.up_proj = self.down_proj = self.gate_up = None

    def param_specs(self):
        D, F = self.hidden_size, self.intermediate_size
        return {"gate_proj": ParamSpec((F, D)), "up_proj": ParamSpec((F, D)), "down_proj": ParamSpec((D, F))}

    def load(self, tensors):
        gate, up = tensors["gate_proj"], tensors["up_proj"]
        if gate.dtype == torch.bfloat16 and gate.is_cuda:
            # one tiled weight for both factors, their tiles in turn: the fused kernels stream it once
            from ..kernels.packing import pack_gate_up

            self.gate_up, self.gate_proj, self.up_proj = pack_gate_up(gate, up), None, None
        else:
            self.gate_up, self.gate_proj, self.up_proj = None, gate, up
        self.down_proj = as_product_weight(tensors["down_proj"])

    def forward(self, x: torch.Tensor, ctx=None, defer_sum=False) -> torch.Tensor:
        # gelu(x.Wg^T) * (x.Wu^T), one kernel
        if self.gate_up is not None:
            z = project(x, self.gate_up, activation=self.activation_code, limit=self.limit)
        else:
            if isinstance(x, PendingNorm):
                x = x.materialize()
            z = ops.gemm(x, self.gate_proj, w2=self.up_proj, activation=self.activation_code, limit=self.limit)
        return ops.gemm(z, self.down_proj, defer_sum=defer_sum)


@FEED_FORWARDS.register("routed_experts")
class RoutedExperts(FeedForward):
    """A mixture of experts: `num_experts` feed-forwards without biases, of which every token uses the `top` ones that
    the router chooses; an expert's result is weighted by its score times `router_scale`.

      gated       True: an expert is down(act(gate x) * (up x)); False: down(act(up x)), and there are no gate tensors
      activation  of the gated form also 'clamped_glu', with `limit` (`shared_limit` for the shared feed-forward)
      router      scores (32-bit) are the softmax of the router's logits over all experts ('softmax'), sigmoids of the
                  logits ('sigmoid'), or ('chosen_softmax') the logits themselves, and the weights are then the softmax
                  over the chosen experts' logits alone; the choice goes by score + a stored correction per expert (`correction`), and the
                  weights are the scores without the correction
      router_bias a stored bias per expert, added to the logits (32-bit)
      num_groups  equal groups of neighbouring experts; only experts of the `keep_groups` best can be chosen.  A group's
                  score: `group_score` 'two_largest', the sum of its two largest choice scores, or 'largest'
      renormalize None, or a small constant e: the weights are the chosen scores divided by their sum + e
      shared_size one more feed-forward of the experts' form runs for every token and is added, times sigmoid(w . x)
                  (one number per token) if `shared_gate`."""

    def __init__(self, hidden_size: int, num_experts: int, top: int, expert_size: int, router_scale: float = 1.0,
                 activation: str = "silu", shared_size: int | None = None, shared_gate: bool = True, gated: bool = True,
                 router: str = "softmax", correction: bool = False, num_groups: int = 1, keep_groups: int = 1,
                 group_score: str = "two_largest", renormalize: float | None = None, limit: float | None = None,
                 shared_limit: float | None = None, router_bias: bool = False):
        self.hidden_size, self.num_experts, self.top = int(hidden_size), int(num_experts), int(top)
        self.expert_size, self.router_scale = int(expert_size), float(router_scale)
        if not 1 <= self.top <= self.num_experts:
            raise ValueError(f"routed_experts: top {top} of {num_experts} experts")
        if router not in ("softmax", "sigmoid", "chosen_softmax"):
            raise ValueError(f"routed_experts: the router is 'softmax', 'sigmoid' or 'chosen_softmax', not {router!r}")
        if router == "chosen_softmax" and renormalize is not None:
            raise ValueError("routed_experts: weights that are the chosen logits' softmax sum to one by themselves")
        self.router_kind, self.correction, self.router_bias = router, bool(correction), bool(router_bias)
        self.num_groups, self.keep_groups = int(num_groups), int(keep_groups)
        if group_score not in ("two_largest", "largest"):
            raise ValueError(f"routed_experts: a group's score is its 'two_largest' or its 'largest', not {group_score!r}")
        self.group_best = 1 if group_score == "largest" else 2
        self.renormalize = None if renormalize is None else float(renormalize)
        if self.num_groups < 1 or self.num_experts % self.num_groups or not 1 <= self.keep_groups <= self.num_groups \
                or self.top > self.keep_groups * (self.num_experts // self.num_groups):
            raise ValueError(f"routed_experts: {num_experts} experts in {num_groups} groups of which {keep_groups} stay "
                             f"do not give {top} choices")
        self.gated = bool(gated)
        self.activation_code = int(ACTIVATIONS.get(activation))
        self.limit = check_limit(activation, limit)
        self.shared = None
        if shared_size and self.gated:
            self.shared = GatedDense(hidden_size, int(shared_size), activation, shared_limit)
        elif shared_size:
            self.shared = Dense(hidden_size, int(shared_size), activation)
        self.shared_gate = bool(shared_gate) and self.shared is not None
        self.router = self.gate_w = self.up_w = self.down_w = self.correction_w = self.router_bias_w = None

    def param_specs(self):
        D, F, E = self.hidden_size, self.expert_size, self.num_experts
        specs = {"router": ParamSpec((E, D))}
        if self.correction:
            specs["correction"] = ParamSpec((E,), role="vector", init="norm")
        if self.router_bias:
            specs["router_bias"] = ParamSpec((E,), role="vector", init="norm")
        for e in range(E):
            if self.gated:
                specs[f"e{e}.gate"] = ParamSpec((F, D))
            specs.update({f"e{e}.up": ParamSpec((F, D)), f"e{e}.down": ParamSpec((D, F))})
        if self.shared is not None:
            specs.update({"shared." + n: s for n, s in self.shared.param_specs().items()})
            if self.shared_gate:
                specs["shared.score"] = ParamSpec((1, D))
        return specs

    def load(self, tensors):
        from ..kernels.packing import stack_experts

        E = self.num_experts
        rows = [tensors["router"]] + ([tensors["shared.score"]] if self.shared_gate else [])
        # the router (and the shared expert's score) are one product, its result 32-bit
        self.router = as_product_weight(torch.cat(rows, dim=0).contiguous())
        self.gate_w = stack_experts(tensors[f"e{e}.gate"] for e in range(E)) if self.gated else None
        self.up_w = stack_experts(tensors[f"e{e}.up"] for e in range(E))
        self.down_w = stack_experts(tensors[f"e{e}.down"] for e in range(E))
        self.correction_w = tensors["correction"].contiguous() if self.correction else None
        self.router_bias_w = tensors["router_bias"].contiguous() if self.router_bias else None
        if self.shared is not None:
            self.shared.load({n: tensors["shared." + n] for n in self.shared.param_specs()})

    def forward(self, x: torch.Tensor, ctx=None) -> torch.Tensor:
        E = self.num_experts
        logits = ops.gemm(x, self.router, out_dtype=torch.float32)
        plain = self.router_kind == "softmax" and not self.correction and self.num_groups == 1 and self.renormalize is None \
            and not self.router_bias
        if not plain:
            experts, weights = ops.route_choice(logits[:, :E], self.top, self.router_scale, correction=self.correction_w,
                                                groups=self.num_groups, keep=self.keep_groups,
                                                softmax={"softmax": True, "sigmoid": False}.get(self.router_kind, "chosen"),
                                                group_best=self.group_best, renorm=self.renormalize,
                                                bias=self.router_bias_w)
        else:
            experts, weights = ops.route(logits[:, :E], self.top, self.router_scale)
        shared = self.shared.forward(x, ctx) if self.shared is not None else None
        return ops.routed_experts(x, experts, weights, self.gate_w, self.up_w, self.down_w, self.activation_code,
                                  shared=shared, shared_gate=logits[:, E:E + 1] if self.shared_gate else None, limit=self.limit)
