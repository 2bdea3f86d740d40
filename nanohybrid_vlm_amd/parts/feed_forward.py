"""Feed-forward parts. ``SwiGLU`` follows nanovllm/models/qwen3.py:91-117."""
from __future__ import annotations

import torch

from ..native import ops
from .base import FEED_FORWARDS, ParamSpec, Part


@FEED_FORWARDS.register("swiglu")
class SwiGLU(Part):
    """down(silu(gate(x)) * up(x)); gate and up are one packed matrix whose first
    ``intermediate_size`` rows are the gate (nanovllm/layers/linear.py:102-108,
    nanovllm/layers/activation.py:10-11)."""

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "silu", bias: bool = False,
                 limit: float | None = None, alpha: float = 1.0, offset: float = 0.0):
        """``activation``: what the gate passes, "silu" (the reference's), "gelu_tanh", or "clamped_swish": with
        g' = min(g, ``limit``) and u' = clamp(u, -limit, limit), the result is g' sigmoid(``alpha`` g') (u' + ``offset``).
        ``bias``: all three projections have biases."""
        if activation == "clamped_swish":
            if limit is None or not limit > 0:
                raise ValueError(f"a clamped gate needs a positive limit, got {limit}")
            self.gate = ops.Gate(2, float(limit), float(alpha), float(offset))
        elif activation in ops.ACTIVATIONS:
            self.gate = ops.gate_of(activation)
        else:
            raise ValueError(f"activation {activation!r} is not known ({sorted(ops.ACTIVATIONS)} and 'clamped_swish' are)")
        self.hidden_size = hidden_size
        self.intermediate_size = intermediate_size
        self.activation, self.bias = activation, bool(bias)
        self.gate_up_weight = self.gate_up_bias = None
        self.down_weight = self.down_bias = None

    def param_specs(self):
        specs = {
            "gate_up.weight": ParamSpec((2 * self.intermediate_size, self.hidden_size)),
            "down.weight": ParamSpec((self.hidden_size, self.intermediate_size)),
        }
        if self.bias:
            specs["gate_up.bias"] = ParamSpec((2 * self.intermediate_size,), init="zeros")
            specs["down.bias"] = ParamSpec((self.hidden_size,), init="zeros")
        return specs

    takes_deferred_norm = True    # x goes straight into a product, which can norm it
    adds_to_residual = True       # the down projection can make the addition to the residual stream

    def first_product(self):
        """(weight, gated) of the product that x goes into."""
        return self.gate_up_weight, True

    def forward(self, x, step, add_to=None):
        y = ops.gated_linear(x, self.gate_up_weight, self.gate, self.gate_up_bias)
        return ops.linear(y, self.down_weight, self.down_bias, add_to=add_to)


@FEED_FORWARDS.register("plain_mlp")
class PlainMLP(Part):
    """down(act(up(x))) without a gate and without biases; ``activation``: "relu2" (the square of max(z, 0)), "silu"
    or "gelu_tanh". The activation is taken in float: on the up projection's finished sums where a step of few rows
    does both in one kernel, else on its rounded rows."""

    def __init__(self, hidden_size: int, intermediate_size: int, activation: str = "relu2"):
        if activation not in ops.PLAIN_ACTIVATIONS:
            raise ValueError(f"activation {activation!r} is not known ({sorted(ops.PLAIN_ACTIVATIONS)} are)")
        if min(hidden_size, intermediate_size) <= 0:
            raise ValueError(f"a feed-forward of {hidden_size} x {intermediate_size}")
        self.hidden_size, self.intermediate_size, self.activation = hidden_size, intermediate_size, activation
        self.up_weight = self.down_weight = None

    def param_specs(self):
        return {"up.weight": ParamSpec((self.intermediate_size, self.hidden_size)),
                "down.weight": ParamSpec((self.hidden_size, self.intermediate_size))}

    def forward(self, x, step):
        return ops.linear(ops.activated_linear(x, self.up_weight, self.activation), self.down_weight)


@FEED_FORWARDS.register("routed_experts")
class RoutedExperts(Part):
    """``num_experts`` feed-forwards (gated, unless ``gated`` says False) of inner size ``expert_size`` without biases, of which every token uses the
    ``top`` with the largest router logit z_e = router_e . x (+ b_e with ``router_bias``; summed and kept in float32).
    ``scoring`` "sigmoid": the score s_e = sigmoid(z_e), taken as it is (not renormalised); "softmax_of_chosen": the
    scores are the softmax over the chosen logits alone. ``scores_on`` "input": the score multiplies the expert's input,
    y = sum over chosen e of D_e (act(G_e s_e x) * (U_e s_e x)); "output": it weighs the expert's output,
    y = sum over chosen e of s_e D_e (act(G_e x) * (U_e x)). ``shared``: the description of one more feed-forward that
    every token uses and whose result is added (its tensors lie under ``shared.``).
    ``gated`` False: an expert is D_e act(U_e x). ``scoring`` "softmax": the scores are the softmax over all experts' logits,
    taken as they are; only with it: ``correction``, a float32 number per expert that is added to the scores for the choice
    alone; ``groups`` (count, keep), the choice is made among the experts of the ``keep`` best of ``count`` equal runs of
    neighbours (by their largest score with its correction); ``identity`` n, the router's last n outputs stand for experts
    without tensors that hand their input on.
    All experts' matrices lie in two tensors, [experts * 2 expert_size, width] (per expert its gate rows, then its
    up rows; without a gate [experts * expert_size, width]) and [experts * width, expert_size]."""

    def __init__(self, hidden_size: int, num_experts: int, top: int, expert_size: int, activation: str = "silu",
                 scoring: str = "sigmoid", scores_on: str = "input", router_bias: bool = False, shared: dict | None = None,
                 gated: bool = True, correction: bool = False, groups: tuple | None = None, identity: int = 0, **offered):
        if not 0 < top <= num_experts + identity or identity < 0 or min(hidden_size, expert_size) <= 0:
            raise ValueError(f"{top} of {num_experts} experts of size {expert_size}")
        known = ops.ACTIVATIONS if gated else ops.PLAIN_ACTIVATIONS
        if activation not in known:
            raise ValueError(f"activation {activation!r} is not known ({sorted(known)} are)")
        if scoring not in (*ops.ROUTER_SCORES, "softmax"):
            raise ValueError(f"scoring {scoring!r} is not known ({sorted((*ops.ROUTER_SCORES, 'softmax'))} are)")
        if scoring == "softmax":
            count, keep = groups if groups is not None else (1, 1)
            if router_bias or scores_on != "output":
                raise ValueError("scores over all experts weigh the outputs, and their logits have no bias")
            if not 0 < keep <= count or (num_experts + identity) % count or top > keep * ((num_experts + identity) // count):
                raise ValueError(f"{top} of {num_experts} experts and {identity} identities, {keep} of {count} groups")
            self.groups = (count, keep)
        elif correction or groups is not None or identity:
            raise ValueError("a correction, groups and identity experts go with scoring 'softmax'")
        if scores_on not in ("input", "output"):
            raise ValueError(f"scores on {scores_on!r}: 'input' and 'output' are known")
        self.hidden_size, self.num_experts, self.top, self.expert_size = hidden_size, num_experts, top, expert_size
        self.activation, self.scoring, self.scores_on, self.has_router_bias = activation, scoring, scores_on, bool(router_bias)
        self.shared = FEED_FORWARDS.build(shared, offered=offered) if shared is not None else None
        self.gated, self.has_correction, self.identity = bool(gated), bool(correction), int(identity)
        self.router_bias = self.correction = None

    def children(self):
        return {"shared": self.shared} if self.shared is not None else {}

    def param_specs(self):
        E, F, W = self.num_experts, self.expert_size, self.hidden_size
        specs = {"router.weight": ParamSpec((E + self.identity, W)),
                 ("gate_up.weight" if self.gated else "up.weight"): ParamSpec((E * (2 if self.gated else 1) * F, W)),
                 "down.weight": ParamSpec((E * W, F))}
        if self.has_router_bias:
            specs["router.bias"] = ParamSpec((E,), init="zeros", always_float32=True)
        if self.has_correction:
            specs["router.correction"] = ParamSpec((E + self.identity,), always_float32=True, init_mean=0.0, init_std=0.02)
        return specs

    def bind(self, params):
        E, F, W = self.num_experts, self.expert_size, self.hidden_size
        self.router_weight = params["router.weight"]
        self.router_bias, self.correction = params.get("router.bias"), params.get("router.correction")
        self.gate_up_weight = params["gate_up.weight"].view(E, 2 * F, W) if self.gated else params["up.weight"].view(E, F, W)
        self.down_weight = params["down.weight"].view(E, W, F)

    def forward(self, x, step):
        logits = ops.linear(x, self.router_weight, out_dtype=torch.float32)
        if self.scoring == "softmax":
            ids, scores = ops.route_groups(logits, self.top, self.correction, *self.groups)
        else:
            ids, scores = ops.route_topk(logits, self.top, bias=self.router_bias, scoring=self.scoring)
        if self.shared is None and self.scores_on == "input":
            return ops.routed_experts(x, ids, scores, self.gate_up_weight, self.down_weight, self.activation)
        add = self.shared.forward(x, step) if self.shared is not None else None
        return ops.routed_experts(x, ids, scores, self.gate_up_weight, self.down_weight, self.activation,
                                  scores_on=self.scores_on, add=add, **({} if self.gated else {"gated": False}),
                                  **({"identity": True} if self.identity else {}))
