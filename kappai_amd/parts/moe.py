"""Mixture of experts: ``experts`` small gated feed-forward layers, of which every token uses
``top``.  Router logits ``W_router h`` in float32; the ``top`` largest are chosen and their
weights are the softmax over the chosen logits alone; the output is the weighted sum of the
chosen experts' ``W_down (silu(W_gate h) * W_up h)``.  Experts have no biases.  ``activation``
"relu_squared": the experts have no gate, ``W_down relu(W_up h)^2``.  ``router_bias``: a bias [E]
on the router's logits.  ``scoring`` "sigmoid": the router squashes every logit by itself, ``s =
sigmoid(z)``; the choice goes by ``s`` plus a learned ``correction`` [E] (where there is one), among
the experts of the ``keep_groups`` best of ``groups`` equal groups of neighbours (a group's worth:
the sum of its ``group_best`` largest such values), and the weights are the chosen experts' ``s`` times
``weight_scale``, without the correction and not renormalised.  ``scoring`` "softmax_all": the same
with ``s = softmax(z)`` over all experts.  ``activation`` "clamped": the gated form with ``g = min(W_gate
h, limit)``, ``u = clamp(W_up h, -limit, limit)`` and ``g sigmoid(slope g) (u + shift)``
(``ops.ClampedGate``).  ``identity``: the router counts that many more experts behind the others, whose
result is their input itself; they have no tensors, and their pairs take part in no product.
``shared_hidden``: one more expert of that size and the same form (``<prefix>shared.``) runs for every
row, and its result is added with weight one, or with ``shared_gate`` times ``sigmoid(W_sg h)``, one
number a row (a row more of the router's product, in float32).

The step's (row, choice) pairs are sorted by expert on the GPU and the experts' products run
over that order tile by tile, so nothing of the routing is read by the host.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..kernels import ops, profile, tuning
from ..weights.spec import INIT_NORMAL, INIT_SMALL, MATRIX, VECTOR, TensorSpec
from .base import FeedForward, register_part
from .feed_forward import SwiGLU
from .linear import Linear


class MixtureOfExperts(FeedForward):
    SCORINGS = ("softmax", "sigmoid", "softmax_all")
    ACTIVATIONS = ("silu_gated", "relu_squared", "clamped")

    def __init__(self, prefix: str, width: int, hidden: int, experts: int, top: int,
                 dtype: torch.dtype, names=None, weight_suffix: str = ".weight",
                 activation: str = "silu_gated", router_bias: bool = False,
                 shared_hidden: Optional[int] = None, bias_suffix: str = ".bias",
                 scoring: str = "softmax", correction: bool = False, groups: int = 1,
                 keep_groups: int = 1, weight_scale: float = 1.0, group_best: int = 2,
                 identity: int = 0, clamp: Optional[ops.ClampedGate] = None,
                 shared_clamp: Optional[ops.ClampedGate] = None, shared_gate: bool = False):
        n = {"router": "router", "expert": "e{}.", "gate": "gate", "up": "up", "down": "down",
             "shared": "shared.", "correction": "correction", "shared_gate": "sg"}
        n.update(names or {})
        if scoring not in self.SCORINGS:
            raise ValueError(f"{prefix}: unknown router scoring {scoring!r}; known: "
                             f"{', '.join(self.SCORINGS)}")
        if scoring == "softmax" and (correction or groups != 1 or weight_scale != 1.0):
            raise ValueError(f"{prefix}: a correction, groups and a weight scale go with the "
                             "sigmoid or the softmax_all scoring")
        if identity < 0 or group_best not in (1, 2):
            raise ValueError(f"{prefix}: {identity} experts that hand their input on, {group_best} "
                             "values a group")
        routed = experts + identity
        if not (groups >= 1 and routed % groups == 0 and 1 <= keep_groups <= groups
                and top <= routed // groups * keep_groups):
            raise ValueError(f"{prefix}: {top} experts a token from the best {keep_groups} of "
                             f"{groups} groups of {routed} experts")
        if activation not in self.ACTIVATIONS:
            raise ValueError(f"{prefix}: unknown expert activation {activation!r}; known: "
                             f"{', '.join(self.ACTIVATIONS)}")
        if not 1 <= top <= min(routed, ops.MOE_MAX_TOP):
            raise ValueError(f"{prefix}: {top} of {routed} experts a token; the kernels take 1 to "
                             f"{ops.MOE_MAX_TOP}")
        if (activation == "clamped") != (clamp is not None):
            raise ValueError(f"{prefix}: the clamped gate comes with its constants")
        if shared_gate and (not shared_hidden or scoring == "softmax"):
            raise ValueError(f"{prefix}: a gate on the shared expert goes with a shared expert and "
                             "the sigmoid or the softmax_all scoring")
        self.prefix, self.width, self.hidden, self.dtype = prefix, width, hidden, dtype
        self.E, self.top = int(experts), int(top)
        self.identity, self.group_best, self.clamp = int(identity), int(group_best), clamp
        self.gated = activation != "relu_squared"
        self._kinds = ("gate", "up", "down") if self.gated else ("up", "down")
        self._router = prefix + n["router"] + weight_suffix
        self._router_bias = prefix + n["router"] + bias_suffix if router_bias else None
        self.scoring, self.weight_scale = scoring, float(weight_scale)
        self.groups, self.keep_groups = int(groups), int(keep_groups)
        self._correction = prefix + n["correction"] if correction else None
        self.correction: Optional[torch.Tensor] = None
        self._expert = [{k: prefix + n["expert"].format(e) + n[k] + weight_suffix
                         for k in self._kinds} for e in range(self.E)]
        self.router_bias: Optional[torch.Tensor] = None
        self.shared_up = self.shared_down = self.shared = self._shared_gate = None
        sp = prefix + n["shared"]
        if shared_gate:
            self._shared_gate = sp + n["shared_gate"] + weight_suffix
        if shared_hidden and self.gated:
            self.shared = SwiGLU(sp, width, int(shared_hidden), dtype,
                                 names={k: n[k] for k in ("gate", "up", "down")},
                                 activation="clamped" if clamp else "silu",
                                 weight_suffix=weight_suffix, clamp=shared_clamp or clamp)
        elif shared_hidden:
            self.shared_up = Linear([sp + n["up"]], width, [int(shared_hidden)],
                                    stage="matmul_ffn_gate_up", weight_suffix=weight_suffix)
            self.shared_down = Linear([sp + n["down"]], int(shared_hidden), [width],
                                      stage="matmul_ffn_down", weight_suffix=weight_suffix)
        self.router: Optional[torch.Tensor] = None
        self.w_gate = self.w_up = self.w_down = None

    def tensor_specs(self) -> List[TensorSpec]:
        routed = self.E + self.identity
        specs = [TensorSpec(self._router, (routed, self.width), MATRIX, INIT_NORMAL)]
        if self._router_bias:
            specs.append(TensorSpec(self._router_bias, (routed,), VECTOR, INIT_SMALL))
        if self._correction:
            specs.append(TensorSpec(self._correction, (routed,), VECTOR, INIT_SMALL))
        if self._shared_gate:
            specs.append(TensorSpec(self._shared_gate, (1, self.width), MATRIX, INIT_NORMAL))
        if self.shared is not None:
            specs += self.shared.tensor_specs()
        for names in self._expert:
            if self.gated:
                specs.append(TensorSpec(names["gate"], (self.hidden, self.width), MATRIX,
                                        INIT_NORMAL))
            specs.append(TensorSpec(names["up"], (self.hidden, self.width), MATRIX, INIT_NORMAL))
            specs.append(TensorSpec(names["down"], (self.width, self.hidden), MATRIX, INIT_NORMAL))
        if self.shared_up is not None:
            specs += self.shared_up.tensor_specs() + self.shared_down.tensor_specs()
        return specs

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.router = tensors[self._router].to(torch.float32).contiguous()
        if self._shared_gate:
            self.router = torch.cat([self.router, tensors[self._shared_gate].to(torch.float32)])
        if self.shared is not None:
            self.shared.bind(tensors)

        def stacked(key):
            w = torch.stack([tensors[names[key]].to(self.dtype) for names in self._expert]
                            ).contiguous()
            # bfloat16 matrices whose shape allows it are kept in the order the matrix-core
            # kernel loads them, and only so
            if w.is_cuda and tuning.FRAGMENT_ORDER and ops.ExpertFragments.fits(w):
                return ops.ExpertFragments.of(w)
            return w
        if self._router_bias:
            self.router_bias = tensors[self._router_bias].to(torch.float32).contiguous()
        if self._correction:
            self.correction = tensors[self._correction].to(torch.float32).contiguous()
        self.w_gate = stacked("gate") if self.gated else None
        self.w_up = stacked("up")
        self.w_down = stacked("down")
        if self.shared_up is not None:
            self.shared_up.bind(tensors)
            self.shared_down.bind(tensors)

    # ``forward(..., terms=True)`` leaves the sum over the chosen experts to the caller
    # (``ops.ExpertTerms``)
    hands_on_terms = True

    def _route(self, x):
        """(experts, weights, gate of the shared expert or None)"""
        if self.scoring == "softmax":
            return *ops.moe_route(x, self.router, self.top, bias=self.router_bias), None
        out = ops.moe_route_scored(x, self.router, self.top, self.weight_scale,
                                   correction=self.correction, groups=self.groups,
                                   keep_groups=self.keep_groups, bias=self.router_bias,
                                   score="sigmoid" if self.scoring == "sigmoid" else "softmax",
                                   group_best=self.group_best, gate=bool(self._shared_gate))
        return out if self._shared_gate else (*out, None)

    def forward(self, x, batch, terms: bool = False):
        with profile.scope("router"):
            chosen, weights, gate = self._route(x)
            plan = ops.moe_plan(chosen, self.E)
        also = None
        if self.shared is not None:
            also = self.shared.forward(x, batch)
        if self.shared_up is not None:
            hidden = self.shared_up.forward(x)
            with profile.scope("ffn_act"):
                hidden = ops.activate(hidden, ops.ACT_RELU_SQUARED)
            also = self.shared_down.forward(hidden, partial_sums=True)
        with profile.scope("matmul_ffn_gate_up", 0):
            act = (ops.moe_experts_gated(x, self.w_gate, self.w_up, plan, clamp=self.clamp)
                   if self.gated else ops.moe_experts_activated(x, self.w_up, plan))
        with profile.scope("matmul_ffn_down", 0):
            y = ops.moe_experts_down(act, self.w_down, plan)
            out = ops.ExpertTerms(y, weights, plan, also=also, also_gate=gate,
                                  rows=x if self.identity else None)
            return out if terms else out.combined()

    def weight_bytes(self) -> int:
        """What a step of one row reads: the router and ``top`` experts."""
        per_expert = len(self._kinds) * self.hidden * self.width * self.w_up.element_size()
        shared = 0
        if self.shared_up is not None:
            shared = self.shared_up.weight_bytes() + self.shared_down.weight_bytes()
        elif self.shared is not None:
            shared = self.shared.weight_bytes()
        return self.router.numel() * 4 + self.top * per_expert + shared


register_part("feed_forward", "moe", MixtureOfExperts)
