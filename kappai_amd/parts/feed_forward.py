"""SwiGLU feed-forward: ``W2 (silu(W1 x) * W3 x)`` (kappai: src/recipe/builders.c:344-370,
383-386; silu at src/backend/cpu/quants.h:369-371).  W1 and W3 are stacked into one
product; in bfloat16 their rows are interleaved so that the product's epilogue applies the
gate and the [T, 2F] intermediate never reaches memory."""
from __future__ import annotations

from typing import Dict, List

import torch

from ..kernels import ops, profile
from ..weights.spec import TensorSpec
from ctypes import Structure, c_int

from .base import FeedForward, register_part
from .cdesc import LinearDesc
from .linear import Linear


class SwiGLUDesc(Structure):
    """``kappai_swiglu`` of csrc/engine_parts.h."""
    _fields_ = [("gate_up", LinearDesc), ("down", LinearDesc), ("hidden", c_int),
                ("fused", c_int)]


class SwiGLU(FeedForward):
    takes_deferred_rows = True     # its first product takes what ops.linear takes
    adds_residual = True           # its last product can add into the residual stream

    ACTIVATIONS = {"silu": ops.GLU_SILU, "gelu_tanh": ops.GLU_GELU_TANH,
                   "clamped": ops.GLU_CLAMPED}

    def __init__(self, prefix: str, width: int, hidden: int, dtype: torch.dtype, names=None,
                 activation: str = "silu", weight_suffix: str = ".weight", bias: bool = False,
                 bias_suffix: str = ".bias", clamp=None):
        """``activation``: what the gate passes through, "silu" or "gelu_tanh" (the tanh form of
        GELU): ``W_down (act(W_gate x + b_gate) * (W_up x + b_up)) + b_down``; or "clamped", the
        clamped gate with the constants ``clamp`` (``ops.ClampedGate``).  ``bias``: whether the three
        maps have biases (the gate then runs as a kernel of its own behind the first product, which
        adds the biases)."""
        n = {"gate": "w1", "up": "w3", "down": "w2"}
        n.update(names or {})
        if activation not in self.ACTIVATIONS:
            raise ValueError(f"unknown gate activation {activation!r}; known: "
                             f"{', '.join(self.ACTIVATIONS)}")
        if (activation == "clamped") != (clamp is not None):
            raise ValueError(f"{prefix}: the clamped gate comes with its constants")
        self.width, self.hidden, self.dtype = width, hidden, dtype
        self.activation, self.clamp = activation, clamp
        self.fused = False
        self.has_bias = bool(bias)
        self.gate_up = Linear([prefix + n["gate"], prefix + n["up"]], width, [hidden, hidden],
                              stage="matmul_ffn_gate_up", weight_suffix=weight_suffix, bias=bias,
                              bias_suffix=bias_suffix)
        self.down = Linear([prefix + n["down"]], hidden, [width], stage="matmul_ffn_down",
                           weight_suffix=weight_suffix, bias=bias, bias_suffix=bias_suffix)

    def tensor_specs(self) -> List[TensorSpec]:
        return self.gate_up.tensor_specs() + self.down.tensor_specs()

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        def interleaved(w):
            # the fused product wants gate and up rows in turns of 16
            self.fused = (w.dtype == torch.bfloat16 and self.hidden % ops.SWIGLU_GROUP == 0
                          and self.width % 8 == 0 and not self.has_bias)
            return ops.interleave_gate_up(w[:self.hidden], w[self.hidden:]) if self.fused else None

        self.gate_up.bind(tensors, arrange=interleaved)
        if self.clamp is not None and self.gate_up.weight.device.type == "cuda":
            self.clamp.on(self.gate_up.weight.device)      # (before any step is captured)
        self.down.bind(tensors)

    def forward(self, x, batch, into=None):
        if self.fused and x.dtype == torch.bfloat16:
            with profile.scope("matmul_ffn_gate_up", self.gate_up.weight_bytes()):
                act = ops.linear_swiglu(x, self.gate_up.weight, out_fragment=True,
                                        activation=self.ACTIVATIONS[self.activation],
                                        clamp=self.clamp)
            return self.down.forward(act, partial_sums=True, add_into=into)
        gate_up = self.gate_up.forward(x)
        with profile.scope("ffn_act"):
            act = (ops.swiglu(gate_up) if self.activation == "silu"
                   else ops.glu(gate_up, self.ACTIVATIONS[self.activation], self.clamp))
        return self.down.forward(act, partial_sums=not self.has_bias, add_into=into)

    def c_part(self, plan, view=None, shared_cache: bool = False):
        """The runner "feed_forward.swiglu" (csrc/engine_parts.hip) makes the same choices as
        ``forward``."""
        if self.activation != "silu" or self.has_bias:
            return None            # the runner on the C side knows the SiLU gate without biases only
        first = plan.linear(self.gate_up)
        desc = SwiGLUDesc(first, plan.linear(self.down), self.hidden, 1 if self.fused else 0)
        return plan.part("feed_forward.swiglu", desc, takes_deferred_rows=True,
                         adds_residual=True, first=first)

    def weight_bytes(self) -> int:
        return self.gate_up.weight_bytes() + self.down.weight_bytes()


register_part("feed_forward", "swiglu", SwiGLU)
