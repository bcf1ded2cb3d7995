"""State-space mixer with one decay a head and token ("Mamba-2", state-space duality).

With ``inner = heads * vdim``, one product gives ``[z: inner | x: inner | B: groups * state | C:
groups * state | dt: heads]``.  x, B and C together pass a causal convolution per channel over the
last ``taps`` tokens with a bias, then SiLU.  ``dt = softplus(dt + dt_bias)`` per head, and with
the head's group's B and C (head h reads group ``h // (heads / groups)``)

    S <- exp(-exp(A_log[h]) dt) S + dt B x^T,     y = S^T C + D[h] x

from a zero state ``S`` [state, vdim].  The heads side by side are multiplied by ``silu(z)``, then
RMS-normed in ``norm_groups`` equal parts of the row with a weight [inner], then ``W_o``.

The product's and the convolution's results are stored in the compute dtype; step sizes, decays,
the state, y and the norm are float32.  The state is a slot of ``heads * vdim * state`` floats a
request; the convolution's last ``taps - 1`` inputs are state too.
"""
from __future__ import annotations

from typing import Dict, List

import torch

from ..cache.specs import CacheBundle, FixedState
from ..kernels import ops, profile, tuning
from ..weights.spec import INIT_ONES, INIT_SMALL, VECTOR, TensorSpec
from .base import Mixer, register_part
from .linear import Linear
from .mingru import ScanChunks


class StateSpaceDual(Mixer):
    def __init__(self, prefix: str, width: int, num_heads: int, vdim: int, state: int, groups: int,
                 taps: int, norm_groups: int, norm_eps: float, dtype: torch.dtype, names=None,
                 weight_suffix: str = ".weight", bias_suffix: str = ".bias"):
        n = {"in": "in", "conv": "conv", "dt_bias": "dt_bias", "A_log": "A_log", "D": "D",
             "norm": "norm", "o": "o"}
        n.update(names or {})
        if num_heads % groups:
            raise ValueError(f"{prefix}: {num_heads} heads cannot be shared out over {groups} groups")
        if norm_groups < 1 or num_heads * vdim % norm_groups:
            raise ValueError(f"{prefix}: {num_heads * vdim} values cannot be normed in {norm_groups} "
                             "equal parts")
        if not 1 <= taps <= ops.CONV_SILU_MAX_TAPS:
            raise ValueError(f"{prefix}: {taps} taps; the kernel takes 1 to "
                             f"{ops.CONV_SILU_MAX_TAPS}")
        if not 1 <= state <= ops.STATE_SPACE_MAX_STATE:
            raise ValueError(f"{prefix}: a state of {state}; the kernel takes 1 to "
                             f"{ops.STATE_SPACE_MAX_STATE}")
        self.prefix, self.width, self.dtype = prefix, width, dtype
        self.H, self.dv, self.N, self.G = num_heads, vdim, state, groups
        self.taps, self.norm_groups, self.norm_eps = int(taps), int(norm_groups), float(norm_eps)
        self.inner = num_heads * vdim
        self.channels = self.inner + 2 * groups * state        # what the convolution runs over
        self.inputs = Linear([prefix + n["in"]], width, [self.inner + self.channels + num_heads],
                             stage="matmul_in_proj", weight_suffix=weight_suffix)
        self.out = Linear([prefix + n["o"]], self.inner, [width], stage="matmul_out_proj",
                          weight_suffix=weight_suffix)
        self._conv = prefix + n["conv"] + weight_suffix
        self._conv_bias = prefix + n["conv"] + bias_suffix
        self._vectors = {k: prefix + n[k] for k in ("dt_bias", "A_log", "D")}
        self._norm = prefix + n["norm"] + weight_suffix
        self.conv_taps = self.conv_bias = self.dt_bias = self.rate = self.skip = None
        self.norm_w = None

    @property
    def step_tables(self) -> ScanChunks:
        return ScanChunks(ops.STATE_SPACE_CHUNK_ROWS)

    def cache_spec(self):
        state = FixedState((self.H, self.dv, self.N), "float32")
        if self.taps == 1:
            return state
        return CacheBundle((("state", state),
                            ("conv", FixedState((self.taps - 1, self.channels), "float32"))))

    def tensor_specs(self) -> List[TensorSpec]:
        specs = self.inputs.tensor_specs() + self.out.tensor_specs()
        specs += [TensorSpec(self._conv, (self.channels, self.taps), VECTOR, INIT_SMALL),
                  TensorSpec(self._conv_bias, (self.channels,), VECTOR, INIT_SMALL)]
        specs += [TensorSpec(name, (self.H,), VECTOR, INIT_ONES if k == "D" else INIT_SMALL)
                  for k, name in self._vectors.items()]
        specs.append(TensorSpec(self._norm, (self.inner,), VECTOR, INIT_ONES))
        return specs

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.inputs.bind(tensors)
        self.out.bind(tensors)
        self.conv_taps = tensors[self._conv].to(torch.float32).contiguous()
        self.conv_bias = tensors[self._conv_bias].to(torch.float32).contiguous()
        self.dt_bias = tensors[self._vectors["dt_bias"]].to(torch.float32).contiguous()
        self.rate = torch.exp(tensors[self._vectors["A_log"]].to(torch.float64)).to(
            torch.float32).contiguous()
        self.skip = tensors[self._vectors["D"]].to(torch.float32).contiguous()
        self.norm_w = tensors[self._norm].to(torch.float32).reshape(
            self.norm_groups, -1).contiguous()

    def forward(self, x, batch, cache, shared_cache: bool = False):
        if shared_cache:
            raise ValueError("a recurrent state cannot be read by another layer")
        inner, C = self.inner, self.channels
        proj = self.inputs.forward(x)                      # [T, z | x B C | dt]
        if self.taps > 1:
            state, conv_state = cache.part("state").state, cache.part("conv").state
        else:
            state = cache.state
            conv_state = torch.empty((state.shape[0], 0, C), dtype=torch.float32,
                                     device=state.device)
        with profile.scope("short_conv"):
            xbc = ops.conv_silu(proj[:, inner:inner + C], self.conv_taps, conv_state,
                                batch.row_pos, batch.row_seg, batch.seg_start, batch.seg_pos0,
                                batch.seg_slot, bias=self.conv_bias)
        chunked = batch.max_segment_rows > tuning.STATE_SPACE_CHUNKS_FROM_ROWS
        with profile.scope("scan"):
            y = ops.state_space(
                xbc, proj[:, inner + C:], self.H, self.G, self.N, self.dv, self.dt_bias, self.rate,
                self.skip, state, batch.seg_start, batch.seg_pos0, batch.seg_slot,
                chunks=batch.extra.get("scan_chunks") if chunked else None,
                seg_chunk0=batch.extra.get("scan_seg_chunk0") if chunked else None,
                chunk_rows=ops.STATE_SPACE_CHUNK_ROWS)
            y = ops.head_norm_gate(y, self.norm_w, self.norm_eps, proj[:, :inner], ops.GATE_SILU,
                                   self.norm_groups, inner // self.norm_groups, self.dtype,
                                   gate_first=True)
        return self.out.forward(y, partial_sums=True)

    def weight_bytes(self) -> int:
        return self.inputs.weight_bytes() + self.out.weight_bytes()


register_part("mixer", "state_space_dual", StateSpaceDual)
