"""A short causal convolution over the residual sum in front of a branch."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..cache.spec import StateSpec
from ..ops.profile import section
from .base import ParamSpec, Part, ResidualStream, StepContext, TensorSource
from .norm import LayerNorm


class ResidualConv(Part):
    """What a branch reads of the residual sum h: h + conv(h), conv(h)_t = sum_j w[:, j] h_(t - taps + 1 + j) per channel, zeros
    before the sequence.  All in float; the result in the activations' storage type.  A request keeps its last
    inputs in a ring of `taps` rows in its state slot (position p at row p mod taps).

    In steps of single tokens the norm behind the branch before, its addition to the sum and this convolution are one
    launch; in others a branch output that waits behind its norm is added first."""

    def __init__(self, hidden: int, taps: int, name: str = ""):
        if not 1 <= taps <= ops.RESIDUAL_CONV_MAX_TAPS:
            raise ValueError(f"a convolution of {taps} taps is not taken: 1 to {ops.RESIDUAL_CONV_MAX_TAPS}")
        self.hidden, self.taps, self.name = int(hidden), int(taps), name
        self.w: Optional[torch.Tensor] = None         # float32 [hidden, taps]

    def cache_spec(self) -> Optional[StateSpec]:
        return StateSpec((self.taps, self.hidden), torch.float32) if self.taps > 1 else None

    def param_specs(self, prefix: str) -> Dict[str, ParamSpec]:
        return {prefix + self.name: ParamSpec((self.hidden, self.taps))}

    def load(self, prefix: str, source: TensorSource) -> None:
        self.w = source.get(prefix + self.name).float().contiguous()

    def forward(self, stream: ResidualStream, ctx: StepContext, ring: Optional[torch.Tensor]) -> torch.Tensor:
        if ctx.n_entries != ctx.n_tokens or not (stream.pending_norm is None or isinstance(stream.pending_norm, LayerNorm)):
            stream.settle()
        if stream.pending is not None and stream.pending_norm is None:
            raise ValueError("a convolution over the residual sum cannot follow a block that leaves its output pending")
        T = ctx.n_tokens
        width = 2 if ctx.act_dtype == torch.bfloat16 else 4
        if ctx.n_entries != T:
            with section("input convolution", nbytes=T * self.hidden * (4 + width)):
                return ops.residual_conv(stream.h, self.w, ring, ctx, ctx.act_dtype)
        norm, delta = stream.pending_norm, stream.pending
        stream.pending = stream.pending_norm = None
        with section("norm", nbytes=T * self.hidden * (8 + 2 * width + 4 * self.taps)):
            return ops.layer_norm(stream.h, LayerNorm.foldable(delta), norm.weight if norm else None, norm.bias if norm else None,
                                  norm.eps if norm else 1.0, out_dtype=ctx.act_dtype, conv=(self.w, ring, ctx))
