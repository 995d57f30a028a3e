"""Embeddings that are more than the token's row."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..cache.spec import StateSpec
from .base import INIT_NORMAL, LayerCache, ParamSpec, Part, ResidualStream, StepContext, TensorSource
from .norm import LayerNorm


class BigramEmbedding(Part):
    """table[token] * scale + pairs[(previous token * mul_prev + token * mul_cur) mod buckets], in float; a sequence's first
    token, which has none before it, takes the row behind the last bucket.  The previous token of a request's next
    one is kept in its state slot (two int32, position p at p mod 2)."""

    def __init__(self, hidden: int, buckets: int, mul_prev: int, mul_cur: int, name: str = "bigram"):
        if buckets < 1:
            raise ValueError("a table of token pairs needs at least one bucket")
        self.hidden, self.buckets, self.mul_prev, self.mul_cur, self.name = int(hidden), int(buckets), int(mul_prev), int(mul_cur), name
        self.pairs: Optional[torch.Tensor] = None

    def cache_spec(self) -> StateSpec:
        return StateSpec((2,), torch.int32)

    def param_specs(self, prefix: str = "") -> Dict[str, ParamSpec]:
        return {prefix + self.name: ParamSpec((self.buckets + 1, self.hidden), INIT_NORMAL)}

    def load(self, prefix: str, source: TensorSource) -> None:
        self.pairs = source.get(prefix + self.name)

    def forward(self, ctx: StepContext, table: torch.Tensor, scale: float, cache: LayerCache) -> torch.Tensor:
        return ops.embed_bigram(ctx, table, self.pairs, self.mul_prev, self.mul_cur, cache.states[0], scale)


class NormedEmbedding(Part):
    """A layer norm of table[token] * scale, in float, with the copy that the first branch reads (``norm``: the norm, its
    tensors under its own names).  Keeps nothing."""

    def __init__(self, norm: LayerNorm):
        self.norm = norm

    def cache_spec(self) -> None:
        return None

    def param_specs(self, prefix: str = "") -> Dict[str, ParamSpec]:
        return self.norm.param_specs(prefix)

    def load(self, prefix: str, source: TensorSource) -> None:
        self.norm.load(prefix, source)

    def forward(self, ctx: StepContext, table: torch.Tensor, scale: float, cache: LayerCache) -> ResidualStream:
        copy = ctx.act_dtype if ctx.act_dtype != torch.float32 else None
        h, act = ops.embed_norm(ctx.token_ids, table, self.norm.weight, self.norm.bias, self.norm.eps, scale, copy)
        stream = ResidualStream(h)
        stream.act = h if copy is None else act
        return stream
