"""Embeddings that read more than the token itself."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..cache.spec import StateSpec
from .base import INIT_NORMAL, LayerCache, ParamSpec, Part, StepContext, TensorSource


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
