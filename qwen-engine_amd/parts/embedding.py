"""Embeddings that are more than a row of one table."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..cache.plan import StateNeed
from ..kernels import ops
from .base import CacheBinding, Runtime, TensorInfo
from .registry import register_part


class PairEmbedding:
    """``PairEmbeddingSpec``: the scaled row of the embedding table plus a row of a second table that the token and the one
    before it choose, in one kernel.  State: a request's last token."""
    graph_safe = True

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self._pairs: Optional[torch.Tensor] = None      # (a step reads a few rows of it)

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        return {spec.name: TensorInfo((int(spec.buckets) + 1, hidden))}

    @staticmethod
    def state_need(spec, hidden: int) -> StateNeed:
        return StateNeed(shape=(1,), dtype="int32")

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        self._pairs = rt.place_matrix(tensors[self.spec.name])

    def embed(self, table: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        """The 32-bit stream [T, H] of the step's tokens."""
        if binding.state is None:
            raise RuntimeError("the embedding of pairs was given no state")
        pairs = self._pairs if self._pairs.dtype == table.dtype else self._pairs.to(table.dtype)
        return ops.embedding_pairs(ctx.token_ids, ctx.positions, ctx.tok_seq, binding.state, table, pairs, self.spec.scale,
                                   self.spec.mul_prev, self.spec.mul_cur, single_rows=ctx.single_rows)


register_part("pair_embedding", PairEmbedding)
