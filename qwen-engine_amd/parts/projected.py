"""Mixers that say which products stand before and behind them, so that mixers side by side share both.

A *projected* mixer defines
  inputs(tensors) -> ([(matrix, bias | None)], [matrix])   its projections of the mixer's input: those whose results are
                                  activations, and those whose results enter 32-bit arithmetic and stay 32-bit
  output(tensors) -> matrix [H, K]   its output projection
  output_width(spec) -> K
  mix(y, gates, ctx, binding, out, factor)   y [T, n] the first kind's results (columns of wider rows, in the activation
                                  type or float32), gates float32 [T, n'], or [S, T, n'] partial products, the second's (or
                                  None); leaves factor * the result before the output projection in out [T, K] (columns of
                                  wider rows)
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from ..kernels import ops
from .base import Runtime

# Up to this many rows the products before a mixer are one product whose results all stay 32-bit (a step of few rows is a
# chain of short kernels: one launch less counts for more than the results' bytes).
ONE_PRODUCT_MAX_ROWS = 64


class InputProducts:
    """The products before one projected mixer, or several that read the same rows."""
    holds_weights = True

    def __init__(self, sets, rt: Runtime):
        """sets: per mixer what its ``inputs`` gave."""
        self.main_cols: List[Tuple[int, int]] = []      # per mixer: its columns among the activations, among the 32-bit results
        self.gate_cols: List[Tuple[int, int]] = []
        mats, gates, biases = [], [], []
        any_bias = any(b is not None for main, _ in sets for _, b in main)
        at = 0
        for main, _ in sets:
            first = at
            for w, b in main:
                mats.append(w)
                biases.append(torch.zeros(w.shape[0]) if b is None else b.float())
                at += w.shape[0]
            self.main_cols.append((first, at))
        self.n_main = at
        at = 0
        for _, extra in sets:
            first = at
            for w in extra:
                gates.append(w)
                at += w.shape[0]
            self.gate_cols.append((first, at))
        every = mats + gates
        if len({m.dtype for m in every}) > 1:
            every = [m.float() for m in every]
        self.w = rt.place_matrix(torch.cat(every, dim=0))
        self.b = rt.place_vector(torch.cat(biases + [torch.zeros(at)])) if any_bias else None
        self._w_main, self._w_gates = self.w[:self.n_main], (self.w[self.n_main:] if at else None)
        self._b_main = self.b[:self.n_main] if any_bias else None

    def run(self, x: torch.Tensor, rt: Runtime):
        """[(y, gates or None)] per mixer."""
        if rt.dtype == torch.float32 or x.shape[0] <= ONE_PRODUCT_MAX_ROWS:
            y = ops.gemm(x, self.w, self.b, out_dtype=torch.float32)
            gates = y[:, self.n_main:]
        else:
            y = ops.gemm(x, self._w_main, self._b_main)
            gates = self._few_columns(x) if self._w_gates is not None else None
        return [(y[:, a:b], gates[..., c:d] if d > c else None) for (a, b), (c, d) in zip(self.main_cols, self.gate_cols)]


    def _few_columns(self, x: torch.Tensor) -> torch.Tensor:
        """The 32-bit results against many rows: a product of so few columns has few tiles, each a walk over all of K, so
        it is cut along K (in the order of the cuts the consumer adds the parts)."""
        tiles = -(-x.shape[0] // 64) * -(-self._w_gates.shape[0] // 128)
        splits = max(1, min(8, 256 // tiles, x.shape[1] // 256))
        K = x.shape[1]
        while splits > 1 and (splits - 1) * (-(-(-(-K // splits)) // 64) * 64) >= K:      # (every cut has some of K)
            splits -= 1
        if splits > 1 and ops.gemm_splits_supported(x, self._w_gates):
            return ops.gemm(x, self._w_gates, epilogue=ops.EPI_PARTIAL, splits=splits)
        return ops.gemm(x, self._w_gates, out_dtype=torch.float32)


class OutputProduct:
    """The product behind one projected mixer, or several whose results lie side by side in one row.  The row is filled up with
    zeros to a multiple of 32, which the kernels for few rows want."""
    holds_weights = True

    def __init__(self, mats: List[torch.Tensor], rt: Runtime):
        self.cols: List[Tuple[int, int]] = []
        at = 0
        for w in mats:
            self.cols.append((at, at + w.shape[1]))
            at += w.shape[1]
        self.n, pad = at, -at % 32
        if len({m.dtype for m in mats}) > 1:
            mats = [m.float() for m in mats]
        self.w = rt.place_matrix(torch.cat(mats + ([torch.zeros((mats[0].shape[0], pad), dtype=mats[0].dtype)] if pad else []), dim=1))

    def rows(self, T: int, rt: Runtime, device) -> torch.Tensor:
        o = torch.empty((T, self.w.shape[1]), dtype=rt.dtype, device=device)
        if self.w.shape[1] > self.n:
            o[:, self.n:].zero_()
        return o

    def run(self, o: torch.Tensor) -> torch.Tensor:
        """[T, H] in o's type, or float32 partial products [S, T, H]."""
        splits = ops.gemm_branch_splits(o, self.w)
        if splits:
            return ops.gemm(o, self.w, epilogue=ops.EPI_PARTIAL, splits=splits)
        return ops.gemm(o, self.w)


class ProjectedMixer:
    """A projected mixer on its own."""
    graph_safe = True
    products_in: Optional[InputProducts] = None
    products_out: Optional[OutputProduct] = None

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        self.load_own(tensors, rt)
        self.products_in = InputProducts([self.inputs(tensors)], rt)
        self.products_out = OutputProduct([self.output(tensors)], rt)

    def load_own(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        """The mixer's tensors beside its projections."""
        raise NotImplementedError

    def forward(self, x: torch.Tensor, ctx, binding) -> torch.Tensor:
        (y, gates), = self.products_in.run(x, ctx.rt)
        o = self.products_out.rows(x.shape[0], ctx.rt, x.device)
        self.mix(y, gates, ctx, binding, o[:, :self.products_out.n], 1.0)
        return self.products_out.run(o)
