"""Dense gated feed-forward: down(silu(gate x) * up x), with biases if the spec says so
(src/models/qwen3/model.py:232-237; silu.mul as src/layers/fused_ops/silumul.py:46-53,
with the product formed in 32-bit before the one rounding).  gate and up are one
product with the two weights stacked."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..kernels import ops
from .base import Runtime, StreamInput, TensorInfo
from .registry import register_part


class SwiGLU:
    takes_stream = True       # forward may get a StreamInput: residual sum and norm are then the gate|up product's prologue

    def __init__(self, spec, hidden_size: int):
        self.hidden = int(hidden_size)
        self.inter = int(spec.intermediate_size)
        self.names = tuple(spec.names)
        self.bias = bool(getattr(spec, "bias", False))
        self.bias_suffix = getattr(spec, "bias_suffix", ".b")
        self.w_gu = self.w_down = self.b_gu = self.b_down = None
        self.interleaved = False

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        i = spec.intermediate_size
        gate, up, down = spec.names
        t = {
            gate: TensorInfo((i, hidden)),
            up: TensorInfo((i, hidden)),
            down: TensorInfo((hidden, i)),
        }
        if getattr(spec, "bias", False):
            for name, n in ((gate, i), (up, i), (down, hidden)):
                t[name + spec.bias_suffix] = TensorInfo((n,), "zeros", "vector")
        return t

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        n_gate, n_up, n_down = self.names
        g, u = tensors[n_gate], tensors[n_up]
        if g.dtype != u.dtype:
            g, u = g.float(), u.float()
        # gate and up rows in alternating blocks of 32, so that a product's epilogue finds the gate
        # and the up of an output side by side; widths that are no multiple of 32 keep gate | up
        self.interleaved = self.inter % 32 == 0
        self.w_gu = rt.place_matrix(ops.interleave_gate_up(g, u) if self.interleaved else torch.cat([g, u], dim=0))
        self.w_down = rt.place_matrix(tensors[n_down])
        if self.bias:                # (gate's and up's in the order of their rows)
            bg, bu = (tensors[n + self.bias_suffix].float() for n in (n_gate, n_up))
            self.b_gu = rt.place_vector(ops.interleave_gate_up(bg.view(-1, 1), bu.view(-1, 1)).view(-1) if self.interleaved
                                        else torch.cat([bg, bu]))
            self.b_down = rt.place_vector(tensors[n_down + self.bias_suffix])

    def activation(self, x) -> torch.Tensor:
        """silu(gate x) * up x [T, I] in the activation type, for x [T, H] (not a StreamInput)."""
        if self.interleaved and ops.gemm_silu_supported(x, self.w_gu):
            return ops.gemm(x, self.w_gu, self.b_gu, epilogue=ops.EPI_SILU_MUL_IL)
        if not self.interleaved and ops.gemm_fused_supported(x, self.w_gu):
            return ops.gemm(x, self.w_gu, self.b_gu, epilogue=ops.EPI_SILU_MUL)
        return ops.silu_mul(ops.gemm(x, self.w_gu, self.b_gu), interleaved=self.interleaved)

    def forward(self, x, ctx) -> torch.Tensor:
        """Returns the feed-forward output [T, H], or float32 partial products [S, T, H] of it.
        x: the normed rows, or a StreamInput."""
        a = None
        if isinstance(x, StreamInput):
            if x.prefers_prologue(ops, self.w_gu):
                a = x.gemm(ops, self.w_gu, self.b_gu, epilogue=ops.EPI_SILU_MUL_IL if self.interleaved else ops.EPI_SILU_MUL)
            else:
                x = x.materialize()
        if a is None:
            a = self.activation(x)                                     # (silu.mul in the product's epilogue where it can be)
        splits = ops.gemm_branch_splits(a, self.w_down)
        if splits:   # partial products along K, added by the norm that follows
            return ops.gemm(a, self.w_down, self.b_down, epilogue=ops.EPI_PARTIAL, splits=splits)
        return ops.gemm(a, self.w_down, self.b_down)


class GeluMLP:
    """down(gelu(up x)), the exact gelu; the up product's result stays 32-bit until the activation has been applied
    (one rounding), and the output is handed on in 32-bit for the residual sum."""

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.inter = int(spec.intermediate_size)
        self.w_up = self.w_down = None

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        up, down = spec.names
        return {up: TensorInfo((spec.intermediate_size, hidden)), down: TensorInfo((hidden, spec.intermediate_size))}

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        up, down = self.spec.names
        self.w_up = rt.place_matrix(tensors[up])
        self.w_down = rt.place_matrix(tensors[down])

    def forward(self, x: torch.Tensor, ctx) -> torch.Tensor:
        z = ops.gemm(x, self.w_up, out_dtype=torch.float32)
        a = ops.unary(z, ops.UNARY_GELU, out_dtype=ctx.rt.dtype)
        return ops.gemm(a, self.w_down, out_dtype=torch.float32)


register_part("swiglu", SwiGLU)
register_part("gelu_mlp", GeluMLP)
