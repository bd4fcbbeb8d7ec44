"""A short causal convolution over time on each channel, added to its input, in front of a mixer:
out_t = x_t + sum_j w[:, j] x_(t - taps + 1 + j), zeros before the request's start.  It reads the 32-bit
stream and writes the activation type.  A request's last ``taps - 1`` inputs are its state, kept in a
state slot in 32-bit, so that a portion cut anywhere continues where the last one ended.  Behind a norm
(``after_norm``) the convolution's input is the normed row, formed in 32-bit on the way and never stored."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..cache.plan import StateNeed
from ..kernels import ops
from .base import BranchSum, Runtime, TensorInfo
from .registry import register_part


class ShortConv:
    graph_safe = True        # one launch (two with the state's update) whose grid follows the rows alone

    def __init__(self, spec, hidden_size: int):
        self.taps = int(spec.taps)
        self.hidden = int(hidden_size)
        if self.taps < 1:
            raise ValueError(f"a convolution of {self.taps} taps")
        self.weight: Optional[torch.Tensor] = None
        self._weight_t: Optional[torch.Tensor] = None      # [taps, H]: what the kernels behind a norm read

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        return {"": TensorInfo((hidden, int(spec.taps)), "normal", "vector")}

    @staticmethod
    def state_need(spec, hidden: int) -> Optional[StateNeed]:
        return StateNeed(shape=(int(spec.taps) - 1, hidden), dtype="float32") if int(spec.taps) > 1 else None

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        self.weight = rt.place_vector(tensors[""])
        self._weight_t = self.weight.t().contiguous()

    def forward(self, x: torch.Tensor, ctx, state: Optional[torch.Tensor]) -> torch.Tensor:
        """x: the 32-bit stream [T, H]; state [slots, taps - 1, H], read and brought up to date."""
        # (a step in which every request brings one token: convolution and the state's shift in one launch)
        single = all(s.q_len == 1 for s in ctx.seqs) and len(ctx.seqs) == x.shape[0]
        return ops.short_conv(x, self.weight, state, ctx.tok_seq, ctx.rt.dtype, single_rows=single)


    def after_norm(self, norm, h: torch.Tensor, pending, ctx, state: Optional[torch.Tensor]) -> torch.Tensor:
        """The convolution of norm(h + what is pending), the sum written back to the 32-bit stream h.  ``norm``: a part
        with ``weight``, ``eps`` and ``center``."""
        if pending is None:
            pending = BranchSum(None)
        elif not isinstance(pending, BranchSum):
            pending = BranchSum(pending)
        single = all(s.q_len == 1 for s in ctx.seqs) and len(ctx.seqs) == h.shape[0]
        return ops.stream_norm(h, norm.weight, norm.eps, ctx.rt.dtype, center=norm.center, conv_w=self._weight_t, state=state,
                               tok_seq=ctx.tok_seq, single_rows=single, **pending.kernel_args())


register_part("short_conv", ShortConv)
