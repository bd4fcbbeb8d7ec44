"""Half-split rotary position encoding.  The table is built as the reference builds
it (src/models/qwen3/model.py:75-86): 32-bit inverse frequencies 1 / theta^(2i/D),
32-bit outer product with the positions, then cos and sin, row = [cos | sin]."""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch

from .base import Runtime, TensorInfo
from .registry import register_part


class RotaryHalf:
    fused = True   # the q/k kernel applies it from table()

    def __init__(self, spec, hidden_size: int = 0):
        self.theta = float(spec.theta)
        self.rotary_dim = int(spec.rotary_dim)
        self.max_positions = int(spec.max_positions)
        if self.rotary_dim % 2:
            raise ValueError(f"rotary_dim {self.rotary_dim} is odd")
        self._table: Optional[torch.Tensor] = None

    @staticmethod
    def expected_tensors(spec, hidden_size: int) -> Dict[str, TensorInfo]:
        return {}

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        d = self.rotary_dim
        inv_freq = 1.0 / (self.theta ** (torch.arange(0, d, 2, dtype=torch.float32) / d))
        t = torch.arange(self.max_positions, dtype=torch.float32)
        freqs = torch.outer(t, inv_freq)
        self._table = torch.cat([torch.cos(freqs), torch.sin(freqs)], dim=-1).contiguous().to(rt.device)

    def table(self) -> torch.Tensor:
        return self._table


class RotaryPairs:
    """Rotation of neighbouring pairs (2i, 2i + 1) by position * theta^(-2i / rotary_dim).  The kernels
    that rotate form the angle, its sine and cosine in 32-bit from ``inv_freq()`` and multiply the latter two by
    ``gain``; the frequencies are computed in 64-bit, scaled as the spec says (``banded_frequencies``,
    ``yarn_frequencies``), and rounded once."""
    neighbours = True

    def __init__(self, spec, hidden_size: int = 0):
        self.theta = float(spec.theta)
        self.rotary_dim = int(spec.rotary_dim)
        if self.rotary_dim % 2:
            raise ValueError(f"rotary_dim {self.rotary_dim} is odd")
        self.band_scaling = getattr(spec, "band_scaling", None)
        self.yarn = getattr(spec, "yarn", None)
        if self.band_scaling is not None and self.yarn is not None:
            raise ValueError("frequencies scaled by bands and by YaRN at once")
        self.gain = 1.0 if self.yarn is None else 0.1 * math.log(float(self.yarn[0])) + 1.0
        self._inv_freq: Optional[torch.Tensor] = None

    @staticmethod
    def expected_tensors(spec, hidden_size: int) -> Dict[str, TensorInfo]:
        return {}

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        d = self.rotary_dim
        i = torch.arange(0, d, 2, dtype=torch.float64)
        f = torch.pow(torch.tensor(self.theta, dtype=torch.float64), -i / d)
        if self.band_scaling is not None:
            f = banded_frequencies(f, *(float(v) for v in self.band_scaling))
        if self.yarn is not None:
            f = yarn_frequencies(f, self.theta, d, *(float(v) for v in self.yarn))
        self._inv_freq = f.to(torch.float32).to(rt.device)

    def inv_freq(self) -> torch.Tensor:
        return self._inv_freq


def banded_frequencies(f: torch.Tensor, factor: float, low: float, high: float, original: float) -> torch.Tensor:
    """Frequencies f (64-bit) for longer contexts: with r = original / wavelength, f where r > high, f / factor where
    r < low, and between the two (1 - s) f / factor + s f with s = (r - low) / (high - low)."""
    turns = original * f / (2.0 * math.pi)
    if high > low:
        s = ((turns - low) / (high - low)).clamp(0.0, 1.0)
    else:                                     # (no band between: either side of the one edge)
        s = (turns > high).to(f.dtype)
    return (1.0 - s) * f / factor + s * f


def yarn_frequencies(f: torch.Tensor, theta: float, dims: int, factor: float, original: float, fast: float,
                     slow: float) -> torch.Tensor:
    """Frequencies f (64-bit, f[i] = theta^(-2 i / dims)) blended with f / factor along a ramp over i, between the
    index that turns ``fast`` times in ``original`` positions (rounded down) and the one that turns ``slow`` times
    (rounded up)."""
    def index(turns: float) -> float:
        return dims * math.log(original / (turns * 2.0 * math.pi)) / (2.0 * math.log(theta))
    low, high = max(math.floor(index(fast)), 0), min(math.ceil(index(slow)), dims - 1)
    i = torch.arange(f.shape[0], dtype=torch.float64)
    ramp = ((i - low) / max(high - low, 0.001)).clamp(0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp)


class RotaryHalfAngles:
    """Half-split rotation of a head's first ``rotary_dim`` numbers (number i pairs with i + rotary_dim / 2) by
    position * theta^(-2i / rotary_dim).  The kernels that rotate form the angle, its sine and cosine in 32-bit from
    ``inv_freq()``; the frequencies are computed in 64-bit, divided by the spec's scaling factor, scaled by bands of
    wavelengths if the spec asks for it (``banded_frequencies``), and rounded once.
    No table: no limit of positions."""
    neighbours = False
    gain = 1.0

    def __init__(self, spec, hidden_size: int = 0):
        self.theta = float(spec.theta)
        self.rotary_dim = int(spec.rotary_dim)
        if self.rotary_dim % 2 or self.rotary_dim <= 0:
            raise ValueError(f"rotary_dim {self.rotary_dim} is odd or not positive")
        self.scaling_factor = float(getattr(spec, "scaling_factor", 1.0))
        if not self.scaling_factor > 0:
            raise ValueError(f"a scaling factor of {self.scaling_factor}")
        self.band_scaling = getattr(spec, "band_scaling", None)
        self._inv_freq: Optional[torch.Tensor] = None

    @staticmethod
    def expected_tensors(spec, hidden_size: int) -> Dict[str, TensorInfo]:
        return {}

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        d = self.rotary_dim
        i = torch.arange(0, d, 2, dtype=torch.float64)
        f = torch.pow(torch.tensor(self.theta, dtype=torch.float64), -i / d) / self.scaling_factor
        if self.band_scaling is not None:
            f = banded_frequencies(f, *(float(v) for v in self.band_scaling))
        self._inv_freq = f.to(torch.float32).to(rt.device)

    def inv_freq(self) -> torch.Tensor:
        return self._inv_freq


register_part("rope_half", RotaryHalf)
register_part("rope_half_angles", RotaryHalfAngles)
register_part("rope_pairs", RotaryPairs)
