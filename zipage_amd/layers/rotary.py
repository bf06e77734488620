"""Frequencies of rotary positions."""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch


@dataclass(frozen=True)
class Rotary:
    """The first `dims` dimensions turn, i with i + dims / 2.  `stretch` (factor, low, high, original): wave
    lengths beyond original / low grow by the factor, those below original / high stay, and between the two
    the frequencies are mixed linearly in original / wave length."""
    base: float
    dims: int
    stretch: tuple[float, float, float, float] | None = None

    def frequencies(self, device) -> torch.Tensor:
        """(dims / 2,) fp32, computed in double precision."""
        out = []
        for i in range(self.dims // 2):
            f = self.base ** (-2.0 * i / self.dims)
            if self.stretch is not None:
                factor, low, high, original = self.stretch
                turns = original * f / (2.0 * math.pi)           # of this pair within `original` positions
                if turns < low:
                    f /= factor
                elif turns <= high and high > low:
                    s = (turns - low) / (high - low)
                    f *= (1.0 - s) / factor + s
            out.append(f)
        return torch.tensor(out, dtype=torch.float64).to(device=device, dtype=torch.float32)
