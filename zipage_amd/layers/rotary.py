"""Frequencies of rotary positions."""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch


@dataclass(frozen=True)
class Rotary:
    """The first `dims` dimensions turn, i with i + dims / 2, or 2 i with 2 i + 1 if `interleaved`.  `stretch` (factor, low, high, original): wave
    lengths beyond original / low grow by the factor, those below original / high stay, and between the two
    the frequencies are mixed linearly in original / wave length."""
    base: float
    dims: int
    stretch: tuple[float, float, float, float] | None = None
    interleaved: bool = False

    def order(self, dim: int) -> list[int]:
        """The dimensions of a head of `dim` so that i and i + dims / 2 are a pair, which is how the kernels turn
        them: rows of weights are put into this order at load."""
        if not self.interleaved:
            return list(range(dim))
        return [*range(0, self.dims, 2), *range(1, self.dims, 2), *range(self.dims, dim)]

    def adjacent_order(self, dim: int) -> list[int]:
        """The same so that pairs are neighbours, which is how the kernels turn values (dims = dim)."""
        if self.interleaved:
            return list(range(dim))
        return [i + j * (dim // 2) for i in range(dim // 2) for j in (0, 1)]

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
