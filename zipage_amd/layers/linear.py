"""Library matrix products whose result goes straight into a residual add."""
from __future__ import annotations

import torch
import torch.nn.functional as F


def pad_to_multiple(n: int, to: int) -> int:
    return -(-n // to) * to


def fit(t: torch.Tensor, *shape: int) -> torch.Tensor:
    """`t` in the corner of a zero tensor of `shape`."""
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(0, n) for n in t.shape)] = t
    return out


class ResidualLinear:
    """y = W x, returned as planes of partial sums (planes, N, out) that `residual_norm` adds up in
    fp32.

    A product with few rows, few outputs and a long contraction leaves most of the chip idle unless
    the contraction is split; the library does not do that by itself here (4096 x 18432 at 64 rows:
    130 us whole, 37 us in four parts).  So a long bfloat16 contraction is kept in a second layout,
    one contiguous (in / 4, out) matrix per part, and steps of up to `SPLIT_ROWS` rows run the four
    parts as one batched product.  Rounding the parts to 16 bits costs no accuracy: each is half as
    large, in the root mean square, as the whole."""

    PARTS, MIN_CONTRACTION, SPLIT_ROWS = 4, 4096, 1024

    def __init__(self, w: torch.Tensor):
        self.w = w
        out, inn = w.shape
        self.parts = None
        if w.dtype == torch.bfloat16 and inn >= self.MIN_CONTRACTION and inn % (8 * self.PARTS) == 0:
            self.parts = w.t().contiguous().view(self.PARTS, inn // self.PARTS, out)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        N = x.shape[0]
        if self.parts is None or N > self.SPLIT_ROWS:
            return F.linear(x, self.w).unsqueeze(0)
        P, k, _ = self.parts.shape
        return torch.bmm(x.view(N, P, k).transpose(0, 1), self.parts)
