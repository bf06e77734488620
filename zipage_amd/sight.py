"""What a token of an attention layer sees of its sequence: an int is a window of that many tokens, the
own one included; a Chunk is the token's own block of positions; None is everything before it."""
from __future__ import annotations

from dataclasses import dataclass


# how far back a token looks that sees everything, for rules that take a number of tokens
EVERYTHING = 1 << 40


@dataclass(frozen=True)
class Chunk:
    """Blocks of `size` positions, counted from position 0 of the sequence."""
    size: int


def first_seen(position: int, sight) -> int:
    """The first position that the token at `position` sees."""
    if sight is None:
        return 0
    if isinstance(sight, Chunk):
        return position // sight.size * sight.size
    return max(0, position - sight + 1)
