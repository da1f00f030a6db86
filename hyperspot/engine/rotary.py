"""Rotary frequencies and pair layouts.

The kernels turn neighbouring dimensions (2i, 2i + 1).  A checkpoint whose
pairs lie half the rotated size apart is brought into that order once, when
its tensors are loaded: rows of the query and key projections alike, which
leaves every score as it is, and rows of the value projection together with
the columns of the output projection.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import List, Union

import torch


@dataclass(frozen=True)
class Yarn:
    """Pairs that turn at least `fast` times within `original` positions keep
    their frequency, those that turn at most `slow` times are slowed down by
    `factor`, with a ramp between."""

    factor: float
    original: float
    fast: float
    slow: float

    def check(self) -> None:
        if not (self.factor > 0 and self.original > 0 and self.fast > 0
                and self.slow > 0):
            raise ValueError("rotation: YaRN constants must be positive")

    def ramp(self, dims: int, base: float) -> List[float]:
        """How far every pair is on the way to the slowed frequency."""
        def pair(turns):
            return dims * math.log(self.original / (2 * math.pi * turns)) \
                / (2 * math.log(base))

        lo = max(math.floor(pair(self.fast)), 0)
        hi = min(math.ceil(pair(self.slow)), dims - 1)
        return [min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
                for i in range(dims // 2)]


# what slows a rotation down: one factor for all pairs, or YaRN
Stretch = Union[float, Yarn]


def frequencies(dims: int, base: float,
                stretch: Stretch = 1.0) -> torch.Tensor:
    """Angle per position of every pair, float64 [dims / 2]."""
    i = torch.arange(0, dims, 2, dtype=torch.float64)
    f = base ** (-i / dims) if dims else i
    if isinstance(stretch, Yarn):
        ramp = torch.tensor(stretch.ramp(dims, base) if dims else [],
                            dtype=torch.float64)
        return f / stretch.factor * ramp + f * (1.0 - ramp)
    return f / stretch


def gain(stretch: Stretch) -> float:
    """What cosine and sine are multiplied by."""
    return 0.1 * math.log(stretch.factor) + 1.0 \
        if isinstance(stretch, Yarn) else 1.0


def pair_order(size: int, dims: int, halves: bool, first: int = 0) -> list:
    """Order that brings the pairs of dimensions [first, first + dims) of
    `size` next to each other: new dimension j is the old one order[j]."""
    order = list(range(size))
    if halves:
        n = dims // 2
        order[first:first + dims] = [first + i + h * n for i in range(n)
                                     for h in (0, 1)]
    return order


def head_order(heads: int, size: int, order: list) -> torch.Tensor:
    """The same order within every one of `heads` blocks of `size`."""
    return (torch.arange(heads)[:, None] * size
            + torch.tensor(order, dtype=torch.long)).flatten()
