"""Buckets of distances: which row of a learned table of biases a key n positions back reads.

Half of the B buckets hold one distance each; the other half grow with the distance's logarithm
up to ``far``, behind which everything is the last bucket's.  The rule's floor is decided in whole
numbers, so that a distance that lies on a bucket's edge falls on the same side everywhere.
"""
from __future__ import annotations

import math
from fractions import Fraction
from typing import List

from ..errors import ConfigError


def bucket_starts(buckets: int, far: float) -> List[int]:
    """The first distance of every bucket, in order (a bucket may be empty: two equal starts)."""
    if buckets < 2:
        raise ConfigError(f"a table of biases by distance needs at least 2 rows, got {buckets}")
    near, grown = buckets // 2, buckets - buckets // 2
    ratio = Fraction(far) / near
    if not ratio > 1:
        raise ConfigError(f"biases by distance: {buckets} buckets reach {near} positions back one "
                          f"by one, the largest distance {far} must be larger")
    starts = list(range(near))
    for k in range(grown):
        # the smallest n with (n / near)^grown >= ratio^k
        def reached(n: int) -> bool:
            return Fraction(n, near) ** grown >= ratio ** k
        n = max(near, math.floor(near * float(ratio) ** (k / grown)))
        while reached(n) and n > near:
            n -= 1
        while not reached(n):
            n += 1
        starts.append(n)
    return starts


def bucket_of_distances(buckets: int, far: float) -> List[int]:
    """Entry n: the bucket of distance n, up to the first distance of the last bucket (every
    larger distance is the last bucket's too)."""
    starts = bucket_starts(buckets, far)
    out, b = [], 0
    for n in range(starts[-1] + 1):
        while b + 1 < buckets and starts[b + 1] <= n:
            b += 1
        out.append(b)
    return out
