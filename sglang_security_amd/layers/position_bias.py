"""Positions that enter attention without a rotation: learned biases by distance and a temperature on the query."""
from __future__ import annotations

import math
from fractions import Fraction
from typing import List, Optional

import torch

LOG2E = 1 / math.log(2)


def bucket_starts(buckets: int, longest) -> List[int]:
    """The shortest distance of every bucket: one distance each for the first half of the buckets (rounded down), then
    half + floor(ln(n / half) / ln(longest / half) * (buckets - half)), at most buckets - 1.  Exact: the logarithms are
    compared as powers."""
    half = buckets // 2
    rest = buckets - half
    if half < 1 or Fraction(longest) <= half:
        raise ValueError(f"{buckets} buckets for distances up to {longest}")
    ratio = Fraction(longest) / half
    starts, n = list(range(half)), half
    for k in range(rest):
        while Fraction(n, half) ** rest < ratio ** k:
            n += 1
        starts.append(n)
    return starts


def distance_table(rel: torch.Tensor, longest, max_context: int) -> torch.Tensor:
    """rel [buckets, heads] -> fp32 [heads, distances] in the base-2 domain; the last column holds for everything
    further away."""
    starts = bucket_starts(rel.shape[0], longest)
    columns = max(1, min(starts[-1] + 1, max_context))
    bucket = torch.bucketize(torch.arange(columns), torch.tensor(starts), right=True) - 1
    return (rel.double().t()[:, bucket.to(rel.device)] * LOG2E).float().contiguous()


def temperature_table(coef: float, every, positions: int, device) -> torch.Tensor:
    """1 + coef ln(floor((p + 1) / every) + 1) per position; formed in double precision, rounded once."""
    steps = torch.tensor([(Fraction(p + 1) / Fraction(every)).__floor__() for p in range(positions)], dtype=torch.float64) \
        if not float(every).is_integer() else torch.div(torch.arange(1, positions + 1), int(every), rounding_mode="floor").double()
    return (1 + coef * torch.log(steps + 1)).float().to(device).contiguous()


def no_temperature(positions: int, device) -> torch.Tensor:
    return torch.ones(positions, dtype=torch.float32, device=device)


def temperature(c: Optional[dict], positions: int, device) -> torch.Tensor:
    return temperature_table(c["coef"], c["every"], positions, device) if c else no_temperature(positions, device)
