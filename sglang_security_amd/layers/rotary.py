"""Rotary tables: cos | sin per position, fp32, for the 'rotate half' pairing (element i with element i + dims / 2)."""
from __future__ import annotations

import math
from typing import Optional

import torch


def yarn_blend(dims: int, base: float, scaling: dict) -> torch.Tensor:
    """Per pair, how much of the stretched frequency (f / factor) replaces the plain one: 0 for pairs that turn more than
    `fast` times over the original context, 1 for pairs that turn less than `slow` times, linear between."""
    def pair_at(turns):
        return dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(pair_at(scaling["fast"])), 0)
    hi = min(math.ceil(pair_at(scaling["slow"])), dims - 1)
    i = torch.arange(dims // 2, dtype=torch.float64)
    return ((i - lo) / max(hi - lo, 0.001)).clamp(0, 1)


def rotary_table(dims: int, base: float, positions: int, device, scaling: Optional[dict] = None) -> torch.Tensor:
    """[positions, dims] = cos[dims / 2] | sin[dims / 2]; angles are formed in double precision and rounded once."""
    f = torch.tensor(float(base), dtype=torch.float64) ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)
    mag = 1.0
    if scaling:
        blend = yarn_blend(dims, base, scaling)
        f = f / scaling["factor"] * blend + f * (1 - blend)
        mag = 0.1 * math.log(scaling["factor"]) + 1.0
    a = torch.arange(positions, dtype=torch.float64)[:, None] * f[None, :]
    return (torch.cat([a.cos(), a.sin()], -1) * mag).float().to(device).contiguous()
