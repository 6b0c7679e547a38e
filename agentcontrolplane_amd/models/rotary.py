"""Rotation tables: frequencies base^(-2i/dims), plain or slowed for long contexts."""
from __future__ import annotations

import math
from typing import Tuple

import torch

from ..engine.config import RotaryScaling, WavelengthScaling, YarnScaling


def frequencies(base: float, dims: int, scaling: RotaryScaling = None) -> Tuple[torch.Tensor, float]:
    """[dims / 2] angles per position (double) and the factor on cos and sin."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = base ** (-2.0 * i / dims)
    if scaling is None:
        return f, 1.0
    s = scaling
    if isinstance(s, WavelengthScaling):
        wavelength = 2 * math.pi / f
        blend = ((s.original / wavelength - s.low) / (s.high - s.low)).clamp(0.0, 1.0)
        return (1 - blend) * f / s.factor + blend * f, 1.0
    if isinstance(s, YarnScaling):
        def dim_of(turns: float) -> float:
            return dims * math.log(s.original / (2 * math.pi * turns)) / (2 * math.log(base))

        lo = max(math.floor(dim_of(s.fast)), 0)
        hi = min(math.ceil(dim_of(s.slow)), dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        return f / s.factor * ramp + f * (1 - ramp), 0.1 * math.log(s.factor) + 1.0
    raise TypeError(f"unknown rotary scaling {scaling!r}")


def rotation_table(positions: int, base: float, dims: int, scaling: RotaryScaling,
                   device) -> torch.Tensor:
    """[2, positions, dims / 2] fp32 cos and sin, angles in double."""
    f, mult = frequencies(base, dims, scaling)
    angles = torch.outer(torch.arange(positions, dtype=torch.float64, device=device), f.to(device))
    return (mult * torch.stack([angles.cos(), angles.sin()])).float()
