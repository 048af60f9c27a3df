"""Rotary frequency tables: computed in float64, rounded to fp32 once."""

from __future__ import annotations

import math
from typing import Optional

import torch

from llmq_amd.engine.model_specs import RotaryScaling, YarnScaling


def _plain(base: float, dims: int) -> torch.Tensor:
    i = torch.arange(dims // 2, dtype=torch.float64)
    return torch.pow(torch.tensor(base, dtype=torch.float64), -2.0 * i / dims)


def rotary_inv_freq(base: float, dims: int) -> torch.Tensor:
    """fp32 table base^(-2i/dims), i < dims/2, rounded once from float64."""
    return _plain(base, dims).to(torch.float32)


def scaled_inv_freq(base: float, dims: int, scaling: Optional[RotaryScaling]) -> torch.Tensor:
    """fp32 rotary table base^(-2i/dims) with the wavelength-dependent
    slowdown applied in float64 and rounded once."""
    if scaling is None:
        return rotary_inv_freq(base, dims)
    f = _plain(base, dims)
    wave = 2.0 * math.pi / f
    blend = (scaling.original / wave - scaling.low) / (scaling.high - scaling.low) \
        if scaling.high != scaling.low else torch.zeros_like(f)
    mid = (1.0 - blend) * f / scaling.factor + blend * f
    out = torch.where(wave < scaling.original / scaling.high, f,
                      torch.where(wave > scaling.original / scaling.low, f / scaling.factor, mid))
    return out.to(torch.float32)


def yarn_inv_freq(base: float, dims: int, scaling: Optional[YarnScaling]) -> torch.Tensor:
    """fp32 rotary table base^(-2i/dims) blended towards its factor-th part by
    a linear ramp over the pair index: the ramp's ends are the (floored /
    ceiled) indices of the pairs that turn `fast` and `slow` times within the
    original context."""
    if scaling is None:
        return rotary_inv_freq(base, dims)

    def index(turns: float) -> float:
        return dims * math.log(scaling.original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index(scaling.fast)), 0)
    hi = min(math.ceil(index(scaling.slow)), dims - 1)
    i = torch.arange(dims // 2, dtype=torch.float64)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp_(0.0, 1.0)
    f = _plain(base, dims)
    return (f / scaling.factor * ramp + f * (1.0 - ramp)).to(torch.float32)
