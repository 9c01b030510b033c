"""The angular steps of rotations whose frequencies are stretched, made in 64-bit when a model is loaded (the kernels
multiply the 32-bit step by the position)."""
from __future__ import annotations

import math

import torch


def banded_frequencies(rot_dims: int, base: float, scaling: dict | None) -> torch.Tensor:
    """[rot_dims / 2] float64: base^(-2 i / rot_dims), stretched by wavelength band where `scaling` is given."""
    i = torch.arange(rot_dims // 2, dtype=torch.float64)
    freq = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / rot_dims)
    if scaling and "low" not in scaling:
        freq = freq / float(scaling["factor"])            # (every wave slowed down alike)
    elif scaling:
        factor, low, high, orig = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
        wave = 2.0 * math.pi / freq
        blend = (orig / wave - low) / (high - low) if high != low else torch.zeros_like(freq)
        mixed = (1.0 - blend) * freq / factor + blend * freq
        freq = torch.where(wave < orig / high, freq, torch.where(wave > orig / low, freq / factor, mixed))
    return freq


def ramped_frequencies(dims: int, base: float, scaling: dict | None) -> tuple[torch.Tensor, float]:
    """([dims / 2] float64 angular steps, the factor on cos and sin)."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / dims)
    if not scaling:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def pair_of(turns: float) -> float:
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(pair_of(float(scaling["slow"]))), dims - 1)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp_(0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0
