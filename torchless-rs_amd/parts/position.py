"""Rotary position encoding.

inv_freq[i] = 1 / theta^(i / (r/2)) for the r rotated channels of a head; pair i
is rotated by the angle pos * inv_freq[i].  The reference rotates the whole head
(r = d) in pairs (i, i + d/2) (src/kernels/mod.rs:572-608); `rotary_dim` < d
rotates the first channels only and `interleaved` pairs (2i, 2i+1) instead.
Angles, cosines and sines are float32.  The table of inverse frequencies is made
once on the host in float64 and rounded to float32.

`scaling` = {factor, original, fast, slow} stretches the rotation for contexts longer than the
`original` positions (Peng et al., YaRN: Efficient Context Window Extension of Large Language
Models): a pair that turns `fast` times or more within `original` positions keeps its frequency,
one that turns `slow` times or fewer has it divided by `factor`, and between the two (as indices
of pairs, rounded outwards) a linear ramp leads from the one to the other; cosines and sines
are multiplied by 0.1 ln(factor) + 1 (`ops.Rotation.magnitude`).

`scaling` = {factor, original, low, high} stretches by wavelength l = 2 pi / f, as Llama 3.1 does: a pair with
l > original / low has its frequency divided by `factor`, one with l < original / high keeps it, and between the two
f -> (1 - s) f / factor + s f with s = (original / l - low) / (high - low).  Cosines and sines stay as they are.
"""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch

from ..kernels import ops
from .base import Position, register_part


class Rotary(Position):
    SCALING = ("factor", "original", "fast", "slow")
    BY_WAVELENGTH = ("factor", "original", "low", "high")

    def __init__(self, head_dim: int, theta: float, rotary_dim: Optional[int] = None, interleaved: bool = False,
                 scaling: Optional[Dict[str, float]] = None):
        if scaling is not None and (set(scaling) not in (set(self.SCALING), set(self.BY_WAVELENGTH))
                                    or any(not float(v) > 0 for v in scaling.values())):
            raise ValueError(f"rotary: scaling takes the positive numbers {self.SCALING} or {self.BY_WAVELENGTH}, got {scaling}")
        self.scaling = None if scaling is None else {k: float(v) for k, v in scaling.items()}
        self.head_dim = int(head_dim)
        self.rotary_dim = self.head_dim if rotary_dim is None else int(rotary_dim)
        if self.rotary_dim % 2 or not (0 < self.rotary_dim <= self.head_dim):
            raise ValueError(f"rotary: {self.rotary_dim} rotated channels of a head of {self.head_dim} "
                             "(even, at most the head)")
        self.theta = float(theta)
        self.interleaved = bool(interleaved)
        self._rotation = {}

    def inv_freq_host(self) -> torch.Tensor:
        half = self.rotary_dim // 2
        i = torch.arange(half, dtype=torch.float64)
        f = 1.0 / torch.pow(torch.tensor(self.theta, dtype=torch.float64), i / half)
        if self.by_wavelength:
            k = self.scaling
            turns = k["original"] * f / (2.0 * math.pi)                 # original / wavelength
            s = ((turns - k["low"]) / max(k["high"] - k["low"], 1e-30)).clamp(0.0, 1.0)
            f = torch.where(turns > k["high"], f, torch.where(turns < k["low"], f / k["factor"], (1.0 - s) * f / k["factor"] + s * f))
        elif self.scaling is not None:
            lo, hi = self._pair_of(self.scaling["fast"]), self._pair_of(self.scaling["slow"])
            lo, hi = max(math.floor(lo), 0), min(math.ceil(hi), self.rotary_dim - 1)
            ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
            f = f / self.scaling["factor"] * ramp + f * (1.0 - ramp)
        return f.to(torch.float32)

    def _pair_of(self, turns: float) -> float:
        """The pair (not a whole number) that turns `turns` times within the original positions."""
        return self.rotary_dim * math.log(self.scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(self.theta))

    @property
    def by_wavelength(self) -> bool:
        return self.scaling is not None and set(self.scaling) == set(self.BY_WAVELENGTH)

    @property
    def magnitude(self) -> float:
        return 1.0 if self.scaling is None or self.by_wavelength else 0.1 * math.log(self.scaling["factor"]) + 1.0

    def rotation(self, device) -> ops.Rotation:
        key = str(device)
        if key not in self._rotation:
            self._rotation[key] = ops.Rotation(self.inv_freq_host().to(device), self.rotary_dim, self.interleaved,
                                              self.magnitude)
        return self._rotation[key]

    def inv_freq(self, device) -> torch.Tensor:
        """The frequencies alone (float32 [rotary_dim / 2] on `device`)."""
        return self.rotation(device).inv_freq


class NoPosition(Position):
    """Queries and keys are used as they are (the base class's answer)."""

    def __init__(self, head_dim: int = 0):
        self.head_dim = int(head_dim)


register_part("position", "rotary", Rotary)
register_part("position", "none", NoPosition)
