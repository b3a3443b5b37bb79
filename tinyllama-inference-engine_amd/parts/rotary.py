"""Rotary positions, half-split pairing: the pair (i, i + d/2) of every head is turned by
angle = float(position) * theta^(-2i/d) (src/operators.cpp:58-73 of the reference).  The
frequencies are made once, in float32 as the reference forms them (`std::pow` on floats,
:63-64); the angle, sine and cosine are float32 in the kernel."""
from __future__ import annotations

import math

import torch

from ..config.spec import PartSpec
from ..errors import invalid_config
from ..registry import register
from .base import PositionEncoding


@register("position_encoding", "rotary")
class Rotary(PositionEncoding):
    """spec: head_dim, theta, optionally rot_dim (default head_dim: the whole head turns), linear_factor (every
    frequency is divided by it: positions counted in steps of 1 / factor; default 1) and wavelength_scaling, a mapping
    with factor, low, high and original: a frequency f of wavelength l = 2 pi / f stays where l < original / high, becomes
    f / factor where l > original / low, and between the two (1 - s) f / factor + s f, s = (original / l - low) / (high - low)."""
    graph_safe = True

    def __init__(self, spec: PartSpec, dtype, device):
        super().__init__(spec, dtype, device)
        self.head_dim = int(spec["head_dim"])
        self.rot_dim = int(spec.get("rot_dim", self.head_dim))
        self.theta = float(spec["theta"])
        if self.rot_dim % 2 != 0 or not 0 < self.rot_dim <= self.head_dim:
            raise invalid_config(f"rotary: rot_dim {self.rot_dim} must be even and at most head_dim {self.head_dim}")
        if not self.theta > 0:
            raise invalid_config("rotary: theta must be positive")
        self.linear_factor = float(spec.get("linear_factor", 1.0))
        if not self.linear_factor > 0:
            raise invalid_config("rotary: linear_factor must be positive")
        index = torch.arange(self.rot_dim // 2, dtype=torch.float32)
        exponent = (-2.0 * index) / float(self.rot_dim)
        inv_freq = torch.pow(torch.tensor(self.theta, dtype=torch.float32), exponent)
        if self.linear_factor != 1.0:
            # formed in double and rounded once, so that the division costs the table no second rounding
            inv_freq = (torch.pow(torch.tensor(self.theta, dtype=torch.float64), exponent.double()) / self.linear_factor).float()
        scaling = spec.get("wavelength_scaling")
        if scaling is not None:
            inv_freq = self._scaled(torch.pow(torch.tensor(self.theta, dtype=torch.float64), -2.0 * index.double() / float(self.rot_dim))
                                    / self.linear_factor, scaling).float()
        self.inv_freq = inv_freq.to(device)

    @staticmethod
    def _scaled(freq: torch.Tensor, scaling) -> torch.Tensor:
        """In double, so that the table is rounded once."""
        factor, low, high, original = (float(scaling[key]) for key in ("factor", "low", "high", "original"))
        if not (factor > 0.0 and 0.0 < low < high and original > 0.0):
            raise invalid_config("rotary: a scaling by wavelengths needs positive numbers with low below high")
        turns = original * freq / (2.0 * math.pi)                     # original / wavelength
        share = (turns - low) / (high - low)
        between = (1.0 - share) * freq / factor + share * freq
        return torch.where(turns > high, freq, torch.where(turns < low, freq / factor, between))

    def rotary_table(self):
        return self.inv_freq, self.rot_dim


@register("position_encoding", "none")
class NoPositions(PositionEncoding):
    """No position encoding in the mixer (keys are cached as projected)."""
    graph_safe = True
