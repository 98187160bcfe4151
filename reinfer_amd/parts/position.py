"""Position encodings. A mixer holds one and passes its constants to its kernel.

Rotation: pair (j, j + R/2) ("rope_neox", half split) or (2j, 2j + 1)
("rope_interleaved") is turned by the angle pos * theta^(-2j/R)
(crates/cuda/kernels/dense_kernels.cu:125-139; crates/kernels/src/refs.rs:25-37).
The reference computes theta^(-2j/R) with powf in the kernel; here the table of
R/2 inverse frequencies is made once, in double precision, and rounded to float.
The angle itself (position times frequency) and its sine and cosine are float.
With ``scaling`` (a YarnSpec) the table is fitted to longer contexts, and ``amplitude`` is the factor on sine and cosine
that goes with it (1 otherwise), for the kernels that take one.
"""
from __future__ import annotations

import math

import torch

from ..config.schema import PositionSpec, YarnSpec
from .registry import register_position


def yarn_frequencies(freq: torch.Tensor, dims: int, theta: float, y: YarnSpec) -> torch.Tensor:
    """The frequencies (float64, one a pair) of ``dims`` turned entries under ``y``."""
    def turns(t: float) -> float:                  # the entry whose pair turns t times over the original context
        return dims * math.log(y.original / (2.0 * math.pi * t)) / (2.0 * math.log(theta))
    lo = max(math.floor(turns(y.fast)), 0)
    hi = min(math.ceil(turns(y.slow)), dims - 1)
    i = torch.arange(freq.numel(), dtype=torch.float64)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return freq / y.factor * ramp + freq * (1.0 - ramp)


class _Rotary:
    style = 0
    amplitude = 1.0

    def __init__(self, spec: PositionSpec, device: torch.device):
        if spec.rotary_dim <= 0 or spec.rotary_dim % 2 != 0:
            raise ValueError(f"rotation needs an even, positive width, got {spec.rotary_dim}")
        self.rotary_dim = spec.rotary_dim
        self.theta = float(spec.theta)
        j = torch.arange(spec.rotary_dim // 2, dtype=torch.float64)
        inv = torch.pow(torch.tensor(self.theta, dtype=torch.float64), -2.0 * j / spec.rotary_dim)
        if spec.scaling is not None:
            inv = yarn_frequencies(inv, spec.rotary_dim, self.theta, spec.scaling)
            self.amplitude = 0.1 * math.log(spec.scaling.factor) + 1.0
        self.inv_freq = inv.to(torch.float32).to(device)


@register_position("rope_neox")
class RotaryHalfSplit(_Rotary):
    style = 0


@register_position("rope_interleaved")
class RotaryInterleaved(_Rotary):
    style = 1


@register_position("none")
class NoPosition:
    style = 0
    amplitude = 1.0
    rotary_dim = 0

    def __init__(self, spec: PositionSpec, device: torch.device):
        self.inv_freq = torch.zeros(1, dtype=torch.float32, device=device)
