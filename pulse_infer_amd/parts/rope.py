"""Rotary position encoding: pairs of channels rotated by position * theta^(-2i/rotary_dim).

The reference rotates ADJACENT pairs (x[2i], x[2i+1])
(src/ops/kernels/cuda/rope_kernel.cu:100-126); ``pairing: "half"`` rotates
(x[i], x[i + rotary_dim/2]) instead.  Channels beyond ``rotary_dim`` pass unchanged.
Once per step this part makes the cos/sin tables for the step's positions (angles in
float64, tables float32); the mixer's fused kernel applies them to q and k.
``scaling_factor`` f (default 1) divides every frequency by f ("linear scaling": position p turns like p / f).
``yarn`` = {"factor", "original", "fast", "slow"} divides the slow frequencies by ``factor`` and leaves the fast ones as
they are: with t(n) = rotary_dim ln(original / (2 pi n)) / (2 ln theta), the index of the frequency that makes n turns over
``original`` positions, a ramp over i goes from 0 at max(floor(t(fast)), 0) to 1 at min(ceil(t(slow)), rotary_dim - 1),
and frequency i becomes f_i (ramp / factor + 1 - ramp); the tables are multiplied by 0.1 ln(factor) + 1.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict

import torch

from ..ops import kernels
from .base import POSITIONS, BuildContext, Part, StepContext

PAIRINGS = {"interleaved": 0, "half": 1}


@dataclass
class RotationTables:
    cos: torch.Tensor   # float32 [T, rotary_dim / 2]
    sin: torch.Tensor
    rotary_dim: int
    pairing: int


@POSITIONS.register("rope")
class RotaryEmbedding(Part):
    records_cleanly = True

    def __init__(self, params: Dict[str, Any], build: BuildContext):
        self.theta = float(params["theta"])
        self.rotary_dim = int(params["rotary_dim"])
        self.head_dim = int(params.get("head_dim", self.rotary_dim))
        pairing = params.get("pairing", "interleaved")
        if pairing not in PAIRINGS:
            raise ValueError(f"unknown rotary pairing '{pairing}', choose from {sorted(PAIRINGS)}")
        if self.rotary_dim <= 0 or self.rotary_dim % 2 or self.rotary_dim > self.head_dim:
            raise ValueError(f"rotary_dim {self.rotary_dim} must be even, positive and at most head_dim {self.head_dim}")
        if not self.theta > 0:
            raise ValueError(f"rope theta must be positive, got {self.theta}")
        self.pairing = PAIRINGS[pairing]
        half = self.rotary_dim // 2
        exponent = torch.arange(half, dtype=torch.float64) * (2.0 / self.rotary_dim)
        self.scaling_factor = float(params.get("scaling_factor", 1.0))
        if not self.scaling_factor > 0:
            raise ValueError(f"a rope scaling factor must be positive, got {self.scaling_factor}")
        freq = torch.pow(torch.tensor(self.theta, dtype=torch.float64), -exponent) / self.scaling_factor
        self.magnitude = 1.0
        if params.get("yarn") is not None:
            freq, self.magnitude = self.yarn(freq, params["yarn"])
        self.inv_freq = freq.to(build.device)
        self.name = params.get("name", "rope")

    def yarn(self, freq: torch.Tensor, params: Dict[str, Any]):
        """(frequencies, magnitude) under the ``yarn`` scaling."""
        factor, original, fast, slow = (float(params[k]) for k in ("factor", "original", "fast", "slow"))
        if min(factor, original, fast, slow) <= 0 or self.theta == 1.0:
            raise ValueError(f"yarn scaling needs positive numbers and a theta other than 1, got {params}, theta {self.theta}")
        n = self.rotary_dim
        index = lambda turns: n * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(self.theta))
        low, high = max(math.floor(index(fast)), 0), min(math.ceil(index(slow)), n - 1)
        ramp = ((torch.arange(n // 2, dtype=torch.float64) - low) / max(high - low, 0.001)).clamp(0.0, 1.0)
        return freq / factor * ramp + freq * (1.0 - ramp), 0.1 * math.log(factor) + 1.0

    def prepare(self, ctx: StepContext) -> RotationTables:
        half = self.rotary_dim // 2
        cos = ctx.workspace.buffer(f"{self.name}.cos", ctx.num_tokens, half, torch.float32)
        sin = ctx.workspace.buffer(f"{self.name}.sin", ctx.num_tokens, half, torch.float32)
        kernels.rope_table(ctx.positions, self.inv_freq, cos, sin, self.magnitude)
        return RotationTables(cos, sin, self.rotary_dim, self.pairing)


@POSITIONS.register("none")
class NoPositionEncoding(Part):
    """Attention that learns order from the causal mask alone."""

    records_cleanly = True

    def __init__(self, params: Dict[str, Any], build: BuildContext):
        pass

    def prepare(self, ctx: StepContext) -> None:
        return None
