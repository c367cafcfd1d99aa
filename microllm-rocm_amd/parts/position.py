"""Rotary position encoding in the split-half layout, and in the layout of neighbours.

For pair ``i`` of a head: ``theta = p * base^(-2i/d)``;
``x'[i] = x[i] cos - x[i+d/2] sin``; ``x'[i+d/2] = x[i] sin + x[i+d/2] cos``
(src/ops/ops.cpp:863-878). The part owns the table of inverse frequencies, held
in float64 so that the angle of any position is exact before cos and sin are
rounded to float32. cos and sin of a step's positions are computed once and
shared by the layers whose encoding has the same parameters; the attention
mixer's fused kernels apply the rotation. With ``scaling_factor`` every rate is
divided by that number (positions stretched linearly). With ``scaling_bands``
(``factor``, ``low``, ``high``, ``original``) only slow rates are divided by the
factor (``stretched_by_bands``). With ``scaling_ramp`` (``factor``, ``original``,
``fast``, ``slow``, ``magnitude_slope``) slow pairs' rates are divided by the
factor along a ramp over the pairs (``stretched_by_ramp``), and what is turned is
multiplied by ``magnitude_slope * ln(factor) + 1``: the table's cos and sin are.

``rope_neighbours`` pairs channel ``2i`` with ``2i + 1`` instead. Moving channel
``2i`` to ``i`` and ``2i + 1`` to ``i + d/2`` makes it the split-half rule, and a
dot product of two vectors does not change when both are reordered alike: a
mixer whose turned queries and keys only ever meet in their dot product reorders
the rows of the weights that produce them once, at load (``split_half_order``),
and runs the split-half kernels.
"""
from __future__ import annotations

import math

import torch

from ..ops import kernels
from .base import PositionEncoding, Runtime
from .registry import register_part
from .spec import PartSpec


def stretched_by_bands(rates: torch.Tensor, factor: float, low: float, high: float, original: float) -> torch.Tensor:
    """Rates (angle a position, float64) stretched by how often they turn over ``original`` positions, ``n = original *
    rate / (2 pi)``: below ``low`` turns a rate is divided by ``factor``, above ``high`` it stays, between the two the
    stretched and the plain rate are blended, linearly in ``n``."""
    turns = original * rates / (2.0 * math.pi)
    blend = ((turns - low) / (high - low)).clamp(0.0, 1.0) if high > low else (turns > high).to(rates.dtype)
    mixed = (1.0 - blend) * rates / factor + blend * rates
    return torch.where(turns < low, rates / factor, torch.where(turns > high, rates, mixed))


def stretched_by_ramp(rates: torch.Tensor, base: float, factor: float, original: float, fast: float, slow: float) -> torch.Tensor:
    """Rates ``base^(-2i/n)`` (float64, ``n / 2`` of them) of which those of pairs that turn ``slow`` times or less over
    ``original`` positions are divided by ``factor``, those of pairs that turn ``fast`` times or more stay, and between the
    two the stretched and the plain rate are blended, linearly in the pair's number ``i``. A pair that turns ``t`` times has
    the number ``n ln(original / (2 pi t)) / (2 ln base)``; the ramp's ends are rounded outwards to whole numbers and kept
    within ``0 .. n - 1``."""
    n = 2 * rates.shape[0]

    def pair_that_turns(times: float) -> float:
        return n * math.log(original / (2.0 * math.pi * times)) / (2.0 * math.log(base))

    low = max(math.floor(pair_that_turns(fast)), 0)
    high = min(math.ceil(pair_that_turns(slow)), n - 1)
    ramp = ((torch.arange(n // 2, dtype=rates.dtype) - low) / max(high - low, 0.001)).clamp(0.0, 1.0)
    return rates / factor * ramp + rates * (1.0 - ramp)


class RopeSplitHalf(PositionEncoding):
    graph_safe = True
    fused_split_half = True

    def __init__(self, spec: PartSpec, runtime: Runtime):
        super().__init__(spec, runtime)
        self.theta = float(spec.params["theta"])
        self.head_dim = int(spec.params["head_dim"])
        self.rotary_dim = int(spec.params.get("rotary_dim", self.head_dim))
        if self.rotary_dim % 2 != 0 or not 0 < self.rotary_dim <= self.head_dim:
            raise ValueError("rotary_dim must be even and at most head_dim")
        self.scaling_factor = float(spec.params.get("scaling_factor") or 1.0)
        if self.scaling_factor <= 0.0:
            raise ValueError("scaling_factor must be positive")
        exponents = torch.arange(0, self.rotary_dim, 2, dtype=torch.float64) / self.rotary_dim
        rates = (self.theta ** -exponents) / self.scaling_factor
        bands = spec.params.get("scaling_bands")
        self.scaling_bands = tuple(float(bands[key]) for key in ("factor", "low", "high", "original")) if bands is not None else None
        if self.scaling_bands is not None:
            rates = stretched_by_bands(rates, *self.scaling_bands)
        ramp = spec.params.get("scaling_ramp")
        self.scaling_ramp = tuple(float(ramp[key]) for key in ("factor", "original", "fast", "slow")) if ramp is not None else None
        self.magnitude = 1.0        # of what is turned
        if self.scaling_ramp is not None:
            rates = stretched_by_ramp(rates, self.theta, *self.scaling_ramp)
            self.magnitude = float(ramp.get("magnitude_slope", 0.0)) * math.log(self.scaling_ramp[0]) + 1.0
        self.inv_freq = rates.to(runtime.device)

    def table(self, ctx) -> torch.Tensor:
        """``[tokens, rotary_dim / 2, 2]`` float32: cos and sin for the step's tokens."""
        key = ("rope_split_half", self.theta, self.rotary_dim, self.scaling_factor, self.scaling_bands, self.scaling_ramp, self.magnitude)
        if key not in ctx.memo:
            ctx.memo[key] = kernels.rope_table(ctx.positions, self.inv_freq, self.magnitude)
        return ctx.memo[key]


class RopeNeighbours(RopeSplitHalf):
    """Channel ``2i`` turns with channel ``2i + 1`` by ``p * base^(-2i/d)``. The mixer brings the turned channels into
    ``split_half_order`` at load; from there on this is the split-half encoding with the same rates."""

    def split_half_order(self) -> torch.Tensor:
        """``order[new] = old``: the even channels of the turned part first, then the odd ones."""
        return torch.cat([torch.arange(0, self.rotary_dim, 2), torch.arange(1, self.rotary_dim, 2)])


register_part("position", "rope_split_half", RopeSplitHalf)
register_part("position", "rope_neighbours", RopeNeighbours)
