"""RMSNorm over the float32 residual stream.

``y = x * (1 / sqrt(mean(x^2) + eps)) * w`` with eps inside the root and the
weight multiplied last (src/ops/ops.cpp:687-698); fused with the residual sum as
the reference's ``add_rms_norm`` is (src/ops/hip/basic_kernels.hip:393-418).
With ``groups`` the vector is cut into that many equal runs of neighbouring
channels and the mean of squares is taken over each. ``unnormed`` is what stands
where an arrangement has a norm and a design has none: the sum is made and handed
on as it is, in the engine's element type.
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..ops import kernels
from .base import Norm, Runtime, TensorDecl, VECTOR
from .registry import register_part
from .spec import PartSpec


class NormedDelta:
    """A sublayer's result that is still to be RMS-normed with a weight of its own and multiplied by ``mult`` before
    it joins the residual stream: ``h += mult * values / sqrt(mean(values^2) + eps) * weight``. The norm that reads the
    stream next does both in one kernel. ``values`` is ``[tokens, hidden]`` or float32 partial sums ``[parts, tokens,
    hidden]``, which are added in order first; with ``groups`` the mean is over each run of ``hidden / groups``. ``extra``: float32 rows ``[tokens, hidden]`` that join the stream after
    it, unnormed (``with_extra``)."""

    def __init__(self, values: torch.Tensor, weight: torch.Tensor, eps: float, mult: float, extra: Optional[torch.Tensor] = None,
                 groups: int = 1):
        self.groups = int(groups)
        self.values = values
        self.weight = weight
        self.eps = float(eps)
        self.mult = float(mult)
        self.extra = extra

    def with_extra(self, rows: torch.Tensor) -> "NormedDelta":
        if self.extra is not None:
            raise ValueError("this delta already takes further rows along")
        return NormedDelta(self.values, self.weight, self.eps, self.mult, rows, self.groups)

    def resolved(self) -> torch.Tensor:
        """What joins the stream, as a float32 tensor ``[tokens, hidden]`` (for observers; a step never needs it)."""
        shape = self.values.shape[-2:]
        joined = torch.zeros(shape, dtype=torch.float32, device=self.values.device)
        kernels.rms_norm_after(joined, self.values, self.weight, self.eps, self.mult, None, 1.0, self.values.dtype, write_h=True,
                               extra=self.extra, groups=self.groups)
        return joined


class SummedDelta:
    """What several sublayers add to the residual stream at once: tensors ``[tokens, hidden]`` or partial sums ``[parts, tokens,
    hidden]``, each in a place of its own. The norm that reads the stream next adds them all in its kernel."""

    def __init__(self, sources):
        self.sources = [source if source.dtype == torch.float32 else source.to(torch.float32) for source in sources]

    def with_extra(self, rows: torch.Tensor) -> "SummedDelta":
        return SummedDelta([*self.sources, rows])

    def resolved(self) -> torch.Tensor:
        """The sum as one float32 tensor ``[tokens, hidden]`` (for observers, and for norms that take no several sources)."""
        total = torch.zeros(self.sources[0].shape[-2:], dtype=torch.float32, device=self.sources[0].device)
        for source in self.sources:
            for part in (source if source.dim() == 3 else (source,)):
                kernels.residual_add(total, part)
        return total


class RMSNorm(Norm):
    graph_safe = True
    def __init__(self, spec: PartSpec, runtime: Runtime):
        super().__init__(spec, runtime)
        self.size = int(spec.params["size"])
        self.eps = float(spec.params["eps"])
        # ``unit_offset``: the file stores the gain's distance from one; the gain ``1 + w`` is formed once, at load,
        # in float32 (the sum a float32 evaluation of ``x * (1 + w)`` forms for every element).
        self.unit_offset = bool(spec.params.get("unit_offset", False))
        self.groups = int(spec.params.get("groups", 1))
        if self.groups < 1 or self.size % self.groups != 0:
            raise ValueError("a norm in groups cuts its vector into equal parts")
        self.weight: Optional[torch.Tensor] = None

    def tensors(self) -> Dict[str, TensorDecl]:
        return {self.name("weight"): TensorDecl((self.size,), VECTOR)}

    def bind(self, tensors: Mapping[str, torch.Tensor]) -> None:
        self.weight = tensors[self.name("weight")]
        if self.unit_offset:
            self.weight = (self.weight.to(torch.float32) + 1.0).contiguous()

    def weight_then_factor(self):
        whole = self.weight is not None and self.weight.dtype == torch.float32 and self.groups == 1
        return (self.weight, self.size, self.eps) if whole else None

    def delayed(self, values: torch.Tensor, mult: float) -> NormedDelta:
        """``mult`` times this norm of ``values``, for the norm that reads the stream next to form and add."""
        if self.weight is None or self.weight.dtype != torch.float32:
            raise TypeError("the norm after a sublayer must have a float32 weight")
        return NormedDelta(values, self.weight, self.eps, mult, groups=self.groups)

    def forward(self, h, delta=None, write_h=True, rows=None):
        dtype = self.runtime.dtype
        if isinstance(delta, SummedDelta):
            if self.groups == 1 and len(delta.sources) <= kernels.DELTA_SOURCES:
                return kernels.rms_norm_sum(h, self.weight, self.eps, dtype, delta.sources, rows=rows, write_h=write_h and rows is None)
            delta = delta.resolved()
        if self.groups != (delta.groups if isinstance(delta, NormedDelta) else 1):
            # the sum's own norm has other runs than the delta's (or a plain delta joins a norm in groups): the sum first
            keeps = write_h and rows is None
            if isinstance(delta, NormedDelta):
                h = add_normed(h, delta, rows, keeps)
            elif delta is not None:
                h = h if keeps else h.clone()
                delta = delta.to(torch.float32)
                kernels.residual_add(h, delta.sum(0) if delta.dim() == 3 else delta)
            taken = rows if not isinstance(delta, NormedDelta) else None        # ``add_normed`` has taken the rows out
            return kernels.rms_norm_after(h, None, None, 0.0, 1.0, self.weight, self.eps, dtype, rows=taken, groups=self.groups)
        if isinstance(delta, NormedDelta):
            return kernels.rms_norm_after(h, delta.values, delta.weight, delta.eps, delta.mult, self.weight, self.eps,
                                          self.runtime.dtype, rows=rows, write_h=write_h and rows is None, extra=delta.extra,
                                          groups=self.groups)
        return kernels.rms_norm(h, self.weight, self.eps, dtype, delta=delta, rows=rows,
                                write_h=write_h and delta is not None and rows is None)


def add_normed(h: torch.Tensor, delta: NormedDelta, rows: Optional[torch.Tensor], write_h: bool) -> torch.Tensor:
    """The stream with ``delta`` in it, float32: ``h`` itself with ``write_h``, else new rows (those of ``rows``, if given)."""
    sums = kernels.rms_norm_after(h, delta.values, delta.weight, delta.eps, delta.mult, None, 1.0, torch.float32, rows=rows,
                                  write_h=write_h, extra=delta.extra, groups=delta.groups, raw=not write_h)
    return h if write_h else sums


class Unnormed(Norm):
    """No norm: ``h + delta`` in the engine's element type. In float32 that is the stream itself, which nothing writes
    before the product that reads it has run."""
    graph_safe = True
    weight = None

    def forward(self, h, delta=None, write_h=True, rows=None):
        dtype = self.runtime.dtype
        if isinstance(delta, SummedDelta):
            delta = delta.resolved()
        if delta is not None and not isinstance(delta, NormedDelta):
            delta = delta.to(torch.float32)
            if not write_h:
                h = h.clone()
            kernels.residual_add(h, delta.sum(0) if delta.dim() == 3 else delta)
            delta = None
        if delta is None:
            if dtype == torch.float32 and rows is None:
                return h
            return kernels.rms_norm_after(h, None, None, 0.0, 1.0, None, 1.0, dtype, rows=rows, raw=True)
        write_h = write_h and rows is None
        if dtype == torch.float32:
            return add_normed(h, delta, rows, write_h)
        return kernels.rms_norm_after(h, delta.values, delta.weight, delta.eps, delta.mult, None, 1.0, dtype, rows=rows, write_h=write_h,
                                      extra=delta.extra, groups=delta.groups, raw=True)


register_part("norm", "rms_norm", RMSNorm)
register_part("norm", "unnormed", Unnormed)
