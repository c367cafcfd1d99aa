"""How a layer's parts are arranged around the residual stream.

``pre_norm`` is the reference's block: ``h' = h + Mixer(Norm1(h))``,
``h'' = h' + FFN(Norm2(h'))`` (src/model/model.cpp:851-860). The residual stream
``h`` is float32 and every sum into it is a float32 sum; the sum is fused with
the norm that follows it, so a block hands its last delta on instead of adding
it (the decode path of the reference does the same, src/model/model.cpp:867).
Where a step has few rows, the part before a norm and the part after it can
take the norm between them: the first adds its result to the stream in its last
product's epilogue and multiplies by the norm's weight, the second multiplies
its first product's rows by the norm's factors (``linear.UnscaledRows``).
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from .base import Part, Runtime, TensorDecl
from .linear import Residual, UnscaledRows
from .norm import NormedDelta, SummedDelta
from .registry import build_part, register_part
from .spec import LayerSpec


class Block:
    """One layer built from a ``LayerSpec``. ``forward`` returns the delta still to be added to ``h``."""
    ffn_has_norm = True     # the feed-forward stands behind a norm of its own

    def __init__(self, spec: LayerSpec, runtime: Runtime):
        self.spec = spec
        self.mixer_norm = build_part("norm", spec.mixer_norm, runtime)
        self.mixer = build_part("mixer", spec.mixer, runtime)
        if self.ffn_has_norm and (spec.ffn is None) != (spec.ffn_norm is None):
            raise ValueError("a layer has a feed-forward and its norm, or neither")
        if not self.ffn_has_norm and spec.ffn_norm is not None:
            raise ValueError("in this arrangement the feed-forward has no norm of its own")
        self.ffn_norm = build_part("norm", spec.ffn_norm, runtime) if spec.ffn_norm is not None else None
        self.ffn = build_part("ffn", spec.ffn, runtime) if spec.ffn is not None else None
        self.extra: Dict[str, Part] = {name: build_part(category, part_spec, runtime)
                                       for name, (category, part_spec) in spec.extra.items()}

    def parts(self):
        """Every part of the layer (the cache manager asks ``mixer`` alone for a cache)."""
        own = (self.mixer_norm, self.mixer, self.ffn_norm, self.ffn)
        return tuple(part for part in own if part is not None) + tuple(self.extra.values())

    def tensors(self) -> Dict[str, TensorDecl]:
        decls: Dict[str, TensorDecl] = {}
        for part in self.parts():
            decls.update(part.tensors())
        return decls

    def bind(self, tensors: Mapping[str, torch.Tensor]) -> None:
        for part in self.parts():
            part.bind(tensors)

    def forward(self, h: torch.Tensor, pending, ctx, cache, next_block: Optional["Block"] = None):
        """``pending`` is the delta the block before left to be added, or that block's ``UnscaledRows``: then the
        sum and this block's first norm are done. ``next_block`` is the block that runs after this one."""
        raise NotImplementedError

    def first_norm_after(self, producer, rows: int, h: torch.Tensor) -> Optional[Residual]:
        """What ``producer`` needs to add its delta to ``h`` itself and begin this block's first norm, if the norm,
        the producer and this block's mixer can all do their part for this many rows; else None."""
        return residual_for(producer, self.mixer_norm, self.mixer, rows, h)


def residual_for(producer, norm, consumer, rows: int, h: torch.Tensor) -> Optional[Residual]:
    if not getattr(producer, "fuses_residual", False) or not consumer.takes_unscaled(rows):
        return None
    pieces = norm.weight_then_factor()
    if pieces is None:
        return None
    weight, width, eps = pieces
    return Residual(h, weight, width, eps)


class PreNormBlock(Block):
    def forward(self, h, pending, ctx, cache, next_block=None):
        rows = h.shape[0]
        x = pending if isinstance(pending, UnscaledRows) else self.mixer_norm.forward(h, delta=pending, write_h=True)
        if self.ffn is None:        # no feed-forward: the mixer's delta goes to whatever norm comes next
            residual = next_block.first_norm_after(self.mixer, rows, h) if next_block is not None else None
            return self.mixer.forward(x, ctx, cache, residual=residual) if residual is not None else self.mixer.forward(x, ctx, cache)
        residual = residual_for(self.mixer, self.ffn_norm, self.ffn, rows, h)
        mixed = self.mixer.forward(x, ctx, cache, residual=residual) if residual is not None else self.mixer.forward(x, ctx, cache)
        x = mixed if isinstance(mixed, UnscaledRows) else self.ffn_norm.forward(h, delta=mixed, write_h=True)
        residual = next_block.first_norm_after(self.ffn, rows, h) if next_block is not None else None
        return self.ffn.forward(x, ctx, residual=residual) if residual is not None else self.ffn.forward(x, ctx)


class SandwichNormBlock(Block):
    """A norm before and a norm after each sublayer, and a factor on what joins the stream:
    ``h' = h + m * NormA(Mixer(Norm1(h)))``, ``h'' = h' + m * NormB(FFN(Norm2(h')))``. The norms after are RMS norms
    named ``mixer_after`` and ``ffn_after`` in ``LayerSpec.extra``; ``m`` is ``LayerSpec.params["residual_mult"]``
    (1 if absent). A design without norms before its sublayers names ``unnormed`` there. With ``side`` in
    ``LayerSpec.extra`` (and ``side_norm`` before it, ``side_after`` after it) one more sublayer of that kind follows, which
    needs the step's token ids beside the stream. A sublayer's result is handed on as a ``NormedDelta``: the norm that reads the stream next norms
    and adds it in the same kernel, so no product adds into the stream itself here."""

    def __init__(self, spec: LayerSpec, runtime: Runtime):
        super().__init__(spec, runtime)
        self.mult = float(spec.params.get("residual_mult", 1.0))
        self.mixer_after = self.extra["mixer_after"]
        self.ffn_after = self.extra.get("ffn_after")
        self.side = self.extra.get("side")
        if (self.ffn is None) != (self.ffn_after is None):
            raise ValueError("a feed-forward and the norm after it come together")
        if self.side is not None and not ("side_norm" in self.extra and "side_after" in self.extra):
            raise ValueError("a side sublayer comes with what stands before and after it")

    def _normed(self, values, norm) -> NormedDelta:
        if not hasattr(norm, "delayed"):
            raise TypeError("the norm after a sublayer must be an RMS norm")
        return norm.delayed(values, self.mult)

    def forward(self, h, pending, ctx, cache, next_block=None):
        x = pending if isinstance(pending, UnscaledRows) else self.mixer_norm.forward(h, delta=pending, write_h=True)
        pending = self._normed(self.mixer.forward(x, ctx, cache), self.mixer_after)
        if self.ffn is not None:
            x = self.ffn_norm.forward(h, delta=pending, write_h=True)
            pending = self._normed(self.ffn.forward(x, ctx), self.ffn_after)
        if self.side is not None:
            x = self.extra["side_norm"].forward(h, delta=pending, write_h=True)
            pending = self._normed(self.side.forward(x, ctx), self.extra["side_after"])
        return pending


class ParallelSublayersBlock(Block):
    """One norm that both sublayers read: ``h' = h + (Mixer(Norm(h)) + FFN(Norm(h)))``; a layer may have no feed-forward. What
    the sublayers leave is handed on as a ``SummedDelta`` of their partial sums, which the norm that reads the stream next
    adds in one kernel: no product adds into the stream itself here."""
    ffn_has_norm = False

    def first_norm_after(self, producer, rows, h):
        return None         # both sublayers want the normed rows themselves

    def forward(self, h, pending, ctx, cache, next_block=None):
        x = self.mixer_norm.forward(h, delta=pending, write_h=True)
        sums = [self.mixer.forward(x, ctx, cache)]
        if self.ffn is not None:
            sums += self.ffn.forward_sums(x, ctx)
        return SummedDelta(sums)


_ARRANGEMENTS = {"pre_norm": PreNormBlock, "sandwich_norm": SandwichNormBlock, "parallel_sublayers": ParallelSublayersBlock}


def register_arrangement(name: str, block_class, replace: bool = False) -> None:
    if name in _ARRANGEMENTS and not replace:
        raise ValueError(f"arrangement {name!r} is already registered")
    _ARRANGEMENTS[name] = block_class


def build_block(spec: LayerSpec, runtime: Runtime) -> Block:
    if spec.arrangement not in _ARRANGEMENTS:
        raise KeyError(f"unknown arrangement {spec.arrangement!r}; registered: {', '.join(sorted(_ARRANGEMENTS))}")
    return _ARRANGEMENTS[spec.arrangement](spec, runtime)
