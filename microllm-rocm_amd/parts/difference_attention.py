"""Differential attention: every head is two attentions over the same values, and gives their difference.

Query head ``h`` is a pair of vectors ``(q1, q2)`` of ``dim`` channels, laid out side by side, and so is key head ``g = h //
(heads / kv_heads)``. Map ``m`` is an ordinary causal softmax attention of ``scale * q_m . k_m`` over the values of head ``g``.
With ``l = exp(sum(lq1 * lk1)) - exp(sum(lq2 * lk2)) + difference`` (four vectors ``[dim]`` of the layer, one number in all) the
head's result is ``a_1 - l a_2``, divided by its root mean square over the head's ``value_dim`` channels (no weight) and
multiplied by ``1 - difference``; then the output projection. Everything else (a convolution over time on q, k and v, pages,
padding to one width) is the softmax attention's that this part extends.

The maps are query heads of one attention: a key head caches ``[k1 | k2]`` as one key of ``2 dim`` channels, and the two
queries of a head are written as ``[q1 | 0]`` and ``[0 | q2]``, so ``2 * heads`` query heads over ``kv_heads`` key/value heads run
on the attention kernels as they are, and every key and value is cached and read once. The kernels leave the maps' results in
float32; the difference, its norm and the factor are formed where the split kernel's splits meet (single tokens) or by one
kernel more, and rounded once.
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..ops import kernels
from .base import Runtime, TensorDecl, VECTOR
from .bias_attention import BucketBiasAttention
from .registry import register_part
from .spec import PartSpec

MAPS = 2


class DifferentialAttention(BucketBiasAttention):
    def __init__(self, spec: PartSpec, runtime: Runtime):
        p = spec.params
        self.dim = int(p["dim"])
        self.difference = float(p["difference"])
        self.factor_on_second: Optional[float] = None
        super().__init__(PartSpec(spec.kind, {"qk_norm": False, "sink": False, "pad_heads": True, **p, "heads": MAPS * int(p["heads"]),
                                              "key_dim": MAPS * self.dim, "maps": MAPS}, spec.names), runtime)

    @property
    def inner_width(self) -> int:
        return self.result_heads * self.value_dim

    def tensors(self) -> Dict[str, TensorDecl]:
        decls = super().tensors()
        decls.update({self.name(role): TensorDecl((self.dim,), VECTOR) for role in ("lq1", "lk1", "lq2", "lk2")})
        return decls

    def bind(self, tensors: Mapping[str, torch.Tensor]) -> None:
        super().bind(tensors)
        first, second = (float(torch.exp((tensors[self.name(f"lq{m}")].double() * tensors[self.name(f"lk{m}")].double()).sum())) for m in (1, 2))
        self.factor_on_second = first - second + self.difference

    def forward_inner(self, x, ctx, cache, out: Optional[torch.Tensor] = None, out_scale: float = 1.0) -> torch.Tensor:
        q, _, pages = self._store(x, ctx, cache)
        combined = kernels.HeadDifference(self.value_dim, self.factor_on_second, self.eps, (1.0 - self.difference) * out_scale)
        if self.tiled:
            result = kernels.paged_attention(q, pages.k, pages.v, ctx.paged[pages.group], ctx, self.scale, self.window, self.heads, self.kv_heads,
                                             self.stored_dim, planner=self.planner, extras=kernels.AttentionExtras(difference=combined))
        else:
            maps = torch.empty((x.shape[0], self.heads * self.result_dim), dtype=torch.float32, device=x.device)
            self._attend(q, None, pages, ctx, maps, 1.0)
            result = kernels.attention_difference(maps, self.result_heads, combined.value_dim, combined.on_second, combined.eps, combined.factor,
                                                  self.runtime.dtype)
        if out is None:
            return result
        out.copy_(result)
        return out


register_part("mixer", "differential_attention", DifferentialAttention)
