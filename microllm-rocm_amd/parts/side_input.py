"""A sublayer that feeds every layer a vector of the token's own.

One table beside the embedding holds, for every token id, a row of ``dim`` numbers a layer, side by side. Layer ``i``
takes ``e``, its ``dim`` columns of the token's row, and adds ``P (gelu(G x) * e)`` to the stream, ``G`` being ``[dim,
hidden]``, ``P`` ``[hidden, dim]`` and gelu its tanh form (what stands before and after it is the arrangement's). The
table is one tensor that all layers name; each reads its own columns of the step's rows where it multiplies (for few
rows in the gate product's epilogue). The gate's
sums, its activation and the product with ``e`` are float32 and rounded once.
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..ops import kernels
from .base import FeedForward, MATRIX, Runtime, TensorDecl
from .linear import SKINNY_ROWS, Weight, linear
from .registry import register_part
from .spec import PartSpec


class TokenSideInput(FeedForward):
    graph_safe = True

    def __init__(self, spec: PartSpec, runtime: Runtime):
        super().__init__(spec, runtime)
        self.hidden = int(spec.params["hidden_size"])
        self.vocab = int(spec.params["vocab_size"])
        self.dim = int(spec.params["dim"])
        self.table_columns = int(spec.params["table_columns"])      # of the whole table: dim times the layers that read it
        self.column_at = int(spec.params["column_at"])
        if not 0 <= self.column_at <= self.table_columns - self.dim:
            raise ValueError("the layer's columns lie inside the side table")
        self.table: Optional[torch.Tensor] = None
        self.gate_weight: Optional[Weight] = None
        self.out_weight: Optional[Weight] = None

    def tensors(self) -> Dict[str, TensorDecl]:
        return {self.name("table"): TensorDecl((self.vocab, self.table_columns), MATRIX),
                self.name("gate"): TensorDecl((self.dim, self.hidden), MATRIX),
                self.name("proj"): TensorDecl((self.hidden, self.dim), MATRIX)}

    def bind(self, tensors: Mapping[str, torch.Tensor]) -> None:
        keep = self.runtime.keep_plain_weights
        self.table = tensors[self.name("table")]
        self.gate_weight = Weight(tensors[self.name("gate")], keep_plain=keep)
        self.out_weight = Weight(tensors[self.name("proj")], keep_plain=keep)

    def weight_bytes_read(self, rows: int) -> int:
        """Both products' weights and the rows' columns of the table (not the table)."""
        weights = sum((weight.tensor if weight.tensor is not None else weight.packed).element_size() * weight.out_features * weight.in_features
                      for weight in (self.gate_weight, self.out_weight))
        return weights + rows * self.dim * self.table.element_size()

    def forward(self, x, ctx):
        if x.shape[0] <= SKINNY_ROWS and self.gate_weight.packed is not None and x.dtype == torch.bfloat16:
            g = kernels.gemm_skinny_side(x, self.gate_weight.packed, self.dim, self.table, self.column_at, ctx.tokens)
            return linear(g, self.out_weight, out_dtype=torch.float32, partials=True)
        z = linear(x, self.gate_weight, out_dtype=torch.float32, partials=True)
        g = kernels.token_side_gate(z, self.table, self.column_at, ctx.tokens, self.runtime.dtype)
        return linear(g, self.out_weight, out_dtype=torch.float32, partials=True)


register_part("ffn", "token_side_input", TokenSideInput)
