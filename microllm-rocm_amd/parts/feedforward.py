"""The SwiGLU feed-forward: ``down(silu(gate(x)) * up(x))``, no biases; ``activation`` may name the tanh form of gelu
for the gate instead (``gelu_tanh``).

``z = g * sigmoid(g) * u`` with the sigmoid evaluated branch-stably
(src/ops/ops.cpp:72-76, 779-783; src/model/model.cpp:787-789). Gate and up are
stacked into one weight at bind time so the input is read once.
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..ops import kernels
from .base import FeedForward, MATRIX, Runtime, TensorDecl
from .linear import Weight, linear, linear_clamped_glu, linear_into_stream, takes_unscaled
from .registry import register_part
from .spec import PartSpec


class SwiGLU(FeedForward):
    graph_safe = True
    fuses_residual = True
    def __init__(self, spec: PartSpec, runtime: Runtime):
        super().__init__(spec, runtime)
        self.hidden = int(spec.params["hidden_size"])
        self.intermediate = int(spec.params["intermediate_size"])
        self.activation = str(spec.params.get("activation", "silu"))
        if self.activation not in kernels.GATED_ACTIVATIONS:
            raise ValueError(f"a gate's activation is one of {', '.join(sorted(kernels.GATED_ACTIVATIONS))}")
        self.gate_up_weight: Optional[torch.Tensor] = None
        self.down_weight: Optional[torch.Tensor] = None

    def tensors(self) -> Dict[str, TensorDecl]:
        return {
            self.name("gate_proj.weight"): TensorDecl((self.intermediate, self.hidden), MATRIX),
            self.name("up_proj.weight"): TensorDecl((self.intermediate, self.hidden), MATRIX),
            self.name("down_proj.weight"): TensorDecl((self.hidden, self.intermediate), MATRIX),
        }

    def bind(self, tensors: Mapping[str, torch.Tensor]) -> None:
        gate = tensors[self.name("gate_proj.weight")]
        up = tensors[self.name("up_proj.weight")]
        if gate.dtype != up.dtype:
            raise TypeError("the gate and up weights of one layer must share a dtype to be stacked")
        self.gate_up_weight = Weight(torch.cat([gate, up], dim=0).contiguous(), gated=True, keep_plain=self.runtime.keep_plain_weights)
        del gate, up
        self.down_weight = Weight(tensors[self.name("down_proj.weight")], keep_plain=self.runtime.keep_plain_weights)

    def takes_unscaled(self, rows: int) -> bool:
        return takes_unscaled(self.gate_up_weight, rows)

    def forward(self, x, ctx, residual=None):
        z = linear(x, self.gate_up_weight, gated=True, activation=self.activation)
        if residual is not None:
            begun = linear_into_stream(z, self.down_weight, residual)
            if begun is not None:
                return begun
        return linear(z, self.down_weight, out_dtype=torch.float32, partials=True)


register_part("ffn", "swiglu", SwiGLU)


class ClampedGLU(FeedForward):
    """A gated feed-forward with clamped inputs: ``g = min(gate(x), limit)``, ``u = clamp(up(x), -limit, limit)``,
    ``down(g * sigmoid(slope * g) * (u + 1))``, no biases. Gate and up are one stacked product; its float32 sums pass the
    activation (in the product's epilogue for few rows) and are rounded once."""
    graph_safe = True

    def __init__(self, spec: PartSpec, runtime: Runtime):
        super().__init__(spec, runtime)
        self.hidden = int(spec.params["hidden_size"])
        self.intermediate = int(spec.params["intermediate_size"])
        self.limit = float(spec.params["limit"])
        self.slope = float(spec.params.get("slope", 1.702))
        self.gate_up_weight: Optional[Weight] = None
        self.down_weight: Optional[Weight] = None

    def tensors(self) -> Dict[str, TensorDecl]:
        return {self.name("gate"): TensorDecl((self.intermediate, self.hidden), MATRIX),
                self.name("up"): TensorDecl((self.intermediate, self.hidden), MATRIX),
                self.name("down"): TensorDecl((self.hidden, self.intermediate), MATRIX)}

    def bind(self, tensors: Mapping[str, torch.Tensor]) -> None:
        gate, up = tensors[self.name("gate")], tensors[self.name("up")]
        if gate.dtype != up.dtype:
            raise TypeError("the gate and up weights of one layer must share a dtype to be stacked")
        self.gate_up_weight = Weight(torch.cat([gate, up], dim=0).contiguous(), gated=True, keep_plain=self.runtime.keep_plain_weights)
        del gate, up
        self.down_weight = Weight(tensors[self.name("down")], keep_plain=self.runtime.keep_plain_weights)

    def forward(self, x, ctx):
        z = linear_clamped_glu(x, self.gate_up_weight, self.limit, self.slope)
        return linear(z, self.down_weight, out_dtype=torch.float32, partials=True)


register_part("ffn", "clamped_glu", ClampedGLU)
