"""Sums over depth: what a layer hands on is not its own result alone but a weighted sum of the embedding's output and of the
results of all layers so far, x = sum_j w[j] X_j, j = 0 .. i + 1 for layer i (X_0 the embedding's output, X_(i + 1) the
layer's own result).  The step keeps every X_j of its rows, in 32-bit; nothing is kept from step to step."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from .base import Part, TensorSpec


class DepthAverage(Part):
    """The weights of the sum behind one layer: ``weight`` [inputs], inputs = the layer's number + 2."""
    replayable = True
    taped = True

    def __init__(self, inputs: int):
        if inputs < 2:
            raise ValueError("a sum over depth has the embedding's output and a layer's result at least")
        self.inputs = int(inputs)
        self.weight: Optional[torch.Tensor] = None

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        return {"weight": TensorSpec((self.inputs,), kind="f32", init="ones")}

    def load(self, tensors):
        self.weight = tensors["weight"].float().contiguous()

    def spec(self, history: torch.Tensor, out: torch.Tensor) -> tuple:
        """``(hist, coef, out)`` for ``ops.residual_rows`` on the layer's result: ``history`` [>= inputs - 1, n, width] holds the
        inputs before it."""
        return (history[:self.inputs - 1], self.weight, out)

    def forward(self, ctx, x, history, out, y=None, slices: int = 1) -> None:
        """x += y (a sublayer's rows, float32, or ``slices`` pieces of them); out = the sum that ends with x."""
        ops.residual_rows(x, y, slices, self.spec(history, out))
