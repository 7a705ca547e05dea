"""Joins of the residual rows with the embedding output in front of a run-order entry, for stacks that pass some of
their layers several times and feed the input in again.

`linear_join`: x <- W [x ; x0] with a learnt matrix W [width, 2 width], x the residual rows (first) and x0 the
embedding output; no norm, no bias.  The product's operand rows [x | x0] live in the compute dtype, the right half
written once a step; the product leaves float sums, which are the new residual rows.  The reference has no repeated
layers."""
from __future__ import annotations

from typing import Dict, List

import torch

from .. import kernels as K
from ..weights import TensorSpec
from .base import InputJoin, Runtime, register_part
from .linear import linear, stream_layout


class LinearJoin(InputJoin):
    graph_safe = True

    def __init__(self, hidden_size: int, tensor: str = "weight"):
        """`tensor`: the piece of the matrix's name behind the part's prefix ("" where the prefix is the whole name)."""
        self.H, self.tensor = int(hidden_size), tensor
        self.w = None

    def weight_specs(self, prefix: str) -> List[TensorSpec]:
        return [TensorSpec(prefix + self.tensor, (self.H, 2 * self.H))]

    def load(self, tensors: Dict[str, torch.Tensor], prefix: str, rt: Runtime) -> None:
        self.rt = rt
        self.w = stream_layout(tensors[prefix + self.tensor], rt)

    def _rows(self, step) -> torch.Tensor:
        return step.ws.get(f"join_rows_{id(self)}", (step.n_tokens, 2 * self.H), self.rt.dtype)

    def begin(self, x, step) -> None:
        K.rows_into(x, self._rows(step)[:, self.H:])

    def forward(self, x, step) -> None:
        rows = self._rows(step)
        K.rows_into(x, rows[:, :self.H])
        linear(rows, self.w, x, step.ws)


register_part("input_join", "linear_join", LinearJoin, replace=True)
