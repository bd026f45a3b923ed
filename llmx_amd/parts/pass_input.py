"""What happens to the residual at the start of a pass of a repeated run of layers.

"pass_vector": x <- (x + embedding rows) + table[index], the embedding rows only where the part says so (every pass but a
loop's first), table a tensor [passes, hidden] with one learned vector a pass.  All float32.
"pass_projection": x <- W [x ; embedding rows], W [hidden, 2 hidden]: the residual is replaced by a product that reads it and
the embedding's rows side by side (rounded, where products read rounded rows; its sum and x are float32).
"""

from __future__ import annotations

import torch

from .. import ops
from .base import ResidualInput, register
from .spec import TensorSpec


class PassVector(ResidualInput):
    """params: hidden, passes (rows of the table), index (the pass), add_embedding (bool).  Tensor: the prefix itself,
    (passes, hidden); every pass's part lists it, and all read the one device tensor."""
    graph_safe = True

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.hidden = int(params["hidden"])
        self.passes = int(params["passes"])
        self.index = int(params["index"])
        if not 0 <= self.index < self.passes:
            raise ValueError(f"pass vector: pass {self.index} outside the table's {self.passes}")
        self.wants_embedding = bool(params.get("add_embedding", False))
        self.vector = None

    def tensor_specs(self, available):
        if self.index:          # the table is listed once, by the first pass's part
            return []
        return [TensorSpec(self.prefix, (self.passes, self.hidden), "bias", init=("normal", 0.0, 0.02))]

    def load(self, tensors):
        self.vector = tensors[self.prefix][self.index]

    def forward(self, step, x, embedding_rows):
        ops.add_rows_vector(x, embedding_rows if self.wants_embedding else None, self.vector)


class PassProjection(ResidualInput):
    """params: hidden.  Tensor: the prefix itself, (hidden, 2 * hidden), the residual's columns first."""
    graph_safe = True
    wants_embedding = True

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.hidden = int(params["hidden"])
        self.weight = None

    def tensor_specs(self, available):
        return [TensorSpec(self.prefix, (self.hidden, 2 * self.hidden))]

    def load(self, tensors):
        self.weight = tensors[self.prefix]

    def forward(self, step, x, embedding_rows):
        T, E = x.shape
        rows = step.buf("pass.rows", (T, 2 * E), step.act_dtype)
        there = step.shared("pass.embedding_half", dict)      # the embedding's half stays from a step's first pass on
        ops.join_rows(x, None if there else embedding_rows, rows)
        there["written"] = True
        ops.gemm(rows, self.weight, x, scratch=step.buf)


register("residual_input", "pass_vector", PassVector)
register("residual_input", "pass_projection", PassProjection)
