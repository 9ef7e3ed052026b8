"""Stages: changes of the residual stream before one entry of the run order.

``add_vector`` adds one row of a stored table to every row of the stream, ``x += table[row]``: what tells the passes of
layers that run several times apart. Parameters: ``hidden``, ``table`` (tensor name), ``rows`` (of the table), ``row``.
"""

from __future__ import annotations

from typing import List

import torch

from .. import kernels
from ..errors import InvalidArgument
from .base import Stage, StepContext, TensorSpec, register_part


@register_part("stage", "add_vector")
class AddVector(Stage):
    capturable = True

    def __init__(self, params):
        super().__init__(params)
        self.hidden = int(params["hidden"])
        self.table_name = params["table"]
        self.rows, self.row = int(params["rows"]), int(params["row"])
        if not 0 <= self.row < self.rows:
            raise InvalidArgument(f"row {self.row} of a table of {self.rows} rows")
        self.vector: torch.Tensor = None

    def tensors(self) -> List[TensorSpec]:
        return [TensorSpec(self.table_name, (self.rows, self.hidden), "vector", ("normal", 0.02))]

    def load(self, fetch, mode, device) -> None:
        self.vector = fetch(self.table_name, "vector")[self.row].to(torch.float32).contiguous()

    def forward(self, ctx: StepContext, x: torch.Tensor) -> None:
        # sums commute: products and partial sums still owed to the stream stay owed
        ctx.run_late()
        kernels.add_bias(x, self.vector)
