"""Token embedding: ``x[t, :] = float32(E[tokens[t], :]) * scale`` (``scale`` 1 unless the spec gives one).

Reference: ``src/model/qwen3.cpp:75,213`` and ``src/backend/cpu/cpu_backend.cpp:51-76``.
Token ids are checked against the vocabulary when a batch is built, before
anything runs. Parameters: ``vocab``, ``hidden``, ``weight`` (tensor name), ``scale`` (optional), ``norm`` (optional: a
PartSpec of a norm the embedded rows pass, its result the float32 stream; a norm that reads rows of either type
gathers them from the table itself, in one launch).
"""

from __future__ import annotations

from typing import List

import torch

from .. import kernels
from .base import Embedding, Part, StepContext, TensorSpec, build_part, register_part


@register_part("embedding", "token_embedding")
class TokenEmbedding(Embedding):
    capturable = True      # reads the step on the device only: may be recorded into a HIP graph

    def __init__(self, params):
        super().__init__(params)
        self.vocab = int(params["vocab"])
        self.hidden = int(params["hidden"])
        self.weight_name = params["weight"]
        self.scale = float(params.get("scale") or 1.0)
        self.norm = build_part("norm", params["norm"]) if params.get("norm") else None
        self.weight: torch.Tensor = None

    def children(self) -> List[Part]:
        return [self.norm] if self.norm is not None else []

    def tensors(self) -> List[TensorSpec]:
        return [TensorSpec(self.weight_name, (self.vocab, self.hidden), "matrix", ("normal", 0.02))]

    def load(self, fetch, mode, device) -> None:
        self.weight = fetch(self.weight_name, "matrix")

    def forward(self, ctx: StepContext, token_ids: torch.Tensor) -> torch.Tensor:
        x = ctx.scratch("residual", (token_ids.numel(), self.hidden), torch.float32)
        if self.norm is None:
            kernels.embed(self.weight, token_ids, x, self.scale)
            return x
        if self.scale == 1.0 and self.norm.reads_either_type:
            return self.norm.forward(ctx, self.weight, rows=token_ids, out_name="residual", out_dtype=torch.float32)
        rows = ctx.scratch("embedding.rows", x.shape, torch.float32)
        kernels.embed(self.weight, token_ids, rows, self.scale)
        return self.norm.forward(ctx, rows, out_name="residual", out_dtype=torch.float32)
