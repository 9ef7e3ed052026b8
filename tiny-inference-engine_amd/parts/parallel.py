"""Two (or more) mixers side by side: all read the same rows, their outputs are added with a factor each.

``y = sum_i scale_i * mixer_i(h)``. A branch is any registered mixer; its factor is handed to it as the parameter
``output_scale``, and the branch folds it into something it computes in float32 anyway (a convolution's weights, a
norm's weights), so that no pass over the rows is spent on it. The branches' cache needs are declared together, in
order (``Mixer.cache_need`` as a tuple), and every branch is bound to its own. Branches that name their first product
(``Part.first_product``) have it formed as one over their weights side by side. Parameters: ``hidden``, ``branches``
(a list of ``(PartSpec of the mixer family, scale)``) and, for designs that have them, ``output_norms`` ``{"eps",
"weights"}`` (a tensor name a branch): ``y = sum_i scale_i * mixer_i(h) / rms(mixer_i(h)) * w_i`` over the model width.
Nothing is folded into the branches then; the factor joins the norm's weight, and what is added to the stream is left
for the next norm's own pass over it.
"""

from __future__ import annotations

from typing import List, Optional

import torch

from .. import kernels
from ..errors import InvalidArgument
from .base import Mixer, Part, PartSpec, StepContext, TensorSpec, build_part, register_part
from .linear import Linear


def _needs_of(mixer) -> tuple:
    need = mixer.cache_need()
    if need is None:
        return ()
    return tuple(need) if isinstance(need, (tuple, list)) else (need,)


@register_part("mixer", "parallel")
class ParallelMixer(Mixer):
    capturable = True
    replayable = True
    returns_result = True

    def __init__(self, params):
        super().__init__(params)
        self.hidden = int(params["hidden"])
        self.branches: List[Mixer] = []
        self.norms = dict(params["output_norms"]) if params.get("output_norms") else None
        self.scales = [float(scale) for _, scale in params["branches"]]
        for spec, scale in params["branches"]:
            branch_params = dict(spec.params)
            if self.norms is None:
                branch_params["output_scale"] = float(scale) * float(branch_params.get("output_scale", 1.0))
            self.branches.append(build_part("mixer", PartSpec(spec.kind, branch_params)))
        if not self.branches:
            raise InvalidArgument("a parallel mixer needs at least one branch")
        self.counts = [len(_needs_of(b)) for b in self.branches]
        self.norm_weights: List[torch.Tensor] = []
        self.first = None              # the branches' first products as one Linear
        if self.norms is not None:
            if len(self.norms["weights"]) != len(self.branches) or len(self.branches) > 2:
                raise InvalidArgument("norms behind the branches: one weight a branch, and at most two branches")
            if not all(getattr(b, "returns_result", False) for b in self.branches):
                raise InvalidArgument("a norm behind a branch needs a mixer that returns its result")

    def tensors(self) -> List[TensorSpec]:
        if self.norms is None:
            return []
        return [TensorSpec(name, (self.hidden,), "vector", ("one_plus_uniform", 0.1)) for name in self.norms["weights"]]

    def load(self, fetch, mode, device) -> None:
        if self.norms is not None:
            self.norm_weights = [(fetch(name, "vector").to(torch.float32) * scale).contiguous()
                                 for name, scale in zip(self.norms["weights"], self.scales)]

    def load_all(self, fetch, mode, device) -> None:
        super().load_all(fetch, mode, device)
        linears = [b.first_product() for b in self.branches]
        self.first = Linear.joined(linears) if len(linears) > 1 and None not in linears else None

    def children(self) -> List[Part]:
        return list(self.branches)

    def cache_need(self):
        needs = tuple(n for b in self.branches for n in _needs_of(b))
        return needs or None

    def _caches(self, cache):
        """Every branch's own binding(s), in the shape it declared them."""
        bindings = () if cache is None else (tuple(cache) if isinstance(cache, tuple) else (cache,))
        out, at = [], 0
        for branch, count in zip(self.branches, self.counts):
            mine = bindings[at:at + count]
            at += count
            declared = branch.cache_need()
            out.append(None if count == 0 else (mine if isinstance(declared, (tuple, list)) else mine[0]))
        return out

    def forward(self, ctx: StepContext, h: torch.Tensor, cache, residual: Optional[torch.Tensor]):
        caches = self._caches(cache)
        if self.first is not None:
            both = ctx.scratch("parallel.first_products", (h.shape[0], self.first.total_out), torch.float32)
            self.first(h, both, ctx=ctx)
            at = 0
            for branch in self.branches:
                linear = branch.first_product()
                ctx.give_product(linear, both[:, at:at + linear.total_out])
                at += linear.total_out
        if self.norms is not None:
            return self._normed(ctx, h, caches, residual)
        target = residual
        first = 0
        if target is None:
            # The first branch's result becomes the sum the others add to.
            y = self.branches[0].forward(ctx, h, caches[0], None) \
                if getattr(self.branches[0], "returns_result", False) else None
            ctx.settle()
            if isinstance(y, torch.Tensor) and y.dim() == 2:
                target, first = y, 1
            else:
                target = ctx.scratch("parallel.result", (h.shape[0], self.hidden), torch.float32)
                target.zero_()
                if isinstance(y, torch.Tensor):
                    kernels.add_partials(target, y)
                    first = 1
        for branch, binding in zip(self.branches[first:], caches[first:]):
            branch.forward(ctx, h, binding, target)
        if residual is None:
            ctx.settle()
            return target
        return None

    def _normed(self, ctx: StepContext, h: torch.Tensor, caches, residual: Optional[torch.Tensor]):
        eps = float(self.norms["eps"])
        left = [(branch.forward(ctx, h, binding, None), weight, eps)
                for branch, binding, weight in zip(self.branches, caches, self.norm_weights)]
        if residual is not None:
            ctx.leave_late(("normed_results",) + tuple(residual.shape),
                           lambda results: kernels.add_normed_results(residual, results), left)
            return None
        ctx.settle()
        target = ctx.scratch("parallel.result", (h.shape[0], self.hidden), torch.float32)
        target.zero_()
        kernels.add_normed_results(target, left)
        return target
