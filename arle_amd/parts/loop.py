"""The entry of a run of layers that is repeated with the same weights and reminded of the embedding in every pass.

The block `loop_entry` stands in the schedule once in front of all layers, where it keeps the residual as it then is, and
once in front of every pass, where it replaces the residual by a projection of it beside what was kept, plus a row of its
own for each pass:

    x <- W [x; x_kept] + step_t           t = 0, 1, ...: the passes that began before this one

Operands of the product are in the activation type, its sums and the residual 32-bit.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import Part, Pending, WeightDecl, register
from .linear import Linear

def _terms(delta) -> list:
    terms = delta if isinstance(delta, list) else ([] if delta is None else [(delta, None)])
    if any(bias is not None for _, bias in terms):
        raise ValueError("a loop's entry adds terms without biases")
    return [term for term, _ in terms]


@register("feed_forward", "joined_input")
class JoinedInput(Part):
    """The tensors of a loop's entry.  params: width, times (rows of `step`)."""

    graph_safe = True  # launches depend on shapes only, never on the values of a step

    @classmethod
    def declare_weights(cls, params):
        w = params["width"]
        return {"in": WeightDecl((w, 2 * w)), "step": WeightDecl((params["times"], w), init="normal")}

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.width, self.times = int(params["width"]), int(params["times"])
        self.proj = Linear(tensors["in"], rt.weight_tiles)
        self.step = tensors["step"].float().contiguous()

    def products(self):
        if self.proj.weight.dtype != torch.bfloat16:
            return []
        return [("in", self.proj.out_features, self.proj.in_features, False, "norm")]

    def forward(self, joined):
        """[T, 2W] -> float32 [T, W], or a float32 stack [S, T, W] to be added in order (see Linear)."""
        return self.proj(joined, out_dtype=torch.float32, partials_ok=True)


@register("block", "loop_entry")
class LoopEntryBlock:
    """A further part `join` (a `joined_input`).  Between its runs it keeps [T, 2W] of the activation type in `batch.carry`,
    what it kept in the right half.  In front of a pass, the first summand (a whole product, or the first of its partial
    sums) becomes the residual; the other partial sums and the pass's row are left for the next norm to add."""

    mixer = feed_forward = None

    def __init__(self, mixer, feed_forward, norms: dict, extra: dict):
        self.join = extra["join"]

    def forward(self, residual, delta, batch, cache_view):
        width = residual.shape[1]
        joined, begun = batch.carry.get(self, (None, 0))
        if joined is None:
            if delta is not None:
                raise ValueError("a loop's entry keeps the residual before any layer has run")
            joined = torch.empty((residual.shape[0], 2 * width), dtype=self.join.rt.act_dtype, device=residual.device)
            ops.add_terms_into(residual, (), joined[:, width:])
            batch.carry[self] = (joined, 0)
            return residual, None
        if begun >= self.join.times:
            raise ValueError("a loop runs more often than it has rows for its passes")
        batch.carry[self] = (joined, begun + 1)
        ops.add_terms_into(residual, _terms(delta), joined[:, :width])
        y = self.join.forward(joined)
        left = Pending()
        if y.dim() == 3:
            if y.shape[0] > 1:
                left.append((y[1:], None))
            y = y[0]
        left.append((ops.EveryRow(self.join.step[begun]), None))
        return y, left
