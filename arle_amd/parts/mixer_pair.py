"""Two mixers side by side on one input.

`mixer_pair`: each one's output is RMS-normed over the model width with a weight of its own, and the result is `coef` times
their sum (the mean, by default).

    out = coef * (left(h) / rms(left(h)) * w_left + right(h) / rms(right(h)) * w_right)

`mixer_sum`: each one's output counts a number of times, left_scale * left(h) + right_scale * right(h).  The pair owns the
projections of both: one product makes what the two read (the rows of both input projections), and, since a factor on a
mixer's output is one on what its output projection reads, one product with the two output projections side by side makes
the sum.

Each mixer keeps the cache or state it declares; a pair's need is the dictionary {"left": ..., "right": ...}.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import Part, WeightDecl, lookup, register
from .linear import Linear


class _TwoMixers(Part):
    """What both kinds share: params left and right (PartSpecs of mixers), the need of each under its name."""

    @classmethod
    def children(cls, params):
        return {"left": ("mixer", params["left"]), "right": ("mixer", params["right"])}

    @classmethod
    def _need(cls, left, right):
        need = {name: n for name, n in (("left", left), ("right", right)) if n is not None}
        return need or None

    @classmethod
    def declare_cache(cls, params):
        return cls._need(*(lookup("mixer", params[s].kind).declare_cache(params[s].params) for s in ("left", "right")))

    def cache_need(self):
        return self._need(self.left.cache_need(), self.right.cache_need())

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.left, self.right = children["left"], children["right"]
        self.graph_safe = all(bool(getattr(m, "graph_safe", False)) for m in (self.left, self.right))

    def decode_launch_class(self, rows, max_context):
        found = tuple(m.decode_launch_class(rows, max_context) for m in (self.left, self.right))
        return None if all(f is None for f in found) else found


@register("mixer", "mixer_pair")
class MixerPair(_TwoMixers):
    """params: width, eps, left (PartSpec of a mixer), right (PartSpec of a mixer), coef (default 0.5)."""

    @classmethod
    def declare_weights(cls, params):
        return {"left_out": WeightDecl((params["width"],), init="ones"), "right_out": WeightDecl((params["width"],), init="ones")}

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.eps = float(params["eps"])
        self.coef = float(params.get("coef", 0.5))
        self.w_left = tensors["left_out"].float().contiguous()
        self.w_right = tensors["right_out"].float().contiguous()

    def products(self):
        return self.left.products() + self.right.products()

    def forward(self, x, batch, cache):
        """x [T, W] -> float32 [T, W]."""
        cache = cache or {}
        a = self.left.forward(x, batch, cache.get("left"))
        b = self.right.forward(x, batch, cache.get("right"))
        return ops.pair_norm(a, b, self.w_left, self.w_right, self.eps, self.coef)


def _columns(weights, widths) -> torch.Tensor:
    """Matrices [W, n_i] side by side, each followed by zero columns up to a width of widths[i]."""
    return torch.cat([torch.nn.functional.pad(w, (0, n - w.shape[1])) for w, n in zip(weights, widths)], dim=1).contiguous()


@register("mixer", "mixer_sum")
class MixerSum(_TwoMixers):
    """params: width, left, right (PartSpecs of mixers with `heads`, built with project_out False), left_scale,
    right_scale."""

    @classmethod
    def declare_weights(cls, params):
        widths = {s: lookup("mixer", params[s].kind).output_width(params[s].params) for s in ("left", "right")}
        return {s + "_o": WeightDecl((params["width"], n)) for s, n in widths.items()}

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.scales = (float(params["left_scale"]), float(params["right_scale"]))
        both = (self.left, self.right)
        if len({m.in_weight.dtype for m in both} | {tensors[n].dtype for n in ("left_o", "right_o")}) != 1:
            raise ValueError("the projections of a joined pair must be stored in one type")
        # each mixer's columns begin at a multiple of 16 entries; what lies between is zero on both sides
        pad16 = lambda n: -(-n // 16) * 16
        self.out_widths = tuple(pad16(m.heads_width) for m in both)
        self.padded = any(p != m.heads_width for p, m in zip(self.out_widths, both))
        self.in_at = pad16(self.left.in_width)
        rows = [torch.nn.functional.pad(m.in_weight, (0, 0, 0, pad16(m.in_width) - m.in_width)) for m in both]
        self.proj = Linear(torch.cat(rows, dim=0).contiguous(), rt.weight_tiles)
        for m in both:
            m.in_weight = None      # held here
        self.o = Linear(_columns([tensors["left_o"], tensors["right_o"]], self.out_widths), rt.weight_tiles)

    def products(self):
        if self.proj.weight.dtype != torch.bfloat16:
            return []
        return [("in", self.proj.out_features, self.proj.in_features, False, None),
                ("o", self.o.out_features, self.o.in_features, False, "norm")]

    def forward(self, x, batch, cache):
        """x [T, W] -> float32 [T, W], or a float32 stack [S, T, W] to be added in order (see Linear)."""
        cache = cache or {}
        sums = all(m.takes_sums(x, batch) for m in (self.left, self.right))     # decoded rows: no pass that adds the partial sums
        y = self.proj(x, out_dtype=torch.float32, partials_ok=True) if sums else self.proj(x)
        make = torch.zeros if self.padded else torch.empty
        out = make((x.shape[0], sum(self.out_widths)), dtype=x.dtype, device=x.device)
        first, at = 0, 0
        for name, m, factor, width in zip(("left", "right"), (self.left, self.right), self.scales, self.out_widths):
            view = out[:, at:at + m.heads_width]
            if sums:
                m.heads_of_sums(y, first, batch, cache.get(name), view, factor)
            else:
                m.heads(y[:, first:first + m.in_width], x, batch, cache.get(name), view, factor)
            first, at = self.in_at, at + width
        return self.o(out, out_dtype=torch.float32, partials_ok=True)   # it goes into the 32-bit residual unrounded
