"""A state-space mixer with one decay a head and token (state-space duality): what enters the state and what reads it are
made from the token and shared by groups of heads.

Per token, with h the mixer's input, H heads of P values, G groups (head j belongs to group j // (H / G)), N state rows:

    [z | x | B | C | dt] = W_in h                              z, x [H, P];  B, C [G, N];  dt [H]
    x, B, C <- silu(conv(x | B | C) + b)                       causal, per channel
    dt <- softplus(dt + dt_bias)
    S <- exp(-exp(A_log) dt) S + dt B x^T;   y = S^T C + D x   per head, S [N, P]
    out = W_o (norm(y * silu(z)) * w)                          norm: in equal parts, each by its own root mean square

S starts at zero and lives in a 32-bit state slot `[H, N, P]` of the request; the convolution's last taps - 1 inputs are
state too.  Step sizes leave their projection as 32-bit sums; decays, recurrence, gate and norm are 32-bit in every mode;
the other projections and the convolution run in the activation type.  A float32 engine works row by row, in one order however a
prompt is cut; a bfloat16 engine takes decoded rows from the projection's sums to the gated norm in two kernels, and longer
portions in chunks on the matrix cores (see csrc/state_space.hip).
"""
from __future__ import annotations

import torch

from ..cache.manager import StateNeed
from ..kernels import ops
from .base import Part, WeightDecl, register
from .linear import Linear
from .short_conv import ShortConv


@register("mixer", "state_space")
class StateSpaceMixer(Part):
    """params: hidden_size, heads, value_dim, state, groups, conv_taps, norm_groups, eps, project_out (bool, default True;
    False: one of a joined pair of mixers, which owns the products in front and behind, and calls `heads`)."""

    CHUNKS_FROM = 72    # rows of the longest portion from which on the form over chunks is ahead of the one row by row

    graph_safe = True  # rows, slots and lengths are read on the GPU; launches depend on shapes only

    @classmethod
    def _widths(cls, params):
        """(values of all heads, channels of the convolution, outputs of the input projection)."""
        inner = params["heads"] * params["value_dim"]
        channels = inner + 2 * params["groups"] * params["state"]
        return inner, channels, inner + channels + params["heads"]

    @classmethod
    def output_width(cls, params):
        return cls._widths(params)[0]

    @classmethod
    def declare_weights(cls, params):
        w, h = params["hidden_size"], params["heads"]
        inner, channels, outputs = cls._widths(params)
        decl = {"in": WeightDecl((outputs, w)), "conv": WeightDecl((channels, params["conv_taps"])),
                "conv_bias": WeightDecl((channels,), init="normal"), "dt_bias": WeightDecl((h,), init="normal"),
                "A_log": WeightDecl((h,), init="zeros"), "D": WeightDecl((h,), init="ones"),
                "norm": WeightDecl((inner,), init="ones"), "o": WeightDecl((w, inner))}
        if not params.get("project_out", True):
            del decl["o"]
        return decl

    @classmethod
    def declare_cache(cls, params):
        need = {"S": StateNeed((int(params["heads"]), int(params["state"]), int(params["value_dim"])), torch.float32)}
        conv = ShortConv.state_need(cls._widths(params)[1], int(params["conv_taps"]))
        if conv is not None:
            need["conv"] = conv
        return need

    def cache_need(self):
        return self.declare_cache(self.params)

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.H, self.P, self.N = int(params["heads"]), int(params["value_dim"]), int(params["state"])
        self.G, self.norm_groups = int(params["groups"]), int(params["norm_groups"])
        if self.G < 1 or self.H % self.G:
            raise ValueError("heads must be a multiple of the groups")
        if not 0 < self.N <= ops.DECAY_SCAN_MAX_KEY_DIM:
            raise ValueError(f"a state of {self.N} rows is not supported: the kernels take 1..{ops.DECAY_SCAN_MAX_KEY_DIM}")
        self.eps = float(params["eps"])
        self.inner, self.channels, outputs = self._widths(params)
        self.heads_width = self.inner
        self.in_weight, self.in_width = tensors["in"], outputs
        # step sizes enter the recurrence: their rows once more, as a product that hands over its 32-bit sums (padded with
        # zero rows to whole tiles of 16 outputs where it runs on the matrix cores)
        dt = tensors["in"][outputs - self.H:]
        if dt.dtype == torch.bfloat16 and not rt.is_f32:
            self.dt = Linear(torch.nn.functional.pad(dt, (0, 0, 0, -self.H % 16)).contiguous(), rt.weight_tiles)
        else:
            self.dt = Linear(dt.float().contiguous())
        self.conv = ShortConv(tensors["conv"], out_bias=tensors["conv_bias"])
        f32 = lambda n: tensors[n].float().contiguous()
        self.dt_bias, self.a_log, self.skip, self.norm = f32("dt_bias"), f32("A_log"), f32("D"), f32("norm")
        self.proj = self.o = None
        if params.get("project_out", True):
            self.proj, self.o = Linear(self.in_weight, rt.weight_tiles), Linear(tensors["o"], rt.weight_tiles)

    def products(self):
        if self.proj is None or self.proj.weight.dtype != torch.bfloat16:
            return []
        return [("in", self.proj.out_features, self.proj.in_features, False, None),
                ("o", self.o.out_features, self.o.in_features, False, "norm")]

    def forward(self, x, batch, cache):
        """x [T, W] -> float32 [T, W], or a float32 stack [S, T, W] to be added in order (see Linear)."""
        out = torch.empty((x.shape[0], self.heads_width), dtype=x.dtype, device=x.device)
        if self.takes_sums(x, batch):
            self.heads_of_sums(self.proj(x, out_dtype=torch.float32, partials_ok=True), 0, batch, cache, out)
        else:
            self.heads(self.proj(x), x, batch, cache, out)
        return self.o(out, out_dtype=torch.float32, partials_ok=True)   # into the 32-bit residual unrounded

    def heads(self, y, x, batch, cache, out, factor: float = 1.0):
        """From y [T, in_width], the product of `in_weight` with x, what the output projection reads, times `factor`, into
        the view out [T, heads_width]."""
        inner, gn = self.inner, self.G * self.N
        dt = self.dt(x, out_dtype=torch.float32)
        u = self.conv(y[:, inner:inner + self.channels], batch, cache.get("conv"), silu=True)
        rest = (dt, self.a_log, self.dt_bias, self.skip, cache["S"].state, batch.seg_row0, batch.seg_slot)
        sizes = dict(heads=self.H, groups=self.G, state=self.N, value_dim=self.P)
        if (not self.rt.is_f32 and batch.max_qlen >= self.CHUNKS_FROM
                and ops.state_space_chunks_supported(u.dtype, x.shape[0], batch.seg_slot.numel(), self.H, self.N, self.P)):
            o = ops.state_space_chunks(u, *rest, **sizes)
        else:
            o = ops.state_space_rows(u[:, :inner], u[:, inner:inner + gn], u[:, inner + gn:], *rest, **sizes)
        ops.gated_group_norm(o, y[:, :inner], self.norm, self.eps, groups=self.norm_groups, factor=factor, out=out)

    def takes_sums(self, x, batch) -> bool:
        """Whether this step is one of decoded rows that `heads_of_sums` takes."""
        return (not self.rt.is_f32 and batch.max_qlen == 1 and x.shape[0] == batch.seg_slot.numel()
                and ops.state_space_decode_supported(self.N, self.P))

    def heads_of_sums(self, y, first, batch, cache, out, factor: float = 1.0):
        """`heads` of decoded rows from the product's 32-bit sums (a tensor or a stack of partial ones), whose columns from
        `first` on are this mixer's."""
        conv = cache.get("conv")
        ops.state_space_decode(y, first, self.conv.weight, self.conv.out_bias, conv.state if conv is not None else None, self.a_log,
                               self.dt_bias, self.skip, self.norm, cache["S"].state, batch.seg_row0, batch.seg_slot, self.eps, out,
                               heads=self.H, groups=self.G, state=self.N, value_dim=self.P, norm_groups=self.norm_groups,
                               factor=factor)
