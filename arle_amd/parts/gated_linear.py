"""Gated linear attention: linear attention whose state decays by a number for every head and key entry, made from the
token through a narrow middle.

Per token, with h the mixer's input, H heads, key size D, value size Dv:

    q = D^(-1/2) W_q h,  k = W_k h,  v = W_v h;   decay = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)     [H, D]
    S <- diag(decay) S + k v^T;   o = S^T q                                                        (per head, S [D, Dv])
    out = W_o ((o / rms(o) per head) * w_norm * silu(W_g h))

S starts at zero and lives in a 32-bit state slot `[H, D, Dv]` of the request.  One fused product makes q, k, v, the gate
and the narrow middle and hands over its 32-bit sums; decays, recurrence and head norm are 32-bit in every mode (at a
request's first rows o is a few terms, whose signs the norm magnifies).  The middle's width is the tensors' own.  A float32
engine works row by row, in one order however a prompt is cut; a bfloat16 engine takes decoded rows in one kernel and
longer portions in chunks on the matrix cores (see csrc/gated_linear.hip).
"""
from __future__ import annotations

import torch

from ..cache.manager import StateNeed
from ..kernels import ops
from .base import Part, WeightDecl, register
from .linear import Linear


@register("mixer", "gated_linear")
class GatedLinearMixer(Part):
    """params: hidden_size, heads, key_dim, value_dim, tau, eps, decay_rank (int, or None: whatever the tensors have)."""

    CHUNKS_FROM = 128    # rows of the longest portion from which on the form over chunks is ahead of the one row by row

    graph_safe = True  # rows, slots and lengths are read on the GPU; launches depend on shapes only

    @classmethod
    def declare_weights(cls, params):
        w, h, d, dv, r = (params["hidden_size"], params["heads"], params["key_dim"], params["value_dim"],
                          params.get("decay_rank"))
        return {"q": WeightDecl((h * d, w)), "k": WeightDecl((h * d, w)), "v": WeightDecl((h * dv, w)),
                "g": WeightDecl((h * dv, w)), "a1": WeightDecl((r, w)), "a2": WeightDecl((h * d, r)),
                "a2_bias": WeightDecl((h * d,), init="normal"), "norm": WeightDecl((dv,), init="ones"),
                "o": WeightDecl((w, h * dv))}

    @classmethod
    def declare_cache(cls, params):
        return StateNeed((int(params["heads"]), int(params["key_dim"]), int(params["value_dim"])), torch.float32)

    def cache_need(self):
        return self.declare_cache(self.params)

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.H, self.D, self.Dv = int(params["heads"]), int(params["key_dim"]), int(params["value_dim"])
        if not 0 < self.D <= ops.DECAY_SCAN_MAX_KEY_DIM:
            raise ValueError(f"key_dim {self.D} is not supported: the kernels take 1..{ops.DECAY_SCAN_MAX_KEY_DIM}")
        self.eps, self.tau = float(params["eps"]), float(params["tau"])
        fused = [tensors[n] for n in ("q", "k", "v", "g", "a1")]
        if len({t.dtype for t in fused}) != 1:
            raise ValueError("q, k, v, gate and decay projections must be stored in one type")
        if tensors["a1"].shape[0] != tensors["a2"].shape[1]:
            raise ValueError("the two projections of the decay do not meet in one width")
        self.rank = int(tensors["a1"].shape[0])
        fused = torch.cat(fused, dim=0)
        self.proj = Linear(torch.nn.functional.pad(fused, (0, 0, 0, -fused.shape[0] % 16)).contiguous(), rt.weight_tiles)
        self.a2 = tensors["a2"].contiguous()
        self.a2_bias = tensors["a2_bias"].float().contiguous()
        self.norm = tensors["norm"].float().contiguous()
        self.o = Linear(tensors["o"], rt.weight_tiles)

    def products(self):
        if self.proj.weight.dtype != torch.bfloat16:
            return []
        return [("qkvga", self.proj.out_features, self.proj.in_features, False, "norm"),
                ("o", self.o.out_features, self.o.in_features, False, "norm")]

    def forward(self, x, batch, cache):
        """x [T, W] -> float32 [T, W], or a float32 stack [S, T, W] to be added in order (see Linear)."""
        rows, segments = x.shape[0], batch.seg_slot.numel()
        y = self.proj(x, out_dtype=torch.float32, partials_ok=True)
        form = ops.gated_linear_rows
        if not self.rt.is_f32 and batch.max_qlen == 1 and rows == segments and ops.gated_linear_decode_supported(self.Dv, self.rank):
            form = ops.gated_linear_decode
        else:
            if y.dim() == 3:
                y = ops.sum_partials(y, torch.float32)
            if (not self.rt.is_f32 and batch.max_qlen >= self.CHUNKS_FROM
                    and ops.gated_linear_chunks_supported(rows, segments, self.H, self.D, self.Dv)):
                form = ops.gated_linear_chunks
        out = form(y, self.a2, self.a2_bias, self.norm, cache.state, batch.seg_row0, batch.seg_slot, self.eps, self.rt.act_dtype,
                   tau=self.tau, heads=self.H, key_dim=self.D, value_dim=self.Dv)
        return self.o(out, out_dtype=torch.float32, partials_ok=True)   # into the 32-bit residual unrounded
