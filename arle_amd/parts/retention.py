"""Retention: linear attention with one fixed decay a head, without a softmax or a denominator.

Per token at position p, with h the mixer's input, H heads, key size D, value size Dv:

    q = turn_p(W_q h),  k = turn_p(W_k h) * D^(-1/2),  v = W_v h         (turn: a rotate-half rotation, optional)
    S' = decay_h S + k v^T;   o = S'^T q                                  (per head)
    out = W_o ((o / rms(o) per head) * silu(W_g h))

S starts at zero and lives in a 32-bit state slot `[H, D, Dv]` of the request.  One fused product makes q, k, v and the
gate and hands over its 32-bit sums; the rotation, the recurrence and the head norm are 32-bit in every mode (at a
request's first rows o is a single term, whose sign alone the norm keeps: what rounding q and k costs there is many
times a usual row's error).  A float32 engine works row by row, in one order however a prompt is cut; a bfloat16 engine
takes decoded rows in one kernel and longer portions in chunks on the matrix cores (see csrc/retention.hip).
"""
from __future__ import annotations

import torch

from ..cache.manager import StateNeed
from ..kernels import ops
from .base import Part, PartSpec, WeightDecl, register
from .linear import Linear


@register("mixer", "retention")
class RetentionMixer(Part):
    """params: hidden_size, heads, key_dim, value_dim, decay (a number for every head), eps, position (PartSpec of a
    rotation of the rotate-half layout, or None)."""

    graph_safe = True  # rows, slots and positions are read on the GPU; launches depend on shapes only

    CHUNKS_FROM = 192    # rows of the longest portion from which on the form over chunks is ahead of the one row by row

    @classmethod
    def declare_weights(cls, params):
        w, h, d, dv = params["hidden_size"], params["heads"], params["key_dim"], params["value_dim"]
        return {"q": WeightDecl((h * d, w)), "k": WeightDecl((h * d, w)), "v": WeightDecl((h * dv, w)),
                "g": WeightDecl((h * dv, w)), "o": WeightDecl((w, h * dv))}

    @classmethod
    def children(cls, params):
        return {"position": ("position", params.get("position") or PartSpec("none"))}

    @classmethod
    def declare_cache(cls, params):
        return StateNeed((int(params["heads"]), int(params["key_dim"]), int(params["value_dim"])), torch.float32)

    def cache_need(self):
        return self.declare_cache(self.params)

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.H, self.D, self.Dv = int(params["heads"]), int(params["key_dim"]), int(params["value_dim"])
        if not 0 < self.D <= ops.RETENTION_MAX_KEY_DIM:
            raise ValueError(f"key_dim {self.D} is not supported: the retention kernels take 1..{ops.RETENTION_MAX_KEY_DIM}")
        decay = torch.tensor([float(g) for g in params["decay"]], dtype=torch.float64)
        if decay.numel() != self.H:
            raise ValueError(f"{decay.numel()} decays for {self.H} heads")
        self.decay = decay.float().to(rt.device)
        self.powers = (decay[:, None] ** torch.arange(ops.RETENTION_CHUNK + 1, dtype=torch.float64)).float().to(rt.device)
        self.eps = float(params["eps"])
        self.position = children["position"]
        if self.position.kind not in ("rope_neox", "none"):
            raise ValueError("the retention kernels rotate in the rotate-half layout")
        fused = [tensors[n] for n in ("q", "k", "v", "g")]
        if len({t.dtype for t in fused}) != 1:
            raise ValueError("q, k, v and gate projections must be stored in one type")
        self.qkvg = Linear(torch.cat(fused, dim=0).contiguous(), rt.weight_tiles)
        self.o = Linear(tensors["o"], rt.weight_tiles)

    def products(self):
        if self.qkvg.weight.dtype != torch.bfloat16:
            return []
        return [("qkvg", self.qkvg.out_features, self.qkvg.in_features, False, "norm"),
                ("o", self.o.out_features, self.o.in_features, False, "norm")]

    def forward(self, x, batch, cache):
        """x [T, W] -> float32 [T, W], or a float32 stack [S, T, W] to be added in order (see Linear)."""
        self.position.ensure_positions(batch.max_position + 1)
        cos, sin, rot = self.position.fused_rotary()
        rows, segments = x.shape[0], batch.seg_slot.numel()
        y = self.qkvg(x, out_dtype=torch.float32, partials_ok=True)
        common = dict(positions=batch.positions, cos=cos, sin=sin, rotary_dims=rot, heads=self.H, key_dim=self.D,
                      value_dim=self.Dv)
        where = (cache.state, batch.seg_row0, batch.seg_slot, self.eps, self.rt.act_dtype)
        if not self.rt.is_f32 and batch.max_qlen == 1 and rows == segments and ops.retention_decode_supported(self.Dv):
            out = ops.retention_decode(y, self.decay, *where, **common)
        else:
            if y.dim() == 3:
                y = ops.sum_partials(y, torch.float32)
            if (not self.rt.is_f32 and batch.max_qlen >= self.CHUNKS_FROM
                    and ops.retention_chunks_supported(rows, segments, self.H, self.D, self.Dv, rot)):
                out = ops.retention_chunks(y, self.powers, *where, **common)
            else:
                out = ops.retention_rows(y, self.decay, *where, **common)
        return self.o(out, out_dtype=torch.float32, partials_ok=True)   # into the 32-bit residual unrounded
