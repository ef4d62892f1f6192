"""A mixture of experts with a sigmoid or softmax router, and an optional shared expert that every token uses.

    z = W_r h + bias (32-bit; the bias optional),  s = sigmoid(z), softmax(z) or (score "softmax_chosen") z itself;  the `top` experts with the largest s + correction are chosen,
    with `groups`: only among the experts of the `keep_groups` groups of neighbours that hold the largest such numbers;
    weight_e = s_e / (sum of the chosen s + 1e-20) * scale, or without `normalize` s_e * scale; where s is z, the softmax
    over the chosen z alone, times scale;
    expert: down(silu(gate h) * (up h)), or (form "squared_relu") down(max(up h, 0)^2), no biases; the last `identity` outputs of the router stand for experts without
    tensors that hand back h itself;
    out = sum over the chosen experts of weight_e expert_e(h) (weigh "input": of expert_e(weight_e h))  +  shared(h), or with `shared_gate` sigmoid(W_s h) shared(h),
    one number a token

The router's kernel leaves the chosen experts and their weights on the GPU; the experts' kernel finds, workgroup by
workgroup, the rows that chose its expert, so no step sorts rows or reads anything back and its launches follow the
number of rows alone.  The experts' outputs stay apart, one row a (token, choice), in float32: the norm behind the
feed-forward weighs and adds them in the order of the choices, in the pass that computes its statistics
(`forward` returns the addends, not their sum).
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import Part, PartSpec, WeightDecl, register


# how an expert is made -> the dense feed-forward of the same form (the shared expert's)
EXPERT_FORMS = {"gated_silu": "swiglu", "squared_relu": "squared_relu"}


@register("feed_forward", "sigmoid_moe")
class SigmoidMoE(Part):
    """params: hidden_size, experts (those with tensors), top, expert_size, scale, correction (bool),
    shared_size (int | None), shared_gate (bool), form ("gated_silu", the default, or "squared_relu": of the experts and
    the shared one), bias (bool: of the router), score ("sigmoid", the default, "softmax" or "softmax_chosen"), normalize (bool, default True),
    weigh ("output", the default, or "input": what a chosen expert's weight multiplies), groups (default 1), keep_groups (default 1), identity (default 0: router outputs behind the experts' that stand
    for experts which hand back their input; groups and the softmax run over experts and these together)."""

    graph_safe = True  # launches depend on shapes only; what a token chose is read on the GPU

    @classmethod
    def declare_weights(cls, params):
        h, i, E = params["hidden_size"], params["expert_size"], params["experts"]
        outputs = E + int(params.get("identity") or 0)
        decl = {"router": WeightDecl((outputs, h))}
        if params.get("correction"):
            decl["correction"] = WeightDecl((outputs,), init="normal")
        if params.get("bias"):
            decl["bias"] = WeightDecl((outputs,), init="normal")
        if params.get("shared_gate"):
            decl["shared_gate"] = WeightDecl((1, h))
        gated = cls._form(params) == "gated_silu"
        for e in range(E):
            if gated:
                decl[f"gate{e}"] = WeightDecl((i, h))
            decl.update({f"up{e}": WeightDecl((i, h)), f"down{e}": WeightDecl((h, i))})
        return decl

    @staticmethod
    def _form(params) -> str:
        form = params.get("form") or "gated_silu"
        if form not in EXPERT_FORMS:
            raise ValueError(f"unknown form of expert {form!r} (known: {', '.join(EXPERT_FORMS)})")
        return form

    @classmethod
    def children(cls, params):
        if not params.get("shared_size"):
            return {}
        shared = PartSpec(EXPERT_FORMS[cls._form(params)], {"hidden_size": params["hidden_size"], "intermediate_size": params["shared_size"],
                                     "float32_out": True}, params["shared_weights"])
        return {"shared": ("feed_forward", shared)}

    def __init__(self, params, tensors, rt, children=None):
        super().__init__(params, tensors, rt, children)
        self.E, self.top = int(params["experts"]), int(params["top"])
        self.identity = int(params.get("identity") or 0)
        outputs = self.E + self.identity
        self.score = params.get("score") or "sigmoid"
        self.normalize = bool(params.get("normalize", True))
        self.groups, self.keep_groups = int(params.get("groups") or 1), int(params.get("keep_groups") or 1)
        if self.score not in ops.MOE_SCORES:
            raise ValueError(f"a router's scores are one of {', '.join(ops.MOE_SCORES)}")
        if self.E < 1 or self.identity < 0 or not 1 <= self.top <= outputs:
            raise ValueError("a token chooses between 1 and all of the experts")
        if outputs > ops.MOE_MAX_EXPERTS or self.top > ops.MOE_MAX_TOP:
            raise ValueError(f"up to {ops.MOE_MAX_EXPERTS} experts and {ops.MOE_MAX_TOP} choices a token are taken")
        if (self.groups < 1 or outputs % self.groups or not 1 <= self.keep_groups <= self.groups
                or self.top > self.keep_groups * (outputs // self.groups)):
            raise ValueError("groups divide the router's outputs evenly, and the kept groups hold at least `top` of them")
        self.scale = float(params.get("scale", 1.0))
        self.router = tensors["router"]
        self.correction = tensors.get("correction")
        self.bias = tensors.get("bias")
        self.shared_gate = tensors.get("shared_gate")
        self.weigh = params.get("weigh") or "output"
        if self.weigh not in ("output", "input"):
            raise ValueError("an expert's weight multiplies its output or its input")
        if self.weigh == "input" and self.identity:
            raise ValueError("experts that hand back their input take their weight on the output")
        E = self.E
        self.gated = self._form(params) == "gated_silu"
        names = ("gate", "up", "down") if self.gated else ("up", "down")
        kinds = {tensors[f"{n}{e}"].dtype for n in names for e in range(E)}
        if len(kinds) != 1:
            raise ValueError("the experts' projections must be stored in one type")
        # one tensor for all experts: [E, 2I, H] (an expert's gate rows, then its up rows; without a gate [E, I, H]) and
        # [E, H, I]
        self.up = torch.stack([torch.cat([tensors[f"{n}{e}"] for n in names[:-1]], dim=0) for e in range(E)]).contiguous()
        self.down = torch.stack([tensors[f"down{e}"] for e in range(E)]).contiguous()
        self.shared = (children or {}).get("shared")
        if self.shared_gate is not None and self.shared is None:
            raise ValueError("a shared expert's gate without a shared expert")

    def forward(self, x):
        """x [T, H] -> the addends of the output: [(outputs float32 [T, top, H], weights float32 [T, top] or None)] and, with
        a shared expert, its output (float32 [T, H] or a float32 stack of partial sums; with a gate, `ops.Scaled`)."""
        w_dtype = self.up.dtype
        xe = x if x.dtype == w_dtype else x.to(w_dtype)
        ids, weights, *gate = ops.moe_route(x, self.router, self.correction, top=self.top, scale=self.scale,
                                            score=self.score, groups=self.groups, keep_groups=self.keep_groups,
                                            normalize=self.normalize, bias=self.bias, shared_gate=self.shared_gate)
        on_input = self.weigh == "input"
        act = ops.moe_expert(xe, self.up, ids, ops.MOE_GATE_UP if self.gated else ops.MOE_UP, weights if on_input else None)
        outs = ops.moe_expert(act, self.down, ids, ops.MOE_DOWN)
        if self.identity:
            ops.moe_identity(x, ids, outs, self.E)
        terms = [(outs.view(x.shape[0], self.top, -1), None if on_input else weights)]
        if self.shared is not None:
            y = self.shared.forward(x)
            terms.append(ops.Scaled(y, gate[0]) if gate else y)
        return terms
