"""Recipe of the Pozirax decoder: its configuration written out as a ModelSpec.

Every layer is a `parallel` block with one norm (`group_rmsnorm` of one group) of the residual, read by the mixer and the
feed-forward, whose outputs are added together.  Mixers: `mixer_sum` of a `rotary_attention` (normed, then rotated in
neighbouring pairs, a window, a sink of score 0) and a `state_space`; or `gated_linear`.  The feed-forward is a `sigmoid_moe`
whose weights are the chosen sigmoids themselves and multiply the experts' inputs.  With a loop the schedule names its
layers once a pass, behind a `loop_entry` (which also runs in front of all layers, to keep the embedding): the passes share weights and each has its own cache and state.  Tensor names:
`embed`, `loop.in`, `loop.step`, `l<i>.norm1`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`, `head`.
"""
from __future__ import annotations

from ..config.pozirax import ARCHITECTURE, AttentionConfig, GatedLinearConfig, MoEConfig, PairConfig, PoziraxConfig, StateSpaceConfig
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

# the rotation's table is made for the longest request the engine is built for, not for a number of the model's
MAX_POSITIONS = 1 << 30


def _attention(c: PoziraxConfig, m: AttentionConfig, p: str) -> PartSpec:
    position = None
    if m.rot is not None:
        position = PartSpec("rope_interleaved", {"head_dim": m.dim, "rotary_dim": m.rot.dims, "theta": m.rot.base,
                                                 "max_positions": 1})
    params = {"hidden_size": c.width, "num_q_heads": m.heads, "num_kv_heads": m.kv_heads, "key_dim": m.dim,
              "value_dim": m.vdim, "eps": c.eps, "scale": m.scale, "softcap": 0.0, "qk_norm": "weighted_before",
              "sink": "zero", "position": position, "window": m.window, "project_out": False}
    return PartSpec("rotary_attention", params, {"q": p + "q", "k": p + "k", "v": p + "v", "q_norm": p + "q.norm",
                                                 "k_norm": p + "k.norm"})


def _state_space(c: PoziraxConfig, m: StateSpaceConfig, p: str) -> PartSpec:
    params = {"hidden_size": c.width, "heads": m.heads, "value_dim": m.vdim, "state": m.state, "groups": m.groups,
              "conv_taps": m.conv, "norm_groups": m.norm_groups, "eps": c.eps, "project_out": False}
    return PartSpec("state_space", params, {"in": p + "in", "conv": p + "conv", "conv_bias": p + "conv.b",
                                            "dt_bias": p + "dt_bias", "A_log": p + "A_log", "D": p + "D", "norm": p + "norm"})


def _pair(c: PoziraxConfig, m: PairConfig, p: str) -> PartSpec:
    return PartSpec("mixer_sum", {"width": c.width, "left": _attention(c, m.left, p + "left."),
                                  "right": _state_space(c, m.right, p + "right."), "left_scale": m.left_scale,
                                  "right_scale": m.right_scale},
                    {"left_o": p + "left.o", "right_o": p + "right.o"})


def _gated_linear(c: PoziraxConfig, m: GatedLinearConfig, p: str) -> PartSpec:
    params = {"hidden_size": c.width, "heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "tau": m.tau, "eps": c.eps,
              "decay_rank": m.decay_rank}
    weights = {n: p + n for n in ("q", "k", "v", "g", "a1", "a2", "norm", "o")}
    return PartSpec("gated_linear", params, dict(weights, a2_bias=p + "a2.b"))


def _feed_forward(c: PoziraxConfig, m: MoEConfig, p: str) -> PartSpec:
    params = {"hidden_size": c.width, "experts": m.experts, "top": m.top, "expert_size": m.expert_ff, "score": "sigmoid",
              "normalize": False, "weigh": "input", "correction": False, "shared_size": m.shared_ff,
              "shared_weights": {n: f"{p}shared.{n}" for n in ("gate", "up", "down")}}
    weights = {"router": p + "router"}
    for e in range(m.experts):
        weights.update({f"{n}{e}": f"{p}e{e}.{n}" for n in ("gate", "up", "down")})
    return PartSpec("sigmoid_moe", params, weights)


_MIXERS = {PairConfig: _pair, GatedLinearConfig: _gated_linear}


def pozirax_spec(config: PoziraxConfig, stop_token_ids=()) -> ModelSpec:
    c = config
    norm = lambda tensor: PartSpec("group_rmsnorm", {"width": c.width, "groups": 1, "eps": c.eps}, {"weight": tensor})
    layers = []
    for i, layer in enumerate(c.layers):
        p = f"l{i}."
        ffn = _feed_forward(c, layer.mlp, p + "mlp.") if layer.mlp is not None else None
        layers.append(LayerSpec("parallel", _MIXERS[type(layer.mixer)](c, layer.mixer, p + "mix."), ffn,
                                {"mixer_in": norm(p + "norm1")}))
    order = list(range(len(layers)))
    if c.loop is not None:
        start, stop, times = c.loop
        join = PartSpec("joined_input", {"width": c.width, "times": times}, {"in": "loop.in", "step": "loop.step"})
        entry = len(layers)
        layers.append(LayerSpec("loop_entry", parts={"join": ("feed_forward", join)}))
        order = [entry] + order[:start] + ([entry] + order[start:stop]) * times + order[stop:]
    sizes = {"vocab_size": c.vocab, "hidden_size": c.width}
    return ModelSpec(hidden_size=c.width, vocab_size=c.vocab, max_positions=MAX_POSITIONS,
                     embedding=PartSpec("token_table", dict(sizes, scale=c.embedding_scale), {"table": "embed"}),
                     layers=layers, schedule=[ScheduleEntry(i) for i in order],
                     final_norm=norm("final.norm"),
                     head=PartSpec("linear", dict(sizes, softcap=c.logit_softcap), {"weight": "head"}),
                     stop_token_ids=tuple(stop_token_ids))


register_architecture(ARCHITECTURE, PoziraxConfig, pozirax_spec)
