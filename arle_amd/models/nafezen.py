"""Recipe of the Nafezen decoder: its configuration written out as a ModelSpec.

Every layer is a `parallel` block with one norm: `group_rmsnorm` of the residual, read by the mixer and the feed-forward,
whose outputs are added together.  Mixers: `latent_attention` with a latent for the queries too (`q_rank`) and a
rotate-half rotation of the rotated part, over all earlier positions; `retention`.  Feed-forwards: `swiglu`, or
`sigmoid_moe` with squared-relu experts, a router with a bias whose weights are the softmax over the chosen logits, and a
shared expert behind a sigmoid gate.  The embedding passes a norm of the same kind; the head is the embedding table.
Tensor names: `embed`, `embed.norm`, `l<i>.norm1`, `l<i>.mix.*`, `l<i>.mlp.*`, `final.norm`.
"""
from __future__ import annotations

from ..config.nafezen import ARCHITECTURE, DenseConfig, LatentConfig, MoEConfig, NafezenConfig, RetentionConfig
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

# the rotation's table is made for the longest request the engine is built for, not for a number of the model's
MAX_POSITIONS = 1 << 30


def _rotation(head_dim: int, rot) -> PartSpec | None:
    if rot is None:
        return None
    return PartSpec("rope_neox", {"head_dim": head_dim, "rotary_dim": rot.dims, "theta": rot.base, "max_positions": 1})


def _latent(c: NafezenConfig, m: LatentConfig, p: str) -> PartSpec:
    params = {"hidden_size": c.width, "heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "value_dim": m.vdim,
              "rank": m.kv_rank, "q_rank": m.q_rank, "eps": c.eps, "scale": m.scale, "window": None, "sink": False,
              "gate": False, "position": _rotation(m.rot_dim, m.rot)}
    return PartSpec("latent_attention", params,
                    {"dq": p + "dq", "q_norm": p + "dq.norm", "uq": p + "uq", "dkv": p + "dkv", "c_norm": p + "dkv.norm",
                     "uk": p + "uk", "uv": p + "uv", "o": p + "o"})


def _retention(c: NafezenConfig, m: RetentionConfig, p: str) -> PartSpec:
    params = {"hidden_size": c.width, "heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "decay": m.decay,
              "eps": c.eps, "position": _rotation(m.dim, m.rot)}
    return PartSpec("retention", params, {n: p + n for n in ("q", "k", "v", "g", "o")})


def _feed_forward(c: NafezenConfig, m, p: str) -> PartSpec:
    if isinstance(m, DenseConfig):
        return PartSpec("swiglu", {"hidden_size": c.width, "intermediate_size": m.ff, "float32_out": True},
                        {"gate": p + "gate", "up": p + "up", "down": p + "down"})
    assert isinstance(m, MoEConfig)
    params = {"hidden_size": c.width, "experts": m.experts, "top": m.top, "expert_size": m.expert_ff,
              "form": "squared_relu", "score": "softmax_chosen", "bias": True, "correction": False,
              "shared_size": m.shared_ff, "shared_gate": m.shared_ff is not None,
              "shared_weights": {"up": p + "shared.up", "down": p + "shared.down"}}
    weights = {"router": p + "router", "bias": p + "router.b", "shared_gate": p + "shared.sg"}
    for e in range(m.experts):
        weights.update({f"up{e}": f"{p}e{e}.up", f"down{e}": f"{p}e{e}.down"})
    return PartSpec("sigmoid_moe", params, weights)


_MIXERS = {LatentConfig: _latent, RetentionConfig: _retention}


def nafezen_spec(config: NafezenConfig, stop_token_ids=()) -> ModelSpec:
    c = config
    norm = lambda tensor: PartSpec("group_rmsnorm", {"width": c.width, "groups": c.groups, "eps": c.eps}, {"weight": tensor})
    layers = []
    for i, layer in enumerate(c.layers):
        p = f"l{i}."
        ffn = _feed_forward(c, layer.mlp, p + "mlp.") if layer.mlp is not None else None
        layers.append(LayerSpec("parallel", _MIXERS[type(layer.mixer)](c, layer.mixer, p + "mix."), ffn,
                                {"mixer_in": norm(p + "norm1")}))
    sizes = {"vocab_size": c.vocab, "hidden_size": c.width}
    return ModelSpec(hidden_size=c.width, vocab_size=c.vocab, max_positions=MAX_POSITIONS,
                     embedding=PartSpec("token_table", dict(sizes, norm=norm("embed.norm")), {"table": "embed"}),
                     layers=layers, schedule=[ScheduleEntry(i) for i in range(len(layers))],
                     final_norm=norm("final.norm"), head=PartSpec("linear", sizes, {"weight": "embed"}),
                     stop_token_ids=tuple(stop_token_ids))


register_architecture(ARCHITECTURE, NafezenConfig, nafezen_spec)
