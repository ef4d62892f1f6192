"""Typed configuration of the Pozirax decoder: a list of parallel layers (one RMS norm whose output the mixer and the
feed-forward both read), each with a mixer (a windowed rotary attention beside a state-space layer, or gated linear
attention) and an optional mixture of experts; a run of layers may be repeated with the same weights, every pass
beginning with a projection of the residual beside the embedding's output.

config.json names the design under `architecture` (one string).  Every size and every constant that can differ
between two models of the design is read here and nowhere else: `vocab`, `width`, `embedding.scale`, `norm.eps`,
`logit_softcap`, `loop` (`start`, `stop`, `times`), and per layer `type`, `mixer.*` (a pair's `left`, `right`,
`left_scale`, `right_scale`) and `mlp` (null, or `kind` with `expert.ff`, `router.experts|top` and `shared.ff`).
"""
from __future__ import annotations

import math
from dataclasses import dataclass

from .base import ConfigError, Key, read_section, require_positive

ARCHITECTURE = "Pozirax"

_TOP = (Key("vocab", int), Key("width", int), Key("norm", dict), Key("layers", list), Key("embedding", dict, default=None),
        Key("logit_softcap", float, default=0.0), Key("loop", dict, default=None))
_PAIR = (Key("left", dict), Key("right", dict), Key("left_scale", float, default=1.0), Key("right_scale", float, default=1.0))
_ATTENTION = (Key("heads", int), Key("kv_heads", int, default=None), Key("dim", int), Key("vdim", int),
              Key("scale", float), Key("mask", dict, default=None), Key("rot", dict, default=None))
_ROT = (Key("base", float), Key("dims", int))
_STATE_SPACE = (Key("heads", int), Key("vdim", int), Key("state", int), Key("groups", int, default=1), Key("conv", int),
                Key("norm_groups", int, default=1))
_GLA = (Key("heads", int), Key("dim", int), Key("vdim", int), Key("tau", float),
        Key("decay_rank", int, default=None))
_MLP = (Key("kind", str), Key("expert", dict), Key("router", dict), Key("shared", dict, default=None))
_ROUTER = (Key("experts", int), Key("top", int))
_FF = (Key("ff", int),)
_LOOP = (Key("start", int), Key("stop", int), Key("times", int))

LAYER_TYPES = ("parallel", "gla")
MLP_KINDS = ("moe",)


@dataclass(frozen=True)
class RotaryConfig:
    base: float
    dims: int

    def to_dict(self) -> dict:
        return {"base": self.base, "dims": self.dims}


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int | None         # a token sees itself and the window - 1 tokens before it; None: all of them
    rot: RotaryConfig | None

    def to_dict(self) -> dict:
        body = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window is not None:
            body["mask"] = {"size": self.window}
        if self.rot is not None:
            body["rot"] = self.rot.to_dict()
        return body


@dataclass(frozen=True)
class StateSpaceConfig:
    heads: int
    vdim: int                  # values a head
    state: int                 # rows of a head's state
    groups: int                # groups of heads that share what enters and reads the state
    conv: int                  # taps of the short convolution
    norm_groups: int           # equal parts of the output that are normed each by itself

    def to_dict(self) -> dict:
        return {"heads": self.heads, "vdim": self.vdim, "state": self.state, "groups": self.groups, "conv": self.conv,
                "norm_groups": self.norm_groups}


@dataclass(frozen=True)
class PairConfig:
    left: AttentionConfig
    right: StateSpaceConfig
    left_scale: float
    right_scale: float

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


@dataclass(frozen=True)
class GatedLinearConfig:
    heads: int
    dim: int
    vdim: int
    tau: float                 # the decays are sigmoids to the power 1 / tau
    # width of the decay's narrow middle where weights are made from nothing; None: whatever the checkpoint's tensors have
    decay_rank: int | None = None

    def to_dict(self) -> dict:
        body = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}
        if self.decay_rank is not None:
            body["decay_rank"] = self.decay_rank
        return body


@dataclass(frozen=True)
class MoEConfig:
    experts: int
    top: int
    expert_ff: int
    shared_ff: int | None      # hidden size of the shared expert; None: there is none

    def to_dict(self) -> dict:
        body = {"kind": "moe", "expert": {"ff": self.expert_ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            body["shared"] = {"ff": self.shared_ff}
        return body


@dataclass(frozen=True)
class PoziraxLayer:
    type: str                  # one of LAYER_TYPES
    mixer: object
    mlp: MoEConfig | None

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


def _finite(where: str, **values) -> None:
    for name, v in values.items():
        if not math.isfinite(v):
            raise ConfigError(f"{where}: `{name}` must be a finite number")


def _read_attention(raw, where: str) -> AttentionConfig:
    a = read_section(raw, _ATTENTION, where)
    kv = a["kv_heads"] if a["kv_heads"] is not None else a["heads"]
    require_positive(where, heads=a["heads"], kv_heads=kv, dim=a["dim"], vdim=a["vdim"])
    if a["heads"] % kv:
        raise ConfigError(f"{where}: heads must be divisible by kv_heads")
    _finite(where, scale=a["scale"])
    window = None
    if a["mask"] is not None:
        window = read_section(a["mask"], (Key("size", int),), where + ".mask")["size"]
        require_positive(where + ".mask", size=window)
    rot = None
    if a["rot"] is not None:
        r = read_section(a["rot"], _ROT, where + ".rot")
        require_positive(where + ".rot", dims=r["dims"])
        if r["dims"] % 2 or r["dims"] > a["dim"]:
            raise ConfigError(f"{where}.rot: `dims` must be even and at most the head's `dim`")
        if not r["base"] > 0:
            raise ConfigError(f"{where}.rot: `base` must be positive")
        rot = RotaryConfig(r["base"], r["dims"])
    return AttentionConfig(a["heads"], kv, a["dim"], a["vdim"], a["scale"], window, rot)


def _read_state_space(raw, where: str) -> StateSpaceConfig:
    a = read_section(raw, _STATE_SPACE, where)
    require_positive(where, **a)
    if a["heads"] % a["groups"]:
        raise ConfigError(f"{where}: heads must be divisible by `groups`")
    if a["heads"] * a["vdim"] % a["norm_groups"]:
        raise ConfigError(f"{where}: `norm_groups` must divide heads times vdim")
    return StateSpaceConfig(a["heads"], a["vdim"], a["state"], a["groups"], a["conv"], a["norm_groups"])


def _read_pair(raw, where: str) -> PairConfig:
    p = read_section(raw, _PAIR, where)
    _finite(where, left_scale=p["left_scale"], right_scale=p["right_scale"])
    return PairConfig(_read_attention(p["left"], where + ".left"), _read_state_space(p["right"], where + ".right"),
                      p["left_scale"], p["right_scale"])


def _read_gla(raw, where: str) -> GatedLinearConfig:
    a = read_section(raw, _GLA, where)
    require_positive(where, heads=a["heads"], dim=a["dim"], vdim=a["vdim"])
    if a["decay_rank"] is not None:
        require_positive(where, decay_rank=a["decay_rank"])
    if not (a["tau"] > 0 and math.isfinite(a["tau"])):
        raise ConfigError(f"{where}: `tau` must be positive")
    return GatedLinearConfig(a["heads"], a["dim"], a["vdim"], a["tau"], a["decay_rank"])


def _read_mlp(raw, where: str) -> MoEConfig | None:
    if raw is None:
        return None
    if isinstance(raw, dict) and isinstance(raw.get("kind"), str) and raw["kind"] not in MLP_KINDS:
        raise ConfigError(f"{where}: unknown kind {raw['kind']!r} (known: {', '.join(MLP_KINDS)})")
    m = read_section(raw, _MLP, where)
    ff = read_section(m["expert"], _FF, where + ".expert")["ff"]
    r = read_section(m["router"], _ROUTER, where + ".router")
    require_positive(where, ff=ff, experts=r["experts"], top=r["top"])
    if r["top"] > r["experts"]:
        raise ConfigError(f"{where}.router: `top` = {r['top']} is more than the {r['experts']} experts a token can choose among")
    shared = None
    if m["shared"] is not None:
        shared = read_section(m["shared"], _FF, where + ".shared")["ff"]
        require_positive(where + ".shared", ff=shared)
    return MoEConfig(r["experts"], r["top"], ff, shared)


_READERS = {"parallel": _read_pair, "gla": _read_gla}


def _read_layer(i: int, raw) -> PoziraxLayer:
    where = f"layers[{i}]"
    if not isinstance(raw, dict) or not isinstance(raw.get("mixer"), dict) or not isinstance(raw.get("type"), str):
        raise ConfigError(f"{where}: a layer is an object with `type`, `mixer` and `mlp`")
    kind = raw["type"]
    if kind not in _READERS:
        raise ConfigError(f"{where}: unknown layer type {kind!r} (known: {', '.join(LAYER_TYPES)})")
    return PoziraxLayer(kind, _READERS[kind](raw["mixer"], where + ".mixer"), _read_mlp(raw.get("mlp"), where + ".mlp"))


@dataclass(frozen=True)
class PoziraxConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    logit_softcap: float       # 0: logits are not capped
    loop: tuple | None         # (start, stop, times): layers start..stop-1 run `times` times in a row
    layers: tuple

    architecture = ARCHITECTURE
    eos_token_id = None

    @classmethod
    def from_dict(cls, raw: dict) -> "PoziraxConfig":
        top = read_section(raw, _TOP, "config.json")
        eps = read_section(top["norm"], (Key("eps", float),), "norm")["eps"]
        scale = 1.0
        if top["embedding"] is not None:
            scale = read_section(top["embedding"], (Key("scale", float, default=1.0),), "embedding")["scale"]
        if len(top["layers"]) > 65535:
            raise ConfigError(f"{len(top['layers'])} layers: more than 65,535 are not taken")
        loop = None
        if top["loop"] is not None:
            lp = read_section(top["loop"], _LOOP, "loop")
            loop = (lp["start"], lp["stop"], lp["times"])
        config = cls(top["vocab"], top["width"], eps, scale, top["logit_softcap"], loop,
                     tuple(_read_layer(i, layer) for i, layer in enumerate(top["layers"])))
        config.validate()
        return config

    def validate(self) -> None:
        require_positive("config.json", vocab=self.vocab, width=self.width)
        if not self.eps >= 0.0:
            raise ConfigError("norm.eps must not be negative")
        _finite("embedding", scale=self.embedding_scale)
        if not self.logit_softcap >= 0.0:
            raise ConfigError("`logit_softcap` must not be negative")
        if not self.layers:
            raise ConfigError("`layers` must name at least one layer")
        if self.loop is not None:
            start, stop, times = self.loop
            if not 0 <= start < stop <= len(self.layers):
                raise ConfigError("loop: `start` and `stop` must lie within the layers, start < stop")
            if times < 1 or times * (stop - start) > 65535:
                raise ConfigError("loop: `times` must be at least 1, and the passes at most 65,535 layer runs")

    def to_dict(self) -> dict:
        """A config.json body that `from_dict` reads back to an equal object."""
        body = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
                "embedding": {"scale": self.embedding_scale}, "logit_softcap": self.logit_softcap,
                "layers": [layer.to_dict() for layer in self.layers]}
        if self.loop is not None:
            body["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return body
