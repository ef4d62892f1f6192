"""Typed configuration of the Nafezen decoder: a list of parallel layers (one grouped RMS norm whose output the mixer and
the feed-forward both read), each with a mixer (a latent attention whose queries go through a latent of their own, or a
retention with one fixed decay a head) and an optional feed-forward (gated dense, or a mixture of squared-relu experts
with a shared one behind a sigmoid gate); the embedding is normed, and the head is the embedding table.

config.json names the design under `architecture` (one string).  Every size and every constant that can differ
between two models of the design is read here and nowhere else: `vocab`, `width`, `norm.eps`, `norm.groups`, and per layer
`type`, `mixer.*` (with `rot.base`, `rot.dims`, a retention's list `decay`) and `mlp` (null, or `kind` with `ff`, or with
`expert.ff`, `router.experts|top` and `shared.ff`).
"""
from __future__ import annotations

import math
from dataclasses import dataclass

from .base import ConfigError, Key, read_keys

ARCHITECTURE = "Nafezen"

_TOP = (Key("vocab", int), Key("width", int), Key("norm", dict), Key("layers", list))
_NORM = (Key("eps", float), Key("groups", int, default=1))
_ROT = (Key("base", float), Key("dims", int))
_LATENT = (Key("heads", int), Key("dim", int), Key("rot_dim", int), Key("vdim", int), Key("kv_rank", int),
           Key("q_rank", int), Key("scale", float), Key("rot", dict))
_RETENTION = (Key("heads", int), Key("dim", int), Key("vdim", int), Key("decay", list), Key("rot", dict, default=None))
_MLP = (Key("kind", str), Key("ff", int, default=None), Key("expert", dict, default=None),
        Key("router", dict, default=None), Key("shared", dict, default=None))
_ROUTER = (Key("experts", int), Key("top", int))
_FF = (Key("ff", int),)

LAYER_TYPES = ("latent_attention", "retention")
MLP_KINDS = ("dense", "moe")


def _positive(where: str, **values) -> None:
    for name, v in values.items():
        if v <= 0:
            raise ConfigError(f"{where}: `{name}` must be positive")
        if v > 2 ** 31 - 1:
            raise ConfigError(f"{where}: `{name}` = {v} is beyond what a 32-bit index reaches")


def _sub(raw, keys, where: str) -> dict:
    try:
        return read_keys(raw, keys)
    except ConfigError as exc:
        raise ConfigError(f"{where}: {exc}") from None


@dataclass(frozen=True)
class RotaryConfig:
    base: float
    dims: int

    def to_dict(self) -> dict:
        return {"base": self.base, "dims": self.dims}


def _read_rot(raw, most: int, where: str):
    if raw is None:
        return None
    r = _sub(raw, _ROT, where)
    _positive(where, dims=r["dims"])
    if r["dims"] % 2 or r["dims"] > most:
        raise ConfigError(f"{where}: `dims` must be even and at most the size of what is rotated ({most})")
    if not r["base"] > 0:
        raise ConfigError(f"{where}: `base` must be positive")
    return RotaryConfig(r["base"], r["dims"])


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int                   # unrotated query/key entries a head
    rot_dim: int               # rotated ones (the key's are shared by the heads)
    vdim: int
    kv_rank: int               # size of the latent that keys and values are made of
    q_rank: int                # size of the latent that queries are made of
    scale: float
    rot: RotaryConfig

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "kv_rank": self.kv_rank,
                "q_rank": self.q_rank, "scale": self.scale, "rot": self.rot.to_dict()}


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple               # what is kept of a head's state from one token to the next
    rot: RotaryConfig | None

    def to_dict(self) -> dict:
        body = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}
        if self.rot is not None:
            body["rot"] = self.rot.to_dict()
        return body


@dataclass(frozen=True)
class DenseConfig:
    ff: int

    def to_dict(self) -> dict:
        return {"kind": "dense", "ff": self.ff}


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
class NafezenLayer:
    type: str                  # one of LAYER_TYPES
    mixer: object
    mlp: object                # DenseConfig, MoEConfig or None

    def to_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


def _read_latent(raw, where: str) -> LatentConfig:
    a = _sub(raw, _LATENT, where)
    _positive(where, heads=a["heads"], dim=a["dim"], rot_dim=a["rot_dim"], vdim=a["vdim"], kv_rank=a["kv_rank"],
              q_rank=a["q_rank"])
    return LatentConfig(a["heads"], a["dim"], a["rot_dim"], a["vdim"], a["kv_rank"], a["q_rank"], a["scale"],
                        _read_rot(a["rot"], a["rot_dim"], where + ".rot"))


def _read_retention(raw, where: str) -> RetentionConfig:
    a = _sub(raw, _RETENTION, where)
    _positive(where, heads=a["heads"], dim=a["dim"], vdim=a["vdim"])
    if len(a["decay"]) != a["heads"]:
        raise ConfigError(f"{where}: `decay` must list one number for each of the {a['heads']} heads")
    for g in a["decay"]:
        if isinstance(g, bool) or not isinstance(g, (int, float)) or not math.isfinite(g):
            raise ConfigError(f"{where}: `decay` holds {g!r}, which is no number")
    return RetentionConfig(a["heads"], a["dim"], a["vdim"], tuple(float(g) for g in a["decay"]),
                           _read_rot(a["rot"], a["dim"], where + ".rot"))


def _read_mlp(raw, where: str):
    if raw is None:
        return None
    m = _sub(raw, _MLP, where)
    if m["kind"] == "dense":
        if m["ff"] is None:
            raise ConfigError(f"{where}: missing or invalid config field `ff`")
        _positive(where, ff=m["ff"])
        return DenseConfig(m["ff"])
    if m["kind"] != "moe":
        raise ConfigError(f"{where}: unknown kind {m['kind']!r} (known: {', '.join(MLP_KINDS)})")
    if m["expert"] is None or m["router"] is None:
        raise ConfigError(f"{where}: a mixture of experts names `expert` and `router`")
    ff = _sub(m["expert"], _FF, where + ".expert")["ff"]
    r = _sub(m["router"], _ROUTER, where + ".router")
    _positive(where, ff=ff, experts=r["experts"], top=r["top"])
    if r["top"] > r["experts"]:
        raise ConfigError(f"{where}.router: `top` = {r['top']} is more than the {r['experts']} experts a token can choose among")
    shared = None
    if m["shared"] is not None:
        shared = _sub(m["shared"], _FF, where + ".shared")["ff"]
        _positive(where + ".shared", ff=shared)
    return MoEConfig(r["experts"], r["top"], ff, shared)


def _read_layer(i: int, raw) -> NafezenLayer:
    where = f"layers[{i}]"
    if not isinstance(raw, dict) or not isinstance(raw.get("mixer"), dict) or not isinstance(raw.get("type"), str):
        raise ConfigError(f"{where}: a layer is an object with `type`, `mixer` and `mlp`")
    kind = raw["type"]
    readers = {"latent_attention": _read_latent, "retention": _read_retention}
    if kind not in readers:
        raise ConfigError(f"{where}: unknown layer type {kind!r} (known: {', '.join(LAYER_TYPES)})")
    return NafezenLayer(kind, readers[kind](raw["mixer"], where + ".mixer"), _read_mlp(raw.get("mlp"), where + ".mlp"))


@dataclass(frozen=True)
class NafezenConfig:
    vocab: int
    width: int
    eps: float
    groups: int                # equal parts of the width that a norm treats each by itself
    layers: tuple

    architecture = ARCHITECTURE
    eos_token_id = None

    @classmethod
    def from_dict(cls, raw: dict) -> "NafezenConfig":
        top = read_keys(raw, _TOP)
        norm = _sub(top["norm"], _NORM, "norm")
        if len(top["layers"]) > 65535:
            raise ConfigError(f"{len(top['layers'])} layers: more than 65,535 are not taken")
        config = cls(top["vocab"], top["width"], norm["eps"], norm["groups"],
                     tuple(_read_layer(i, layer) for i, layer in enumerate(top["layers"])))
        config.validate()
        return config

    def validate(self) -> None:
        _positive("config.json", vocab=self.vocab, width=self.width)
        _positive("norm", groups=self.groups)
        if not self.eps >= 0.0:
            raise ConfigError("norm.eps must not be negative")
        if self.width % self.groups:
            raise ConfigError(f"norm.groups = {self.groups} must divide the width {self.width} evenly")
        if not self.layers:
            raise ConfigError("`layers` must name at least one layer")

    def to_dict(self) -> dict:
        """A config.json body that `from_dict` reads back to an equal object."""
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width,
                "norm": {"eps": self.eps, "groups": self.groups}, "layers": [layer.to_dict() for layer in self.layers]}
