"""Tiny Pozirax configurations for tests, and helpers that make model folders from them.

P: both mixers: groups of query heads and of state-space heads, key and value sizes that differ everywhere, a rotation of
   fewer entries than a key has, norm groups that cross heads, six experts of which two are chosen beside a shared one, a
   layer without feed-forward; the middle layers run twice.
Q: what models often make equal differs and what is often large is 1: one head, one tap, a window of one token, one expert
   chosen, no shared expert, no rotation, sizes that are no multiples of 4 or 8, factors below 0 and above 1, decays that
   forget within a few tokens; the loop is one layer, three times.
R: sizes the matrix cores take, one kv head, every expert chosen, pages of 16; all layers run twice.
S: state sizes that are multiples of 8 but of nothing more, heads of 40 values, nine experts of which three are chosen, pages
   of 16; no loop.
T: wide heads: a state of 136 rows, 72 values a head, keys of 132 over 136 values in the gated linear attention; the last
   layer runs once in a loop of one pass.
"""
from __future__ import annotations

import copy
import os

import torch
from safetensors.torch import load_file, save_file

from arle_amd.config import PoziraxConfig
from arle_amd.weights import write_random_model

ARCH = "Pozirax"


def rot(base, dims):
    return {"base": base, "dims": dims}


def attention(heads, kv_heads, dim, vdim, window, scale=0.3, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window}}
    if rot is not None:
        m["rot"] = rot
    return m


def state_space(heads, vdim, state, groups, conv=4, norm_groups=1):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def pair(left, right, left_scale=0.7, right_scale=0.6):
    return {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def gla(heads, dim, vdim, tau=16.0, rank=16):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}


def moe(experts, top, ff, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def loop(start, stop, times):
    return {"start": start, "stop": stop, "times": times}


def model(vocab, width, eps, layers, loop=None, scale=0.7, cap=20.0):
    raw = {"architecture": ARCH, "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "logit_softcap": cap, "layers": layers}
    if loop is not None:
        raw["loop"] = loop
    return raw


TINY_P = model(211, 72, 2e-5, [
    layer("parallel", pair(attention(4, 2, 16, 12, 9, 0.35, rot(500.0, 12)), state_space(6, 8, 12, 3, 4, 2), 0.8, 0.5), moe(6, 2, 40, 56)),
    layer("gla", gla(3, 16, 24, 4.0, 5), moe(5, 3, 24, 24)),
    layer("parallel", pair(attention(2, 2, 24, 20, 30, 0.25, rot(20000.0, 24)), state_space(4, 12, 16, 1, 3, 6), 0.4, 0.9), None),
    layer("gla", gla(2, 24, 12, 8.0, 7), moe(4, 2, 32, 48))], loop(1, 3, 2))

TINY_Q = model(97, 42, 1e-6, [
    layer("gla", gla(1, 10, 6, 0.25, 3), moe(4, 1, 30)),
    layer("parallel", pair(attention(1, 1, 10, 14, 1, 0.4), state_space(1, 6, 10, 1, 1, 1), -0.6, 1.3), moe(3, 2, 18)),
    layer("parallel", pair(attention(5, 1, 6, 10, 7, 0.5, rot(20.0, 4)), state_space(5, 10, 6, 5, 2, 10), 1.2, -0.7), None)],
    loop(1, 2, 3), scale=1.5, cap=7.0)

TINY_R = model(300, 96, 1e-5, [
    layer("parallel", pair(attention(4, 1, 32, 48, 40, 0.18, rot(250000.0, 32)), state_space(4, 32, 64, 2, 3, 4)), moe(7, 7, 48, 64)),
    layer("gla", gla(2, 64, 128, 16.0, 16), moe(3, 3, 40, 32)),
    layer("parallel", pair(attention(6, 2, 48, 32, 65, 0.15, rot(1000.0, 16)), state_space(2, 64, 32, 1, 4, 1)), moe(2, 2, 64, 72))],
    loop(0, 3, 2))

TINY_S = model(150, 80, 1e-5, [
    layer("gla", gla(2, 36, 20, 2.0, 20), moe(9, 3, 40, 72)),
    layer("parallel", pair(attention(2, 1, 40, 16, 17, 0.2, rot(10000.0, 40)), state_space(2, 40, 24, 1, 4, 5)), moe(4, 2, 40, 8)),
    layer("parallel", pair(attention(3, 3, 16, 32, 16, 0.3, rot(100.0, 8)), state_space(3, 16, 72, 3, 5, 1)), None)])

TINY_T = model(130, 64, 1e-5, [
    layer("parallel", pair(attention(1, 1, 64, 64, 33, 0.15, rot(10000.0, 64)), state_space(2, 72, 136, 2, 4, 2)), moe(3, 3, 32, 32)),
    layer("gla", gla(1, 132, 136, 16.0, 16), moe(2, 2, 40, 24))], loop(1, 2, 1))

# name -> (config, page size, weight std, norm std, seed)
TINY = {"P": (TINY_P, 4, 0.2, 0.2, 5), "Q": (TINY_Q, 8, 0.25, 0.3, 6), "R": (TINY_R, 16, 0.12, 0.2, 7),
        "S": (TINY_S, 16, 0.12, 0.2, 9), "T": (TINY_T, 16, 0.12, 0.2, 11)}


def spread(key: str, t: torch.Tensor, g: torch.Generator) -> torch.Tensor:
    """Tensors whose usual random values would hide a mistake: decays from fast to slow, step sizes about one, biases and skips
    that count, rows for the passes as large as the residual."""
    r = torch.randn(t.shape, generator=g)
    if key.endswith(".A_log"):
        return torch.log(torch.rand(t.shape, generator=g) * 2.0 + 0.02)
    if key.endswith((".dt_bias", ".conv.b")):
        return 0.7 * r - 0.3
    if key.endswith(".D"):
        return r
    if key.endswith(".a2.b"):
        return 1.5 * r + 1.0
    if key.endswith((".q.norm", ".k.norm")):
        return 1.0 + 0.5 * r
    if key.endswith((".conv", "loop.step")):
        return 0.6 * r
    return t


def make_model_dir(tmp_path, name: str, every_expert: bool = False) -> str:
    """every_expert: the same model with routers that choose all of their experts."""
    raw, _, std, norm_std, seed = TINY[name]
    d = os.path.join(str(tmp_path), f"pozirax_{name}{'_all' if every_expert else ''}")
    if every_expert:
        raw = copy.deepcopy(raw)
        for lay in raw["layers"]:
            if lay["mlp"]:
                lay["mlp"]["router"]["top"] = lay["mlp"]["router"]["experts"]
    write_random_model(d, ARCH, PoziraxConfig.from_dict(raw), seed=seed, std=std, norm_std=norm_std)
    path = os.path.join(d, "model.safetensors")
    tensors = load_file(path)
    g = torch.Generator().manual_seed(seed)
    save_file({k: spread(k, t, g).to(t.dtype).contiguous() for k, t in sorted(tensors.items())}, path)
    return d
