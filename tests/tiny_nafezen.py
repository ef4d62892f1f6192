"""Tiny Nafezen configurations for tests, and helpers that make model folders from them.

P: both mixers and both feed-forwards: norms in three groups, key and value sizes that differ everywhere, a rotation of
   fewer entries than a retention's key has, three decays, six experts of which two are chosen beside a shared one, a
   layer without feed-forward.
Q: what models often make equal differs and what is often large is 1: one head, one expert chosen, no shared expert, a
   retention without rotation, groups of six entries, sizes that are no multiples of 4 or 8, a latent whose rotated part
   turns only in its first entries.
R: sizes the matrix cores take (retention heads of 64 over values of 128, a latent of 64 + 32), one group, every expert
   chosen, a head that never forgets beside one that forgets at once, pages of 16.
S: groups of four entries, a retention with key size 128 over values of 36, nine experts of which three are chosen, a
   latent whose keys and values are wider than the queries' latent, pages of 16.
"""
from __future__ import annotations

import os

import torch
from safetensors.torch import load_file, save_file

from arle_amd.config import NafezenConfig
from arle_amd.weights import write_random_model

ARCH = "Nafezen"


def rot(base, dims):
    return {"base": base, "dims": dims}


def latent(heads, dim, rot_dim, vdim, rank, q_rank, scale=0.3, rot=None):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": scale,
            "rot": rot}


def retention(heads, dim, vdim, decay, rot=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}
    if rot is not None:
        m["rot"] = rot
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


TINY_P = {"architecture": ARCH, "vocab": 211, "width": 72, "norm": {"eps": 2e-5, "groups": 3},
          "layers": [layer("retention", retention(3, 16, 24, (0.5, 0.9, 0.99), rot(10000.0, 12)), moe(6, 2, 40, shared=56)),
                     layer("latent_attention", latent(4, 16, 8, 12, 24, 20, scale=0.35, rot=rot(500.0, 8)), dense(96)),
                     layer("retention", retention(2, 24, 12, (0.97, 0.75), rot(100.0, 24)), None),
                     layer("latent_attention", latent(3, 8, 16, 20, 36, 28, scale=0.25, rot=rot(20000.0, 16)),
                           moe(5, 3, 24, shared=24))]}

TINY_Q = {"architecture": ARCH, "vocab": 97, "width": 42, "norm": {"eps": 1e-6, "groups": 7},
          "layers": [layer("latent_attention", latent(1, 10, 6, 14, 18, 9, scale=0.4, rot=rot(50.0, 4)), moe(4, 1, 30)),
                     layer("retention", retention(1, 10, 6, (0.9375,)), None),
                     layer("retention", retention(5, 6, 10, (0.6, 0.7, 0.8, 0.9, 0.95), rot(20.0, 6)), dense(50)),
                     layer("latent_attention", latent(5, 6, 2, 6, 10, 30, scale=0.5, rot=rot(30.0, 2)), moe(3, 2, 18, shared=10))]}

TINY_R = {"architecture": ARCH, "vocab": 300, "width": 96, "norm": {"eps": 1e-5, "groups": 1},
          "layers": [layer("latent_attention", latent(4, 32, 32, 48, 64, 48, scale=0.12, rot=rot(250000.0, 32)),
                           moe(7, 7, 48, shared=64)),
                     layer("retention", retention(2, 64, 128, (1.0, 0.0), rot(250000.0, 32)), dense(128)),
                     layer("retention", retention(4, 32, 64, (0.98, 0.998, 0.9, 0.6), rot(1000.0, 32)), moe(3, 3, 40, shared=32))]}

TINY_S = {"architecture": ARCH, "vocab": 150, "width": 80, "norm": {"eps": 1e-5, "groups": 20},
          "layers": [layer("retention", retention(2, 128, 36, (0.99, 0.8), rot(800.0, 64)), moe(9, 3, 40, shared=72)),
                     layer("latent_attention", latent(2, 24, 16, 40, 40, 16, scale=0.2, rot=rot(10000.0, 16)), dense(70)),
                     layer("retention", retention(1, 40, 20, (0.95,), rot(800.0, 8)), moe(2, 2, 40, shared=8))]}

# name -> (config, page size, weight std, norm std, seed)
TINY = {"P": (TINY_P, 4, 0.2, 0.2, 5), "Q": (TINY_Q, 8, 0.25, 0.3, 6), "R": (TINY_R, 16, 0.12, 0.2, 7),
        "S": (TINY_S, 16, 0.12, 0.2, 9)}


def make_model_dir(tmp_path, name: str) -> str:
    raw, _, std, norm_std, seed = TINY[name]
    d = os.path.join(str(tmp_path), f"nafezen_{name}")
    write_random_model(d, ARCH, NafezenConfig.from_dict(raw), seed=seed, std=std, norm_std=norm_std)
    # large enough that leaving one out or misplacing one shows: router biases that change who is chosen, shared gates
    # away from a half, latents' norm weights that differ by halves
    path = os.path.join(d, "model.safetensors")
    tensors = load_file(path)
    g = torch.Generator().manual_seed(seed)
    for key, t in tensors.items():
        if key.endswith(".router.b"):
            tensors[key] = torch.randn(t.shape, generator=g).to(t.dtype)
        elif key.endswith(".shared.sg"):
            tensors[key] = (t.float() * 2.0).to(t.dtype)
        elif key.endswith((".dq.norm", ".dkv.norm")):
            tensors[key] = (1.0 + 0.5 * torch.randn(t.shape, generator=g)).to(t.dtype)
    save_file(tensors, path)
    return d
