"""A plain, slow implementation of the Nafezen decoder in float64 on the CPU: one function a mechanism, whole
sequences at once, no cache, no kernels.  It shares no code with the engine; the tests compare the two.

`config` is the config.json body as a dictionary, `tensors` a dictionary name -> torch tensor (any float type).
"""
from __future__ import annotations

import torch

F = torch.float64

# a test may set this to a function of a matrix product's result (to move every entry by a rounding, say)
after_product = None


def t64(x):
    return x.to(F)


def mm(x, w):
    """x [.., K] times w [N, K] transposed: every projection goes through here."""
    y = x @ w.T
    return after_product(y) if after_product is not None else y


def silu(z):
    return z * torch.sigmoid(z)


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, weight, groups, eps):
    """The last axis in `groups` equal consecutive parts, each divided by its own root mean square, times a weight."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return unit_rms(parts, eps).reshape(x.shape) * weight


def rotate_half(x, positions, dims, base):
    """x [T, heads, D]: the first `dims` entries of every head turn, entry i with entry i + dims / 2."""
    if not dims:
        return x
    half = dims // 2
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=F)
    ang = positions.to(F)[:, None] * freq[None, :]            # [T, half]
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def latent_attention(h, m, w, eps):
    """Attention whose queries go through a normed latent of their own, and whose keys and values are linear maps of
    one normed vector a token, with a rotated key part that all heads share.  m: the layer's `mixer` dictionary,
    w(name) -> tensor of the mixer."""
    T = h.shape[0]
    H, D, R, Dv, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = unit_rms(mm(h, w("dq")), eps) * w("dq.norm")
    q = mm(cq, w("uq")).view(T, H, D + R)
    d = mm(h, w("dkv"))
    c = unit_rms(d[:, :C], eps) * w("dkv.norm")
    pos = torch.arange(T)
    rot = m["rot"]
    q_rot = rotate_half(q[..., D:], pos, rot["dims"], rot["base"])
    k_rot = rotate_half(d[:, C:].view(T, 1, R), pos, rot["dims"], rot["base"]).expand(T, H, R)
    k = torch.cat([mm(c, w("uk")).view(T, H, D), k_rot], dim=-1)
    v = mm(c, w("uv")).view(T, H, Dv)
    q = torch.cat([q[..., :D], q_rot], dim=-1)
    out = torch.zeros(T, H, Dv, dtype=F)
    for j in range(H):
        s = q[:, j] @ k[:, j].T * m["scale"]
        s = s.masked_fill(torch.arange(T)[None, :] > torch.arange(T)[:, None], float("-inf"))
        out[:, j] = torch.softmax(s, dim=-1) @ v[:, j]
    return mm(out.reshape(T, H * Dv), w("o"))


def retention(h, m, w, eps):
    """Linear attention with one fixed decay a head; the read-out is divided by its root mean square, head by head."""
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q, k, v = mm(h, w("q")).view(T, H, D), mm(h, w("k")).view(T, H, D), mm(h, w("v")).view(T, H, Dv)
    rot = m.get("rot")
    if rot:
        pos = torch.arange(T)
        q, k = rotate_half(q, pos, rot["dims"], rot["base"]), rotate_half(k, pos, rot["dims"], rot["base"])
    k = k * D ** -0.5
    decay = torch.tensor(m["decay"], dtype=F)
    out = torch.zeros(T, H, Dv, dtype=F)
    S = torch.zeros(H, D, Dv, dtype=F)
    for t in range(T):
        S = S * decay[:, None, None] + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    out = unit_rms(out, eps).reshape(T, H * Dv) * silu(mm(h, w("g")))
    return mm(out, w("o"))


def gated_ff(h, gate, up, down):
    return mm(silu(mm(h, gate)) * mm(h, up), down)


def squared_relu_ff(h, up, down):
    return mm(torch.relu(mm(h, up)) ** 2, down)


# every call of `route` leaves here, a token, how far its choice was from another one: the smallest chosen logit less
# the largest that was not chosen, over the root mean square of the token's logits (infinity where all are chosen)
route_margins: list = []


def route(h, top, router, bias):
    """-> (chosen [T, top] indices, weights [T, top]): the largest logits, and the softmax over just those."""
    z = mm(h, router) + (bias if bias is not None else 0.0)
    ordered = torch.sort(z, dim=-1, descending=True).values
    size = torch.sqrt((z * z).mean(-1))
    route_margins.append((ordered[:, top - 1] - ordered[:, top]) / size if top < z.shape[1]
                         else torch.full((h.shape[0],), float("inf"), dtype=F))
    best = torch.topk(z, top, dim=-1)
    return best.indices, torch.softmax(best.values, dim=-1)


def mixture(h, mlp, w):
    """Experts e0.. of which each token uses a few, and a shared expert behind a sigmoid of one number a token."""
    chosen, weights = route(h, mlp["router"]["top"], w("router"), w("router.b"))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, f in zip(chosen[t].tolist(), weights[t]):
            out[t] = out[t] + f * squared_relu_ff(h[t], w(f"e{e}.up"), w(f"e{e}.down"))
    if mlp.get("shared"):
        out = out + torch.sigmoid(mm(h, w("shared.sg"))) * squared_relu_ff(h, w("shared.up"), w("shared.down"))
    return out


def feed_forward(h, mlp, w):
    if mlp["kind"] == "dense":
        return gated_ff(h, w("gate"), w("up"), w("down"))
    return mixture(h, mlp, w)


MIXERS = {"latent_attention": latent_attention, "retention": retention}


def forward(config, tensors, tokens, return_layers=False):
    """tokens: a list of ids -> float64 logits [T, vocab] (and the residual after every layer)."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps, groups = config["norm"]["eps"], config["norm"]["groups"]
    table = t64(tensors["embed"])
    x = group_norm(table[tokens], t64(tensors["embed.norm"]), groups, eps)
    seen = []
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        w_mix = lambda name, p=p: t64(tensors[p + "mix." + name]) if (p + "mix." + name) in tensors else None
        w_mlp = lambda name, p=p: t64(tensors[p + "mlp." + name]) if (p + "mlp." + name) in tensors else None
        h = group_norm(x, t64(tensors[p + "norm1"]), groups, eps)
        y = MIXERS[layer["type"]](h, layer["mixer"], w_mix, eps)
        if layer.get("mlp") is not None:
            y = y + feed_forward(h, layer["mlp"], w_mlp)
        x = x + y
        seen.append(x)
    logits = mm(group_norm(x, t64(tensors["final.norm"]), groups, eps), table)
    return (logits, torch.stack(seen)) if return_layers else logits
