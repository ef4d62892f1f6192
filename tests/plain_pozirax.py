"""A plain, slow implementation of the Pozirax decoder in float64 on the CPU: one function a mechanism, whole
sequences at once, no cache, no kernels.  It shares no code with the engine; the tests compare the two.

`config` is the config.json body as a dictionary, `tensors` a dictionary name -> torch tensor (any float type).
"""
from __future__ import annotations

import math

import torch

F = torch.float64

# a test may set this to a function (x, w) -> product (one that moves every entry by a rounding, say)
around_product = None


def t64(x):
    return x.to(F)


def mm(x, w):
    """x [.., K] times w [N, K] transposed: every projection goes through here."""
    return around_product(x, w) if around_product is not None else x @ w.T


def silu(z):
    return z * torch.sigmoid(z)


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rotate_pairs(x, positions, dims, base):
    """x [T, heads, D]: of every head's first `dims` entries, entry 2i turns with entry 2i + 1."""
    if not dims:
        return x
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F)
    ang = positions.to(F)[:, None] * freq[None, :]
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    turned = torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1).flatten(-2)
    return torch.cat([turned, x[..., dims:]], dim=-1)


def window_attention_heads(h, m, w, eps):
    """Attention over the last `mask.size` positions with normed, then rotated queries and keys and one more in the
    softmax's denominator -> what the output projection reads, [T, heads * vdim]."""
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads") or H
    q = unit_rms(mm(h, w("q")).view(T, H, D), eps) * w("q.norm")
    k = unit_rms(mm(h, w("k")).view(T, G, D), eps) * w("k.norm")
    v = mm(h, w("v")).view(T, G, Dv)
    rot = m.get("rot")
    if rot:
        pos = torch.arange(T)
        q, k = rotate_pairs(q, pos, rot["dims"], rot["base"]), rotate_pairs(k, pos, rot["dims"], rot["base"])
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if m.get("mask"):
        seen &= i - j < m["mask"]["size"]
    out = torch.zeros(T, H, Dv, dtype=F)
    for n in range(H):
        s = (q[:, n] @ k[:, n // (H // G)].T) * m["scale"]
        s = torch.cat([torch.zeros(T, 1, dtype=F), s.masked_fill(~seen, float("-inf"))], dim=1)   # the sink's score: 0
        out[:, n] = torch.softmax(s, dim=-1)[:, 1:] @ v[:, n // (H // G)]
    return out.reshape(T, H * Dv)


def causal_conv(u, taps, bias):
    """y_t = bias + sum_j taps[:, j] u_(t - K + 1 + j), a channel at a time, zeros before the start."""
    T, K = u.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros(K - 1, u.shape[1], dtype=F), u])
    y = sum(padded[j:j + T] * taps[:, j] for j in range(K))
    return y + bias if bias is not None else y


def state_space_heads(h, m, w, eps):
    """A state-space layer with one decay a head and token: -> what the output projection reads, [T, heads * vdim]."""
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = torch.split(mm(h, w("in")), [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, w("conv"), w("conv.b")))
    x, B, C = xbc[:, :inner].view(T, H, P), xbc[:, inner:inner + G * N].view(T, G, N), xbc[:, inner + G * N:].view(T, G, N)
    dt = torch.nn.functional.softplus(dt + w("dt_bias"), threshold=1e9)
    keep = torch.exp(-torch.exp(w("A_log")) * dt)
    group = torch.arange(H) // (H // G)
    S = torch.zeros(H, N, P, dtype=F)
    y = torch.zeros(T, H, P, dtype=F)
    for t in range(T):
        S = S * keep[t][:, None, None] + dt[t][:, None, None] * B[t][group][:, :, None] * x[t][:, None, :]
        y[t] = torch.einsum("hnp,hn->hp", S, C[t][group]) + w("D")[:, None] * x[t]
    y = y.reshape(T, inner) * silu(z)
    return unit_rms(y.view(T, m["norm_groups"], -1), eps).reshape(T, inner) * w("norm")


def parallel(h, m, w, eps):
    """Two mixers on one input, each times a number of its own."""
    left, right = (lambda n: w("left." + n)), (lambda n: w("right." + n))
    return (m["left_scale"] * mm(window_attention_heads(h, m["left"], left, eps), left("o"))
            + m["right_scale"] * mm(state_space_heads(h, m["right"], right, eps), right("o")))


def gla(h, m, w, eps):
    """Gated linear attention: a decay for every key entry of every head; the read-out normed head by head."""
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q, k, v = mm(h, w("q")).view(T, H, D) * D ** -0.5, mm(h, w("k")).view(T, H, D), mm(h, w("v")).view(T, H, Dv)
    z = mm(mm(h, w("a1")), w("a2")) + w("a2.b")
    keep = torch.exp(torch.nn.functional.logsigmoid(z) / m["tau"]).view(T, H, D)
    S = torch.zeros(H, D, Dv, dtype=F)
    o = torch.zeros(T, H, Dv, dtype=F)
    for t in range(T):
        S = keep[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = torch.einsum("hde,hd->he", S, q[t])
    o = (unit_rms(o, eps) * w("norm")).reshape(T, H * Dv) * silu(mm(h, w("g")))
    return mm(o, w("o"))


def gated_ff(h, gate, up, down):
    return mm(silu(mm(h, gate)) * mm(h, up), down)


# every call of `route` leaves here, a token, how far its choice was from another one: the smallest chosen logit less
# the largest that was not chosen, over the root mean square of the token's logits (infinity where all are chosen)
route_margins: list = []


def route(h, top, router):
    """-> (chosen [T, top] indices, weights [T, top]): the largest sigmoids, as they are."""
    z = mm(h, router)
    ordered = torch.sort(z, dim=-1, descending=True).values
    size = torch.sqrt((z * z).mean(-1))
    route_margins.append((ordered[:, top - 1] - ordered[:, top]) / size if top < z.shape[1]
                         else torch.full((h.shape[0],), math.inf, dtype=F))
    best = torch.topk(z, top, dim=-1)
    return best.indices, torch.sigmoid(best.values)


def mixture(h, mlp, w):
    """Experts e0.. of which each token uses a few, each on the token's input times its weight, and a shared expert."""
    chosen, weights = route(h, mlp["router"]["top"], w("router"))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, f in zip(chosen[t].tolist(), weights[t]):
            out[t] = out[t] + gated_ff(f * h[t], w(f"e{e}.gate"), w(f"e{e}.up"), w(f"e{e}.down"))
    if mlp.get("shared"):
        out = out + gated_ff(h, w("shared.gate"), w("shared.up"), w("shared.down"))
    return out


MIXERS = {"parallel": parallel, "gla": gla}


def forward(config, tensors, tokens, return_layers=False):
    """tokens: a list of ids -> float64 logits [T, vocab] (and the residual after every layer run)."""
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = config["norm"]["eps"]
    norm = lambda x, name: unit_rms(x, eps) * t64(tensors[name])
    x0 = t64(tensors["embed"])[tokens] * config["embedding"]["scale"]
    x = x0
    n, loop = len(config["layers"]), config.get("loop")
    runs = [(i, None) for i in range(n)]
    if loop:
        a, b = loop["start"], loop["stop"]
        once = lambda t: [(i, t if i == a else None) for i in range(a, b)]
        runs = runs[:a] + [r for t in range(loop["times"]) for r in once(t)] + runs[b:]
    seen = []
    for i, begins in runs:
        if begins is not None:      # the first layer of a pass
            x = mm(torch.cat([x, x0], dim=-1), t64(tensors["loop.in"])) + t64(tensors["loop.step"])[begins]
        layer, p = config["layers"][i], f"l{i}."
        w_mix = lambda name, p=p: t64(tensors[p + "mix." + name])
        w_mlp = lambda name, p=p: t64(tensors[p + "mlp." + name])
        h = norm(x, p + "norm1")
        y = MIXERS[layer["type"]](h, layer["mixer"], w_mix, eps)
        if layer.get("mlp") is not None:
            y = y + mixture(h, layer["mlp"], w_mlp)
        x = x + y
        seen.append(x)
    cap = config["logit_softcap"]
    logits = cap * torch.tanh(mm(norm(x, "final.norm"), t64(tensors["head"])) / cap)
    return (logits, torch.stack(seen)) if return_layers else logits
