"""Pozirax's configuration, recipe and cache needs, and the plain implementation's own consistency (no GPU)."""
import copy

import pytest
import torch

import plain_pozirax as plain
from arle_amd.cache.manager import PagedNeed, StateNeed
from arle_amd.config import ConfigError, PoziraxConfig, detect_architecture
from arle_amd.models.decoder import declared_cache_needs, expected_checkpoint_tensors
from tiny import read_folder
from tiny_pozirax import TINY, attention, gla, make_model_dir, rot, state_space

F = torch.float64


@pytest.mark.parametrize("name", list(TINY))
def test_a_configuration_reads_back_equal_and_names_its_tensors(name):
    raw = TINY[name][0]
    config = PoziraxConfig.from_dict(raw)
    assert PoziraxConfig.from_dict(config.to_dict()) == config
    arch = detect_architecture(raw)
    assert arch.name == "Pozirax"
    expected = expected_checkpoint_tensors(arch.recipe(config, ()))
    W, V = raw["width"], raw["vocab"]
    found = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    if "loop" in raw:
        found.update({"loop.in": (W, 2 * W), "loop.step": (raw["loop"]["times"], W)})
    for i, lay in enumerate(raw["layers"]):
        m, p, mlp = lay["mixer"], f"l{i}.", lay["mlp"]
        found[p + "norm1"] = (W,)
        if lay["type"] == "parallel":
            a, s = m["left"], m["right"]
            kv, inner = a["kv_heads"], s["heads"] * s["vdim"]
            channels = inner + 2 * s["groups"] * s["state"]
            left = {"q": (a["heads"] * a["dim"], W), "k": (kv * a["dim"], W), "v": (kv * a["vdim"], W), "q.norm": (a["dim"],),
                    "k.norm": (a["dim"],), "o": (W, a["heads"] * a["vdim"])}
            right = {"in": (inner + channels + s["heads"], W), "conv": (channels, s["conv"]), "conv.b": (channels,),
                     "dt_bias": (s["heads"],), "A_log": (s["heads"],), "D": (s["heads"],), "norm": (inner,), "o": (W, inner)}
            found.update({p + "mix.left." + n: x for n, x in left.items()})
            found.update({p + "mix.right." + n: x for n, x in right.items()})
        else:
            k, v, r = m["heads"] * m["dim"], m["heads"] * m["vdim"], m["decay_rank"]
            found.update({p + "mix." + n: x for n, x in {"q": (k, W), "k": (k, W), "v": (v, W), "g": (v, W), "o": (W, v), "a1": (r, W),
                                                         "a2": (k, r), "a2.b": (k,), "norm": (m["vdim"],)}.items()})
        if mlp:
            E, f = mlp["router"]["experts"], mlp["expert"]["ff"]
            found[p + "mlp.router"] = (E, W)
            for e in [f"e{e}" for e in range(E)] + (["shared"] if mlp.get("shared") else []):
                n = mlp["shared"]["ff"] if e == "shared" else f
                found.update({f"{p}mlp.{e}.gate": (n, W), f"{p}mlp.{e}.up": (n, W), f"{p}mlp.{e}.down": (W, n)})
    assert {n: tuple(d.shape) for n, d in expected.items()} == found


def test_the_loop_repeats_its_layers_behind_an_entry_each_time():
    spec = detect_architecture(TINY["P"][0]).recipe(PoziraxConfig.from_dict(TINY["P"][0]), ())
    entry = len(spec.layers) - 1
    assert spec.layers[entry].block == "loop_entry"
    assert [e.layer for e in spec.schedule] == [entry, 0, entry, 1, 2, entry, 1, 2, 3]
    spec = detect_architecture(TINY["R"][0]).recipe(PoziraxConfig.from_dict(TINY["R"][0]), ())
    assert [e.layer for e in spec.schedule] == [3, 3, 0, 1, 2, 3, 0, 1, 2]
    spec = detect_architecture(TINY["S"][0]).recipe(PoziraxConfig.from_dict(TINY["S"][0]), ())
    assert [e.layer for e in spec.schedule] == [0, 1, 2]


def test_every_pass_has_caches_and_states_of_its_own():
    needs = declared_cache_needs(detect_architecture(TINY["P"][0]).recipe(PoziraxConfig.from_dict(TINY["P"][0]), ()))
    assert [n is None for n in needs] == [True, False, True, False, False, True, False, False, False]
    left, right = needs[1]["left"], needs[1]["right"]
    assert isinstance(left, PagedNeed) and left.window == 9
    assert [t.shape for t in left.tensors] == [(2, "page", 16), (2, 12, "page")]
    assert right["S"].shape == (6, 12, 8) and right["S"].dtype == torch.float32
    assert right["conv"].shape == (3, 6 * 8 + 2 * 3 * 12)
    assert isinstance(needs[3], StateNeed) and needs[3].shape == (3, 16, 24)
    assert needs[4]["left"].window == 30 and needs[7]["left"].window == 30
    # one tap keeps nothing
    needs = declared_cache_needs(detect_architecture(TINY["Q"][0]).recipe(PoziraxConfig.from_dict(TINY["Q"][0]), ()))
    assert set(needs[3]["right"]) == {"S"}


BAD = [
    (lambda r: r["layers"][0].update(type="parallel_9"), "unknown layer type"),
    (lambda r: r["layers"][0]["mixer"].pop("right"), "right"),
    (lambda r: r["layers"][0]["mixer"]["left"].update(kv_heads=3), "divisible"),
    (lambda r: r["layers"][0]["mixer"]["left"]["rot"].update(dims=11), "even"),
    (lambda r: r["layers"][0]["mixer"]["left"]["rot"].update(dims=18), "at most"),
    (lambda r: r["layers"][0]["mixer"]["left"]["mask"].update(size=0), "positive"),
    (lambda r: r["layers"][0]["mixer"]["left"].pop("scale"), "scale"),
    (lambda r: r["layers"][0]["mixer"]["right"].update(groups=4), "groups"),
    (lambda r: r["layers"][0]["mixer"]["right"].update(norm_groups=5), "norm_groups"),
    (lambda r: r["layers"][0]["mixer"]["right"].pop("conv"), "conv"),
    (lambda r: r["layers"][0]["mixer"]["right"].update(state=0), "positive"),
    (lambda r: r["layers"][0]["mixer"].update(left_scale=float("nan")), "finite"),
    (lambda r: r["layers"][1]["mixer"].update(tau=0.0), "tau"),
    (lambda r: r["layers"][1]["mixer"].pop("vdim"), "vdim"),
    (lambda r: r["layers"][0]["mlp"].update(kind="dense"), "unknown kind"),
    (lambda r: r["layers"][0]["mlp"]["router"].update(top=7), "top"),
    (lambda r: r["layers"][0]["mlp"].pop("expert"), "expert"),
    (lambda r: r["layers"][0]["mlp"]["shared"].update(ff=0), "positive"),
    (lambda r: r["loop"].update(stop=5), "within"),
    (lambda r: r["loop"].update(stop=1), "start < stop"),
    (lambda r: r["loop"].update(times=0), "times"),
    (lambda r: r.update(logit_softcap=-1.0), "softcap"),
    (lambda r: r["norm"].update(eps=-1.0), "eps"),
    (lambda r: r.update(layers=[]), "at least one"),
    (lambda r: r.pop("width"), "width"),
]


@pytest.mark.parametrize("case", range(len(BAD)))
def test_a_configuration_that_cannot_be_used_is_refused_with_its_key(case):
    change, word = BAD[case]
    raw = copy.deepcopy(TINY["P"][0])
    change(raw)
    with pytest.raises(ConfigError, match=word):
        PoziraxConfig.from_dict(raw)


def test_the_plain_implementation_agrees_with_itself():
    """Rotation, attention, both recurrences, convolution and router written a second way."""
    g = torch.Generator().manual_seed(1)
    r = lambda *s: torch.randn(*s, generator=g, dtype=F)
    x = r(3, 2, 10)
    y = plain.rotate_pairs(x, torch.tensor([0, 1, 7]), 6, 100.0)
    assert torch.equal(y[0], x[0]) and torch.equal(y[..., 6:], x[..., 6:])
    for i in range(3):
        turn = torch.polar(torch.ones((), dtype=F), torch.tensor(7 * 100.0 ** (-2.0 * i / 6), dtype=F))
        z = torch.complex(x[2, :, 2 * i], x[2, :, 2 * i + 1]) * turn
        assert torch.allclose(y[2, :, 2 * i], z.real) and torch.allclose(y[2, :, 2 * i + 1], z.imag)
    # attention, one row and head at a time
    m, T, W = attention(4, 2, 6, 5, 3, 0.4, rot(30.0, 4)), 8, 7
    w = {"q": r(24, W), "k": r(12, W), "v": r(10, W), "q.norm": r(6), "k.norm": r(6)}
    h = r(T, W)
    got = plain.window_attention_heads(h, m, w.__getitem__, 1e-5)
    unit = lambda v: v / (v.pow(2).mean() + 1e-5).sqrt()
    for t in range(T):
        for n in range(4):
            turn = lambda v, p: plain.rotate_pairs(v.view(1, 1, 6), torch.tensor([p]), 4, 30.0).view(6)
            q = turn(unit((h[t] @ w["q"].T)[6 * n:6 * n + 6]) * w["q.norm"], t)
            s, v = [], []
            for j in range(max(0, t - 2), t + 1):
                s.append(torch.dot(q, turn(unit((h[j] @ w["k"].T)[6 * (n // 2):6 * (n // 2) + 6]) * w["k.norm"], j)) * 0.4)
                v.append((h[j] @ w["v"].T)[5 * (n // 2):5 * (n // 2) + 5])
            e = torch.exp(torch.stack(s))
            assert torch.allclose(got[t, 5 * n:5 * n + 5], (e[:, None] * torch.stack(v)).sum(0) / (1 + e.sum()))
    # the state-space layer as an attention whose weights fall with the sum of the steps between two tokens
    m = state_space(4, 3, 5, 2, 3, 2)
    inner, C = 12, 12 + 2 * 2 * 5
    w = {"in": r(inner + C + 4, W), "conv": r(C, 3), "conv.b": r(C), "dt_bias": r(4), "A_log": r(4) * 0.5, "D": r(4), "norm": r(inner)}
    got = plain.state_space_heads(h, m, w.__getitem__, 1e-5)
    p = h @ w["in"].T
    u = torch.nn.functional.conv1d(torch.nn.functional.pad(p[:, inner:inner + C].T[None], (2, 0)), w["conv"][:, None], w["conv.b"],
                                   groups=C)[0].T
    u = u * torch.sigmoid(u)
    dt = torch.log1p(torch.exp(p[:, inner + C:] + w["dt_bias"]))
    y = torch.zeros(T, 4, 3, dtype=F)
    for n in range(4):
        k = u[:, inner + 5 * (n // 2):][:, :5]
        q = u[:, inner + 10 + 5 * (n // 2):][:, :5]
        L = torch.cumsum(-torch.exp(w["A_log"][n]) * dt[:, n], 0)
        a = (q @ k.T) * torch.exp(L[:, None] - L[None, :]) * dt[None, :, n]
        y[:, n] = torch.tril(a) @ u[:, 3 * n:3 * n + 3] + w["D"][n] * u[:, 3 * n:3 * n + 3]
    z = p[:, :inner]
    y = (y.reshape(T, inner) * z * torch.sigmoid(z)).view(T, 2, 6)
    want = (y / (y.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt()).view(T, inner) * w["norm"]
    assert torch.allclose(got, want)
    # gated linear attention likewise, a decay an entry
    m = gla(2, 4, 3, 5.0)
    w = {"q": r(8, W), "k": r(8, W), "v": r(6, W), "g": r(6, W), "o": r(W, 6), "a1": r(2, W), "a2": r(8, 2), "a2.b": r(8), "norm": r(3)}
    got = plain.gla(h, m, w.__getitem__, 1e-5)
    L = torch.cumsum(torch.log(torch.sigmoid(h @ w["a1"].T @ w["a2"].T + w["a2.b"]) ** 0.2), 0).view(T, 2, 4)
    q, k, v = (h @ w["q"].T).view(T, 2, 4) / 2.0, (h @ w["k"].T).view(T, 2, 4), (h @ w["v"].T).view(T, 2, 3)
    o = torch.zeros(T, 2, 3, dtype=F)
    for t in range(T):
        for j in range(t + 1):
            o[t] += ((q[t] * k[j] * torch.exp(L[t] - L[j])).sum(-1)[:, None]) * v[j]
    o = o / (o.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * w["norm"]
    z = h @ w["g"].T
    assert torch.allclose(got, (o.reshape(T, 6) * z * torch.sigmoid(z)) @ w["o"].T)
    # the router: sorted by hand
    h, router = r(20, 8), r(6, 8)
    chosen, weights = plain.route(h, 2, router)
    for t in range(20):
        z = h[t] @ router.T
        order = sorted(range(6), key=lambda e: -z[e])[:2]
        assert chosen[t].tolist() == order and torch.allclose(weights[t], 1 / (1 + torch.exp(-z[order])))


def test_a_mechanism_left_out_or_misread_would_show_in_the_test_models(tmp_path):
    """Each planted mistake moves the plain logits of a test model by far more than any tolerance."""
    cfg, weights = read_folder(make_model_dir(tmp_path, "P"))
    toks = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(3)).tolist()
    want = plain.forward(cfg, weights, toks)

    def differs(change_cfg=None, change_weights=None, **patched):
        c, w = copy.deepcopy(cfg), dict(weights)
        if change_cfg:
            change_cfg(c)
        if change_weights:
            change_weights(w)
        before = {n: getattr(plain, n) for n in patched}
        try:
            for n, f in patched.items():
                setattr(plain, n, f)
            return float((plain.forward(c, w, toks) - want).abs().max()) / float(want.abs().max())
        finally:
            for n, f in before.items():
                setattr(plain, n, f)

    right_route, right_conv = plain.route, plain.causal_conv

    def normalized(h, top, router):
        chosen, s = right_route(h, top, router)
        return chosen, s / s.sum(-1, keepdim=True)

    def on_the_output(h, mlp, w):
        chosen, s = right_route(h, mlp["router"]["top"], w("router"))
        out = plain.gated_ff(h, w("shared.gate"), w("shared.up"), w("shared.down"))
        for t in range(h.shape[0]):
            for e, f in zip(chosen[t].tolist(), s[t]):
                out[t] = out[t] + f * plain.gated_ff(h[t], w(f"e{e}.gate"), w(f"e{e}.up"), w(f"e{e}.down"))
        return out

    def halves(x, positions, dims, base):
        order = torch.arange(x.shape[-1])
        order[:dims] = torch.arange(dims).view(2, -1).T.flatten()
        return right_rotate(x[..., order], positions, dims, base)[..., order.argsort()]

    right_rotate = plain.rotate_pairs
    fill = lambda value, suffix: lambda w: [w.__setitem__(k, torch.full_like(v, value)) for k, v in list(w.items()) if k.endswith(suffix)]
    every = lambda f: lambda c: [f(l["mixer"]) for l in c["layers"] if l["type"] == "parallel"]
    mistakes = {
        "a window one token longer": differs(every(lambda m: m["left"]["mask"].update(size=m["left"]["mask"]["size"] + 1))),
        "no rotation": differs(rotate_pairs=lambda x, *a: x),
        "rotation of halves": differs(rotate_pairs=halves),
        "no query norm weight": differs(None, fill(1.0, ".q.norm")),
        "another attention scale": differs(every(lambda m: m["left"].update(scale=0.1))),
        "scales exchanged": differs(every(lambda m: m.update(left_scale=m["right_scale"], right_scale=m["left_scale"]))),
        "no convolution bias": differs(None, fill(0.0, ".conv.b")),
        "taps in reverse": differs(causal_conv=lambda u, taps, b: right_conv(u, taps.flip(1), b)),
        "no step bias": differs(None, fill(0.0, ".dt_bias")),
        "one decay for all": differs(None, fill(0.0, ".A_log")),
        "no skip": differs(None, fill(0.0, ".D")),
        "one norm group": differs(every(lambda m: m["right"].update(norm_groups=1))),
        "no decay bias": differs(None, fill(0.0, ".a2.b")),
        "another tau": differs(lambda c: [l["mixer"].update(tau=1.0) for l in c["layers"] if l["type"] == "gla"]),
        "no head norm weight": differs(None, fill(1.0, ".mix.norm")),
        "weights normalized": differs(route=normalized),
        "weights on the output": differs(mixture=on_the_output),
        "no row for the passes": differs(None, fill(0.0, "loop.step")),
        "one pass": differs(lambda c: c["loop"].update(times=1)),
        "another embedding scale": differs(lambda c: c["embedding"].update(scale=1.0)),
        "no cap": differs(lambda c: c.update(logit_softcap=1e9)),
    }
    for what, d in mistakes.items():
        assert d > 0.03, f"{what}: moves the logits by {d:.1e} only"
