"""Pozirax on the GPU against the plain implementation (`plain_pozirax.py`): every mechanism alone as the part or the
operation the engine runs, in cuts of every size, and whole models through `Engine.step`, the scheduler and
`LLM.generate`.

Tolerances.  float32: 5e-5 of the largest plain logit for whole models, 5e-5 of the largest plain output for a mechanism
alone (the plain side is float64; the engine adds in 32 bits).  bfloat16: 3e-2 of the largest plain logit for whole
models, 2.5e-2 of the largest plain output for a mechanism alone.
"""
import pytest
import torch

import plain_pozirax as plain
import replay
from arle_amd import LLM
from arle_amd.cache import CacheManager
from arle_amd.config import PoziraxConfig
from arle_amd.engine import Engine, StepEntry
from arle_amd.engine.batch import build_step_batch
from arle_amd.kernels import ops
from arle_amd.models.pozirax import pozirax_spec
from arle_amd.parts.base import Runtime, build_part, expected_tensors
from arle_amd.parts.position import rope_table
from arle_amd.parts.spec import PartSpec
from tiny import random_tokens, read_folder
from tiny_pozirax import ARCH, TINY, attention, gla, layer, make_model_dir, moe, pair, rot, spread, state_space

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 5e-5, BF16: 2.5e-2}
EPS = 1e-5


def rnd(shape, seed, std=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * std).to(BF16).float()     # values that bfloat16 holds exactly


def close(got, want, dtype, what, tol=None):
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all(), what
    err = float((got - want).abs().max()) / float(want.abs().max())
    assert err <= (tol or TOL[dtype]), f"{what}: {err:.3e}"


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def one_layer(kind, mixer, mlp=None, width=40):
    """(config dictionary, ModelSpec) of a model of one layer."""
    raw = {"architecture": ARCH, "vocab": 50, "width": width, "norm": {"eps": EPS}, "layers": [layer(kind, mixer, mlp)]}
    return raw, pozirax_spec(PoziraxConfig.from_dict(raw))


def alone(spec, output: str):
    """One of a pair's mixers as a mixer by itself, with the output projection `output`."""
    return PartSpec(spec.kind, dict(spec.params, project_out=True), dict(spec.weights, o=output))


def random_part(role, spec, dtype, seed, std=0.3):
    """A part of `spec` with random tensors; returns (part, {checkpoint name: float32 CPU tensor})."""
    tensors = {}
    for i, (name, decl) in enumerate(sorted(expected_tensors(role, spec).items())):
        t = 1 + rnd(tuple(decl.shape), seed + i, 0.3) if decl.init == "ones" else rnd(tuple(decl.shape), seed + i, std)
        tensors[name] = spread(name, t, torch.Generator().manual_seed(seed + i)).to(BF16).float()
    rt = Runtime(device=torch.device(DEV), act_dtype=dtype)
    held = {k: v.to(DEV, dtype) for k, v in tensors.items()}
    return build_part(role, spec, held.__getitem__, rt), tensors


def poison(state, slot):
    for view in (state.values() if isinstance(state, dict) else [state]):
        if isinstance(view, dict):
            poison(view, slot)
        elif getattr(view, "state", None) is not None:
            view.state[slot] = float("nan")


def run_mixer(part, x, cuts, *, page=4, dtype=F32):
    """Feed x [T, W] of one request to a mixer in portions of the given sizes (repeating), through a cache in which
    another request's pages and slot lie between, every page starts as NaN and the other request's state is rubbish.
    Returns the concatenated outputs."""
    T = x.shape[0]
    part.prepare(T + page)
    cache = CacheManager([part.cache_need()], page_size=page, num_pages=2 * (-(-T // page)) + 4, max_slots=3,
                         max_request_tokens=T + page, device=torch.device(DEV), dtype=dtype)
    cache.admit("other")
    cache.append([("other", page + 1)])
    for group in cache.page_buffers:
        for t in group.values():
            t.fill_(float("nan"))
    cache.admit("r")
    poison(cache.view(0), cache.slot_of["other"])
    outs, at, k = [], 0, 0
    xd = x.to(DEV, dtype)
    while at < T:
        n = min(cuts[k % len(cuts)], T - at)
        k += 1
        before = cache.length("r")
        cache.append([("r", n)])
        cache.sync_tables()
        batch = build_step_batch([StepEntry("r", [0] * n, [])], cache.slot_of.__getitem__, lambda _r, b=before: b, 10, DEV)
        y = part.forward(xd[at:at + n].contiguous(), batch, cache.view(0))
        outs.append((y.float().sum(0) if y.dim() == 3 else y.float()).cpu())
        at += n
    cache.check()
    return torch.cat(outs)


CUTS = [(1000,), (1,), (2,), (5, 2, 7, 3, 1, 16, 2)]


def rounded_products(dtype, trial):
    """Products whose operands and results are rounded (trial 0), or move at random by up to half a unit in the last place."""
    unit = 2.0 ** -24 if dtype == F32 else 2.0 ** -9
    g = torch.Generator().manual_seed(50 + trial)
    move = lambda y: y * (1 + (torch.rand(y.shape, generator=g, dtype=torch.float64) - 0.5) * 2 * unit) if trial else y.to(dtype).double()
    return lambda x, w: move(move(x) @ w.T)


def mixer_case(spec, function, dtype, seed, T, *, width=40, page=4, loud=(), std=0.3, cuts=CUTS, tol=None, jitter=True, setup=None):
    """A mixer alone against its plain function(x, w), in every cutting; in float32 the cuttings agree bit for bit.
    loud: positions whose input dwarfs the others', so that a key seen or hidden by mistake shows.  jitter: a row may be
    wrong by eight times what moving every operand and result of every product by up to half a unit in the last place, or
    rounding them, does to it (norms on a recurrence's read-out magnify rounding where its terms nearly cancel, most at a request's first
    rows)."""
    part, tensors = random_part("mixer", spec, dtype, seed, std)
    if setup is not None:
        setup(part)
    x = rnd((T, width), seed + 100)
    for p in loud:
        if 0 <= p < T:
            x[p] *= 6.0
    w = lambda name: tensors["l0.mix." + name].double()
    want = function(x.double(), w)
    bound = torch.full((T,), tol or TOL[dtype], dtype=torch.float64)
    if jitter:
        for trial in range(4):
            plain.around_product = rounded_products(dtype, trial)
            try:
                moved = function(x.double(), w)
            finally:
                plain.around_product = None
            bound = torch.maximum(bound, 8.0 * (moved - want).abs().max(1).values / want.abs().max())
    first = None
    for c in cuts:
        got = run_mixer(part, x, c, page=page, dtype=dtype)
        assert torch.isfinite(got).all()
        err = (got.double() - want).abs().max(1).values / want.abs().max()
        worst = int((err / bound).argmax())
        assert err[worst] <= bound[worst], f"{spec.kind} {dtype} cut {c}: row {worst} is off by {float(err[worst]):.3e}"
        if dtype == F32:
            first = got if first is None else first
            assert torch.equal(got, first), f"{spec.kind}: cut {c} differs in bits from the whole prompt"


# ----------------------------------------------------------------------------------- the windowed attention

ATTENTIONS = [
    # (mixer, page, T)
    (attention(4, 2, 16, 12, 9, 0.35, rot(500.0, 12)), 4, 40),
    (attention(1, 1, 10, 14, 1, 0.4), 8, 20),
    (attention(5, 1, 6, 10, 7, 0.5, rot(20.0, 4)), 4, 30),
    (attention(4, 1, 32, 48, 40, 0.18, rot(250000.0, 32)), 16, 150),
    (attention(6, 6, 48, 32, 16, 0.2, rot(100.0, 48)), 16, 70),
    (attention(2, 2, 24, 16, 64, 0.2, rot(1000.0, 2)), 16, 140),
    (attention(3, 3, 128, 128, 65, 0.1, rot(1e6, 128)), 64, 140),
    # heads of one size: in bfloat16 the kernels of the plain softmax
    (attention(4, 2, 16, 16, 9, 0.35, rot(500.0, 12)), 4, 40),
    (attention(6, 2, 48, 48, 41, 0.2, rot(3e5, 48)), 16, 150),
    (attention(8, 1, 64, 64, 17, 0.15, rot(1e4, 64)), 16, 90),
    (attention(2, 1, 256, 256, 33, 0.08, rot(1e4, 32)), 16, 70),
    (attention(5, 5, 32, 32, 1, 0.2), 8, 30),
]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", range(len(ATTENTIONS)))
def test_the_windowed_attention_equals_plain_in_every_cut(dtype, case):
    m, page, T = ATTENTIONS[case]
    window = m["mask"]["size"]
    raw, spec = one_layer("parallel", pair(m, state_space(1, 4, 4, 1)))
    left = alone(spec.layers[0].mixer.params["left"], "l0.mix.left.o")
    function = lambda x, w: plain.mm(plain.window_attention_heads(x, m, lambda n: w("left." + n), EPS), w("left.o"))
    mixer_case(left, function, dtype, 20 + 9 * case, T, page=page, loud=(0, window - 1, window, page, T // 2), jitter=False,
               tol=4e-2 if dtype == BF16 else None)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("window,page", [(16, 16), (17, 16), (33, 4), (5, 8)])
def test_a_key_inside_and_outside_of_the_window(dtype, window, page):
    """A key that would take most of the softmax stands where the last row just sees it, just does not, and near it."""
    T, W = 90, 40
    m = attention(2, 1, 16, 16, window, 1.5, rot(1e6, 4))
    raw, spec = one_layer("parallel", pair(m, state_space(1, 4, 4, 1)))
    part, tensors = random_part("mixer", alone(spec.layers[0].mixer.params["left"], "l0.mix.left.o"), dtype, 77, 0.3)
    w = lambda name: tensors["l0.mix.left." + name].double()
    function = lambda x: plain.window_attention_heads(x.double(), m, w, EPS) @ w("o").T
    base = rnd((T, W), 5, 0.5)
    quiet = function(base)[-1]
    for target in (T - window, T - window - 1, T - window + 1, T - 2):
        seen = T - 1 - target < window
        best, moved = None, -1.0
        for trial in range(60):       # of sixty random inputs at the target, the one that the last row hears most
            x = base.clone()
            x[target] = rnd((W,), 1000 + trial)
            d = float((function(x)[-1] - quiet).abs().max()) if seen else float(trial == 0)
            if d > moved:
                best, moved = x, d
        want = function(best)
        assert not seen or moved > 0.3 * float(quiet.abs().max()), "the test's own inputs must make it matter"
        if not seen:
            best[target] *= 1e3       # nothing of it may be heard
            want = function(best)
            assert torch.equal(want[-1], quiet)
        for c in ((1000,), (7, 1), (T - 1, 1)):
            close(run_mixer(part, best, c, page=page, dtype=dtype)[-1], want[-1], dtype, f"key at {target}, window {window}, cut {c}",
                  tol=4e-2 if dtype == BF16 else 1e-4)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_the_sink_takes_its_share_and_scores_below_it_leave_nothing(dtype):
    """Keys whose scores are far below the sink's 0: the attention hands out almost nothing, where a softmax without the
    sink would hand out whole values."""
    m = attention(2, 2, 16, 16, 12, 1.0)
    raw, spec = one_layer("parallel", pair(m, state_space(1, 4, 4, 1)))
    left = alone(spec.layers[0].mixer.params["left"], "l0.mix.left.o")
    part, tensors = random_part("mixer", left, dtype, 3, 0.3)
    tensors["l0.mix.left.k"] = -tensors["l0.mix.left.q"]           # every key points away from its own query
    held = {k: v.to(DEV, dtype) for k, v in tensors.items()}
    part = build_part("mixer", left, held.__getitem__, Runtime(device=torch.device(DEV), act_dtype=dtype))
    tensors = {k: v.double() for k, v in tensors.items()}
    x = rnd((1, 40), 8).expand(30, 40).contiguous()
    w = lambda n: tensors["l0.mix.left." + n]
    want = plain.window_attention_heads(x.double(), m, w, EPS) @ w("o").T
    whole = x.double() @ w("v").T @ w("o").T
    assert float(want.abs().max()) < 0.05 * float(whole.abs().max())
    for c in ((1000,), (1,), (4,)):
        got = run_mixer(part, x, c, dtype=dtype)
        assert float((got.double() - want).abs().max()) < 1e-3 * float(whole.abs().max())


SINK_OPS = [
    # (q heads, kv heads, head size, page, window, segments: (rows now, position of the first), portions' keys in parts)
    (4, 2, 64, 16, 0, [(300, 0), (1, 200), (5, 63)], 1),
    (8, 2, 128, 64, 100, [(300, 40), (1, 700), (40, 0), (1, 99), (1, 100)], 1),
    (6, 3, 48, 16, 17, [(97, 0), (2, 31), (1, 0), (1, 500)], 1),
    (8, 8, 128, 64, 0, [(200, 300), (150, 0)], 4),
    (16, 2, 64, 32, 65, [(64, 500)], 3),
    (2, 1, 256, 16, 33, [(50, 0), (1, 80)], 1),
    (4, 4, 128, 16, 1, [(140, 3), (1, 5)], 1),
]


@pytest.mark.parametrize("single", [False, True])
@pytest.mark.parametrize("case", range(len(SINK_OPS)))
def test_the_plain_softmax_with_a_sink_a_factor_and_a_window_equals_float64(case, single):
    """Segments of several requests on pages in a shuffled order, sinks of several sizes, rows of the output far apart; decoded
    rows with their keys split several ways."""
    nq, nkv, D, page, window, segments, parts = SINK_OPS[case]
    if single:
        segments = [(1, start + n - 1) for n, start in segments]
    S, T = len(segments), sum(n for n, _ in segments)
    g = torch.Generator().manual_seed(case)
    per = -(-max(n + start for n, start in segments) // page)
    order = torch.randperm(S * per + 2, generator=g).to(torch.int32)
    table = torch.full((S, per), -1, dtype=torch.int32)
    k_pages = torch.full((S * per + 2, nkv, page, D), float("nan"))
    v_pages = torch.full((S * per + 2, nkv, D, page), float("nan"))
    q, sink = rnd((T, nq, D), 3 + case), rnd((nq,), 5, 2.0)
    sink[0] = 0.0
    want = torch.zeros(T, nq, D, dtype=torch.float64)
    row0, at, scale, factor = [0], 0, 1.5 / D ** 0.5, -0.7
    for s, (n, start) in enumerate(segments):
        k, v = rnd((start + n, nkv, D), 100 + 10 * case + s), rnd((start + n, nkv, D), 500 + 10 * case + s)
        first = max(0, start - window + 1) if window else 0
        for p in range(first // page, -(-(start + n) // page)):
            pid = int(order[s * per + p])
            table[s, p] = pid
            m = min(page, start + n - p * page)
            k_pages[pid, :, :m] = k[p * page:p * page + m].transpose(0, 1)
            v_pages[pid, :, :, :m] = v[p * page:p * page + m].permute(1, 2, 0)
        for t in range(n):
            pos = start + t
            lo = max(0, pos - window + 1) if window else 0
            for h in range(nq):
                z = (k[lo:pos + 1, h // (nq // nkv)].double() @ q[at + t, h].double()) * scale
                p = torch.softmax(torch.cat([z, sink[h:h + 1].double()]), dim=0)[:-1]
                want[at + t, h] = factor * (p @ v[lo:pos + 1, h // (nq // nkv)].double())
        at += n
        row0.append(at)
    lengths = [n for n, _ in segments]
    for splits in (1, 2, 8) if max(lengths) == 1 else (None,):
        out = torch.full((T, nq * D + 24), 9.0, dtype=BF16, device=DEV)
        ops.attn_paged_mfma(q.reshape(T, nq * D).to(DEV, BF16), out[:, 8:8 + nq * D], k_pages.to(DEV, BF16), v_pages.to(DEV, BF16),
                            table.to(DEV), i32(row0), i32(list(range(S))), i32([start for _, start in segments]),
                            max_qlen=max(lengths), min_qlen=min(lengths), max_kv_len=max(n + start for n, start in segments),
                            num_q_heads=nq, num_kv_heads=nkv, head_dim=D, page_size=page, scale=scale, window=window, splits=splits,
                            portion_splits=None if single else parts, sink=sink.to(DEV), out_scale=factor)
        close(out[:, 8:8 + nq * D].reshape(T, nq, D), want, BF16, f"splits {splits}", tol=1.2e-2)
        assert bool((out[:, :8] == 9).all()) and bool((out[:, 8 + nq * D:] == 9).all())


def test_decoded_rows_are_prepared_from_the_sums_with_the_same_bits():
    """The preparation from partial sums against the one from rounded projections."""
    for nq, nkv, Dk, Dv, R, inter, unit, S in ((4, 2, 16, 24, 12, True, False, 3), (6, 3, 48, 16, 48, True, False, 1),
                                               (8, 1, 128, 128, 64, False, True, 5), (2, 2, 8, 8, 0, True, False, 9)):
        T, page, slots, first = 7, 16, 9, 32
        width = first + (nq + nkv) * Dk + nkv * Dv
        width += -width % 16
        stack = rnd((S, T, width), 3 + Dk).to(DEV)
        y = ops.sum_partials(stack, BF16) if S > 1 else stack[0].to(BF16)
        cos, sin = (t.to(DEV) for t in rope_table(R, 500.0, 64)) if R else (None, None)
        wq, wk = (1 + rnd((Dk,), 5, 0.3)).to(DEV, BF16), (1 + rnd((Dk,), 6, 0.3)).to(DEV, BF16)
        pages = lambda: (torch.zeros(slots * 4, nkv, page, Dk, dtype=BF16, device=DEV), torch.zeros(slots * 4, nkv, Dv, page, dtype=BF16, device=DEV))
        common = dict(num_q_heads=nq, num_kv_heads=nkv, key_dim=Dk, value_dim=Dv, eps=EPS, q_weight=None if unit else wq,
                      k_weight=None if unit else wk, unit_after=unit, cos=cos, sin=sin, rotary_dim=R, interleaved=inter,
                      positions=i32([3, 0, 17, 40, 63, 16, 15]), slot_of_token=i32([8, 1, 0, 3, 2, 5, 4]),
                      block_table=torch.randperm(slots * 4, generator=torch.Generator().manual_seed(1)).to(torch.int32).view(slots, 4).to(DEV),
                      page_size=page)
        ka, va = pages()
        q = y[:, first:first + nq * Dk].clone()
        ops.rotary_qkv_store(q, y[:, first + nq * Dk:first + (nq + nkv) * Dk], y[:, first + (nq + nkv) * Dk:first + (nq + nkv) * Dk + nkv * Dv],
                             k_pages=ka, v_pages=va, **common)
        kb, vb = pages()
        got = ops.rotary_sums_store(stack if S > 1 else stack[0], first, k_pages=kb, v_pages=vb, **common)
        assert torch.equal(got, q) and torch.equal(ka, kb) and torch.equal(va, vb)


# ----------------------------------------------------------------------------------- the state-space layer

STATE_SPACES = [
    # (mixer, T)
    (state_space(6, 8, 12, 3, 4, 2), 60),              # a state that the chunks' form refuses
    (state_space(1, 6, 10, 1, 1, 1), 50),              # one tap; sizes that both fast forms refuse
    (state_space(5, 10, 6, 5, 2, 10), 40),
    (state_space(4, 32, 64, 2, 3, 4), 200),
    (state_space(2, 40, 24, 1, 4, 5), 140),
    (state_space(3, 16, 72, 3, 5, 1), 130),
    (state_space(2, 72, 136, 2, 4, 2), 150),
    (state_space(2, 136, 8, 1, 2, 4), 129),
    (state_space(8, 8, 16, 4, 16, 8), 90),
]
SCAN_CUTS = CUTS + [(64, 1), (63, 65, 2), (17, 1, 1, 33), (128, 3)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", range(len(STATE_SPACES)))
def test_the_state_space_layer_equals_plain_in_every_cut(dtype, case):
    m, T = STATE_SPACES[case]
    raw, spec = one_layer("parallel", pair(attention(1, 1, 4, 4, 4), m))
    right = alone(spec.layers[0].mixer.params["right"], "l0.mix.right.o")
    function = lambda x, w: plain.mm(plain.state_space_heads(x, m, lambda n: w("right." + n), EPS), w("right.o"))
    for chunks_from in (2, 10 ** 6) if dtype == BF16 else (None,):
        mixer_case(right, function, dtype, 100 + 20 * case, T, loud=(0, 63, 64), cuts=SCAN_CUTS, std=0.25,
                   tol=2e-4 if dtype == F32 else 3e-2, setup=lambda part: chunks_from and setattr(part, "CHUNKS_FROM", chunks_from))


SS_OPS = [
    # (heads, groups, state, values, segments)
    (2, 1, 64, 64, [64]),
    (4, 2, 32, 16, [1, 65, 1, 128, 2]),
    (3, 3, 128, 72, [200, 63]),
    (2, 1, 256, 256, [31, 97]),
    (6, 2, 40, 8, [129, 16, 17]),
    (2, 2, 8, 128, [70, 64]),
    (4, 4, 136, 200, [64, 128, 1]),
]


@pytest.mark.parametrize("fast", [False, True])
@pytest.mark.parametrize("form", ["rows", "rows32", "chunks"])
@pytest.mark.parametrize("case", range(len(SS_OPS)))
def test_the_forms_of_the_state_space_recurrence_agree_with_float64_from_a_state_on(case, form, fast):
    """Segments of several requests with states of their own in slots out of order, bfloat16 (or 32-bit) in, 32-bit out.
    fast: steps so large that a state is forgotten within a few tokens."""
    H, G, N, P, segments = SS_OPS[case]
    T, S = sum(segments), len(segments)
    u = rnd((T, H * P + 2 * G * N), 7 + case)
    dt = rnd((T, H + 3), 8 + case) + (4.0 if fast else -1.5)
    a_log = rnd((H,), 1) + (1.0 if fast else -1.0)
    dt_bias, skip = rnd((H,), 2, 0.5), rnd((H,), 3)
    slots = [2 * i + 1 for i in reversed(range(S))]
    state = rnd((2 * S + 1, H, N, P), 9 + case, 0.5)
    row0 = [0]
    for n in segments:
        row0.append(row0[-1] + n)
    want, after = torch.zeros(T, H * P, dtype=torch.float64), state.double().clone()
    step = torch.log1p(torch.exp((dt[:, :H] + dt_bias).double()))
    keep = torch.exp(-torch.exp(a_log.double()) * step)
    group = torch.arange(H) // (H // G)
    for s in range(S):
        for t in range(row0[s], row0[s + 1]):
            x, B, C = u[t, :H * P].view(H, P).double(), u[t, H * P:H * P + G * N].view(G, N).double(), u[t, H * P + G * N:].view(G, N).double()
            after[slots[s]] = after[slots[s]] * keep[t][:, None, None] + step[t][:, None, None] * B[group][:, :, None] * x[:, None, :]
            want[t] = (torch.einsum("hnp,hn->hp", after[slots[s]], C[group]) + skip.double()[:, None] * x).reshape(-1)
    d = lambda t: t.to(DEV)
    held, dtype = d(state).clone(), F32 if form == "rows32" else BF16
    ud = u.to(DEV, dtype)
    rest = (d(dt), d(a_log), d(dt_bias), d(skip), held, i32(row0), i32(slots))
    sizes = dict(heads=H, groups=G, state=N, value_dim=P)
    if form == "chunks":
        assert ops.state_space_chunks_supported(BF16, T, S, H, N, P)
        got = ops.state_space_chunks(ud, *rest, **sizes)
    else:
        got = ops.state_space_rows(ud[:, :H * P], ud[:, H * P:H * P + G * N], ud[:, H * P + G * N:], *rest, **sizes)
    close(got, want, F32, f"{form}", tol=2e-5)
    close(held, after, F32, "the states", tol=2e-5)
    untouched = [s for s in range(state.shape[0]) if s not in slots]
    assert torch.equal(held.cpu()[untouched], state[untouched]), "other slots keep theirs"


@pytest.mark.parametrize("H,G,N,P,taps,norm_groups,parts", [(6, 3, 12, 8, 4, 2, 3), (4, 2, 64, 32, 3, 4, 1), (2, 1, 256, 256, 2, 1, 9),
                                                            (5, 5, 7, 4, 1, 5, 4), (3, 1, 136, 72, 16, 27, 2), (80, 8, 128, 64, 4, 8, 4)])
def test_a_decoded_row_of_the_state_space_layer_goes_from_the_sums_to_the_gated_norm(H, G, N, P, taps, norm_groups, parts):
    inner, T, first = H * P, 5, 16
    C = inner + 2 * G * N
    width = first + inner + C + H
    width += -width % 16
    stack = torch.zeros(parts, T, width)
    total = rnd((T, width), 2)
    for i in range(parts):                       # exact parts: halves, quarters, ... of bfloat16 numbers
        stack[i] = total * (0.5 ** (i + 1) if i + 1 < parts else 0.5 ** i)
    conv, conv_bias = rnd((C, taps), 3, 0.5), rnd((C,), 4, 0.5)
    a_log, dt_bias, skip, norm = rnd((H,), 5, 0.5), rnd((H,), 6, 0.5), rnd((H,), 7), 1 + rnd((inner,), 8, 0.3)
    slots, row_slots = 9, [8, 1, 0, 3, 5]
    state, conv_state = rnd((slots, H, N, P), 9, 0.5), rnd((slots, max(taps - 1, 1), C), 10)
    out = torch.full((T, inner + 24), 7.0, dtype=BF16, device=DEV)
    held, held_conv = state.to(DEV), conv_state.to(DEV, BF16)
    d = lambda t: t.to(DEV)
    ops.state_space_decode(d(stack) if parts > 1 else d(stack[0]), first, conv.to(DEV, BF16), conv_bias.to(DEV, BF16),
                           held_conv if taps > 1 else None, d(a_log), d(dt_bias), d(skip), d(norm), held, i32(list(range(T + 1))),
                           i32(row_slots), EPS, out[:, 8:8 + inner], heads=H, groups=G, state=N, value_dim=P, norm_groups=norm_groups,
                           factor=-0.5)
    assert bool((out[:, :8] == 7).all()) and bool((out[:, 8 + inner:] == 7).all())
    want, after, after_conv = torch.zeros(T, inner, dtype=torch.float64), state.double().clone(), conv_state.clone()
    group = torch.arange(H) // (H // G)
    for t, slot in enumerate(row_slots):
        r = total[t, first:].double()
        z, now, raw = r[:inner], r[inner:inner + C], r[inner + C:inner + C + H]
        u = conv[:, -1].double() * now + conv_bias.double()
        for b in range(1, taps):
            u = u + conv[:, taps - 1 - b].double() * conv_state[slot, taps - 1 - b].double()
        if taps > 1:
            after_conv[slot] = torch.cat([conv_state[slot, 1:], now[None].float()])
        u = plain.silu(u).to(BF16).double()
        x, B, Cc = u[:inner].view(H, P), u[inner:inner + G * N].view(G, N), u[inner + G * N:].view(G, N)
        step = torch.log1p(torch.exp(raw + dt_bias.double()))
        S = after[slot] * torch.exp(-torch.exp(a_log.double()) * step)[:, None, None] + step[:, None, None] * B[group][:, :, None] * x[:, None, :]
        after[slot] = S
        y = (torch.einsum("hnp,hn->hp", S, Cc[group]) + skip.double()[:, None] * x).reshape(-1) * plain.silu(z)
        want[t] = -0.5 * plain.unit_rms(y.view(norm_groups, -1), EPS).reshape(-1) * norm.double()
    close(out[:, 8:8 + inner], want, BF16, "the output", tol=1.2e-2)
    close(held, after, F32, "the states", tol=8e-3)          # (a value of the convolution may round the other way)
    assert torch.equal(held_conv.float().cpu()[:, :taps - 1], after_conv[:, :taps - 1]), "the convolution's inputs"


def test_the_gated_group_norm_writes_into_a_view():
    for T, width, groups in ((3, 48, 2), (5, 60, 10), (2, 5120, 8), (300, 256, 1), (2, 16384, 1), (4, 7, 7)):
        y, z, w = rnd((T, width), 1, 2.0), rnd((T, width + 8), 2), 1 + rnd((width,), 3, 0.3)
        gated = y.double() * plain.silu(z[:, 8:].double())
        want = 0.7 * plain.unit_rms(gated.view(T, groups, -1), EPS).reshape(T, width) * w.double()
        for dtype in (F32, BF16):
            out = torch.full((T, width + 16), 3.0, dtype=dtype, device=DEV)
            zd = z.to(DEV, dtype)
            ops.gated_group_norm(y.to(DEV), zd[:, 8:], w.to(DEV), EPS, groups=groups, factor=0.7, out=out[:, 16:])
            close(out[:, 16:], want, dtype, f"{width} in {groups}", tol=1e-2 if dtype == BF16 else 1e-5)
            assert bool((out[:, :16] == 3).all())


# ----------------------------------------------------------------------------------- gated linear attention

GLAS = [
    # (mixer, T)
    (gla(3, 16, 24, 4.0, 5), 60),
    (gla(1, 10, 6, 0.25, 3), 70),            # sizes that both fast forms refuse; decays that forget at once
    (gla(2, 64, 128, 16.0, 16), 200),
    (gla(2, 36, 20, 2.0, 20), 150),
    (gla(1, 132, 136, 16.0, 16), 140),
    (gla(1, 256, 256, 8.0, 70), 130),
    (gla(4, 32, 64, 0.1, 9), 140),           # blocks of rows forget more than a factor may grow
    (gla(3, 20, 4, 1.0, 1), 129),
]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", range(len(GLAS)))
def test_gated_linear_attention_equals_plain_in_every_cut(dtype, case):
    m, T = GLAS[case]
    raw, spec = one_layer("gla", m)
    for chunks_from in (2, 10 ** 6) if dtype == BF16 else (None,):
        mixer_case(spec.layers[0].mixer, lambda x, w: plain.gla(x, m, w, EPS), dtype, 300 + 20 * case, T, loud=(0, 63, 64),
                   cuts=SCAN_CUTS, std=0.25, tol=2e-4 if dtype == F32 else 3e-2,
                   setup=lambda part: chunks_from and setattr(part, "CHUNKS_FROM", chunks_from))


GLA_OPS = [
    # (heads, key size, value size, middle, tau, bias, segments)
    (2, 64, 128, 16, 16.0, 0.0, [64]),
    (3, 32, 64, 8, 16.0, 1.0, [1, 65, 1, 128, 2]),
    (1, 128, 256, 16, 4.0, 0.0, [200, 63]),
    (2, 256, 40, 33, 16.0, -2.0, [31, 97]),
    (2, 24, 20, 100, 1.0, 0.0, [129, 16, 17]),
    (5, 4, 4, 1, 0.05, 0.0, [70]),                   # nothing is left after a token
    (2, 64, 64, 16, 0.5, -3.0, [150, 64]),           # forgets within a token or two
    (1, 72, 32, 16, 0.02, 6.0, [130]),               # most entries hardly forget, some all at once
]


@pytest.mark.parametrize("case", range(len(GLA_OPS)))
@pytest.mark.parametrize("form", ["rows", "chunks", "decode"])
def test_the_forms_of_gated_linear_attention_agree_with_float64_from_a_state_on(case, form):
    """Segments of several requests with states of their own in slots out of order, 32-bit in and out."""
    H, D, Dv, rank, tau, bias, segments = GLA_OPS[case]
    if form == "decode":
        segments = [1 for _ in segments] + [1]
    T, S = sum(segments), len(segments)
    width = 2 * H * (D + Dv) + rank
    width += -width % 16
    y = rnd((T, width), 7 + case)
    a2, a2_bias, norm = rnd((H * D, rank), 3, rank ** -0.5), bias + rnd((H * D,), 4), 1 + rnd((Dv,), 5, 0.3)
    slots = [2 * i + 1 for i in reversed(range(S))]
    state = rnd((2 * S + 1, H, D, Dv), 9 + case, 0.5)
    row0 = [0]
    for n in segments:
        row0.append(row0[-1] + n)
    want, after = torch.zeros(T, H * Dv, dtype=torch.float64), state.double().clone()
    qw, vw = H * D, H * Dv
    middle = y[:, 2 * qw + 2 * vw:2 * qw + 2 * vw + rank].double()
    keep = torch.exp(torch.nn.functional.logsigmoid(middle @ a2.double().T + a2_bias.double()) / tau).view(T, H, D)
    for s in range(S):
        for t in range(row0[s], row0[s + 1]):
            r = y[t].double()
            k, v = r[qw:2 * qw].view(H, D), r[2 * qw:2 * qw + vw].view(H, Dv)
            after[slots[s]] = after[slots[s]] * keep[t][:, :, None] + k[:, :, None] * v[:, None, :]
            o = torch.einsum("hde,hd->he", after[slots[s]], r[:qw].view(H, D)) * D ** -0.5
            want[t] = (plain.unit_rms(o, EPS) * norm.double()).reshape(-1) * plain.silu(r[2 * qw + vw:2 * qw + 2 * vw])
    d = lambda t: t.to(DEV)
    for out_dtype, w_dtype in ((F32, F32), (BF16, BF16)):
        held = d(state).clone()
        args = (a2.to(DEV, w_dtype), d(a2_bias), d(norm), held, i32(row0), i32(slots), EPS, out_dtype)
        sizes = dict(tau=tau, heads=H, key_dim=D, value_dim=Dv)
        if form == "chunks":
            assert ops.gated_linear_chunks_supported(T, S, H, D, Dv)
            got = ops.gated_linear_chunks(d(y), *args, **sizes)
        elif form == "rows":
            got = ops.gated_linear_rows(d(y), *args, **sizes)
        else:
            stack = torch.stack([d(y) * 0.5, d(y) * 0.25, d(y) * 0.25])      # partial sums of the product, exact halves
            got = ops.gated_linear_decode(stack, *args, **sizes)
            assert torch.equal(ops.gated_linear_decode(d(y), args[0], args[1], args[2], d(state).clone(), *args[4:], **sizes), got)
        close(got, want, out_dtype, f"{form} {out_dtype}", tol=1e-2 if out_dtype == BF16 else 2e-4)
        close(held, after, F32, "the states", tol=3e-5)
        untouched = [s for s in range(state.shape[0]) if s not in slots]
        assert torch.equal(held.cpu()[untouched], state[untouched]), "other slots keep theirs"


def test_both_recurrences_over_long_decoding():
    ss, gl = state_space(4, 16, 24, 2, 4, 2), gla(2, 32, 16, 16.0, 8)
    raw, spec = one_layer("parallel", pair(attention(2, 2, 16, 16, 20, 0.3, rot(1000.0, 16)), ss))
    _, other = one_layer("gla", gl)
    x = rnd((460, raw["width"]), 91)
    cases = ((spec.layers[0].mixer, lambda w: plain.parallel(x.double(), raw["layers"][0]["mixer"], w, EPS)),
             (other.layers[0].mixer, lambda w: plain.gla(x.double(), gl, w, EPS)))
    for mixer, function in cases:
        for dtype in (F32, BF16):
            part, tensors = random_part("mixer", mixer, dtype, 90, 0.25)
            want = function(lambda name: tensors["l0.mix." + name].double())
            got = run_mixer(part, x, (60,) + (1,) * 400, dtype=dtype)
            close(got[60:], want[60:], dtype, f"{mixer.kind}: 400 rows decoded one by one", tol=2e-4 if dtype == F32 else 3e-2)


# ----------------------------------------------------------------------------------- the pair

PAIRS = [
    (pair(attention(4, 2, 16, 12, 9, 0.35, rot(500.0, 12)), state_space(6, 8, 12, 3, 4, 2), 0.8, 0.5), 4, 50),
    (pair(attention(1, 1, 10, 14, 3, 0.4), state_space(1, 6, 10, 1, 1, 1), -0.6, 1.3), 8, 40),
    (pair(attention(4, 1, 32, 48, 40, 0.18, rot(250000.0, 32)), state_space(4, 32, 64, 2, 3, 4), 1.0, 1.0), 16, 150),
    (pair(attention(2, 2, 16, 16, 20, 0.3, rot(10.0, 6)), state_space(2, 40, 24, 1, 4, 5), 0.0, 0.9), 16, 90),
    (pair(attention(2, 1, 16, 16, 20, 0.3, rot(10.0, 6)), state_space(2, 16, 24, 1, 4, 1), 1.1, 0.0), 16, 90),
]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", range(len(PAIRS)))
def test_a_pair_of_mixers_counts_each_by_its_factor(dtype, case):
    m, page, T = PAIRS[case]
    raw, spec = one_layer("parallel", m)
    mixer_case(spec.layers[0].mixer, lambda x, w: plain.parallel(x, m, w, EPS), dtype, 500 + 20 * case, T, page=page,
               loud=(0, page, m["left"]["mask"]["size"]), std=0.25, tol=2e-4 if dtype == F32 else 3e-2)


# ----------------------------------------------------------------------------------- the feed-forward

ROUTERS = [
    # (experts, top, width, ff, shared)
    (6, 2, 72, 40, 56), (5, 3, 40, 24, 24), (4, 1, 42, 30, None), (7, 7, 96, 48, 64), (9, 3, 80, 40, 72), (2, 2, 64, 16, 8),
    (70, 6, 128, 64, 128), (1, 1, 48, 32, 10), (8, 1, 160, 56, 72),
]


def added(terms):
    """The sum of what a mixture of experts leaves to be added."""
    total = 0.0
    for t in terms:
        if isinstance(t, tuple):
            assert t[1] is None
            total = total + t[0].double().sum(1)
        else:
            total = total + (t.double().sum(0) if t.dim() == 3 else t.double())
    return total


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("case", range(len(ROUTERS)))
def test_the_chosen_sigmoids_weigh_the_experts_inputs(dtype, case):
    experts, top, width, ff, shared = ROUTERS[case]
    mlp = moe(experts, top, ff, shared)
    raw, spec = one_layer("gla", gla(1, 8, 8), mlp, width=width)
    part, tensors = random_part("feed_forward", spec.layers[0].feed_forward, dtype, 300 + 7 * case, width ** -0.5 * 1.5)
    w = lambda name: tensors["l0.mlp." + name].double()
    for rows in (1, 9, 70, 300):
        x = rnd((rows, width), 7 + rows)
        chosen, weights = plain.route(x.double(), top, w("router"))
        ids, found = ops.moe_route(x.to(DEV, dtype), tensors["l0.mlp.router"].to(DEV, dtype), None, top=top, scale=1.0, normalize=False)
        z = x.double() @ w("router").T
        gaps = (z[:, :, None] - z[:, None, :]).abs() + 10.0 * torch.eye(experts)
        clear = gaps.flatten(1).min(1).values > 1e-5      # (the router's sums are 32-bit in both modes, from the same inputs)
        assert clear.sum() >= rows // 2 or rows == 1
        assert torch.equal(ids.cpu().long()[clear], chosen[clear]), "the chosen experts, in the order they were chosen"
        close(found.cpu()[clear], weights[clear], F32, "their weights")
        if bool(clear.all()):
            want = plain.mixture(x.double(), mlp, w)
            close(added(part.forward(x.to(DEV, dtype))), want, dtype, f"the mixture at {rows} rows")


def test_factors_on_the_experts_inputs_in_all_forms():
    """Few rows, many rows, 32-bit; with a gate and without; factors of both signs and zero."""
    for tokens, E, top, N, K in ((1, 3, 2, 40, 64), (33, 4, 2, 72, 264), (64, 5, 1, 130, 40), (65, 2, 2, 16, 24), (300, 3, 1, 200, 64),
                                 (600, 4, 3, 257, 128), (40, 3, 2, 18, 42)):
        x, up, gate_up = rnd((tokens, K), 1), rnd((E, N, K), 2, K ** -0.5), rnd((E, 2 * N, K), 3, K ** -0.5)
        ids = torch.stack([torch.randperm(E, generator=torch.Generator().manual_seed(t))[:top] for t in range(tokens)]).to(torch.int32)
        f = rnd((tokens, top), 4)
        f[0, 0] = 0.0
        pick = lambda w: torch.einsum("tjk,tjnk->tjn", f.double()[:, :, None] * x.double()[:, None, :], w.double()[ids.long()])
        z, u = pick(gate_up), pick(up)
        for dtype in (F32, BF16):
            d = lambda t: t.to(DEV, dtype)
            got = ops.moe_expert(d(x), d(gate_up), ids.to(DEV), ops.MOE_GATE_UP, f.to(DEV))
            close(got.view(tokens, top, N), plain.silu(z[..., :N]) * z[..., N:], dtype, f"gated {tokens}", tol=1e-2 if dtype == BF16 else None)
            got = ops.moe_expert(d(x), d(up), ids.to(DEV), ops.MOE_UP, f.to(DEV))
            close(got.view(tokens, top, N), torch.relu(u) ** 2, dtype, f"up {tokens}", tol=1e-2 if dtype == BF16 else None)


# ----------------------------------------------------------------------------------- what is added, and the loop's entry

@pytest.mark.parametrize("width,rows", [(72, 5), (42, 3), (2560, 300), (1001, 2), (16384, 2)])
def test_terms_go_into_a_view_and_into_a_norm(width, rows):
    res, y, stack, outs, row = rnd((rows, width), 1), rnd((rows, width), 2), rnd((4, rows, width), 3), rnd((rows, 3, width), 4), rnd((width,), 5)
    d = lambda t: t.to(DEV)
    cases = [([], torch.zeros(rows, width)), ([d(y)], y), ([d(stack), ops.EveryRow(d(row))], stack.sum(0) + row),
             ([d(stack), (d(outs), None), d(y)], stack.sum(0) + outs.sum(1) + y), ([ops.EveryRow(d(row))], row.expand(rows, width))]
    w = 1 + rnd((width,), 6, 0.3)
    for terms, total in cases:
        want = res.double() + total.double()
        for dtype in (F32, BF16):
            out = torch.full((rows, 2 * width), 5.0, dtype=dtype, device=DEV)
            held = d(res).clone()
            ops.add_terms_into(held, terms, out[:, width:])
            close(out[:, width:], want, dtype, f"{len(terms)} terms", tol=5e-3 if dtype == BF16 else 1e-6)
            assert bool((out[:, :width] == 5).all()) and torch.equal(held.cpu(), res)
        held = d(res).clone()
        got = ops.group_norm(held, d(w), 1, EPS, F32, terms=terms)
        close(got, plain.unit_rms(want, EPS) * w.double(), F32, f"{len(terms)} terms normed", tol=1e-5)
        close(held, want if terms else res, F32, "the residual", tol=1e-6)


@pytest.mark.parametrize("taps,channels", [(1, 24), (2, 40), (3, 42), (4, 64), (6, 16)])
def test_a_bias_behind_the_convolution(taps, channels):
    """In front of the silu; rows that follow a state and rows of two requests."""
    u, w, b = rnd((11, channels), 1), rnd((channels, taps), 2, 0.6), rnd((channels,), 3)
    state = rnd((3, max(taps - 1, 1), channels), 4)
    slot_of = [2] * 6 + [0] * 5
    want = torch.zeros(11, channels, dtype=torch.float64)
    for slot, rows in ((2, range(0, 6)), (0, range(6, 11))):
        seen = torch.cat([state[slot, :taps - 1], u[rows[0]:rows[-1] + 1]]).double()
        for i, t in enumerate(rows):
            want[t] = plain.silu((seen[i:i + taps] * w.double().T).sum(0) + b.double())
    for dtype in (F32, BF16):
        d = lambda t: t.to(DEV, dtype)
        got = ops.causal_conv(d(u), d(w), d(state) if taps > 1 else None, i32(slot_of), out_bias=d(b), silu=True)
        close(got, want, dtype, f"{taps} taps", tol=1e-2 if dtype == BF16 else 1e-5)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("width,rows", [(72, 5), (42, 3), (96, 70), (2560, 8)])
def test_a_loop_s_entry_joins_the_residual_with_the_kept_input(dtype, width, rows):
    from arle_amd.parts.base import lookup

    times = 3
    spec = PartSpec("joined_input", {"width": width, "times": times}, {"in": "loop.in", "step": "loop.step"})
    part, tensors = random_part("feed_forward", spec, dtype, 5, (2 * width) ** -0.5)
    block = lookup("block", "loop_entry")(None, None, {}, {"join": part})
    x0 = rnd((rows, width), 1)
    batch = type("Batch", (), {"carry": {}})()
    x, delta = block.forward(x0.to(DEV), None, batch, None)
    want = x0.double()
    for t in range(times):
        if t:       # a layer ran in between: it changed the residual in place and left a term
            term = rnd((rows, width), 20 + t)
            x, delta, want = x.clone(), [(term.to(DEV), None)], want + term.double()
        x, left = block.forward(x, delta, batch, None)
        joined = torch.cat([want, x0.double()], dim=1)
        if dtype == BF16:
            joined = joined.to(BF16).double()
        want = joined @ tensors["loop.in"].double().T + tensors["loop.step"].double()[t]
        norm = ops.group_norm(x, torch.ones(width, device=DEV), 1, EPS, F32, terms=[term for term, _ in left])
        close(x, want, dtype, f"pass {t}", tol=1e-2 if dtype == BF16 else 1e-5)
        close(norm, plain.unit_rms(want, EPS), dtype, f"pass {t} normed", tol=1e-2 if dtype == BF16 else 1e-5)
        want = x.double().cpu()
    with pytest.raises(ValueError, match="more often"):
        block.forward(x, None, batch, None)


# ----------------------------------------------------------------------------------- whole models

@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("pozirax")
    # in bfloat16 with routers that choose every expert: rounding a hidden state by a hundredth may decide a close call
    # between experts the other way, and another expert is another function
    return {(name, dtype): make_model_dir(base, name, every_expert=dtype == "bfloat16")
            for name in TINY for dtype in ("float32", "bfloat16")}


def requests_for(cfg, lengths, seed):
    return {f"r{i}": random_tokens(n, cfg["vocab"], seed + i) for i, n in enumerate(lengths)}


def engine_for(folder, name, dtype, tokens, slots=4, **kw):
    return Engine.from_folder(folder, dtype=dtype, page_size=TINY[name][1], max_tokens=tokens, max_slots=slots, **kw)


def references(cfg, weights, reqs):
    return {rid: plain.forward(cfg, weights, toks) for rid, toks in reqs.items()}


MODEL_TOL = {"float32": 5e-5, "bfloat16": 3e-2}


def row_limits(cfg, weights, reqs, ref, dtype, floor=None):
    """What rounding may do to each row: the norms on the recurrences' read-outs magnify the rounding of what lies in front
    where terms nearly cancel, most at a request's first rows.  A row's limit is eight times what the plain logits of
    that row change by when every operand and result of every matrix product is rounded, or moves by up to half a unit in
    the last place, and no less than the usual tolerance."""
    limits = {rid: torch.full((len(toks),), floor or MODEL_TOL[dtype], dtype=torch.float64) for rid, toks in reqs.items()}
    for trial in range(5):
        plain.around_product = rounded_products(F32 if dtype == "float32" else BF16, trial)
        try:
            for rid, toks in reqs.items():
                err = (plain.forward(cfg, weights, toks) - ref[rid]).abs().max(1).values / ref[rid].abs().max()
                limits[rid] = torch.maximum(limits[rid], 8.0 * err)
        finally:
            plain.around_product = None
    return limits


def check(got, ref, limits, dtype, what, floor=None):
    """Every row within its limit, and the median row within the usual tolerance."""
    errors = []
    for rid, want in ref.items():
        scale = float(want.abs().max())
        for p in range(want.shape[0]):
            row = got[(rid, p)].double()
            assert torch.isfinite(row).all(), f"{what}: non-finite logits at {rid}:{p}"
            err = float((row - want[p]).abs().max()) / scale
            errors.append(err)
            assert err <= float(limits[rid][p]), f"{what}: row {rid}:{p} is off by {err:.3e}, its limit is {float(limits[rid][p]):.3e}"
    assert sorted(errors)[len(errors) // 2] <= (floor or MODEL_TOL[dtype]), f"{what}: the median row is off by more than the tolerance"


CASES = [(name, dtype) for name in TINY for dtype in ("float32", "bfloat16")]


@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_prompts_decoding_and_portions_equal_the_plain_logits(folders, name, dtype):
    cfg, weights = read_folder(folders[name, dtype])
    reqs = requests_for(cfg, (1, 2, 23, 61, 130), 100)
    ref = references(cfg, weights, reqs)
    eng = engine_for(folders[name, dtype], name, dtype, 160)
    limits = row_limits(cfg, weights, reqs, ref, dtype)
    for how, make in (("whole", replay.whole), ("decode", lambda r, t: replay.prefill_then_decode(r, t, tail=80)),
                      ("portions", replay.portions), ("pairs", lambda r, t: replay.portions(r, t, sizes=(2,))),
                      ("chunk borders", lambda r, t: replay.portions(r, t, sizes=(63, 2, 64))),
                      ("single tokens", lambda r, t: replay.portions(r, t, sizes=(1,)))):
        got = {}
        for rid, toks in reqs.items():
            got.update(replay.run_steps(eng, make(rid, toks)))
        check(got, ref, limits, dtype, f"pozirax {name} {dtype} {how}")
        assert eng.cache.free_tokens() == eng.cache.pool_tokens()


@pytest.mark.parametrize("name,dtype", CASES)
def test_mixed_batches_with_pages_and_slots_used_again(folders, name, dtype):
    cfg, weights = read_folder(folders[name, dtype])
    reqs = requests_for(cfg, (40, 7, 75, 2, 33, 58, 19, 90), 210)
    ref = references(cfg, weights, reqs)
    # three slots and a pool that just holds the three longest live requests: every slot and page is used again
    eng = engine_for(folders[name, dtype], name, dtype, 90 + 75 + 58 + 3 * TINY[name][1], slots=3)
    alone = engine_for(folders[name, dtype], name, dtype, 128, slots=1)
    limits = row_limits(cfg, weights, reqs, ref, dtype)
    for seed, portion in ((1, 17), (2, 40)):
        steps = replay.mixed(reqs, max_live=3, seed=seed, decode_tail=12, max_portion=portion)
        got = replay.run_steps(eng, steps)
        check(got, ref, limits, dtype, f"pozirax {name} {dtype} mixed {seed}")
        assert eng.cache.free_slot_count == 3 and eng.cache.free_tokens() == eng.cache.pool_tokens()
    if dtype == "float32":      # in 32 bits a row is the same bits in a batch and alone
        for rid in ("r0", "r3", "r5"):
            solo = replay.run_steps(alone, replay.whole(rid, reqs[rid]))
            for key, row in solo.items():
                assert torch.equal(row, got[key]), f"{key} differs between the batch and the request alone"


def test_a_long_prompt_and_long_decoding_stay_with_the_plain_logits(folders):
    for name, dtype in (("P", "float32"), ("R", "float32"), ("R", "bfloat16")):
        cfg, weights = read_folder(folders[name, dtype])
        toks = random_tokens(450, cfg["vocab"], 31)
        ref = {"a": plain.forward(cfg, weights, toks)}
        eng = engine_for(folders[name, dtype], name, dtype, 480)
        got = replay.run_steps(eng, replay.prefill_then_decode("a", toks, tail=280))
        floor = 1e-4 if dtype == "float32" else None      # a thousand steps of a 32-bit recurrence
        check(got, ref, row_limits(cfg, weights, {"a": toks}, ref, dtype, floor), dtype, f"long {name} {dtype}", floor)


@pytest.mark.parametrize("name", ["P", "R"])
def test_captured_steps_give_the_bits_of_eager_ones(folders, name):
    folder = folders[name, "bfloat16"]
    cfg, _ = read_folder(folder)
    reqs = requests_for(cfg, (54, 54, 71), 300)
    steps = []
    for rid, toks in reqs.items():      # equal portions, then decoding: shapes repeat and are captured
        steps += [{"entries": [(rid, toks[i:i + 24], list(range(len(toks[i:i + 24]))))], "end": []} for i in range(0, 48, 24)]
    live = list(reqs)
    for i in range(48, 54):
        steps.append({"entries": [(rid, reqs[rid][i:i + 1], [0]) for rid in live], "end": live if i == 53 else []})
    out = {}
    for graphs in (False, True):
        eng = engine_for(folder, name, "bfloat16", 240, cuda_graph=graphs)
        out[graphs] = replay.run_steps(eng, steps)
        assert (eng.graph_replays > 0) == graphs
    assert all(torch.equal(out[True][k], out[False][k]) for k in out[False])


def _plain_greedy(cfg, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(plain.forward(cfg, weights, toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("name", ["P", "Q"])
def test_greedy_generation_through_the_scheduler_equals_the_plain_implementation(folders, name):
    folder = folders[name, "float32"]
    cfg, weights = read_folder(folder)
    prompts = [random_tokens(n, cfg["vocab"], 400 + n) for n in (3, 12, 29, 18, 7)]
    want = [_plain_greedy(cfg, weights, p, 24) for p in prompts]
    # two slots for five requests, portions of at most eight tokens: slots and pages are used again
    llm = LLM(folder, dtype="float32", page_size=TINY[name][1], kv_cache_tokens=160, max_seq_len=64, num_slots=2,
              chunked_prefill_size=8)
    outs = llm.generate(prompts, max_tokens=24)
    assert [o.response_token_ids for o in outs] == want
    assert all(o.finish_reason == "length" for o in outs)
