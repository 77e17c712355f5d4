"""Fikevik models on the GPU through the framework's entry points, against the plain implementation: whole prompts, portions, batches,
cells and states that are given back and used again, window edges, long decoding, greedy generation through the scheduler and the captured loop."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_fikevik as o
from fikevik_models import attention, config, dense, even_config, gla, memory, odd_config, parallel, tall_config, weights
from lerasun_models import row_errors, tokens
from powerinfer_amd import checkpoint, fikevik, lib as pl, registry, serve

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
MODELS = {"even": even_config, "odd": odd_config, "tall": tall_config}
CASES = [(m, c) for m in MODELS.values() for c in (pl.BF16, pl.F32)]
IDS = [f"{n}-{c}" for n in MODELS for c in ("bf16", "f32")]


class Shaken(o.PlainModel):
    """The plain model with every sublayer's input off by up to 2^-7 of itself, two places in bf16: how much rounding moves a position.  (The first
    tokens' recurrences are a product of one query and one key over its own size, of which little more than a sign is left.)"""

    def __init__(self, cfg, w, seed):
        super().__init__(cfg, w)
        self.rng = np.random.default_rng(seed)

    def operand(self, x):
        return x * (1 + self.rng.uniform(-2.0 ** -7, 2.0 ** -7, x.shape))


class Oracle:
    """Logits, streams and what rounding does to them, of token sequences, one plain model per call."""
    cache = {}

    def __init__(self, make):
        self.make, self.cfg = make, make()
        self.w = weights(self.cfg, 17)

    def run(self, toks):
        key = (self.make.__name__, tuple(toks))
        if key not in Oracle.cache:
            p = o.PlainModel(self.cfg, self.w)
            want, streams = p.feed(toks), p.streams
            moved, n = np.zeros(len(toks)), min(len(toks), 20)           # the first tokens
            for seed in range(12):
                d = Shaken(self.cfg, self.w, seed).feed(toks[:n]) - want[:n]
                d -= d.mean(axis=1, keepdims=True)
                moved[:n] = np.maximum(moved[:n], np.sqrt((d ** 2).mean(axis=1)) / want.std())
            Oracle.cache[key] = (want, streams, moved)
        return Oracle.cache[key]

    def logits(self, toks):
        return self.run(toks)[0]


def model(orc, compute, n_ctx=512, max_batch=0):
    return fikevik.build(orc.cfg, orc.w, compute=compute, n_ctx=n_ctx, max_batch=max_batch)


def check(got, orc, toks, compute, rows=slice(None)):
    """Rows of the logits of `toks`."""
    want, _, moved = orc.run(toks)
    want, moved = want[rows], moved[rows]
    assert got.shape == want.shape
    e = row_errors(got, want)
    limit = np.maximum(2e-5, 2.0 ** -11 * moved) if compute == pl.F32 else np.maximum(0.06, 2 * moved)
    late = e[moved == 0]
    assert (e < (1 if compute == pl.F32 else 1.5) * limit).all() and (e > limit).mean() <= 0.01 and (compute == pl.F32 or late.size == 0 or np.median(late) < 0.02), (np.median(e), (e / limit).max(), int((e / limit).argmax()))


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_whole_prompts_and_streams(make, compute):
    orc = Oracle(make)
    m = model(orc, compute)
    m.set_capture(True)
    st = serve.Stepper(m, 400)
    for n, rid in ((1, "a"), (2, "b"), (17, "c"), (64, "e"), (65, "f"), (170, "d")):
        toks = tokens(orc.cfg, n, n)
        got, _ = st.run([(rid, toks, list(range(n)))])
        check(got, orc, toks, compute)
        s, want = m.get_streams(), orc.run(toks)[1]
        assert s.shape == (len(want), n, orc.cfg["width"])
        e = np.max([np.abs(a - b).max(axis=1) / np.abs(b).max() for a, b in zip(s, want)], axis=0)
        assert (e < np.maximum(1e-5, 2.0 ** -11 * orc.run(toks)[2]) if compute == pl.F32 else e < np.maximum(0.1, 3 * orc.run(toks)[2])).all()
        st.end(rid)
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
@pytest.mark.parametrize("cut", ["ones", "twos", "mixed", "tail"])
def test_portions(make, compute, cut):
    """The same prompt token by token, two at a time, in portions of changing size, and as one portion with a decoded tail."""
    orc = Oracle(make)
    n = 150
    toks = tokens(orc.cfg, n, 5)
    sizes = {"ones": [1] * n, "twos": [2] * (n // 2), "mixed": [2, 3, 31, 1, 17, 16, 2, 64, 1, 13], "tail": [n - 12] + [1] * 12}[cut]
    assert sum(sizes) == n
    m = model(orc, compute)
    st = serve.Stepper(m, n)
    got, at = [], 0
    for k in sizes:
        got.append(st.run([("r", toks[at:at + k], list(range(k)))])[0])
        at += k
    check(np.vstack(got), orc, toks, compute)
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_mixed_batches_against_each_alone(make, compute):
    """Four requests of unequal length, portions beside single tokens, some left out of a step, ends at different times, and two more
    requests on the cells, states and sequences the first ones gave back - in a pool that holds exactly what is live."""
    orc = Oracle(make)
    lens = {"a": 140, "b": 3, "c": 66, "d": 90, "e": 75, "f": 120}
    toks = {k: tokens(orc.cfg, n, ord(k)) for k, n in lens.items()}
    plan = [{"a": 70, "b": 1}, {"a": 2, "c": 16, "b": 1, "d": 1}, {"d": 70, "c": 1}, {"a": 1, "b": 1, "c": 33, "d": 1}, {"a": 66, "c": 16, "e": 2},
            {"a": 1, "d": 17, "e": 70}, {"f": 100, "d": 1, "e": 3}, {"f": 20}]
    at, live, peak = {k: 0 for k in lens}, {}, 0
    for step in plan:                                   # what the pool has to hold
        for k, n in step.items():
            live[k] = live.get(k, 0) + n
        peak = max(peak, sum(live.values()))
        live = {k: n for k, n in live.items() if n < lens[k]}
    m = model(orc, compute)
    st = serve.Stepper(m, peak, max_live=4)
    got = {k: [] for k in lens}
    for step in plan:
        lg, _ = st.run([(k, toks[k][at[k]:at[k] + n], list(range(n))) for k, n in step.items()])
        row = 0
        for k, n in step.items():
            got[k].append(lg[row:row + n])
            row += n
            at[k] += n
            if at[k] == lens[k]:
                st.end(k)
    assert at == lens and st.free_cells == peak
    for k in lens:
        check(np.vstack(got[k]), orc, toks[k], compute)
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_many_requests_on_slots_used_again(compute):
    """More live requests than the states there is room for at the start, then fewer, then others in their places, in steps of 16 and more."""
    orc = Oracle(odd_config)
    m = model(orc, compute)
    st = serve.Stepper(m, 400, max_live=20)
    t = {i: tokens(orc.cfg, 12, 200 + i) for i in range(30)}
    got = {i: [] for i in t}

    def step(ids, a, b):
        lg, _ = st.run([(i, t[i][a:b], list(range(b - a))) for i in ids])
        for k, i in enumerate(ids):
            got[i].append(lg[k * (b - a):(k + 1) * (b - a)])

    step(range(3), 0, 5)
    step(range(3, 20), 0, 5)                            # the states are moved to a larger place while three requests hold some
    step(range(0, 20), 5, 6)
    for i in range(0, 20, 2):
        st.end(i)
    step(range(20, 30), 0, 6)                           # in the places of the ended ones
    step(list(range(1, 20, 2)) + list(range(20, 30)), 6, 12)
    for i in range(0, 20, 2):
        check(np.vstack(got[i]), orc, t[i][:6], compute)
    for i in list(range(1, 20, 2)) + list(range(20, 30)):
        check(np.vstack(got[i]), orc, t[i], compute)
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_fragmented_pool(compute):
    """Requests that grow token by token side by side, so that every sequence's cells are scattered, then holes taken by a long prompt."""
    orc = Oracle(even_config)
    m = model(orc, compute)
    st = serve.Stepper(m, 160, max_live=4)
    t = {k: tokens(orc.cfg, 40, i) for i, k in enumerate("wxyz")}
    for i in range(40):
        st.run([(k, [t[k][i]], []) for k in "wxyz"], logits=False)
    st.end("x")
    st.end("z")
    long = tokens(orc.cfg, 80, 9)
    got, _ = st.run([("n", long, list(range(80)))])
    check(got, orc, long, compute)
    more = tokens(orc.cfg, 3, 8)
    st.end("y")
    got, _ = st.run([("w", more, [0, 1, 2])])
    check(got, orc, t["w"] + more, compute, slice(-3, None))
    with pytest.raises(pl.PiError, match="free cells"):
        st.m.kv_cells_step([1] * 50, range(50), [1 << 9] * 50, [49])
    st.end("n")                                         # the refused step has left nothing behind
    assert (st.m.kv_cells_state()[0] >= 0).sum() == 43
    got, _ = st.run([("w", more, [2])])
    check(got, orc, t["w"] + more + more, compute, slice(-1, None))
    m.close()


@pytest.mark.parametrize("make,compute", CASES[:4], ids=IDS[:4])
def test_long_steps_run_in_passes(make, compute):
    orc = Oracle(make)
    m = model(orc, compute, max_batch=48)
    st = serve.Stepper(m, 300)
    a, b = tokens(orc.cfg, 130, 1), tokens(orc.cfg, 61, 2)
    got, _ = st.run([("a", a, list(range(130))), ("b", b, list(range(61)))])
    check(got[:130], orc, a, compute)
    check(got[130:], orc, b, compute)
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_a_decoded_token_beside_a_long_prompt(make, compute):
    """A token far into its sequence in one batch with a long run, and the other way round."""
    orc = Oracle(make)
    m = model(orc, compute, n_ctx=1024)
    st = serve.Stepper(m, 760)
    a, b = tokens(orc.cfg, 340, 1), tokens(orc.cfg, 400, 2)
    st.run([("a", a[:330], [])])
    got, _ = st.run([("a", a[330:331], [0]), ("b", b[:399], list(range(399)))])
    check(got[:1], orc, a, compute, slice(330, 331))
    check(got[1:], orc, b, compute, slice(0, 399))
    got, _ = st.run([("b", b[399:], [0]), ("a", a[331:], list(range(9)))])
    check(got[:1], orc, b, compute, slice(399, None))
    check(got[1:], orc, a, compute, slice(331, None))
    m.close()


def looking_model(window, kv_heads=1):
    """One layer whose attention makes token 32 + k look for token 42 + k and for nothing else; the memory beside it is all but shut out."""
    rng = np.random.default_rng(0)
    cfg = config(64, 64, [parallel(attention(2, kv_heads, 64, 48, window, rot=0, scale=0.5), memory(1, 8, 8), 1.0, 1e-3)], scale=1.0, alpha=0.1)
    w = weights(cfg, 3)
    bf = lambda a: checkpoint.bf16_floats(checkpoint.bf16_bits(a)).reshape(a.shape)  # noqa: E731
    emb = np.linalg.qr(rng.standard_normal((64, 64)))[0].T
    look = sum(np.outer(emb[42 + k], emb[32 + k]) for k in range(12)) + 0.05 * np.eye(64)
    code = np.linalg.qr(rng.standard_normal((64, 64)))[0]
    w["embed"] = bf(emb.astype(np.float32))
    w["l0.mix.left.k"], w["l0.mix.left.q"] = bf(np.concatenate([code] * kv_heads)), bf(np.concatenate([code @ look] * 2))
    for x in ("q.norm", "k.norm", "temp"):
        w["l0.mix.left." + x] = np.ones_like(w["l0.mix.left." + x])
    w["l0.rg1.b"] += 2
    return cfg, w


@pytest.mark.parametrize("window", [63, 64, 65, 130])
def test_window_edges_in_prompts_and_decoding(window):
    """Keys just inside and just outside the window, at edges of tiles of cells, the first position, and the token's own place: each decides the
    result where it is seen and changes nothing where it is not."""
    cfg, w = looking_model(window)
    rng, n = np.random.default_rng(window), 330
    toks = [int(v) for v in rng.integers(1, 32, n)]
    far, inside, outside = window - 1, [], []
    # (key place, asking place): the last ones are decoded singly below
    pairs = [(0, far), (95, 95 + far), (96, 96 + far + 1), (n - 4 - far, n - 4), (n - 2 - far - 1, n - 2), (n - 1 - far, n - 1), (140, 141)]
    assert len({x for p in pairs for x in p}) == 14
    for k, (key, ask) in enumerate(pairs):
        toks[key], toks[ask] = 42 + k, 32 + k
        (inside if ask - key <= far else outside).append((k, key, ask))
    assert len(inside) == 5 and len(outside) == 2
    want = o.PlainModel(cfg, w).feed(toks)
    for pairs, seen in ((inside, True), (outside, False)):
        for k, key, ask in pairs:
            blind = list(toks)
            blind[key] = 3
            e = row_errors(o.PlainModel(cfg, w).feed(blind)[ask:ask + 1], want[ask:ask + 1])[0]
            assert (e > 0.2) == seen and (seen or e < 0.01), (key, ask, e)         # (what is not seen still is in the memory)
    for compute, limit in ((pl.F32, 2e-5), (pl.BF16, 0.05)):
        for sizes in ([n], [n - 12] + [1] * 12, [64] * 5 + [10], [99, 2, 2] + [1] * 227, [17] * 19 + [7]):
            m = fikevik.build(cfg, w, compute=compute)
            st = serve.Stepper(m, 352)
            got, at = [], 0
            for k in sizes:
                got.append(st.run([("r", toks[at:at + k], list(range(k)))])[0])
                at += k
            e = row_errors(np.vstack(got), want)
            assert e.max() < limit, (compute, sizes[:2], e.max(), int(e.argmax()))
            m.close()


def test_windows_follow_positions():
    """Positions with gaps: a window counts positions, not cells."""
    cfg, w = looking_model(20)
    toks = [int(v) for v in np.random.default_rng(1).integers(1, 32, 40)]
    pos = list(range(0, 10)) + list(range(15, 25)) + list(range(40, 60))
    for k, (key, ask) in enumerate([(5, 14), (4, 15), (16, 21), (20, 39), (8, 18)]):        # distances 14, 16, 20 (unseen), 19, 15
        toks[key], toks[ask] = 42 + k, 32 + k
    assert pos[21] - pos[16] == 20 and pos[39] - pos[20] == 19
    p = o.PlainModel(cfg, w)
    t = {k[3:]: v for k, v in p.t.items() if k.startswith("l0.")}
    x = p.t["embed"][toks]
    a, r = cfg["layers"][0]["mixer"]["left"], cfg["layers"][0]["mixer"]["right"]
    q, k, v = o.queries_and_cells(x, np.asarray(pos), {n[9:]: y for n, y in t.items() if n.startswith("mix.left.")}, a, 1e-5)
    left = o.window_attention(q, k, v, pos, pos, o.head_scale(t["mix.left.temp"], 0.5), 20).reshape(40, -1) @ t["mix.left.o"].T
    right, _ = o.matrix_memory(x, {n[10:]: y for n, y in t.items() if n.startswith("mix.right.")}, r, 1e-5, o.empty_memory(r))
    y = o.gated(o.side_by_side(left, right, cfg["layers"][0]["mixer"]), x, t["rg1"], t["rg1.b"])
    want = o.rms_norm(o.norm_after_sum(x, y, cfg["postln_alpha"], t["norm1"], 1e-5), p.t["final.norm"], 1e-5) @ p.t["head"].T
    for compute, limit in ((pl.F32, 2e-5), (pl.BF16, 0.05)):
        for sizes in ([40], [11, 29], [1] * 40):
            m = fikevik.build(cfg, w, compute=compute)
            m.kv_cells_init(64)
            got, at = [], 0
            for n in sizes:
                got.append(m.kv_cells_step(toks[at:at + n], pos[at:at + n], [1] * n, range(n))[1])
                at += n
            assert row_errors(np.vstack(got), want).max() < limit, (compute, sizes[:2])
            m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_first_tokens(compute):
    """Every start of a sequence, alone and beside others that have begun already."""
    orc = Oracle(even_config)
    m = model(orc, compute)
    st = serve.Stepper(m, 400, max_live=8)
    old = tokens(orc.cfg, 60, 1)
    st.run([("old", old[:50], [])])
    for n in (1, 2, 3, 5, 16, 17):
        t = tokens(orc.cfg, n, 70 + n)
        got, _ = st.run([("old", old[50:51], []), (n, t, list(range(n)))])
        check(got, orc, t, compute)
        st.end(n)
        st.end("old")
        st.run([("old", old[:50], [])])
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_small_variants_of_the_configuration(compute):
    """One layer of one kind only, sizes of one, no feed-forward at all, layers that share weights with others in between, widths below and
    beyond a kernel's step, factors of the sums that are one, zero or negative."""
    a, b = parallel(attention(2, 2, 24, 16, 9, rot=10), memory(1, 16, 16)), gla(2, 16, 16, mlp=dense(40))
    one = parallel(attention(1, 1, 2, 1, 5, rot=2), memory(1, 1, 1, cap=1.0), 1.0, 1.0)
    for width, layers, kw in ((72, [a], {}), (72, [b], {}), (40, [one, gla(1, 1, 1, tau=1.0)], dict(alpha=1.0, scale=1.0)), (300, [a, b, dict(a, weights_of=0), a, dict(b, weights_of=1)], {}),
                              (1100, [b, dict(b, weights_of=0)], dict(eps=1e-2)), (24, [dict(b, weights_of=1), b], dict(alpha=-0.5)), (33, [a, gla(3, 7, 5)], dict(alpha=0.0)),
                              (64, [parallel(attention(4, 1, 32, 64, 1000), memory(2, 8, 24), 0.0, 1.0), parallel(attention(4, 4, 8, 8, 3), memory(2, 8, 24), -1.0, 0.0)], {})):
        cfg = config(width, 60, layers, **kw)
        w = weights(cfg, 8)
        toks = tokens(cfg, 90, 3)
        want = o.PlainModel(cfg, w).feed(toks)
        m = fikevik.build(cfg, w, compute=compute)
        st = serve.Stepper(m, 200)
        got = np.vstack([st.run([("r", toks[i:j], list(range(j - i)))])[0] for i, j in ((0, 70), (70, 79), (79, 80), (80, 90))])
        e = row_errors(got, want)
        # (with the residual's factor 0 or a width below 40 little averages out)
        assert e.max() < (5e-5 if compute == pl.F32 else 0.1), (width, len(layers), np.sort(e)[-5:])
        m.close()


def greedy(orc, prompt, n):
    """Greedy continuation of the oracle with the gap between the best two logits at every step."""
    p = o.PlainModel(orc.cfg, orc.w)
    lg, out, gaps = p.feed(prompt)[-1], [], []
    for _ in range(n):
        s = np.sort(lg)
        out.append(int(lg.argmax()))
        gaps.append((s[-1] - s[-2]) / lg.std())
        lg = p.feed(out[-1:])[-1]
    return out, gaps


@pytest.mark.parametrize("make", MODELS.values(), ids=MODELS)
def test_greedy_generation_through_the_scheduler(make):
    """fp32: the scheduler's tokens are the oracle's, in a pool that makes requests wait for each other and prompts arrive in portions."""
    orc = Oracle(make)
    prompts = [tokens(orc.cfg, n, 40 + n) for n in (1, 7, 40, 90, 3, 21)]
    want = [greedy(orc, p, 10) for p in prompts]
    assert min(min(g) for _, g in want) > 1e-4, "a tie in the test's own model"
    m = model(orc, pl.F32)
    got = serve.generate(m, prompts, 10, n_cells=128, max_live=3, budget=24)
    assert got == [w for w, _ in want]
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_long_decoding_in_the_captured_loop(make, compute):
    """pi_model_decode + pi_model_generate (one captured step replayed, several calls) against token-by-token steps and, position by
    position, the oracle."""
    orc = Oracle(make)
    m = model(orc, compute, n_ctx=320)
    prompt = tokens(orc.cfg, 37, 77)
    first, lg = m.decode(prompt, 0)
    check(lg[None], orc, prompt, compute, slice(-1, None))
    out = [first] + [int(v) for n in (3, 120, 77) for v in m.generate(n)[0]]
    assert len(out) == 201
    full = orc.logits(prompt + out[:-1])[len(prompt) - 1:]
    if compute == pl.F32:
        assert [int(v) for v in full.argmax(axis=1)] == out
    else:                                               # every chosen token is within rounding of the best one
        short = (full.max(axis=1) - full[np.arange(201), out]) / full.std()
        assert short.max() < 0.1, np.sort(short)[-8:]
    again, lg2 = m.decode(out[-1:], len(prompt) + 200)  # and the cache and states it left are the right ones
    check(lg2[None], orc, prompt + out, compute, slice(-1, None))
    with pytest.raises(pl.PiError, match="go back"):    # a recurrent state has no earlier positions
        m.decode([1], len(prompt))
    m.kv_clear()
    assert m.decode(prompt, 0)[0] == first
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_lockstep_batches(compute):
    """batch_init / batch_decode / batch_generate: five sequences, each as if it were alone; a prefix handed on with its states."""
    orc = Oracle(even_config)
    m = model(orc, compute, n_ctx=128)
    m.batch_init(5)
    toks = [tokens(orc.cfg, 30, 60 + s) for s in range(5)]
    rows = []
    for p in range(30):
        nxt, lg = m.batch_decode([t[p] for t in toks], [p] * 5)
        rows.append(lg)
    for s in range(5):
        check(np.stack([r[s] for r in rows]), orc, toks[s], compute)
    out, _ = m.batch_generate(40)
    assert out.shape == (40, 5)
    for s in range(5):
        seq = [int(nxt[s])] + [int(v) for v in out[:, s]]
        full = orc.logits(toks[s] + seq[:-1])[29:]
        short = (full.max(axis=1) - full[np.arange(41), seq]) / full.std()
        assert short.max() < (1e-4 if compute == pl.F32 else 0.1)
    assert m.batch_kv_seq_rm(0, 0, -1) == 0
    with pytest.raises(pl.PiError, match="recurrent"):
        m.batch_kv_seq_cp(1, 0, 0, 30)                  # a part of a sequence
    assert m.batch_kv_seq_cp(1, 0, 0, -1) == 70
    nxt, lg = m.batch_decode([3] * 5, [70] * 5)
    check(lg[:1], orc, toks[1] + [int(rows[-1][1].argmax())] + [int(v) for v in out[:-1, 1]] + [3], compute, slice(-1, None))
    assert np.abs(lg[0] - lg[1]).max() < 1e-5 * np.abs(lg[1]).max()
    m.close()


def test_sequences_with_states_are_whole_or_empty():
    """kv_cells_*: a sequence's cells and states are handed to another one and go on separately; what would take part of a state apart is
    refused and changes nothing."""
    orc = Oracle(odd_config)
    m = model(orc, pl.F32)
    m.kv_cells_init(100)
    p, a, b = tokens(orc.cfg, 50, 1), tokens(orc.cfg, 9, 2), tokens(orc.cfg, 9, 3)
    m.kv_cells_step(p, range(50), [1] * 50, [])
    m.kv_cells_seq_cp(0, 1, 0, -1)
    for refused in (lambda: m.kv_cells_seq_rm(0, 10, 20), lambda: m.kv_cells_seq_shift(0, 0, -1, 4), lambda: m.kv_cells_seq_cp(0, 2, 0, 30), lambda: m.kv_cells_seq_cp(0, 1, 0, -1),
                    lambda: m.kv_cells_step([3], [50], [3], [0]), lambda: m.kv_cells_step([3], [20], [1], [0]), lambda: m.kv_cells_step([3, 4, 5], [50, 50, 51], [1, 2, 1], [0])):
        with pytest.raises(pl.PiError, match="recurrent|follow"):
            refused()
    _, lg = m.kv_cells_step(a + b, list(range(50, 59)) * 2, [1] * 9 + [2] * 9, range(18))
    check(lg[:9], orc, p + a, pl.F32, slice(50, None))
    check(lg[9:], orc, p + b, pl.F32, slice(50, None))
    m.kv_cells_seq_rm(0, -1, -1)
    _, lg = m.kv_cells_step([5], [59], [2], [0])
    check(lg, orc, p + b + [5], pl.F32, slice(-1, None))
    m.kv_cells_seq_keep(1)
    _, lg = m.kv_cells_step([7], [0], [1], [0])
    check(lg, orc, [7], pl.F32)
    m.close()


def save(folder, cfg, w):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    checkpoint.write_safetensors(os.path.join(folder, "model.safetensors"), {k: checkpoint.bf16_bits(v) for k, v in w.items()})


def test_files_and_trace_replay_and_command_line(tmp_path):
    orc = Oracle(odd_config)
    folder = str(tmp_path / "m")
    save(folder, orc.cfg, orc.w)
    m = registry.load_model(folder, "float32", n_ctx=128)
    toks = tokens(orc.cfg, 20, 4)
    check(m.decode(toks, 0)[1][None], orc, toks, pl.F32, slice(-1, None))
    m.close()
    steps = [{"step": 0, "entries": [{"id": "p", "tokens": toks[:11], "want": [0, 10]}, {"id": "q", "tokens": toks[:2], "want": []}], "end": ["q"]},
             {"step": 1, "entries": [{"id": "p", "tokens": toks[11:12], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "r", "tokens": toks[:3], "want": [2]}, {"id": "p", "tokens": toks[12:], "want": [7]}], "end": ["p", "r"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"], r.stderr[-800:]
    full, v = orc.logits(toks), orc.cfg["vocab"]
    for name, rows in (("0.f32", [0, 10]), ("2.f32", [2, 19])):
        assert row_errors(np.fromfile(tmp_path / name, "<f4").reshape(2, v), full[rows]).max() < 2e-5
    assert not (tmp_path / "1.f32").exists()
    r = subprocess.run([sys.executable, "-m", "powerinfer_amd", "generate", "--model", folder, "--dtype", "float32", "--prompt", ",".join(map(str, toks)), "--new", "5"],
                       cwd=ROOT, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-800:]
    assert [int(t) for t in r.stdout.split()[-1].split(",")] == greedy(orc, toks, 5)[0]


def test_bad_models_are_refused():
    cfg = odd_config()
    w = weights(cfg, 1)
    for name, why in (("l1.mix.a2", "mix_a2"), ("l0.mix.right.i", "mem_i"), ("l0.rg2", "res_gate_ffn"), ("l3.mix.left.temp", "mix_temp")):
        bad = dict(w)
        bad[name] = w[name][:-1]
        with pytest.raises(pl.PiError, match=why):
            fikevik.build(cfg, bad)
    for spoil, why in ((lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=4), "grouped-query"), (lambda c: c["layers"][1]["mixer"].update(tau=0.0), "key decays"),
                       (lambda c: c["layers"][0]["mixer"]["right"].update(gate_cap=0.0), "memory"), (lambda c: c["layers"][3]["mixer"]["left"]["rot"].update(dims=18), "grouped-query"),
                       (lambda c: c["layers"][4].update(weights_of=1), "weights_of")):
        c = odd_config()
        spoil(c)
        with pytest.raises(pl.PiError, match=why):
            fikevik.build(c, w)
