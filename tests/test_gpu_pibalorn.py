"""Pibalorn models on the GPU through the framework's entry points, against the plain implementation: whole prompts, portions, batches,
cells and states that are given back and used again, long decoding, greedy generation through the scheduler and the captured loop."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_pibalorn as o
from lerasun_models import row_errors, tokens
from pibalorn_models import attention, config, dense, even_config, lightning, moe, odd_config, tall_config, weights
from powerinfer_amd import checkpoint, lib as pl, pibalorn, registry, serve

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CASES = [(m, c) for m in (even_config, odd_config, tall_config) for c in (pl.BF16, pl.F32)]
IDS = [f"{n}-{c}" for n in ("even", "odd", "tall") for c in ("bf16", "f32")]


class Oracle:
    """Logits and routing margins of token sequences, one plain model per call."""
    cache = {}

    def __init__(self, make):
        self.make, self.cfg = make, make()
        self.w = weights(self.cfg, 17)

    def run(self, toks):
        key = (self.make.__name__, tuple(toks))
        if key not in Oracle.cache:
            p = o.PlainModel(self.cfg, self.w)
            Oracle.cache[key] = (p.feed(toks), p.margins, p.streams)
        return Oracle.cache[key]

    def logits(self, toks):
        return self.run(toks)[0]


def model(orc, compute, n_ctx=512, max_batch=0):
    return pibalorn.build(orc.cfg, orc.w, compute=compute, n_ctx=n_ctx, max_batch=max_batch)


def check(got, orc, toks, compute, rows=slice(None)):
    """Rows of the logits of `toks`.  fp32: every position.  bf16: the positions whose routing decisions were not close calls (those may fall
    the other way, and a token that looks at such a token hears of it)."""
    want, margins, _ = orc.run(toks)
    want, margins = want[rows], margins[rows]
    assert got.shape == want.shape
    e = row_errors(got, want)
    if compute == pl.F32:
        assert e.max() < 2e-5, (e.max(), int(e.argmax()))
    else:
        e = e[margins > 0.03]
        assert e.size == 0 or (np.median(e) < 0.025 and (e > 0.06).mean() <= 0.08 and (e > 0.12).mean() <= 0.03), (np.median(e), np.sort(e)[-5:], np.argsort(e)[-5:])


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
        if compute == pl.F32:
            s, want = m.get_streams(), orc.run(toks)[2]
            assert s.shape == (len(want), n, orc.cfg["width"])
            assert max(np.abs(a - b).max() / np.abs(b).max() for a, b in zip(s, want)) < 1e-5
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
    orc = Oracle(even_config)
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
    """A token far into its sequence (its cells split over workgroups) in one batch with a long run."""
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


def test_far_keys_in_prompts_and_decoding():
    """One layer in which token 32 + k looks for token 42 + k and for nothing else: that key decides the result hundreds of tokens back, at
    the first positions, at edges of tiles of cells - and not at all one position before it appears."""
    rng = np.random.default_rng(0)
    cfg = config(64, 64, [attention(2, 1, 64, rot=2, base=1e12, scale=0.5)], scale=1.0, bigram=(5, 1, 1))
    w = weights(cfg, 3)
    bf = lambda a: checkpoint.bf16_floats(checkpoint.bf16_bits(a)).reshape(a.shape)  # noqa: E731
    basis = np.linalg.qr(np.concatenate([np.ones((64, 1)), rng.standard_normal((64, 63))], 1))[0].T[1:]       # rows without a mean
    emb = np.concatenate([basis, -basis[:1]]).astype(np.float32)
    w["embed"], w["bigram"], w["l0.norm1"] = bf(emb), np.zeros((6, 64), np.float32), np.ones(64, np.float32)
    look = sum(np.outer(emb[42 + k], emb[32 + k]) for k in range(10)) + np.outer(emb[62], emb[61]) + 0.05 * np.eye(64)
    code = np.linalg.qr(rng.standard_normal((64, 64)))[0]
    w["l0.mix.k"], w["l0.mix.q"] = bf(code), bf(np.concatenate([code @ look] * 2))
    n = 330
    toks = [int(v) for v in rng.integers(1, 32, n)]
    for k, p in enumerate([0, 1, 31, 32, 63, 64, 127, 128, 255, 256]):
        toks[p], toks[n - 12 + k] = 42 + k, 32 + k
    toks[100], toks[99], toks[101], toks[200] = 62, 61, 61, 61
    want = o.PlainModel(cfg, w).feed(toks)
    for key, asks, seen in ((0, n - 12, True), (256, n - 3, True), (100, 99, False), (100, 101, True), (100, 200, True)):
        blind = list(toks)
        blind[key] = 3
        e = row_errors(o.PlainModel(cfg, w).feed(blind)[asks:asks + 1], want[asks:asks + 1])[0]
        assert (e > 0.2) == seen and (seen or e == 0), (key, asks, e)        # the far key does decide
    for compute, limit in ((pl.F32, 2e-5), (pl.BF16, 0.05)):
        for sizes in ([n], [n - 12] + [1] * 12, [64] * 5 + [10], [99, 2, 2] + [1] * 227):
            m = pibalorn.build(cfg, w, compute=compute)
            st = serve.Stepper(m, 352)
            got, at = [], 0
            for k in sizes:
                got.append(st.run([("r", toks[at:at + k], list(range(k)))])[0])
                at += k
            e = row_errors(np.vstack(got), want)
            assert e.max() < limit, (compute, sizes[:2], e.max(), int(e.argmax()))
            m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_small_variants_of_the_configuration(compute):
    """What the other configurations do not have: no bigram table, no loop, a loop that runs once, one layer of one kind only, a layer
    without feed-forward, more choices per token than the fused step takes."""
    a, b = attention(2, 2, 24, rot=10, mlp=dense(40)), lightning(2, 16, 16, (0.9, 1.0), mlp=moe(20, 17, 8, shared=(24, 0.6)))
    for layers, loop, bigram in (([a], None, False), ([b], (0, 1, 2), True), ([b, lightning(1, 40, 24, (0.5,)), a], (1, 2, 1), True), ([a, a], (1, 2, 3), False)):
        cfg = config(72, 60, layers, loop=loop)
        w = weights(cfg, 8)
        plain = dict(w)
        if not bigram:
            plain["bigram"] = np.zeros_like(w["bigram"])
            cfg["embedding"].pop("bigram")
        p = o.PlainModel(dict(cfg, embedding=dict(cfg["embedding"], bigram=dict(buckets=97, mul_prev=1, mul_cur=1))) if not bigram else cfg, plain)
        toks = tokens(cfg, 90, 3)
        want = p.feed(toks)
        m = pibalorn.build(cfg, w, compute=compute)
        st = serve.Stepper(m, 200)
        got = np.vstack([st.run([("r", toks[i:j], list(range(j - i)))])[0] for i, j in ((0, 70), (70, 79), (79, 80), (80, 90))])
        e = row_errors(got, want)
        e = e if compute == pl.F32 else e[p.margins > 0.03]
        assert e.max() < 2e-5 if compute == pl.F32 else np.median(e) < 0.025 and (e > 0.06).mean() < 0.1, (loop, np.sort(e)[-5:])
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


@pytest.mark.parametrize("make", [even_config, odd_config, tall_config])
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
        assert (short > 0.1).mean() <= 0.05, np.sort(short)[-8:]
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
        assert (short > (1e-4 if compute == pl.F32 else 0.1)).mean() <= (0 if compute == pl.F32 else 0.05)
    assert m.batch_kv_seq_rm(0, 0, -1) == 0
    with pytest.raises(pl.PiError, match="recurrent"):
        m.batch_kv_seq_cp(1, 0, 0, 30)                  # a part of a sequence
    assert m.batch_kv_seq_cp(1, 0, 0, -1) == 70
    nxt, lg = m.batch_decode([3] * 5, [70] * 5)
    check(lg[:1], orc, toks[1] + [int(v) for v in [full_first(rows, 1)] + list(out[:-1, 1])] + [3], compute, slice(-1, None))
    assert np.abs(lg[0] - lg[1]).max() < 1e-5 * np.abs(lg[1]).max()
    m.close()


def full_first(rows, s):
    return rows[-1][s].argmax()


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


def test_removed_and_shifted_cells():
    """A model without recurrent layers: cells removed in the middle and the rest moved up, the keys turn with them, values stay.  The
    oracle is given the same cells at their new positions."""
    cfg = config(64, 50, [attention(4, 2, 32, rot=20)])
    w = weights(cfg, 5)
    toks = tokens(cfg, 40, 1)
    for compute, limit in ((pl.F32, 2e-5), (pl.BF16, 0.05)):
        m = pibalorn.build(cfg, w, compute=compute)
        m.decode(toks, 0, want_logits=False)
        assert m.kv_seq_rm(4, 14) == 30
        with pytest.raises(pl.PiError):
            m.decode([7], 30)                           # a gap is open
        assert m.kv_seq_shift(14, -1, -10) == 30
        _, lg = m.decode([7], 30)
        p = o.PlainModel(cfg, w)
        p.feed(toks)
        k, v = p.kv[0]
        keep = [i for i in range(40) if not 4 <= i < 14]
        p.kv[0], p.n = (o.rotate_halves(k[keep], np.array([0] * 4 + [-10] * 26), 20, 10000.0), v[keep]), 30
        assert row_errors(lg[None], p.feed([7]))[0] < limit
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
    cfg = even_config()
    w = weights(cfg, 1)
    bad = dict(w)
    bad["l1.mix.g"] = w["l1.mix.g"][:-1]
    with pytest.raises(pl.PiError, match="mix_g"):
        pibalorn.build(cfg, bad)
    for spoil, why in ((lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "grouped-query"), (lambda c: c["loop"].update(stop=9), "loop"),
                       (lambda c: c["layers"][1]["mlp"]["router"].update(top=19), "experts"), (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=66), "grouped-query")):
        c = even_config()
        spoil(c)
        with pytest.raises(pl.PiError, match=why):
            pibalorn.build(c, w)
