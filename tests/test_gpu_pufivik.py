"""Pufivik models on the GPU through the framework's entry points, against the plain implementation: whole prompts, portions, batches, cells and
convolution states that are given back and used again, keys far away, first tokens, long decoding, greedy generation through the scheduler and the
captured loop."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_pufivik as o
from lerasun_models import row_errors, tokens
from powerinfer_amd import checkpoint, lib as pl, pufivik, registry, serve
from pufivik_models import capped, config, even_config, moe, odd_config, talking, tall_config, weights

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
MODELS = {"even": even_config, "odd": odd_config, "tall": tall_config}
CASES = [(m, c) for m in MODELS.values() for c in (pl.BF16, pl.F32)]
IDS = [f"{n}-{c}" for n in MODELS for c in ("bf16", "f32")]


class Oracle:
    """Logits and streams of token sequences, one plain model per call."""
    cache = {}

    def __init__(self, make, compute):
        self.make, self.compute, self.cfg = make, compute, make()
        self.w = weights(self.cfg, 17, compute == pl.BF16)

    def run(self, toks):
        key = (self.make.__name__, self.compute, tuple(toks))
        if key not in Oracle.cache:
            p = o.PlainModel(self.cfg, self.w)
            Oracle.cache[key] = (p.feed(toks), p.streams)
        return Oracle.cache[key]

    def logits(self, toks):
        return self.run(toks)[0]


def model(orc, compute, n_ctx=512, max_batch=0):
    return pufivik.build(orc.cfg, orc.w, compute=compute, n_ctx=n_ctx, max_batch=max_batch)


def check(got, orc, toks, compute, rows=slice(None)):
    """Rows of the logits of `toks`.  (In bf16 models no choice of experts is a close call.)"""
    want = orc.run(toks)[0][rows]
    assert got.shape == want.shape
    e = row_errors(got, want)
    if compute == pl.F32:
        assert e.max() < 2e-5, (e.max(), int(e.argmax()))
    else:
        assert (e.size < 10 or np.median(e) < 0.03) and (e > 0.06).mean() <= 0.02 and e.max() < 0.12, (np.median(e), np.sort(e)[-5:], np.argsort(e)[-5:])


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_whole_prompts_and_streams(make, compute):
    orc = Oracle(make, compute)
    m = model(orc, compute)
    m.set_capture(True)
    st = serve.Stepper(m, 400)
    for n, rid in ((1, "a"), (2, "b"), (17, "c"), (64, "e"), (65, "f"), (170, "d")):
        toks = tokens(orc.cfg, n, n)
        got, _ = st.run([(rid, toks, list(range(n)))])
        check(got, orc, toks, compute)
        if compute == pl.F32:
            s, want = m.get_streams(), orc.run(toks)[1]
            assert s.shape == (len(want), n, orc.cfg["width"])
            assert max(np.abs(a - b).max() / np.abs(b).max() for a, b in zip(s, want)) < 1e-5
        st.end(rid)
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
@pytest.mark.parametrize("cut", ["ones", "twos", "mixed", "tail"])
def test_portions(make, compute, cut):
    """The same prompt token by token, two at a time, in portions of changing size, and as one portion with a decoded tail."""
    orc = Oracle(make, compute)
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
    orc = Oracle(make, compute)
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
    orc = Oracle(odd_config, compute)
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
    orc = Oracle(even_config, compute)
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
    got, _ = st.run([("w", more, [2])])
    check(got, orc, t["w"] + more + more, compute, slice(-1, None))
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_long_steps_run_in_passes(make, compute):
    """A step that is cut into passes, in the middle of the convolution's reach as well."""
    orc = Oracle(make, compute)
    for batch in (48, 33):
        m = model(orc, compute, max_batch=batch)
        st = serve.Stepper(m, 300)
        a, b = tokens(orc.cfg, 130, 1), tokens(orc.cfg, 61, 2)
        got, _ = st.run([("a", a, list(range(130))), ("b", b, list(range(61)))])
        check(got[:130], orc, a, compute)
        check(got[130:], orc, b, compute)
        m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_a_decoded_token_beside_a_long_prompt(make, compute):
    """A token far into its sequence in one batch with a long run, and the other way round."""
    orc = Oracle(make, compute)
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


@pytest.mark.parametrize("groups", [1, 2, 4])
def test_prompts_of_many_cells(groups):
    """Prompts whose later tokens' cells are shared out between workgroups, in one step and with a start that has been read already."""
    def make():
        f = moe(6, 2, 32)
        return config(96, 120, [talking(4, groups, 32, 24, f, original=300), capped(4, groups, 32, 24, 20.0, f), talking(4, groups, 40, 24)], groups=3)

    make.__name__ = f"many_cells_{groups}"
    orc = Oracle(make, pl.BF16)
    toks = tokens(orc.cfg, 1100, 3)
    m = model(orc, pl.BF16, n_ctx=1200)
    st = serve.Stepper(m, 1200)
    for cuts in ([0, 1100], [0, 300, 1099, 1100]):
        got = np.vstack([st.run([("r", toks[a:b], list(range(b - a)))])[0] for a, b in zip(cuts, cuts[1:])])
        check(got, orc, toks, pl.BF16)
        st.end("r")
    m.close()


def looking_model(layer):
    """One layer whose attention makes token 32 + k look for token 42 + k and for nothing else."""
    rng = np.random.default_rng(0)
    cfg = config(64, 64, [layer], scale=1.0, mult=1.5, taps=3)
    w = weights(cfg, 3)
    bf = lambda a: checkpoint.bf16_floats(checkpoint.bf16_bits(a)).reshape(a.shape)  # noqa: E731
    emb = np.linalg.qr(rng.standard_normal((64, 64)))[0].T
    look = sum(np.outer(emb[42 + k], emb[32 + k]) for k in range(12)) + 0.05 * np.eye(64)
    code = np.linalg.qr(rng.standard_normal((64, 64)))[0]
    w["embed"], w["l0.norm1"] = bf(emb.astype(np.float32)), np.ones(64, np.float32)
    w["l0.canon1"] = 0.25 * w["l0.canon1"]
    w["l0.mix.k"], w["l0.mix.q"] = bf(np.concatenate([code] * layer["mixer"]["kv_heads"])), bf(np.concatenate([code @ look] * layer["mixer"]["heads"]))
    return cfg, w


FAR = {"talking": talking(4, 2, 64, 48, rot=0, scale=0.5), "capped": capped(2, 1, 64, 48, 20.0, rot=0, scale=0.5)}


@pytest.mark.parametrize("kind", FAR)
def test_far_keys_in_prompts_and_decoding(kind):
    """One key among hundreds decides a token's result: the first, at edges of tiles of cells, the token before, asked for in a portion and singly."""
    cfg, w = looking_model(FAR[kind])
    rng, n = np.random.default_rng(7), 330
    toks = [int(v) for v in rng.integers(1, 32, n)]
    pairs = [(0, 300), (1, n - 5), (63, 200), (64, n - 3), (127, 280), (128, n - 1), (254, 255), (31, 32), (4, 180), (256, n - 7)]
    assert len({x for p in pairs for x in p}) == 20
    for k, (key, ask) in enumerate(pairs):
        toks[key], toks[ask] = 42 + k, 32 + k
    want = o.PlainModel(cfg, w).feed(toks)
    for key, ask in pairs:
        blind = list(toks)
        blind[key] = 3
        e = row_errors(o.PlainModel(cfg, w).feed(blind)[ask:ask + 1], want[ask:ask + 1])[0]
        assert e > 0.2, (key, ask, e)
    for compute, limit in ((pl.F32, 2e-5), (pl.BF16, 0.06)):
        for sizes in ([n], [n - 12] + [1] * 12, [64] * 5 + [10], [99, 2, 2] + [1] * 227, [17] * 19 + [7]):
            m = pufivik.build(cfg, w, compute=compute)
            st = serve.Stepper(m, 352)
            got, at = [], 0
            for k in sizes:
                got.append(st.run([("r", toks[at:at + k], list(range(k)))])[0])
                at += k
            e = row_errors(np.vstack(got), want)
            assert e.max() < limit, (compute, sizes[:2], e.max(), int(e.argmax()))
            m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_first_tokens(compute):
    """Every start of a sequence, alone and beside others that have begun already."""
    orc = Oracle(even_config, compute)
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
    """One layer of one kind only, sizes of one, no feed-forward at all, one tap and many, groups of one value, one expert of which all are chosen, plain
    rotations, none, and part of one, widths below and beyond a kernel's step, a factor of the sums that is zero or negative."""
    t, c = talking(4, 2, 24, 16, moe(4, 4, 24), rot=10), capped(2, 2, 16, 40, 3.0, moe(1, 1, 40))
    plain = capped(2, 1, 32, 32, 9.0)
    plain["mixer"]["rot"].pop("scaling")
    bare = talking(2, 1, 32, 32)
    bare["mixer"]["rot"] = None
    one = talking(1, 1, 2, 1, moe(1, 1, 1), rot=2)
    for width, layers, kw in ((72, [t], dict(taps=1)), (72, [c], dict(taps=2)), (40, [one, capped(1, 1, 1, 1, 1.0)], dict(taps=5, scale=1.0, mult=1.0)), (300, [dict(t, mlp=None)] * 3, dict(groups=6)),
                              (1100, [plain, bare], dict(eps=1e-2, groups=10)), (48, [c, c], dict(mult=-0.5, groups=16)), (33, [bare, plain], dict(mult=0.0, groups=11, taps=9)),
                              (64, [talking(4, 4, 8, 8, moe(6, 3, 16), original=8, v_mix=False), plain], dict(groups=8, taps=6))):
        cfg = config(width, 60, layers, **kw)
        w = weights(cfg, 8, compute == pl.BF16)
        toks = tokens(cfg, 90, 3)
        want = o.PlainModel(cfg, w).feed(toks)
        m = pufivik.build(cfg, w, compute=compute)
        st = serve.Stepper(m, 200)
        got = np.vstack([st.run([("r", toks[i:j], list(range(j - i)))])[0] for i, j in ((0, 70), (70, 79), (79, 80), (80, 90))])
        e = row_errors(got, want)
        assert e.max() < (5e-5 if compute == pl.F32 else 0.1), (width, len(layers), np.median(e), np.sort(e)[-5:])
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
    orc = Oracle(make, pl.F32)
    prompts = [tokens(orc.cfg, n, 40 + n) for n in (1, 7, 40, 90, 3, 21)]
    want = [greedy(orc, p, 10) for p in prompts]
    assert min(min(g) for _, g in want) > 1e-4, "a tie in the test's own model"
    m = model(orc, pl.F32)
    got = serve.generate(m, prompts, 10, n_cells=128, max_live=3, budget=24)
    assert got == [w for w, _ in want]
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_long_decoding_in_the_captured_loop(make, compute):
    """pi_model_decode + pi_model_generate (one captured step replayed, several calls) against the oracle, position by position."""
    orc = Oracle(make, compute)
    m = model(orc, compute, n_ctx=320)
    prompt = tokens(orc.cfg, 37, 77)
    first, lg = m.decode(prompt, 0)
    check(lg[None], orc, prompt, compute, slice(-1, None))
    out = [first] + [int(v) for n in (3, 120, 77) for v in m.generate(n)[0]]
    assert len(out) == 201
    full = orc.logits(prompt + out[:-1])[len(prompt) - 1:]
    short = (full.max(axis=1) - full[np.arange(201), out]) / full.std()
    assert short.max() < (1e-4 if compute == pl.F32 else 0.12), np.sort(short)[-8:]          # a chosen token is within rounding of the best one
    again, lg2 = m.decode(out[-1:], len(prompt) + 200)  # and the cache and states it left are the right ones
    check(lg2[None], orc, prompt + out, compute, slice(-1, None))
    with pytest.raises(pl.PiError, match="go back"):    # a convolution's last inputs have no earlier positions
        m.decode([1], len(prompt))
    m.kv_clear()
    assert m.decode(prompt, 0)[0] == first
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_lockstep_batches(compute):
    """batch_init / batch_decode / batch_generate: five sequences, each as if it were alone; a prefix handed on with its states."""
    orc = Oracle(even_config, compute)
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
        assert short.max() < (1e-4 if compute == pl.F32 else 0.12)
    assert m.batch_kv_seq_rm(0, 0, -1) == 0
    with pytest.raises(pl.PiError, match="recurrent"):
        m.batch_kv_seq_cp(1, 0, 0, 30)                  # a part of a sequence
    assert m.batch_kv_seq_cp(1, 0, 0, -1) == 70
    nxt, lg = m.batch_decode([3] * 5, [70] * 5)
    check(lg[:1], orc, toks[1] + [int(rows[-1][1].argmax())] + [int(v) for v in out[:-1, 1]] + [3], compute, slice(-1, None))
    assert np.abs(lg[0] - lg[1]).max() < 1e-5 * np.abs(lg[1]).max()
    m.close()


def test_sequences_are_moved_where_nothing_is_convolved():
    """One tap leaves no state: cells may be dropped and their keys turned to other positions, with scaled frequencies."""
    cfg = config(80, 70, [capped(2, 2, 32, 12, 4.0), talking(4, 2, 32, 12, original=30)], taps=1)
    w = weights(cfg, 2)
    toks = tokens(cfg, 40, 3)
    p = o.PlainModel(cfg, w)
    want = p.feed(toks[:10] + toks[20:])[-1:]
    m = pufivik.build(cfg, w, compute=pl.F32)
    m.kv_cells_init(64)
    # one layer deep the dropped tokens leave no trace; here the second layer's cells have seen them, so only positions are compared
    m.kv_cells_step(toks[:10], range(10), [1] * 10, [])
    m.kv_cells_step(toks[20:39], range(20, 39), [1] * 19, [])
    _, lg0 = m.kv_cells_step(toks[39:], [39], [1], [0])
    m.kv_cells_seq_rm(0, 39, 40)
    m.kv_cells_seq_shift(0, 0, -1, 7)                   # all keys move: scores depend on distances alone
    _, lg1 = m.kv_cells_step(toks[39:], [46], [1], [0])
    assert row_errors(lg1, lg0).max() < 2e-5
    assert row_errors(lg1, want).max() > 1e-3           # (with the gap closed the result would be another one)
    m.close()


def save(folder, cfg, w):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    checkpoint.write_safetensors(os.path.join(folder, "model.safetensors"), {k: checkpoint.bf16_bits(v).reshape(np.shape(v)) for k, v in w.items()})


def test_files_and_trace_replay_and_command_line(tmp_path):
    orc = Oracle(odd_config, pl.F32)
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
    for name, why in (("l1.mix.talk", "mix_talk"), ("l1.mix.sink", "mix_sink"), ("l4.mix.g", "mix_head_gate"), ("l0.canon1", "mix_conv"), ("l2.norm2b", "ffn_norm_after"), ("l3.norm1b", "attn_norm_after")):
        bad = dict(w)
        bad[name] = w[name][:-1]
        with pytest.raises(pl.PiError, match=why):
            pufivik.build(cfg, bad)
    for spoil, why in ((lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "grouped-query"), (lambda c: c["norm"].update(groups=3), "norm_groups"),
                       (lambda c: c["layers"][0]["mixer"].update(softcap=-1.0), "soft cap"), (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0.0), "rotation"),
                       (lambda c: c["layers"][4]["mixer"].update(vdim=25), "mix values"), (lambda c: c["layers"][1]["mlp"]["router"].update(top=6), "experts")):
        c = odd_config()
        spoil(c)
        with pytest.raises(pl.PiError, match=why):
            pufivik.build(c, w)
