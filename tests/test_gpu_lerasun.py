"""Lerasun models on the GPU through the framework's entry points, against the plain implementation: whole prompts, portions, batches,
cells that are given back and used again, long decoding, greedy generation through the scheduler and the captured loop."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_latent as o
from lerasun_models import config, even_config, layer, odd_config, row_errors, tokens, weights
from powerinfer_amd import checkpoint, lerasun, lib as pl, registry, serve

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
CASES = [(even_config, pl.BF16), (even_config, pl.F32), (odd_config, pl.BF16), (odd_config, pl.F32)]
IDS = ["even-bf16", "even-f32", "odd-bf16", "odd-f32"]


class Oracle:
    """Logits of token sequences, one plain model per call."""
    cache = {}

    def __init__(self, make):
        self.cfg = make()
        self.w = weights(self.cfg, 17)
        self.make = make

    def logits(self, toks):
        key = (self.make.__name__, tuple(toks))
        if key not in Oracle.cache:
            p = o.PlainModel(self.cfg, self.w)
            Oracle.cache[key] = Logits(p.feed(toks), p.margins)
        return Oracle.cache[key]


class Logits(np.ndarray):
    """Logits that remember how far each position's closest routing decision was."""

    def __new__(cls, a, margins):
        x = np.asarray(a).view(cls)
        x.margins = margins
        return x

    def __array_finalize__(self, src):
        self.margins = getattr(src, "margins", None)

    def __getitem__(self, k):
        x = super().__getitem__(k)
        if isinstance(x, Logits) and isinstance(k, (slice, list)):
            x.margins = self.margins[k]
        return x


def model(orc, compute, n_ctx=512, max_batch=0):
    return lerasun.build(orc.cfg, orc.w, compute=compute, n_ctx=n_ctx, max_batch=max_batch)


def check(got, want, compute):
    """fp32: every position.  bf16: the positions whose routing decisions were not close calls (those may fall the other way, and a token
    that looks at such a token hears of it)."""
    assert got.shape == want.shape
    e = row_errors(got, np.asarray(want))
    if compute == pl.F32:
        assert e.max() < 2e-5, (e.max(), int(e.argmax()))
    else:
        e = e[want.margins > 0.015]
        assert e.size == 0 or (np.median(e) < 0.02 and (e > 0.06).mean() <= 0.08 and (e > 0.1).mean() <= 0.03), (np.median(e), np.sort(e)[-5:], np.argsort(e)[-5:])


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_whole_prompts_and_streams(make, compute):
    orc = Oracle(make)
    m = model(orc, compute)
    m.set_capture(True)
    st = serve.Stepper(m, 400)
    for n, rid in ((1, "a"), (2, "b"), (17, "c"), (170, "d")):
        toks = tokens(orc.cfg, n, n)
        got, _ = st.run([(rid, toks, list(range(n)))])
        check(got, orc.logits(toks), compute)
        if compute == pl.F32:
            p = o.PlainModel(orc.cfg, orc.w)
            p.feed(toks)
            s = m.get_streams()
            assert s.shape == (len(orc.cfg["layers"]), n, orc.cfg["width"])
            assert max(np.abs(a - b).max() / np.abs(b).max() for a, b in zip(s, p.streams)) < 1e-5
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
    check(np.vstack(got), orc.logits(toks), compute)
    m.close()


@pytest.mark.parametrize("make,compute", CASES, ids=IDS)
def test_mixed_batches_against_each_alone(make, compute):
    """Four requests of unequal length, portions beside single tokens, some left out of a step, ends at different times, and two more
    requests on the cells and sequences the first ones gave back - in a pool that holds exactly what is live."""
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
        entries = [(k, toks[k][at[k]:at[k] + n], list(range(n))) for k, n in step.items()]
        lg, _ = st.run(entries)
        row = 0
        for k, n in step.items():
            got[k].append(lg[row:row + n])
            row += n
            at[k] += n
            if at[k] == lens[k]:
                st.end(k)
    assert at == lens and st.free_cells == peak
    for k in lens:
        check(np.vstack(got[k]), orc.logits(toks[k]), compute)
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
    check(got, orc.logits(long), compute)
    more = tokens(orc.cfg, 3, 8)
    st.end("y")
    got, _ = st.run([("w", more, [0, 1, 2])])
    check(got, orc.logits(t["w"] + more)[-3:], compute)
    with pytest.raises(pl.PiError, match="free cells"):
        st.m.kv_cells_step([1] * 50, range(50), [1 << 9] * 50, [49])
    st.end("n")                                         # the refused step has left nothing behind
    assert (st.m.kv_cells_state()[0] >= 0).sum() == 43
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_long_steps_run_in_passes(compute):
    orc = Oracle(even_config)
    m = model(orc, compute, max_batch=48)
    st = serve.Stepper(m, 300)
    a, b = tokens(orc.cfg, 130, 1), tokens(orc.cfg, 61, 2)
    got, _ = st.run([("a", a, list(range(130))), ("b", b, list(range(61)))])
    check(got[:130], orc.logits(a), compute)
    check(got[130:], orc.logits(b), compute)
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_a_decoded_token_beside_a_long_prompt(compute):
    """A token far into its sequence (its cells split over workgroups) in one batch with a long run on expanded keys and values."""
    orc = Oracle(even_config)
    m = model(orc, compute, n_ctx=1024)
    st = serve.Stepper(m, 760)
    a, b = tokens(orc.cfg, 340, 1), tokens(orc.cfg, 400, 2)
    st.run([("a", a[:330], [])])
    got, _ = st.run([("a", a[330:331], [0]), ("b", b[:399], list(range(399)))])
    check(got[:1], orc.logits(a)[330:331], compute)
    check(got[1:], orc.logits(b)[:399], compute)
    got, _ = st.run([("b", b[399:], [0]), ("a", a[331:], list(range(9)))])
    check(got[:1], orc.logits(b)[399:], compute)
    check(got[1:], orc.logits(a)[331:], compute)
    m.close()


def test_far_keys_in_prompts_and_decoding():
    """One layer in which token 32 + k looks for token 42 + k and for nothing else: that key decides the result hundreds of tokens back, at
    the first positions, at edges of 32- and 64-cell tiles - and not at all one position before it appears."""
    cfg = config(64, 64, [layer(2, 32, 8, 32, 64, scale=1.0)], logit_scale=1.0)
    w = weights(cfg, 3)
    rng = np.random.default_rng(0)
    bf = lambda a: checkpoint.bf16_floats(checkpoint.bf16_bits(a)).reshape(a.shape)  # noqa: E731
    emb = np.linalg.qr(rng.standard_normal((64, 64)))[0].astype(np.float32)
    w["embed"] = bf(emb)
    for k in ("embed.norm", "l0.norm1"):
        w[k] = np.zeros(64, np.float32)
    w["l0.mix.dkv.norm"] = np.ones(64, np.float32)
    w["l0.mix.dkv"] = np.zeros((72, 64), np.float32)
    w["l0.mix.dkv"][:64] = np.eye(64)
    look = sum(np.outer(emb[42 + k], emb[32 + k]) for k in range(10)) + np.outer(emb[63], emb[62])
    uk = (rng.integers(0, 2, (2, 32, 64)) * 2 - 1).astype(np.float32) / 4
    q = np.zeros((2, 40, 64), np.float32)
    q[:, :32] = uk @ look / 2
    w["l0.mix.q"], w["l0.mix.uk"] = bf(q.reshape(80, 64)), uk.reshape(64, 64)
    n = 330
    toks = [int(v) for v in rng.integers(0, 32, n)]
    for k, p in enumerate([0, 1, 31, 32, 63, 64, 127, 128, 255, 256]):
        toks[p], toks[n - 12 + k] = 42 + k, 32 + k
    toks[100], toks[99], toks[101], toks[200] = 63, 62, 62, 62
    want = o.PlainModel(cfg, w).feed(toks)
    for key, asks, seen in ((0, n - 12, True), (256, n - 3, True), (100, 99, False), (100, 101, True), (100, 200, True)):
        blind = list(toks)
        blind[key] = 3
        other = o.PlainModel(cfg, w).feed(blind)
        e = row_errors(other[asks:asks + 1], want[asks:asks + 1])[0]
        assert (e > 0.2) == seen and (seen or e == 0), (key, asks, e)        # the far key does decide
    for compute, limit in ((pl.F32, 2e-5), (pl.BF16, 0.05)):
        for sizes in ([n], [n - 12] + [1] * 12, [64] * 5 + [10], [99, 2, 2] + [1] * 227):
            m = lerasun.build(cfg, w, compute=compute)
            st = serve.Stepper(m, 352)
            got, at = [], 0
            for k in sizes:
                got.append(st.run([("r", toks[at:at + k], list(range(k)))])[0])
                at += k
            e = row_errors(np.vstack(got), want)
            assert e.max() < limit, (compute, sizes[:2], e.max(), int(e.argmax()))
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


@pytest.mark.parametrize("make", [even_config, odd_config])
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
    check(lg[None], orc.logits(prompt)[-1:], compute)
    out = [first] + [int(v) for n in (3, 120, 77) for v in m.generate(n)[0]]
    assert len(out) == 201
    full = orc.logits(prompt + out[:-1])[len(prompt) - 1:]
    if compute == pl.F32:
        assert [int(v) for v in full.argmax(axis=1)] == out
    else:                                               # every chosen token is within rounding of the best one
        short = np.asarray((full.max(axis=1) - full[np.arange(201), out]) / full.std())
        assert (short > 0.1).mean() <= 0.05, np.sort(short)[-8:]
    again, lg2 = m.decode(out[-1:], len(prompt) + 200)  # and the cache it left is the right one
    check(lg2[None], orc.logits(prompt + out)[-1:], compute)
    m.kv_clear()
    assert m.decode(prompt, 0)[0] == first
    m.close()


@pytest.mark.parametrize("compute", [pl.BF16, pl.F32])
def test_lockstep_batches(compute):
    """batch_init / batch_decode / batch_generate: five sequences at unequal positions, each as if it were alone; a prefix handed on."""
    orc = Oracle(even_config)
    m = model(orc, compute, n_ctx=128)
    m.batch_init(5)
    toks = [tokens(orc.cfg, 30, 60 + s) for s in range(5)]
    rows = []
    for p in range(30):
        nxt, lg = m.batch_decode([t[p] for t in toks], [p] * 5)
        rows.append(lg)
    for s in range(5):
        check(np.stack([r[s] for r in rows]), orc.logits(toks[s]), compute)
    out, _ = m.batch_generate(40)
    assert out.shape == (40, 5)
    for s in range(5):
        seq = [int(nxt[s])] + [int(v) for v in out[:, s]]
        full = orc.logits(toks[s] + seq[:-1])[29:]
        short = (full.max(axis=1) - full[np.arange(41), seq]) / full.std()
        assert (short > (1e-4 if compute == pl.F32 else 0.1)).mean() <= (0 if compute == pl.F32 else 0.05)
    assert m.batch_kv_seq_rm(0, 0, -1) == 0 and m.batch_kv_seq_cp(1, 0, 0, 30) == 30           # the prefix is shared, not copied
    nxt, lg = m.batch_decode([3] * 5, [30] + [70] * 4)
    check(lg[:1], orc.logits(toks[1] + [3])[-1:], compute)
    m.close()


def test_removed_and_shifted_cells():
    """Cells removed in the middle and the rest moved up: the rotated key parts turn with them (what the reference's context shift does
    to K rows), latents stay.  The oracle is given the same latents at their new positions."""
    cfg = config(64, 50, [layer(2, 16, 8, 16, 32)], logit_scale=1.0)
    w = weights(cfg, 5)
    toks = tokens(cfg, 40, 1)
    for compute, limit in ((pl.F32, 2e-5), (pl.BF16, 0.05)):
        m = lerasun.build(cfg, w, compute=compute)
        m.decode(toks, 0, want_logits=False)
        assert m.kv_seq_rm(4, 14) == 30
        with pytest.raises(pl.PiError):
            m.decode([7], 30)                           # a gap is open
        assert m.kv_seq_shift(14, -1, -10) == 30
        _, lg = m.decode([7], 30)
        p = o.PlainModel(cfg, w)
        p.feed(toks)
        lat, kr = p.kv[0]
        keep = [i for i in range(40) if not 4 <= i < 14]
        back = np.array([0] * 4 + [-10] * 26)
        p.kv[0], p.n = (lat[keep], o.rotate_pairs(kr[keep], back, 10000.0)), 30
        assert row_errors(lg[None], p.feed([7]))[0] < limit
        m.close()


def test_a_sequence_of_shared_cells():
    """kv_cells_seq_cp: a prompt evaluated once serves two continuations; ending one leaves the other's cells alone."""
    orc = Oracle(odd_config)
    m = model(orc, pl.F32)
    m.kv_cells_init(100)
    p, a, b = tokens(orc.cfg, 50, 1), tokens(orc.cfg, 9, 2), tokens(orc.cfg, 9, 3)
    m.kv_cells_step(p, range(50), [1] * 50, [])
    m.kv_cells_seq_cp(0, 1, 0, -1)
    _, lg = m.kv_cells_step(a + b, list(range(50, 59)) * 2, [1] * 9 + [2] * 9, range(18))
    check(lg[:9], orc.logits(p + a)[50:], pl.F32)
    check(lg[9:], orc.logits(p + b)[50:], pl.F32)
    m.kv_cells_seq_rm(0, -1, -1)
    _, lg = m.kv_cells_step([5], [59], [2], [0])
    check(lg, orc.logits(p + b + [5])[-1:], pl.F32)
    m.close()


def test_existing_models_run_through_the_same_scheduler():
    """kv_cells_step and the scheduler on a sparse LLaMA model: the tokens of its own token loop."""
    from powerinfer_amd import synth
    from powerinfer_amd.model import Model
    hp = synth.hparams("llama-tiny", n_embd=512, n_ff=1024, n_rank=128, n_head=8, n_head_kv=8, n_layer=2, n_ctx=128, seed=3)
    data = synth.make_model(hp)
    prompt = [5, 9, 200, 31, 7, 4, 4, 90, 12, 33, 1, 2, 3, 8, 100, 101, 102, 103, 104]
    m = Model(hp).load(data)
    m.kv_cells_init(128)
    nxt, lg = m.kv_cells_step(prompt, range(len(prompt)), [1] * len(prompt), [3, len(prompt) - 1])
    m.close()
    m = Model(hp).load(data)
    for k, at in ((0, 4), (1, len(prompt))):
        tok, want = m.decode(prompt[:at], 0)
        assert np.abs(lg[k] - want).max() / np.abs(want).max() < 2e-2
    m.close()
    m = Model(hp).load(data)
    out = serve.generate(m, [prompt, prompt[:5]], 6, n_cells=128)
    assert [len(v) for v in out] == [6, 6] and all(0 <= t < hp.n_vocab for v in out for t in v)
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
    check(m.decode(toks, 0)[1][None], orc.logits(toks)[-1:], pl.F32)
    m.close()
    steps = [{"step": 0, "entries": [{"id": "p", "tokens": toks[:11], "want": [0, 10]}, {"id": "q", "tokens": toks[:2], "want": []}], "end": ["q"]},
             {"step": 1, "entries": [{"id": "p", "tokens": toks[11:12], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "r", "tokens": toks[:3], "want": [2]}, {"id": "p", "tokens": toks[12:], "want": [7]}], "end": ["p", "r"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"], r.stderr[-800:]
    full, v = orc.logits(toks), orc.cfg["vocab"]
    check(np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, v), full[[0, 10]], pl.F32)
    check(np.fromfile(tmp_path / "2.f32", "<f4").reshape(2, v), full[[2, 19]], pl.F32)
    assert not (tmp_path / "1.f32").exists()
    r = subprocess.run([sys.executable, "-m", "powerinfer_amd", "generate", "--model", folder, "--dtype", "float32", "--prompt", ",".join(map(str, toks)), "--new", "5"],
                       cwd=ROOT, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-800:]
    assert [int(t) for t in r.stdout.split()[-1].split(",")] == greedy(orc, toks, 5)[0]


def test_bad_models_are_refused():
    cfg = even_config()
    w = weights(cfg, 1)
    bad = dict(w)
    bad["l0.mix.uk"] = w["l0.mix.uk"][:-1]
    with pytest.raises(pl.PiError, match="mix_uk"):
        lerasun.build(cfg, bad)
    c = even_config()
    c["layers"][2]["mixer"]["kv_from"] = 1              # names a layer without cells of its own
    with pytest.raises(pl.PiError, match="kv_from"):
        lerasun.build(c, w)
    c = even_config()
    c["layers"][0]["mlp"]["router"]["groups"]["count"] = 5
    with pytest.raises(pl.PiError, match="experts"):
        lerasun.build(c, w)
