"""Operators of layers whose norms come after the sums, one by one against the plain implementations (tests/plain_fikevik.py): linear
attention with key decays and with exponential gates, windows, norms of queries, keys and values, gated residuals, the GLU of a step."""
import ctypes as C

import numpy as np
import pytest

import plain_fikevik as o
from plain_pibalorn import rotate_halves
from powerinfer_amd import lib as pl
from test_gpu_gqa_ops import attend, filled
from test_gpu_latent_ops import TYPES, as_stored, dev, fetch, i32, padded, rounded, store, tol

pytestmark = pytest.mark.gpu
KEYED, GATED = pl.DECAY_KEYED, pl.DECAY_GATED


class Run:
    """One call of the operator on random projections.  runs: (tokens, slot, starts at zero)."""

    def __init__(self, kind, t, runs, H, dim, vdim, chunked, seed=0, slots=5, rank=11, tau=3.0, cap=6.0, bias=0.0, spread=2.0, beside=None, edit=None, exact=False):
        L, rng = pl.init(), np.random.default_rng(seed)
        T, Cn, dim_ld, vdim_ld = sum(n for n, _, _ in runs), L.pi_k_linear_chunk(), (dim + 31) // 32 * 32, (vdim + 63) // 64 * 64
        at, off = 0, {}
        if beside:                                           # the attention's rows come first
            off["att"], at = 0, beside["rows"]
        for name, n in (("q", H * dim), ("k", H * dim), ("v", H * vdim), ("a", rank), ("i", H), ("f", H)):
            off[name], at = at, (at + n + 2 + 15) // 16 * 16
        ldz = at
        z = rng.standard_normal((T, ldz)).astype(np.float32)
        if exact:                                            # projections that bf16 holds
            z = rounded(z)
        a2, a2b = rounded(rng.standard_normal((H * dim, rank)) / np.sqrt(rank)), (bias + spread * rng.standard_normal(H * dim)).astype(np.float32)
        ib, fb = (2 * rng.standard_normal((2, H)) + [[0], [bias]]).astype(np.float32)
        if edit:
            edit(z, off, a2b, ib, fb)
        copies, n_s, n_k = L.pi_k_linear_copies(vdim), H * dim * vdim, H * dim
        slot = L.pi_k_linear_slot_floats(kind, H, dim, vdim)
        state = np.zeros((slots, slot + 3), np.float32)
        state[:, :n_s] = rng.standard_normal((slots, n_s))
        if kind == GATED:
            state[:, n_s:n_s + n_k] = rng.standard_normal((slots, n_k))
            state[:, n_s + n_k:slot] = np.repeat(rng.standard_normal((slots, H)), copies, axis=1)
        else:
            assert slot == n_s
        items, chunks, first, row = [], [], [], 0
        for n, s, fresh in runs:
            items.append([row, n, s, fresh])
            first.append(len(chunks))
            chunks += [[row + c, min(Cn, n - c), int(fresh and c == 0)] for c in range(0, n, Cn)]
            row += n
        rank_ld = (rank + 7) // 8 * 8
        b = dict(z=dev(z), state=dev(state), runs=i32(items), o=pl.DevBuf.zeros(4 * T * H * vdim), q=pl.DevBuf(2 * T * H * dim_ld), k=pl.DevBuf(2 * T * H * dim_ld),
                 v=pl.DevBuf(2 * T * H * vdim_ld), states=pl.DevBuf(L.pi_k_linear_states_bytes(len(chunks), H, dim_ld, vdim_ld)), chunks=i32(chunks), first_chunk=i32(first),
                 a2=store(padded(a2, rank_ld), pl.BF16), a2_b=dev(a2b), i_b=dev(ib), f_b=dev(fb), den=pl.DevBuf.zeros(4 * T * H),
                 gates=pl.DevBuf(4 * L.pi_k_linear_gate_floats(kind, T, len(chunks), H, dim_ld)))
        p = filled(pl.Linear, ldz=ldz, T=T, n_head=H, dim=dim, vdim=vdim, off_q=off["q"], off_k=off["k"], off_v=off["v"], n_runs=len(items), dim_ld=dim_ld, vdim_ld=vdim_ld, n_chunks=len(chunks),
                   decay_kind=kind, plain=1, q_scale=dim ** -0.5, slot_ld=slot + 3, off_a=off["a"], rank=rank, rank_ld=rank_ld, tau=tau, off_i=off["i"], off_f=off["f"], cap=cap, **b)
        if chunked:
            pl.check(L.pi_k_linear_prep(t, C.byref(p), None, None))
            pl.check(L.pi_k_linear_chunks(C.byref(p), None))
        elif beside:
            prep = beside["prep"](b["z"], ldz, T)
            pl.check(L.pi_k_linear_step_beside(t, C.byref(p), C.byref(prep), None))
        else:
            pl.check(L.pi_k_linear_step(t, C.byref(p), None, None))
        pl.sync()
        z64 = z.astype(np.float64)
        self.z = z64
        part = lambda name, n, f=1.0: as_stored(z[:, off[name]:off[name] + n] * np.float32(f), t if chunked else pl.F32).astype(np.float64).reshape(T, H, -1)  # noqa: E731
        q, k, v = part("q", H * dim, dim ** -0.5), part("k", H * dim), part("v", H * vdim)
        self.want, ends, wden = np.empty((T, H, vdim)), state[:, :slot].astype(np.float64), np.ones((T, H))
        row = 0
        for n, s, fresh in runs:
            x, st = slice(row, row + n), ends[s] * (not fresh)
            S = st[:n_s].reshape(H, dim, vdim)
            if kind == KEYED:
                decay = o.key_decays(z64[x, off["a"]:off["a"] + rank], np.eye(rank), a2.astype(np.float64), a2b, tau).reshape(n, H, dim)
                self.want[x], S = o.keyed_sums(q[x], k[x], v[x], decay, S)
                ends[s] = S.ravel()
            else:
                ts = {"i": np.eye(H), "i.b": ib.astype(np.float64)}
                i, _ = o.memory_gates(z64[x, off["i"]:off["i"] + H], dict(ts, f=np.eye(H), **{"f.b": fb.astype(np.float64)}), cap)
                _, f = o.memory_gates(z64[x, off["f"]:off["f"] + H], dict(ts, f=np.eye(H), **{"f.b": fb.astype(np.float64)}), cap)
                mem = (S, st[n_s:n_s + n_k].reshape(H, dim), st[n_s + n_k:].reshape(H, copies)[:, 0])
                reads, (S, key, top) = o.memory_reads(q[x], k[x], v[x], i, f, mem)
                wden[x] = o.memory_reads.den
                self.want[x] = reads * wden[x][:, :, None]
                ends[s] = np.concatenate([S.ravel(), key.ravel(), np.repeat(top, copies)])
            row += n
        self.got = b["o"].download(np.float32).reshape(T, H, vdim)
        self.den, self.wden = b["den"].download(np.float32).reshape(T, H), wden
        got = b["state"].download(np.float32).reshape(state.shape)
        assert np.array_equal(got[:, slot:], state[:, slot:])
        assert all(np.array_equal(got[s], state[s]) for s in range(slots) if s not in [r[1] for r in runs])
        self.states, self.ends, self.split = got[:, :slot], ends, (n_s, n_s + n_k)

    def check(self, limit, per_token=None):
        close = lambda a, b: np.abs(a - b).max() <= limit * np.abs(b).max()  # noqa: E731
        assert np.isfinite(self.got).all() and close(self.got, self.want), np.abs(self.got - self.want).max() / np.abs(self.want).max()
        cuts = (0,) + self.split + (self.states.shape[1],)
        for a, b in zip(cuts[:-1], cuts[1:]):
            if b > a and (self.states.shape[1] > self.split[0] or a == 0):
                assert close(self.states[:, a:b], self.ends[:, a:b]), (a, b)
        if (self.wden != 1).any():
            assert close(self.den, self.wden)
        if per_token:                                            # no token is off, also where the sums are small
            e = np.abs(self.got - self.want).max(axis=(1, 2)) - per_token * np.abs(self.want).max(axis=(1, 2))
            assert (e <= 1e-4).all(), int(e.argmax())


SHAPES = [(3, 20, 36), (4, 64, 64), (5, 33, 9), (1, 128, 128), (2, 256, 70), (2, 90, 256), (1, 1, 1), (2, 256, 256)]
LONG = [[(64, 0, True)], [(17, 1, True), (63, 0, False), (65, 3, True), (200, 2, False)], [(128, 4, False), (1, 0, True), (129, 1, True)]]


@pytest.mark.parametrize("kind", [KEYED, GATED])
@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("H,dim,vdim", SHAPES)
def test_token_by_token(kind, t, H, dim, vdim):
    Run(kind, t, [(1, 3, False), (16, 0, True), (2, 4, True), (1, 1, True), (40, 2, False)], H, dim, vdim, False, seed=dim).check(2e-5)


@pytest.mark.parametrize("kind", [KEYED, GATED])
@pytest.mark.parametrize("H,dim,vdim", SHAPES)
@pytest.mark.parametrize("runs", LONG)
def test_chunks(kind, H, dim, vdim, runs):
    Run(kind, pl.BF16, runs, H, dim, vdim, True, seed=vdim).check(1e-4, 1e-3)


@pytest.mark.parametrize("bias,spread,tau", [(-40.0, 20.0, 0.5), (-10.0, 10.0, 1.0), (0.0, 30.0, 0.3), (20.0, 0.0, 16.0), (-300.0, 0.0, 0.2), (0.0, 300.0, 1.0)])
def test_key_decays_of_any_size(bias, spread, tau):
    """From channels that keep everything to channels that forget within a token, also side by side: no overflow, nothing lost."""
    for runs in LONG:
        Run(KEYED, pl.BF16, runs, 2, 64, 64, True, tau=tau, bias=bias, spread=spread).check(1e-4, 1e-3)
        Run(KEYED, pl.BF16, runs, 2, 64, 64, False, tau=tau, bias=bias, spread=spread).check(2e-5)


def test_a_reset_in_the_middle_of_a_chunk():
    """One token wipes a channel's state; what comes behind it decays hardly at all."""
    for at in (0, 5, 15, 16, 40, 63):
        def edit(z, off, a2b, ib, fb, at=at):
            z[:, off["a"]:off["a"] + 11] = 0
            z[at, off["a"]:off["a"] + 11] = 900.0
        Run(KEYED, pl.BF16, [(150, 0, False)], 2, 32, 64, True, tau=1.0, bias=6.0, spread=0.5, edit=edit).check(1e-4, 1e-3)


@pytest.mark.parametrize("cap,bias", [(40.0, 0.0), (15.0, 30.0), (15.0, -30.0), (2.0, 0.0), (60.0, 50.0), (40.0, -60.0)])
def test_exponential_gates_of_any_size(cap, bias):
    """Large and small input gates after one another, memories that keep and that forget everything: the running maximum holds them together."""
    def edit(z, off, a2b, ib, fb):
        z[:, off["i"]:off["i"] + 2] *= cap / 2
    for runs in LONG:
        Run(GATED, pl.BF16, runs, 2, 64, 64, True, cap=cap, bias=bias, edit=edit).check(1e-4)
        Run(GATED, pl.BF16, runs, 2, 64, 64, False, cap=cap, bias=bias, edit=edit).check(3e-5)


@pytest.mark.parametrize("kind", [KEYED, GATED])
def test_chunks_and_steps_agree_closely(kind):
    runs = [(150, 0, False)]
    a, b = Run(kind, pl.BF16, runs, 3, 64, 96, True, exact=True), Run(kind, pl.BF16, runs, 3, 64, 96, False, exact=True)
    for x, y in ((a.got, b.got), (a.states, b.states), (a.den, b.den)):
        assert np.abs(x - y).max() <= 5e-5 * np.abs(y).max()


@pytest.mark.parametrize("kind", [KEYED, GATED])
@pytest.mark.parametrize("chunked", [False, True])
def test_state_far_back_decides(kind, chunked):
    """Only the first token writes, and it is hundreds of tokens later that its value is asked for."""
    def edit(z, off, a2b, ib, fb):
        z[:, off["k"]:off["k"] + 32], z[:, off["q"]:off["q"] + 32] = 0, 0
        z[0, off["k"]:off["k"] + 32], z[-1, off["q"]:off["q"] + 32] = 2.0, 2.0
        z[:, off["a"]:off["a"] + 11], a2b[:] = 0, 60.0
        ib[:], fb[:] = 0, 1000.0
        z[:, [off["i"], off["f"]]] = 0
    r = Run(kind, pl.BF16, [(300, 0, True)], 1, 32, 40, chunked, seed=4, cap=30.0, edit=edit)
    r.check(1e-4)
    assert np.abs(r.want[-1]).max() > 10 * np.abs(r.want[1:-1]).max() and np.abs(r.got[-1] - r.want[-1]).max() < 1e-3 * np.abs(r.want[-1]).max()


PREPS = [(6, 2, 96, 130, 96), (5, 1, 17, 9, 6), (4, 2, 128, 64, 32), (3, 3, 256, 256, 0), (8, 2, 40, 72, 40)]


def prepared(L, t, z, ldz, T, at, H, G, dim, vdim, rot, rng, n_cells=40, pairs=1):
    """(pi_gqa_prep with every option, a check of what it should leave given z)."""
    off_k, off_v, hd = at + H * dim + 1, at + H * dim + 1 + G * dim + 2, L.pi_k_gqa_head_ld(t, dim, vdim)
    pos, cells = rng.integers(0, 5000, T).astype(np.int32), rng.permutation(n_cells)[:T]
    qn, kn = (1 + 0.3 * rng.standard_normal((2, dim))).astype(np.float32)
    temp = (1 + 0.5 * rng.standard_normal(H)).astype(np.float32)
    b = dict(cs=pl.DevBuf.zeros(8 * T * max(rot // 2, 1)), q=pl.DevBuf.zeros(4 * T * H * hd), cache=pl.DevBuf.zeros(4 * n_cells * G * 2 * hd), cell=i32(cells), q_norm=dev(qn), k_norm=dev(kn),
             temp=dev(temp))
    pb = i32(pos)
    if rot:
        pl.check(L.pi_k_rope_angles(pb.ptr, T, rot, 700.0, b["cs"].ptr, None))
        pl.sync()
    p = filled(pl.GqaPrep, z=z, ldz=ldz, T=T, n_head=H, n_kv=G, dim=dim, vdim=vdim, rot_dim=rot, off_k=off_k, off_v=off_v, hd=hd, eps=1e-5, rot_pairs=pairs, unit_v=1, **b)

    def check(z64):
        tail = {"q": np.eye(H * dim), "k": np.eye(G * dim), "v": np.eye(G * vdim)}
        rows = np.concatenate([z64[:, at:at + H * dim], z64[:, off_k:off_k + G * dim], z64[:, off_v:off_v + G * vdim]], 1)
        n = rows.shape[1]
        for x, (a, w) in (("q", (0, H * dim)), ("k", (H * dim, G * dim)), ("v", (H * dim + G * dim, G * vdim))):
            full = np.zeros((w, n))
            full[:, a:a + w] = tail[x]
            tail[x] = full
        tail.update({"q.norm": qn, "k.norm": kn})
        wq, wk, wv = o.queries_and_cells(rows, pos, tail, dict(heads=H, kv_heads=G, dim=dim, vdim=vdim, rot={"dims": rot, "base": 700.0}), 1e-5)
        wq = wq * temp[None, :, None]
        got_q, got_c = fetch(b["q"], t, (T, H, hd)), fetch(b["cache"], t, (n_cells, G, 2, hd))
        for got, want in ((got_q[..., :dim], wq), (got_c[cells][:, :, 0, :dim], wk), (got_c[cells][:, :, 1, :vdim], wv)):
            assert np.abs(got - want).max() <= tol(t) * np.abs(want).max()
        assert not got_q[..., dim:].any() and not got_c[:, :, 0, dim:].any() and not got_c[:, :, 1, vdim:].any()
        assert not got_c[[c for c in range(n_cells) if c not in cells]].any()
    return p, check


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,pairs", [(6, 1), (33, 1), (6, 0)])
@pytest.mark.parametrize("H,G,dim,vdim,rot", PREPS)
def test_queries_and_cells(monkeypatch, t, T, pairs, H, G, dim, vdim, rot):
    """In steps and in prompts (several heads a wave), and for the rotation of the other designs."""
    if not pairs:
        monkeypatch.setattr(o, "rotate_neighbours", rotate_halves)
    L, rng = pl.init(), np.random.default_rng(dim)
    ldz = (H * dim + G * (dim + vdim) + 20) // 16 * 16
    z = (2 * rng.standard_normal((T, ldz))).astype(np.float32)
    zb = dev(z)
    p, check = prepared(L, t, zb, ldz, T, 0, H, G, dim, vdim, rot, rng, pairs=pairs)
    pl.check(L.pi_k_gqa_prep(t, C.byref(p), None, None))
    pl.sync()
    check(z.astype(np.float64))


@pytest.mark.parametrize("kind", [KEYED, GATED])
@pytest.mark.parametrize("t", TYPES)
def test_state_step_beside_queries_and_cells(kind, t):
    """Both in one launch, each as if it were alone."""
    rng, checks = np.random.default_rng(8), []
    H, G, dim, vdim, rot = 6, 2, 40, 72, 24

    def prep(z, ldz, T):
        p, check = prepared(pl.init(), t, z, ldz, T, 0, H, G, dim, vdim, rot, rng)
        checks.append(check)
        return p
    r = Run(kind, t, [(1, 3, False), (5, 0, True), (2, 4, True)], 3, 48, 80, False, beside=dict(rows=H * dim + G * (dim + vdim) + 3, prep=prep))
    r.check(2e-5)
    checks[0](r.z)


@pytest.mark.parametrize("t,parts,wide", [(pl.F32, 1, 0), (pl.BF16, 1, 0), (pl.BF16, 5, 0), (pl.BF16, 1, 1), (pl.BF16, 3, 1)])
@pytest.mark.parametrize("window", [1, 2, 17, 64, 65, 128, 200, 1000])
def test_attention_in_a_window(t, parts, wide, window):
    seqs = [(70, 0), (9, 190), (1, 300), (130, 61)] if wide else [(1, 0), (3, 126), (1, 127), (1, 700), (17, 30), (2, 0)]
    for H, G, dim, vdim in ((6, 2, 64, 40), (4, 1, 128, 128)):
        got, want = attend(t, np.random.default_rng(window), seqs, H, G, dim, vdim, parts, wide, dim ** -0.5, -np.inf, window=window, out_scale=0.6)
        assert np.abs(got - want).max() <= tol(t, 1.5) * np.abs(want).max()


@pytest.mark.parametrize("t,parts,wide", [(pl.F32, 1, 0), (pl.BF16, 1, 0), (pl.BF16, 7, 0), (pl.BF16, 1, 1), (pl.BF16, 4, 1)])
@pytest.mark.parametrize("window", [63, 64, 65, 127, 128, 129, 200])
def test_the_edge_of_a_window(t, parts, wide, window):
    """A score that stands out sits on the last cell a token sees, and for another token one cell further back."""
    n, b = (40 if wide else 6), 400
    spike = [(0, 0, b + 1 - window, 1), (0, 2, b + 2 - window, 2)]
    got, want = attend(t, np.random.default_rng(1), [(n, b)], 4, 2, 64, 64, parts, wide, 64 ** -0.5, -np.inf, spike, window=window)
    assert np.abs(want[0, 1]).max() > 2 > 1.5 > np.abs(want[2, 2]).max()
    assert np.abs(got - want).max() <= tol(t, 1.5) * np.abs(want).max()


@pytest.mark.parametrize("t,parts,wide", [(pl.F32, 1, 0), (pl.BF16, 1, 0), (pl.BF16, 3, 0), (pl.BF16, 2, 1)])
def test_first_cells_given(t, parts, wide):
    """What a token sees first as a list, for positions with gaps."""
    first = lambda s, i: [0, 57, 3][s] + (i * (1 + s)) // 2  # noqa: E731
    got, want = attend(t, np.random.default_rng(5), [(33, 100), (40, 60), (1, 9)], 4, 2, 32, 64, parts, wide, 0.3, -np.inf, window=7, first=first)
    assert np.abs(got - want).max() <= tol(t, 1.5) * np.abs(want).max()


@pytest.mark.parametrize("t", TYPES)
def test_shifted_keys_in_neighbouring_pairs(t):
    L, rng = pl.init(), np.random.default_rng(4)
    n, G, dim, rot = 9, 2, 40, 24
    hd = L.pi_k_gqa_head_ld(t, dim, dim)
    k = rng.standard_normal((n, G, dim))
    pos, delta = rng.integers(50, 900, n), np.array([0, 5, -7, 0, 1, -50, 300, 2, 0], np.int32)
    cells = np.zeros((n, G, 2, hd), np.float32)
    cells[:, :, 0, :dim], cells[:, :, 1, :dim] = o.rotate_neighbours(k, pos, rot, 800.0), k
    cb, db = store(cells, t), i32(delta)
    pl.check(L.pi_k_gqa_shift(t, cb.ptr, n, G, hd, rot, 800.0, 1, db.ptr, None))
    pl.sync()
    got = fetch(cb, t, cells.shape)
    assert np.abs(got[:, :, 0, :dim] - o.rotate_neighbours(k, pos + delta, rot, 800.0)).max() < (4e-2 if t == pl.BF16 else 1e-5)
    assert np.array_equal(got[:, :, 1], as_stored(cells[:, :, 1], t))


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,H,vd,silu,den", [(1, 3, 50, 0, 1), (7, 8, 128, 1, 0), (3, 5, 256, 0, 0), (16, 1, 9, 1, 1)])
def test_gated_norm_of_heads(t, T, H, vd, silu, den):
    L, rng = pl.init(), np.random.default_rng(vd)
    n = H * vd
    x, z, w = rng.standard_normal((T, n)).astype(np.float32) * 4, rng.standard_normal((T, n + 9)).astype(np.float32), rng.random(n).astype(np.float32)
    d = (0.01 + rng.random((T, H))).astype(np.float32)
    xb, zb, wb, db, att = dev(x), dev(z), dev(w), dev(d), pl.DevBuf.zeros(4 * T * (n + 4))
    g = filled(pl.GateNorm, o=xb, z=zb, w=wb, ldz=n + 9, off_gate=4, n=n, T=T, eps=1e-3, att=att, ld_att=n + 4, scale=0.7, heads=H, silu=silu, den=db if den else None)
    pl.check(L.pi_k_gate_norm(t, C.byref(g), None))
    pl.sync()
    heads = x.astype(np.float64).reshape(T, H, vd) / (d[:, :, None] if den else 1)
    want = 0.7 * o.unit(heads, 1e-3).reshape(T, n) * w * (o.silu if silu else o.sigmoid)(z[:, 4:4 + n].astype(np.float64))
    got = fetch(att, t, (T, n + 4))
    assert np.abs(got[:, :n] - want).max() <= tol(t) * np.abs(want).max() and not got[:, n:].any()


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,cols,ol", [(1, 100, 0), (5, 3000, 0), (3, 5001, 0), (16, 256, 1), (7, 72, 1), (4, 4096, 0), (2, 8192, 0), (2, 12000, 0), (3, 33, 0)])
@pytest.mark.parametrize("mix,gate,norm", [(1, 1, 1), (1, 0, 1), (0, 0, 1), (0, 0, 0), (1, 1, 0)])
def test_residual_norm(t, T, cols, ol, mix, gate, norm):
    if ol and t == pl.F32:
        pytest.skip("the operand layout is a bf16 layout")
    L, rng = pl.init(), np.random.default_rng(T + cols)
    x, y, z = rng.standard_normal((3, T, cols + 8)).astype(np.float32)
    x, y, gb, w, ld = x[:, :cols].copy(), y[:, :cols].copy(), rng.standard_normal(cols).astype(np.float32), (1 + 0.3 * rng.standard_normal(cols)).astype(np.float32), (cols + 63) // 64 * 64
    xb, yb, zb, bb, wb, keep, h = dev(x), dev(y), dev(z), dev(gb), dev(w), pl.DevBuf.zeros(4 * T * cols), pl.DevBuf.zeros(4 * max(T, 16) * ld)
    p = filled(pl.ResNorm, x=xb, mix=yb if mix else None, gate_z=zb if gate else None, gate_b=bb if gate else None, w=wb if norm else None, ld_gate=cols + 8, off_gate=4, T=T, cols=cols,
               alpha=1.3, eps=1e-4, out=xb, keep=keep, h=h, ld=ld, ol=ol)
    pl.check(L.pi_k_res_norm(t, C.byref(p), None))
    pl.sync()
    x64 = x.astype(np.float64)
    s = 1.3 * x64 + y * (o.sigmoid(z[:, 4:4 + cols].astype(np.float64) + gb) if gate else 1) if mix else x64
    want = o.rms_norm(s, w, 1e-4) if norm else s
    got = xb.download(np.float32).reshape(T, cols)
    assert np.abs(got - want).max() <= 3e-6 * np.abs(want).max() and np.array_equal(got, keep.download(np.float32).reshape(T, cols))
    oper = fetch(h, t, (ld // 8, 16, 8)).transpose(1, 0, 2).reshape(16, ld)[:T, :cols] if ol else fetch(h, t, (T, ld))[:, :cols]
    assert np.array_equal(oper, as_stored(got, t))


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,ff", [(1, 9), (30, 1100), (3, 4097)])
def test_plain_glu(t, T, ff):
    L, rng = pl.init(), np.random.default_rng(ff)
    ldz, ff_ld = (2 * ff + 15) // 16 * 16 + 16, (ff + 127) // 128 * 128
    z = (2 * rng.standard_normal((T, ldz))).astype(np.float32)
    zb, act = dev(z), pl.DevBuf.zeros(4 * T * ff_ld)
    f = filled(pl.FfnFront, off_glu=16, ff=ff, ff_ld=ff_ld, off_score=-1, limit=np.inf, gain=1.0, act=act, ld_act=ff_ld, plain_up=1)
    pl.check(L.pi_k_ffn_front(t, zb.ptr, ldz, T, C.byref(f), None))
    pl.sync()
    g = z[:, 16:16 + 2 * ff].reshape(T, ff, 2).astype(np.float64)
    want, got = o.silu(g[..., 0]) * g[..., 1], fetch(act, t, (T, ff_ld))
    assert np.abs(got[:, :ff] - want).max() <= tol(t) * np.abs(want).max() and not got[:, ff:].any()


@pytest.mark.parametrize("T,ff,cols,rows2", [(1, 24, 256, 0), (16, 1000, 512, 100), (5, 33, 768, 300), (3, 3000, 1024, 1024), (2, 9000, 256, 40)])
@pytest.mark.parametrize("one,limit", [(0.0, np.inf), (1.0, 0.8)])
def test_glu_of_a_step(T, ff, cols, rows2, one, limit):
    L, rng = pl.init(), np.random.default_rng(ff)
    W, W2 = rounded(2 * rng.standard_normal((ff, 2, cols)) / np.sqrt(cols)), rounded(rng.standard_normal((max(rows2, 1), cols)) / np.sqrt(cols))
    x = rounded(rng.standard_normal((T, cols)))
    ol = np.zeros((cols // 8, 16, 8), np.float32)
    ol[:, :T] = x.reshape(T, cols // 8, 8).transpose(1, 0, 2)
    wb, w2b, xb, ld, y2 = store(W, pl.BF16), store(W2, pl.BF16), store(ol, pl.BF16), (ff + 127) // 128 * 128, pl.DevBuf.zeros(4 * T * max(rows2, 1))
    act = pl.DevBuf.zeros(2 * T * ld)
    pl.check(L.pi_k_gemm_bf16_ol_glu(wb.ptr, ff, xb.ptr, limit, 1.0, one, act.ptr, ld, w2b.ptr if rows2 else None, rows2, y2.ptr, cols, T, None))
    pl.sync()
    x64 = x.astype(np.float64)
    g, u = np.minimum(x64 @ W[:, 0].T, limit), np.clip(x64 @ W[:, 1].T, -limit, limit)
    want, got = o.silu(g) * (u + one), fetch(act, pl.BF16, (T, ld))
    assert np.abs(got[:, :ff] - want).max() <= tol(pl.BF16) * np.abs(want).max() and not got[:, ff:].any()
    if rows2:
        want = x64 @ W2.T
        assert np.abs(y2.download(np.float32).reshape(T, rows2) - want).max() <= 1e-5 * np.abs(want).max()


@pytest.mark.parametrize("T,rows,ld", [(1, 100, 128), (16, 256, 640), (7, 5000, 256)])
@pytest.mark.parametrize("gate", [0, 1])
def test_gated_sum_of_a_step(T, rows, ld, gate):
    L, rng = pl.init(), np.random.default_rng(rows)
    W, a = rounded(rng.standard_normal((rows, ld)) / np.sqrt(ld)), rounded(rng.standard_normal((T, ld)))
    x, z, b = rng.standard_normal((T, rows)).astype(np.float32), rng.standard_normal((T, rows + 9)).astype(np.float32), rng.standard_normal(rows).astype(np.float32)
    wb, ab, xb, zb, bb, out = store(W, pl.BF16), store(a, pl.BF16), dev(x), dev(z), dev(b), pl.DevBuf.zeros(4 * T * rows)
    s = filled(pl.LayerOut, x=xb, wo=wb, att=ab, rows=rows, ld_att=ld, T=T, out=out, scaled=1, alpha=-0.4, gate_z=zb if gate else None, gate_b=bb if gate else None, ld_gate=rows + 9, off_gate=7)
    pl.check(L.pi_k_layer_out_step(C.byref(s), None))
    pl.sync()
    want = -0.4 * x.astype(np.float64) + a.astype(np.float64) @ W.T * (o.sigmoid(z[:, 7:7 + rows].astype(np.float64) + b) if gate else 1)
    assert np.abs(out.download(np.float32).reshape(T, rows) - want).max() <= 1e-5 * np.abs(want).max()


def test_bad_arguments_are_errors():
    L, buf = pl.init(), pl.DevBuf.zeros(1 << 16)
    base = dict(z=buf, ldz=256, T=1, n_head=2, dim=16, vdim=16, off_q=0, off_k=32, off_v=64, state=buf, runs=buf, n_runs=1, o=buf, q_scale=1.0, plain=1)
    keyed = dict(base, decay_kind=KEYED, a2=buf, a2_b=buf, off_a=96, rank=8, rank_ld=8, tau=1.0)
    gated = dict(base, decay_kind=GATED, i_b=buf, f_b=buf, den=buf, off_i=96, off_f=98, cap=1.0)
    for good, spoils in ((keyed, (dict(rank_ld=4), dict(off_a=250), dict(tau=0.0), dict(a2=None), dict(rank=600, rank_ld=600), dict(slot_ld=5))),
                         (gated, (dict(off_f=255), dict(cap=0.0), dict(den=None), dict(slot_ld=520))), (base, (dict(decay_kind=7),))):
        for spoil in spoils:
            p = filled(pl.Linear, **{k: v for k, v in dict(good, **spoil).items() if v is not None})
            assert L.pi_k_linear_step(pl.BF16, C.byref(p), None, None) != 0, spoil
    p = filled(pl.Linear, **keyed)
    assert L.pi_k_linear_step_beside(pl.BF16, C.byref(p), None, None) != 0
    r = filled(pl.ResNorm, x=buf, out=buf, T=1, cols=8, h=buf, ld=4)
    assert L.pi_k_res_norm(pl.BF16, C.byref(r), None) != 0                        # operand rows shorter than the columns
    assert L.pi_k_gemm_bf16_ol_glu(buf.ptr, 8, buf.ptr, 1.0, 1.0, 0.0, buf.ptr, 8, None, 0, None, 128, 1, None) != 0
    g = filled(pl.GateNorm, o=buf, z=buf, w=buf, ldz=64, off_gate=0, n=30, T=1, att=buf, ld_att=32, scale=1.0, heads=4)
    assert L.pi_k_gate_norm(pl.BF16, C.byref(g), None) != 0                       # heads of unequal size
