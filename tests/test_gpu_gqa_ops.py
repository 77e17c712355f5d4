"""Operators of layers with one norm: embedding, layer norm, clamped GLU, expert choice, grouped-query attention - one by one against the
plain implementations (tests/plain_pibalorn.py) in bf16 and fp32."""
import ctypes as C

import numpy as np
import pytest

import plain_pibalorn as o
from powerinfer_amd import lib as pl
from powerinfer_amd.checkpoint import bf16_bits
from test_gpu_latent_ops import TYPES, as_stored, dev, fetch, group_args, i32, padded, rounded, store, tol

pytestmark = pytest.mark.gpu


def filled(cls, **kw):
    s = cls()
    for k, v in kw.items():
        assert any(k == f[0] for f in cls._fields_), k
        setattr(s, k, v.ptr if isinstance(v, pl.DevBuf) else v)
    return s


@pytest.mark.parametrize("cols,buckets,muls", [(64, 11, (29, 13)), (300, 1, (3, 5)), (1000, 50, (1 << 33, 1000003))])
def test_embed_bigram(cols, buckets, muls):
    L, rng = pl.init(), np.random.default_rng(cols)
    table, bg = rounded(rng.standard_normal((40000, cols)))[:40000], rounded(rng.standard_normal((buckets + 1, cols)))
    toks, prev = [39999, 0, 3, 39998, 5], [-1, 39999, 0, 39997, -1]
    x, x0, tb, bb, ib, pb = pl.DevBuf(4 * 5 * cols), pl.DevBuf(4 * 5 * cols), store(table, pl.BF16), store(bg, pl.BF16), i32(toks), i32(prev)
    for with_bigram, carry in ((True, 0), (False, 1)):
        pl.check(L.pi_k_embed_bigram(tb.ptr, cols, ib.ptr, pb.ptr, 5, 2.5, bb.ptr if with_bigram else None, buckets, *muls, carry, x.ptr, x0.ptr, None))
        pl.sync()
        rows = [o.bigram_rows([t], None if p < 0 else p, buckets, *muls)[0] for t, p in zip(toks, prev)]
        want = table[toks].astype(np.float64) * 2.5 + (bg[rows] if with_bigram else 0)
        got = x.download(np.float32).reshape(5, cols)
        assert np.abs(got - want).max() < 1e-6 * np.abs(want).max() and np.array_equal(got, x0.download(np.float32).reshape(5, cols))
        assert pb.download(np.int32).tolist() == (toks if carry else prev)


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,cols,ol,adds", [(1, 100, 0, 0), (5, 3000, 0, 3), (3, 5000, 0, 1), (3, 4500, 0, 2), (16, 256, 1, 3), (7, 72, 1, 0), (9, 640, 0, 2)])
def test_layer_norm(t, T, cols, ol, adds):
    if ol and t == pl.F32:
        pytest.skip("the operand layout is a bf16 layout")
    L, rng = pl.init(), np.random.default_rng(T + cols)
    x, x0 = (5 + 3 * rng.standard_normal((2, T + 2, cols))).astype(np.float32)
    w, step = (1 + 0.3 * rng.standard_normal((2, cols))).astype(np.float32)
    rows = rng.permutation(T + 2)[:T].astype(np.int32) if not adds else np.arange(T, dtype=np.int32)
    ld = (cols + 63) // 64 * 64
    xb, rb, wb, ab, sb, out = dev(x), i32(rows), dev(w), dev(x0), dev(step), pl.DevBuf.zeros(4 * max(T, 16) * ld)
    pl.check(L.pi_k_layer_norm(t, xb.ptr, None if adds else rb.ptr, T, cols, 1e-5, wb.ptr, ab.ptr if adds & 1 else None, sb.ptr if adds & 2 else None, out.ptr, ld, ol, None))
    pl.sync()
    src = x.astype(np.float64) + (x0 if adds & 1 else 0) + (step if adds & 2 else 0)
    want = o.layer_norm(src[rows], w, 1e-5)
    got = fetch(out, t, (ld // 8, 16, 8)).transpose(1, 0, 2).reshape(16, ld)[:T, :cols] if ol else fetch(out, t, (T, ld))[:, :cols]
    assert np.abs(got - want).max() <= tol(t) * np.abs(want).max()
    assert np.abs(xb.download(np.float32).reshape(x.shape)[:T] - src[:T]).max() < 1e-5        # what was added stays in the residual stream


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("tile", [0, 64, 128])
@pytest.mark.parametrize("ff,cols,T,y_f32,limit", [(25, 100, 1, 0, 1.0), (96, 64, 37, 0, 0.5), (130, 192, 300, 1, 2.0), (33, 320, 129, 0, 1e9)])
def test_group_gemm_clamped_glu(t, tile, ff, cols, T, y_f32, limit):
    if tile and t == pl.F32:
        pytest.skip("the tiled product is bf16")
    L, rng = pl.init(), np.random.default_rng(ff)
    G, ld = 3, (cols + 63) // 64 * 64
    W, x = rounded(2 * rng.standard_normal((G, ff, 2, cols)) / np.sqrt(cols)), as_stored(rng.standard_normal((T, G, cols)), t)
    wb, xb, ldy = store(padded(W.reshape(-1, cols), ld), pl.BF16), store(padded(x.reshape(-1, cols), ld), t), G * ff + 3
    y = pl.DevBuf.zeros(4 * T * ldy)
    g = group_args(W=wb.ptr, w_gs=2 * ff * ld, rows=2 * ff, cols=ld, ldw=ld, n_group=G, x=xb.ptr, x_gs=ld, ldx=G * ld, T=T, y=y.ptr, y_gs=ff, ldy=ldy,
                   y_f32=y_f32, alpha=1.0, glu=1, glu_limit=limit, glu_gain=1.702)
    pl.check(L.pi_k_group_gemm_tile(C.byref(g), tile, None) if tile else L.pi_k_group_gemm(t, C.byref(g), None))
    pl.sync()
    got = fetch(y, pl.F32 if y_f32 else t, (T, ldy))[:, :G * ff].reshape(T, G, ff)
    want = np.stack([o.clamped_glu(x[:, k].astype(np.float64), W[k, :, 0], W[k, :, 1], np.eye(ff), limit) for k in range(G)], 1)
    assert np.abs(got - want).max() <= (tol(t) if not y_f32 else 1e-5) * np.abs(want).max()


def front(z, t, ff, off_glu, off_score, limit, E, off_router, top):
    """(pi_ffn_front, its buffers) for z [T, ldz]."""
    T, ff_ld = z.shape[0], (ff + 63) // 64 * 64
    act, ids, wts = pl.DevBuf.zeros(4 * T * (ff_ld + 8)), i32(np.zeros((T, max(top, 1)))), dev(np.zeros((T, max(top, 1)), np.float32))
    return filled(pl.FfnFront, off_glu=off_glu, ff=ff, ff_ld=ff_ld if ff else 0, off_score=off_score, limit=limit, gain=1.702, act=act, ld_act=ff_ld + 8, off_router=off_router,
                  n_expert=E, n_top=top, ids=ids, weights=wts), (act, ids, wts, ff_ld + 8)


def check_front(z, t, f, bufs):
    act, ids, wts, ld = bufs
    T = z.shape[0]
    if f.ff:
        g = z[:, f.off_glu:f.off_glu + 2 * f.ff].reshape(T, f.ff, 2).astype(np.float64)
        want = np.stack([o.clamped_glu(g[i], np.array([[1.0, 0.0]]), np.array([[0.0, 1.0]]), np.eye(1), f.limit)[:, 0] for i in range(T)])
        if f.off_score >= 0:
            want *= o.sigmoid(z[:, f.off_score:f.off_score + 1].astype(np.float64))
        got = fetch(act, t, (T, ld))
        assert np.abs(got[:, :f.ff] - want).max() <= tol(t) * np.abs(want).max() and not got[:, f.ff:f.ff_ld].any()
    if f.n_expert:
        e, w = o.route_softmax(z[:, f.off_router:f.off_router + f.n_expert].astype(np.float64), np.eye(f.n_expert), f.n_top)
        assert np.array_equal(ids.download(np.int32).reshape(T, -1), e) and np.abs(wts.download(np.float32).reshape(T, -1) - w).max() < 2e-6


def prepped(q, k, v, pos, m, eps):
    """Oracle's (queries, keys, values) of projections q [T, H, D], k, v [T, G, ..]."""
    turn = lambda x: o.unit(o.rotate_halves(x, pos, m["rot"], m["base"]), eps) if m["unit"] else o.rotate_halves(x, pos, m["rot"], m["base"])  # noqa: E731
    return turn(q), turn(k), v


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("H,G,dim,vdim,rot,unit,ff,E,top", [(6, 2, 96, 96, 96, 1, 0, 0, 0), (5, 1, 17, 17, 6, 1, 30, 5, 2), (4, 2, 128, 64, 32, 0, 2100, 0, 0), (3, 3, 256, 256, 0, 1, 7, 300, 8),
                                                            (8, 2, 40, 72, 40, 1, 0, 64, 6)])
def test_gqa_prep_and_front(t, H, G, dim, vdim, rot, unit, ff, E, top):
    L, rng = pl.init(), np.random.default_rng(dim)
    T, n_cells, eps, own = 6, 40, 1e-5, vdim != dim
    off_k = H * dim + 3
    off_v = off_k + G * dim + 1 if own else off_k
    off_glu = (off_v + G * vdim + 15) // 16 * 16
    ldz = (off_glu + 2 * ff + 8 + E + 15) // 16 * 16
    z = (2 * rng.standard_normal((T, ldz))).astype(np.float32)
    pos, cells = rng.integers(0, 5000, T).astype(np.int32), rng.permutation(n_cells)[:T]
    hd = L.pi_k_gqa_head_ld(t, dim, vdim)
    assert hd >= max(dim, vdim) and hd % 32 == 0
    f, bufs = front(z, t, ff, off_glu, off_glu + 2 * ff if ff == 30 else -1, 1.1, E, off_glu + 2 * ff + 1, top)
    zb, cb, pb, q = dev(z), i32(cells), i32(pos), pl.DevBuf.zeros(4 * T * H * hd)
    cs, cache = pl.DevBuf.zeros(8 * T * max(rot // 2, 1)), pl.DevBuf.zeros(4 * n_cells * G * 2 * hd)
    if rot:
        pl.check(L.pi_k_rope_angles(pb.ptr, T, rot, 700.0, cs.ptr, None))
    p = filled(pl.GqaPrep, z=zb, ldz=ldz, T=T, n_head=H, n_kv=G, dim=dim, vdim=vdim, rot_dim=rot, off_k=off_k, off_v=off_v, hd=hd, unit=unit, cs=cs, eps=eps, q=q, cache=cache, cell=cb)
    pl.check(L.pi_k_gqa_prep(t, C.byref(p), C.byref(f), None))
    pl.sync()
    m = dict(rot=rot, base=700.0, unit=unit)
    z64 = z.astype(np.float64)
    wq, wk, wv = prepped(z64[:, :H * dim].reshape(T, H, dim), z64[:, off_k:off_k + G * dim].reshape(T, G, dim), z64[:, off_v:off_v + G * vdim].reshape(T, G, vdim), pos, m, eps)
    got_q, got_c = fetch(q, t, (T, H, hd)), fetch(cache, t, (n_cells, G, 2, hd))
    for got, want in ((got_q[..., :dim], wq), (got_c[cells][:, :, 0, :dim], wk), (got_c[cells][:, :, 1, :vdim], wv)):
        assert np.abs(got - want).max() <= tol(t) * np.abs(want).max()
    assert not got_q[..., dim:].any() and not got_c[:, :, 0, dim:].any() and not got_c[:, :, 1, vdim:].any()
    assert not got_c[[c for c in range(n_cells) if c not in cells]].any()
    check_front(z, t, f, bufs)


def attend(t, rng, seqs, H, G, dim, vdim, parts, wide, scale, sink, spike=(), window=0, first=None, out_scale=1.0):
    """seqs: (tokens of the step, cells before them) per sequence.  Runs pi_k_gqa_attn on scattered cells; returns (got, want) [T, H, vdim].
    spike: (sequence, token, cell, head) whose score is made to stand out.  window, first (a function of sequence and token): what the tokens
    see (without the soft-max's own entry)."""
    L = pl.init()
    hd, per, T = L.pi_k_gqa_head_ld(t, dim, vdim), H // G, sum(n for n, _ in seqs)
    pool = sum(n + b for n, b in seqs) + 7
    free = list(rng.permutation(pool))
    list_ld = max(n + b for n, b in seqs) + 2
    lists = np.zeros((len(seqs), list_ld), np.int32)
    q, cache = as_stored(rng.standard_normal((T, H, dim)), t), as_stored(rng.standard_normal((pool, G, 2, max(dim, vdim))), t)
    work, seq_of, vis, at = [], [], [], 0
    want = np.empty((T, H, vdim))
    for s, (n, b) in enumerate(seqs):
        cells = [free.pop() for _ in range(n + b)]
        lists[s, :n + b] = cells
        for x in spike:
            if x[0] == s:
                cache[cells[x[2]], x[3] // per, 0, :dim] = as_stored(4 * q[at + x[1], x[3]], t)
        rows, step = n * per, L.pi_k_gqa_rows(wide)
        work += [[at, r, min(step, rows - r), s] for r in range(0, rows, step)]
        seq_of += [s] * n
        vis += list(range(b + 1, b + n + 1))
        k, v = cache[cells][:, :, 0, :dim].astype(np.float64), cache[cells][:, :, 1, :vdim].astype(np.float64)
        if sink == -np.inf:
            for a in range(H):
                lo = np.array([first(s, i) if first else max(b + i + 1 - window, 0) if window else 0 for i in range(n)])[:, None]
                sc = np.where((np.arange(n + b)[None] <= np.arange(b, b + n)[:, None]) & (np.arange(n + b)[None] >= lo), q[at:at + n, a].astype(np.float64) @ k[:, a // per].T * scale, -np.inf)
                e = np.exp(sc - sc.max(1, keepdims=True))
                want[at:at + n, a] = e / e.sum(1, keepdims=True) @ v[:, a // per]
        else:
            want[at:at + n] = o.grouped_attention(q[at:at + n].astype(np.float64), k, v, np.arange(b, b + n), np.arange(n + b), scale)
        at += n
    pad = np.zeros((pool, G, 2, hd), np.float32)
    pad[:, :, 0, :dim], pad[:, :, 1, :vdim] = cache[:, :, 0, :dim], cache[:, :, 1, :vdim]
    qp = np.zeros((T, H, hd), np.float32)
    qp[..., :dim] = q
    ld = H * vdim + 5
    qb, cb, lb, vb, att = store(qp, t), store(pad, t), i32(lists), i32(vis), pl.DevBuf.zeros(4 * T * ld)
    wb = i32(work if t == pl.BF16 else seq_of)
    fb = i32([first(s, i) for s, (n, _) in enumerate(seqs) for i in range(n)]) if first else None
    scratch = pl.DevBuf(4 * max(L.pi_k_gqa_scratch_floats(len(work), wide, G, hd, parts), 1))
    a = filled(pl.GqaAttn, out_scale=out_scale, window=window, first=fb, q=qb, cache=cb, lists=lb, list_ld=list_ld, work=wb, n_vis=vb, n_work=len(work), T=T, n_head=H, n_kv=G, dim=dim, vdim=vdim, hd=hd, n_parts=parts, wide=wide,
               scale=scale, sink=sink, scratch=scratch, att=att, ld_att=ld)
    pl.check(L.pi_k_gqa_attn(t, C.byref(a), None))
    pl.sync()
    got = fetch(att, t, (T, ld))
    assert not got[:, H * vdim:].any()
    return got[:, :H * vdim].reshape(T, H, vdim), want * out_scale


SHAPES = [(6, 2, 96, 96), (5, 1, 17, 17), (4, 4, 32, 20), (8, 1, 64, 64), (16, 2, 128, 128), (3, 3, 130, 130), (40, 2, 40, 64), (2, 1, 256, 250)]


@pytest.mark.parametrize("t,parts,wide", [(pl.F32, 1, 0), (pl.BF16, 1, 0), (pl.BF16, 5, 0), (pl.BF16, 64, 0), (pl.BF16, 1, 1), (pl.BF16, 3, 1)])
@pytest.mark.parametrize("H,G,dim,vdim", SHAPES)
def test_grouped_attention(t, parts, wide, H, G, dim, vdim):
    rng = np.random.default_rng(dim)
    seqs = [(70, 0), (9, 190), (1, 300), (130, 61)] if wide else [(1, 0), (3, 126), (1, 127), (1, 700), (17, 30), (2, 0)]
    got, want = attend(t, rng, seqs, H, G, dim, vdim, parts, wide, dim ** -0.5, 0.0)
    assert np.abs(got - want).max() <= tol(t, 1.5) * np.abs(want).max()


@pytest.mark.parametrize("t,parts,wide", [(pl.F32, 1, 0), (pl.BF16, 1, 0), (pl.BF16, 7, 0), (pl.BF16, 1, 1), (pl.BF16, 4, 1)])
def test_one_key_among_hundreds(t, parts, wide):
    """One score stands out: the first cell, the edges of the tiles, the token's own cell, and one just beyond what the token sees."""
    rng = np.random.default_rng(1)
    n = 40 if wide else 6
    spike = [(0, 0, c, 1) for c in (0,)] + [(0, 1, 63, 2), (0, 2, 64, 3), (0, 3, 127, 0), (0, 4, 128, 1), (0, 5, 400 + 5, 2), (0, 2, 400 + 3, 0)]
    got, want = attend(t, rng, [(n, 400)], 4, 2, 64, 64, parts, wide, 64 ** -0.5, 0.0, spike)
    assert np.abs(want[:6]).max() > 2 > 1.5 > np.abs(want[2, 0]).max()                # one value comes out whole; an average of hundreds does not
    assert np.abs(got - want).max() <= tol(t, 1.5) * np.abs(want).max()


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("wide", [0, 1])
def test_soft_max_without_the_entry(t, wide):
    for parts in (1, 4) if t == pl.BF16 else (1,):
        got, want = attend(t, np.random.default_rng(2), [(33, 100), (1, 0)], 4, 2, 32, 32, parts, wide, 0.3, -np.inf)
        assert np.abs(got - want).max() <= tol(t, 1.5) * np.abs(want).max()
        other, _ = attend(t, np.random.default_rng(2), [(33, 100), (1, 0)], 4, 2, 32, 32, parts, wide, 0.3, 0.0)
        assert np.abs(got - other)[33].max() > 0.1                                      # a token that sees only itself


@pytest.mark.parametrize("t", TYPES)
def test_scores_of_any_size(t):
    """Large scores (no overflow) and tiny ones (the added entry outweighs a lonely key)."""
    for scale in (30.0, 1e-3, -2.0):
        got, want = attend(t, np.random.default_rng(3), [(2, 0), (20, 50)], 2, 1, 64, 64, 1, 0, scale, 0.0)
        assert np.isfinite(got).all() and np.abs(got - want).max() <= tol(t, 3) * np.abs(want).max()


@pytest.mark.parametrize("t", TYPES)
def test_shifted_keys(t):
    """Rotating a stored key by a distance gives the key of the other position (the division by its size commutes with it)."""
    L, rng = pl.init(), np.random.default_rng(4)
    n, G, dim, rot = 9, 2, 40, 24
    hd = L.pi_k_gqa_head_ld(t, dim, dim)
    k = rng.standard_normal((n, G, dim))
    pos, delta = rng.integers(50, 900, n), np.array([0, 5, -7, 0, 1, -50, 300, 2, 0], np.int32)
    cells = np.zeros((n, G, 2, hd), np.float32)
    cells[:, :, 0, :dim] = o.unit(o.rotate_halves(k, pos, rot, 800.0), 1e-5)
    cells[:, :, 1, :dim] = k
    cb, db = store(cells, t), i32(delta)
    pl.check(L.pi_k_gqa_shift(t, cb.ptr, n, G, hd, rot, 800.0, 0, db.ptr, None))
    pl.sync()
    got = fetch(cb, t, cells.shape)
    assert np.abs(got[:, :, 0, :dim] - o.unit(o.rotate_halves(k, pos + delta, rot, 800.0), 1e-5)).max() < (2e-2 if t == pl.BF16 else 1e-5)
    assert np.array_equal(got[:, :, 1], as_stored(cells[:, :, 1], t))


@pytest.mark.parametrize("T,E,top,ff,cols,what", [(1, 6, 2, 24, 256, "gate"), (16, 40, 16, 72, 512, "merge"), (5, 3, 3, 33, 256, "both"), (7, 9, 1, 100, 768, "none"), (4, 0, 0, 0, 256, "merge")])
def test_step_launch_beside_the_experts(T, E, top, ff, cols, what):
    """pi_k_mix_up_step: experts' clamped GLU for the step's pairs, beside a gated norm and the merge of a split attention."""
    L, rng = pl.init(), np.random.default_rng(T)
    h = rounded(rng.standard_normal((T, cols)))
    ol = np.zeros((cols // 8, 16, 8), np.float32)
    ol[:, :T] = h.reshape(T, cols // 8, 8).transpose(1, 0, 2)
    up = rounded(2 * rng.standard_normal((max(E, 1), max(ff, 1), 2, cols)) / np.sqrt(cols))
    ids = np.stack([rng.permutation(E)[:top] for _ in range(T)]).astype(np.int32) if E else np.zeros((T, 1), np.int32)
    wts, ld = rng.random((T, max(top, 1))).astype(np.float32), (ff + 63) // 64 * 64 + 8
    hb, ub, ib, wb, act = store(ol, pl.BF16), store(up, pl.BF16), i32(ids), dev(wts), pl.DevBuf.zeros(2 * T * max(top, 1) * ld)
    n, hv = 90, 3 * 20
    og, zg, wg, attg = rng.standard_normal((T, n)).astype(np.float32), rng.standard_normal((T, n + 7)).astype(np.float32), rng.random(n).astype(np.float32), pl.DevBuf.zeros(2 * T * (n + 6))
    ob, zb, nb = dev(og), dev(zg), dev(wg)
    gate = filled(pl.GateNorm, scale=1.0, o=ob, z=zb, w=nb, ldz=n + 7, off_gate=5, n=n, T=T, eps=1e-5, att=attg, ld_att=n + 6)
    # parts of an attention: 3 heads of one group, 5 parts, one of them empty
    P, hd = 5, 32
    work = np.array([[t, 0, 3, 0] for t in range(T)], np.int32)
    acc, ml = rng.standard_normal((T, 16, P, hd)).astype(np.float32), np.stack([3 * rng.standard_normal((T, 16, P)), 1 + rng.random((T, 16, P))], -1).astype(np.float32)
    ml[:, :, 2], acc[:, :, 2] = [-np.inf, 0], 0
    sb, kb, attm = dev(np.concatenate([acc.ravel(), ml.ravel()])), i32(work), pl.DevBuf.zeros(2 * T * (hv + 2))
    merge = filled(pl.GqaAttn, out_scale=1.0, work=kb, n_work=T, T=T, n_head=3, n_kv=1, dim=20, vdim=20, hd=hd, n_parts=P, wide=0, scale=1.0, sink=0.0, scratch=sb, att=attm, ld_att=hv + 2)
    with_gate, with_merge = what in ("gate", "both"), what in ("merge", "both")
    pl.check(L.pi_k_mix_up_step(C.byref(merge) if with_merge else None, C.byref(gate) if with_gate else None, ub.ptr, E, ff, cols, 0.9, 1.702, hb.ptr, T, ib.ptr if E else None, wb.ptr,
                                top, act.ptr, ld, None))
    pl.sync()
    if E:
        got = fetch(act, pl.BF16, (T, top, ld))
        want = np.stack([[w * o.clamped_glu(h[t:t + 1].astype(np.float64), up[e, :, 0], up[e, :, 1], np.eye(ff), 0.9)[0] for e, w in zip(ids[t], wts[t])] for t in range(T)])
        assert np.abs(got[..., :ff] - want).max() <= tol(pl.BF16) * np.abs(want).max() and not got[..., ff:].any()
    want = o.unit(og.astype(np.float64), 1e-5) * wg * o.sigmoid(zg[:, 5:5 + n].astype(np.float64))
    got = fetch(attg, pl.BF16, (T, n + 6))
    assert np.abs(got[:, :n] - want * with_gate).max() <= tol(pl.BF16) * np.abs(want).max()
    e = np.exp(np.float64(ml[:, :3, :, 0]))
    want = (np.einsum("trp,trpc->trc", e, acc[:, :3]) / (1 + (e * ml[:, :3, :, 1]).sum(-1))[..., None])[..., :20].reshape(T, hv)
    got = fetch(attm, pl.BF16, (T, hv + 2))
    assert np.abs(got[:, :hv] - want * with_merge).max() <= tol(pl.BF16) * np.abs(want).max()


def test_place():
    L, rng = pl.init(), np.random.default_rng(6)
    a, b = bf16_bits(rng.standard_normal((5, 7))).reshape(5, 7), bf16_bits(rng.standard_normal((5, 7))).reshape(5, 7)
    out, ab, bb = pl.DevBuf.zeros(2 * 12 * 24), dev(a), dev(b)
    pl.check(L.pi_k_place_bf16(ab.ptr, 5, 7, out.ptr, 24, 8, 12, 1, 2, None))
    pl.check(L.pi_k_place_bf16(bb.ptr, 5, 7, out.ptr, 24, 8, 12, 2, 2, None))
    pl.sync()
    want = np.zeros((12, 24), np.uint16)
    want[1:11:2, 8:15], want[2:12:2, 8:15] = a, b
    assert np.array_equal(out.download(np.uint16).reshape(12, 24), want)


def test_bad_arguments_are_errors():
    L = pl.init()
    buf = pl.DevBuf.zeros(1 << 16)
    a = filled(pl.GqaAttn, out_scale=1.0, q=buf, cache=buf, lists=buf, list_ld=8, work=buf, n_vis=buf, n_work=1, T=1, n_head=3, n_kv=2, dim=32, vdim=32, hd=32, n_parts=1, scale=1.0, att=buf, ld_att=96)
    assert L.pi_k_gqa_attn(pl.BF16, C.byref(a), None) != 0                 # heads are no multiple of the groups
    a.n_kv, a.hd = 3, 64
    assert L.pi_k_gqa_attn(pl.BF16, C.byref(a), None) != 0                 # not the row length of this head size
    a.hd, a.n_parts = 32, 2
    assert L.pi_k_gqa_attn(pl.BF16, C.byref(a), None) != 0                 # parts without scratch
    assert L.pi_k_gqa_head_ld(pl.BF16, 257, 16) == 0 and L.pi_k_linear_supported(257, 4) == 0
    assert L.pi_k_layer_norm(pl.BF16, buf.ptr, buf.ptr, 1, 8, 1e-5, buf.ptr, buf.ptr, None, buf.ptr, 8, 0, None) != 0          # rows and additions
    g = group_args(W=buf.ptr, rows=5, cols=32, ldw=32, n_group=1, x=buf.ptr, ldx=32, T=1, y=buf.ptr, ldy=8, alpha=1.0, glu=1)
    assert L.pi_k_group_gemm(pl.F32, C.byref(g), None) != 0                # gate and up rows come in pairs
