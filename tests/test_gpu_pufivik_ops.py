"""Operators of the Pufivik path one by one against the plain implementations (tests/plain_pufivik.py) in bf16 and fp32: norms in groups, sums and
convolutions around a sublayer, scaled rotations, mixed values, attention with sinks, soft caps, mixed and gated heads, experts weighted at their input."""
import ctypes as C

import numpy as np
import pytest

import plain_pufivik as o
from powerinfer_amd import lib as pl
from test_gpu_gqa_ops import filled
from test_gpu_latent_ops import TYPES, as_stored, dev, fetch, group_args, i32, padded, rounded, store, tol

pytestmark = pytest.mark.gpu


def f64(a):
    return pl.DevBuf(host=np.asarray(a, np.float64))


def operand(buf, t, T, cols, ld, ol):
    return fetch(buf, t, (ld // 8, 16, 8)).transpose(1, 0, 2).reshape(16, ld)[:T, :cols] if ol else fetch(buf, t, (T, ld))[:, :cols]


def in_layout(x):
    """Rows of up to 16 tokens in the operand layout."""
    T, cols = x.shape
    out = np.zeros((cols // 8, 16, 8), np.float32)
    out[:, :T] = x.reshape(T, cols // 8, 8).transpose(1, 0, 2)
    return out


# ---- norms, sums, convolution -------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,cols,groups,ol", [(1, 100, 5, 0), (5, 3000, 8, 0), (3, 99, 3, 0), (16, 256, 4, 1), (7, 72, 1, 1), (2, 12000, 12, 0), (4, 64, 64, 0), (1, 1, 1, 0), (40, 520, 2, 0)])
@pytest.mark.parametrize("what", ["sum", "experts", "weighted experts", "norm only", "sum only"])
def test_sums_and_norms_in_groups(t, T, cols, groups, ol, what):
    if ol and t == pl.F32:
        pytest.skip("the operand layout is a bf16 layout")
    L, rng = pl.init(), np.random.default_rng(T + cols)
    ld, top, n = (cols + 63) // 64 * 64, 3, T + 2
    spread = np.repeat(10.0 ** rng.uniform(-1, 1, groups), cols // groups)             # groups of different sizes, so that one norm of all differs
    x, mix = rng.standard_normal((n, cols)).astype(np.float32) * spread.astype(np.float32), (rng.standard_normal((T, cols)) * spread[::-1]).astype(np.float32)
    y, inv, y_w = as_stored(rng.standard_normal((T * top, cols)) * spread, t), rng.permutation(T * top).astype(np.int32), rng.random(T * top).astype(np.float32)
    w, w2, rows = (1 + 0.3 * rng.standard_normal(cols)).astype(np.float32), (1 + 0.3 * rng.standard_normal(cols)).astype(np.float32), rng.permutation(n)[:T].astype(np.int32)
    bufs = [dev(a) for a in (x, mix, w, w2, y_w)]
    xb, mb, wb, w2b, yw = bufs
    yb, ib, rb, keep, h = store(y, t), i32(inv), i32(rows), pl.DevBuf.zeros(4 * T * cols), pl.DevBuf.zeros(4 * max(T, 16) * ld)
    add, out = what != "norm only", what != "sum only"
    kw = dict(x=xb, T=T, cols=cols, groups=groups, eps=1e-3, mult=-0.6, ld=ld, ol=ol, top=top)
    if add:
        kw.update(w=wb, keep=keep)
        kw.update(dict(y=yb, inv=ib) if "experts" in what else dict(mix=mb))
        if what == "weighted experts":
            kw.update(y_w=yw)
    else:
        kw.update(rows=rb)
    if out:
        kw.update(h=h, w_next=w2b)
    p = filled(pl.SumNorm, **kw)
    pl.check(L.pi_k_sum_norm(t, C.byref(p), None))
    pl.sync()
    x64 = x.astype(np.float64)
    s = (y.astype(np.float64)[inv] * (y_w if what == "weighted experts" else np.ones(T * top))[:, None]).reshape(T, top, cols).sum(1) if "experts" in what else mix.astype(np.float64)
    want = o.add_normed(x64[:T], s, -0.6, w, groups, 1e-3) if add else x64[rows]
    got = xb.download(np.float32).reshape(n, cols)
    if add:
        size = np.abs(want).reshape(T, groups, -1).max(axis=(0, 2))
        assert (np.abs(got[:T] - want).reshape(T, groups, -1) / size[None, :, None]).max() < 5e-6 and np.array_equal(got[:T], keep.download(np.float32).reshape(T, cols))
        assert np.array_equal(got[T:], x[T:])
    else:
        assert np.array_equal(got, x)
    if out:
        wn = o.group_norm(want, w2, groups, 1e-3)
        assert np.abs(operand(h, t, T, cols, ld, ol) - wn).max() <= tol(t, 2) * np.abs(wn).max()


def convolve(t, runs, cols, groups, taps, ol, rng, steps):
    """Runs as (slot, tokens of each step) through steps, each step one call; checks every result and the states behind the last one."""
    L = pl.init()
    w, tw = (1 + 0.3 * rng.standard_normal(cols)).astype(np.float32), (0.5 * rng.standard_normal((taps, cols))).astype(np.float32)
    back, slots, slot_ld, ld = taps - 1, max(s for s, _ in runs) + 2, (taps - 1) * cols + 12, (cols + 63) // 64 * 64
    state = np.full((slots, slot_ld), 7.0, np.float32)                                  # what an earlier sequence left: a fresh run does not read it
    sb, wb, tb = dev(state), dev(w), dev(tw)
    past = {s: np.zeros((back, cols)) for s, _ in runs}
    seen = set()
    for step in range(steps):
        live = [(s, n[step]) for s, n in runs if n[step] > 0]
        T = sum(n for _, n in live)
        x = (rng.standard_normal((T, cols)) * np.repeat(10.0 ** rng.uniform(-1, 1, groups), cols // groups)).astype(np.float32)
        per, items, at = L.pi_k_conv_tokens(T, taps), [], 0
        for s, n in live:
            c = 0
            while c < n:
                k = min(max(per, back) if c == 0 else per, n - c)
                items.append([at + c, k, c, n, s, int(s not in seen), 0, 0])
                c += k
            at += n
            seen.add(s)
        xb, ib, h = dev(x), i32(items), pl.DevBuf.zeros(4 * max(T, 16) * ld)
        p = filled(pl.ConvNorm, x=xb, w=wb, taps_w=tb, T=T, cols=cols, groups=groups, taps=taps, eps=1e-4, state=sb, slot_ld=slot_ld, items=ib, n_items=len(items), h=h, ld=ld, ol=ol)
        pl.check(L.pi_k_conv_norm(t, C.byref(p), None))
        pl.sync()
        u, at, want = o.group_norm(x.astype(np.float64), w, groups, 1e-4), 0, np.empty((T, cols))
        for s, n in live:
            want[at:at + n] = o.convolved(u[at:at + n], past[s], tw.T.astype(np.float64))
            past[s] = o.past_inputs(past[s], u[at:at + n], taps)
            at += n
        assert np.abs(operand(h, t, T, cols, ld, ol) - want).max() <= tol(t) * np.abs(want).max(), step
    left = sb.download(np.float32).reshape(slots, slot_ld)
    for s in range(slots):
        if s in past:
            assert np.abs(left[s, :back * cols].reshape(back, cols) - past[s]).max(initial=0) < 2e-5
            assert (left[s, back * cols:] == 7).all()
        else:
            assert (left[s] == 7).all()


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("cols,groups,taps", [(96, 4, 4), (100, 5, 3), (99, 3, 4), (72, 1, 1), (64, 16, 2), (260, 5, 5), (64, 4, 1), (136, 2, 7), (4096, 8, 4), (1, 1, 3), (1500, 2, 12)])
def test_norm_and_convolution(t, cols, groups, taps):
    """Prompts, portions shorter than the convolution reaches, single tokens and runs side by side, on states an earlier sequence left."""
    runs = [(2, [37, 1, 2, 1, 20]), (0, [1, 1, 1, 1, 1]), (4, [2, 60, 0, 1, 3]), (1, [0, 5, 1, 1, 1])]
    convolve(t, runs, cols, groups, taps, 0, np.random.default_rng(cols + taps), 5)


@pytest.mark.parametrize("cols,groups,taps", [(96, 4, 4), (104, 13, 3), (264, 11, 6), (2048, 8, 4)])
def test_norm_and_convolution_into_the_operand_layout(cols, groups, taps):
    convolve(pl.BF16, [(3, [9, 1, 2, 1]), (0, [1, 1, 1, 13]), (1, [6, 2, 0, 2])], cols, groups, taps, 1, np.random.default_rng(cols), 4)


# ---- rotations and values -----------------------------------------------------------------------------------------------------------
def test_angles_of_given_frequencies():
    L = pl.init()
    pos = np.array([0, 1, 77, 4095, 131071], np.int32)
    for f, length in ((o.wavelength_frequencies(24, 500.0, dict(factor=8.0, low=1.0, high=4.0, original=300)), 1.0), (o.ramp_frequencies(64, 10000.0, dict(factor=4.0, slow=1.0, fast=32.0, original=512)), 1.1386)):
        pb, fb, cs = i32(pos), f64(f), pl.DevBuf(8 * pos.size * f.size)
        pl.check(L.pi_k_rope_angles_table(pb.ptr, pos.size, 2 * f.size, fb.ptr, length, cs.ptr, None))
        pl.sync()
        a = pos[:, None] * f[None]
        want = length * np.stack([np.cos(a), np.sin(a)], -1)
        assert np.abs(cs.download(np.float32).reshape(want.shape) - want).max() < 3e-7


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("pairs", [0, 1])
def test_shifted_keys_with_given_frequencies(t, pairs):
    L, rng = pl.init(), np.random.default_rng(4)
    n, G, dim = 9, 2, 40
    hd, turn, f = L.pi_k_gqa_head_ld(t, dim, dim), (o.rotate_neighbours if pairs else o.rotate_halves), o.ramp_frequencies(24, 800.0, dict(factor=4.0, slow=1.0, fast=32.0, original=100))
    k = rng.standard_normal((n, G, dim))
    pos, delta = rng.integers(50, 900, n), np.array([0, 5, -7, 0, 1, -50, 300, 2, 0], np.int32)
    cells = np.zeros((n, G, 2, hd), np.float32)
    cells[:, :, 0, :dim], cells[:, :, 1, :dim] = turn(k, pos, f, 1.2), k
    cb, db, fb = store(cells, t), i32(delta), f64(f)
    pl.check(L.pi_k_gqa_shift_table(t, cb.ptr, n, G, hd, 24, fb.ptr, pairs, db.ptr, None))
    pl.sync()
    got = fetch(cb, t, cells.shape)
    assert np.abs(got[:, :, 0, :dim] - turn(k, pos + delta, f, 1.2)).max() < (4e-2 if t == pl.BF16 else 1e-5)
    assert np.array_equal(got[:, :, 1], as_stored(cells[:, :, 1], t))


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T", [6, 33])
@pytest.mark.parametrize("pairs", [0, 1])
@pytest.mark.parametrize("H,G,dim,vdim,rot", [(6, 2, 40, 24, 24), (5, 1, 17, 33, 6), (4, 4, 128, 128, 64), (3, 3, 2, 1, 2), (8, 4, 96, 40, 32), (2, 1, 256, 200, 256)])
def test_queries_cells_and_mixed_values(t, T, pairs, H, G, dim, vdim, rot):
    """A layer that keeps its values, then one that mixes them into its own; rotations longer than one."""
    L, rng = pl.init(), np.random.default_rng(dim + T)
    hd, n_cells, off_k = L.pi_k_gqa_head_ld(t, dim, vdim), 50, H * dim
    off_v = off_k + G * dim
    ldz, ld_first = (off_v + G * vdim + 15) // 16 * 16, G * vdim + 3
    f, turn, lam = o.ramp_frequencies(rot, 700.0, dict(factor=3.0, slow=1.0, fast=16.0, original=600)), (o.rotate_neighbours if pairs else o.rotate_halves), np.float32(0.3)
    pos = rng.integers(0, 5000, T).astype(np.int32)
    pb, fb, cs, first, lb = i32(pos), f64(f), pl.DevBuf(8 * T * (rot // 2)), pl.DevBuf.zeros(4 * T * ld_first), dev(np.full(1, lam))
    pl.check(L.pi_k_rope_angles_table(pb.ptr, T, rot, fb.ptr, 1.25, cs.ptr, None))
    kept = None
    for keeps in (True, False):
        z = (2 * rng.standard_normal((T, ldz))).astype(np.float32)
        cells = rng.permutation(n_cells)[:T]
        zb, cb, q, cache = dev(z), i32(cells), pl.DevBuf.zeros(4 * T * H * hd), pl.DevBuf.zeros(4 * n_cells * G * 2 * hd)
        p = filled(pl.GqaPrep, z=zb, ldz=ldz, T=T, n_head=H, n_kv=G, dim=dim, vdim=vdim, rot_dim=rot, off_k=off_k, off_v=off_v, hd=hd, eps=1e-5, rot_pairs=pairs, cs=cs, q=q, cache=cache, cell=cb,
                   ld_first=ld_first, v_keep=first if keeps else None, v_first=None if keeps else first, v_mix=None if keeps else lb)
        pl.check(L.pi_k_gqa_prep(t, C.byref(p), None, None))
        pl.sync()
        z64 = z.astype(np.float64)
        wq, wk = turn(z64[:, :H * dim].reshape(T, H, dim), pos, f, 1.25), turn(z64[:, off_k:off_v].reshape(T, G, dim), pos, f, 1.25)
        v = z64[:, off_v:off_v + G * vdim].reshape(T, G, vdim)
        wv = v if keeps else o.blended_values(v, kept, np.float64(lam))
        kept = v
        got_q, got_c = fetch(q, t, (T, H, hd)), fetch(cache, t, (n_cells, G, 2, hd))
        for got, want in ((got_q[..., :dim], wq), (got_c[cells][:, :, 0, :dim], wk), (got_c[cells][:, :, 1, :vdim], wv)):
            assert np.abs(got - want).max() <= tol(t) * np.abs(want).max()
        assert not got_q[..., dim:].any() and not got_c[:, :, 0, dim:].any() and not got_c[:, :, 1, vdim:].any()
        assert not got_c[[c for c in range(n_cells) if c not in cells]].any()
        if keeps:
            assert np.array_equal(first.download(np.float32).reshape(T, ld_first)[:, :G * vdim], z[:, off_v:off_v + G * vdim])


# ---- attention ----------------------------------------------------------------------------------------------------------------------
def attend(t, seqs, H, G, dim, vdim, route, parts=1, wide=0, scale=None, cap=0.0, sinks=None, talk=None, gate=True, spike=(), seed=0, blind=False, split=1):
    """seqs: (tokens of the step, cells before them) per sequence, on scattered cells.  route: "own" (a head meets its own group's values), "all" (every
    group's, then the mixture) or "passes" (soft-max denominators first, then weights mixed as they are formed).  spike: (sequence, token,
    cell, head) whose score stands out.  split: parts of an item's cells, for the passes.  Returns (got, want) [T, H, vdim]; blind: the oracle does not see the spikes' keys."""
    L, rng = pl.init(), np.random.default_rng(seed)
    hd, per, T = L.pi_k_gqa_head_ld(t, dim, vdim), H // G, sum(n for n, _ in seqs)
    scale = dim ** -0.5 if scale is None else scale
    pool = sum(n + b for n, b in seqs) + 7
    free, list_ld = list(rng.permutation(pool)), max(n + b for n, b in seqs) + 2
    lists = np.zeros((len(seqs), list_ld), np.int32)
    q, cache = as_stored(rng.standard_normal((T, H, dim)), t), as_stored(rng.standard_normal((pool, G, 2, max(dim, vdim))), t)
    z = rng.standard_normal((T, H + 9)).astype(np.float32)
    work, seq_of, vis, items, at, want = [], [], [], [], 0, np.empty((T, H, vdim))
    most = L.pi_k_gqa_talk_tokens(H, G, dim, vdim)
    for s, (n, b) in enumerate(seqs):
        cells = [free.pop() for _ in range(n + b)]
        lists[s, :n + b] = cells
        for x in spike:
            if x[0] == s:
                cache[cells[x[2]], x[3] // per, 0, :dim] = as_stored(4 * q[at + x[1], x[3]], t)
        rows, step = n * per, L.pi_k_gqa_rows(wide)
        work += [[at, r, min(step, rows - r), s] for r in range(0, rows, step)]
        if route == "passes":
            items += [[at + i, min(most, n - i), s, split << 16 | j if split > 1 and i % (2 * most) == 0 else 0] for i in range(0, n, most) for j in range(split if i % (2 * most) == 0 else 1)]
        seq_of += [s] * n
        vis += list(range(b + 1, b + n + 1))
        k, v = cache[cells][:, :, 0, :dim].astype(np.float64), cache[cells][:, :, 1, :vdim].astype(np.float64)
        if blind:
            k[[x[2] for x in spike if x[0] == s]] = 0
        sc = o.scores(q[at:at + n].astype(np.float64), k, scale)
        w = o.softmax(o.causal(o.capped(sc, cap) if cap else sc, np.arange(b, b + n), np.arange(n + b)), None if sinks is None else sinks.astype(np.float64))
        r = o.weighted_values(w if talk is None else o.mixed_heads(w, talk), v)
        want[at:at + n] = o.gated_heads(r, z[at:at + n, 4:4 + H].astype(np.float64), np.eye(H)) if gate and route != "own" else r
        at += n
    pad = np.zeros((pool, G, 2, hd), np.float32)
    pad[:, :, 0, :dim], pad[:, :, 1, :vdim] = cache[:, :, 0, :dim], cache[:, :, 1, :vdim]
    qp = np.zeros((T, H, hd), np.float32)
    qp[..., :dim] = q
    ld, every = H * vdim + 5, route == "all"
    qb, cb, lb, vb, att, zb = store(qp, t), store(pad, t), i32(lists), i32(vis), pl.DevBuf.zeros(4 * T * ld), dev(z)
    heads = pl.DevBuf.zeros(4 * T * H * G * vdim) if every else None
    wb, sb, tb = i32(work if t == pl.BF16 else seq_of), (dev(sinks) if sinks is not None else None), (dev(talk.astype(np.float32)) if talk is not None else None)
    scratch = pl.DevBuf(4 * max(L.pi_k_gqa_scratch_floats(len(work), wide, G * G if every else G, hd, parts), 1))
    a = filled(pl.GqaAttn, out_scale=1.0, q=qb, cache=cb, lists=lb, list_ld=list_ld, work=wb, n_vis=vb, n_work=len(work), T=T, n_head=H, n_kv=G, dim=dim, vdim=vdim, hd=hd, n_parts=parts,
               wide=wide, scale=scale, sink=-np.inf, sinks=sb, softcap=cap, scratch=scratch, att=heads if every else att, ld_att=ld, all_values=int(every))
    m = filled(pl.GqaMix, a=heads, talk=tb, z=zb, ldz=H + 9, off_gate=4 if gate else -1, T=T, n_head=H, n_kv=G, vdim=vdim, att=att, ld_att=ld)
    if route == "passes":
        assert most > 0
        stats, ib, some = pl.DevBuf.zeros(4 * T * H), i32(items), pl.DevBuf(4 * split * T * H * vdim)
        m.parts, m.n_parts = some.ptr, split
        pl.check(L.pi_k_gqa_stats(C.byref(a), stats.ptr, None))
        pl.check(L.pi_k_gqa_talk(C.byref(a), C.byref(m), stats.ptr, ib.ptr, len(items), None))
    else:
        pl.check(L.pi_k_gqa_attn(t, C.byref(a), None))
        if every:
            pl.check(L.pi_k_gqa_mix(t, C.byref(m), None))
    pl.sync()
    got = fetch(att, t, (T, ld))
    assert not got[:, H * vdim:].any()
    return got[:, :H * vdim].reshape(T, H, vdim), want


def mixture(H, seed=1):
    rng = np.random.default_rng(seed)
    return rounded(np.eye(H) + 0.6 * rng.standard_normal((H, H))).astype(np.float64), rng.uniform(-3, 6, H).astype(np.float32)


def near(got, want, t, scale=1.5):
    assert np.abs(got - want).max() <= tol(t, scale) * np.abs(want).max(), np.abs(got - want).max() / np.abs(want).max()


SHORT, LONG = [(1, 0), (3, 126), (1, 127), (1, 700), (17, 30), (2, 0)], [(70, 0), (9, 190), (1, 300), (130, 61)]
SHAPES = [(6, 2, 40, 24), (5, 1, 17, 33), (4, 4, 32, 20), (8, 2, 64, 64), (16, 2, 128, 128), (3, 3, 96, 90), (1, 1, 2, 1), (14, 7, 24, 30), (20, 2, 128, 64)]
WAYS = [(pl.F32, 1, 0), (pl.BF16, 1, 0), (pl.BF16, 5, 0), (pl.BF16, 64, 0), (pl.BF16, 1, 1), (pl.BF16, 3, 1)]


@pytest.mark.parametrize("t,parts,wide", WAYS)
@pytest.mark.parametrize("cap", [0.7, 20.0])
@pytest.mark.parametrize("H,G,dim,vdim", SHAPES + [(2, 1, 256, 250), (4, 2, 160, 160)])
def test_soft_capped_scores(t, parts, wide, cap, H, G, dim, vdim):
    near(*attend(t, LONG if wide else SHORT, H, G, dim, vdim, "own", parts, wide, cap=cap, scale=2 * dim ** -0.5), t)


@pytest.mark.parametrize("t,parts,wide", WAYS)
def test_a_sink_per_head(t, parts, wide):
    sinks = np.array([-np.inf, 8.0, -4.0, 0.0, 2.0, 60.0], np.float32)
    got, want = attend(t, LONG if wide else SHORT, 6, 2, 40, 24, "own", parts, wide, sinks=sinks)
    for h in range(5):
        near(got[:, h], want[:, h], t)
    assert np.abs(got[:, 5]).max() < 1e-6 and np.abs(want[:, 1]).max() < 0.2 < np.abs(want[:, 0]).max()        # a sink that takes all, and much


@pytest.mark.parametrize("t,parts,wide", WAYS)
@pytest.mark.parametrize("H,G,dim,vdim", SHAPES + [(2, 2, 256, 250), (18, 9, 32, 32), (128, 1, 16, 10), (100, 50, 8, 2)])
def test_mixed_heads(t, parts, wide, H, G, dim, vdim):
    talk, sinks = mixture(H)
    near(*attend(t, LONG if wide else SHORT, H, G, dim, vdim, "all", parts, wide, sinks=sinks, talk=talk), t)


@pytest.mark.parametrize("cap,sink,gate,split", [(0.0, True, True, 1), (0.0, False, False, 2), (1.5, True, True, 5)])
@pytest.mark.parametrize("H,G,dim,vdim", SHAPES)
def test_mixed_heads_in_two_passes(H, G, dim, vdim, cap, sink, gate, split):
    talk, sinks = mixture(H)
    seqs = LONG + [(2, 0), (1, 0), (33, 500), (1, 31), (5, 32)]
    near(*attend(pl.BF16, seqs, H, G, dim, vdim, "passes", 1, 1, cap=cap, sinks=sinks if sink else None, talk=talk, gate=gate, split=split), pl.BF16, 2)


def test_sizes_two_passes_do_not_take():
    L = pl.init()
    assert L.pi_k_gqa_talk_tokens(9, 9, 64, 64) == 0 and L.pi_k_gqa_talk_tokens(17, 1, 64, 64) == 0 and L.pi_k_gqa_talk_tokens(4, 2, 130, 64) == 0
    assert L.pi_k_gqa_talk_tokens(16, 1, 64, 64) == 2 and L.pi_k_gqa_talk_tokens(3, 3, 128, 1) == 32


@pytest.mark.parametrize("t,parts,wide,route", [(*w, "all") for w in WAYS] + [(pl.BF16, 1, 1, "passes")])
def test_one_key_among_hundreds(t, parts, wide, route):
    """One score of one head stands out and reaches all heads through the mixture: the first cell, the edges of tiles of 32 and 64 cells, the token's
    own cell; a key just beyond what a token sees stays out of sight."""
    n = 40 if wide else 6
    talk, sinks = mixture(4, 3)
    spike = [(0, 0, 0, 1), (0, 1, 31, 2), (0, 2, 32, 3), (0, 3, 63, 0), (0, 4, 64, 1), (0, 5, 400 + 5, 2), (0, 2, 400 + 3, 0)]
    kw = dict(scale=64 ** -0.5, sinks=sinks, talk=talk, spike=spike)
    got, want = attend(t, [(n, 400)], 4, 2, 64, 64, route, parts, wide, **kw)
    near(got, want, t, 2)
    if route == "passes":
        near(attend(t, [(n, 400)], 4, 2, 64, 64, route, parts, wide, split=3, **kw)[0], want, t, 2)
    _, blind = attend(t, [(n, 400)], 4, 2, 64, 64, route, parts, wide, blind=True, **kw)
    assert (np.abs(blind - want)[:6].max(axis=(1, 2)) > 0.3).all()


@pytest.mark.parametrize("t", TYPES)
def test_scores_of_any_size(t):
    talk, sinks = mixture(4)
    for scale, cap in ((30.0, 0.0), (-2.0, 0.0), (1e-3, 5.0), (30.0, 4.0)):
        for route, wide in (("all", 0), ("all", 1), ("passes", 1)) if t == pl.BF16 else (("all", 0),):
            got, want = attend(t, [(2, 0), (40, 50)], 4, 2, 64, 64, route, 1, wide, scale=scale, cap=cap, sinks=sinks, talk=talk)
            assert np.isfinite(got).all()
            near(got, want, t, 3)


def test_the_mixture_of_some_tokens():
    """Only the listed tokens are written."""
    L, rng = pl.init(), np.random.default_rng(2)
    T, H, G, vd = 7, 6, 3, 20
    a, talk, z = rng.standard_normal((T, H, G, vd)).astype(np.float32), rng.standard_normal((H, H)).astype(np.float32), rng.standard_normal((T, H)).astype(np.float32)
    ab, tb, zb, att, some = dev(a), dev(talk), dev(z), pl.DevBuf.zeros(4 * T * H * vd), i32([1, 4, 6])
    m = filled(pl.GqaMix, a=ab, talk=tb, z=zb, ldz=H, off_gate=0, T=T, n_head=H, n_kv=G, vdim=vd, att=att, ld_att=H * vd, tokens=some, n_tokens=3)
    pl.check(L.pi_k_gqa_mix(pl.F32, C.byref(m), None))
    pl.sync()
    want = np.stack([np.einsum("g,tgc->tc", talk[h].astype(np.float64), a[:, :, h // 2]) for h in range(H)], 1) * o.sigmoid(z.astype(np.float64))[..., None]
    got = fetch(att, pl.F32, (T, H, vd))
    assert np.abs(got[[1, 4, 6]] - want[[1, 4, 6]]).max() < 1e-5 and not got[[0, 2, 3, 5]].any()


# ---- experts ------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("E,top", [(10, 2), (1, 1), (64, 6), (5, 5), (160, 6), (300, 8), (16, 1)])
def test_choice_by_scores(E, top):
    L, rng = pl.init(), np.random.default_rng(E)
    T = 33
    z = (rng.standard_normal((T, E)) * 2).astype(np.float32)
    zb, ids, w = dev(z), pl.DevBuf(4 * T * top), pl.DevBuf(4 * T * top)
    pl.check(L.pi_k_route_scores(zb.ptr, T, E, top, ids.ptr, w.ptr, None))
    pl.sync()
    want, sc = o.choice(z.astype(np.float64), np.eye(E), top)
    assert np.array_equal(ids.download(np.int32).reshape(T, top), want) and np.abs(w.download(np.float32).reshape(T, top) - sc).max() < 1e-6


def weighted_acts(h, up, ids, wts):
    """silu(w gate h) * (w up h) of every choice, [T, top, ff]."""
    return np.stack([[o.silu(up[e, :, 0] @ (w * h[i])) * (up[e, :, 1] @ (w * h[i])) for e, w in zip(ids[i], wts[i])] for i in range(len(h))])


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,E,top,tile,ff,d", [(3, 5, 2, 0, 24, 64), (200, 7, 3, 64, 33, 64), (150, 2, 1, 128, 96, 128), (64, 40, 4, 64, 130, 192)])
def test_sorted_experts_weighted_at_their_input(t, T, E, top, tile, ff, d):
    L, rng = pl.init(), np.random.default_rng(T)
    ids, wts = np.stack([rng.permutation(E)[:top] for _ in range(T)]).astype(np.int32), (0.05 + rng.random((T, top))).astype(np.float32)
    up, h, n, ld = rounded(3 * rng.standard_normal((E, ff, 2, d)) / np.sqrt(d)), as_stored(rng.standard_normal((T, d)), t), T * top, ff + 3
    off, perm, inv, tiles, nt = i32(np.zeros(E + 1)), i32(np.zeros(n)), i32(np.zeros(n)), i32(np.zeros(2 * (n // 64 + E + 1))), i32([0])
    ib, wb, tn = i32(ids), dev(wts), tile or 64
    pl.check(L.pi_k_moe_sort(ib.ptr, n, E, off.ptr, perm.ptr, inv.ptr, tn, tiles.ptr, nt.ptr, None))
    ub, hb, act = store(up.reshape(-1, d), pl.BF16), store(h, t), pl.DevBuf.zeros(4 * n * ld)
    g = group_args(W=ub.ptr, w_gs=2 * ff * d, rows=2 * ff, cols=d, ldw=d, n_group=E, x=hb.ptr, ldx=d, T=T, y=act.ptr, ldy=ld, alpha=1.0, off=off.ptr, gather=perm.ptr, gather_div=top, tiles=tiles.ptr,
                   n_tiles=nt.ptr, max_tiles=n // tn + E, glu=1, glu_limit=np.inf, glu_gain=1.0, glu_plain_up=1, pair_w=wb.ptr)
    pl.check(L.pi_k_group_gemm_tile(C.byref(g), tile, None) if tile and t == pl.BF16 else L.pi_k_group_gemm(t, C.byref(g), None))
    pl.sync()
    got = fetch(act, t, (n, ld))[inv.download(np.int32)][:, :ff].reshape(T, top, ff)
    want = weighted_acts(h.astype(np.float64), up.astype(np.float64), ids, wts)
    assert np.abs(got - want).max() <= tol(t) * np.abs(want).max()
    late = want / 1 - weighted_acts(h.astype(np.float64), up.astype(np.float64), ids, np.ones_like(wts)) * wts[..., None]
    assert np.abs(late).max() > 0.1 * np.abs(want).max()                                # (weights behind the activation give something else)


@pytest.mark.parametrize("T,E,top,ff,cols", [(1, 6, 2, 24, 256), (16, 40, 8, 72, 512), (5, 3, 3, 33, 256), (7, 9, 1, 100, 768), (2, 1, 1, 1, 64)])
def test_experts_of_a_step(T, E, top, ff, cols):
    """Both halves of a step's experts: what they read weighted, and the sum of their results without a residual."""
    L, rng = pl.init(), np.random.default_rng(T)
    h, up = rounded(rng.standard_normal((T, cols))), rounded(2 * rng.standard_normal((E, ff, 2, cols)) / np.sqrt(cols))
    ids, wts, ld = np.stack([rng.permutation(E)[:top] for _ in range(T)]).astype(np.int32), (0.05 + rng.random((T, top))).astype(np.float32), (ff + 63) // 64 * 64
    hb, ub, ib, wb, act = store(in_layout(h), pl.BF16), store(up, pl.BF16), i32(ids), dev(wts), pl.DevBuf.zeros(2 * T * top * ld)
    pl.check(L.pi_k_expert_up_step(ub.ptr, E, ff, cols, np.inf, 1.0, 1, 1, hb.ptr, T, ib.ptr, wb.ptr, top, act.ptr, ld, None))
    pl.sync()
    want, got = weighted_acts(h.astype(np.float64), up.astype(np.float64), ids, wts), fetch(act, pl.BF16, (T, top, ld))
    assert np.abs(got[..., :ff] - want).max() <= tol(pl.BF16) * np.abs(want).max() and not got[..., ff:].any()
    rows = cols + 40
    down, out = rounded(rng.standard_normal((E, rows, ff)) / np.sqrt(ff)), pl.DevBuf(4 * T * rows)
    db = store(padded(down.reshape(-1, ff), ld), pl.BF16)
    s = filled(pl.LayerOut, rows=rows, T=T, out=out, down=db, act=act, ids=ib, ld_act=ld, top=top, n_expert=E)
    pl.check(L.pi_k_layer_out_step(C.byref(s), None))
    pl.sync()
    total = np.stack([sum(down[e].astype(np.float64) @ got[i, k, :ff] for k, e in enumerate(ids[i])) for i in range(T)])
    assert np.abs(out.download(np.float32).reshape(T, rows) - total).max() <= 1e-5 * np.abs(total).max()


def test_bad_arguments_are_errors():
    L, b = pl.init(), pl.DevBuf.zeros(1 << 16)
    s = dict(x=b, mix=b, w=b, w_next=b, T=1, cols=24, groups=4, eps=1e-5, h=b, ld=24)
    for spoil in (dict(groups=5), dict(groups=0), dict(y=b), dict(mix=None), dict(ld=23), dict(w_next=None), dict(rows=b), dict(mix=None, y=b, top=2), dict(ol=1, T=17), dict(cols=40000, groups=1, ld=40000)):
        p = filled(pl.SumNorm, **{k: v for k, v in dict(s, **spoil).items() if v is not None})
        assert L.pi_k_sum_norm(pl.BF16, C.byref(p), None) != 0, spoil
    c = dict(x=b, w=b, taps_w=b, T=1, cols=24, groups=4, taps=3, eps=1e-5, state=b, slot_ld=48, items=b, n_items=1, h=b, ld=24)
    for spoil in (dict(groups=5), dict(taps=0), dict(state=None), dict(slot_ld=47), dict(items=None), dict(ld=20), dict(groups=24, taps=2000, slot_ld=1999 * 24)):
        p = filled(pl.ConvNorm, **{k: v for k, v in dict(c, **spoil).items() if v is not None})
        assert L.pi_k_conv_norm(pl.BF16, C.byref(p), None) != 0, spoil
    m = dict(a=b, talk=b, z=b, ldz=8, off_gate=4, T=1, n_head=4, n_kv=2, vdim=8, att=b, ld_att=32)
    for spoil in (dict(n_kv=3), dict(off_gate=5), dict(ld_att=31), dict(tokens=b), dict(n_head=200, off_gate=-1, ld_att=1600)):
        p = filled(pl.GqaMix, **dict(m, **spoil))
        assert L.pi_k_gqa_mix(pl.BF16, C.byref(p), None) != 0, spoil
    assert L.pi_k_rope_angles_table(b.ptr, 1, 4, None, 1.0, b.ptr, None) != 0
    assert L.pi_k_gqa_shift_table(pl.F32, b.ptr, 1, 1, 32, 4, None, 0, b.ptr, None) != 0
    assert L.pi_k_expert_up_step(b.ptr, 1, 8, 40, 1.0, 1.0, 1, 1, b.ptr, 1, b.ptr, b.ptr, 1, b.ptr, 8, None) != 0          # columns are no multiple of 32
    o_ = filled(pl.LayerOut, out=b, rows=8, T=1)
    assert L.pi_k_layer_out_step(C.byref(o_), None) != 0                                # neither a product nor experts
