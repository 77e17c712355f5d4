"""Operators of the models described layer by layer, one by one against the plain implementations (tests/plain_latent.py) in bf16 and fp32."""
import ctypes as C

import numpy as np
import pytest

import plain_latent as o
from powerinfer_amd import lib as pl
from powerinfer_amd.checkpoint import bf16_bits, bf16_floats

pytestmark = pytest.mark.gpu
TYPES = [pl.BF16, pl.F32]


def rounded(a):
    a = np.asarray(a, np.float32)
    return bf16_floats(bf16_bits(a)).reshape(a.shape)


def store(a, t):
    return pl.DevBuf(host=bf16_bits(a) if t == pl.BF16 else np.asarray(a, np.float32))


def fetch(buf, t, shape):
    n = int(np.prod(shape))
    return bf16_floats(buf.download(np.uint16, n)).reshape(shape) if t == pl.BF16 else buf.download(np.float32, n).reshape(shape)


def as_stored(a, t):
    return rounded(a) if t == pl.BF16 else np.asarray(a, np.float32)


def tol(t, scale=1.0):
    return (6e-3 if t == pl.BF16 else 3e-6) * scale


def dev(a):
    return pl.DevBuf(host=a)


def i32(a):
    return pl.DevBuf(host=np.asarray(a, np.int32))


def padded(w, ld):
    out = np.zeros((w.shape[0], ld), np.float32)
    out[:, :w.shape[1]] = w
    return out


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,cols,ol", [(1, 100, 0), (5, 3000, 0), (3, 5000, 0), (16, 256, 1), (7, 72, 1)])
def test_norm_pair(t, T, cols, ol):
    if ol and t == pl.F32:
        pytest.skip("the operand layout is a bf16 layout")
    L, rng = pl.init(), np.random.default_rng(T + cols)
    x = (rng.standard_normal((T + 2, cols)) * 3).astype(np.float32)
    wa, wb = (1 + 0.3 * rng.standard_normal((2, cols))).astype(np.float32)
    rows = rng.permutation(T + 2)[:T].astype(np.int32)
    ld = (cols + 63) // 64 * 64
    a, b = pl.DevBuf.zeros(16 * max(T, 16) * ld), pl.DevBuf.zeros(16 * max(T, 16) * ld)
    bufs = [dev(x), i32(rows), dev(wa), dev(wb)]
    pl.check(L.pi_k_norm_pair(t, bufs[0].ptr, bufs[1].ptr, T, cols, 1e-5, bufs[2].ptr, a.ptr, bufs[3].ptr, b.ptr, ld, ol, None))
    pl.sync()
    for buf, w in ((a, wa), (b, wb)):
        want = o.rms_norm_plain(x[rows].astype(np.float64), w, 1e-5)
        if ol:
            got = fetch(buf, t, (ld // 8, 16, 8)).transpose(1, 0, 2).reshape(16, ld)[:T, :cols]
        else:
            got = fetch(buf, t, (T, ld))[:, :cols]
        assert np.abs(got - want).max() <= tol(t) * np.abs(want).max()


@pytest.mark.parametrize("cols", [64, 300, 4096, 9000])
def test_embed_norm(cols):
    L, rng = pl.init(), np.random.default_rng(cols)
    table, w = rounded(rng.standard_normal((9, cols))), rng.standard_normal(cols).astype(np.float32)
    toks = [8, 0, 3, 3]
    x = pl.DevBuf(4 * 4 * cols)
    tb, wb, ib = store(table, pl.BF16), dev(w), i32(toks)
    pl.check(L.pi_k_embed_norm(tb.ptr, cols, ib.ptr, 4, wb.ptr, 1e-6, x.ptr, None))
    pl.sync()
    want = o.rms_norm_plain(table[toks].astype(np.float64), w, 1e-6)
    assert np.abs(x.download(np.float32).reshape(4, cols) - want).max() < 3e-6 * np.abs(want).max()


def test_rope_angles_far_out():
    L = pl.init()
    pos, dims, base = np.array([0, 1, 77, 4095, 131071, 2000003], np.int32), 64, 10000.0
    cs, pb = pl.DevBuf(8 * pos.size * dims // 2), i32(pos)
    pl.check(L.pi_k_rope_angles(pb.ptr, pos.size, dims, base, cs.ptr, None))
    pl.sync()
    a = pos[:, None] * base ** (-2.0 * np.arange(dims // 2) / dims)
    want = np.stack([np.cos(a), np.sin(a)], -1)
    assert np.abs(cs.download(np.float32).reshape(want.shape) - want).max() < 2e-7


def group_args(**kw):
    g = pl.GroupGemm()
    for k, v in kw.items():
        setattr(g, k, v)
    return g


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("tile", [0, 64, 128])
@pytest.mark.parametrize("groups,rows,cols,T,relu2,y_f32", [(3, 50, 100, 1, 0, 0), (5, 130, 64, 37, 1, 0), (1, 260, 192, 300, 0, 1), (2, 33, 320, 129, 1, 1)])
def test_group_gemm_per_group_inputs(t, tile, groups, rows, cols, T, relu2, y_f32):
    if tile and t == pl.F32:
        pytest.skip("the tiled product is bf16")
    L, rng = pl.init(), np.random.default_rng(rows)
    ld = (cols + 63) // 64 * 64
    W = rounded(rng.standard_normal((groups, rows, cols)) / np.sqrt(cols))
    x = as_stored(rng.standard_normal((T, groups, cols)), t)
    wb = store(padded(W.reshape(-1, cols), ld), pl.BF16)
    xb = store(padded(x.reshape(-1, cols), ld), t)
    ldy = groups * rows + 4
    y = pl.DevBuf.zeros(4 * T * ldy)
    g = group_args(W=wb.ptr, w_gs=rows * ld, rows=rows, cols=ld, ldw=ld, n_group=groups, x=xb.ptr, x_gs=ld, ldx=groups * ld, T=T, y=y.ptr, y_gs=rows, ldy=ldy,
                   y_f32=y_f32, relu2=relu2, alpha=1.5)
    pl.check(L.pi_k_group_gemm_tile(C.byref(g), tile, None) if tile else L.pi_k_group_gemm(t, C.byref(g), None))
    pl.sync()
    got = fetch(y, pl.F32 if y_f32 else t, (T, ldy))[:, :groups * rows].reshape(T, groups, rows)
    want = 1.5 * np.einsum("tgc,grc->tgr", x.astype(np.float64), W)
    if relu2:
        want = np.maximum(want, 0) ** 2
    assert np.abs(got - want).max() <= (tol(t) if not y_f32 else 1e-5) * np.abs(want).max()


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,E,top,tile", [(3, 5, 2, 0), (200, 7, 3, 64), (150, 2, 1, 128), (64, 40, 4, 64)])
def test_sorted_experts_and_combine(t, T, E, top, tile):
    """moe_sort's places and tiles, both grouped products over them, and the weighted sum."""
    L, rng = pl.init(), np.random.default_rng(T)
    d, ff, D = 64, 40, 72
    ids = np.stack([rng.permutation(E)[:top] for _ in range(T)]).astype(np.int32)
    wts = rng.random((T, top)).astype(np.float32)
    up, down = rounded(rng.standard_normal((E, ff, d)) / 8), rounded(rng.standard_normal((E, D, ff)) / 6)
    h, x, mix = as_stored(rng.standard_normal((T, d)), t), rng.standard_normal((T, D)).astype(np.float32), rng.standard_normal((T, D)).astype(np.float32)
    n = T * top
    off, perm, inv, tiles, nt = i32(np.zeros(E + 1)), i32(np.zeros(n)), i32(np.zeros(n)), i32(np.zeros(2 * (n // 64 + E + 1))), i32([0])
    ib, wb = i32(ids), dev(wts)
    tn = tile or 64
    pl.check(L.pi_k_moe_sort(ib.ptr, n, E, off.ptr, perm.ptr, inv.ptr, tn, tiles.ptr, nt.ptr, None))
    pl.sync()
    offs, perms, invs = off.download(np.int32), perm.download(np.int32), inv.download(np.int32)
    assert np.array_equal(np.diff(offs), np.bincount(ids.ravel(), minlength=E)) and sorted(perms) == list(range(n)) and np.array_equal(perms[invs], np.arange(n))
    assert all((ids.ravel()[perms[offs[e]:offs[e + 1]]] == e).all() for e in range(E))
    k = int(nt.download(np.int32)[0])
    assert sorted(map(tuple, tiles.download(np.int32).reshape(-1, 2)[:k])) == sorted((e, p) for e in range(E) for p in range(offs[e], offs[e + 1], tn))
    upb, dnb = store(up.reshape(-1, d), pl.BF16), store(padded(down.reshape(-1, ff), 64), pl.BF16)
    hb, act, y = store(h, t), pl.DevBuf.zeros(4 * n * 64), pl.DevBuf.zeros(4 * n * D)
    a = group_args(W=upb.ptr, w_gs=ff * d, rows=ff, cols=d, ldw=d, n_group=E, x=hb.ptr, ldx=d, T=T, y=act.ptr, ldy=64, relu2=1, alpha=1.0, off=off.ptr, gather=perm.ptr,
                   gather_div=top, tiles=tiles.ptr, n_tiles=nt.ptr, max_tiles=n // tn + E)
    b = group_args(W=dnb.ptr, w_gs=D * 64, rows=D, cols=64, ldw=64, n_group=E, x=act.ptr, ldx=64, T=T, y=y.ptr, ldy=D, alpha=1.0, off=off.ptr, tiles=tiles.ptr, n_tiles=nt.ptr,
                   max_tiles=n // tn + E)
    for g in (a, b):
        pl.check(L.pi_k_group_gemm_tile(C.byref(g), tile, None) if tile and t == pl.BF16 else L.pi_k_group_gemm(t, C.byref(g), None))
    out, keep, xb, mb = pl.DevBuf(4 * T * D), pl.DevBuf(4 * T * D), dev(x), dev(mix)
    pl.check(L.pi_k_moe_combine(t, xb.ptr, mb.ptr, y.ptr, inv.ptr, wb.ptr, top, T, D, out.ptr, keep.ptr, None))
    pl.sync()
    want = x.astype(np.float64) + mix
    for i in range(T):
        for e, w in zip(ids[i], wts[i]):
            want[i] += w * o.expert(h[i:i + 1].astype(np.float64), up[e].astype(np.float64), down[e].astype(np.float64))[0]
    got = out.download(np.float32).reshape(T, D)
    assert np.abs(got - want).max() <= tol(t) * np.abs(want).max() and np.array_equal(got, keep.download(np.float32).reshape(T, D))


@pytest.mark.parametrize("E,top,G,keep", [(10, 2, 5, 3), (6, 2, 3, 1), (64, 6, 8, 4), (5, 5, 1, 1), (160, 6, 8, 3), (4, 2, 4, 2), (300, 8, 1, 1), (640, 6, 8, 4)])
def test_route(E, top, G, keep):
    L, rng = pl.init(), np.random.default_rng(E)
    T = 33
    z = (rng.standard_normal((T, E)) * 2).astype(np.float32)
    for bias in (rng.standard_normal(E).astype(np.float32), (-3 - rng.random(E)).astype(np.float32), np.zeros(E, np.float32)):
        zb, bb, ids, w = dev(z), dev(bias), pl.DevBuf(4 * T * top), pl.DevBuf(4 * T * top)
        pl.check(L.pi_k_route(zb.ptr, T, E, top, G, keep, bb.ptr, ids.ptr, w.ptr, None))
        pl.sync()
        want_ids, _ = o.route(z.astype(np.float64), np.eye(E), bias, top, G, keep)
        got = ids.download(np.int32).reshape(T, top)
        choice = 1 / (1 + np.exp(-z.astype(np.float64))) + bias
        assert np.abs(np.take_along_axis(choice, got, 1) - np.take_along_axis(choice, want_ids, 1)).max() < 1e-6      # the same ones, up to fp32 ties
        assert all(len(set(r)) == top for r in got) and (got == want_ids).mean() > 0.98
        sc = np.take_along_axis(choice - bias, got, 1)
        assert np.abs(w.download(np.float32).reshape(T, top) - sc / (sc.sum(1, keepdims=True) + 1e-20)).max() < 1e-6


class Case:
    """Queries of several sequences against shuffled cells, with the operands of every attention kernel."""

    def __init__(self, t, H, dim, rot, vdim, rank, lens, ask, seed, sink=0.5, scale=None, spike=()):
        """lens: cells of each sequence; ask[s]: the positions of sequence s that query; spike: (sequence, query index, head, key
        position) - that key is made to match that query so well that its value is nearly the whole result."""
        rng = np.random.default_rng(seed)
        self.t, self.H, self.dim, self.rot, self.vdim, self.rank = t, H, dim, rot, vdim, rank
        self.rank_ld, self.dim_ld = (rank + 63) // 64 * 64, (dim + 63) // 64 * 64
        self.kd = self.rank_ld + (rot + 31) // 32 * 32
        self.scale = (dim + rot) ** -0.5 if scale is None else scale
        self.n_cells = sum(lens) + 19
        self.cells = np.zeros((self.n_cells, self.kd), np.float32)
        self.cells[:, :rank] = as_stored(rng.standard_normal((self.n_cells, rank)), t)
        self.cells[:, self.rank_ld:self.rank_ld + rot] = as_stored(rng.standard_normal((self.n_cells, rot)), t)
        order = rng.permutation(self.n_cells)
        self.lists = np.full((len(lens), self.n_cells), 0, np.int32)
        at = 0
        for s, n in enumerate(lens):
            self.lists[s, :n] = order[at:at + n]
            at += n
        self.seq = np.concatenate([np.full(len(a), s) for s, a in enumerate(ask)]).astype(np.int32)
        self.pos = np.concatenate([np.asarray(a) for a in ask]).astype(np.int32)
        self.T = self.seq.size
        self.uk = rounded(rng.standard_normal((H, dim, rank)) / np.sqrt(rank))
        self.uv = rounded(rng.standard_normal((H, vdim, rank)) / np.sqrt(rank))
        self.q = as_stored(rng.standard_normal((self.T, H, dim + rot)), t)
        self.sink = (sink + rng.standard_normal(H)).astype(np.float32)
        for s, qi, h, key in spike:
            c = self.cells[self.lists[s, key]]
            k = np.concatenate([self.uk[h] @ c[:rank], c[self.rank_ld:self.rank_ld + rot]])
            self.q[qi, h] = as_stored(k / np.linalg.norm(k) * 40 / self.scale / np.linalg.norm(k), t)

    def want(self):
        """[T, H, vdim] heads in float64, the query rotation left out (q is taken as rotated)."""
        out = np.empty((self.T, self.H, self.vdim))
        for i in range(self.T):
            c = self.cells[self.lists[self.seq[i], :self.pos[i] + 1]].astype(np.float64)
            lat, kr = c[:, :self.rank], c[:, self.rank_ld:self.rank_ld + self.rot]
            for h in range(self.H):
                s = (lat @ self.uk[h].T.astype(np.float64) @ self.q[i, h, :self.dim] + kr @ self.q[i, h, self.dim:]) * self.scale
                out[i, h] = o.sink_softmax(s[None], self.sink[h:h + 1])[0] @ (lat @ self.uv[h].T.astype(np.float64))
        return out

    def latent_queries(self):
        q = np.zeros((self.T, self.H, self.kd), np.float32)
        q[..., :self.rank] = np.einsum("thd,hdr->thr", self.q[..., :self.dim], self.uk)
        q[..., self.rank_ld:self.rank_ld + self.rot] = self.q[..., self.dim:]
        return as_stored(q, self.t)

    def work(self):
        if self.t == pl.F32:
            return self.seq
        rows, items, t0 = pl.load().pi_k_latent_attn_rows(self.t), [], 0
        while t0 < self.T:
            t1 = t0 + 1
            while t1 < self.T and self.seq[t1] == self.seq[t0] and self.pos[t1] >= self.pos[t1 - 1]:
                t1 += 1
            n = (t1 - t0) * self.H
            items += [[t0, r, min(rows, n - r), self.seq[t0]] for r in range(0, n, rows)]
            t0 = t1
        return np.asarray(items, np.int32)

    def args(self, parts):
        self.bufs = [store(self.latent_queries(), self.t), store(self.cells, self.t), i32(self.lists), i32(self.work()), i32(self.pos + 1), dev(self.sink)]
        n = pl.load().pi_k_latent_attn_scratch_floats(max(self.T * self.H, len(self.work()) * 32), self.rank_ld, parts)
        self.scratch, self.out = pl.DevBuf(4 * max(n, 1)), pl.DevBuf.zeros(4 * self.T * self.H * self.rank_ld)
        a = pl.LatentAttn()
        a.q_lat, a.cache, a.lists, a.work, a.n_vis, a.sink = (b.ptr for b in self.bufs)
        a.list_ld, a.n_work, a.T, a.n_head, a.kv_rank, a.rank_ld, a.kd, a.n_parts = self.n_cells, len(self.work()), self.T, self.H, self.rank, self.rank_ld, self.kd, parts
        a.scale, a.scratch, a.out_lat = self.scale, self.scratch.ptr, self.out.ptr
        return a

    def run(self, parts):
        a = self.args(parts)
        pl.check(pl.load().pi_k_latent_attn(self.t, C.byref(a), None))
        pl.sync()
        lat = fetch(self.out, self.t, (self.T, self.H, self.rank_ld))[..., :self.rank]
        return np.einsum("thr,hvr->thv", lat.astype(np.float64), self.uv)


def close(got, want, t):
    err = np.abs(got - want).max() / np.abs(want).max()
    assert err < (2e-2 if t == pl.BF16 else 1e-5), err


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("parts", [1, 3, 16])
@pytest.mark.parametrize("H,dim,rot,vdim,rank", [(8, 16, 8, 24, 40), (3, 32, 32, 16, 128), (33, 24, 6, 8, 200), (1, 64, 64, 64, 512), (5, 16, 34, 16, 600)])
def test_latent_attention(t, parts, H, dim, rot, vdim, rank):
    if t == pl.F32 and parts > 1:
        pytest.skip("parts are a bf16 form")
    # first tokens, edges of the 32-cell tiles, portions in the middle of a sequence, single tokens
    c = Case(t, H, dim, rot, vdim, rank, [1, 97, 33, 64], [[0], list(range(40, 71)), [31, 32], [63]], 5)
    close(c.run(parts), c.want(), t)


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("parts", [1, 5])
def test_one_key_among_many(t, parts):
    """One score stands out of 700: at either end, at the edges of tiles and parts, and - unseen - just past the query's own position."""
    if t == pl.F32 and parts > 1:
        pytest.skip("parts are a bf16 form")
    at = [0, 1, 31, 32, 63, 64, 127, 128, 350, 511, 512, 698, 699, 700, 701]
    n = len(at)
    c = Case(t, 2, 32, 16, 16, 64, [760], [[699] * n], 11, spike=[(0, k, h, p) for k, p in enumerate(at) for h in range(2)])
    got, want = c.run(parts), c.want()
    close(got, want, t)
    for k, p in enumerate(at):                  # and it is that key's value, where it is visible
        v = c.uv[0] @ c.cells[c.lists[0, p], :64]
        near = np.abs(got[k, 0] - v).max() < 0.05 * np.abs(v).max()
        assert near == (p <= 699), p


@pytest.mark.parametrize("t", TYPES)
def test_sinks_of_any_size(t):
    for sink in (-50.0, 0.0, 4.0, 60.0):
        c = Case(t, 3, 16, 8, 16, 32, [40], [[0, 1, 39]], 3, sink=sink)
        got, want = c.run(1), c.want()
        assert np.abs(got - want).max() < (2e-2 if t == pl.BF16 else 1e-5) * max(np.abs(want).max(), 1e-3)


@pytest.mark.parametrize("H,dim,rot,vdim,rank,T,start", [(2, 32, 16, 32, 64, 64, 0), (3, 64, 48, 56, 120, 130, 0), (9, 128, 64, 128, 64, 200, 77), (4, 160, 96, 72, 96, 70, 190), (5, 40, 8, 24, 40, 129, 63)])
def test_expanded_attention(H, dim, rot, vdim, rank, T, start):
    """A long run over expanded keys and values against the plain form and against the latent form."""
    L, t = pl.init(), pl.BF16
    n = start + T
    ask = list(range(start, n))
    spike = [(0, T - 1, 0, 0), (0, T // 2, H - 1, start), (0, T - 2, 0, min(63, n - 2)), (0, 5, 0, start + 5), (0, 6, 0, start + 7)]
    c = Case(t, H, dim, rot, vdim, rank, [n + 3], [ask], T, spike=spike)
    lat = c.cells[c.lists[0, :n], :rank]
    keys = store(np.einsum("nr,hdr->nhd", lat, c.uk), t)
    vals = store(np.einsum("nr,hvr->nhv", lat, c.uv), t)
    q_un = np.zeros((T, H, c.dim_ld), np.float32)
    q_un[..., :dim] = c.q[..., :dim]
    ql, qu, cache, lst, nv, sk = store(c.latent_queries(), t), store(q_un, t), store(c.cells, t), i32(c.lists[0]), i32(c.pos + 1), dev(c.sink)
    ld = (H * vdim + 127) // 128 * 128
    att = pl.DevBuf.zeros(2 * T * ld)
    a = pl.LatentExpanded()
    a.q_un, a.q_lat, a.keys, a.values, a.cache, a.list, a.n_vis, a.sink, a.att = (b.ptr for b in (qu, ql, keys, vals, cache, lst, nv, sk, att))
    a.tok0, a.T, a.n_head, a.dim, a.dim_ld, a.rot_dim, a.vdim, a.rank_ld, a.kd, a.ld_att, a.scale = 0, T, H, dim, c.dim_ld, rot, vdim, c.rank_ld, c.kd, ld, c.scale
    pl.check(L.pi_k_latent_attn_expanded(C.byref(a), None))
    pl.sync()
    got = fetch(att, t, (T, ld))[:, :H * vdim].reshape(T, H, vdim)
    want = c.want()
    close(got, want, t)
    close(c.run(1), want, t)


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("own", [True, False])
def test_latent_prep(t, own):
    L, rng = pl.init(), np.random.default_rng(8)
    T, H, dim, rot, rank, base, eps = 5, 3, 17, 6, 50, 700.0, 1e-4
    rank_ld, dim_ld, kd = 64, 64, 96
    z = rng.standard_normal((T, H * (dim + rot) + rank + rot)).astype(np.float32)
    pos, cell, w = np.array([0, 5, 6, 999, 70000], np.int32), np.array([7, 0, 3, 2, 9], np.int32), rng.standard_normal(rank).astype(np.float32)
    cs, qu, ql, cache = pl.DevBuf(8 * T * rot // 2), pl.DevBuf.zeros(4 * T * H * dim_ld), pl.DevBuf.zeros(4 * T * H * kd), pl.DevBuf.zeros(4 * 10 * kd)
    pb, zb, wb, cb = i32(pos), dev(z), dev(w), i32(cell)
    pl.check(L.pi_k_rope_angles(pb.ptr, T, rot, base, cs.ptr, None))
    p = pl.LatentPrep()
    p.z, p.ldz, p.T, p.n_head, p.dim, p.dim_ld, p.rot_dim, p.kv_rank, p.rank_ld, p.kd = zb.ptr, z.shape[1], T, H, dim, dim_ld, rot, rank, rank_ld, kd
    p.cs, p.norm_w, p.eps, p.q_un, p.q_lat, p.cache, p.cell = cs.ptr, wb.ptr, eps, qu.ptr, ql.ptr, cache.ptr if own else None, cb.ptr
    pl.check(L.pi_k_latent_prep(t, C.byref(p), None))
    pl.sync()
    q = z[:, :H * (dim + rot)].reshape(T, H, dim + rot).astype(np.float64)
    assert np.abs(fetch(qu, t, (T, H, dim_ld))[..., :dim] - q[..., :dim]).max() <= tol(t, 4)
    rot_q = np.stack([o.rotate_pairs(q[:, h, dim:], pos, base) for h in range(H)], 1)
    assert np.abs(fetch(ql, t, (T, H, kd))[..., rank_ld:rank_ld + rot] - rot_q).max() <= tol(t, 4)
    got = fetch(cache, t, (10, kd))
    want = np.zeros((10, kd))
    if own:
        c = z[:, H * (dim + rot):].astype(np.float64)
        want[cell, :rank] = o.rms_norm_plain(c[:, :rank], w, eps)
        want[cell, rank_ld:rank_ld + rot] = o.rotate_pairs(c[:, rank:], pos, base)
    assert np.abs(got - want).max() <= tol(t, np.abs(want).max() + 1e-9)


@pytest.mark.parametrize("t", TYPES)
def test_latent_shift(t):
    L, rng = pl.init(), np.random.default_rng(2)
    cells, delta = as_stored(rng.standard_normal((6, 96)), t), np.array([0, 3, -2, 0, 100, 1], np.int32)
    b, db = store(cells, t), i32(delta)
    pl.check(L.pi_k_latent_shift(t, b.ptr, 6, 96, 64, 10, 300.0, db.ptr, None))
    pl.sync()
    want = cells.astype(np.float64)
    want[:, 64:74] = o.rotate_pairs(want[:, 64:74], delta, 300.0)
    assert np.abs(fetch(b, t, (6, 96)) - want).max() <= tol(t, 3)


@pytest.mark.parametrize("T,H,dim,rot,vdim,rank,E,top,ff,D,parts", [(1, 4, 16, 8, 24, 40, 6, 2, 24, 70, 4), (16, 3, 32, 16, 64, 128, 40, 8, 72, 256, 1), (5, 2, 24, 6, 80, 72, 3, 3, 300, 100, 7)])
def test_step_kernels(T, H, dim, rot, vdim, rank, E, top, ff, D, parts):
    """The fused launches of a step against the plain pieces: absorbed queries, cells and expert choice; merge + values + experts' first
    matrices; the layer's closing sum."""
    L, t, rng = pl.init(), pl.BF16, np.random.default_rng(T)
    base, eps = 1000.0, 1e-5
    c = Case(t, H, dim, rot, vdim, rank, [60 + 7 * s for s in range(T)], [[59 + 7 * s] for s in range(T)], 3 * T)
    z = rng.standard_normal((T, H * (dim + rot) + rank + rot)).astype(np.float32)
    zr, bias, w = (rng.standard_normal((T, E)) * 2).astype(np.float32), rng.standard_normal(E).astype(np.float32), rng.standard_normal(rank).astype(np.float32)
    pos, cell = np.arange(T, dtype=np.int32) * 50, rng.permutation(T + 4)[:T].astype(np.int32)
    ukt = np.zeros((H, rank, c.dim_ld), np.float32)
    ukt[..., :dim] = c.uk.transpose(0, 2, 1)
    cs, ql, cache = pl.DevBuf(8 * T * rot // 2), pl.DevBuf.zeros(2 * T * H * c.kd), pl.DevBuf.zeros(2 * (T + 4) * c.kd)
    ids, wts = pl.DevBuf(4 * T * top), pl.DevBuf(4 * T * top)
    pb, zb, wb, cb, ub, rb, bb = i32(pos), dev(z), dev(w), i32(cell), store(ukt, t), dev(zr), dev(bias)
    pl.check(L.pi_k_rope_angles(pb.ptr, T, rot, base, cs.ptr, None))
    p = pl.LatentPrep()
    p.z, p.ldz, p.T, p.n_head, p.dim, p.dim_ld, p.rot_dim, p.kv_rank, p.rank_ld, p.kd = zb.ptr, z.shape[1], T, H, dim, c.dim_ld, rot, rank, c.rank_ld, c.kd
    p.cs, p.norm_w, p.eps, p.q_un, p.q_lat, p.cache, p.cell = cs.ptr, wb.ptr, eps, None, ql.ptr, cache.ptr, cb.ptr
    pl.check(L.pi_k_latent_step(C.byref(p), ub.ptr, rb.ptr, E, top, 1, 1, bb.ptr, ids.ptr, wts.ptr, None))
    pl.sync()
    q = z[:, :H * (dim + rot)].reshape(T, H, dim + rot)
    got = fetch(ql, t, (T, H, c.kd))
    lat = np.einsum("thd,hdr->thr", rounded(q[..., :dim]).astype(np.float64), c.uk)
    assert np.abs(got[..., :rank] - lat).max() <= tol(t) * np.abs(lat).max()
    rq = np.stack([o.rotate_pairs(q[:, h, dim:].astype(np.float64), pos, base) for h in range(H)], 1)
    assert np.abs(got[..., c.rank_ld:c.rank_ld + rot] - rq).max() <= tol(t) * np.abs(rq).max()
    lt, kr = o.rms_norm_plain(z[:, H * (dim + rot):][:, :rank].astype(np.float64), w, eps), o.rotate_pairs(z[:, H * (dim + rot) + rank:].astype(np.float64), pos, base)
    gc = fetch(cache, t, (T + 4, c.kd))[cell]
    assert np.abs(gc[:, :rank] - lt).max() <= tol(t) * np.abs(lt).max() and np.abs(gc[:, c.rank_ld:c.rank_ld + rot] - kr).max() <= tol(t) * np.abs(kr).max()
    want_ids, want_w = o.route(zr.astype(np.float64), np.eye(E), bias, top, 1, 1)
    idh, wth = ids.download(np.int32).reshape(T, top), wts.download(np.float32).reshape(T, top)
    assert np.array_equal(idh, want_ids) and np.abs(wth - want_w).max() < 1e-6

    cols, ff_ld, ld_att = (D + 31) // 32 * 32, (ff + 63) // 64 * 64, (H * vdim + 127) // 128 * 128
    h = rounded(rng.standard_normal((T, D)))
    h_ol = np.zeros((cols // 8, 16, 8), np.float32)
    h_ol[:, :T] = padded(h, cols).reshape(T, cols // 8, 8).transpose(1, 0, 2)
    up, down, wo = rounded(rng.standard_normal((E, ff, D)) / np.sqrt(D)), rounded(rng.standard_normal((E, D, ff)) / np.sqrt(ff)), rounded(rng.standard_normal((D, H * vdim)) / 8)
    uvp = np.zeros((H, vdim, c.rank_ld), np.float32)
    uvp[..., :rank] = c.uv
    hb, upb, uvb, att, act = store(h_ol, t), store(padded(up.reshape(-1, D), cols), t), store(uvp, t), pl.DevBuf.zeros(2 * T * ld_att), pl.DevBuf.zeros(2 * T * top * ff_ld)
    a = c.args(parts)
    pl.check(L.pi_k_latent_attn_parts(C.byref(a), None))
    pl.check(L.pi_k_value_up_step(C.byref(a), uvb.ptr, vdim, att.ptr, ld_att, upb.ptr, E, ff, cols, hb.ptr, ids.ptr, wts.ptr, top, act.ptr, ff_ld, None))
    pl.sync()
    heads = fetch(att, t, (T, ld_att))[:, :H * vdim]
    close(heads.reshape(T, H, vdim), c.want(), t)
    acts = fetch(act, t, (T, top, ff_ld))[..., :ff]
    want = np.stack([[wth[i, k] * np.maximum(up[idh[i, k]].astype(np.float64) @ h[i], 0) ** 2 for k in range(top)] for i in range(T)])
    assert np.abs(acts - want).max() <= tol(t) * np.abs(want).max()

    x = rng.standard_normal((T, D)).astype(np.float32)
    xb, wob, dnb, out, keep = dev(x), store(padded(wo, ld_att), t), store(padded(down.reshape(-1, ff), ff_ld), t), pl.DevBuf(4 * T * D), pl.DevBuf(4 * T * D)
    for experts in (True, False):
        s = pl.LayerOut()
        s.x, s.wo, s.att, s.rows, s.ld_att, s.T, s.out, s.keep = xb.ptr, wob.ptr, att.ptr, D, ld_att, T, out.ptr, keep.ptr
        if experts:
            s.down, s.act, s.ids, s.ld_act, s.top, s.n_expert = dnb.ptr, act.ptr, ids.ptr, ff_ld, top, E
        pl.check(L.pi_k_layer_out_step(C.byref(s), None))
        pl.sync()
        want = x + heads.astype(np.float64) @ wo.T
        if experts:
            for i in range(T):
                for k in range(top):
                    want[i] += down[idh[i, k]].astype(np.float64) @ acts[i, k]
        got = out.download(np.float32).reshape(T, D)
        assert np.abs(got - want).max() < 2e-5 * np.abs(want).max() and np.array_equal(got, keep.download(np.float32).reshape(T, D))


@pytest.mark.parametrize("rows,cols,T", [(70, 256, 1), (700, 512, 16), (6000, 128, 7), (130, 384, 3)])
def test_bf16_mat_muls(rows, cols, T):
    L, t, rng = pl.init(), pl.BF16, np.random.default_rng(rows)
    W, x = rounded(rng.standard_normal((rows, cols)) / np.sqrt(cols)), rounded(rng.standard_normal((T, cols)))
    want = x.astype(np.float64) @ W.T
    wb, xb, y = store(W, t), store(x, t), pl.DevBuf(4 * T * rows)
    ol = np.zeros((cols // 8, 16, 8), np.float32)
    ol[:, :T] = x.reshape(T, cols // 8, 8).transpose(1, 0, 2)
    xo = store(ol, t)
    calls = [lambda: L.pi_k_gemm_bf16(wb.ptr, rows, cols, xb.ptr, T, 0, None, None, y.ptr, None, None),
             lambda: L.pi_k_gemm_bf16_ol(wb.ptr, rows, cols, xo.ptr, T, 0, None, None, y.ptr, None, None),
             lambda: L.pi_k_gemm_tile_bf16(wb.ptr, rows, cols, xb.ptr, T, 0, None, None, y.ptr, None, 0, None)]
    for call in calls:
        pl.check(call())
        pl.sync()
        assert np.abs(y.download(np.float32).reshape(T, rows) - want).max() < 1e-5 * np.abs(want).max()
    if cols % 256 == 0:
        y2 = pl.DevBuf(4 * T * 30)
        pl.check(L.pi_k_gemm_bf16_ol_two(wb.ptr, rows, xo.ptr, y.ptr, wb.ptr, 30, xo.ptr, y2.ptr, cols, T, None))
        pl.sync()
        assert np.abs(y.download(np.float32).reshape(T, rows) - want).max() < 1e-5 * np.abs(want).max()
        assert np.abs(y2.download(np.float32).reshape(T, 30) - want[:, :30]).max() < 1e-5 * np.abs(want).max()


def test_bf16_library_mat_mul():
    L, t, rng = pl.init(), pl.BF16, np.random.default_rng(1)
    rows, cols, T = 1024, 1024, 300
    W, x = rounded(rng.standard_normal((rows, cols)) / 32), rounded(rng.standard_normal((T, cols)))
    wb, xb, y, y16 = store(W, t), store(x, t), pl.DevBuf(4 * T * rows), pl.DevBuf(2 * T * rows)
    g = L.pi_gemm_lib_create(1 << 24)
    pl.check(L.pi_gemm_lib_bf16(g, wb.ptr, rows, cols, xb.ptr, T, pl.EPI_RELU, None, None, y.ptr, y16.ptr, None))
    pl.sync()
    want = np.maximum(x.astype(np.float64) @ W.T, 0)
    assert np.abs(y.download(np.float32).reshape(T, rows) - want).max() < 1e-5 * np.abs(want).max()
    assert np.abs(fetch(y16, t, (T, rows)) - want).max() < 5e-3 * np.abs(want).max()
    L.pi_gemm_lib_destroy(g)


def test_bad_arguments_are_errors():
    L = pl.init()
    g = group_args(rows=4, cols=33, ldw=33, n_group=1, ldx=33, T=1, ldy=4)
    assert L.pi_k_group_gemm(pl.BF16, C.byref(g), None) < 0
    assert L.pi_k_latent_attn(pl.BF16, C.byref(pl.LatentAttn()), None) < 0
    assert L.pi_k_latent_attn_supported(pl.BF16, 2048, 2080) == 0 and L.pi_k_latent_attn_supported(pl.BF16, 512, 576) == 1
    assert L.pi_k_route(None, 1, 4, 2, 3, 1, None, None, None, None) < 0
