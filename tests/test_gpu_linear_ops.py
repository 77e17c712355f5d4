"""Decayed linear attention: token by token and in chunks against the plain recurrence (tests/plain_pibalorn.py)."""
import ctypes as C

import numpy as np
import pytest

import plain_pibalorn as o
from powerinfer_amd import lib as pl
from test_gpu_gqa_ops import check_front, filled, front
from test_gpu_latent_ops import TYPES, as_stored, dev, fetch, i32, tol

pytestmark = pytest.mark.gpu


def run(t, rng, runs, H, dim, vdim, decay, chunked, slots=5, gap=3, ff=0, E=0):
    """runs: (tokens, slot, starts at zero).  Returns (outputs, wanted outputs, states, wanted states)."""
    L = pl.init()
    T = sum(n for n, _, _ in runs)
    off_k = (H * dim + gap + 15) // 16 * 16
    off_v = (off_k + H * dim + gap + 15) // 16 * 16
    off_glu = (off_v + H * vdim + 15) // 16 * 16
    ldz = (off_glu + 2 * ff + E + 15) // 16 * 16
    z = rng.standard_normal((T, ldz)).astype(np.float32)
    state = rng.standard_normal((slots, H, dim, vdim)).astype(np.float32)
    dec = np.asarray(decay, np.float32)
    Cn = L.pi_k_linear_chunk()
    powers = np.stack([dec.astype(np.float64) ** k for k in range(Cn + 1)], 1).astype(np.float32)
    items, chunks, first, at = [], [], [], 0
    for n, s, fresh in runs:
        items.append([at, n, s, fresh])
        first.append(len(chunks))
        chunks += [[at + c, min(Cn, n - c), int(fresh and c == 0)] for c in range(0, n, Cn)]
        at += n
    dim_ld, vdim_ld = (dim + 31) // 32 * 32, (vdim + 63) // 64 * 64
    f, bufs = front(z, t, ff, off_glu, -1, 1.2, E, off_glu + 2 * ff, min(E, 2))
    b = dict(z=dev(z), decay=dev(dec), powers=dev(powers), state=dev(state), runs=i32(items), o=pl.DevBuf.zeros(4 * T * H * vdim), q=pl.DevBuf(2 * T * H * dim_ld),
             k=pl.DevBuf(2 * T * H * dim_ld), v=pl.DevBuf(2 * T * H * vdim_ld), states=pl.DevBuf(L.pi_k_linear_states_bytes(len(chunks), H, dim_ld, vdim_ld)), chunks=i32(chunks),
             first_chunk=i32(first))
    p = filled(pl.Linear, ldz=ldz, T=T, n_head=H, dim=dim, vdim=vdim, off_k=off_k, off_v=off_v, n_runs=len(items), dim_ld=dim_ld, vdim_ld=vdim_ld, n_chunks=len(chunks), **b)
    if chunked:
        pl.check(L.pi_k_linear_prep(t, C.byref(p), C.byref(f), None))
        pl.check(L.pi_k_linear_chunks(C.byref(p), None))
    else:
        pl.check(L.pi_k_linear_step(t, C.byref(p), C.byref(f), None))
    pl.sync()
    check_front(z, t, f, bufs)
    parts = [as_stored(o.silu(z[:, a:a + w].astype(np.float64)), t).astype(np.float64).reshape(T, H, -1) for a, w in ((0, H * dim), (off_k, H * dim), (off_v, H * vdim))]
    if chunked:
        for name, w, ld in (("q", parts[0], dim_ld), ("k", parts[1], dim_ld), ("v", parts[2], vdim_ld)):
            got = fetch(b[name], pl.BF16, (T, H, ld))
            assert np.abs(got[..., :w.shape[2]] - w).max() <= 6e-3 * np.abs(w).max() and not got[..., w.shape[2]:].any()
    want, ends, at = np.empty((T, H, vdim)), state.astype(np.float64), 0
    for n, s, fresh in runs:
        want[at:at + n], ends[s] = o.decayed_sums(*[x[at:at + n] for x in parts], dec, ends[s] * (not fresh))
        at += n
    return b["o"].download(np.float32).reshape(T, H, vdim), want, b["state"].download(np.float32).reshape(state.shape), ends


def close(got, want, limit):
    return np.abs(got - want).max() <= limit * np.abs(want).max()


SHAPES = [(3, 20, 36, (1.0, 0.5, 0.03)), (4, 64, 64, (0.997, 0.7, 0.95, 0.4)), (5, 33, 9, (0.999, 0.9, 0.0, 0.7, 0.97)), (1, 128, 128, (0.98,)), (2, 256, 70, (0.9, 1.0)), (2, 90, 256, (0.99, 0.5)),
          (1, 1, 1, (0.9,))]


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("H,dim,vdim,decay", SHAPES)
def test_token_by_token(t, H, dim, vdim, decay):
    runs = [(1, 3, False), (16, 0, True), (2, 4, True), (1, 1, True), (40, 2, False)]
    got, want, states, ends = run(t, np.random.default_rng(dim), runs, H, dim, vdim, decay, False, ff=20, E=5)
    # (bf16: silu may fall on the other side of a rounding boundary than the oracle's)
    assert close(got, want, 2e-3 if t == pl.BF16 else 1e-5) and close(states, ends, 2e-3 if t == pl.BF16 else 1e-5)


@pytest.mark.parametrize("H,dim,vdim,decay", SHAPES)
@pytest.mark.parametrize("runs", [[(64, 0, True)], [(17, 1, True), (63, 0, False), (65, 3, True), (200, 2, False)], [(128, 4, False), (1, 0, True), (129, 1, True)]])
def test_chunks(H, dim, vdim, decay, runs):
    got, want, states, ends = run(pl.BF16, np.random.default_rng(vdim), runs, H, dim, vdim, decay, True, ff=1100, E=9)
    assert close(got, want, 2e-3) and close(states, ends, 2e-3)
    at = 0
    for n, _, _ in runs:                                                       # no token is off, also where the sums are small
        for i in range(at, at + n):
            assert np.abs(got[i] - want[i]).max() <= 4e-3 * np.abs(want[i]).max() + 1e-4, (i - at, n)
        at += n


def test_chunks_and_steps_agree_closely():
    """The same tokens in chunks and one by one: what fp32 numbers lose as sums of two bf16 is far below bf16's own rounding."""
    runs, rng = [(150, 0, False)], lambda: np.random.default_rng(9)
    a, _, sa, _ = run(pl.BF16, rng(), runs, 3, 64, 64, (0.999, 1.0, 0.8), True)
    b, _, sb, _ = run(pl.BF16, rng(), runs, 3, 64, 64, (0.999, 1.0, 0.8), False)
    assert close(a, b, 3e-5) and close(sa, sb, 3e-5)


def test_state_far_back_decides():
    """With nothing but the first token's pair in the state, decay 1, hundreds of tokens later its value is what comes out."""
    L, n, dim, vdim = pl.init(), 300, 32, 32
    rng = np.random.default_rng(3)
    z = np.full((n, 3 * 32), -40.0, np.float32)                                # silu: nothing
    z[0, 32:64], z[0, 64:] = 5.0, 5 * rng.random(32)
    z[-1, :32] = 5.0
    for chunked in (False, True):
        b = dict(z=dev(z), decay=dev(np.ones(1, np.float32)), powers=dev(np.ones(65, np.float32)), state=dev(np.full((1, 1, 32, 32), 7, np.float32)), runs=i32([0, n, 0, 1]),
                 o=pl.DevBuf.zeros(4 * n * 32), q=pl.DevBuf(2 * n * 32), k=pl.DevBuf(2 * n * 32), v=pl.DevBuf(2 * n * 64), states=pl.DevBuf(L.pi_k_linear_states_bytes(5, 1, 32, 64)),
                 chunks=i32([[c, min(64, n - c), int(c == 0)] for c in range(0, n, 64)]), first_chunk=i32([0]))
        p = filled(pl.Linear, ldz=96, T=n, n_head=1, dim=dim, vdim=vdim, off_k=32, off_v=64, n_runs=1, dim_ld=32, vdim_ld=64, n_chunks=5, **b)
        if chunked:
            pl.check(L.pi_k_linear_prep(pl.BF16, C.byref(p), None, None))
            pl.check(L.pi_k_linear_chunks(C.byref(p), None))
        else:
            pl.check(L.pi_k_linear_step(pl.BF16, C.byref(p), None, None))
        pl.sync()
        got = b["o"].download(np.float32).reshape(n, 32)[-1]
        want = o.silu(5.0) ** 2 * 32 * o.silu(z[0, 64:].astype(np.float64))
        assert np.abs(got - want).max() < 1e-2 * want.max()


@pytest.mark.parametrize("t", TYPES)
@pytest.mark.parametrize("T,n", [(1, 50), (7, 4096), (3, 5000)])
def test_gate_norm(t, T, n):
    L, rng = pl.init(), np.random.default_rng(n)
    x, z, w = rng.standard_normal((T, n)).astype(np.float32) * 4, rng.standard_normal((T, n + 9)).astype(np.float32), rng.random(n).astype(np.float32)
    xb, zb, wb, att = dev(x), dev(z), dev(w), pl.DevBuf.zeros(4 * T * (n + 4))
    g = filled(pl.GateNorm, scale=1.0, o=xb, z=zb, w=wb, ldz=n + 9, off_gate=4, n=n, T=T, eps=1e-5, att=att, ld_att=n + 4)
    pl.check(L.pi_k_gate_norm(t, C.byref(g), None))
    pl.sync()
    want = o.unit(x.astype(np.float64), 1e-5) * w * o.sigmoid(z[:, 4:4 + n].astype(np.float64))
    got = fetch(att, t, (T, n + 4))
    assert np.abs(got[:, :n] - want).max() <= tol(t) * np.abs(want).max() and not got[:, n:].any()
