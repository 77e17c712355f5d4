// Linear attention with a constant decay per head over a fp32 state per sequence: token by token for steps (any storage type), and in
// chunks on the matrix cores for long prompt portions.  With d the decay and S the state before a chunk, token i of the chunk has
//   o_i = d^(i+1) S^T q_i + sum over j <= i of d^(i-j) (q_i . k_j) v_j,     S' = d^n S + sum over j of d^(n-1-j) k_j v_j^T.
// Whatever is fp32 (states, decayed keys, decayed scores) enters the matrix cores as the sum of two bf16, which keeps 16 bits of mantissa.
#include "mixers.hpp"

namespace {

constexpr int kLinCols = 32;             // value columns of a workgroup of the token-by-token kernel
constexpr int kLinBlock = 16;            // tokens staged at a time
constexpr int kLinMax = 256;

// a thread keeps J consecutive rows of one column of the state in registers; 8 groups of rows x 32 columns
template <typename ST, int J>
__global__ __launch_bounds__(256) void linear_step_kernel(pi_linear p, pi_ffn_front f, int n_state, int slices, int per) {
    constexpr int D = 8 * J;
    extern __shared__ __align__(16) float sm[];
    if ((int)blockIdx.x >= n_state) {
        const int b = blockIdx.x - n_state;
        front_block<ST>(f, p.z, p.ldz, b / per, b % per, sm);
        return;
    }
    float * qs = sm, * ks = qs + kLinBlock * D, * vs = ks + kLinBlock * D, * part = vs + kLinBlock * kLinCols;      // [16][D], [16][D], [16][32], [4][16][32]
    const int slice = blockIdx.x % slices, h = (int)blockIdx.x / slices % p.n_head, tid = threadIdx.x;
    const int4 run = reinterpret_cast<const int4 *>(p.runs)[(int)blockIdx.x / slices / p.n_head];
    const int c = tid % kLinCols, rg = tid / kLinCols, col = slice * kLinCols + c, wave = tid >> 6;
    const float d = p.decay[h];
    float * S = p.state + ((size_t)run.z * p.n_head + h) * p.dim * p.vdim;
    float s[J];
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int r = rg * J + j;
        s[j] = !run.w && r < p.dim && col < p.vdim ? S[(size_t)r * p.vdim + col] : 0.0f;
    }
    for (int t0 = 0; t0 < run.y; t0 += kLinBlock) {
        const int n = min(kLinBlock, run.y - t0);
        if (t0) __syncthreads();
        for (int e = tid; e < n * D; e += 256) {
            const int t = e / D, r = e % D;
            const float * z = p.z + (size_t)(run.x + t0 + t) * p.ldz + h * p.dim + r;
            qs[e] = r < p.dim ? from_st(to_st<ST>(silu_f32(z[0]))) : 0.0f;
            ks[e] = r < p.dim ? from_st(to_st<ST>(silu_f32(z[p.off_k]))) : 0.0f;
        }
        for (int e = tid; e < n * kLinCols; e += 256) {
            const int t = e / kLinCols, v = slice * kLinCols + e % kLinCols;
            vs[e] = v < p.vdim ? from_st(to_st<ST>(silu_f32(p.z[(size_t)(run.x + t0 + t) * p.ldz + p.off_v + h * p.vdim + v]))) : 0.0f;
        }
        __syncthreads();
        for (int t = 0; t < n; ++t) {
            const float v = vs[t * kLinCols + c];
            float a = 0.0f;
#pragma unroll
            for (int j = 0; j < J; j += 4) {
                const float4 k = *reinterpret_cast<const float4 *>(ks + t * D + rg * J + j), q = *reinterpret_cast<const float4 *>(qs + t * D + rg * J + j);
                s[j] = fmaf(k.x, v, d * s[j]); a = fmaf(q.x, s[j], a);
                s[j + 1] = fmaf(k.y, v, d * s[j + 1]); a = fmaf(q.y, s[j + 1], a);
                s[j + 2] = fmaf(k.z, v, d * s[j + 2]); a = fmaf(q.z, s[j + 2], a);
                s[j + 3] = fmaf(k.w, v, d * s[j + 3]); a = fmaf(q.w, s[j + 3], a);
            }
            a += __shfl_xor(a, 32, PI_WAVE);
            if ((tid & 63) < kLinCols) part[(wave * kLinBlock + t) * kLinCols + c] = a;
        }
        __syncthreads();
        for (int e = tid; e < n * kLinCols; e += 256) {
            const int t = e / kLinCols, v = slice * kLinCols + e % kLinCols;
            if (v < p.vdim) p.o[(size_t)(run.x + t0 + t) * p.n_head * p.vdim + h * p.vdim + v] =
                part[e] + part[kLinBlock * kLinCols + e] + part[2 * kLinBlock * kLinCols + e] + part[3 * kLinBlock * kLinCols + e];
        }
    }
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int r = rg * J + j;
        if (r < p.dim && col < p.vdim) S[(size_t)r * p.vdim + col] = s[j];
    }
}

// silu of the projections as bf16 operands, rows padded with zeros: a block covers 4096 values of a token's [q | k | v], a thread four of
// every 1024
constexpr int kLinPrep = 4096;
__global__ __launch_bounds__(256) void linear_prep_kernel(pi_linear p, pi_ffn_front f, int n_val, int per) {
    extern __shared__ __align__(16) float sm[];
    const int t = blockIdx.x / per, b = blockIdx.x % per;
    if (b >= n_val) { front_block<bf16>(f, p.z, p.ldz, t, b - n_val, sm); return; }
    const int nq = p.n_head * p.dim_ld, all = 2 * nq + p.n_head * p.vdim_ld;
    constexpr int Q = kLinPrep / 1024;
    float v[Q][4];
    bf16 * o[Q];
#pragma unroll
    for (int i = 0; i < Q; ++i) {
        const int e = min(b * kLinPrep + i * 1024 + (int)threadIdx.x * 4, all - 4);      // past the end: the last four again, the same values
        const int what = e < nq ? 0 : e < 2 * nq ? 1 : 2, k = e - what * nq, ld = what == 2 ? p.vdim_ld : p.dim_ld, dim = what == 2 ? p.vdim : p.dim, h = k / ld, r = k % ld;
        const float * z = p.z + (size_t)t * p.ldz + (what == 0 ? 0 : what == 1 ? p.off_k : p.off_v) + h * dim + r;
        o[i] = (bf16 *)(what == 0 ? p.q : what == 1 ? p.k : p.v) + (size_t)t * p.n_head * ld + k;
        if (r + 4 <= dim && ((uintptr_t)z & 15) == 0) {
            const float4 a = *reinterpret_cast<const float4 *>(z);
            v[i][0] = a.x; v[i][1] = a.y; v[i][2] = a.z; v[i][3] = a.w;
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j) v[i][j] = r + j < dim ? z[j] : 0.0f;
        }
    }
#pragma unroll
    for (int i = 0; i < Q; ++i) {
#pragma unroll
        for (int j = 0; j < 4; ++j) v[i][j] = silu_f32(v[i][j]);            // (silu(0) = 0)
        store4(o[i], v[i], true, 4);
    }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// chunks
// ---------------------------------------------------------------------------------------------------------------------------------
constexpr int kLinC = 64;                // tokens of a chunk
typedef short pi_s4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ pi_u32x2 lin_tr(const unsigned char * q) {
    return __builtin_bit_cast(pi_u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) pi_s4 *)(__attribute__((address_space(3))) void *)q));
}
// operand with 32 rows of LDS as its inner dimension: lane (column i, rows 8 g ..)
__device__ __forceinline__ pi_u32x4 lin_frag(const unsigned char * rows, int stride, int col) {
    const int lane = threadIdx.x & 63, g = lane >> 4, li = lane & 15;
    const unsigned char * a = rows + (8 * g + (li >> 2)) * stride + (col + (li & 3) * 4) * 2;
    const pi_u32x2 lo = lin_tr(a), hi = lin_tr(a + 4 * stride);
    return pi_u32x4{lo.x, lo.y, hi.x, hi.y};
}
__device__ __forceinline__ void split_bf16(float v, bf16 & hi, bf16 & lo) { hi = (bf16)v; lo = (bf16)(v - (float)hi); }

// states: per (chunk, head) the state before the chunk, transposed, as two bf16 matrices [vdim_ld][dim_ld].  A workgroup owns 32 rows x 64
// value columns of one head's state and walks the run's chunks; the next chunk's keys and values are requested while one is multiplied.
__global__ __launch_bounds__(256) void linear_states_kernel(pi_linear p, int tiles_d, int tiles_v) {
    constexpr int KROW = 32 * 2 + 16, VROW = 64 * 2 + 16;
    __shared__ __align__(16) unsigned char kh[kLinC * KROW], kl[kLinC * KROW], vs[kLinC * VROW];
    const int tile = blockIdx.x % (tiles_d * tiles_v), h = blockIdx.x / (tiles_d * tiles_v), ri = blockIdx.y;
    const int d0 = tile / tiles_v * 32, v0 = tile % tiles_v * 64;
    const int4 run = reinterpret_cast<const int4 *>(p.runs)[ri];
    const int chunk0 = p.first_chunk[ri], n_chunk = (run.y + kLinC - 1) / kLinC;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    const float * pw = p.powers + (size_t)h * (kLinC + 1);
    float * S = p.state + ((size_t)run.z * p.n_head + h) * p.dim * p.vdim;
    const int vcol = v0 + wave * 16 + i;
    pi_f4 acc[2];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = d0 + m * 16 + 4 * g + r;
            acc[m][r] = !run.w && row < p.dim && vcol < p.vdim ? S[(size_t)row * p.vdim + vcol] : 0.0f;
        }
    const int kt = tid / 4, kc = (tid % 4) * 8, vt = tid / 8, vc = (tid % 8) * 8;
    const size_t ldk = (size_t)p.n_head * p.dim_ld, ldv = (size_t)p.n_head * p.vdim_ld;
    const uint16_t * kp = (const uint16_t *)p.k + h * p.dim_ld + d0 + kc, * vp = (const uint16_t *)p.v + h * p.vdim_ld + v0 + vc;
    const int last = run.x + run.y - 1;
    pi_u32x4 rk, rv[2];
    auto fetch = [&](int t0) {
        rk = pi_ld16(kp + (size_t)min(t0 + kt, last) * ldk);
        rv[0] = pi_ld16(vp + (size_t)min(t0 + vt, last) * ldv);
        rv[1] = pi_ld16(vp + (size_t)min(t0 + 32 + vt, last) * ldv);
    };
    fetch(run.x);
    for (int ck = 0; ck < n_chunk; ++ck) {
        const int n = min(kLinC, run.y - ck * kLinC);
        __syncthreads();
        {
            const bf16 * kb = reinterpret_cast<const bf16 *>(&rk);
            const float w = kt < n ? pw[n - 1 - kt] : 0.0f;
            bf16 hi[8], lo[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) split_bf16((float)kb[j] * w, hi[j], lo[j]);
            *reinterpret_cast<pi_u32x4 *>(kh + kt * KROW + kc * 2) = __builtin_bit_cast(pi_u32x4, hi);
            *reinterpret_cast<pi_u32x4 *>(kl + kt * KROW + kc * 2) = __builtin_bit_cast(pi_u32x4, lo);
            *reinterpret_cast<pi_u32x4 *>(vs + vt * VROW + vc * 2) = rv[0];
            *reinterpret_cast<pi_u32x4 *>(vs + (32 + vt) * VROW + vc * 2) = rv[1];
        }
        __syncthreads();
        fetch(run.x + (ck + 1) * kLinC);                         // past the last chunk: its last token again, not used
        bf16 * out = (bf16 *)p.states + ((size_t)(chunk0 + ck) * p.n_head + h) * 2 * p.vdim_ld * p.dim_ld + (size_t)vcol * p.dim_ld + d0 + 4 * g;
        const float dn = pw[n];
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            bf16 hi[4], lo[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) { split_bf16(acc[m][r], hi[r], lo[r]); acc[m][r] *= dn; }
            *reinterpret_cast<pi_u32x2 *>(out + m * 16) = __builtin_bit_cast(pi_u32x2, hi);
            *reinterpret_cast<pi_u32x2 *>(out + (size_t)p.vdim_ld * p.dim_ld + m * 16) = __builtin_bit_cast(pi_u32x2, lo);
        }
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const pi_u32x4 b = lin_frag(vs + s * 32 * VROW, VROW, wave * 16);
#pragma unroll
            for (int m = 0; m < 2; ++m) {
                acc[m] = mfma_bf16(lin_frag(kh + s * 32 * KROW, KROW, m * 16), b, acc[m]);
                acc[m] = mfma_bf16(lin_frag(kl + s * 32 * KROW, KROW, m * 16), b, acc[m]);
            }
        }
    }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = d0 + m * 16 + 4 * g + r;
            if (row < p.dim && vcol < p.vdim) S[(size_t)row * p.vdim + vcol] = acc[m][r];
        }
}

// outputs of one chunk of one head.  Wave w forms the decayed scores of tokens 16 w .. (as columns, keys x tokens) and leaves them in LDS in
// operand order; then every wave owns a quarter of the value columns for all tokens of the chunk.
template <int VPW>                       // 16-column value tiles per wave
__global__ __launch_bounds__(256) void linear_out_kernel(pi_linear p) {
    extern __shared__ __align__(16) unsigned char smem[];
    const int qrow = p.dim_ld * 2 + 16, vrow = p.vdim_ld * 2 + 16;
    unsigned char * qs = smem, * ks = qs + kLinC * qrow, * vs = ks + kLinC * qrow;
    pi_u32x4 * pp = reinterpret_cast<pi_u32x4 *>(vs + kLinC * vrow);          // [4 column tiles][2 steps][hi, lo][64]
    float * pw = reinterpret_cast<float *>(pp + 4 * 2 * 2 * 64);              // [kLinC + 1]
    const int h = blockIdx.x % p.n_head, ck = blockIdx.x / p.n_head;
    const int tok0 = p.chunks[3 * ck], n = p.chunks[3 * ck + 1], fresh = p.chunks[3 * ck + 2];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    for (int e = tid; e <= kLinC; e += 256) pw[e] = p.powers[(size_t)h * (kLinC + 1) + e];
    const int qp = p.dim_ld / 8, vp = p.vdim_ld / 8;
    for (int e = tid; e < kLinC * qp; e += 256) {
        const int t = e / qp, c = (e % qp) * 8;
        const size_t o = (size_t)(tok0 + min(t, n - 1)) * p.n_head * p.dim_ld + h * p.dim_ld + c;
        *reinterpret_cast<pi_u32x4 *>(qs + t * qrow + c * 2) = pi_ld16((const uint16_t *)p.q + o);
        *reinterpret_cast<pi_u32x4 *>(ks + t * qrow + c * 2) = pi_ld16((const uint16_t *)p.k + o);
    }
    for (int e = tid; e < kLinC * vp; e += 256) {
        const int t = e / vp, c = (e % vp) * 8;
        *reinterpret_cast<pi_u32x4 *>(vs + t * vrow + c * 2) = pi_ld16((const uint16_t *)p.v + (size_t)(tok0 + min(t, n - 1)) * p.n_head * p.vdim_ld + h * p.vdim_ld + c);
    }
    __syncthreads();
    const int nk = p.dim_ld / 32;
    {
        pi_f4 s[4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) s[kt] = pi_f4{0, 0, 0, 0};
        for (int k = 0; k < nk; ++k) {
            const pi_u32x4 q = *reinterpret_cast<const pi_u32x4 *>(qs + (wave * 16 + i) * qrow + k * 64 + g * 16);
#pragma unroll
            for (int kt = 0; kt < 4; ++kt)
                if (kt <= wave) s[kt] = mfma_bf16(*reinterpret_cast<const pi_u32x4 *>(ks + (kt * 16 + i) * qrow + k * 64 + g * 16), q, s[kt]);
        }
        const int ti = wave * 16 + i;                             // this lane's token
#pragma unroll
        for (int st = 0; st < 2; ++st) {
            bf16 hi[8], lo[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int kt = 2 * st + (j >> 2), tj = kt * 16 + 4 * g + (j & 3);
                split_bf16(tj <= ti ? s[kt][j & 3] * pw[max(ti - tj, 0)] : 0.0f, hi[j], lo[j]);
            }
            pp[((wave * 2 + st) * 2) * 64 + lane] = __builtin_bit_cast(pi_u32x4, hi);
            pp[((wave * 2 + st) * 2 + 1) * 64 + lane] = __builtin_bit_cast(pi_u32x4, lo);
        }
    }
    __syncthreads();
    pi_f4 acc[VPW][4];
#pragma unroll
    for (int v = 0; v < VPW; ++v)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[v][c] = pi_f4{0, 0, 0, 0};
    const int n_vt = p.vdim_ld / 16;
    if (!fresh) {
        const bf16 * S = (const bf16 *)p.states + ((size_t)ck * p.n_head + h) * 2 * p.vdim_ld * p.dim_ld;
        const size_t half = (size_t)p.vdim_ld * p.dim_ld;
        for (int k = 0; k < nk; ++k) {
            pi_u32x4 q[4];
#pragma unroll
            for (int c = 0; c < 4; ++c) q[c] = *reinterpret_cast<const pi_u32x4 *>(qs + (c * 16 + i) * qrow + k * 64 + g * 16);
#pragma unroll
            for (int v = 0; v < VPW; ++v) {
                const int vt = min(wave + 4 * v, n_vt - 1);
                const bf16 * a = S + (size_t)(vt * 16 + i) * p.dim_ld + k * 32 + g * 8;
                const pi_u32x4 hi = pi_ld16(a), lo = pi_ld16(a + half);
#pragma unroll
                for (int c = 0; c < 4; ++c) { acc[v][c] = mfma_bf16(hi, q[c], acc[v][c]); acc[v][c] = mfma_bf16(lo, q[c], acc[v][c]); }
            }
        }
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const float w = pw[c * 16 + i + 1];
#pragma unroll
            for (int v = 0; v < VPW; ++v) acc[v][c] *= w;
        }
    }
#pragma unroll
    for (int st = 0; st < 2; ++st)
#pragma unroll
        for (int v = 0; v < VPW; ++v) {
            const int vt = min(wave + 4 * v, n_vt - 1);
            // slot (g, j) of the step: token 4 g + j of its first 16 (j < 4) or of its second 16, as the scores came out
            const unsigned char * a = vs + (st * 32 + 4 * g + (i >> 2)) * vrow + (vt * 16 + (i & 3) * 4) * 2;
            const pi_u32x2 x = lin_tr(a), y = lin_tr(a + 16 * vrow);
            const pi_u32x4 f{x.x, x.y, y.x, y.y};
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                if (2 * st > c) continue;                         // tokens before the step's keys
                acc[v][c] = mfma_bf16(f, pp[((c * 2 + st) * 2) * 64 + lane], acc[v][c]);
                acc[v][c] = mfma_bf16(f, pp[((c * 2 + st) * 2 + 1) * 64 + lane], acc[v][c]);
            }
        }
    const bool quads = (p.vdim & 3) == 0;
#pragma unroll
    for (int v = 0; v < VPW; ++v) {
        const int vt = wave + 4 * v, vr = vt * 16 + 4 * g;
        if (vt >= n_vt || vr >= p.vdim) continue;
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int t = c * 16 + i;
            if (t >= n) continue;
            const float w[4] = {acc[v][c][0], acc[v][c][1], acc[v][c][2], acc[v][c][3]};
            store4(p.o + (size_t)(tok0 + t) * p.n_head * p.vdim + h * p.vdim + vr, w, quads, p.vdim - vr);
        }
    }
}

template <typename ST>
__global__ __launch_bounds__(256) void gate_norm_kernel(pi_gate_norm p) {
    __shared__ double red[4];
    gate_norm_token<ST>(p, blockIdx.x, red);
}

template <typename ST, int J> int launch_step(const pi_linear * p, const pi_ffn_front & f, hipStream_t st) {
    const int slices = (p->vdim + kLinCols - 1) / kLinCols, n_state = p->n_runs * p->n_head * slices, per = front_blocks(f);
    const size_t own = sizeof(float) * (2 * kLinBlock * 8 * J + kLinBlock * kLinCols + 4 * kLinBlock * kLinCols), lds = own > front_lds_bytes(f) ? own : front_lds_bytes(f);
    if (n_state + per * p->T <= 0) return PI_OK;
    hipLaunchKernelGGL((linear_step_kernel<ST, J>), dim3(n_state + per * p->T), dim3(256), lds, st, *p, f, n_state, slices, per);
    return pi::check_launch("pi_k_linear_step");
}
template <typename ST> int step_of_type(const pi_linear * p, const pi_ffn_front & f, hipStream_t st) {
    if (p->dim <= 32) return launch_step<ST, 4>(p, f, st);
    if (p->dim <= 64) return launch_step<ST, 8>(p, f, st);
    if (p->dim <= 96) return launch_step<ST, 12>(p, f, st);
    if (p->dim <= 128) return launch_step<ST, 16>(p, f, st);
    return launch_step<ST, 32>(p, f, st);
}

bool linear_ok(const pi_linear * p, const pi_ffn_front & f) {
    return p && p->z && p->T > 0 && p->n_head > 0 && pi_k_linear_supported(p->dim, p->vdim) && p->off_k >= 0 && p->off_v >= 0 && p->off_k + p->n_head * p->dim <= p->ldz &&
           p->n_head * p->dim <= p->ldz && p->off_v + p->n_head * p->vdim <= p->ldz && front_ok(f, p->ldz) && (long long)p->T * (front_blocks(f) + 3 * (p->n_head + 1)) < (1 << 30);
}
bool operands_ok(const pi_linear * p) {
    return p->q && p->k && p->v && p->dim_ld >= p->dim && p->dim_ld % 32 == 0 && p->vdim_ld >= p->vdim && p->vdim_ld % 64 == 0 && p->dim_ld <= kLinMax && p->vdim_ld <= kLinMax;
}

template <int VPW> int launch_out(const pi_linear * p, hipStream_t st) {
    const size_t lds = (size_t)kLinC * (2 * (p->dim_ld * 2 + 16) + p->vdim_ld * 2 + 16) + 4 * 2 * 2 * 64 * 16 + sizeof(float) * (kLinC + 4);
    static bool raised = false;
    if (!raised) { PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&linear_out_kernel<VPW>), hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024)); raised = true; }
    hipLaunchKernelGGL(linear_out_kernel<VPW>, dim3(p->n_chunks * p->n_head), dim3(256), lds, st, *p);
    return pi::check_launch("pi_k_linear_chunks out");
}

}  // namespace

extern "C" {

int pi_k_linear_chunk(void) { return kLinC; }
int pi_k_linear_supported(int dim, int vdim) { return dim > 0 && vdim > 0 && dim <= kLinMax && vdim <= kLinMax; }
size_t pi_k_linear_states_bytes(int n_chunks, int n_head, int dim_ld, int vdim_ld) { return (size_t)n_chunks * n_head * dim_ld * vdim_ld * 4; }

int pi_k_linear_step(int type, const pi_linear * p, const pi_ffn_front * front, pi_stream_t stream) {
    const pi_ffn_front f = front ? *front : pi_ffn_front{};
    if (!linear_ok(p, f) || p->n_runs < 0 || (p->n_runs > 0 && (!p->decay || !p->state || !p->runs || !p->o)) || (long long)p->n_runs * p->n_head * 8 > (1 << 29))
        return pi::fail(PI_E_ARG, "pi_k_linear_step: bad arguments");
    if (type == PI_TYPE_BF16) return step_of_type<bf16>(p, f, (hipStream_t)stream);
    if (type == PI_TYPE_F32) return step_of_type<float>(p, f, (hipStream_t)stream);
    return pi::fail(PI_E_UNSUPPORTED, "pi_k_linear_step: type");
}

int pi_k_linear_prep(int type, const pi_linear * p, const pi_ffn_front * front, pi_stream_t stream) {
    const pi_ffn_front f = front ? *front : pi_ffn_front{};
    if (type != PI_TYPE_BF16) return pi::fail(PI_E_UNSUPPORTED, "pi_k_linear_prep: type");
    if (!linear_ok(p, f) || !operands_ok(p)) return pi::fail(PI_E_ARG, "pi_k_linear_prep: bad arguments");
    const int n_val = (p->n_head * (2 * p->dim_ld + p->vdim_ld) + kLinPrep - 1) / kLinPrep, per = n_val + front_blocks(f);
    hipLaunchKernelGGL(linear_prep_kernel, dim3(per * p->T), dim3(256), front_lds_bytes(f), (hipStream_t)stream, *p, f, n_val, per);
    return pi::check_launch("pi_k_linear_prep");
}

int pi_k_linear_chunks(const pi_linear * p, pi_stream_t stream) {
    if (!linear_ok(p, pi_ffn_front{}) || !operands_ok(p) || !p->powers || !p->state || !p->runs || p->n_runs <= 0 || p->n_runs > 65535 || !p->o || !p->states || p->n_chunks <= 0 || !p->chunks ||
        !p->first_chunk || (long long)p->n_chunks * p->n_head > (1 << 30))
        return pi::fail(PI_E_ARG, "pi_k_linear_chunks: bad arguments");
    hipStream_t st = (hipStream_t)stream;
    const int td = p->dim_ld / 32, tv = p->vdim_ld / 64;
    hipLaunchKernelGGL(linear_states_kernel, dim3(td * tv * p->n_head, p->n_runs), dim3(256), 0, st, *p, td, tv);
    const int rc = pi::check_launch("pi_k_linear_chunks states");
    if (rc != PI_OK) return rc;
    return p->vdim_ld <= 64 ? launch_out<1>(p, st) : p->vdim_ld <= 128 ? launch_out<2>(p, st) : p->vdim_ld <= 192 ? launch_out<3>(p, st) : launch_out<4>(p, st);
}

int pi_k_gate_norm(int type, const pi_gate_norm * p, pi_stream_t stream) {
    if (!p || !gate_norm_ok(*p)) return pi::fail(PI_E_ARG, "pi_k_gate_norm: bad arguments");
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(gate_norm_kernel<bf16>, dim3(p->T), dim3(256), 0, (hipStream_t)stream, *p);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(gate_norm_kernel<float>, dim3(p->T), dim3(256), 0, (hipStream_t)stream, *p);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_gate_norm: type");
    return pi::check_launch("pi_k_gate_norm");
}

}  // extern "C"
