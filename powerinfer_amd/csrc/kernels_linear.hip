// Linear attention over a fp32 state per sequence: token by token for steps (any storage type), and in chunks on the matrix cores for long
// prompt portions.  What becomes of the state S from token to token (pi_linear::decay_kind): a constant factor per head, a factor per
// key channel and token, or factors per head and token from exponential gates.  With A_i the product of a chunk's factors up to token i
// (d^(i+1), a diagonal matrix, or exp of the sum of log forget gates) and S the state before the chunk, token i of the chunk has
//   o_i = (A_i S)^T q_i + sum over j <= i of (q_i . A_i / A_j k_j) v_j,     S' = A_n S + sum over j of A_n / A_j k_j v_j^T.
// Whatever is fp32 (states, decayed keys, queries and scores) enters the matrix cores as the sum of two bf16, which keeps 16 bits of mantissa.
#include "mixers.hpp"

namespace {

constexpr int kConst = PI_DECAY_CONST, kKeyed = PI_DECAY_KEYED, kGated = PI_DECAY_GATED;
constexpr int kLinCols = 32;             // value columns of a workgroup of the token-by-token kernel
constexpr int kLinBlock = 16;            // tokens staged at a time
constexpr int kLinMax = 256;
constexpr int kLinMaxRank = 512;         // of the projection that key decays come from
constexpr float kLog2E = 1.44269504088896340736f;

__device__ __forceinline__ float log_sigmoid_f32(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float lin_exp2(float v) { return __builtin_amdgcn_exp2f(v); }
// log2 of the decay of a key channel; the quick form's error is of the order of fp32's last place of one, not of the result
__device__ __forceinline__ float keyed_log2(float u, float tau) { return log_sigmoid_f32(u) / tau * kLog2E; }
__device__ __forceinline__ float keyed_log2_quick(float u, float per_tau) {
    const float a = u * kLog2E;
    return (fminf(a, 0.0f) - __builtin_amdgcn_logf(1.0f + lin_exp2(-fabsf(a)))) * per_tau;
}
__device__ __forceinline__ float soft_cap(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_input_gate(const pi_linear & p, const float * z, int h) { return soft_cap(z[p.off_i + h] + p.i_b[h], p.cap); }
__device__ __forceinline__ float log_forget_gate(const pi_linear & p, const float * z, int h) { return log_sigmoid_f32(soft_cap(z[p.off_f + h] + p.f_b[h], p.cap)); }
// the value of a projection as the recurrence takes it; walked token by token it is rounded to the activations' storage only behind an activation
__device__ __forceinline__ float lin_value(const pi_linear & p, float z, bool query) { return p.plain ? (query ? z * p.q_scale : z) : silu_f32(z); }
template <typename ST> __device__ __forceinline__ float lin_operand(const pi_linear & p, float z, bool query) {
    const float v = lin_value(p, z, query);
    return p.plain ? v : from_st(to_st<ST>(v));
}
__device__ __forceinline__ float lin_den(float nq, float m) { return fmaxf(fabsf(nq), expf(-m)) + 1e-6f; }
// places of the sum of keys and of the copies of the running maximum inside a slot
__host__ __device__ inline int lin_copies(int vdim) { return (vdim + kLinCols - 1) / kLinCols; }
__host__ __device__ inline size_t lin_slot_floats(int kind, int n_head, int dim, int vdim) {
    return (size_t)n_head * dim * vdim + (kind == kGated ? (size_t)n_head * (dim + lin_copies(vdim)) : 0);
}
__device__ __forceinline__ float * lin_slot(const pi_linear & p, int slot) { return p.state + (size_t)slot * (p.slot_ld ? p.slot_ld : lin_slot_floats(p.decay_kind, p.n_head, p.dim, p.vdim)); }
__device__ __forceinline__ float * lin_keys(const pi_linear & p, float * slot, int h) { return slot + (size_t)p.n_head * p.dim * p.vdim + (size_t)h * p.dim; }
__device__ __forceinline__ float * lin_tops(const pi_linear & p, float * slot, int h) {
    return slot + (size_t)p.n_head * p.dim * (p.vdim + 1) + (size_t)h * lin_copies(p.vdim);
}

// A thread keeps J consecutive rows of one column of the state in registers; 8 groups of rows x 32 columns.  Exponential gates: every
// workgroup follows the running maximum by itself and keeps a copy of it, the first slice of a head the sum of keys.
__host__ __device__ constexpr int lin_step_floats(int D, int mode) {
    return 2 * kLinBlock * D + kLinBlock * kLinCols + 4 * kLinBlock * kLinCols + (mode == kKeyed ? kLinBlock * D : mode == kGated ? 7 * kLinBlock : 0);
}
template <typename ST, int J, int MODE>
__global__ __launch_bounds__(256) void linear_step_kernel(pi_linear p, pi_ffn_front f, pi_gqa_prep beside, int n_state, int n_front, int slices, int per, int per_beside) {
    constexpr int D = 8 * J;
    extern __shared__ __align__(16) float sm[];
    if ((int)blockIdx.x >= n_state) {
        const int b = blockIdx.x - n_state;
        if (b < n_front) front_block<ST>(f, p.z, p.ldz, b / per, b % per, sm);
        else if (MODE == kConst) return;                         // (asks for nothing beside it: checked by the launcher)
        else if (beside.rot_pairs) gqa_prep_block<ST, true>(beside, (b - n_front) / per_beside, (b - n_front) % per_beside);
        else gqa_prep_block<ST, false>(beside, (b - n_front) / per_beside, (b - n_front) % per_beside);
        return;
    }
    float * qs = sm, * ks = qs + kLinBlock * D, * vs = ks + kLinBlock * D, * part = vs + kLinBlock * kLinCols;      // [16][D], [16][D], [16][32], [4][16][32]
    float * more = part + 4 * kLinBlock * kLinCols;          // keyed: decays [16][D]; gated: log gates [2][16], tops [16], parts of n . q [4][16]
    float * fl = more, * il = fl + kLinBlock, * tops = il + kLinBlock, * partn = tops + kLinBlock;
    const int slice = blockIdx.x % slices, h = (int)blockIdx.x / slices % p.n_head, tid = threadIdx.x;
    const int4 run = reinterpret_cast<const int4 *>(p.runs)[(int)blockIdx.x / slices / p.n_head];
    const int c = tid % kLinCols, rg = tid / kLinCols, col = slice * kLinCols + c, wave = tid >> 6;
    const float d = MODE == kConst ? p.decay[h] : 0.0f;
    float * slot = lin_slot(p, run.z), * S = slot + (size_t)h * p.dim * p.vdim;
    float s[J], nk[MODE == kGated ? J : 1], top = 0.0f;
    const bool sums = MODE == kGated && slice == 0;
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int r = min(rg * J + j, p.dim - 1);              // (no guard around a load)
        s[j] = S[(size_t)r * p.vdim + min(col, p.vdim - 1)];
        if constexpr (MODE == kGated) nk[j] = lin_keys(p, slot, h)[r];
    }
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int r = rg * J + j;
        if (run.w || r >= p.dim || col >= p.vdim) s[j] = 0.0f;
        if constexpr (MODE == kGated) if (run.w || r >= p.dim || !sums) nk[j] = 0.0f;
    }
    if constexpr (MODE == kGated) top = run.w ? 0.0f : lin_tops(p, slot, h)[slice];
    for (int t0 = 0; t0 < run.y; t0 += kLinBlock) {
        const int n = min(kLinBlock, run.y - t0);
        if (t0) __syncthreads();
        for (int e = tid; e < n * D; e += 256) {
            const int t = e / D, r = e % D;
            const float * zt = p.z + (size_t)(run.x + t0 + t) * p.ldz, * z = zt + h * p.dim + r;
            qs[e] = r < p.dim ? lin_operand<ST>(p, z[p.off_q], true) : 0.0f;
            ks[e] = r < p.dim ? lin_operand<ST>(p, z[p.off_k], false) : 0.0f;
            if constexpr (MODE == kKeyed) {
                float a = 0.0f;
                if (r < p.dim) {
                    const uint16_t * w = (const uint16_t *)p.a2 + (size_t)(h * p.dim + r) * p.rank_ld;
                    const float * u = zt + p.off_a;
                    float b = p.a2_b[h * p.dim + r];
                    for (int k = 0; k < p.rank_ld; k += 8) {
                        const Frag<float> wf = frag_weights<float>(w + k);
#pragma unroll
                        for (int i = 0; i < 8; ++i) b = fmaf(wf.v[i], u[k + i], b);        // (behind the rank: zeros of a2)
                    }
                    a = exp2f(keyed_log2(b, p.tau));
                }
                more[e] = a;
            }
        }
        for (int e = tid; e < n * kLinCols; e += 256) {
            const int t = e / kLinCols, v = slice * kLinCols + e % kLinCols;
            vs[e] = v < p.vdim ? lin_operand<ST>(p, p.z[(size_t)(run.x + t0 + t) * p.ldz + p.off_v + h * p.vdim + v], false) : 0.0f;
        }
        if (MODE == kGated && tid < n) {
            const float * z = p.z + (size_t)(run.x + t0 + tid) * p.ldz;
            fl[tid] = log_forget_gate(p, z, h);
            il[tid] = log_input_gate(p, z, h);
        }
        __syncthreads();
        for (int t = 0; t < n; ++t) {
            float v = vs[t * kLinCols + c], keep = d, add = 1.0f;
            if constexpr (MODE == kGated) {
                const float next = fmaxf(fl[t] + top, il[t]);
                keep = expf(fl[t] + top - next);
                add = expf(il[t] - next);
                top = next;
                v *= add;
            }
            float a = 0.0f, an = 0.0f;
#pragma unroll
            for (int j = 0; j < J; j += 4) {
                const float4 k = *reinterpret_cast<const float4 *>(ks + t * D + rg * J + j), q = *reinterpret_cast<const float4 *>(qs + t * D + rg * J + j);
                float4 dk = make_float4(keep, keep, keep, keep);
                if constexpr (MODE == kKeyed) dk = *reinterpret_cast<const float4 *>(more + t * D + rg * J + j);
                s[j] = fmaf(k.x, v, dk.x * s[j]); a = fmaf(q.x, s[j], a);
                s[j + 1] = fmaf(k.y, v, dk.y * s[j + 1]); a = fmaf(q.y, s[j + 1], a);
                s[j + 2] = fmaf(k.z, v, dk.z * s[j + 2]); a = fmaf(q.z, s[j + 2], a);
                s[j + 3] = fmaf(k.w, v, dk.w * s[j + 3]); a = fmaf(q.w, s[j + 3], a);
                if constexpr (MODE == kGated) {
                    if (sums) {
                        nk[j] = fmaf(k.x, add, keep * nk[j]); an = fmaf(q.x, nk[j], an);
                        nk[j + 1] = fmaf(k.y, add, keep * nk[j + 1]); an = fmaf(q.y, nk[j + 1], an);
                        nk[j + 2] = fmaf(k.z, add, keep * nk[j + 2]); an = fmaf(q.z, nk[j + 2], an);
                        nk[j + 3] = fmaf(k.w, add, keep * nk[j + 3]); an = fmaf(q.w, nk[j + 3], an);
                    }
                }
            }
            a += __shfl_xor(a, 32, PI_WAVE);
            if ((tid & 63) < kLinCols) part[(wave * kLinBlock + t) * kLinCols + c] = a;
            if constexpr (MODE == kGated) {
                an += __shfl_xor(an, 32, PI_WAVE);
                if ((tid & 63) == 0) partn[wave * kLinBlock + t] = an;
                if (tid == 0) tops[t] = top;
            }
        }
        __syncthreads();
        for (int e = tid; e < n * kLinCols; e += 256) {
            const int t = e / kLinCols, v = slice * kLinCols + e % kLinCols;
            if (v < p.vdim) p.o[(size_t)(run.x + t0 + t) * p.n_head * p.vdim + h * p.vdim + v] =
                part[e] + part[kLinBlock * kLinCols + e] + part[2 * kLinBlock * kLinCols + e] + part[3 * kLinBlock * kLinCols + e];
        }
        if (sums && tid < n)
            p.den[(size_t)(run.x + t0 + tid) * p.n_head + h] =
                lin_den(partn[tid] + partn[kLinBlock + tid] + partn[2 * kLinBlock + tid] + partn[3 * kLinBlock + tid], tops[tid]);
    }
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int r = rg * J + j;
        if (r < p.dim && col < p.vdim) S[(size_t)r * p.vdim + col] = s[j];
        if constexpr (MODE == kGated) if (sums && c == 0 && r < p.dim) lin_keys(p, slot, h)[r] = nk[j];
    }
    if (MODE == kGated && tid == 0) lin_tops(p, slot, h)[slice] = top;
}

// the projections as bf16 operands, rows padded with zeros: a block covers 4096 values of a token's [q | k | v], a thread four of every 1024
constexpr int kLinPrep = 4096;
__global__ __launch_bounds__(256) void linear_prep_kernel(pi_linear p, pi_ffn_front f, int n_val, int per) {
    extern __shared__ __align__(16) float sm[];
    const int t = blockIdx.x / per, b = blockIdx.x % per;
    if (b >= n_val) { front_block<bf16>(f, p.z, p.ldz, t, b - n_val, sm); return; }
    const int nq = p.n_head * p.dim_ld, all = 2 * nq + p.n_head * p.vdim_ld;
    constexpr int Q = kLinPrep / 1024;
    float v[Q][4];
    bf16 * o[Q];
    bool query[Q];
#pragma unroll
    for (int i = 0; i < Q; ++i) {
        const int e = min(b * kLinPrep + i * 1024 + (int)threadIdx.x * 4, all - 4);      // past the end: the last four again, the same values
        const int what = e < nq ? 0 : e < 2 * nq ? 1 : 2, k = e - what * nq, ld = what == 2 ? p.vdim_ld : p.dim_ld, dim = what == 2 ? p.vdim : p.dim, h = k / ld, r = k % ld;
        const float * z = p.z + (size_t)t * p.ldz + (what == 0 ? p.off_q : what == 1 ? p.off_k : p.off_v) + h * dim + r;
        query[i] = what == 0;
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
        for (int j = 0; j < 4; ++j) v[i][j] = lin_value(p, v[i][j], query[i]);            // (zeros stay zeros)
        store4(o[i], v[i], true, 4);
    }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// decays of long runs, per chunk
// ---------------------------------------------------------------------------------------------------------------------------------
constexpr int kLinC = 64;                // tokens of a chunk
// what pi_linear::gates holds.  Keyed: [T][n_head][dim_ld] sums of log2 decays from the chunk's start on (fp32).  Gated: with F the sum of log
// forget gates from the chunk's start on and i the log input gate, per (token, head) {F, i - F, largest i - F since the chunk's start, -},
// and behind them the running maximum m ahead of every chunk [n_chunks][n_head].  With m0 ahead of the chunk the maximum at a token is
// m = F + max(m0, largest i - F), so that only the few numbers per chunk depend on what came before it.
__device__ __forceinline__ const float4 * lin_gates(const pi_linear & p) { return (const float4 *)p.gates; }
__device__ __forceinline__ float * lin_chunk_tops(const pi_linear & p) { return p.gates + (size_t)4 * p.T * p.n_head; }
// sums of keys ahead of every chunk, behind the states: [chunk][head][hi, lo][dim_ld]
__device__ __forceinline__ bf16 * lin_chunk_keys(const pi_linear & p) { return (bf16 *)p.states + (size_t)p.n_chunks * p.n_head * 2 * p.vdim_ld * p.dim_ld; }

// log2 of the smallest decay of one token: what it leaves is far below fp32's last place, and the sums stay small enough to tell the
// decays of the tokens behind it apart
constexpr float kLinForgotten = -100.0f;
// a workgroup per (chunk, 256 key channels of all heads): the second factor of the low-rank projection, 16 tokens at a time
__global__ __launch_bounds__(256) void linear_decays_kernel(pi_linear p, int n_blocks) {
    extern __shared__ __align__(16) float us[];              // [64][rank_ld]
    const int ck = blockIdx.x / n_blocks, ch = blockIdx.x % n_blocks * 256 + (int)threadIdx.x, tok0 = p.chunks[3 * ck], n = p.chunks[3 * ck + 1];
    for (int e = threadIdx.x; e < kLinC * p.rank_ld; e += 256) {
        const int t = e / p.rank_ld, k = e % p.rank_ld;
        us[e] = t < n && k < p.rank ? p.z[(size_t)(tok0 + t) * p.ldz + p.off_a + k] : 0.0f;
    }
    __syncthreads();
    const int all = p.n_head * p.dim_ld, h = ch / p.dim_ld, r = ch % p.dim_ld;
    if (ch >= all) return;
    const bool real = r < p.dim;
    const int row = h * p.dim + (real ? r : 0);
    const uint16_t * w = (const uint16_t *)p.a2 + (size_t)row * p.rank_ld;
    const float bias = p.a2_b[row], per_tau = 1.0f / p.tau;
    float * out = p.gates + (size_t)tok0 * all + ch;
    float sum = 0.0f;
    for (int t0 = 0; t0 < n; t0 += 16) {
        float acc[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) acc[t] = bias;
        for (int k = 0; k < p.rank_ld; k += 8) {
            const Frag<float> wf = frag_weights<float>(w + k);
#pragma unroll
            for (int t = 0; t < 16; ++t) {
                const float4 * u = reinterpret_cast<const float4 *>(us + (t0 + t) * p.rank_ld + k);
                const float4 a = u[0], b = u[1];
                acc[t] = fmaf(wf.v[0], a.x, acc[t]); acc[t] = fmaf(wf.v[1], a.y, acc[t]); acc[t] = fmaf(wf.v[2], a.z, acc[t]); acc[t] = fmaf(wf.v[3], a.w, acc[t]);
                acc[t] = fmaf(wf.v[4], b.x, acc[t]); acc[t] = fmaf(wf.v[5], b.y, acc[t]); acc[t] = fmaf(wf.v[6], b.z, acc[t]); acc[t] = fmaf(wf.v[7], b.w, acc[t]);
            }
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            sum += fmaxf(keyed_log2_quick(acc[t], per_tau), kLinForgotten);
            if (t0 + t < n) out[(size_t)(t0 + t) * all] = real ? sum : 0.0f;
        }
    }
}

// a wave per (chunk, head), a lane per token; the workgroups behind them hand the slots' maxima to their runs' first chunks
__global__ __launch_bounds__(256) void linear_gates_kernel(pi_linear p, int h4) {
    const int lane = threadIdx.x & 63;
    if ((int)blockIdx.x >= p.n_chunks * h4) {
        const int ri = blockIdx.x - p.n_chunks * h4;
        const int4 run = reinterpret_cast<const int4 *>(p.runs)[ri];
        for (int h = threadIdx.x; h < p.n_head; h += 256) lin_chunk_tops(p)[(size_t)p.first_chunk[ri] * p.n_head + h] = run.w ? 0.0f : lin_tops(p, lin_slot(p, run.z), h)[0];
        return;
    }
    const int ck = blockIdx.x / h4, h = blockIdx.x % h4 * 4 + (int)(threadIdx.x >> 6), tok0 = p.chunks[3 * ck], n = p.chunks[3 * ck + 1];
    if (h >= p.n_head) return;
    const float * z = p.z + (size_t)(tok0 + min(lane, n - 1)) * p.ldz;
    const float i = log_input_gate(p, z, h);
    float F = log_forget_gate(p, z, h);
#pragma unroll
    for (int o = 1; o < PI_WAVE; o <<= 1) { const float v = __shfl_up(F, o, PI_WAVE); if (lane >= o) F += v; }
    float best = i - F;
#pragma unroll
    for (int o = 1; o < PI_WAVE; o <<= 1) { const float v = __shfl_up(best, o, PI_WAVE); if (lane >= o) best = fmaxf(best, v); }
    if (lane < n) reinterpret_cast<float4 *>(p.gates)[(size_t)(tok0 + lane) * p.n_head + h] = make_float4(F, i - F, best, 0.0f);
}

// ---------------------------------------------------------------------------------------------------------------------------------
// chunks
// ---------------------------------------------------------------------------------------------------------------------------------
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
__device__ __forceinline__ pi_u32x4 lin_ones() { return pi_u32x4{0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u}; }
// eight values times factors, as the sum of two operands
__device__ __forceinline__ void lin_split8(const pi_u32x4 & x, const float (&f)[8], pi_u32x4 & hi, pi_u32x4 & lo) {
    const bf16 * b = reinterpret_cast<const bf16 *>(&x);
    bf16 h[8], l[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) split_bf16((float)b[j] * f[j], h[j], l[j]);
    hi = __builtin_bit_cast(pi_u32x4, h);
    lo = __builtin_bit_cast(pi_u32x4, l);
}

// states: per (chunk, head) the state before the chunk, transposed, as two bf16 matrices [vdim_ld][dim_ld].  A workgroup owns 32 rows x 64
// value columns of one head's state and walks the run's chunks; the next chunk's keys and values are requested while one is multiplied.
template <int MODE>
__global__ __launch_bounds__(256) void linear_states_kernel(pi_linear p, int tiles_d, int tiles_v) {
    constexpr int KROW = 32 * 2 + 16, VROW = 64 * 2 + 16;
    __shared__ __align__(16) unsigned char kh[kLinC * KROW], kl[kLinC * KROW], vs[kLinC * VROW];
    const int tile = blockIdx.x % (tiles_d * tiles_v), h = blockIdx.x / (tiles_d * tiles_v), ri = blockIdx.y;
    const int d0 = tile / tiles_v * 32, v0 = tile % tiles_v * 64;
    const int4 run = reinterpret_cast<const int4 *>(p.runs)[ri];
    const int chunk0 = p.first_chunk[ri], n_chunk = (run.y + kLinC - 1) / kLinC;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    const float * pw = MODE == kConst ? p.powers + (size_t)h * (kLinC + 1) : nullptr;
    float * slot = lin_slot(p, run.z), * S = slot + (size_t)h * p.dim * p.vdim;
    const int vcol = v0 + wave * 16 + i;
    const bool sums = MODE == kGated && v0 == 0 && wave == 0;      // this wave keeps the sums of keys of its rows as well (all of its columns alike)
    const bool keeps = MODE == kGated && v0 == 0 && d0 == 0 && tid == 0;      // this thread reports the running maximum
    pi_f4 acc[2], accn[2];
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = d0 + m * 16 + 4 * g + r;
            acc[m][r] = !run.w && row < p.dim && vcol < p.vdim ? S[(size_t)row * p.vdim + vcol] : 0.0f;
            accn[m][r] = sums && !run.w && row < p.dim ? lin_keys(p, slot, h)[row] : 0.0f;
        }
    const int kt = tid / 4, kc = (tid % 4) * 8, vt = tid / 8, vc = (tid % 8) * 8;
    const size_t ldk = (size_t)p.n_head * p.dim_ld, ldv = (size_t)p.n_head * p.vdim_ld;
    const uint16_t * kp = (const uint16_t *)p.k + h * p.dim_ld + d0 + kc, * vp = (const uint16_t *)p.v + h * p.vdim_ld + v0 + vc;
    const float * gp = p.gates + h * p.dim_ld + d0;              // keyed
    const int last = run.x + run.y - 1;
    pi_u32x4 rk, rv[2];
    float4 gk[2], ge[2], gr[2];                                  // keyed: sums of the key's channels, of the chunk's last token, and of the rows of acc
    float4 tk, te;                                               // gated: the key's and the last token's numbers
    float top = MODE == kGated ? lin_chunk_tops(p)[(size_t)chunk0 * p.n_head + h] : 0.0f;      // the running maximum ahead of the chunk
    auto fetch = [&](int ck) {
        const int t0 = run.x + ck * kLinC, end = min(t0 + kLinC - 1, last);
        rk = pi_ld16(kp + (size_t)min(t0 + kt, last) * ldk);
        rv[0] = pi_ld16(vp + (size_t)min(t0 + vt, last) * ldv);
        rv[1] = pi_ld16(vp + (size_t)min(t0 + 32 + vt, last) * ldv);
        if constexpr (MODE == kKeyed) {
            const float4 * a = reinterpret_cast<const float4 *>(gp + (size_t)min(t0 + kt, last) * ldk + kc), * e = reinterpret_cast<const float4 *>(gp + (size_t)end * ldk + kc);
            gk[0] = a[0]; gk[1] = a[1]; ge[0] = e[0]; ge[1] = e[1];
#pragma unroll
            for (int m = 0; m < 2; ++m) gr[m] = *reinterpret_cast<const float4 *>(gp + (size_t)end * ldk + m * 16 + 4 * g);
        }
        if constexpr (MODE == kGated) {
            tk = lin_gates(p)[(size_t)min(t0 + kt, last) * p.n_head + h];
            te = lin_gates(p)[(size_t)end * p.n_head + h];
        }
    };
    fetch(0);
    for (int ck = 0; ck < n_chunk; ++ck) {
        const int n = min(kLinC, run.y - ck * kLinC);
        float dn[2][4];                                          // what the state's rows are multiplied by
        __syncthreads();
        {
            float w[8];
            if constexpr (MODE == kKeyed) {
                const float a[8] = {gk[0].x, gk[0].y, gk[0].z, gk[0].w, gk[1].x, gk[1].y, gk[1].z, gk[1].w}, e[8] = {ge[0].x, ge[0].y, ge[0].z, ge[0].w, ge[1].x, ge[1].y, ge[1].z, ge[1].w};
#pragma unroll
                for (int j = 0; j < 8; ++j) w[j] = kt < n ? lin_exp2(e[j] - a[j]) : 0.0f;
#pragma unroll
                for (int m = 0; m < 2; ++m) { dn[m][0] = lin_exp2(gr[m].x); dn[m][1] = lin_exp2(gr[m].y); dn[m][2] = lin_exp2(gr[m].z); dn[m][3] = lin_exp2(gr[m].w); }
            } else {
                const float most = MODE == kGated ? fmaxf(top, te.z) : 0.0f;
                const float one = kt < n ? (MODE == kGated ? expf(tk.y - most) : pw[max(n - 1 - kt, 0)]) : 0.0f, all = MODE == kGated ? expf(top - most) : pw[n];
                if constexpr (MODE == kGated) {
                    if (keeps && ck) lin_chunk_tops(p)[(size_t)(chunk0 + ck) * p.n_head + h] = top;
                    top = te.x + most;
                }
#pragma unroll
                for (int j = 0; j < 8; ++j) { w[j] = one; dn[j >> 2][j & 3] = all; }
            }
            pi_u32x4 hi, lo;
            lin_split8(rk, w, hi, lo);
            *reinterpret_cast<pi_u32x4 *>(kh + kt * KROW + kc * 2) = hi;
            *reinterpret_cast<pi_u32x4 *>(kl + kt * KROW + kc * 2) = lo;
            *reinterpret_cast<pi_u32x4 *>(vs + vt * VROW + vc * 2) = rv[0];
            *reinterpret_cast<pi_u32x4 *>(vs + (32 + vt) * VROW + vc * 2) = rv[1];
        }
        __syncthreads();
        fetch(ck + 1);                                           // past the last chunk: its last token again, not used
        bf16 * out = (bf16 *)p.states + ((size_t)(chunk0 + ck) * p.n_head + h) * 2 * p.vdim_ld * p.dim_ld + (size_t)vcol * p.dim_ld + d0 + 4 * g;
        bf16 * outn = lin_chunk_keys(p) + ((size_t)(chunk0 + ck) * p.n_head + h) * 2 * p.dim_ld + d0 + 4 * g;
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            bf16 hi[4], lo[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) { split_bf16(acc[m][r], hi[r], lo[r]); acc[m][r] *= dn[m][r]; }
            *reinterpret_cast<pi_u32x2 *>(out + m * 16) = __builtin_bit_cast(pi_u32x2, hi);
            *reinterpret_cast<pi_u32x2 *>(out + (size_t)p.vdim_ld * p.dim_ld + m * 16) = __builtin_bit_cast(pi_u32x2, lo);
            if (sums) {
#pragma unroll
                for (int r = 0; r < 4; ++r) { split_bf16(accn[m][r], hi[r], lo[r]); accn[m][r] *= dn[m][r]; }
                if (i == 0) {
                    *reinterpret_cast<pi_u32x2 *>(outn + m * 16) = __builtin_bit_cast(pi_u32x2, hi);
                    *reinterpret_cast<pi_u32x2 *>(outn + p.dim_ld + m * 16) = __builtin_bit_cast(pi_u32x2, lo);
                }
            }
        }
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const pi_u32x4 b = lin_frag(vs + s * 32 * VROW, VROW, wave * 16);
#pragma unroll
            for (int m = 0; m < 2; ++m) {
                const pi_u32x4 hi = lin_frag(kh + s * 32 * KROW, KROW, m * 16), lo = lin_frag(kl + s * 32 * KROW, KROW, m * 16);
                acc[m] = mfma_bf16(hi, b, acc[m]);
                acc[m] = mfma_bf16(lo, b, acc[m]);
                if (sums) { accn[m] = mfma_bf16(hi, lin_ones(), accn[m]); accn[m] = mfma_bf16(lo, lin_ones(), accn[m]); }
            }
        }
    }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = d0 + m * 16 + 4 * g + r;
            if (row < p.dim && vcol < p.vdim) S[(size_t)row * p.vdim + vcol] = acc[m][r];
            if (sums && i == 0 && row < p.dim) lin_keys(p, slot, h)[row] = accn[m][r];
        }
    if (keeps) for (int k = 0; k < lin_copies(p.vdim); ++k) lin_tops(p, slot, h)[k] = top;
}

// ---- outputs of one chunk of one head.  Wave w forms the decayed scores of tokens 16 w .. (as columns, keys x tokens) and leaves them in LDS in
// operand order; then every wave owns a quarter of the value columns for all tokens of the chunk -----------------------------------------
template <int VPW> using LinAcc = pi_f4[VPW][4];        // 16-column value tiles per wave x 16-token tiles

// a lane's column of the wave's decayed scores (keys kt * 16 + 4 g + r) as two operands of 32 keys, each the sum of two
__device__ __forceinline__ void lin_store_scores(pi_u32x4 * pp, const float (&s)[4][4], int wave, int lane) {
#pragma unroll
    for (int st = 0; st < 2; ++st) {
        bf16 hi[8], lo[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) split_bf16(s[2 * st + (j >> 2)][j & 3], hi[j], lo[j]);
        pp[((wave * 2 + st) * 2) * 64 + lane] = __builtin_bit_cast(pi_u32x4, hi);
        pp[((wave * 2 + st) * 2 + 1) * 64 + lane] = __builtin_bit_cast(pi_u32x4, lo);
    }
}
// + S^T q for the 64 queries in LDS (ql: their second parts, optional)
template <int VPW, bool LO>
__device__ __forceinline__ void lin_add_state(LinAcc<VPW> & acc, const pi_linear & p, int ck, int h, const unsigned char * qs, const unsigned char * ql, int qrow) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, g = lane >> 4, n_vt = p.vdim_ld / 16;
    const size_t half = (size_t)p.vdim_ld * p.dim_ld;
    const bf16 * S = (const bf16 *)p.states + ((size_t)ck * p.n_head + h) * 2 * half;
    for (int k = 0; k < p.dim_ld / 32; ++k) {
        pi_u32x4 q[4], l[4];
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            q[c] = *reinterpret_cast<const pi_u32x4 *>(qs + (c * 16 + i) * qrow + k * 64 + g * 16);
            if (LO) l[c] = *reinterpret_cast<const pi_u32x4 *>(ql + (c * 16 + i) * qrow + k * 64 + g * 16);
        }
#pragma unroll
        for (int v = 0; v < VPW; ++v) {
            const int vt = min(wave + 4 * v, n_vt - 1);
            const bf16 * a = S + (size_t)(vt * 16 + i) * p.dim_ld + k * 32 + g * 8;
            const pi_u32x4 hi = pi_ld16(a), lo = pi_ld16(a + half);
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                acc[v][c] = mfma_bf16(hi, q[c], acc[v][c]);
                acc[v][c] = mfma_bf16(lo, q[c], acc[v][c]);
                if (LO) acc[v][c] = mfma_bf16(hi, l[c], acc[v][c]);
            }
        }
    }
}
// + values^T x scores
template <int VPW>
__device__ __forceinline__ void lin_add_scores(LinAcc<VPW> & acc, const pi_linear & p, const unsigned char * vs, int vrow, const pi_u32x4 * pp) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, g = lane >> 4, n_vt = p.vdim_ld / 16;
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
}
template <int VPW> __device__ __forceinline__ void lin_zero(LinAcc<VPW> & acc) {
#pragma unroll
    for (int v = 0; v < VPW; ++v)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[v][c] = pi_f4{0, 0, 0, 0};
}
template <int VPW> __device__ __forceinline__ void lin_store(const LinAcc<VPW> & acc, const pi_linear & p, int tok0, int n, int h) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, g = lane >> 4, n_vt = p.vdim_ld / 16;
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

// decays that are numbers per head: the products of queries and keys are decayed
template <int VPW, int MODE>
__global__ __launch_bounds__(256) void linear_out_kernel(pi_linear p) {
    extern __shared__ __align__(16) unsigned char smem[];
    const int qrow = p.dim_ld * 2 + 16, vrow = p.vdim_ld * 2 + 16;
    unsigned char * qs = smem, * ks = qs + kLinC * qrow, * vs = ks + kLinC * qrow;
    pi_u32x4 * pp = reinterpret_cast<pi_u32x4 *>(vs + kLinC * vrow);          // [4 column tiles][2 steps][hi, lo][64]
    float * pw = reinterpret_cast<float *>(pp + 4 * 2 * 2 * 64);              // constant: powers [kLinC + 1]; gated: three numbers a token
    float * fa = pw, * fb = pw + kLinC, * ft = pw + 2 * kLinC;
    const int h = blockIdx.x % p.n_head, ck = blockIdx.x / p.n_head;
    const int tok0 = p.chunks[3 * ck], n = p.chunks[3 * ck + 1], fresh = p.chunks[3 * ck + 2];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    float top = 0.0f;
    if (MODE == kGated) {
        top = lin_chunk_tops(p)[(size_t)ck * p.n_head + h];
        if (tid < kLinC) {
            const float4 v = lin_gates(p)[(size_t)(tok0 + min(tid, n - 1)) * p.n_head + h];
            const float most = fmaxf(top, v.z);
            fa[tid] = -most; fb[tid] = v.y; ft[tid] = v.x + most;
        }
    } else for (int e = tid; e <= kLinC; e += 256) pw[e] = p.powers[(size_t)h * (kLinC + 1) + e];
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
        float w[4][4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int tj = kt * 16 + 4 * g + r;
                w[kt][r] = tj <= ti ? s[kt][r] * (MODE == kGated ? expf(fa[ti] + fb[tj]) : pw[max(ti - tj, 0)]) : 0.0f;
            }
        lin_store_scores(pp, w, wave, lane);
    }
    __syncthreads();
    LinAcc<VPW> acc;
    lin_zero<VPW>(acc);
    pi_f4 den[4];                                                // gated: n . q (every row of the tile alike), by the first wave
#pragma unroll
    for (int c = 0; c < 4; ++c) den[c] = pi_f4{0, 0, 0, 0};
    if (!fresh) {
        lin_add_state<VPW, false>(acc, p, ck, h, qs, nullptr, qrow);
        if (MODE == kGated && wave == 0) {
            const bf16 * nkey = lin_chunk_keys(p) + ((size_t)ck * p.n_head + h) * 2 * p.dim_ld + g * 8;
            for (int k = 0; k < nk; ++k) {
                const pi_u32x4 hi = pi_ld16(nkey + k * 32), lo = pi_ld16(nkey + p.dim_ld + k * 32);
#pragma unroll
                for (int c = 0; c < 4; ++c) {
                    const pi_u32x4 q = *reinterpret_cast<const pi_u32x4 *>(qs + (c * 16 + i) * qrow + k * 64 + g * 16);
                    den[c] = mfma_bf16(hi, q, den[c]);
                    den[c] = mfma_bf16(lo, q, den[c]);
                }
            }
        }
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const float w = MODE == kGated ? expf(fa[c * 16 + i] + top) : pw[c * 16 + i + 1];
#pragma unroll
            for (int v = 0; v < VPW; ++v) acc[v][c] *= w;
            den[c] *= w;
        }
    }
    lin_add_scores<VPW>(acc, p, vs, vrow, pp);
    lin_store<VPW>(acc, p, tok0, n, h);
    if (MODE == kGated && wave == 0) {
#pragma unroll
        for (int st = 0; st < 2; ++st)
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                if (2 * st > c) continue;
                den[c] = mfma_bf16(lin_ones(), pp[((c * 2 + st) * 2) * 64 + lane], den[c]);
                den[c] = mfma_bf16(lin_ones(), pp[((c * 2 + st) * 2 + 1) * 64 + lane], den[c]);
            }
#pragma unroll
        for (int c = 0; c < 4; ++c)
            if (g == 0 && c * 16 + i < n) p.den[(size_t)(tok0 + c * 16 + i) * p.n_head + h] = lin_den(den[c][0], ft[c * 16 + i]);
    }
}

// Decays per key channel: queries and keys are decayed ahead of their product.  For the scores wave w takes the state of affairs before its own 16
// tokens as the point both are decayed to: later queries have decayed since (a factor below one), earlier keys up to it (below one as well),
// and the keys of its own 16 tokens are the only ones that are scaled up.  If that would leave fp32's range the wave forms the scores
// of its own tokens pair by pair.
constexpr float kLinSpan = 80.0f;          // log2 of the largest factor
__host__ __device__ inline size_t lin_keyed_lds(int dim_ld, int vdim_ld) {
    const size_t q = (size_t)kLinC * (dim_ld * 2 + 16), g = (size_t)kLinC * (dim_ld * 4 + 16), v = (size_t)kLinC * (vdim_ld * 2 + 16) + 4 * 2 * 2 * 64 * 16;
    return 2 * q + (g > v ? g : v);
}
template <int VPW>
__global__ __launch_bounds__(256) void linear_out_keyed_kernel(pi_linear p) {
    extern __shared__ __align__(16) unsigned char smem[];
    const int qrow = p.dim_ld * 2 + 16, grow = p.dim_ld * 4 + 16, vrow = p.vdim_ld * 2 + 16;
    unsigned char * qs = smem, * ks = qs + kLinC * qrow, * gs = ks + kLinC * qrow, * vs = gs;      // (values and scores take the place of the sums, queries' second parts that of the keys)
    pi_u32x4 * pp = reinterpret_cast<pi_u32x4 *>(vs + kLinC * vrow);
    const int h = blockIdx.x % p.n_head, ck = blockIdx.x / p.n_head;
    const int tok0 = p.chunks[3 * ck], n = p.chunks[3 * ck + 1], fresh = p.chunks[3 * ck + 2];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    const int qp = p.dim_ld / 8, vp = p.vdim_ld / 8, nk = p.dim_ld / 32;
    for (int e = tid; e < kLinC * qp; e += 256) {
        const int t = e / qp, c = (e % qp) * 8;
        const size_t o = (size_t)(tok0 + min(t, n - 1)) * p.n_head * p.dim_ld + h * p.dim_ld + c;
        *reinterpret_cast<pi_u32x4 *>(qs + t * qrow + c * 2) = pi_ld16((const uint16_t *)p.q + o);
        *reinterpret_cast<pi_u32x4 *>(ks + t * qrow + c * 2) = pi_ld16((const uint16_t *)p.k + o);
        *reinterpret_cast<pi_u32x4 *>(gs + t * grow + c * 4) = pi_ld16(p.gates + o);
        *reinterpret_cast<pi_u32x4 *>(gs + t * grow + c * 4 + 16) = pi_ld16(p.gates + o + 4);
    }
    pi_u32x4 rv[2 * VPW];                                         // a thread's pieces of the values, stored once the sums are done with
#pragma unroll
    for (int k = 0; k < 2 * VPW; ++k) {
        const int e = min(tid + k * 256, kLinC * vp - 1);
        rv[k] = pi_ld16((const uint16_t *)p.v + (size_t)(tok0 + min(e / vp, n - 1)) * p.n_head * p.vdim_ld + h * p.vdim_ld + e % vp * 8);
    }
    __syncthreads();
    const auto sums8 = [&](int t, int c, float (&o)[8]) {        // eight channels of a token's sums; zeros before the chunk
        if (t < 0) {
#pragma unroll
            for (int j = 0; j < 8; ++j) o[j] = 0.0f;
            return;
        }
        const float4 * a = reinterpret_cast<const float4 *>(gs + t * grow + c * 4);
        const float4 x = a[0], y = a[1];
        o[0] = x.x; o[1] = x.y; o[2] = x.z; o[3] = x.w; o[4] = y.x; o[5] = y.y; o[6] = y.z; o[7] = y.w;
    };
    float w[4][4];
    {
        const int ti = wave * 16 + i, ref = wave * 16 - 1;
        float span = 0.0f;                                        // how far the sums fall over the wave's tokens
        for (int c = lane; c < p.dim; c += PI_WAVE)
            span = fmaxf(span, (ref < 0 ? 0.0f : *reinterpret_cast<const float *>(gs + ref * grow + c * 4)) - *reinterpret_cast<const float *>(gs + (wave * 16 + 15) * grow + c * 4));
        const bool pairs = pi_wave_max(span) > kLinSpan;
        pi_f4 s[4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) s[kt] = pi_f4{0, 0, 0, 0};
        for (int k = 0; k < nk; ++k) {
            const int c = k * 32 + g * 8;
            float r[8], f[8], e[8];
            sums8(ref, c, r);
            sums8(ti, c, f);
#pragma unroll
            for (int j = 0; j < 8; ++j) e[j] = lin_exp2(f[j] - r[j]);
            pi_u32x4 qh, ql;
            lin_split8(*reinterpret_cast<const pi_u32x4 *>(qs + ti * qrow + c * 2), e, qh, ql);
#pragma unroll
            for (int kt = 0; kt < 4; ++kt) {
                if (kt > wave || (kt == wave && pairs)) continue;
                sums8(kt * 16 + i, c, f);
#pragma unroll
                for (int j = 0; j < 8; ++j) e[j] = lin_exp2(r[j] - f[j]);
                pi_u32x4 kh, kl;
                lin_split8(*reinterpret_cast<const pi_u32x4 *>(ks + (kt * 16 + i) * qrow + c * 2), e, kh, kl);
                s[kt] = mfma_bf16(kh, qh, s[kt]);
                s[kt] = mfma_bf16(kh, ql, s[kt]);
                s[kt] = mfma_bf16(kl, qh, s[kt]);
            }
        }
        if (pairs) {
            float a[4] = {0.0f, 0.0f, 0.0f, 0.0f};
            for (int c = 0; c < p.dim_ld; c += 8) {
                float f[8], e[8];
                sums8(ti, c, f);
                const pi_u32x4 qv = *reinterpret_cast<const pi_u32x4 *>(qs + ti * qrow + c * 2);
                const bf16 * q = reinterpret_cast<const bf16 *>(&qv);
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int tj = wave * 16 + 4 * g + r;
                    sums8(tj, c, e);
                    const pi_u32x4 kv = *reinterpret_cast<const pi_u32x4 *>(ks + tj * qrow + c * 2);
                    const bf16 * k = reinterpret_cast<const bf16 *>(&kv);
#pragma unroll
                    for (int j = 0; j < 8; ++j) a[r] = fmaf((float)q[j] * (float)k[j], lin_exp2(fminf(f[j] - e[j], 0.0f)), a[r]);
                }
            }
#pragma unroll
            for (int kt = 0; kt < 4; ++kt) if (kt == wave) s[kt] = pi_f4{a[0], a[1], a[2], a[3]};
        }
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) w[kt][r] = kt * 16 + 4 * g + r <= ti ? s[kt][r] : 0.0f;
    }
    __syncthreads();
    for (int e = tid; e < kLinC * qp; e += 256) {                 // queries decayed from the chunk's start on, for the state before it
        const int t = e / qp, c = (e % qp) * 8;
        float f[8];
        sums8(t, c, f);
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] = lin_exp2(f[j]);
        pi_u32x4 hi, lo;
        lin_split8(*reinterpret_cast<const pi_u32x4 *>(qs + t * qrow + c * 2), f, hi, lo);
        *reinterpret_cast<pi_u32x4 *>(qs + t * qrow + c * 2) = hi;
        *reinterpret_cast<pi_u32x4 *>(ks + t * qrow + c * 2) = lo;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 2 * VPW; ++k) {
        const int e = tid + k * 256;
        if (e < kLinC * vp) *reinterpret_cast<pi_u32x4 *>(vs + (e / vp) * vrow + (e % vp) * 16) = rv[k];
    }
    lin_store_scores(pp, w, wave, lane);
    __syncthreads();
    LinAcc<VPW> acc;
    lin_zero<VPW>(acc);
    if (!fresh) lin_add_state<VPW, true>(acc, p, ck, h, qs, ks, qrow);
    lin_add_scores<VPW>(acc, p, vs, vrow, pp);
    lin_store<VPW>(acc, p, tok0, n, h);
}

template <typename ST>
__global__ __launch_bounds__(256) void gate_norm_kernel(pi_gate_norm p) {
    __shared__ double red[4];
    gate_norm_block<ST>(p, blockIdx.x, red);
}

template <typename ST, int J, int MODE> int launch_step(const pi_linear * p, const pi_ffn_front & f, const pi_gqa_prep * beside, hipStream_t st) {
    const int slices = lin_copies(p->vdim), n_state = p->n_runs * p->n_head * slices, per = front_blocks(f), n_front = per * p->T;
    const int per_beside = beside ? gqa_prep_blocks(*beside) : 0, n_beside = per_beside * p->T;
    const size_t own = sizeof(float) * lin_step_floats(8 * J, MODE), lds = own > front_lds_bytes(f) ? own : front_lds_bytes(f);
    if (n_state + n_front + n_beside <= 0) return PI_OK;
    static bool raised = false;
    if (!raised && lds > 64 * 1024) { PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&linear_step_kernel<ST, J, MODE>), hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024)); raised = true; }
    hipLaunchKernelGGL((linear_step_kernel<ST, J, MODE>), dim3(n_state + n_front + n_beside), dim3(256), lds, st, *p, f, beside ? *beside : pi_gqa_prep{}, n_state, n_front, slices, per, per_beside);
    return pi::check_launch("pi_k_linear_step");
}
template <typename ST, int MODE> int step_of_size(const pi_linear * p, const pi_ffn_front & f, const pi_gqa_prep * b, hipStream_t st) {
    if (p->dim <= 32) return launch_step<ST, 4, MODE>(p, f, b, st);
    if (p->dim <= 64) return launch_step<ST, 8, MODE>(p, f, b, st);
    if (p->dim <= 96) return launch_step<ST, 12, MODE>(p, f, b, st);
    if (p->dim <= 128) return launch_step<ST, 16, MODE>(p, f, b, st);
    return launch_step<ST, 32, MODE>(p, f, b, st);
}
template <typename ST> int step_of_type(const pi_linear * p, const pi_ffn_front & f, const pi_gqa_prep * b, hipStream_t st) {
    if (p->decay_kind == kConst) return step_of_size<ST, kConst>(p, f, b, st);
    return p->decay_kind == kKeyed ? step_of_size<ST, kKeyed>(p, f, b, st) : step_of_size<ST, kGated>(p, f, b, st);
}

bool linear_ok(const pi_linear * p, const pi_ffn_front & f) {
    if (!p || !p->z || p->T <= 0 || p->n_head <= 0 || !pi_k_linear_supported(p->dim, p->vdim) || p->off_q < 0 || p->off_k < 0 || p->off_v < 0 || p->off_k + p->n_head * p->dim > p->ldz ||
        p->off_q + p->n_head * p->dim > p->ldz || p->off_v + p->n_head * p->vdim > p->ldz || !front_ok(f, p->ldz) || (long long)p->T * (front_blocks(f) + 3 * (p->n_head + 1)) >= (1 << 30) ||
        (p->slot_ld && p->slot_ld < lin_slot_floats(p->decay_kind, p->n_head, p->dim, p->vdim)))
        return false;
    if (p->decay_kind == kKeyed)
        return p->a2 && p->a2_b && p->rank > 0 && p->rank <= kLinMaxRank && p->rank_ld >= p->rank && p->rank_ld % 8 == 0 && p->rank_ld <= kLinMaxRank && p->off_a >= 0 &&
               p->off_a + p->rank_ld <= p->ldz && p->tau > 0.0f;
    if (p->decay_kind == kGated) return p->i_b && p->f_b && p->den && p->off_i >= 0 && p->off_i + p->n_head <= p->ldz && p->off_f >= 0 && p->off_f + p->n_head <= p->ldz && p->cap > 0.0f;
    return p->decay_kind == kConst;
}
bool operands_ok(const pi_linear * p) {
    return p->q && p->k && p->v && p->dim_ld >= p->dim && p->dim_ld % 32 == 0 && p->vdim_ld >= p->vdim && p->vdim_ld % 64 == 0 && p->dim_ld <= kLinMax && p->vdim_ld <= kLinMax;
}
int linear_step(int type, const pi_linear * p, const pi_ffn_front & f, const pi_gqa_prep * beside, hipStream_t st) {
    if (!linear_ok(p, f) || p->n_runs < 0 || (p->n_runs > 0 && ((p->decay_kind == kConst && !p->decay) || !p->state || !p->runs || !p->o)) || (long long)p->n_runs * p->n_head * 8 > (1 << 29) ||
        (beside && (!gqa_prep_ok(type, *beside) || beside->T != p->T || (long long)beside->T * gqa_prep_blocks(*beside) > (1 << 29))))
        return pi::fail(PI_E_ARG, "pi_k_linear_step: bad arguments");
    if (type == PI_TYPE_BF16) return step_of_type<bf16>(p, f, beside, st);
    if (type == PI_TYPE_F32) return step_of_type<float>(p, f, beside, st);
    return pi::fail(PI_E_UNSUPPORTED, "pi_k_linear_step: type");
}

// raises the kernel's LDS limit once
template <typename K> int big_lds(K * kernel, bool & raised) {
    if (!raised) { PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024)); raised = true; }
    return PI_OK;
}
template <int VPW, int MODE> int launch_out_mode(const pi_linear * p, hipStream_t st) {
    static bool raised = false;
    const dim3 grid(p->n_chunks * p->n_head);
    if constexpr (MODE == kKeyed) {
        const int rc = big_lds(&linear_out_keyed_kernel<VPW>, raised);
        if (rc != PI_OK) return rc;
        hipLaunchKernelGGL(linear_out_keyed_kernel<VPW>, grid, dim3(256), lin_keyed_lds(p->dim_ld, p->vdim_ld), st, *p);
    } else {
        const size_t lds = (size_t)kLinC * (2 * (p->dim_ld * 2 + 16) + p->vdim_ld * 2 + 16) + 4 * 2 * 2 * 64 * 16 + sizeof(float) * (MODE == kGated ? 3 * kLinC : kLinC + 4);
        const int rc = big_lds(&linear_out_kernel<VPW, MODE>, raised);
        if (rc != PI_OK) return rc;
        hipLaunchKernelGGL((linear_out_kernel<VPW, MODE>), grid, dim3(256), lds, st, *p);
    }
    return pi::check_launch("pi_k_linear_chunks out");
}
template <int VPW> int launch_out(const pi_linear * p, hipStream_t st) {
    return p->decay_kind == kConst ? launch_out_mode<VPW, kConst>(p, st) : p->decay_kind == kKeyed ? launch_out_mode<VPW, kKeyed>(p, st) : launch_out_mode<VPW, kGated>(p, st);
}
int launch_decays(const pi_linear * p, hipStream_t st) {
    if (p->decay_kind == kGated) {
        const int h4 = (p->n_head + 3) / 4;
        hipLaunchKernelGGL(linear_gates_kernel, dim3(p->n_chunks * h4 + p->n_runs), dim3(256), 0, st, *p, h4);
        return pi::check_launch("pi_k_linear_chunks gates");
    }
    if (p->decay_kind != kKeyed) return PI_OK;
    static bool raised = false;
    const int rc = big_lds(&linear_decays_kernel, raised), n_blocks = (p->n_head * p->dim_ld + 255) / 256;
    if (rc != PI_OK) return rc;
    hipLaunchKernelGGL(linear_decays_kernel, dim3(p->n_chunks * n_blocks), dim3(256), sizeof(float) * kLinC * p->rank_ld, st, *p, n_blocks);
    return pi::check_launch("pi_k_linear_chunks decays");
}

}  // namespace

extern "C" {

int pi_k_linear_chunk(void) { return kLinC; }
int pi_k_linear_supported(int dim, int vdim) { return dim > 0 && vdim > 0 && dim <= kLinMax && vdim <= kLinMax; }
int pi_k_linear_copies(int vdim) { return lin_copies(vdim); }
size_t pi_k_linear_slot_floats(int decay_kind, int n_head, int dim, int vdim) { return lin_slot_floats(decay_kind, n_head, dim, vdim); }
size_t pi_k_linear_states_bytes(int n_chunks, int n_head, int dim_ld, int vdim_ld) { return (size_t)n_chunks * n_head * dim_ld * (vdim_ld + 1) * 4; }
size_t pi_k_linear_gate_floats(int decay_kind, int T, int n_chunks, int n_head, int dim_ld) {
    return decay_kind == kKeyed ? (size_t)T * n_head * dim_ld : decay_kind == kGated ? ((size_t)4 * T + n_chunks) * n_head : 0;
}

int pi_k_linear_step(int type, const pi_linear * p, const pi_ffn_front * front, pi_stream_t stream) {
    return linear_step(type, p, front ? *front : pi_ffn_front{}, nullptr, (hipStream_t)stream);
}
int pi_k_linear_step_beside(int type, const pi_linear * p, const pi_gqa_prep * prep, pi_stream_t stream) {
    if (!p || !prep || p->decay_kind == kConst) return pi::fail(PI_E_ARG, "pi_k_linear_step_beside: bad arguments (a recurrence with gates)");
    return linear_step(type, p, pi_ffn_front{}, prep, (hipStream_t)stream);
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
    if (!linear_ok(p, pi_ffn_front{}) || !operands_ok(p) || (p->decay_kind == kConst ? !p->powers : !p->gates) || !p->state || !p->runs || p->n_runs <= 0 || p->n_runs > 65535 || !p->o ||
        !p->states || p->n_chunks <= 0 || !p->chunks || !p->first_chunk || (long long)p->n_chunks * p->n_head * p->dim_ld > (1LL << 36))
        return pi::fail(PI_E_ARG, "pi_k_linear_chunks: bad arguments");
    hipStream_t st = (hipStream_t)stream;
    int rc = launch_decays(p, st);
    if (rc != PI_OK) return rc;
    const int td = p->dim_ld / 32, tv = p->vdim_ld / 64;
    const dim3 grid(td * tv * p->n_head, p->n_runs);
    if (p->decay_kind == kConst) hipLaunchKernelGGL(linear_states_kernel<kConst>, grid, dim3(256), 0, st, *p, td, tv);
    else if (p->decay_kind == kKeyed) hipLaunchKernelGGL(linear_states_kernel<kKeyed>, grid, dim3(256), 0, st, *p, td, tv);
    else hipLaunchKernelGGL(linear_states_kernel<kGated>, grid, dim3(256), 0, st, *p, td, tv);
    rc = pi::check_launch("pi_k_linear_chunks states");
    if (rc != PI_OK) return rc;
    return p->vdim_ld <= 64 ? launch_out<1>(p, st) : p->vdim_ld <= 128 ? launch_out<2>(p, st) : p->vdim_ld <= 192 ? launch_out<3>(p, st) : launch_out<4>(p, st);
}

int pi_k_gate_norm(int type, const pi_gate_norm * p, pi_stream_t stream) {
    if (!p || !gate_norm_ok(*p)) return pi::fail(PI_E_ARG, "pi_k_gate_norm: bad arguments");
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(gate_norm_kernel<bf16>, dim3(gate_norm_blocks(*p)), dim3(256), 0, (hipStream_t)stream, *p);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(gate_norm_kernel<float>, dim3(gate_norm_blocks(*p)), dim3(256), 0, (hipStream_t)stream, *p);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_gate_norm: type");
    return pi::check_launch("pi_k_gate_norm");
}

}  // extern "C"
