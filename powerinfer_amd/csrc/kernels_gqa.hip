// Grouped-query attention on cells that lie anywhere in the pool: lists[seq] names a sequence's cells in position order.  A cell of a
// layer is, per key / value head, one row [key | value] of 2 * hd values, so that what a head reads of a cell is contiguous.
#include "mixers.hpp"

namespace {

template <typename ST, bool PAIRS>
__global__ __launch_bounds__(256) void gqa_prep_kernel(pi_gqa_prep p, pi_ffn_front f, int n_heads4, int per) {
    extern __shared__ __align__(16) float sm[];
    const int t = blockIdx.x / per, b = blockIdx.x % per;
    if (b >= n_heads4) front_block<ST>(f, p.z, p.ldz, t, b - n_heads4, sm);
    else gqa_prep_block<ST, PAIRS>(p, t, b);
}
template <typename ST> void launch_prep(const pi_gqa_prep & p, const pi_ffn_front & f, int n4, int per, hipStream_t st) {
    if (p.rot_pairs) hipLaunchKernelGGL((gqa_prep_kernel<ST, true>), dim3(per * p.T), dim3(256), front_lds_bytes(f), st, p, f, n4, per);
    else hipLaunchKernelGGL((gqa_prep_kernel<ST, false>), dim3(per * p.T), dim3(256), front_lds_bytes(f), st, p, f, n4, per);
}

// the first cell a token sees
__device__ __forceinline__ int first_cell(const pi_gqa_attn & p, int t) { return p.first ? p.first[t] : p.window > 0 ? max(p.n_vis[t] - p.window, 0) : 0; }

// ---------------------------------------------------------------------------------------------------------------------------------
// bf16 attention on the matrix cores.  Scores are formed transposed (keys x query rows), so that a lane's scores belong to one row, its
// soft-max needs two shuffles, and its weights are already the column operand of the second product (values^T x weights) - which key a
// slot of that product's inner dimension stands for is free, so the value operand is read (transposed, ds_read_tr16) in the order the
// scores came out.  Query rows are (token, head of the group) pairs, heads innermost: the rows of a token share its cells.
//   WIDE: 128 rows, 32 per wave, against 64 cells at a time (long runs).
//   else: 16 rows, the same in every wave, against 128 cells at a time, 32 per wave; the waves' sums are merged at the end.
// ---------------------------------------------------------------------------------------------------------------------------------
typedef short pi_s4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ pi_s4 tr_read(const unsigned char * q) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) pi_s4 *)(__attribute__((address_space(3))) void *)q);
}

template <int KS, bool WIDE> constexpr size_t gqa_lds() { return (size_t)2 * (WIDE ? 64 : 128) * (KS * 64 + 16); }

// EXT: soft caps, a sink per head, every head against the values of every key / value head (all_values)
__device__ __forceinline__ int gqa_groups(const pi_gqa_attn & p) { return p.all_values ? p.n_kv * p.n_kv : p.n_kv; }
// cap * tanh(v * k / (2 log2 e)): k = 2 log2 e / cap
__device__ __forceinline__ float soft_cap(float v, float k, float cap) { return fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(v * k) + 1.0f), cap); }
constexpr float kTwoLog2E = 2.8853900817779268f;

template <int KS, bool WIDE, bool EXT>      // 32-column steps of a key or value row
__global__ __launch_bounds__(256, WIDE && KS <= 4 ? 2 : 1) void gqa_attn_kernel(pi_gqa_attn p) {
    constexpr int VT = 2 * KS, NK = WIDE ? 64 : 128, R = WIDE ? 128 : 16, U = WIDE ? 2 : 1, KT = WIDE ? 4 : 2, ROW = KS * 64 + 16, NKK = NK / 32, HD = KS * 32;
    extern __shared__ __align__(16) unsigned char smem[];
    unsigned char * ks = smem, * vs = smem + NK * ROW;
    const int n_groups = EXT ? gqa_groups(p) : p.n_kv, vg = blockIdx.x % n_groups, item_index = p.n_work - 1 - (int)blockIdx.x / n_groups, part = blockIdx.y;      // the last items see the most cells
    const int g = EXT && p.all_values ? vg / p.n_kv : vg, gv = EXT && p.all_values ? vg % p.n_kv : vg;      // the group's keys and whose values
    const int4 item = reinterpret_cast<const int4 *>(p.work)[item_index];
    const int tok0 = item.x, first = item.y, rows = min(item.z, R), per = p.n_head / p.n_kv;
    const int32_t * list = p.lists + (size_t)item.w * p.list_ld;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, gq = lane >> 4;
    const int tok_a = tok0 + first / per, tok_z = tok0 + (first + rows - 1) / per;
    const int n_keys = p.n_vis[tok_z], n_all = p.n_vis[tok_a];       // the most and the fewest cells a row here sees
    const int lo_a = first_cell(p, tok_a), lo_z = first_cell(p, tok_z);      // the first cell of the rows' windows: the earliest and the latest
    const int tiles = (n_keys - lo_a + NK - 1) / NK;
    const int c0 = lo_a + (int)((long long)tiles * part / p.n_parts) * NK, c1 = min(lo_a + (int)((long long)tiles * (part + 1) / p.n_parts) * NK, n_keys);
    // the thread's pieces of a tile: eight threads share a cell's row
    const int sub = tid % 8, key0 = tid / 8;
    const uint16_t * cache = (const uint16_t *)p.cache + (size_t)g * 2 * HD + sub * 8;
    int idx[NKK];
    pi_u32x4 pre[NKK][KS];
    auto look_up = [&](int cb) {
#pragma unroll
        for (int k = 0; k < NKK; ++k) idx[k] = list[min(cb + key0 + 32 * k, n_keys - 1)];
    };
    auto fetch = [&]() {
#pragma unroll
        for (int k = 0; k < NKK; ++k)
#pragma unroll
            for (int j = 0; j < KS; ++j) pre[k][j] = pi_ld16(cache + (size_t)idx[k] * p.n_kv * 2 * HD + j * 64 + (EXT && sub + 8 * j >= 4 * KS ? (gv - g) * 2 * HD : 0));
    };
    if (c0 < c1) look_up(c0);
    int row[U], tok[U], head[U], lo[U];
    unsigned nv[U];                                              // cells the row sees, from lo on
    pi_u32x4 qf[U][KS];
#pragma unroll
    for (int u = 0; u < U; ++u) {
        row[u] = (WIDE ? wave * 32 : 0) + u * 16 + i;
        const int rr = first + min(row[u], rows - 1);
        tok[u] = tok0 + rr / per;
        head[u] = g * per + rr % per;
        lo[u] = first_cell(p, tok[u]);
        nv[u] = row[u] < rows ? p.n_vis[tok[u]] - lo[u] : 0;
#pragma unroll
        for (int s = 0; s < KS; ++s) qf[u][s] = pi_ld16((const uint16_t *)p.q + ((size_t)tok[u] * p.n_head + head[u]) * HD + s * 32 + gq * 8);
    }
    if (c0 < c1) { fetch(); look_up(c0 + NK); }
    float m[U], l[U];
    pi_f4 o[U][VT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
        m[u] = -INFINITY; l[u] = 0.0f;
#pragma unroll
        for (int v = 0; v < VT; ++v) o[u][v] = pi_f4{0, 0, 0, 0};
    }
    const int kb = WIDE ? 0 : wave * 32;                         // this wave's cells of a tile
    const float cap_k = EXT && p.softcap > 0.0f ? kTwoLog2E / p.softcap : 0.0f;
    for (int cb = c0; cb < c1; cb += NK) {
        __syncthreads();
#pragma unroll
        for (int k = 0; k < NKK; ++k)
#pragma unroll
            for (int j = 0; j < KS; ++j) {
                const int c = sub + 8 * j;
                *reinterpret_cast<pi_u32x4 *>((c < 4 * KS ? ks + c * 16 : vs + (c - 4 * KS) * 16) + (key0 + 32 * k) * ROW) = pre[k][j];
            }
        __syncthreads();
        fetch();                                                 // past the last tile: rows of the last cell, not used
        look_up(cb + 2 * NK);
        pi_f4 s[U][KT];
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {
#pragma unroll
            for (int u = 0; u < U; ++u) s[u][kt] = pi_f4{0, 0, 0, 0};
#pragma unroll
            for (int c = 0; c < KS; ++c) {
                const pi_u32x4 a = *reinterpret_cast<const pi_u32x4 *>(ks + (kb + kt * 16 + i) * ROW + c * 64 + gq * 16);
#pragma unroll
                for (int u = 0; u < U; ++u) s[u][kt] = mfma_bf16(a, qf[u][c], s[u][kt]);
            }
        }
        pi_u32x4 pb[U][KT / 2];                                  // weights as the column operand
        const bool edge = cb + NK > n_all || cb < lo_z;
#pragma unroll
        for (int u = 0; u < U; ++u) {
            float mx = -INFINITY;
#pragma unroll
            for (int kt = 0; kt < KT; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float v = s[u][kt][r] * p.scale;
                    if (EXT && p.softcap > 0.0f) v = soft_cap(v, cap_k, p.softcap);
                    if (edge && (unsigned)(cb + kb + kt * 16 + 4 * gq + r - lo[u]) >= nv[u]) v = -INFINITY;
                    s[u][kt][r] = v;
                    mx = fmaxf(mx, v);
                }
            mx = fmaxf(mx, __shfl_xor(mx, 16, PI_WAVE));
            mx = fmaxf(mx, __shfl_xor(mx, 32, PI_WAVE));
            const float mn = fmaxf(m[u], mx), base = mn == -INFINITY ? 0.0f : mn;
            const float a = expf(m[u] - base);                   // 0 while nothing has been seen
            m[u] = mn;
            float sum = 0.0f;
            bf16 w[4 * KT];
#pragma unroll
            for (int kt = 0; kt < KT; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) { const float e = expf(s[u][kt][r] - base); sum += e; w[kt * 4 + r] = (bf16)e; }
            l[u] = l[u] * a + sum;
#pragma unroll
            for (int v = 0; v < VT; ++v) { o[u][v][0] *= a; o[u][v][1] *= a; o[u][v][2] *= a; o[u][v][3] *= a; }
#pragma unroll
            for (int k = 0; k < KT / 2; ++k) {
                bf16 b[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) b[j] = w[k * 8 + j];
                pb[u][k] = __builtin_bit_cast(pi_u32x4, b);
            }
        }
        // slot (gq, j) of a 32-cell step: cell 4 gq + j of its first 16 (j < 4) or of its second 16 - two transposing reads
#pragma unroll
        for (int k = 0; k < KT / 2; ++k)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const unsigned char * a = vs + (kb + k * 32 + 4 * gq + (i >> 2)) * ROW + (v * 16 + (i & 3) * 4) * 2;
                const pi_u32x2 lo = __builtin_bit_cast(pi_u32x2, tr_read(a)), hi = __builtin_bit_cast(pi_u32x2, tr_read(a + 16 * ROW));
                const pi_u32x4 fr{lo.x, lo.y, hi.x, hi.y};
#pragma unroll
                for (int u = 0; u < U; ++u) o[u][v] = mfma_bf16(fr, pb[u][k], o[u][v]);
            }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) { l[u] += __shfl_xor(l[u], 16, PI_WAVE); l[u] += __shfl_xor(l[u], 32, PI_WAVE); }
    const bool whole = p.n_parts == 1, quads = ((p.vdim | p.ld_att) & 3) == 0;
    const size_t srow0 = ((size_t)item_index * n_groups + vg) * R;
    float2 * ml = reinterpret_cast<float2 *>(p.scratch + (size_t)p.n_work * n_groups * R * p.n_parts * HD);
    if (WIDE) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (row[u] >= rows) continue;
            if (!whole) {
                float * acc = p.scratch + ((srow0 + row[u]) * p.n_parts + part) * HD;
#pragma unroll
                for (int v = 0; v < VT; ++v) *reinterpret_cast<pi_f4 *>(acc + v * 16 + 4 * gq) = o[u][v];
                if (gq == 0) ml[(srow0 + row[u]) * p.n_parts + part] = make_float2(m[u], l[u]);
                continue;
            }
            const float sink = EXT && p.sinks ? p.sinks[head[u]] : p.sink;
            const float mf = fmaxf(m[u], sink), a = m[u] == -INFINITY ? 0.0f : expf(m[u] - mf), f = a / (l[u] * a + expf(sink - mf)) * p.out_scale;
            if (EXT && p.all_values) {
                float * out = (float *)p.att + (((size_t)tok[u] * p.n_head + head[u]) * p.n_kv + gv) * p.vdim;
#pragma unroll
                for (int v = 0; v < VT; ++v) {
                    const int c = v * 16 + 4 * gq;
                    const float w[4] = {o[u][v][0] * f, o[u][v][1] * f, o[u][v][2] * f, o[u][v][3] * f};
                    if (c < p.vdim) store4(out + c, w, (p.vdim & 3) == 0, p.vdim - c);
                }
                continue;
            }
            bf16 * out = (bf16 *)p.att + (size_t)tok[u] * p.ld_att + head[u] * p.vdim;
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const int c = v * 16 + 4 * gq;
                const float w[4] = {o[u][v][0] * f, o[u][v][1] * f, o[u][v][2] * f, o[u][v][3] * f};
                if (c < p.vdim) store4(out + c, w, quads && c + 4 <= p.vdim, p.vdim - c);
            }
        }
        return;
    }
    // merge of the waves' sums
    __syncthreads();
    constexpr int OLD = HD + 4;
    float * os = reinterpret_cast<float *>(smem);                // [4][16][OLD]
    float2 * wm = reinterpret_cast<float2 *>(os + 4 * 16 * OLD); // [4][16]
#pragma unroll
    for (int v = 0; v < VT; ++v) *reinterpret_cast<pi_f4 *>(os + (wave * 16 + i) * OLD + v * 16 + 4 * gq) = o[0][v];
    if (gq == 0) wm[wave * 16 + i] = make_float2(m[0], l[0]);
    __syncthreads();
    const int r = tid >> 4, cl = tid & 15;
    if (r >= rows) return;
    float mm = -INFINITY, f[4], sum = 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) mm = fmaxf(mm, wm[w * 16 + r].x);
#pragma unroll
    for (int w = 0; w < 4; ++w) { const float2 x = wm[w * 16 + r]; f[w] = x.x == -INFINITY ? 0.0f : expf(x.x - mm); sum += f[w] * x.y; }
    float fin = 1.0f;
    if (whole) {
        const float sink = EXT && p.sinks ? p.sinks[g * per + (first + r) % per] : p.sink;
        const float mf = fmaxf(mm, sink), a = mm == -INFINITY ? 0.0f : expf(mm - mf);
        fin = a / (sum * a + expf(sink - mf)) * p.out_scale;
    } else if (cl == 0) ml[(srow0 + r) * p.n_parts + part] = make_float2(mm, sum);
    const int rr = first + r;
    bf16 * out = (bf16 *)p.att + (size_t)(tok0 + rr / per) * p.ld_att + (g * per + rr % per) * p.vdim;
    float * acc = p.scratch + ((srow0 + r) * p.n_parts + part) * HD;
    for (int c = cl * 4; c < HD; c += 64) {
        float v[4] = {0, 0, 0, 0};
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const pi_f4 x = *reinterpret_cast<const pi_f4 *>(os + (w * 16 + r) * OLD + c);
#pragma unroll
            for (int k = 0; k < 4; ++k) v[k] = fmaf(f[w], x[k], v[k]);
        }
        if (whole) {
#pragma unroll
            for (int k = 0; k < 4; ++k) v[k] *= fin;
            if (EXT && p.all_values) {
                if (c < p.vdim) store4((float *)p.att + (((size_t)(tok0 + rr / per) * p.n_head + g * per + rr % per) * p.n_kv + gv) * p.vdim + c, v, (p.vdim & 3) == 0, p.vdim - c);
            } else if (c < p.vdim) store4(out + c, v, quads && c + 4 <= p.vdim, p.vdim - c);
        } else {
            *reinterpret_cast<float4 *>(acc + c) = make_float4(v[0], v[1], v[2], v[3]);
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// Long runs whose heads' weights are mixed, in two passes over the cells.  The first leaves the soft-max denominator of every (token, head).
// The second has a wave per key / value head: it forms its heads' weights from the denominators, hands them to the others through LDS, mixes those
// of all heads into its own and applies them to its values.  A tile's 16 rows are (token, head of the group) pairs, so the mixture is a product with a
// matrix that is zero between different tokens; the scores come out with rows as the inner dimension of that product, and its result with cells
// as the inner dimension of the product with the values.  Weights are mixed as sums of two bf16.
// ---------------------------------------------------------------------------------------------------------------------------------
constexpr float kLog2E = 1.4426950408889634f;
template <int KS>
__global__ __launch_bounds__(256) void gqa_stats_kernel(pi_gqa_attn p, float * __restrict__ stats) {
    constexpr int NK = 64, ROW = KS * 64 + 16, HD = KS * 32, C = 4 * KS, LD = (NK * C + 255) / 256;      // pieces of 16 bytes of a tile, per thread
    __shared__ __align__(16) unsigned char ks[NK * ROW];
    const int g = blockIdx.x % p.n_kv, item_index = p.n_work - 1 - (int)blockIdx.x / p.n_kv;
    const int4 item = reinterpret_cast<const int4 *>(p.work)[item_index];
    const int tok0 = item.x, first = item.y, rows = min(item.z, 128), per = p.n_head / p.n_kv;
    const int32_t * list = p.lists + (size_t)item.w * p.list_ld;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, gq = lane >> 4;
    const int tok_a = tok0 + first / per, tok_z = tok0 + (first + rows - 1) / per, n_keys = p.n_vis[tok_z], n_all = p.n_vis[tok_a], lo_a = first_cell(p, tok_a), lo_z = first_cell(p, tok_z);
    const uint16_t * cache = (const uint16_t *)p.cache + (size_t)g * 2 * HD;
    pi_u32x4 pre[LD];
    auto fetch = [&](int cb) {
#pragma unroll
        for (int k = 0; k < LD; ++k) {
            const int e = min(tid + 256 * k, NK * C - 1);
            pre[k] = pi_ld16(cache + (size_t)list[min(cb + e / C, n_keys - 1)] * p.n_kv * 2 * HD + (e % C) * 8);
        }
    };
    fetch(lo_a);
    int lo[2], tok[2], head[2], row[2];
    unsigned nv[2];
    pi_u32x4 qf[2][KS];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        row[u] = wave * 32 + u * 16 + i;
        const int rr = first + min(row[u], rows - 1);
        tok[u] = tok0 + rr / per;
        head[u] = g * per + rr % per;
        lo[u] = first_cell(p, tok[u]);
        nv[u] = row[u] < rows ? p.n_vis[tok[u]] - lo[u] : 0;
#pragma unroll
        for (int s = 0; s < KS; ++s) qf[u][s] = pi_ld16((const uint16_t *)p.q + ((size_t)tok[u] * p.n_head + head[u]) * HD + s * 32 + gq * 8);
    }
    const float cap_k = p.softcap > 0.0f ? kTwoLog2E / p.softcap : 0.0f;
    float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.0f, 0.0f};      // of this lane's cells, scores times log2 e
    for (int cb = lo_a; cb < n_keys; cb += NK) {
        __syncthreads();
#pragma unroll
        for (int k = 0; k < LD; ++k) {
            const int e = tid + 256 * k;
            if (e < NK * C) *reinterpret_cast<pi_u32x4 *>(ks + (e / C) * ROW + (e % C) * 16) = pre[k];
        }
        __syncthreads();
        fetch(cb + NK);                                          // past the last tile: rows of the last cell, not used
        pi_f4 s[2][4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
            s[0][kt] = s[1][kt] = pi_f4{0, 0, 0, 0};
#pragma unroll
            for (int c = 0; c < KS; ++c) {
                const pi_u32x4 a = *reinterpret_cast<const pi_u32x4 *>(ks + (kt * 16 + i) * ROW + c * 64 + gq * 16);
#pragma unroll
                for (int u = 0; u < 2; ++u) s[u][kt] = mfma_bf16(a, qf[u][c], s[u][kt]);
            }
        }
        const bool edge = cb + NK > n_all || cb < lo_z;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            float mx = m[u];
#pragma unroll
            for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float v = s[u][kt][r] * p.scale;
                    if (p.softcap > 0.0f) v = soft_cap(v, cap_k, p.softcap);
                    v *= kLog2E;
                    if (edge && (unsigned)(cb + kt * 16 + 4 * gq + r - lo[u]) >= nv[u]) v = -INFINITY;
                    s[u][kt][r] = v;
                    mx = fmaxf(mx, v);
                }
            const float base = mx == -INFINITY ? 0.0f : mx;
            float sum = l[u] * __builtin_amdgcn_exp2f(m[u] - base);
#pragma unroll
            for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) sum += __builtin_amdgcn_exp2f(s[u][kt][r] - base);
            m[u] = mx; l[u] = sum;
        }
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        float mm = fmaxf(m[u], __shfl_xor(m[u], 16, PI_WAVE));
        mm = fmaxf(mm, __shfl_xor(mm, 32, PI_WAVE));
        const float sink = (p.sinks ? p.sinks[head[u]] : p.sink) * kLog2E;
        mm = fmaxf(mm, sink);
        float sum = m[u] == -INFINITY ? 0.0f : l[u] * __builtin_amdgcn_exp2f(m[u] - mm);
        sum += __shfl_xor(sum, 16, PI_WAVE);
        sum += __shfl_xor(sum, 32, PI_WAVE);
        if (row[u] < rows && gq == 0) stats[(size_t)tok[u] * p.n_head + head[u]] = mm + log2f(sum + __builtin_amdgcn_exp2f(sink - mm));
    }
}

constexpr int kTalkTiles = 2, kTalkGroups = 8;      // tiles of 16 rows a wave has; most key / value heads
template <int KS> constexpr size_t talk_values_bytes() { return (size_t)32 * (KS * 64 + 16); }
inline int talk_pairs(int n_kv) { return (n_kv + 1) / 2; }
inline size_t talk_weights_bytes(int n_kv) { return (size_t)2 * kTalkTiles * 2 * talk_pairs(n_kv) * 64 * 16; }

template <int KS>
__global__ __launch_bounds__(64 * kTalkGroups) void gqa_talk_kernel(pi_gqa_attn p, pi_gqa_mix x, const float * __restrict__ stats, const int4 * __restrict__ items, int n_items) {
    constexpr int U = kTalkTiles, VT = 2 * KS, ROW = KS * 64 + 16, HD = KS * 32, C = 4 * KS, LD = 32 * C / 64, MAXP = kTalkGroups / 2;
    extern __shared__ __align__(16) unsigned char smem[];
    const int pairs = (p.n_kv + 1) / 2, groups = 2 * pairs;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, gq = lane >> 4, g = wave;
    pi_u32x4 * ws = reinterpret_cast<pi_u32x4 *>(smem);           // [2 cell tiles][U][groups][64]: four weights as bf16, and what is left of them
    unsigned char * vs = smem + (size_t)2 * U * groups * 64 * 16 + (size_t)wave * talk_values_bytes<KS>();
    const int4 item = items[n_items - 1 - (int)blockIdx.x];       // the last items see the most cells
    const int tok0 = item.x, n_tok = item.y, per = p.n_head / p.n_kv, tpt = 16 / per;      // tokens of a tile
    const int32_t * list = p.lists + (size_t)item.z * p.list_ld;
    const int n_all = p.n_vis[tok0], lo_z = first_cell(p, tok0 + n_tok - 1), parts = min(item.w >> 16, x.n_parts), part = item.w & 0xffff;
    int lo_a = first_cell(p, tok0), n_keys = p.n_vis[tok0 + n_tok - 1];
    if (parts > 1) {                                              // this part's cells
        const int each = ((n_keys - lo_a + parts - 1) / parts + 31) / 32 * 32;
        lo_a = min(lo_a + part * each, n_keys);
        n_keys = min(lo_a + each, n_keys);
    }
    const uint16_t * cache = (const uint16_t *)p.cache + (size_t)g * 2 * HD;
    if (p.n_kv & 1)                                               // the missing group of the last pair: zeros
        for (int k = threadIdx.x; k < 2 * U * 64; k += blockDim.x) ws[((k >> 6) * groups + p.n_kv) * 64 + (k & 63)] = pi_u32x4{0, 0, 0, 0};
    // rows 4 gq + r of the wave's tiles
    float c[U][4];
    int lo[U][4];
    unsigned nv[U][4];
    pi_u32x4 qf[U][KS];
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = 4 * gq + r, tl = u * tpt + row / per;
            const bool in = row < tpt * per && tl < n_tok;
            const int t = tok0 + (in ? tl : 0);
            lo[u][r] = first_cell(p, t);
            nv[u][r] = in ? p.n_vis[t] - lo[u][r] : 0;
            c[u][r] = in ? stats[(size_t)t * p.n_head + g * per + row % per] : 0.0f;
        }
        const int tq = tok0 + (i < tpt * per ? min(u * tpt + i / per, n_tok - 1) : 0), hq = g * per + i % per;
#pragma unroll
        for (int s = 0; s < KS; ++s) qf[u][s] = pi_ld16((const uint16_t *)p.q + ((size_t)tq * p.n_head + hq) * HD + s * 32 + gq * 8);
    }
    // column operand of the mixture: slot (gq, j) is row 4 gq + j of the pair's first group or row 4 gq + j - 4 of its second
    pi_u32x4 tf[MAXP];
#pragma unroll
    for (int q = 0; q < MAXP; ++q) {
        bf16 b[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int row = 4 * gq + (j & 3), from = 2 * q + (j >> 2);
            const bool in = from < p.n_kv && row < tpt * per && i < tpt * per && row / per == i / per;
            const int at = in ? (g * per + i % per) * p.n_head + from * per + row % per : 0;
            b[j] = (bf16)(in ? (x.talk ? x.talk[at] : (float)(at / p.n_head == at % p.n_head)) : 0.0f);
        }
        tf[q] = __builtin_bit_cast(pi_u32x4, b);
    }
    pi_f4 o[U][VT];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
        for (int v = 0; v < VT; ++v) o[u][v] = pi_f4{0, 0, 0, 0};
    const float cap_k = p.softcap > 0.0f ? kTwoLog2E / p.softcap : 0.0f;
    pi_u32x4 kf[2][KS], vf[LD];
    int cell = list[min(lo_a + (lane & 31), n_keys - 1)];
    auto fetch = [&]() {
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            const uint16_t * k = cache + (size_t)__shfl(cell, kt * 16 + i, PI_WAVE) * p.n_kv * 2 * HD + gq * 8;
#pragma unroll
            for (int s = 0; s < KS; ++s) kf[kt][s] = pi_ld16(k + s * 32);
        }
#pragma unroll
        for (int k = 0; k < LD; ++k) {
            const int e = lane + 64 * k;
            vf[k] = pi_ld16(cache + (size_t)__shfl(cell, e / C, PI_WAVE) * p.n_kv * 2 * HD + HD + (e % C) * 8);
        }
    };
    fetch();
    cell = list[min(lo_a + 32 + (lane & 31), n_keys - 1)];
    for (int cb = lo_a; cb < n_keys; cb += 32) {
        const bool edge = cb + 32 > n_all || cb < lo_z;
        __syncthreads();                                         // the last tile's weights and values have been read
#pragma unroll
        for (int k = 0; k < LD; ++k) { const int e = lane + 64 * k; *reinterpret_cast<pi_u32x4 *>(vs + (e / C) * ROW + (e % C) * 16) = vf[k]; }
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
            for (int u = 0; u < U; ++u) {
                pi_f4 s = pi_f4{0, 0, 0, 0};
#pragma unroll
                for (int k = 0; k < KS; ++k) s = mfma_bf16(qf[u][k], kf[kt][k], s);
                bf16 w[8];
                const bool all_rows = !edge;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float v = s[r] * p.scale;
                    if (p.softcap > 0.0f) v = soft_cap(v, cap_k, p.softcap);
                    float e = __builtin_amdgcn_exp2f(fmaf(v, kLog2E, -c[u][r]));
                    if (all_rows ? nv[u][r] == 0 : (unsigned)(cb + kt * 16 + i - lo[u][r]) >= nv[u][r]) e = 0.0f;
                    w[r] = (bf16)e;
                    w[4 + r] = (bf16)(e - (float)w[r]);
                }
                ws[((kt * U + u) * groups + g) * 64 + lane] = __builtin_bit_cast(pi_u32x4, w);
            }
        fetch();                                                 // past the last tile: rows of the last cell, not used
        cell = list[min(cb + 64 + (lane & 31), n_keys - 1)];
        __syncthreads();
        pi_u32x4 pb[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            bf16 b[8];
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
                pi_f4 mix = pi_f4{0, 0, 0, 0};
                const pi_u32x4 * wp = ws + (size_t)(kt * U + u) * groups * 64 + lane;
#pragma unroll
                for (int q = 0; q < MAXP; ++q) {
                    if (q >= pairs) break;
                    const pi_u32x4 a = wp[(2 * q) * 64], d = wp[(2 * q + 1) * 64];
                    mix = mfma_bf16(pi_u32x4{a.x, a.y, d.x, d.y}, tf[q], mix);
                    mix = mfma_bf16(pi_u32x4{a.z, a.w, d.z, d.w}, tf[q], mix);
                }
#pragma unroll
                for (int r = 0; r < 4; ++r) b[kt * 4 + r] = (bf16)mix[r];
            }
            pb[u] = __builtin_bit_cast(pi_u32x4, b);
        }
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const unsigned char * a = vs + (4 * gq + (i >> 2)) * ROW + (v * 16 + (i & 3) * 4) * 2;
            const pi_u32x2 l = __builtin_bit_cast(pi_u32x2, tr_read(a)), h = __builtin_bit_cast(pi_u32x2, tr_read(a + 16 * ROW));
            const pi_u32x4 fr{l.x, l.y, h.x, h.y};
#pragma unroll
            for (int u = 0; u < U; ++u) o[u][v] = mfma_bf16(fr, pb[u], o[u][v]);
        }
    }
    const bool quads = ((x.vdim | x.ld_att) & 3) == 0;
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int tl = u * tpt + i / per, head = g * per + i % per;
        if (i >= tpt * per || tl >= n_tok) continue;
        const int t = tok0 + tl;
        if (parts > 1) {                                          // (gated by gqa_talk_sum_kernel)
            if (part >= parts) continue;
            float * out = x.parts + (((size_t)part * x.T + t) * p.n_head + head) * x.vdim;
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const int col = v * 16 + 4 * gq;
                const float w[4] = {o[u][v][0], o[u][v][1], o[u][v][2], o[u][v][3]};
                if (col < x.vdim) store4(out + col, w, (x.vdim & 3) == 0, x.vdim - col);
            }
            continue;
        }
        const float f = x.off_gate >= 0 ? sigmoid_f32(x.z[(size_t)t * x.ldz + x.off_gate + head]) : 1.0f;
        bf16 * out = (bf16 *)x.att + (size_t)t * x.ld_att + head * x.vdim;
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int col = v * 16 + 4 * gq;
            const float w[4] = {o[u][v][0] * f, o[u][v][1] * f, o[u][v][2] * f, o[u][v][3] * f};
            if (col < x.vdim) store4(out + col, w, quads && col + 4 <= x.vdim, x.vdim - col);
        }
    }
}

// the sum of the parts of split items, with the heads' gates: a workgroup per (item, token of it)
__global__ __launch_bounds__(256) void gqa_talk_sum_kernel(pi_gqa_mix x, const int4 * __restrict__ items) {
    const int4 item = items[blockIdx.x];
    const int parts = min(item.w >> 16, x.n_parts), n = x.n_head * x.vdim;
    if (parts <= 1 || (item.w & 0xffff) != 0 || (int)blockIdx.y >= item.y) return;
    const int t = item.x + blockIdx.y;
    const float * a = x.parts + (size_t)t * n, * gate = x.off_gate >= 0 ? x.z + (size_t)t * x.ldz + x.off_gate : nullptr;
    bf16 * out = (bf16 *)x.att + (size_t)t * x.ld_att;
    const size_t step = (size_t)x.T * n;
    if (((x.vdim | x.ld_att) & 3) == 0) {
        for (int e = threadIdx.x * 4; e < n; e += 1024) {
            float4 s = make_float4(0, 0, 0, 0);
            for (int k = 0; k < parts; ++k) { const float4 v = *reinterpret_cast<const float4 *>(a + k * step + e); s.x += v.x; s.y += v.y; s.z += v.z; s.w += v.w; }
            const float f = gate ? sigmoid_f32(gate[e / x.vdim]) : 1.0f, w[4] = {s.x * f, s.y * f, s.z * f, s.w * f};
            store4(out + e, w, true, 4);
        }
    } else {
        for (int e = threadIdx.x; e < n; e += 256) {
            float s = 0.0f;
            for (int k = 0; k < parts; ++k) s += a[k * step + e];
            out[e] = (bf16)(gate ? s * sigmoid_f32(gate[e / x.vdim]) : s);
        }
    }
}

template <int KS> int launch_talk(const pi_gqa_attn * p, const pi_gqa_mix * x, const float * stats, const int32_t * items, int n, hipStream_t st) {
    const size_t lds = talk_weights_bytes(p->n_kv) + talk_values_bytes<KS>() * p->n_kv;
    static bool raised = false;
    if (!raised) {
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&gqa_talk_kernel<KS>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)(talk_weights_bytes(kTalkGroups) + talk_values_bytes<KS>() * kTalkGroups)));
        raised = true;
    }
    hipLaunchKernelGGL(gqa_talk_kernel<KS>, dim3(n), dim3(64 * p->n_kv), lds, st, *p, *x, stats, (const int4 *)items, n);
    if (x->n_parts > 1) hipLaunchKernelGGL(gqa_talk_sum_kernel, dim3(n, kTalkTiles * (16 / (p->n_head / p->n_kv))), dim3(256), 0, st, *x, (const int4 *)items);
    return pi::check_launch("pi_k_gqa_talk");
}

__global__ __launch_bounds__(256) void gqa_merge_kernel(pi_gqa_attn p) {
    const int R4 = gqa_rows(p.wide) / 4, wg = blockIdx.x, n = p.all_values ? p.n_kv * p.n_kv : p.n_kv;
    gqa_merge_row(p, wg / R4 / n, wg / R4 % n, (wg % R4) * 4 + (threadIdx.x >> 6));
}

// fp32: one workgroup per (token, head), 64 cells at a time (a wave per cell for the scores, a thread per column for the sum)
constexpr int kGfCells = 64;
__global__ __launch_bounds__(256) void gqa_attn_f32_kernel(pi_gqa_attn p) {
    __shared__ float q[kGqaMaxDim], s[kGfCells];
    __shared__ int idx[kGfCells];
    const int vals = p.all_values ? p.n_kv : 1, th = blockIdx.x / vals;
    const int t = th / p.n_head, h = th % p.n_head, g = h / (p.n_head / p.n_kv), gv = p.all_values ? blockIdx.x % vals : g, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int n = p.n_vis[t];
    const int32_t * list = p.lists + (size_t)p.work[t] * p.list_ld;
    const float * cache = (const float *)p.cache + (size_t)g * 2 * p.hd;
    const float * values = (const float *)p.cache + (size_t)gv * 2 * p.hd + p.hd;
    const size_t cell_ld = (size_t)p.n_kv * 2 * p.hd;
    for (int k = tid; k < p.dim; k += 256) q[k] = ((const float *)p.q)[(size_t)th * p.hd + k];
    const float own_sink = p.sinks ? p.sinks[h] : p.sink;
    const bool sink = own_sink != -INFINITY;
    float m = own_sink, l = sink ? 1.0f : 0.0f, acc = 0.0f;              // the sink is the soft-max's first entry: weight exp(0), no value
    for (int c0 = first_cell(p, t); c0 < n; c0 += kGfCells) {
        const int nc = min(kGfCells, n - c0);
        __syncthreads();
        for (int c = tid; c < nc; c += 256) idx[c] = list[c0 + c];
        __syncthreads();
        for (int c = wave; c < nc; c += 4) {
            const float * row = cache + idx[c] * cell_ld;
            float d = 0.0f;
            for (int k = lane; k < p.dim; k += 64) d = fmaf(q[k], row[k], d);
            d = pi_wave_sum(d);
            if (lane == 0) s[c] = p.softcap > 0.0f ? p.softcap * tanhf(d * p.scale / p.softcap) : d * p.scale;
        }
        __syncthreads();
        float mn = m;
        for (int c = 0; c < nc; ++c) mn = fmaxf(mn, s[c]);
        const float a = m == -INFINITY ? 0.0f : expf(m - mn);
        l *= a;
        acc *= a;
        for (int c = 0; c < nc; ++c) {
            const float w = expf(s[c] - mn);
            l += w;
            if (tid < p.vdim) acc = fmaf(w, values[idx[c] * cell_ld + tid], acc);
        }
        m = mn;
    }
    if (tid < p.vdim) ((float *)p.att)[p.all_values ? (size_t)blockIdx.x * p.vdim + tid : (size_t)t * p.ld_att + h * p.vdim + tid] = acc / l * p.out_scale;
}

// heads mixed behind an attention with all_values: 64 values of the key / value heads a workgroup, a quarter of the heads a wave, the query heads of a value's
// group eight at a time
constexpr int kMixAhead = 8, kMixHeads = 128;          // heads a wave requests together; most heads
__host__ __device__ inline int mix_groups(int n_kv, int vdim) { return min(n_kv, 63 / vdim + 2); }      // groups that 64 values can belong to
template <typename ST>
__global__ __launch_bounds__(256) void gqa_mix_kernel(pi_gqa_mix p) {
    extern __shared__ __align__(16) float talk[];      // the rows of the heads of those groups
    __shared__ float sum[4][8][64];
    const int t = p.tokens ? p.tokens[blockIdx.x] : blockIdx.x, per = p.n_head / p.n_kv, n = p.n_kv * p.vdim, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int e0 = blockIdx.y * 64, e = min(e0 + lane, n - 1), kv = e / p.vdim, c = e % p.vdim, kv0 = e0 / p.vdim, each = (p.n_head + 3) / 4;
    const int lo = min(wave * each, p.n_head), hi = min(lo + each, p.n_head);
    const float * a = p.a + (size_t)t * p.n_head * n + e;
    float v[kMixAhead];
    const auto fetch = [&](int g0) {
#pragma unroll
        for (int j = 0; j < kMixAhead; ++j) v[j] = g0 + j < hi ? a[(size_t)(g0 + j) * n] : 0.0f;
    };
    if (p.talk) {
        fetch(lo);
        const int rows = (min(e0 + 63, n - 1) / p.vdim - kv0 + 1) * per;
        for (int i = threadIdx.x; i < rows * p.n_head; i += 256) talk[i] = p.talk[kv0 * per * p.n_head + i];
    }
    __syncthreads();
    const float * gate = p.off_gate >= 0 ? p.z + (size_t)t * p.ldz + p.off_gate : nullptr;
    ST * out = (ST *)p.att + (size_t)t * p.ld_att;
    for (int h0 = 0; h0 < per; h0 += 8) {
        float s[8] = {0, 0, 0, 0, 0, 0, 0, 0};
        if (p.talk) {
            for (int g0 = lo; g0 < hi; g0 += kMixAhead) {
                if (h0 > 0 || g0 > lo) fetch(g0);
#pragma unroll
                for (int k = 0; k < 8; ++k) {
                    const float * row = talk + (size_t)((kv - kv0) * per + min(h0 + k, per - 1)) * p.n_head + g0;
#pragma unroll
                    for (int j = 0; j < kMixAhead; ++j) s[k] = g0 + j < hi ? fmaf(row[j], v[j], s[k]) : s[k];
                }
            }
        } else if (wave == 0) {
#pragma unroll
            for (int k = 0; k < 8; ++k) s[k] = a[(size_t)(kv * per + min(h0 + k, per - 1)) * n];
        }
        if (h0 > 0) __syncthreads();                   // the last eight heads' sums have been read
#pragma unroll
        for (int k = 0; k < 8; ++k) sum[wave][k][lane] = s[k];
        __syncthreads();
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            const int k = wave + 4 * q, h = kv * per + h0 + k;
            if (h0 + k >= per || e0 + lane >= n) continue;
            const float r = (sum[0][k][lane] + sum[1][k][lane]) + (sum[2][k][lane] + sum[3][k][lane]);
            out[h * p.vdim + c] = to_st<ST>(gate ? r * sigmoid_f32(gate[h]) : r);
        }
    }
}

template <typename ST>
__global__ void gqa_shift_kernel(ST * __restrict__ cache, int n_kv, int hd, int rot_dim, double base, const double * __restrict__ freq, int pairs, const int32_t * __restrict__ delta) {
    const int c = blockIdx.x, d = delta[c], half = rot_dim / 2;
    if (d == 0) return;
    for (int e = threadIdx.x; e < n_kv * half; e += blockDim.x) {
        const int g = e / half, i = e % half;
        double sn, cn;
        sincos((double)d * (freq ? freq[i] : pow(base, -2.0 * (double)i / (double)rot_dim)), &sn, &cn);
        ST * r = cache + ((size_t)c * n_kv + g) * 2 * hd + (pairs ? 2 * i : i), * o = r + (pairs ? 1 : half);
        const float u = from_st(*r), v = from_st(*o);
        *r = to_st<ST>(u * (float)cn - v * (float)sn);
        *o = to_st<ST>(v * (float)cn + u * (float)sn);
    }
}

template <int KS, bool WIDE, bool EXT> int launch_gqa_as(const pi_gqa_attn * p, hipStream_t st) {
    constexpr size_t tile = gqa_lds<KS, WIDE>(), merge = WIDE ? 0 : sizeof(float) * (4 * 16 * (KS * 32 + 4) + 2 * 4 * 16), lds = tile > merge ? tile : merge;
    static bool raised = false;
    if (!raised && lds > 64 * 1024) {
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&gqa_attn_kernel<KS, WIDE, EXT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        raised = true;
    }
    hipLaunchKernelGGL((gqa_attn_kernel<KS, WIDE, EXT>), dim3(p->n_work * p->n_kv * (p->all_values ? p->n_kv : 1), p->n_parts), dim3(256), lds, st, *p);
    return pi::check_launch("pi_k_gqa_attn");
}
template <int KS, bool WIDE> int launch_gqa(const pi_gqa_attn * p, hipStream_t st) {
    return p->softcap > 0.0f || p->sinks || p->all_values ? launch_gqa_as<KS, WIDE, true>(p, st) : launch_gqa_as<KS, WIDE, false>(p, st);
}

int gqa_check(int type, const pi_gqa_attn * p) {
    if (!p || !p->q || !p->cache || !p->lists || !p->work || !p->n_vis || !p->att || p->T <= 0 || p->n_head <= 0 || p->n_kv <= 0 || p->n_head % p->n_kv || p->dim <= 0 || p->vdim <= 0 ||
        p->hd < p->dim || p->hd < p->vdim || (!p->all_values && p->ld_att < p->n_head * p->vdim) || p->hd != pi_k_gqa_head_ld(type, p->dim, p->vdim) || p->n_parts <= 0 || p->window < 0)
        return pi::fail(PI_E_ARG, "pi_k_gqa_attn: bad arguments");
    if (type == PI_TYPE_BF16 && (p->n_work <= 0 || (long long)p->n_work * p->n_kv * (p->all_values ? p->n_kv : 1) > (1 << 30) || p->n_parts > 64 || (p->n_parts > 1 && !p->scratch)))
        return pi::fail(PI_E_ARG, "pi_k_gqa_attn: bad work arguments");
    return PI_OK;
}

template <bool WIDE> int gqa_bf16(const pi_gqa_attn * p, hipStream_t st) {
    switch (p->hd) {
        case 32: return launch_gqa<1, WIDE>(p, st);
        case 64: return launch_gqa<2, WIDE>(p, st);
        case 96: return launch_gqa<3, WIDE>(p, st);
        case 128: return launch_gqa<4, WIDE>(p, st);
        case 192: return launch_gqa<6, WIDE>(p, st);
        default: return launch_gqa<8, WIDE>(p, st);
    }
}

}  // namespace

extern "C" {

int pi_k_gqa_head_ld(int type, int dim, int vdim) {
    const int d = dim > vdim ? dim : vdim;
    if (dim <= 0 || vdim <= 0 || d > kGqaMaxDim) return 0;
    if (type == PI_TYPE_F32) return (d + 31) / 32 * 32;
    return d <= 128 ? (d + 31) / 32 * 32 : d <= 192 ? 192 : 256;
}

int pi_k_gqa_prep(int type, const pi_gqa_prep * p, const pi_ffn_front * front, pi_stream_t stream) {
    const pi_ffn_front f = front ? *front : pi_ffn_front{};
    if (!p || !gqa_prep_ok(type, *p) || !front_ok(f, p->ldz))
        return pi::fail(PI_E_ARG, "pi_k_gqa_prep: bad arguments");
    const int n4 = gqa_prep_blocks(*p), per = n4 + front_blocks(f);
    if ((long long)per * p->T > (1 << 30)) return pi::fail(PI_E_ARG, "pi_k_gqa_prep: too many tokens");
    if (type == PI_TYPE_BF16) launch_prep<bf16>(*p, f, n4, per, (hipStream_t)stream);
    else if (type == PI_TYPE_F32) launch_prep<float>(*p, f, n4, per, (hipStream_t)stream);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_gqa_prep: type");
    return pi::check_launch("pi_k_gqa_prep");
}

int pi_k_gqa_rows(int wide) { return gqa_rows(wide); }

size_t pi_k_gqa_scratch_floats(int n_work, int wide, int n_kv, int hd, int n_parts) {
    return n_parts > 1 ? (size_t)n_work * gqa_rows(wide) * n_kv * n_parts * (hd + 2) : 0;
}

int pi_k_gqa_attn_parts(const pi_gqa_attn * p, pi_stream_t stream) {
    const int rc = gqa_check(PI_TYPE_BF16, p);
    if (rc != PI_OK) return rc;
    return p->wide ? gqa_bf16<true>(p, (hipStream_t)stream) : gqa_bf16<false>(p, (hipStream_t)stream);
}

int pi_k_gqa_attn(int type, const pi_gqa_attn * p, pi_stream_t stream) {
    if (type == PI_TYPE_F32) {
        const int rc = gqa_check(type, p);
        if (rc != PI_OK) return rc;
        hipLaunchKernelGGL(gqa_attn_f32_kernel, dim3(p->T * p->n_head * (p->all_values ? p->n_kv : 1)), dim3(256), 0, (hipStream_t)stream, *p);
        return pi::check_launch("pi_k_gqa_attn");
    }
    if (type != PI_TYPE_BF16) return pi::fail(PI_E_UNSUPPORTED, "pi_k_gqa_attn: type");
    const int rc = pi_k_gqa_attn_parts(p, stream);
    if (rc != PI_OK || p->n_parts == 1) return rc;
    hipLaunchKernelGGL(gqa_merge_kernel, dim3(p->n_work * p->n_kv * (p->all_values ? p->n_kv : 1) * (gqa_rows(p->wide) / 4)), dim3(256), 0, (hipStream_t)stream, *p);
    return pi::check_launch("pi_k_gqa_attn merge");
}

int pi_k_gqa_talk_tokens(int n_head, int n_kv, int dim, int vdim) {
    const int hd = pi_k_gqa_head_ld(PI_TYPE_BF16, dim, vdim);
    if (!hd || hd > 128 || n_head <= 0 || n_kv <= 0 || n_kv > kTalkGroups || n_head % n_kv || n_head / n_kv > 16) return 0;
    return kTalkTiles * (16 / (n_head / n_kv));
}

int pi_k_gqa_stats(const pi_gqa_attn * p, float * stats, pi_stream_t stream) {
    if (!p || !p->q || !p->cache || !p->lists || !p->work || !p->n_vis || !stats || p->n_work <= 0 || p->window < 0 || !p->wide || !pi_k_gqa_talk_tokens(p->n_head, p->n_kv, p->dim, p->vdim) ||
        p->hd != pi_k_gqa_head_ld(PI_TYPE_BF16, p->dim, p->vdim))
        return pi::fail(PI_E_ARG, "pi_k_gqa_stats: bad arguments");
    hipStream_t st = (hipStream_t)stream;
    const dim3 grid(p->n_work * p->n_kv);
    switch (p->hd) {
        case 32: hipLaunchKernelGGL(gqa_stats_kernel<1>, grid, dim3(256), 0, st, *p, stats); break;
        case 64: hipLaunchKernelGGL(gqa_stats_kernel<2>, grid, dim3(256), 0, st, *p, stats); break;
        case 96: hipLaunchKernelGGL(gqa_stats_kernel<3>, grid, dim3(256), 0, st, *p, stats); break;
        default: hipLaunchKernelGGL(gqa_stats_kernel<4>, grid, dim3(256), 0, st, *p, stats);
    }
    return pi::check_launch("pi_k_gqa_stats");
}

int pi_k_gqa_talk(const pi_gqa_attn * p, const pi_gqa_mix * x, const float * stats, const int32_t * items, int n_items, pi_stream_t stream) {
    if (!p || !x || !p->q || !p->cache || !p->lists || !p->n_vis || !stats || !items || n_items <= 0 || p->window < 0 || !pi_k_gqa_talk_tokens(p->n_head, p->n_kv, p->dim, p->vdim) ||
        p->hd != pi_k_gqa_head_ld(PI_TYPE_BF16, p->dim, p->vdim) || !x->att || x->vdim != p->vdim || x->ld_att < p->n_head * p->vdim ||
        (x->off_gate >= 0 && (!x->z || x->off_gate + p->n_head > x->ldz)) || x->n_head != p->n_head || x->n_kv != p->n_kv || x->n_parts < 0 || (x->n_parts > 1 && (!x->parts || x->T != p->T)))
        return pi::fail(PI_E_ARG, "pi_k_gqa_talk: bad arguments");
    hipStream_t st = (hipStream_t)stream;
    switch (p->hd) {
        case 32: return launch_talk<1>(p, x, stats, items, n_items, st);
        case 64: return launch_talk<2>(p, x, stats, items, n_items, st);
        case 96: return launch_talk<3>(p, x, stats, items, n_items, st);
        default: return launch_talk<4>(p, x, stats, items, n_items, st);
    }
}

int pi_k_gqa_mix(int type, const pi_gqa_mix * p, pi_stream_t stream) {
    if (!p || !p->a || !p->att || p->T <= 0 || p->n_head <= 0 || p->n_kv <= 0 || p->n_head % p->n_kv || p->vdim <= 0 || p->ld_att < p->n_head * p->vdim ||
        (p->off_gate >= 0 && (!p->z || p->off_gate + p->n_head > p->ldz)))
        return pi::fail(PI_E_ARG, "pi_k_gqa_mix: bad arguments");
    const size_t lds = p->talk ? sizeof(float) * mix_groups(p->n_kv, p->vdim) * (p->n_head / p->n_kv) * p->n_head : 0;
    if (p->tokens && p->n_tokens <= 0) return pi::fail(PI_E_ARG, "pi_k_gqa_mix: bad arguments");
    const dim3 grid(p->tokens ? p->n_tokens : p->T, (p->n_kv * p->vdim + 63) / 64);
    if (p->n_head > kMixHeads || grid.y > 65535) return pi::fail(PI_E_UNSUPPORTED, "pi_k_gqa_mix: up to 128 heads");
    static bool raised = false;
    if (!raised) {
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&gqa_mix_kernel<bf16>), hipFuncAttributeMaxDynamicSharedMemorySize, kMixHeads * kMixHeads * (int)sizeof(float)));
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&gqa_mix_kernel<float>), hipFuncAttributeMaxDynamicSharedMemorySize, kMixHeads * kMixHeads * (int)sizeof(float)));
        raised = true;
    }
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(gqa_mix_kernel<bf16>, grid, dim3(256), lds, (hipStream_t)stream, *p);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(gqa_mix_kernel<float>, grid, dim3(256), lds, (hipStream_t)stream, *p);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_gqa_mix: type");
    return pi::check_launch("pi_k_gqa_mix");
}

static int gqa_shift(int type, void * cache, int n_cells, int n_kv, int hd, int rot_dim, double base, const double * freq, int pairs, const int32_t * delta, pi_stream_t stream) {
    if (!cache || !delta || n_cells <= 0 || n_kv <= 0 || hd <= 0 || rot_dim < 0 || rot_dim % 2 || rot_dim > hd) return pi::fail(PI_E_ARG, "pi_k_gqa_shift: bad arguments");
    if (rot_dim == 0) return PI_OK;
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(gqa_shift_kernel<bf16>, dim3(n_cells), dim3(64), 0, (hipStream_t)stream, (bf16 *)cache, n_kv, hd, rot_dim, base, freq, pairs, delta);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(gqa_shift_kernel<float>, dim3(n_cells), dim3(64), 0, (hipStream_t)stream, (float *)cache, n_kv, hd, rot_dim, base, freq, pairs, delta);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_gqa_shift: type");
    return pi::check_launch("pi_k_gqa_shift");
}

int pi_k_gqa_shift(int type, void * cache, int n_cells, int n_kv, int hd, int rot_dim, double base, int pairs, const int32_t * delta, pi_stream_t stream) {
    return gqa_shift(type, cache, n_cells, n_kv, hd, rot_dim, base, nullptr, pairs, delta, stream);
}

int pi_k_gqa_shift_table(int type, void * cache, int n_cells, int n_kv, int hd, int rot_dim, const double * freq, int pairs, const int32_t * delta, pi_stream_t stream) {
    if (!freq) return pi::fail(PI_E_ARG, "pi_k_gqa_shift_table: bad arguments");
    return gqa_shift(type, cache, n_cells, n_kv, hd, rot_dim, 1.0, freq, pairs, delta, stream);
}

}  // extern "C"
