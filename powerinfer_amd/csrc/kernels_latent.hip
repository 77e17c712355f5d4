// Attention over a cached low-rank latent.  A cell of the cache is one row [latent (padded) | rotated key part (padded)]; with the
// key expansion folded into the query (q_lat = W_uk^T q) every head scores its cells straight on these rows, and the value expansion is
// applied to the weighted sum of latents afterwards, so a cell is read once for all heads and never expanded.  A sequence's cells lie
// anywhere in the pool: lists[seq] names them in position order.
#include "layer_types.hpp"

namespace {

// ---------------------------------------------------------------------------------------------------------------------------------
// behind the joint projection: query parts, rotation, and the token's own cell
// ---------------------------------------------------------------------------------------------------------------------------------
template <typename ST>
__global__ __launch_bounds__(256) void latent_prep_kernel(pi_latent_prep p) {
    __shared__ double red[4];
    const int t = blockIdx.x, hd = p.dim + p.rot_dim, half = p.rot_dim / 2;
    const float * z = p.z + (size_t)t * p.ldz;
    const float2 * cs = (const float2 *)p.cs + (size_t)t * half;
    const int n_q = p.cache ? gridDim.y - 1 : gridDim.y;           // with own cells the last workgroup of a token makes the cell
    if ((int)blockIdx.y == n_q) {
        const float * c = z + p.n_head * hd;
        ST * cell = (ST *)p.cache + (size_t)p.cell[t] * p.kd;
        double s = 0.0;
        for (int i = threadIdx.x; i < p.kv_rank; i += blockDim.x) { const float v = c[i]; s += (double)v * (double)v; }
        s = block_sum_f64(s, red);
        const float sc = pi_inv_sqrt((float)(s / p.kv_rank) + p.eps);
        for (int i = threadIdx.x; i < p.kv_rank; i += blockDim.x) cell[i] = to_st<ST>(c[i] * sc * p.norm_w[i]);
        for (int i = threadIdx.x; i < half; i += blockDim.x) {
            const float u = c[p.kv_rank + 2 * i], v = c[p.kv_rank + 2 * i + 1];
            cell[p.rank_ld + 2 * i] = to_st<ST>(u * cs[i].x - v * cs[i].y);
            cell[p.rank_ld + 2 * i + 1] = to_st<ST>(v * cs[i].x + u * cs[i].y);
        }
        return;
    }
    ST * qu = (ST *)p.q_un + (size_t)t * p.n_head * p.dim_ld, * ql = (ST *)p.q_lat + (size_t)t * p.n_head * p.kd;
    for (int e = blockIdx.y * 256 + threadIdx.x; e < p.n_head * (p.dim + half); e += n_q * 256) {
        const int h = e / (p.dim + half), k = e % (p.dim + half);
        const float * q = z + h * hd;
        if (k < p.dim) {
            qu[h * p.dim_ld + k] = to_st<ST>(q[k]);
        } else {
            const int i = k - p.dim;
            const float u = q[p.dim + 2 * i], v = q[p.dim + 2 * i + 1];
            ST * o = ql + (size_t)h * p.kd + p.rank_ld + 2 * i;
            o[0] = to_st<ST>(u * cs[i].x - v * cs[i].y);
            o[1] = to_st<ST>(v * cs[i].x + u * cs[i].y);
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// bf16 attention on the matrix cores.  A workgroup of four waves owns 16 * RT query rows ((token, head) pairs, heads innermost: the rows
// of a token share its cells) and one part of their cells, 32 cells at a time: rows staged in LDS once, used as the key operand of the
// scores and - read transposed - as the value operand of the weighted sum.  Scores, soft-max and sums are fp32; the weights enter the
// second product as bf16.  Waves split the (row tile, cell tile) pairs of the scores and the latent columns of the sum.
// ---------------------------------------------------------------------------------------------------------------------------------
constexpr int kLaCells = 32;
constexpr int kLaRows = 32;

// B operand of 32 cells x 16 columns from LDS rows of `stride` bytes: lane (column i, cells 8 g ..) - two transposing reads, in each of
// which sixteen lanes fetch 4 cells x 16 columns and swap them so that every lane ends up with its column's four cells
typedef short pi_s4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ pi_s4 tr_read(const unsigned char * q) {
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) pi_s4 *)(__attribute__((address_space(3))) void *)q);
}
__device__ __forceinline__ pi_u32x4 frag_cells(const unsigned char * rows, int stride, int col) {
    const int lane = threadIdx.x & 63, g = lane >> 4, li = lane & 15;
    const unsigned char * a = rows + (8 * g + (li >> 2)) * stride + (col + (li & 3) * 4) * 2;
    const pi_u32x2 lo = __builtin_bit_cast(pi_u32x2, tr_read(a)), hi = __builtin_bit_cast(pi_u32x2, tr_read(a + 4 * stride));
    return pi_u32x4{lo.x, lo.y, hi.x, hi.y};
}

// by_item: parts are kept per work item (row = item * rows per item + row of the item) instead of per (token, head)
template <int RT, int VT, int PF>      // row tiles; latent-column tiles per wave; 16-byte pieces of a cell tile per thread
__global__ __launch_bounds__(256) void latent_attn_bf16_kernel(pi_latent_attn p, int by_item) {
    constexpr int R = 16 * RT, NC = kLaCells, TPR = 256 / R, CPT = NC / TPR;      // threads per row and cells per thread of the soft-max
    extern __shared__ __align__(16) unsigned char smem[];
    const int stride = p.kd * 2 + 16, pieces = p.kd / 8;
    unsigned char * qs = smem;                                   // [R][stride]
    unsigned char * ks = qs + R * stride;                        // [NC][stride]
    float * ss = reinterpret_cast<float *>(ks + NC * stride);    // [R][NC + 1]
    bf16 * ps = reinterpret_cast<bf16 *>(ss + R * (NC + 1) + (R * (NC + 1)) % 4);          // [R][NC + 8]
    float * row_m = reinterpret_cast<float *>(ps + R * (NC + 8)), * row_l = row_m + R, * row_a = row_l + R;
    int * row_n = reinterpret_cast<int *>(row_a + R);
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    const int4 item = reinterpret_cast<const int4 *>(p.work)[blockIdx.x];
    const int tok0 = item.x, first = item.y, rows = min(item.z, R), seq = item.w;
    const size_t qrow0 = (size_t)tok0 * p.n_head + first;        // row of q_lat / out_lat of this workgroup's first row
    const size_t srow0 = by_item ? (size_t)blockIdx.x * R : qrow0;                         // and of the parts it leaves
    const int32_t * list = p.lists + (size_t)seq * p.list_ld;
    const int n_all = p.n_vis[tok0 + (first + rows - 1) / p.n_head];                       // cells of the last row's token: the most of all
    const int tiles = (n_all + NC - 1) / NC, part = blockIdx.y;
    const int c0 = (int)((long long)tiles * part / p.n_parts) * NC, c1 = min((int)((long long)tiles * (part + 1) / p.n_parts) * NC, n_all);
    // thread's pieces of a cell tile
    pi_u32x4 pre[PF];
    int pn[PF], pc[PF];
    const int step_n = 256 / pieces, step_c = 256 - step_n * pieces;
#pragma unroll
    for (int j = 0; j < PF; ++j) {                   // piece tid + 256 j: row and place within it, by carrying instead of dividing
        if (j == 0) { pn[0] = tid / pieces; pc[0] = tid - pn[0] * pieces; continue; }
        const int c = pc[j - 1] + step_c, over = c >= pieces ? 1 : 0;
        pc[j] = c - (over ? pieces : 0);
        pn[j] = pn[j - 1] + step_n + over;
    }
    // pieces past the tile repeat its last row: loads and stores stay unconditional (a guarded load makes the compiler wait for all of
    // them one by one), and what is stored twice is the same
#pragma unroll
    for (int j = 0; j < PF; ++j) { pn[j] = min(pn[j], NC - 1); pc[j] *= 8; }
    const uint16_t * cache = (const uint16_t *)p.cache;
    // a tile's cells are looked up one tile before its rows are requested, the rows one tile before they are used
    int idx[PF];
    auto look_up = [&](int cb) {
#pragma unroll
        for (int j = 0; j < PF; ++j) idx[j] = list[min(cb + pn[j], n_all - 1)];
    };
    auto fetch = [&]() {
#pragma unroll
        for (int j = 0; j < PF; ++j) pre[j] = pi_ld16(cache + (size_t)idx[j] * p.kd + pc[j]);
    };
    if (c0 < c1) look_up(c0);
    // the query rows travel with the first cells: as many pieces per thread as a cell tile has (R == NC rows)
    static_assert(R == NC, "query and cell tiles share the piece layout");
    pi_u32x4 qr[PF];
#pragma unroll
    for (int j = 0; j < PF; ++j)
        qr[j] = pi_ld16((const uint16_t *)p.q_lat + (qrow0 + min(pn[j], rows - 1)) * p.kd + pc[j]);
    if (c0 < c1) { fetch(); look_up(c0 + NC); }
#pragma unroll
    for (int j = 0; j < PF; ++j)
        *reinterpret_cast<pi_u32x4 *>(qs + pn[j] * stride + pc[j] * 2) = qr[j];
    if (tid < R) { row_m[tid] = -INFINITY; row_l[tid] = 0.0f; row_n[tid] = tid < rows ? p.n_vis[tok0 + (first + tid) / p.n_head] : 0; }
    pi_f4 acc[RT][VT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt)
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[rt][v] = pi_f4{0, 0, 0, 0};
    const int n_vt = p.rank_ld / 16;
    for (int cb = c0; cb < c1; cb += NC) {
        __syncthreads();                                         // the previous tile's readers are done (first pass: nothing to wait for)
#pragma unroll
        for (int j = 0; j < PF; ++j)
            *reinterpret_cast<pi_u32x4 *>(ks + pn[j] * stride + pc[j] * 2) = pre[j];
        __syncthreads();
        fetch();                                                 // past the last tile: rows of the last cell, not used
        look_up(cb + 2 * NC);
        // scores: RT x 2 pairs of (row tile, cell tile) over four waves
        for (int pr = wave; pr < RT * 2; pr += 4) {
            const int rt = pr >> 1, ct = pr & 1;
            pi_f4 s = pi_f4{0, 0, 0, 0}, s2 = s;
            const unsigned char * qa = qs + (rt * 16 + i) * stride + g * 16, * kb = ks + (ct * 16 + i) * stride + g * 16;
            // four 32-column steps at a time: their operands are read while the previous four are multiplied
            const int n4 = p.kd / 128;
            pi_u32x4 fa[2][4], fb[2][4];
            auto read4 = [&](pi_u32x4 (&a)[4], pi_u32x4 (&b)[4], int k) {
#pragma unroll
                for (int u = 0; u < 4; ++u) { a[u] = *reinterpret_cast<const pi_u32x4 *>(qa + k * 256 + u * 64); b[u] = *reinterpret_cast<const pi_u32x4 *>(kb + k * 256 + u * 64); }
            };
            auto mul4 = [&](const pi_u32x4 (&a)[4], const pi_u32x4 (&b)[4]) {
                s = mfma_bf16(a[0], b[0], s); s2 = mfma_bf16(a[1], b[1], s2); s = mfma_bf16(a[2], b[2], s); s2 = mfma_bf16(a[3], b[3], s2);
            };
            if (n4 > 0) read4(fa[0], fb[0], 0);
            for (int k = 0; k < n4; k += 2) {
                if (k + 1 < n4) read4(fa[1], fb[1], k + 1);
                mul4(fa[0], fb[0]);
                if (k + 1 < n4) {
                    if (k + 2 < n4) read4(fa[0], fb[0], k + 2);
                    mul4(fa[1], fb[1]);
                }
            }
            for (int k = n4 * 256; k < p.kd * 2; k += 64)
                s = mfma_bf16(*reinterpret_cast<const pi_u32x4 *>(qa + k), *reinterpret_cast<const pi_u32x4 *>(kb + k), s);
            s += s2;
            const int cell = cb + ct * 16 + i;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int row = rt * 16 + 4 * g + r;
                ss[row * (NC + 1) + ct * 16 + i] = cell < c1 && cell < row_n[row] ? s[r] * p.scale : -INFINITY;
            }
        }
        __syncthreads();
        {
            const int row = tid / TPR, sub = tid % TPR;
            float v[CPT], mx = -INFINITY;
#pragma unroll
            for (int c = 0; c < CPT; ++c) { v[c] = ss[row * (NC + 1) + sub * CPT + c]; mx = fmaxf(mx, v[c]); }
#pragma unroll
            for (int o = TPR / 2; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, PI_WAVE));
            const float m_old = row_m[row], m_new = fmaxf(m_old, mx);
            float sum = 0.0f;
#pragma unroll
            for (int c = 0; c < CPT; ++c) {
                const float e = m_new == -INFINITY ? 0.0f : expf(v[c] - m_new);
                sum += e;
                ps[row * (NC + 8) + sub * CPT + c] = (bf16)e;
            }
#pragma unroll
            for (int o = TPR / 2; o > 0; o >>= 1) sum += __shfl_xor(sum, o, PI_WAVE);
            if (sub == 0) {
                const float a = m_old == -INFINITY ? 0.0f : expf(m_old - m_new);
                row_a[row] = a;
                row_l[row] = row_l[row] * a + sum;
                row_m[row] = m_new;
            }
        }
        __syncthreads();
        pi_u32x4 pa[RT];
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) {
            pa[rt] = *reinterpret_cast<const pi_u32x4 *>(ps + (rt * 16 + i) * (NC + 8) + g * 8);
            const float4 a = *reinterpret_cast<const float4 *>(row_a + rt * 16 + 4 * g);
#pragma unroll
            for (int v = 0; v < VT; ++v) { acc[rt][v][0] *= a.x; acc[rt][v][1] *= a.y; acc[rt][v][2] *= a.z; acc[rt][v][3] *= a.w; }
        }
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            if (wave * VT + v >= n_vt) continue;
            const pi_u32x4 b = frag_cells(ks, stride, (wave * VT + v) * 16);
#pragma unroll
            for (int rt = 0; rt < RT; ++rt) acc[rt][v] = mfma_bf16(pa[rt], b, acc[rt][v]);
        }
    }
    __syncthreads();
    const bool whole = p.n_parts == 1;
    if (tid < rows) {
        if (whole) {
            const float sink = p.sink[(first + tid) % p.n_head], m = fmaxf(row_m[tid], sink), a = row_m[tid] == -INFINITY ? 0.0f : expf(row_m[tid] - m);
            row_a[tid] = a / (row_l[tid] * a + expf(sink - m));
        } else {
            float * ml = p.scratch + (by_item ? (size_t)p.n_work * R : (size_t)p.T * p.n_head) * p.n_parts * p.rank_ld;
            const size_t o = ((srow0 + tid) * p.n_parts + part) * 2;
            ml[o] = row_m[tid];
            ml[o + 1] = row_l[tid];
        }
    }
    __syncthreads();
    // the sums leave through LDS (queries and cells are done with), so that the stores are whole lines and the code is short
    float * os = reinterpret_cast<float *>(smem);                // [R][rank_ld]
#pragma unroll
    for (int rt = 0; rt < RT; ++rt)
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int col = (wave * VT + v) * 16 + i;
            if (col >= p.rank_ld) continue;
            float * d = os + (rt * 16 + 4 * g) * p.rank_ld + col;
#pragma unroll
            for (int r = 0; r < 4; ++r) d[r * p.rank_ld] = acc[rt][v][r];
        }
    __syncthreads();
    const int quads = p.rank_ld / 4;
    for (int r = wave; r < rows; r += 4) {                       // a wave per row
        const float f = whole ? row_a[r] : 1.0f;
        for (int c = lane; c < quads; c += 64) {
            const float4 v = *reinterpret_cast<const float4 *>(os + r * p.rank_ld + c * 4);
            if (whole) {
                const bf16 b[4] = {(bf16)(v.x * f), (bf16)(v.y * f), (bf16)(v.z * f), (bf16)(v.w * f)};
                *reinterpret_cast<pi_u32x2 *>((bf16 *)p.out_lat + (qrow0 + r) * p.rank_ld + c * 4) = __builtin_bit_cast(pi_u32x2, b);
            } else {
                *reinterpret_cast<float4 *>(p.scratch + ((srow0 + r) * p.n_parts + part) * p.rank_ld + c * 4) = v;
            }
        }
    }
}

// the parts of one row of a work item and the sink: fixed order
__global__ __launch_bounds__(128) void latent_merge_kernel(pi_latent_attn p) {
    const int4 item = reinterpret_cast<const int4 *>(p.work)[blockIdx.x / kLaRows];
    const int r = blockIdx.x % kLaRows;
    if (r >= item.z) return;
    const size_t row = (size_t)item.x * p.n_head + item.y + r, srow = blockIdx.x;
    const float * ml = p.scratch + (size_t)p.n_work * kLaRows * p.n_parts * p.rank_ld + srow * p.n_parts * 2;
    const float * acc = p.scratch + srow * p.n_parts * p.rank_ld;
    const float sink = p.sink[row % p.n_head];
    float m = sink;
    for (int s = 0; s < p.n_parts; ++s) m = fmaxf(m, ml[2 * s]);
    float l = expf(sink - m);
    for (int s = 0; s < p.n_parts; ++s) if (ml[2 * s] != -INFINITY) l += ml[2 * s + 1] * expf(ml[2 * s] - m);
    for (int c = threadIdx.x; c < p.rank_ld; c += blockDim.x) {
        float v = 0.0f;
        for (int s = 0; s < p.n_parts; ++s) if (ml[2 * s] != -INFINITY) v += acc[(size_t)s * p.rank_ld + c] * expf(ml[2 * s] - m);
        ((bf16 *)p.out_lat)[row * p.rank_ld + c] = (bf16)(v / l);
    }
}

// fp32: one workgroup per row, 64 cells at a time (a wave per cell for the scores, a thread per latent column for the sum)
constexpr int kLfCells = 64;
__global__ __launch_bounds__(256) void latent_attn_f32_kernel(pi_latent_attn p) {
    extern __shared__ __align__(16) unsigned char smem[];
    float * q = reinterpret_cast<float *>(smem), * s = q + p.kd;          // [kd], [64]
    int * idx = reinterpret_cast<int *>(s + kLfCells);
    const int t = blockIdx.x / p.n_head, h = blockIdx.x % p.n_head, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int n = p.n_vis[t];
    const int32_t * list = p.lists + (size_t)p.work[t] * p.list_ld;       // fp32: work holds each token's sequence
    const float * cache = (const float *)p.cache;
    for (int k = tid; k < p.kd; k += 256) q[k] = ((const float *)p.q_lat)[(size_t)blockIdx.x * p.kd + k];
    float m = p.sink[h], l = 1.0f, acc[4] = {0, 0, 0, 0};                 // the sink is the soft-max's first entry: weight exp(0), no value
    for (int c0 = 0; c0 < n; c0 += kLfCells) {
        const int nc = min(kLfCells, n - c0);
        __syncthreads();
        for (int c = tid; c < nc; c += 256) idx[c] = list[c0 + c];
        __syncthreads();
        for (int c = wave; c < nc; c += 4) {
            const float * row = cache + (size_t)idx[c] * p.kd;
            float d = 0.0f;
            for (int k = lane; k < p.kd; k += 64) d = fmaf(q[k], row[k], d);
            d = pi_wave_sum(d);
            if (lane == 0) s[c] = d * p.scale;
        }
        __syncthreads();
        float mn = m;
        for (int c = 0; c < nc; ++c) mn = fmaxf(mn, s[c]);
        const float a = expf(m - mn);
        l *= a;
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] *= a;
        for (int c = 0; c < nc; ++c) {
            const float w = expf(s[c] - mn);
            l += w;
            const float * row = cache + (size_t)idx[c] * p.kd;
#pragma unroll
            for (int j = 0; j < 4; ++j) { const int k = tid + 256 * j; if (k < p.rank_ld) acc[j] = fmaf(w, row[k], acc[j]); }
        }
        m = mn;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) { const int k = tid + 256 * j; if (k < p.rank_ld) ((float *)p.out_lat)[(size_t)blockIdx.x * p.rank_ld + k] = acc[j] / l; }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// Long prompt portions: keys and values of the visible cells are expanded once (two mat-muls over the cells' latents) and a portion's
// tokens attend to them head by head.  A workgroup owns 128 tokens of one head; a wave owns 32 of them as columns: scores are formed
// transposed (keys x tokens), so that a lane's scores belong to one token, its soft-max needs two shuffles, and its weights are already
// the column operand of the second product (values^T x weights) - which key a slot of that product's inner dimension stands for is free,
// so the value operand is read in the order the scores came out.  64 keys at a time through LDS, the next 64 in registers.
// ---------------------------------------------------------------------------------------------------------------------------------
constexpr int kXKeys = 64, kXTok = 128;
template <int KS, int VT>              // 32-column steps of a key row (unrotated | rotated, zero padded); 16-column tiles of a value row
__global__ __launch_bounds__(256, 2) void latent_expanded_attn_kernel(pi_latent_expanded p, int n_qt, int hp) {
    constexpr int KROW = KS * 64 + 16, VROW = VT * 32 + 16, KP = KS * 4 * kXKeys / 256, VP = VT * 2 * kXKeys / 256;      // bytes per LDS row; pieces per thread
    __shared__ __align__(16) unsigned char ks[kXKeys * KROW];
    __shared__ __align__(16) unsigned char vs[kXKeys * VROW];
    const int xcd = blockIdx.x % 8, slot = blockIdx.x / 8, h = xcd + 8 * (slot % hp), qt = n_qt - 1 - slot / hp;            // the longest tiles first; a head stays on one XCD
    if (h >= p.n_head) return;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    const int q0 = qt * kXTok, dk = p.dim + p.rot_dim;
    // the tokens of this lane (column i of two tiles) and the cells they see
    int nv[2], tok[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const int t = q0 + wave * 32 + u * 16 + i;
        tok[u] = p.tok0 + min(t, p.T - 1);
        nv[u] = t < p.T ? p.n_vis[tok[u]] : 0;
    }
    const int n_keys = p.n_vis[p.tok0 + min(q0 + kXTok, p.T) - 1], n_all = p.n_vis[p.tok0 + q0];          // the most and the fewest cells a token here sees
    pi_u32x4 qf[2][KS];
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const int c = s * 32 + g * 8;
            const bf16 * src = c < p.dim ? (const bf16 *)p.q_un + ((size_t)tok[u] * p.n_head + h) * p.dim_ld + c
                                         : (const bf16 *)p.q_lat + ((size_t)tok[u] * p.n_head + h) * p.kd + p.rank_ld + (c - p.dim);
            qf[u][s] = c < dk ? pi_ld16(src) : pi_u32x4{0, 0, 0, 0};
        }
    pi_u32x4 kr[KP], vr[VP];
    auto fetch = [&](int k0) {
#pragma unroll
        for (int j = 0; j < KP; ++j) {
            const int e = tid + 256 * j, key = min(k0 + e / (KS * 4), n_keys - 1), c = (e % (KS * 4)) * 8;
            const bf16 * src = c < p.dim ? (const bf16 *)p.keys + ((size_t)key * p.n_head + h) * p.dim + c
                                         : (const bf16 *)p.cache + (size_t)p.list[key] * p.kd + p.rank_ld + (min(c, dk - 8) - p.dim);
            kr[j] = pi_ld16(src);                      // (unconditional loads: past the end of a row its last piece, zeroed on the way to LDS)
        }
#pragma unroll
        for (int j = 0; j < VP; ++j) {
            const int e = tid + 256 * j, key = min(k0 + e / (VT * 2), n_keys - 1), c = min((e % (VT * 2)) * 8, p.vdim - 8);
            vr[j] = pi_ld16((const bf16 *)p.values + ((size_t)key * p.n_head + h) * p.vdim + c);
        }
    };
    fetch(0);
    float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.0f, 0.0f};
    pi_f4 o[2][VT];
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int v = 0; v < VT; ++v) o[u][v] = pi_f4{0, 0, 0, 0};
    for (int k0 = 0; k0 < n_keys; k0 += kXKeys) {
        __syncthreads();
#pragma unroll
        for (int j = 0; j < KP; ++j) { const int e = tid + 256 * j; *reinterpret_cast<pi_u32x4 *>(ks + (e / (KS * 4)) * KROW + (e % (KS * 4)) * 16) = (e % (KS * 4)) * 8 < dk ? kr[j] : pi_u32x4{0, 0, 0, 0}; }
#pragma unroll
        for (int j = 0; j < VP; ++j) { const int e = tid + 256 * j; *reinterpret_cast<pi_u32x4 *>(vs + (e / (VT * 2)) * VROW + (e % (VT * 2)) * 16) = vr[j]; }
        __syncthreads();
        fetch(k0 + kXKeys);
        pi_f4 s[2][4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
            s[0][kt] = s[1][kt] = pi_f4{0, 0, 0, 0};
#pragma unroll
            for (int c = 0; c < KS; ++c) {
                const pi_u32x4 a = *reinterpret_cast<const pi_u32x4 *>(ks + (kt * 16 + i) * KROW + c * 64 + g * 16);
                s[0][kt] = mfma_bf16(a, qf[0][c], s[0][kt]);
                s[1][kt] = mfma_bf16(a, qf[1][c], s[1][kt]);
            }
        }
        pi_u32x4 pb[2][2];                             // weights as the column operand: [token tile][32 keys]
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            float mx = -INFINITY;
            const bool edge = k0 + kXKeys > n_all;
#pragma unroll
            for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    float v = s[u][kt][r] * p.scale;
                    if (edge && k0 + kt * 16 + 4 * g + r >= nv[u]) v = -INFINITY;
                    s[u][kt][r] = v;
                    mx = fmaxf(mx, v);
                }
            mx = fmaxf(mx, __shfl_xor(mx, 16, PI_WAVE));
            mx = fmaxf(mx, __shfl_xor(mx, 32, PI_WAVE));
            const float mn = fmaxf(m[u], mx), base = mn == -INFINITY ? 0.0f : mn;
            const float a = expf(m[u] - base);         // 0 while nothing has been seen
            m[u] = mn;
            float sum = 0.0f;
            bf16 w[16];
#pragma unroll
            for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                for (int r = 0; r < 4; ++r) { const float e = expf(s[u][kt][r] - base); sum += e; w[kt * 4 + r] = (bf16)e; }
            l[u] = l[u] * a + sum;
#pragma unroll
            for (int v = 0; v < VT; ++v) { o[u][v][0] *= a; o[u][v][1] *= a; o[u][v][2] *= a; o[u][v][3] *= a; }
#pragma unroll
            for (int k = 0; k < 2; ++k) {
                bf16 b[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) b[j] = w[k * 8 + j];
                pb[u][k] = __builtin_bit_cast(pi_u32x4, b);
            }
        }
        // slot (g, j) of a 32-key step: key 4 g + j of its first 16 (j < 4) or of its second 16 - two transposing reads
#pragma unroll
        for (int k = 0; k < 2; ++k)
#pragma unroll
            for (int v = 0; v < VT; ++v) {
                const unsigned char * a = vs + (k * 32 + 4 * g + (i >> 2)) * VROW + (v * 16 + (i & 3) * 4) * 2;
                const pi_u32x2 lo = __builtin_bit_cast(pi_u32x2, tr_read(a)), hi = __builtin_bit_cast(pi_u32x2, tr_read(a + 16 * VROW));
                const pi_u32x4 f{lo.x, lo.y, hi.x, hi.y};
                o[0][v] = mfma_bf16(f, pb[0][k], o[0][v]);
                o[1][v] = mfma_bf16(f, pb[1][k], o[1][v]);
            }
    }
    const float sink = p.sink[h];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        float sum = l[u];
        sum += __shfl_xor(sum, 16, PI_WAVE);
        sum += __shfl_xor(sum, 32, PI_WAVE);
        const float mf = fmaxf(m[u], sink), a = m[u] == -INFINITY ? 0.0f : expf(m[u] - mf), f = a / (sum * a + expf(sink - mf));
        if (q0 + wave * 32 + u * 16 + i >= p.T) continue;
        bf16 * out = (bf16 *)p.att + (size_t)tok[u] * p.ld_att + h * p.vdim;
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const int c = v * 16 + 4 * g;
            if (c >= p.vdim) continue;                 // vdim % 8 == 0: four columns at a time
            bf16 b[4] = {(bf16)(o[u][v][0] * f), (bf16)(o[u][v][1] * f), (bf16)(o[u][v][2] * f), (bf16)(o[u][v][3] * f)};
            *reinterpret_cast<pi_u32x2 *>(out + c) = __builtin_bit_cast(pi_u32x2, b);
        }
    }
}

template <int KS, int VT> int launch_expanded(const pi_latent_expanded * p, hipStream_t st) {
    const int n_qt = (p->T + kXTok - 1) / kXTok, hp = (p->n_head + 7) / 8;
    hipLaunchKernelGGL((latent_expanded_attn_kernel<KS, VT>), dim3(8 * hp * n_qt), dim3(256), 0, st, *p, n_qt, hp);
    return pi::check_launch("pi_k_latent_attn_expanded");
}

template <typename ST>
__global__ void latent_shift_kernel(ST * __restrict__ cache, int kd, int rank_ld, int rot_dim, double base, const int32_t * __restrict__ delta) {
    const int c = blockIdx.x, d = delta[c];
    if (d == 0) return;
    for (int i = threadIdx.x; i < rot_dim / 2; i += blockDim.x) {
        double sn, cn;
        sincos((double)d * pow(base, -2.0 * (double)i / (double)rot_dim), &sn, &cn);
        ST * r = cache + (size_t)c * kd + rank_ld + 2 * i;
        const float u = from_st(r[0]), v = from_st(r[1]);
        r[0] = to_st<ST>(u * (float)cn - v * (float)sn);
        r[1] = to_st<ST>(v * (float)cn + u * (float)sn);
    }
}

size_t attn_lds(int rt, int kd) {
    const int R = 16 * rt, stride = kd * 2 + 16;
    return (size_t)(R + kLaCells) * stride + 4 * (size_t)(R * (kLaCells + 1) + (R * (kLaCells + 1)) % 4) + 2 * (size_t)R * (kLaCells + 8) + 16 * (size_t)R;
}

template <int RT, int VT, int PF> int launch_attn(const pi_latent_attn * p, int by_item, hipStream_t st) {
    const size_t lds = attn_lds(RT, p->kd);
    static bool raised = false;
    if (!raised) {
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_attn_bf16_kernel<RT, VT, PF>), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
        raised = true;
    }
    hipLaunchKernelGGL((latent_attn_bf16_kernel<RT, VT, PF>), dim3(p->n_work, p->n_parts), dim3(256), lds, st, *p, by_item);
    return pi::check_launch("pi_k_latent_attn");
}

}  // namespace

extern "C" {

int pi_k_latent_prep(int type, const pi_latent_prep * p, pi_stream_t stream) {
    if (!p || !p->z || !p->q_un || !p->q_lat || !p->cs || p->T <= 0 || p->n_head <= 0 || p->dim <= 0 || p->rot_dim <= 0 || p->rot_dim % 2 || p->kv_rank <= 0 ||
        p->dim_ld < p->dim || p->rank_ld < p->kv_rank || p->kd < p->rank_ld + p->rot_dim || (p->cache && (!p->cell || !p->norm_w)) ||
        p->ldz < p->n_head * (p->dim + p->rot_dim) + (p->cache ? p->kv_rank + p->rot_dim : 0))
        return pi::fail(PI_E_ARG, "pi_k_latent_prep: bad arguments");
    int n_q = (p->n_head * (p->dim + p->rot_dim / 2) + 1023) / 1024;
    if (n_q > 64) n_q = 64;
    const dim3 grid(p->T, n_q + (p->cache ? 1 : 0));
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(latent_prep_kernel<bf16>, grid, dim3(256), 0, (hipStream_t)stream, *p);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(latent_prep_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, *p);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_latent_prep: type");
    return pi::check_launch("pi_k_latent_prep");
}

int pi_k_latent_attn_rows(int type) { return type == PI_TYPE_BF16 ? kLaRows : 1; }

int pi_k_latent_attn_supported(int type, int rank_ld, int kd) {
    if (rank_ld <= 0 || rank_ld % 32 || kd % 32 || kd <= rank_ld || rank_ld > 1024) return 0;
    return type == PI_TYPE_F32 ? kd <= 8192 : (kd <= 1152 && attn_lds(kLaRows / 16, kd) <= 160 * 1024);
}

size_t pi_k_latent_attn_scratch_floats(int rows, int rank_ld, int n_parts) { return n_parts > 1 ? (size_t)rows * n_parts * (rank_ld + 2) : 0; }

static int attn_bf16(const pi_latent_attn * p, int by_item, hipStream_t st) {
    if (p->rank_ld <= 128 && p->kd <= 256) return launch_attn<2, 2, 4>(p, by_item, st);
    if (p->rank_ld <= 256 && p->kd <= 384) return launch_attn<2, 4, 6>(p, by_item, st);
    if (p->rank_ld <= 512 && p->kd <= 640) return launch_attn<2, 8, 10>(p, by_item, st);
    return launch_attn<2, 16, 18>(p, by_item, st);
}

static int attn_check(int type, const pi_latent_attn * p) {
    if (!p || !p->q_lat || !p->cache || !p->lists || !p->work || !p->n_vis || !p->sink || !p->out_lat || p->n_work <= 0 || p->T <= 0 || p->n_head <= 0 ||
        p->n_parts <= 0 || p->n_parts > 65535 || (p->n_parts > 1 && !p->scratch) || p->kv_rank > p->rank_ld)
        return pi::fail(PI_E_ARG, "pi_k_latent_attn: bad arguments");
    if (!pi_k_latent_attn_supported(type, p->rank_ld, p->kd)) return pi::fail(PI_E_UNSUPPORTED, "pi_k_latent_attn: latent sizes (rank up to 1024)");
    return PI_OK;
}

int pi_k_latent_attn_parts(const pi_latent_attn * p, pi_stream_t stream) {
    const int rc = attn_check(PI_TYPE_BF16, p);
    return rc != PI_OK ? rc : attn_bf16(p, 0, (hipStream_t)stream);
}

int pi_k_latent_attn(int type, const pi_latent_attn * p, pi_stream_t stream) {
    int rc = attn_check(type, p);
    if (rc != PI_OK) return rc;
    hipStream_t st = (hipStream_t)stream;
    if (type == PI_TYPE_F32) {
        hipLaunchKernelGGL(latent_attn_f32_kernel, dim3(p->T * p->n_head), dim3(256), sizeof(float) * (p->kd + kLfCells) + sizeof(int) * kLfCells, st, *p);
        return pi::check_launch("pi_k_latent_attn");
    }
    rc = attn_bf16(p, 1, st);
    if (rc != PI_OK || p->n_parts == 1) return rc;
    hipLaunchKernelGGL(latent_merge_kernel, dim3(p->n_work * kLaRows), dim3(128), 0, st, *p);
    return pi::check_launch("pi_k_latent_attn merge");
}

int pi_k_latent_expanded_supported(int dim, int rot_dim, int vdim) {
    return dim > 0 && rot_dim > 0 && vdim > 0 && dim % 8 == 0 && rot_dim % 8 == 0 && vdim % 8 == 0 && dim + rot_dim <= 256 && vdim <= 128;
}

int pi_k_latent_attn_expanded(const pi_latent_expanded * p, pi_stream_t stream) {
    if (!p || !p->q_un || !p->q_lat || !p->keys || !p->values || !p->cache || !p->list || !p->n_vis || !p->sink || !p->att || p->T <= 0 || p->tok0 < 0 || p->n_head <= 0 ||
        p->dim_ld < p->dim || p->dim_ld % 8 || p->kd % 8 || p->rank_ld % 8 || p->kd < p->rank_ld + p->rot_dim || p->ld_att % 8 || p->ld_att < p->n_head * p->vdim)
        return pi::fail(PI_E_ARG, "pi_k_latent_attn_expanded: bad arguments");
    if (!pi_k_latent_expanded_supported(p->dim, p->rot_dim, p->vdim)) return pi::fail(PI_E_UNSUPPORTED, "pi_k_latent_attn_expanded: head sizes");
    const int dk = p->dim + p->rot_dim;
    hipStream_t st = (hipStream_t)stream;
    if (p->vdim <= 64) return dk <= 128 ? launch_expanded<4, 4>(p, st) : dk <= 192 ? launch_expanded<6, 4>(p, st) : launch_expanded<8, 4>(p, st);
    return dk <= 128 ? launch_expanded<4, 8>(p, st) : dk <= 192 ? launch_expanded<6, 8>(p, st) : launch_expanded<8, 8>(p, st);
}

int pi_k_latent_shift(int type, void * cache, int n_cells, int kd, int rank_ld, int rot_dim, double base, const int32_t * delta, pi_stream_t stream) {
    if (!cache || !delta || n_cells <= 0 || kd <= 0 || rank_ld < 0 || rot_dim <= 0 || rot_dim % 2 || rank_ld + rot_dim > kd) return pi::fail(PI_E_ARG, "pi_k_latent_shift: bad arguments");
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(latent_shift_kernel<bf16>, dim3(n_cells), dim3(64), 0, (hipStream_t)stream, (bf16 *)cache, kd, rank_ld, rot_dim, base, delta);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(latent_shift_kernel<float>, dim3(n_cells), dim3(64), 0, (hipStream_t)stream, (float *)cache, kd, rank_ld, rot_dim, base, delta);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_latent_shift: type");
    return pi::check_launch("pi_k_latent_shift");
}

}  // extern "C"
