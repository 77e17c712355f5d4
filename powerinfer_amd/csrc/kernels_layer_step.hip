// Steps of up to 16 tokens of a model described layer by layer (bf16), as few launches as its dependencies allow: everything behind
// the joint projection (absorbed queries, rotation, cells, expert choice) in one, the merge of a split attention with the value
// expansion together with the experts' first matrices in one, and one for what closes a layer - attention output and the experts' second
// matrices as a single long dot product per row, plus the residual.
#include "layer_types.hpp"
#include "mixers.hpp"
#include "route.hpp"

namespace {

constexpr int kRopePerWg = 512;           // rotated query pairs of a workgroup
// Behind the joint projection: per head the absorbed query (64 latent rows a workgroup), per token the rotated query parts, the cell,
// and the expert choice.
__global__ __launch_bounds__(256) void latent_step_kernel(pi_latent_prep p, const uint16_t * __restrict__ uk_t, RouteArgs r, int n_absorb) {
    extern __shared__ __align__(16) float sm[];
    __shared__ double red[4];
    const int hd = p.dim + p.rot_dim, half = p.rot_dim / 2, tid = threadIdx.x;
    int b = blockIdx.x;
    if (b < n_absorb) {                                       // a head's query in latent coordinates: 64 rows of W_uk^T against the step's tokens
        const int tiles = (p.kv_rank + 63) / 64, h = b / tiles, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
        const int row0 = (b % tiles) * 64 + wave * 16;
        if (row0 >= p.kv_rank) return;
        const uint16_t * W = uk_t + ((size_t)h * p.kv_rank + min(row0 + i, p.kv_rank - 1)) * p.dim_ld + g * 8;
        const float * z = p.z + (size_t)min(i, p.T - 1) * p.ldz + h * hd;
        const bool whole = p.dim % 8 == 0 && hd % 4 == 0 && p.ldz % 4 == 0;        // eight columns are two 16-byte loads
        pi_f4 acc = pi_f4{0, 0, 0, 0};
        for (int k0 = 0; k0 < p.dim_ld; k0 += 128) {          // four steps requested together, unguarded; what is past the end is zeroed
            pi_u32x4 w[4];
            float q[4][8];
#pragma unroll
            for (int s = 0; s < 4; ++s) w[s] = pi_ld16(W + min(k0 + s * 32, p.dim_ld - 32));
            if (whole) {
#pragma unroll
                for (int s = 0; s < 4; ++s) {
                    const float4 * zp = reinterpret_cast<const float4 *>(z + min(k0 + s * 32 + g * 8, p.dim - 8));
                    const float4 a = zp[0], c = zp[1];
                    q[s][0] = a.x; q[s][1] = a.y; q[s][2] = a.z; q[s][3] = a.w; q[s][4] = c.x; q[s][5] = c.y; q[s][6] = c.z; q[s][7] = c.w;
                }
            } else {
#pragma unroll
                for (int s = 0; s < 4; ++s)
#pragma unroll
                    for (int j = 0; j < 8; ++j) q[s][j] = z[min(k0 + s * 32 + g * 8 + j, p.dim - 1)];
            }
#pragma unroll
            for (int s = 0; s < 4; ++s) {
                bf16 v[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) v[j] = (bf16)(k0 + s * 32 + g * 8 + j < p.dim ? q[s][j] : 0.0f);
                acc = mma16<bf16>(w[s], __builtin_bit_cast(pi_u32x4, v), acc);
            }
        }
        if (i >= p.T) return;
        bf16 * o = (bf16 *)p.q_lat + ((size_t)i * p.n_head + h) * p.kd + row0 + 4 * g;
#pragma unroll
        for (int k = 0; k < 4; ++k) if (row0 + 4 * g + k < p.kv_rank) o[k] = (bf16)acc[k];
        return;
    }
    b -= n_absorb;
    const int n_rope = (p.n_head * half + kRopePerWg - 1) / kRopePerWg, kinds = n_rope + (p.cache ? 1 : 0) + (r.ids ? 1 : 0), t = b / kinds, what = b % kinds;
    const float * z = p.z + (size_t)t * p.ldz;
    const float2 * cs = (const float2 *)p.cs + (size_t)t * half;
    if (what < n_rope) {                                      // rotated query parts
        float u[kRopePerWg / 256], v[kRopePerWg / 256];
        const int e0 = what * kRopePerWg + tid, last = p.n_head * half - 1;
#pragma unroll
        for (int k = 0; k < kRopePerWg / 256; ++k) {
            const int e = min(e0 + k * 256, last), h = e / half, i = e - h * half;
            u[k] = z[h * hd + p.dim + 2 * i]; v[k] = z[h * hd + p.dim + 2 * i + 1];
        }
#pragma unroll
        for (int k = 0; k < kRopePerWg / 256; ++k) {
            const int e = e0 + k * 256, h = e / half, i = e - h * half;
            if (e > last) continue;
            bf16 * o = (bf16 *)p.q_lat + ((size_t)t * p.n_head + h) * p.kd + p.rank_ld + 2 * i;
            o[0] = (bf16)(u[k] * cs[i].x - v[k] * cs[i].y);
            o[1] = (bf16)(v[k] * cs[i].x + u[k] * cs[i].y);
        }
    } else if (what == n_rope && p.cache) {                        // the token's cell
        const float * c = z + p.n_head * hd;
        bf16 * cell = (bf16 *)p.cache + (size_t)p.cell[t] * p.kd;
        double s = 0.0;
        for (int i = tid; i < p.kv_rank; i += 256) { const float v = c[i]; s += (double)v * (double)v; }
        s = block_sum_f64(s, red);
        const float sc = pi_inv_sqrt((float)(s / p.kv_rank) + p.eps);
        for (int i = tid; i < p.kv_rank; i += 256) cell[i] = (bf16)(c[i] * sc * p.norm_w[i]);
        for (int i = tid; i < half; i += 256) {
            const float u = c[p.kv_rank + 2 * i], v = c[p.kv_rank + 2 * i + 1];
            cell[p.rank_ld + 2 * i] = (bf16)(u * cs[i].x - v * cs[i].y);
            cell[p.rank_ld + 2 * i + 1] = (bf16)(v * cs[i].x + u * cs[i].y);
        }
    } else {                                                  // the token's experts
        route_token(r, t, sm);
    }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// the parts of a split attention merged (fixed order, the sink in the denominator) and the head's values expanded from the result:
// a workgroup owns 64 value rows of one head, for all tokens of the step
// ---------------------------------------------------------------------------------------------------------------------------------
__host__ __device__ inline size_t value_lds_bytes(int T, int rank_ld, int n_parts) {
    return (size_t)T * (rank_ld + 8) * 2 + sizeof(float) * (((size_t)T * n_parts + 3) / 4 * 4 + 4 * (size_t)rank_ld);
}
__device__ void latent_value(const pi_latent_attn & p, const uint16_t * __restrict__ uv, int vdim, bf16 * __restrict__ att, int ld_att, int h, int rt, unsigned char * smem) {
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
    const int ld = p.rank_ld + 8;
    bf16 * ol = reinterpret_cast<bf16 *>(smem);               // [T][ld]
    float * f = reinterpret_cast<float *>(ol + p.T * ld);     // [T][n_parts] factor of each part
    float * ws = f + (p.T * p.n_parts + 3) / 4 * 4;           // [4][rank_ld] the waves' sums
    const int row0 = rt * 64 + wave * 16;
    // the value matrix does not depend on the attention: its first fragments are requested ahead of everything else
    const uint16_t * W = uv + ((size_t)h * vdim + min(row0 + i, vdim - 1)) * p.rank_ld + g * 8;
    pi_u32x4 w0[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) w0[k] = k * 32 < p.rank_ld ? pi_ld_stream(W + k * 32) : pi_u32x4{0, 0, 0, 0};
    if (p.n_parts == 1) {
        for (int c = tid; c < p.T * (p.rank_ld / 8); c += 256) {
            const int t = c / (p.rank_ld / 8), k = (c % (p.rank_ld / 8)) * 8;
            *reinterpret_cast<pi_u32x4 *>(ol + t * ld + k) = pi_ld16((const uint16_t *)p.out_lat + ((size_t)t * p.n_head + h) * p.rank_ld + k);
        }
    } else {
        const float * ml = p.scratch + (size_t)p.T * p.n_head * p.n_parts * p.rank_ld;
        const float sink = p.sink[h];
        for (int t = wave; t < p.T; t += 4) {                 // a wave per token: n_parts <= 64 lanes
            const float2 v = lane < p.n_parts ? reinterpret_cast<const float2 *>(ml)[((size_t)t * p.n_head + h) * p.n_parts + lane] : make_float2(-INFINITY, 0.0f);
            const float m = fmaxf(pi_wave_max(v.x), sink);
            const float e = v.x == -INFINITY ? 0.0f : expf(v.x - m);
            const float l = pi_wave_sum(e * v.y) + expf(sink - m);
            if (lane < p.n_parts) f[t * p.n_parts + lane] = e / l;
        }
        __syncthreads();
        for (int t = 0; t < p.T; ++t) {                       // a wave takes every fourth part, a lane four columns of a 256-column piece
            const float * a = p.scratch + ((size_t)t * p.n_head + h) * p.n_parts * p.rank_ld;
            for (int c = lane * 4; c < p.rank_ld; c += 256) {
                float4 s = make_float4(0, 0, 0, 0);
                for (int q0 = wave; q0 < p.n_parts; q0 += 32) {
                    float4 v[8];
#pragma unroll
                    for (int u = 0; u < 8; ++u) v[u] = *reinterpret_cast<const float4 *>(a + (size_t)min(q0 + 4 * u, p.n_parts - 1) * p.rank_ld + c);
#pragma unroll
                    for (int u = 0; u < 8; ++u) {
                        const float w = q0 + 4 * u < p.n_parts ? f[t * p.n_parts + q0 + 4 * u] : 0.0f;
                        s.x = fmaf(w, v[u].x, s.x); s.y = fmaf(w, v[u].y, s.y); s.z = fmaf(w, v[u].z, s.z); s.w = fmaf(w, v[u].w, s.w);
                    }
                }
                *reinterpret_cast<float4 *>(ws + wave * p.rank_ld + c) = s;
            }
            __syncthreads();
            for (int c = tid; c < p.rank_ld; c += 256) ol[t * ld + c] = (bf16)(ws[c] + ws[p.rank_ld + c] + ws[2 * p.rank_ld + c] + ws[3 * p.rank_ld + c]);
            __syncthreads();
        }
    }
    __syncthreads();
    if (row0 >= vdim) return;
    const bf16 * x = ol + min(i, p.T - 1) * ld + g * 8;
    pi_f4 acc = pi_f4{0, 0, 0, 0};
#pragma unroll
    for (int k = 0; k < 8; ++k)
        if (k * 32 < p.rank_ld) acc = mma16<bf16>(w0[k], *reinterpret_cast<const pi_u32x4 *>(x + k * 32), acc);
    for (int k0 = 256; k0 < p.rank_ld; k0 += 256) {
#pragma unroll
        for (int k = 0; k < 8; ++k) w0[k] = k0 + k * 32 < p.rank_ld ? pi_ld_stream(W + k0 + k * 32) : pi_u32x4{0, 0, 0, 0};
#pragma unroll
        for (int k = 0; k < 8; ++k) if (k0 + k * 32 < p.rank_ld) acc = mma16<bf16>(w0[k], *reinterpret_cast<const pi_u32x4 *>(x + k0 + k * 32), acc);
    }
    if (i >= p.T) return;
    bf16 * o = att + (size_t)i * ld_att + h * vdim + row0 + 4 * g;
#pragma unroll
    for (int k = 0; k < 4; ++k) if (row0 + 4 * g + k < vdim) o[k] = (bf16)acc[k];
}

// ---------------------------------------------------------------------------------------------------------------------------------
// Weight rows streamed past the step's tokens: a wave reads 2 rows x 512 B per load (16 rows x 256 columns in eight), passes them
// through its own LDS buffer into the matrix cores' operand layout (as gemm_t16_lds_kernel does) and multiplies.  Columns beyond the
// end of a row are not read (the last piece of the row is read again) and meet zeros.
// ---------------------------------------------------------------------------------------------------------------------------------
constexpr int kWsStride = 512 + 16;
struct WaveStream {
    unsigned char * tile;
    int lane, i, g, lr, lc;
    __device__ __forceinline__ WaveStream(unsigned char * t) : tile(t), lane(threadIdx.x & 63), i(lane & 15), g(lane >> 4), lr(lane >> 5), lc(lane & 31) {}
    // rows row0 .. row0 + 15 (clamped to rows), columns c0 .. c0 + 255 of a matrix of `cols` (a multiple of 32) columns
    __device__ __forceinline__ void load(pi_u32x4 (&ld)[8], const bf16 * W, size_t ldw, int row0, int rows, int c0, int cols) const {
        const int c = min(c0 + lc * 8, cols - 8);
#pragma unroll
        for (int j = 0; j < 8; ++j) ld[j] = pi_ld_stream(W + (size_t)min(row0 + 2 * j + lr, rows - 1) * ldw + c);
    }
    __device__ __forceinline__ void multiply(const pi_u32x4 (&ld)[8], const pi_u32x4 (&b)[8], pi_f4 & acc) const {
#pragma unroll
        for (int j = 0; j < 8; ++j) *reinterpret_cast<pi_u32x4 *>(tile + (2 * j + lr) * kWsStride + lc * 16) = ld[j];
#pragma unroll
        for (int st = 0; st < 8; ++st) acc = mma16<bf16>(*reinterpret_cast<const pi_u32x4 *>(tile + i * kWsStride + (4 * st + g) * 16), b[st], acc);
    }
};

// The step's distinct experts in LDS: expert[k] in order of first appearance, slot[k][t] = token t's pair with it or -1.
constexpr int kStepPairs = 256, kStepExperts = 2048;
struct StepExperts {
    int expert[kStepPairs], rank[kStepPairs], sred[16];
    int16_t slot[kStepPairs][16];
};
// first: kStepExperts ints of LDS
__device__ int step_experts(StepExperts & s, int * first, const int32_t * __restrict__ ids, int n, int top, int E) {
    const int tid = threadIdx.x, e = tid < n ? ids[tid] : 0;
    for (int k = tid; k < E; k += blockDim.x) first[k] = n;
    for (int k = tid; k < n * 8; k += blockDim.x) reinterpret_cast<int *>(s.slot)[k] = -1;
    __syncthreads();
    if (tid < n) atomicMin(&first[e], tid);
    __syncthreads();
    const int lead = tid < n ? first[e] : -1, own = lead == tid ? 1 : 0;
    int total;
    const int rank = block_exclusive_scan_i32(own, &total, s.sred);
    if (own) { s.expert[rank] = e; s.rank[tid] = rank; }
    __syncthreads();
    if (tid < n) s.slot[s.rank[lead]][tid / top] = (int16_t)tid;
    __syncthreads();
    return total;
}

// ---------------------------------------------------------------------------------------------------------------------------------
// first matrices of the step's experts: workgroup (row tile, pair) works for the pair's expert if no earlier pair has the same one, for
// every token that chose it; act[pair] = weight * relu(z)^2, or (glu: rows of gate and up in turn, ff of both together) weight * clamped GLU (weigh_input:
// the clamped GLU of the weighted rows)
// ---------------------------------------------------------------------------------------------------------------------------------
struct ExpertUp { const bf16 * up; int ff, cols; const bf16 * x_ol; const int32_t * ids; const float * weights; int T, top; bf16 * act; int ld_act; int glu = 0; float limit = 0.0f, gain = 0.0f, one = 1.0f; int weigh_input = 0; };
constexpr int kUpLds = 4 * 16 * kWsStride;
__device__ void expert_up(const ExpertUp & a, int tile, int p, unsigned char * smem) {
    constexpr int NW = 4;
    unsigned char (*tiles)[16 * kWsStride] = reinterpret_cast<unsigned char (*)[16 * kWsStride]>(smem);
    const bf16 * up = a.up, * x_ol = a.x_ol; const int32_t * ids = a.ids;
    const int ff = a.ff, cols = a.cols, T = a.T, top = a.top;
    const int e = ids[p], tid = threadIdx.x, wave = tid >> 6;
    if (T > 1 && __syncthreads_or(tid < p && ids[tid] == e)) return;            // p < 256: checked by the launcher
    const WaveStream ws(tiles[wave]);
    const int row0 = tile * 16, n_ss = (cols + 255) / 256;
    const bf16 * W = up + (size_t)e * ff * cols;
    pi_u32x4 ld[2][8];
    pi_f4 acc = pi_f4{0, 0, 0, 0};
    if (wave < n_ss) ws.load(ld[0], W, cols, row0, ff, wave * 256, cols);
    if (wave + NW < n_ss) ws.load(ld[1], W, cols, row0, ff, (wave + NW) * 256, cols);
    for (int s0 = wave; s0 < n_ss; s0 += 2 * NW) {
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            const int ss = s0 + b * NW;
            if (ss < n_ss) {
                pi_u32x4 x[8];
#pragma unroll
                for (int st = 0; st < 8; ++st) x[st] = ss * 256 + st * 32 < cols ? pi_ld16(x_ol + ((size_t)(ss * 8 + st) * 64 + ws.g * 16 + ws.i) * 8) : pi_u32x4{0, 0, 0, 0};
                ws.multiply(ld[b], x, acc);
                if (ss + 2 * NW < n_ss) ws.load(ld[b], W, cols, row0, ff, (ss + 2 * NW) * 256, cols);
            }
        }
    }
    float (*cs)[17] = reinterpret_cast<float (*)[17]>(tiles[wave]);
#pragma unroll
    for (int r = 0; r < 4; ++r) cs[4 * ws.g + r][ws.i] = acc[r];
    __syncthreads();
    if (tid >= 256) return;
    const int rr = tid >> 4, t = tid & 15, row = row0 + rr;
    if (row >= ff || t >= T) return;
    if (a.glu) {
        if (rr & 1) return;
        float g = 0.0f, u = 0.0f;
#pragma unroll
        for (int w = 0; w < NW; ++w) { g += reinterpret_cast<float (*)[17]>(tiles[w])[rr][t]; u += reinterpret_cast<float (*)[17]>(tiles[w])[rr + 1][t]; }
        for (int k = 0; k < top; ++k) {
            if (ids[t * top + k] != e) continue;
            const float w = a.weights[t * top + k];
            const float y = a.weigh_input ? clamped_glu(w * g, w * u, a.limit, a.gain, a.one) : w * clamped_glu(g, u, a.limit, a.gain, a.one);
            a.act[(size_t)(t * top + k) * a.ld_act + row / 2] = (bf16)y;
        }
        return;
    }
    float v = 0.0f;
#pragma unroll
    for (int w = 0; w < NW; ++w) v += reinterpret_cast<float (*)[17]>(tiles[w])[rr][t];
    v = fmaxf(v, 0.0f);
    for (int k = 0; k < top; ++k)
        if (ids[t * top + k] == e) a.act[(size_t)(t * top + k) * a.ld_act + row] = (bf16)(a.weights[t * top + k] * v * v);
}

// both in one launch: the value expansion of the attention branch hides behind the experts' weights
__global__ __launch_bounds__(256) void value_and_up_kernel(pi_latent_attn p, const uint16_t * __restrict__ uv, int vdim, bf16 * __restrict__ att, int ld_att, int n_rt, int n_value,
                                                           ExpertUp u, int n_up_tiles) {
    extern __shared__ __align__(16) unsigned char smem[];
    const int b = blockIdx.x;
    if (b < n_value) latent_value(p, uv, vdim, att, ld_att, b / n_rt, b % n_rt, smem);
    else expert_up(u, (b - n_value) % n_up_tiles, (b - n_value) / n_up_tiles, smem);
}

// the merge of a split grouped-query attention (four rows a workgroup) and the gated norm of a linear attention (a token or four heads a
// workgroup) beside the experts' first matrices
__global__ __launch_bounds__(256) void mix_and_up_kernel(pi_gqa_attn p, pi_gate_norm gn, int n_merge, int n_gate, ExpertUp u, int n_up_tiles) {
    extern __shared__ __align__(16) unsigned char smem[];
    int b = blockIdx.x;
    if (b < n_gate) { gate_norm_block<bf16>(gn, b, reinterpret_cast<double *>(smem)); return; }
    b -= n_gate;
    if (b < n_merge) {
        const int r4 = gqa_rows(p.wide) / 4;
        const int n = p.all_values ? p.n_kv * p.n_kv : p.n_kv;
        gqa_merge_row(p, b / r4 / n, b / r4 % n, (b % r4) * 4 + (threadIdx.x >> 6));
        return;
    }
    expert_up(u, (b - n_merge) % n_up_tiles, (b - n_merge) / n_up_tiles, smem);
}

// ---------------------------------------------------------------------------------------------------------------------------------
// what closes a layer: out[t] = x[t] + (W_o att[t] + sum over the token's experts of W_down[e] act[pair]), 16 rows a workgroup (or, what closes a
// sublayer in front of its norm: out[t] = alpha x[t] + gate * W att[t]).  The
// pieces of 256 columns of W_o and of every expert of the step form one list that the waves take in turn.
// ---------------------------------------------------------------------------------------------------------------------------------
template <int NW>
__global__ __launch_bounds__(64 * NW) void layer_out_step_kernel(pi_layer_out a) {
    __shared__ __align__(16) unsigned char tiles[NW][16 * kWsStride];
    __shared__ StepExperts se;
    __shared__ int first[kStepExperts];
    // (eight waves: the workgroup's LDS exceeds half a compute unit's, so that no two share one while others idle)
    static_assert(NW < 8 || sizeof(tiles) + sizeof(se) + sizeof(first) > 80 * 1024, "one workgroup per compute unit");
    const int tid = threadIdx.x, wave = tid >> 6;
    const WaveStream ws(tiles[wave]);
    const int row0 = blockIdx.x * 16, n_o = a.wo ? (a.ld_att + 255) / 256 : 0, n_e = a.ids ? (a.ld_act + 255) / 256 : 1;
    const int tok = min(ws.i, a.T - 1);
    const bf16 * wo = (const bf16 *)a.wo, * down = (const bf16 *)a.down;
    pi_u32x4 ld[2][8];
    pi_f4 acc = pi_f4{0, 0, 0, 0};
    auto load = [&](pi_u32x4 (&l)[8], int ss) {
        if (ss < n_o) { ws.load(l, wo, a.ld_att, row0, a.rows, ss * 256, a.ld_att); return; }
        const int k = (ss - n_o) / n_e, c = (ss - n_o) % n_e;
        ws.load(l, down + (size_t)se.expert[k] * a.rows * a.ld_act, a.ld_act, row0, a.rows, c * 256, a.ld_act);
    };
    // the attention's pieces are requested before the experts are known
    if (wave < n_o) load(ld[0], wave);
    if (wave + NW < n_o) load(ld[1], wave + NW);
    const int n_exp = a.ids ? step_experts(se, first, a.ids, a.T * a.top, a.top, a.n_expert) : 0, n_ss = n_o + n_exp * n_e;
    if (wave >= n_o && wave < n_ss) load(ld[0], wave);
    if (wave + NW >= n_o && wave + NW < n_ss) load(ld[1], wave + NW);
    for (int s0 = wave; s0 < n_ss; s0 += 2 * NW) {
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            const int ss = s0 + b * NW;
            if (ss < n_ss) {
                const bool att = ss < n_o;
                const int k = att ? 0 : (ss - n_o) / n_e, c = (att ? ss : (ss - n_o) % n_e) * 256, cols = att ? a.ld_att : a.ld_act;
                const int pair = att ? 0 : se.slot[k][ws.i];
                const bf16 * xp = att ? (const bf16 *)a.att + (size_t)tok * a.ld_att : (const bf16 *)a.act + (size_t)max(pair, 0) * a.ld_act;
                pi_u32x4 x[8];
#pragma unroll
                for (int st = 0; st < 8; ++st) x[st] = c + st * 32 < cols && pair >= 0 ? pi_ld16(xp + c + st * 32 + ws.g * 8) : pi_u32x4{0, 0, 0, 0};
                ws.multiply(ld[b], x, acc);
                if (ss + 2 * NW < n_ss) load(ld[b], ss + 2 * NW);
            }
        }
    }
    float (*cs)[17] = reinterpret_cast<float (*)[17]>(tiles[wave]);
#pragma unroll
    for (int r = 0; r < 4; ++r) cs[4 * ws.g + r][ws.i] = acc[r];
    __syncthreads();
    if (tid >= 256) return;
    const int t = tid >> 4, row = row0 + (tid & 15);
    if (row >= a.rows || t >= a.T) return;
    float v = 0.0f;
#pragma unroll
    for (int w = 0; w < NW; ++w) v += reinterpret_cast<float (*)[17]>(tiles[w])[tid & 15][t];
    if (a.gate_z) v *= sigmoid_f32(a.gate_z[(size_t)t * a.ld_gate + a.off_gate + row] + a.gate_b[row]);
    const float x = a.x ? a.x[(size_t)t * a.rows + row] : 0.0f;
    v += a.scaled ? a.alpha * x : x;
    a.out[(size_t)t * a.rows + row] = v;
    if (a.keep) a.keep[(size_t)t * a.rows + row] = v;
}

}  // namespace

extern "C" {

int pi_k_layer_step_supported(int T, int n_expert, int n_top) { return T >= 1 && T <= kBtMaxT && n_expert <= kStepExperts && T * n_top <= kStepPairs; }

int pi_k_latent_step(const pi_latent_prep * p, const void * uk_t, const float * z_router, int n_expert, int n_top, int n_group, int n_keep, const float * bias,
                     int32_t * ids, float * weights, pi_stream_t stream) {
    if (!p || !p->z || !p->q_lat || !p->cs || !uk_t || p->T <= 0 || p->T > kBtMaxT || p->n_head <= 0 || p->dim <= 0 || p->dim_ld % 32 || p->dim_ld < p->dim || p->rot_dim <= 0 ||
        p->rot_dim % 2 || p->kv_rank <= 0 || p->rank_ld < p->kv_rank || p->kd < p->rank_ld + p->rot_dim || (p->cache && (!p->cell || !p->norm_w)) ||
        p->ldz < p->n_head * (p->dim + p->rot_dim) + (p->cache ? p->kv_rank + p->rot_dim : 0))
        return pi::fail(PI_E_ARG, "pi_k_latent_step: bad arguments");
    if (ids && (!z_router || !bias || !weights || n_expert <= 0 || n_expert > kStepExperts || n_group <= 0 || n_expert % n_group || n_keep <= 0 || n_keep > n_group || n_top <= 0 ||
                n_top > n_keep * (n_expert / n_group)))
        return pi::fail(PI_E_ARG, "pi_k_latent_step: bad routing arguments");
    const int n_absorb = p->n_head * ((p->kv_rank + 63) / 64), kinds = (p->n_head * (p->rot_dim / 2) + kRopePerWg - 1) / kRopePerWg + (p->cache ? 1 : 0) + (ids ? 1 : 0);
    hipLaunchKernelGGL(latent_step_kernel, dim3(n_absorb + p->T * kinds), dim3(256), ids ? route_lds_bytes(n_expert, n_group, n_top) : 0, (hipStream_t)stream, *p, (const uint16_t *)uk_t,
                       RouteArgs{z_router, n_expert, n_top, n_group, n_keep, bias, ids, weights}, n_absorb);
    return pi::check_launch("pi_k_latent_step");
}

int pi_k_value_up_step(const pi_latent_attn * p, const void * uv, int vdim, void * att, int ld_att, const void * up, int n_expert, int ff, int cols, const void * x_ol,
                       const int32_t * ids, const float * weights, int top, void * act, int ld_act, pi_stream_t stream) {
    if (!p || !uv || !att || p->T <= 0 || p->T > kBtMaxT || p->n_head <= 0 || vdim <= 0 || p->rank_ld <= 0 || p->rank_ld % 64 || p->rank_ld > 1024 || ld_att < p->n_head * vdim || !p->sink ||
        p->n_parts <= 0 || p->n_parts > 64 || (p->n_parts == 1 ? !p->out_lat : !p->scratch))
        return pi::fail(PI_E_ARG, "pi_k_value_up_step: bad arguments");
    if (ids && (!up || !x_ol || !weights || !act || n_expert <= 0 || ff <= 0 || cols <= 0 || cols % 32 || top <= 0 || p->T * top > kStepPairs || ld_act < ff))
        return pi::fail(PI_E_ARG, "pi_k_value_up_step: bad expert arguments");
    const int n_rt = (vdim + 63) / 64, n_value = p->n_head * n_rt, n_up_tiles = ids ? (ff + 15) / 16 : 1, n_up = ids ? n_up_tiles * p->T * top : 0;
    size_t lds = value_lds_bytes(p->T, p->rank_ld, p->n_parts);
    if (ids && lds < (size_t)kUpLds) lds = kUpLds;
    static bool raised = false;
    if (!raised) { PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&value_and_up_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024)); raised = true; }
    hipLaunchKernelGGL(value_and_up_kernel, dim3(n_value + n_up), dim3(256), lds, (hipStream_t)stream, *p, (const uint16_t *)uv, vdim, (bf16 *)att, ld_att, n_rt, n_value,
                       ExpertUp{(const bf16 *)up, ff, cols, (const bf16 *)x_ol, ids, weights, p->T, top, (bf16 *)act, ld_act}, n_up_tiles);
    return pi::check_launch("pi_k_value_up_step");
}

int pi_k_mix_up_step(const pi_gqa_attn * attn, const pi_gate_norm * gate, const void * up, int n_expert, int ff, int cols, float limit, float gain, const void * x_ol, int T,
                     const int32_t * ids, const float * weights, int top, void * act, int ld_act, pi_stream_t stream) {
    const pi_gqa_attn p = attn ? *attn : pi_gqa_attn{};
    const pi_gate_norm g = gate ? *gate : pi_gate_norm{};
    if (T <= 0 || T > kBtMaxT || (attn && (!p.att || !p.scratch || !p.work || p.n_parts <= 1 || p.n_parts > 64 || p.n_work <= 0 || p.n_kv <= 0 || p.n_head % p.n_kv || p.vdim <= 0 || p.hd < p.vdim)) ||
        (gate && (!gate_norm_ok(g) || g.T != T)))
        return pi::fail(PI_E_ARG, "pi_k_mix_up_step: bad arguments");
    if (ids && (!up || !x_ol || !weights || !act || n_expert <= 0 || ff <= 0 || cols <= 0 || cols % 32 || top <= 0 || T * top > kStepPairs || ld_act < ff))
        return pi::fail(PI_E_ARG, "pi_k_mix_up_step: bad expert arguments");
    const int n_merge = attn ? p.n_work * p.n_kv * (p.all_values ? p.n_kv : 1) * (gqa_rows(p.wide) / 4) : 0, n_gate = gate ? gate_norm_blocks(g) : 0, n_up_tiles = ids ? (2 * ff + 15) / 16 : 1, n_up = ids ? n_up_tiles * T * top : 0;
    if (n_merge + n_gate + n_up == 0) return PI_OK;
    ExpertUp u{(const bf16 *)up, 2 * ff, cols, (const bf16 *)x_ol, ids, weights, T, top, (bf16 *)act, ld_act};
    u.glu = 1; u.limit = limit; u.gain = gain;
    hipLaunchKernelGGL(mix_and_up_kernel, dim3(n_merge + n_gate + n_up), dim3(256), ids ? kUpLds : 256, (hipStream_t)stream, p, g, n_merge, n_gate, u, n_up_tiles);
    return pi::check_launch("pi_k_mix_up_step");
}

int pi_k_expert_up_step(const void * up, int n_expert, int ff, int cols, float limit, float gain, int plain_up, int weigh_input, const void * x_ol, int T, const int32_t * ids,
                        const float * weights, int top, void * act, int ld_act, pi_stream_t stream) {
    if (!up || !x_ol || !ids || !weights || !act || T <= 0 || T > kBtMaxT || n_expert <= 0 || ff <= 0 || cols <= 0 || cols % 32 || top <= 0 || T * top > kStepPairs || ld_act < ff)
        return pi::fail(PI_E_ARG, "pi_k_expert_up_step: bad arguments");
    ExpertUp u{(const bf16 *)up, 2 * ff, cols, (const bf16 *)x_ol, ids, weights, T, top, (bf16 *)act, ld_act};
    u.glu = 1; u.limit = limit; u.gain = gain; u.one = plain_up ? 0.0f : 1.0f; u.weigh_input = weigh_input;
    const int tiles = (2 * ff + 15) / 16;
    hipLaunchKernelGGL(mix_and_up_kernel, dim3(tiles * T * top), dim3(256), kUpLds, (hipStream_t)stream, pi_gqa_attn{}, pi_gate_norm{}, 0, 0, u, tiles);
    return pi::check_launch("pi_k_expert_up_step");
}

int pi_k_layer_out_step(const pi_layer_out * a, pi_stream_t stream) {
    if (!a || (a->wo ? !a->att || a->ld_att <= 0 || a->ld_att % 32 : !a->ids) || !a->out || (a->gate_z && (!a->gate_b || a->off_gate < 0 || a->off_gate + a->rows > a->ld_gate)) || a->rows <= 0 || a->T <= 0 || a->T > kBtMaxT ||
        (a->ids && (!a->down || !a->act || a->ld_act <= 0 || a->ld_act % 32 || a->top <= 0 || a->T * a->top > kStepPairs || a->n_expert <= 0 || a->n_expert > kStepExperts)))
        return pi::fail(PI_E_ARG, "pi_k_layer_out_step: bad arguments");
    // eight waves a workgroup when every workgroup has a compute unit to itself, four (and several workgroups a unit) beyond
    const int n = (a->rows + 15) / 16;
    if (n <= pi::compute_units() ) hipLaunchKernelGGL(layer_out_step_kernel<8>, dim3(n), dim3(512), 0, (hipStream_t)stream, *a);
    else hipLaunchKernelGGL(layer_out_step_kernel<4>, dim3(n), dim3(256), 0, (hipStream_t)stream, *a);
    return pi::check_launch("pi_k_layer_out_step");
}

}  // extern "C"
