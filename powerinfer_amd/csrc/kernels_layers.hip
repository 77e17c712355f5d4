// Operators of the models that are described layer by layer, apart from attention: embedding + norm, the pair of norms of a parallel
// layer, grouped mat-muls (heads of a latent attention, experts), rotation angles, expert choice, and the sum that closes a layer.
// Templated on the storage of activations: bf16 (matrix cores on bf16 operands, fp32 accumulation) or fp32.
#include "gemm_tile.hpp"
#include "layer_types.hpp"
#include "mixers.hpp"
#include "route.hpp"

namespace {

// ---------------------------------------------------------------------------------------------------------------------------------
// norms
// ---------------------------------------------------------------------------------------------------------------------------------
// 1 / sqrt(mean(x^2) + eps) of a row the workgroup reads together (squares summed in fp64, fixed order)
template <typename LD> __device__ float row_rms_scale(int cols, float eps, double * red, LD && ld) {
    double s = 0.0;
    for (int i = threadIdx.x; i < cols; i += blockDim.x) { const float v = ld(i); s += (double)v * (double)v; }
    s = block_sum_f64(s, red);
    return pi_inv_sqrt((float)(s / cols) + eps);
}

__global__ __launch_bounds__(1024) void embed_norm_kernel(const uint16_t * __restrict__ table, int cols, const int32_t * __restrict__ tokens,
                                                          const float * __restrict__ w, float eps, float * __restrict__ x) {
    __shared__ double red[16];
    const uint16_t * row = table + (size_t)tokens[blockIdx.x] * cols;
    float * out = x + (size_t)blockIdx.x * cols;
    if (cols <= 8 * (int)blockDim.x) {              // row and weights requested together, kept in registers
        float v[8], wv[8];
        double s = 0.0;
#pragma unroll
        for (int k = 0; k < 8; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            v[k] = i < cols ? bf16_to_f32(row[i]) : 0.0f;
            wv[k] = i < cols ? w[i] : 0.0f;
            s += (double)v[k] * (double)v[k];
        }
        s = block_sum_f64(s, red);
        const float sc = pi_inv_sqrt((float)(s / cols) + eps);
#pragma unroll
        for (int k = 0; k < 8; ++k) { const int i = threadIdx.x + k * blockDim.x; if (i < cols) out[i] = v[k] * sc * wv[k]; }
        return;
    }
    const float sc = row_rms_scale(cols, eps, red, [&](int i) { return bf16_to_f32(row[i]); });
    for (int i = threadIdx.x; i < cols; i += blockDim.x) out[i] = bf16_to_f32(row[i]) * sc * w[i];
}

template <typename ST>
__global__ __launch_bounds__(1024) void norm_pair_kernel(const float * __restrict__ x, const int32_t * __restrict__ rows, int cols, float eps,
                                                        const float * __restrict__ wa, ST * __restrict__ out_a, const float * __restrict__ wb,
                                                        ST * __restrict__ out_b, int ld, int ol) {
    __shared__ double red[16];
    const float * xt = x + (size_t)(rows ? rows[blockIdx.x] : blockIdx.x) * cols;
    auto at = [&](int i) -> size_t { return ol ? pi_ol_index(blockIdx.x, i) : (size_t)blockIdx.x * ld + i; };
    if (cols <= 4 * (int)blockDim.x) {              // one memory round trip: the row and both weight vectors are requested together
        float xv[4], av[4], bv[4];
        double s = 0.0;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            xv[k] = i < cols ? xt[i] : 0.0f;
            av[k] = i < cols ? wa[i] : 0.0f;
            bv[k] = wb && i < cols ? wb[i] : 0.0f;
            s += (double)xv[k] * (double)xv[k];
        }
        s = block_sum_f64(s, red);
        const float sc = pi_inv_sqrt((float)(s / cols) + eps);
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            if (i < cols) {
                out_a[at(i)] = to_st<ST>(xv[k] * sc * av[k]);
                if (wb) out_b[at(i)] = to_st<ST>(xv[k] * sc * bv[k]);
            }
        }
        return;
    }
    const float sc = row_rms_scale(cols, eps, red, [&](int i) { return xt[i]; });
    for (int i = threadIdx.x; i < cols; i += blockDim.x) {
        const float v = xt[i] * sc;
        out_a[at(i)] = to_st<ST>(v * wa[i]);
        if (wb) out_b[at(i)] = to_st<ST>(v * wb[i]);
    }
}

__global__ __launch_bounds__(256) void embed_bigram_kernel(const uint16_t * __restrict__ table, int cols, const int32_t * __restrict__ tokens, int32_t * prev, float scale,
                                                           const uint16_t * __restrict__ bigram, int buckets, long long mul_prev, long long mul_cur, int carry,
                                                           float * __restrict__ x, float * __restrict__ x0) {
    const int t = blockIdx.x, tok = tokens[t], before = prev[t];
    const uint16_t * a = table + (size_t)tok * cols, * b = nullptr;
    if (bigram) b = bigram + (size_t)(before < 0 ? buckets : (int)(((long long)before * mul_prev + (long long)tok * mul_cur) % buckets)) * cols;
    float * o = x + (size_t)t * cols, * o0 = x0 ? x0 + (size_t)t * cols : nullptr;
    if ((cols & 7) == 0) {
        for (int i = threadIdx.x * 8; i < cols; i += 2048) {
            const pi_u32x4 u = pi_ld16(a + i), w = b ? pi_ld16(b + i) : pi_u32x4{0, 0, 0, 0};
            float v[8];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                v[2 * j] = __uint_as_float(u[j] << 16) * scale + __uint_as_float(w[j] << 16);
                v[2 * j + 1] = __uint_as_float(u[j] & 0xffff0000u) * scale + __uint_as_float(w[j] & 0xffff0000u);
            }
#pragma unroll
            for (int j = 0; j < 8; j += 4) {
                *reinterpret_cast<float4 *>(o + i + j) = make_float4(v[j], v[j + 1], v[j + 2], v[j + 3]);
                if (o0) *reinterpret_cast<float4 *>(o0 + i + j) = make_float4(v[j], v[j + 1], v[j + 2], v[j + 3]);
            }
        }
    } else {
        for (int i = threadIdx.x; i < cols; i += 256) {
            const float v = bf16_to_f32(a[i]) * scale + (b ? bf16_to_f32(b[i]) : 0.0f);
            o[i] = v;
            if (o0) o0[i] = v;
        }
    }
    if (carry) {
        __syncthreads();                               // every thread has read prev[t]
        if (threadIdx.x == 0) prev[t] = tok;
    }
}

// layer norm, two passes over the row (held in registers where it fits); x0, step: added to the residual stream first
template <typename ST>
__global__ __launch_bounds__(1024) void layer_norm_kernel(float * __restrict__ x, const int32_t * __restrict__ rows, int cols, float eps, const float * __restrict__ w,
                                                         const float * __restrict__ x0, const float * __restrict__ step, ST * __restrict__ out, int ld, int ol) {
    __shared__ double red[16];
    const size_t base = (size_t)(rows ? rows[blockIdx.x] : blockIdx.x) * cols;
    float * xt = x + base;
    auto at = [&](int i) -> size_t { return ol ? pi_ol_index(blockIdx.x, i) : (size_t)blockIdx.x * ld + i; };
    const bool adds = x0 || step;
    if (cols <= 4 * (int)blockDim.x) {
        float xv[4], wv[4];
        double s = 0.0;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            xv[k] = i < cols ? xt[i] : 0.0f;
            wv[k] = i < cols ? w[i] : 0.0f;
            if (x0 && i < cols) xv[k] += x0[base + i];
            if (step && i < cols) xv[k] += step[i];
            s += (double)xv[k];
        }
        const float mean = (float)(block_sum_f64(s, red) / cols);
        s = 0.0;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            if (i < cols) {
                if (adds) xt[i] = xv[k];
                xv[k] -= mean;
                s += (double)xv[k] * (double)xv[k];
            }
        }
        const float sc = pi_inv_sqrt((float)(block_sum_f64(s, red) / cols) + eps);
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int i = threadIdx.x + k * blockDim.x;
            if (i < cols) out[at(i)] = to_st<ST>(xv[k] * sc * wv[k]);
        }
        return;
    }
    double s = 0.0;
    for (int i = threadIdx.x; i < cols; i += blockDim.x) {
        float v = xt[i];
        if (x0) v += x0[base + i];
        if (step) v += step[i];
        if (adds) xt[i] = v;                           // (read back below by the thread that wrote it)
        s += (double)v;
    }
    const float mean = (float)(block_sum_f64(s, red) / cols);
    s = 0.0;
    for (int i = threadIdx.x; i < cols; i += blockDim.x) { const float v = xt[i] - mean; s += (double)v * (double)v; }
    const float sc = pi_inv_sqrt((float)(block_sum_f64(s, red) / cols) + eps);
    for (int i = threadIdx.x; i < cols; i += blockDim.x) out[at(i)] = to_st<ST>((xt[i] - mean) * sc * w[i]);
}

// what closes a sublayer whose norm comes after the sum (pi_res_norm): Q quads of columns per thread in registers, one trip over the row
template <typename ST, int Q>
__global__ void res_norm_kernel(pi_res_norm p) {
    __shared__ double red[16];
    const int t = blockIdx.x, tid = threadIdx.x, nt = blockDim.x;
    const size_t base = (size_t)t * p.cols;
    const float * gz = p.gate_z ? p.gate_z + (size_t)t * p.ld_gate + p.off_gate : nullptr;
    float v[Q][4], wv[Q][4];
    double s = 0.0;
    const bool quads = ((p.cols | p.ld_gate | p.off_gate) & 3) == 0;
    auto load = [&](const float * a, int c, float (&o)[4]) {      // columns c .. c + 3 of a row (past its end: zeros)
        if (quads && c < p.cols) { const float4 q = *reinterpret_cast<const float4 *>(a + c); o[0] = q.x; o[1] = q.y; o[2] = q.z; o[3] = q.w; }
        else for (int j = 0; j < 4; ++j) o[j] = c + j < p.cols ? a[c + j] : 0.0f;
    };
#pragma unroll
    for (int q = 0; q < Q; ++q) {
        const int c = (tid + q * nt) * 4;
        load(p.x + base, c, v[q]);
        if (p.w) load(p.w, c, wv[q]);
        if (p.mix) {
            float m[4];
            load(p.mix + base, c, m);
            if (gz) {
                float g[4], b[4];
                load(gz, c, g);
                load(p.gate_b, c, b);
#pragma unroll
                for (int j = 0; j < 4; ++j) m[j] *= sigmoid_f32(g[j] + b[j]);
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) v[q][j] = fmaf(p.alpha, v[q][j], m[j]);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) if (c + j < p.cols) s += (double)v[q][j] * (double)v[q][j];
    }
    float sc = 1.0f;
    if (p.w) sc = pi_inv_sqrt((float)(block_sum_f64(s, red) / p.cols) + p.eps);
    ST * h = (ST *)p.h;
#pragma unroll
    for (int q = 0; q < Q; ++q) {
        const int c = (tid + q * nt) * 4;
        if (c >= p.cols) break;
        if (p.w) {
#pragma unroll
            for (int j = 0; j < 4; ++j) v[q][j] *= sc * wv[q][j];
        }
        const bool whole = quads && c + 4 <= p.cols;
        store4(p.out + base + c, v[q], whole, p.cols - c);
        if (p.keep) store4(p.keep + base + c, v[q], whole, p.cols - c);
        if (h) {                                       // (four columns from a multiple of four on lie together in both layouts)
            ST * o = h + (p.ol ? pi_ol_index(t, c) : (size_t)t * p.ld + c);
            store4(o, v[q], ((uintptr_t)o & (4 * sizeof(ST) - 1)) == 0 && c + 4 <= p.cols, p.cols - c);
        }
    }
}
template <typename ST> int launch_res_norm(const pi_res_norm & p, hipStream_t st) {
    const int quads = (p.cols + 3) / 4;
    if (quads <= 256) hipLaunchKernelGGL((res_norm_kernel<ST, 1>), dim3(p.T), dim3(256), 0, st, p);
    else if (quads <= 512) hipLaunchKernelGGL((res_norm_kernel<ST, 1>), dim3(p.T), dim3(512), 0, st, p);
    else if (quads <= 1024) hipLaunchKernelGGL((res_norm_kernel<ST, 2>), dim3(p.T), dim3(512), 0, st, p);
    else if (quads <= 2048) hipLaunchKernelGGL((res_norm_kernel<ST, 4>), dim3(p.T), dim3(512), 0, st, p);
    else if (quads <= 8192) hipLaunchKernelGGL((res_norm_kernel<ST, 8>), dim3(p.T), dim3(1024), 0, st, p);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_res_norm: up to 32768 columns");
    return pi::check_launch("pi_k_res_norm");
}

template <typename ST>
__global__ __launch_bounds__(256) void ffn_front_kernel(pi_ffn_front f, const float * __restrict__ z, int ldz, int per) {
    extern __shared__ __align__(16) float sm[];
    front_block<ST>(f, z, ldz, blockIdx.x / per, blockIdx.x % per, sm);
}

// ---------------------------------------------------------------------------------------------------------------------------------
// grouped mat-mul.  A workgroup of four waves owns 64 rows of one group's matrix x 32 of the group's tokens; each wave holds 16 rows in
// the matrix cores' operand layout (lane l: row l % 16, eight consecutive columns 8 * (l / 16) of a 32-column step) against two token
// tiles.  fp32 storage runs the same steps on v_mfma_f32_16x16x4_f32, eight per 32 columns.
// ---------------------------------------------------------------------------------------------------------------------------------
template <typename ST>
__global__ __launch_bounds__(256) void group_gemm_kernel(pi_group_gemm g) {
    const int grp = blockIdx.z;
    const int lo = g.off ? g.off[grp] : 0, n = g.off ? g.off[grp + 1] - lo : g.T;
    const int t0 = blockIdx.y * 32;
    if (t0 >= n) return;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, q = lane >> 4;
    const int row0 = blockIdx.x * 64 + wave * 16;
    if (row0 >= g.rows) return;
    const uint16_t * W = (const uint16_t *)g.W + (size_t)grp * g.w_gs + (size_t)min(row0 + i, g.rows - 1) * g.ldw + q * 8;
    const ST * xb = (const ST *)g.x + (g.off ? 0 : (size_t)grp * g.x_gs);
    const ST * xp[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const int t = min(t0 + u * 16 + i, n - 1);
        const int xr = g.off ? (g.gather ? g.gather[lo + t] / g.gather_div : lo + t) : t;
        xp[u] = xb + (size_t)xr * g.ldx + q * 8;
    }
    pi_f4 acc[2] = {pi_f4{0, 0, 0, 0}, pi_f4{0, 0, 0, 0}};
    const bool two = t0 + 16 < n;
    for (int k = 0; k < g.cols; k += 32) {
        const Frag<ST> a = frag_weights<ST>(W + k);
        frag_mma(a, frag_load(xp[0] + k), acc[0]);
        if (two) frag_mma(a, frag_load(xp[1] + k), acc[1]);
    }
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const int t = t0 + u * 16 + i;
        if (t >= n) continue;
        const float alpha = g.pair_w ? g.alpha * g.pair_w[g.gather[lo + t]] : g.alpha, one = g.glu_plain_up ? 0.0f : 1.0f;
        const size_t yr = g.off ? (size_t)(lo + t) * g.ldy : (size_t)grp * g.y_gs + (size_t)t * g.ldy;
        if (g.glu) {                                   // rows in (gate, up) pairs: a lane holds two of them
#pragma unroll
            for (int r = 0; r < 4; r += 2) {
                const int row = row0 + 4 * q + r;
                if (row >= g.rows) continue;
                const float v = clamped_glu(acc[u][r] * alpha, acc[u][r + 1] * alpha, g.glu_limit, g.glu_gain, one);
                if (g.y_f32) ((float *)g.y)[yr + row / 2] = v;
                else ((ST *)g.y)[yr + row / 2] = to_st<ST>(v);
            }
            continue;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = row0 + 4 * q + r;
            if (row >= g.rows) continue;
            float v = acc[u][r] * alpha;
            if (g.relu2) { v = fmaxf(v, 0.0f); v *= v; }
            if (g.y_f32) ((float *)g.y)[yr + row] = v;
            else ((ST *)g.y)[yr + row] = to_st<ST>(v);
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// rotation angles: formed and reduced in fp64, so that the fp32 cosine and sine are right at any position
// ---------------------------------------------------------------------------------------------------------------------------------
__global__ void rope_angles_kernel(const int32_t * __restrict__ pos, int T, int dims, double base, float2 * __restrict__ cs) {
    const int half = dims / 2, idx = blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= T * half) return;
    const int t = idx / half, i = idx % half;
    double s, c;
    sincos((double)pos[t] * pow(base, -2.0 * (double)i / (double)dims), &s, &c);
    cs[idx] = make_float2((float)c, (float)s);
}

__global__ void rope_table_kernel(const int32_t * __restrict__ pos, int T, int half, const double * __restrict__ freq, double length, float2 * __restrict__ cs) {
    const int idx = blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= T * half) return;
    double s, c;
    sincos((double)pos[idx / half] * freq[idx % half], &s, &c);
    cs[idx] = make_float2((float)(length * c), (float)(length * s));
}

// expert choice, one workgroup per token
__global__ __launch_bounds__(256) void route_kernel(RouteArgs r) {
    extern __shared__ __align__(16) float sm[];
    route_token(r, blockIdx.x, sm);
}

// Pairs in expert order, one workgroup with the experts' counters in LDS: counts, their prefix sums, places.  The order of the pairs
// within an expert is free (every row of the grouped products is computed on its own).  tiles (optional): {expert, first place} of
// every group of up to tile_n pairs of one expert, n_tiles of them - the token tiles of the grouped products.
__global__ __launch_bounds__(1024) void moe_sort_kernel(const int32_t * __restrict__ ids, int n, int E, int32_t * __restrict__ off, int32_t * __restrict__ perm,
                                                        int32_t * __restrict__ inv, int tile_n, int2 * __restrict__ tiles, int32_t * __restrict__ n_tiles) {
    extern __shared__ int cnt[];
    __shared__ int sred[16];
    for (int e = threadIdx.x; e < E; e += 1024) cnt[e] = 0;
    __syncthreads();
    for (int p = threadIdx.x; p < n; p += 1024) atomicAdd(&cnt[ids[p]], 1);
    __syncthreads();
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < E; e0 += 1024) {
        const int e = e0 + threadIdx.x, c = e < E ? cnt[e] : 0;
        int tot, ttot;
        const int at = base + block_exclusive_scan_i32(c, &tot, sred);
        const int nt = tiles ? (c + tile_n - 1) / tile_n : 0;
        const int ta = tbase + block_exclusive_scan_i32(nt, &ttot, sred);
        if (e < E) {
            off[e] = at;
            cnt[e] = at;
            for (int k = 0; k < nt; ++k) tiles[ta + k] = make_int2(e, at + k * tile_n);
        }
        base += tot; tbase += ttot;
    }
    if (threadIdx.x == 0) { off[E] = base; if (tiles) *n_tiles = tbase; }
    __syncthreads();
    for (int p = threadIdx.x; p < n; p += 1024) {
        const int at = atomicAdd(&cnt[ids[p]], 1);
        perm[at] = p;
        inv[p] = at;
    }
}

// ---------------------------------------------------------------------------------------------------------------------------------
// grouped mat-mul of prompt portions (bf16): GemmTile per (group, token tile, row tile).  Token tiles come from moe_sort's list
// (g.tiles) or, without a list, every group has ceil(T / BN) of them.  The units are dealt out so that an XCD works through a
// contiguous range of them: the row tiles of a token tile, and the token tiles of a group, share that XCD's L2.
// ---------------------------------------------------------------------------------------------------------------------------------
template <int BM, int BN, int WGM, int WGN>
__global__ __launch_bounds__(64 * WGM * WGN, (WGM * WGN > 4 ? 1 : BM + BN <= 192 ? 3 : 2)) void group_tile_kernel(pi_group_gemm g, int nx, int max_units) {
    using Tile = GemmTile<bf16, BM, BN, WGM, WGN>;
    constexpr int WM = Tile::WM, WN = Tile::WN, MT = Tile::MT, NT = Tile::NT;
    extern __shared__ __align__(16) unsigned char smem[];
    const int tt = (g.T + BN - 1) / BN;                       // token tiles of a group without a list
    const int units = g.off ? *g.n_tiles * nx : max_units;
    const int per = (units + 7) / 8, unit = (int)(blockIdx.x % 8) * per + (int)blockIdx.x / 8;
    if ((int)blockIdx.x / 8 >= per || unit >= units) return;
    const int tx = unit % nx, ty = unit / nx;
    int grp, lo, n;                                           // group, first token (place), tokens from there on
    if (g.off) {
        const int2 t = reinterpret_cast<const int2 *>(g.tiles)[ty];
        grp = t.x; lo = t.y; n = g.off[grp + 1] - lo;
    } else {
        grp = ty / tt; lo = (ty % tt) * BN; n = g.T - lo;
    }
    n = min(n, BN);
    const int row0 = tx * BM;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, i = lane & 15, q = lane >> 4;
    const int wm = wave % WGM, wn = wave / WGM;
    const bf16 * W = (const bf16 *)g.W + (size_t)grp * g.w_gs;
    const bf16 * x = (const bf16 *)g.x + (g.off ? 0 : (size_t)grp * g.x_gs);
    const bf16 * ga[Tile::ACH]; const bf16 * gb[Tile::BCH];
#pragma unroll
    for (int j = 0; j < Tile::ACH; ++j) ga[j] = W + (size_t)min(row0 + Tile::chunk_row(j), g.rows - 1) * g.ldw + Tile::chunk_col();
#pragma unroll
    for (int j = 0; j < Tile::BCH; ++j) {
        const int s = lo + min(Tile::chunk_row(j), n - 1);
        gb[j] = x + (size_t)(g.gather ? g.gather[s] / g.gather_div : s) * g.ldx + Tile::chunk_col();
    }
    pi_f4 acc[MT][NT];
    Tile::run(smem, ga, gb, g.cols / kGtBK, acc);
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int nn = 0; nn < NT; ++nn) {
            const int row = row0 + wm * WM + m * 16 + 4 * q, tok = wn * WN + nn * 16 + i;
            if (tok >= n || row >= g.rows) continue;
            const float alpha = g.pair_w ? g.alpha * g.pair_w[g.gather[lo + tok]] : g.alpha;
            if (g.glu) {                               // rows in (gate, up) pairs: a lane holds two of them
                const size_t o = (g.off ? 0 : (size_t)grp * g.y_gs) + (size_t)(lo + tok) * g.ldy + row / 2;
                const float one = g.glu_plain_up ? 0.0f : 1.0f, a = clamped_glu(acc[m][nn][0] * alpha, acc[m][nn][1] * alpha, g.glu_limit, g.glu_gain, one);
                const float b = clamped_glu(acc[m][nn][2] * alpha, acc[m][nn][3] * alpha, g.glu_limit, g.glu_gain, one);
                const bool two = row + 4 <= g.rows;
                if (g.y_f32) {
                    ((float *)g.y)[o] = a;
                    if (two) ((float *)g.y)[o + 1] = b;
                } else if (two && (o & 1) == 0) {
                    const bf16 v[2] = {(bf16)a, (bf16)b};
                    *reinterpret_cast<uint32_t *>((bf16 *)g.y + o) = __builtin_bit_cast(uint32_t, v);
                } else {
                    ((bf16 *)g.y)[o] = (bf16)a;
                    if (two) ((bf16 *)g.y)[o + 1] = (bf16)b;
                }
                continue;
            }
            const size_t o = (g.off ? 0 : (size_t)grp * g.y_gs) + (size_t)(lo + tok) * g.ldy + row;
            float v[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                v[r] = acc[m][nn][r] * alpha;
                if (g.relu2) { v[r] = fmaxf(v[r], 0.0f); v[r] *= v[r]; }
            }
            const bool quad = row + 4 <= g.rows && (o & 3) == 0;
            if (g.y_f32) {
                float * y = (float *)g.y + o;
                if (quad) *reinterpret_cast<float4 *>(y) = make_float4(v[0], v[1], v[2], v[3]);
                else for (int r = 0; r < 4 && row + r < g.rows; ++r) y[r] = v[r];
            } else {
                bf16 * y = (bf16 *)g.y + o;
                bf16 b[4] = {(bf16)v[0], (bf16)v[1], (bf16)v[2], (bf16)v[3]};
                if (quad) *reinterpret_cast<uint2 *>(y) = __builtin_bit_cast(uint2, b);
                else for (int r = 0; r < 4 && row + r < g.rows; ++r) y[r] = b[r];
            }
        }
}

template <int BM, int BN, int WGM, int WGN> int launch_group_tile(const pi_group_gemm & g, hipStream_t st) {
    using Tile = GemmTile<bf16, BM, BN, WGM, WGN>;
    static bool raised = false;
    if (!raised && Tile::kLds > 64 * 1024) {
        PI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(&group_tile_kernel<BM, BN, WGM, WGN>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)Tile::kLds));
        raised = true;
    }
    const int nx = (g.rows + BM - 1) / BM;
    const long long units = (long long)nx * (g.off ? g.max_tiles : (long long)g.n_group * ((g.T + BN - 1) / BN));
    if (units > (1 << 30)) return pi::fail(PI_E_ARG, "pi_k_group_gemm_tile: too many tiles");
    hipLaunchKernelGGL((group_tile_kernel<BM, BN, WGM, WGN>), dim3((unsigned)((units + 7) / 8 * 8)), dim3(64 * WGM * WGN), Tile::kLds, st, g, nx, (int)units);
    return pi::check_launch("pi_k_group_gemm_tile");
}

template <typename ST>
__global__ __launch_bounds__(256) void moe_combine_kernel(const float * __restrict__ x, const float * __restrict__ mix, const ST * __restrict__ y,
                                                          const int32_t * __restrict__ inv, const float * __restrict__ weights, int top, int cols,
                                                          float * __restrict__ out, float * __restrict__ keep) {
    const int t = blockIdx.y, c0 = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (c0 >= cols) return;
    if ((cols & 3) == 0) {                           // four columns a thread
        const size_t o = (size_t)t * cols + c0;
        float s[4] = {0.0f, 0.0f, 0.0f, 0.0f};
        if (weights) for (int k = 0; k < top; ++k) {
            const float w = weights[(size_t)t * top + k];
            struct alignas(4 * sizeof(ST)) Quad { ST v[4]; };
            const Quad q = *reinterpret_cast<const Quad *>(y + (size_t)inv[(size_t)t * top + k] * cols + c0);
#pragma unroll
            for (int j = 0; j < 4; ++j) s[j] = fmaf(w, from_st(q.v[j]), s[j]);
        }
        const float4 a = *reinterpret_cast<const float4 *>(x + o), b = *reinterpret_cast<const float4 *>(mix + o);
        const float4 v = make_float4(a.x + (b.x + s[0]), a.y + (b.y + s[1]), a.z + (b.z + s[2]), a.w + (b.w + s[3]));
        *reinterpret_cast<float4 *>(out + o) = v;
        if (keep) *reinterpret_cast<float4 *>(keep + o) = v;
        return;
    }
    for (int c = c0; c < min(c0 + 4, cols); ++c) {
        const size_t o = (size_t)t * cols + c;
        float s = 0.0f;
        if (weights) for (int k = 0; k < top; ++k) s = fmaf(weights[(size_t)t * top + k], from_st(y[(size_t)inv[(size_t)t * top + k] * cols + c]), s);
        const float v = x[o] + (mix[o] + s);
        out[o] = v;
        if (keep) keep[o] = v;
    }
}

__global__ void pad_cols_kernel(const uint16_t * __restrict__ in, int64_t rows, int cols, uint16_t * __restrict__ out, int ld) {
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < rows * ld; i += (int64_t)gridDim.x * blockDim.x) {
        const int64_t r = i / ld; const int c = (int)(i % ld);
        out[i] = c < cols ? in[r * cols + c] : (uint16_t)0;
    }
}
__global__ void place_kernel(const uint16_t * __restrict__ in, int64_t rows, int cols, uint16_t * __restrict__ out, int ld, int col0, int width, int64_t row0, int row_step) {
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < rows * width; i += (int64_t)gridDim.x * blockDim.x) {
        const int64_t r = i / width; const int c = (int)(i % width);
        out[(size_t)(row0 + r * row_step) * ld + col0 + c] = c < cols ? in[r * cols + c] : (uint16_t)0;
    }
}
__global__ void transpose_pad_kernel(const uint16_t * __restrict__ in, int n_mat, int rows, int cols, uint16_t * __restrict__ out, int ld) {
    const int64_t n = (int64_t)n_mat * cols * ld;
    for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
        const int r = (int)(i % ld); const int64_t mc = i / ld;
        const int64_t mat = mc / cols; const int c = (int)(mc % cols);
        out[i] = r < rows ? in[(mat * rows + r) * cols + c] : (uint16_t)0;
    }
}

__global__ void cells_advance_kernel(int T, const int32_t * __restrict__ seq, const int32_t * __restrict__ lists, size_t list_ld, int32_t * __restrict__ n_vis,
                                     int32_t * __restrict__ cell, int32_t * step) {
    const int t = threadIdx.x;
    if (t < T) {
        const int n = n_vis[t] + 1;
        n_vis[t] = n;
        cell[t] = lists[(size_t)seq[t] * list_ld + min((size_t)n, list_ld) - 1];        // (behind the last step of a full pool: not used)
    }
    if (t == 0) *step += 1;
}

}  // namespace

extern "C" {

int pi_k_embed_norm(const void * table, int cols, const int32_t * tokens, int T, const float * w, float eps, float * x, pi_stream_t stream) {
    if (!table || !tokens || !w || !x || cols <= 0 || T <= 0) return pi::fail(PI_E_ARG, "pi_k_embed_norm: bad arguments");
    hipLaunchKernelGGL(embed_norm_kernel, dim3(T), dim3(cols > 2048 ? 1024 : 256), 0, (hipStream_t)stream, (const uint16_t *)table, cols, tokens, w, eps, x);
    return pi::check_launch("pi_k_embed_norm");
}

int pi_k_embed_bigram(const void * table, int cols, const int32_t * tokens, int32_t * prev, int T, float scale, const void * bigram, int32_t buckets, int64_t mul_prev,
                      int64_t mul_cur, int carry, float * x, float * x0, pi_stream_t stream) {
    if (!table || !tokens || !prev || !x || cols <= 0 || T <= 0 || (bigram && buckets <= 0)) return pi::fail(PI_E_ARG, "pi_k_embed_bigram: bad arguments");
    hipLaunchKernelGGL(embed_bigram_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, (const uint16_t *)table, cols, tokens, prev, scale, (const uint16_t *)bigram, buckets,
                       (long long)mul_prev, (long long)mul_cur, carry, x, x0);
    return pi::check_launch("pi_k_embed_bigram");
}

int pi_k_layer_norm(int type, float * x, const int32_t * rows, int T, int cols, float eps, const float * w, const float * x0, const float * step, void * out, int ld, int ol,
                    pi_stream_t stream) {
    if (!x || !w || !out || T <= 0 || cols <= 0 || ld < cols || (rows && (x0 || step))) return pi::fail(PI_E_ARG, "pi_k_layer_norm: bad arguments");
    if (ol && (type != PI_TYPE_BF16 || T > kBtMaxT || ld % 8)) return pi::fail(PI_E_ARG, "pi_k_layer_norm: operand layout needs BF16, T <= 16, ld % 8 == 0");
    const int block = cols > 2048 ? 1024 : cols > 512 ? 512 : 256;
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(layer_norm_kernel<bf16>, dim3(T), dim3(block), 0, (hipStream_t)stream, x, rows, cols, eps, w, x0, step, (bf16 *)out, ld, ol);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(layer_norm_kernel<float>, dim3(T), dim3(block), 0, (hipStream_t)stream, x, rows, cols, eps, w, x0, step, (float *)out, ld, 0);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_layer_norm: type");
    return pi::check_launch("pi_k_layer_norm");
}

int pi_k_res_norm(int type, const pi_res_norm * p, pi_stream_t stream) {
    if (!p || !p->x || !p->out || p->T <= 0 || p->cols <= 0 || (p->mix && p->gate_z && (!p->gate_b || p->off_gate < 0 || p->off_gate + p->cols > p->ld_gate)) || (p->h && p->ld < p->cols))
        return pi::fail(PI_E_ARG, "pi_k_res_norm: bad arguments");
    if (p->h && p->ol && (type != PI_TYPE_BF16 || p->T > kBtMaxT || p->ld % 8)) return pi::fail(PI_E_ARG, "pi_k_res_norm: operand layout needs BF16, T <= 16, ld % 8 == 0");
    if (type == PI_TYPE_BF16) return launch_res_norm<bf16>(*p, (hipStream_t)stream);
    if (type == PI_TYPE_F32) return launch_res_norm<float>(*p, (hipStream_t)stream);
    return pi::fail(PI_E_UNSUPPORTED, "pi_k_res_norm: type");
}

int pi_k_ffn_front(int type, const float * z, int ldz, int T, const pi_ffn_front * front, pi_stream_t stream) {
    if (!z || !front || T <= 0 || !front_ok(*front, ldz)) return pi::fail(PI_E_ARG, "pi_k_ffn_front: bad arguments");
    const int per = front_blocks(*front);
    if (per == 0) return PI_OK;
    if ((long long)per * T > (1 << 30)) return pi::fail(PI_E_ARG, "pi_k_ffn_front: too many tokens");
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(ffn_front_kernel<bf16>, dim3(per * T), dim3(256), front_lds_bytes(*front), (hipStream_t)stream, *front, z, ldz, per);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(ffn_front_kernel<float>, dim3(per * T), dim3(256), front_lds_bytes(*front), (hipStream_t)stream, *front, z, ldz, per);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_ffn_front: type");
    return pi::check_launch("pi_k_ffn_front");
}

int pi_k_norm_pair(int type, const float * x, const int32_t * rows, int T, int cols, float eps, const float * wa, void * out_a,
                   const float * wb, void * out_b, int ld, int ol, pi_stream_t stream) {
    if (!x || !wa || !out_a || (wb && !out_b) || T <= 0 || cols <= 0 || ld < cols) return pi::fail(PI_E_ARG, "pi_k_norm_pair: bad arguments");
    if (ol && (type != PI_TYPE_BF16 || T > kBtMaxT || ld % 8)) return pi::fail(PI_E_ARG, "pi_k_norm_pair: operand layout needs BF16, T <= 16, ld % 8 == 0");
    const int block = cols > 2048 ? 1024 : cols > 512 ? 512 : 256;
    if (type == PI_TYPE_BF16)
        hipLaunchKernelGGL(norm_pair_kernel<bf16>, dim3(T), dim3(block), 0, (hipStream_t)stream, x, rows, cols, eps, wa, (bf16 *)out_a, wb, (bf16 *)out_b, ld, ol);
    else if (type == PI_TYPE_F32)
        hipLaunchKernelGGL(norm_pair_kernel<float>, dim3(T), dim3(block), 0, (hipStream_t)stream, x, rows, cols, eps, wa, (float *)out_a, wb, (float *)out_b, ld, 0);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_norm_pair: type");
    return pi::check_launch("pi_k_norm_pair");
}

int pi_k_group_gemm(int type, const pi_group_gemm * g, pi_stream_t stream) {
    if (!g || !g->W || !g->x || !g->y || g->rows <= 0 || g->cols <= 0 || g->cols % 32 || g->ldw < g->cols || g->ldw % 8 || g->ldx < g->cols || g->ldx % 8 ||
        g->ldy < (g->glu ? g->rows / 2 : g->rows) || (g->glu && (g->rows % 2 || g->relu2)) || g->T <= 0 || g->n_group <= 0 || g->n_group > 65535 || (g->gather && g->gather_div <= 0) || (g->pair_w && (!g->gather || !g->off)) || g->w_gs % 8 || g->x_gs % 8)
        return pi::fail(PI_E_ARG, "pi_k_group_gemm: bad arguments");
    const dim3 grid((g->rows + 63) / 64, (g->T + 31) / 32, g->n_group);
    if (grid.y > 65535) return pi::fail(PI_E_ARG, "pi_k_group_gemm: too many tokens");
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(group_gemm_kernel<bf16>, grid, dim3(256), 0, (hipStream_t)stream, *g);
    else if (type == PI_TYPE_F32) hipLaunchKernelGGL(group_gemm_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, *g);
    else return pi::fail(PI_E_UNSUPPORTED, "pi_k_group_gemm: type");
    return pi::check_launch("pi_k_group_gemm");
}

int pi_k_rope_angles(const int32_t * pos, int T, int dims, double base, void * cs, pi_stream_t stream) {
    if (!pos || !cs || T <= 0 || dims <= 0 || dims % 2 || !(base > 0.0)) return pi::fail(PI_E_ARG, "pi_k_rope_angles: bad arguments");
    hipLaunchKernelGGL(rope_angles_kernel, dim3((T * (dims / 2) + 63) / 64), dim3(64), 0, (hipStream_t)stream, pos, T, dims, base, (float2 *)cs);
    return pi::check_launch("pi_k_rope_angles");
}

int pi_k_rope_angles_table(const int32_t * pos, int T, int dims, const double * freq, double length, void * cs, pi_stream_t stream) {
    if (!pos || !cs || !freq || T <= 0 || dims <= 0 || dims % 2) return pi::fail(PI_E_ARG, "pi_k_rope_angles_table: bad arguments");
    hipLaunchKernelGGL(rope_table_kernel, dim3((T * (dims / 2) + 63) / 64), dim3(64), 0, (hipStream_t)stream, pos, T, dims / 2, freq, length, (float2 *)cs);
    return pi::check_launch("pi_k_rope_angles_table");
}

int pi_k_route_scores(const float * z, int T, int n_expert, int n_top, int32_t * ids, float * weights, pi_stream_t stream) {
    if (!z || !ids || !weights || T <= 0 || n_expert <= 0 || n_expert > 4096 || n_top <= 0 || n_top > n_expert) return pi::fail(PI_E_ARG, "pi_k_route_scores: bad arguments");
    RouteArgs r{z, n_expert, n_top, 1, 1, nullptr, ids, weights};
    r.raw = true;
    hipLaunchKernelGGL(route_kernel, dim3(T), dim3(n_expert > 128 ? 256 : n_expert > 64 ? 128 : 64), route_lds_bytes(n_expert, 1, n_top), (hipStream_t)stream, r);
    return pi::check_launch("pi_k_route_scores");
}

int pi_k_route(const float * z, int T, int n_expert, int n_top, int n_group, int n_keep, const float * bias, int32_t * ids, float * weights, pi_stream_t stream) {
    if (!z || !bias || !ids || !weights || T <= 0 || n_expert <= 0 || n_expert > 4096 || n_top <= 0 || n_group <= 0 || n_expert % n_group || n_keep <= 0 || n_keep > n_group ||
        n_top > n_keep * (n_expert / n_group))
        return pi::fail(PI_E_ARG, "pi_k_route: bad arguments");
    hipLaunchKernelGGL(route_kernel, dim3(T), dim3(n_expert > 128 ? 256 : n_expert > 64 ? 128 : 64), route_lds_bytes(n_expert, n_group, n_top), (hipStream_t)stream, RouteArgs{z, n_expert, n_top, n_group, n_keep, bias, ids, weights});
    return pi::check_launch("pi_k_route");
}

int pi_k_moe_sort(const int32_t * ids, int n_pairs, int n_expert, int32_t * off, int32_t * perm, int32_t * inv, int tile_n, int32_t * tiles, int32_t * n_tiles,
                  pi_stream_t stream) {
    if (!ids || !off || !perm || !inv || n_pairs <= 0 || n_expert <= 0 || n_expert > 8192 || (tiles && (tile_n <= 0 || !n_tiles))) return pi::fail(PI_E_ARG, "pi_k_moe_sort: bad arguments");
    hipLaunchKernelGGL(moe_sort_kernel, dim3(1), dim3(1024), sizeof(int) * n_expert, (hipStream_t)stream, ids, n_pairs, n_expert, off, perm, inv, tile_n, (int2 *)tiles, n_tiles);
    return pi::check_launch("pi_k_moe_sort");
}

int pi_k_group_gemm_tile(const pi_group_gemm * g, int tile_n, pi_stream_t stream) {
    if (!g || !g->W || !g->x || !g->y || g->rows <= 0 || g->cols <= 0 || g->cols % kGtBK || g->ldw < g->cols || g->ldw % 8 || g->ldx < g->cols || g->ldx % 8 ||
        g->ldy < (g->glu ? g->rows / 2 : g->rows) || (g->glu && (g->rows % 2 || g->relu2)) || g->T <= 0 || g->n_group <= 0 || (g->gather && g->gather_div <= 0) || (g->pair_w && (!g->gather || !g->off)) || g->w_gs % 8 || g->x_gs % 8 || (g->off && (!g->tiles || !g->n_tiles || g->max_tiles <= 0)))
        return pi::fail(PI_E_ARG, "pi_k_group_gemm_tile: bad arguments");
    if ((((uintptr_t)g->W | (uintptr_t)g->x | (uintptr_t)g->y) & 15) != 0) return pi::fail(PI_E_ARG, "pi_k_group_gemm_tile: operands must be 16-byte aligned");
    hipStream_t st = (hipStream_t)stream;
    if (tile_n == 128) return launch_group_tile<128, 128, 2, 2>(*g, st);
    if (tile_n == 64) return g->rows <= 64 ? launch_group_tile<64, 64, 2, 2>(*g, st) : launch_group_tile<128, 64, 2, 2>(*g, st);
    return pi::fail(PI_E_ARG, "pi_k_group_gemm_tile: tile_n must be 64 or 128");
}

int pi_k_moe_combine(int type, const float * x, const float * mix, const void * y, const int32_t * inv, const float * weights, int n_top, int T, int cols,
                     float * out, float * keep, pi_stream_t stream) {
    if (!x || !mix || !out || T <= 0 || T > 65535 || cols <= 0 || (weights && (!y || !inv || n_top <= 0))) return pi::fail(PI_E_ARG, "pi_k_moe_combine: bad arguments");
    const dim3 grid((cols + 1023) / 1024, T);
    if (type == PI_TYPE_BF16) hipLaunchKernelGGL(moe_combine_kernel<bf16>, grid, dim3(256), 0, (hipStream_t)stream, x, mix, (const bf16 *)y, inv, weights, n_top, cols, out, keep);
    else hipLaunchKernelGGL(moe_combine_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, x, mix, (const float *)y, inv, weights, n_top, cols, out, keep);
    return pi::check_launch("pi_k_moe_combine");
}

int pi_k_pad_cols_bf16(const void * in, int64_t rows, int cols, void * out, int ld, pi_stream_t stream) {
    if (!in || !out || rows <= 0 || cols <= 0 || ld < cols) return pi::fail(PI_E_ARG, "pi_k_pad_cols_bf16: bad arguments");
    hipLaunchKernelGGL(pad_cols_kernel, dim3(4096), dim3(256), 0, (hipStream_t)stream, (const uint16_t *)in, rows, cols, (uint16_t *)out, ld);
    return pi::check_launch("pi_k_pad_cols_bf16");
}

int pi_k_place_bf16(const void * in, int64_t rows, int cols, void * out, int ld, int col0, int width, int64_t row0, int row_step, pi_stream_t stream) {
    if (!in || !out || rows <= 0 || cols <= 0 || width < cols || col0 < 0 || col0 + width > ld || row0 < 0 || row_step <= 0) return pi::fail(PI_E_ARG, "pi_k_place_bf16: bad arguments");
    hipLaunchKernelGGL(place_kernel, dim3(4096), dim3(256), 0, (hipStream_t)stream, (const uint16_t *)in, rows, cols, (uint16_t *)out, ld, col0, width, row0, row_step);
    return pi::check_launch("pi_k_place_bf16");
}

int pi_k_transpose_pad_bf16(const void * in, int n_mat, int rows, int cols, void * out, int ld, pi_stream_t stream) {
    if (!in || !out || n_mat <= 0 || rows <= 0 || cols <= 0 || ld < rows) return pi::fail(PI_E_ARG, "pi_k_transpose_pad_bf16: bad arguments");
    hipLaunchKernelGGL(transpose_pad_kernel, dim3(4096), dim3(256), 0, (hipStream_t)stream, (const uint16_t *)in, n_mat, rows, cols, (uint16_t *)out, ld);
    return pi::check_launch("pi_k_transpose_pad_bf16");
}

int pi_k_cells_advance(int T, const int32_t * seq, const int32_t * lists, size_t list_ld, int32_t * n_vis, int32_t * cell, int32_t * step, pi_stream_t stream) {
    if (T <= 0 || T > 64 || !seq || !lists || !n_vis || !cell || !step) return pi::fail(PI_E_ARG, "pi_k_cells_advance: bad arguments");
    hipLaunchKernelGGL(cells_advance_kernel, dim3(1), dim3(64), 0, (hipStream_t)stream, T, seq, lists, list_ld, n_vis, cell, step);
    return pi::check_launch("pi_k_cells_advance");
}

}  // extern "C"
