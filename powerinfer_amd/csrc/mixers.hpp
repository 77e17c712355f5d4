// Pieces of a layer that several launches hold: the clamped GLU, what a layer with one norm computes of its feed-forward straight from the
// joint projection, queries and cells of a grouped-query attention, the merge of a split one, and the gated norm behind a linear attention.
#pragma once
#include "layer_types.hpp"
#include "route.hpp"

namespace {

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z * sigmoid_f32(z); }
__device__ __forceinline__ float clamped_glu(float g, float u, float limit, float gain, float one = 1.0f) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g * sigmoid_f32(gain * g) * (u + one);
}

// four values of activation storage in one store where the place allows it
template <typename ST> __device__ __forceinline__ void store4(ST * p, const float (&v)[4], bool whole, int n) {
    if (whole) {
        struct alignas(4 * sizeof(ST)) Quad { ST v[4]; } q{{to_st<ST>(v[0]), to_st<ST>(v[1]), to_st<ST>(v[2]), to_st<ST>(v[3])}};
        *reinterpret_cast<Quad *>(p) = q;
    } else {
        for (int r = 0; r < 4 && r < n; ++r) p[r] = to_st<ST>(v[r]);
    }
}

// ---- pi_ffn_front: blocks of 256 threads, front_glu_blocks of them and one more for the choice of experts per token -----------------
constexpr int kFrontGlu = 1024;           // values of a workgroup
__host__ __device__ inline int front_glu_blocks(const pi_ffn_front & f) { return f.ff > 0 ? (f.ff_ld + kFrontGlu - 1) / kFrontGlu : 0; }
__host__ __device__ inline int front_blocks(const pi_ffn_front & f) { return front_glu_blocks(f) + (f.n_expert > 0 ? 1 : 0); }
inline size_t front_lds_bytes(const pi_ffn_front & f) { return f.n_expert > 0 ? route_lds_bytes(f.n_expert, 1, f.n_top) : 0; }
inline bool front_ok(const pi_ffn_front & f, int ldz) {
    if (f.ff > 0 && (!f.act || f.off_glu < 0 || f.off_glu + 2 * f.ff > ldz || f.off_score >= ldz || f.ff_ld < f.ff || f.ff_ld % 4 || f.ld_act < f.ff_ld)) return false;
    return f.n_expert <= 0 || (f.ids && f.weights && f.off_router >= 0 && f.off_router + f.n_expert <= ldz && f.n_expert <= 4096 && f.n_top > 0 && f.n_top <= f.n_expert);
}
template <typename ST> __device__ void front_block(const pi_ffn_front & f, const float * __restrict__ z, int ldz, int t, int b, float * sm) {
    const float * row = z + (size_t)t * ldz;
    if (b == front_glu_blocks(f)) {
        route_token(RouteArgs{z + f.off_router, f.n_expert, f.n_top, 1, 1, nullptr, f.ids, f.weights, ldz, true}, t, sm);
        return;
    }
    const int j0 = b * kFrontGlu + threadIdx.x * 4;
    if (j0 >= f.ff_ld) return;
    const float * g = row + f.off_glu + 2 * j0;
    float v[4], w[8];
    if (j0 + 4 <= f.ff && ((f.off_glu | ldz) & 3) == 0) {
        const float4 a = reinterpret_cast<const float4 *>(g)[0], c = reinterpret_cast<const float4 *>(g)[1];
        w[0] = a.x; w[1] = a.y; w[2] = a.z; w[3] = a.w; w[4] = c.x; w[5] = c.y; w[6] = c.z; w[7] = c.w;
    } else {
#pragma unroll
        for (int k = 0; k < 8; ++k) w[k] = j0 + k / 2 < f.ff ? g[k] : 0.0f;
    }
    const float s = f.off_score >= 0 ? sigmoid_f32(row[f.off_score]) : 1.0f, one = f.plain_up ? 0.0f : 1.0f;
#pragma unroll
    for (int k = 0; k < 4; ++k) v[k] = j0 + k < f.ff ? s * clamped_glu(w[2 * k], w[2 * k + 1], f.limit, f.gain, one) : 0.0f;
    ST * o = (ST *)f.act + (size_t)t * f.ld_act + j0;
    store4(o, v, ((uintptr_t)o & (4 * sizeof(ST) - 1)) == 0, 4);
}

// ---- grouped-query attention, behind the joint projection: a wave per head (four heads a block) - norm, rotation, division by the root
// mean square, query row or cell --------------------------------------------------------------------------------------------------------
constexpr int kGqaMaxDim = 256;
// value e of a token's heads: kept for the layers behind, or mixed with the one an earlier layer kept
__device__ __forceinline__ float mixed_value(const pi_gqa_prep & p, float v, int t, int e) {
    if (p.v_keep) p.v_keep[(size_t)t * p.ld_first + e] = v;
    if (p.v_first) { const float l = p.v_mix[0]; v = (1.0f - l) * v + l * p.v_first[(size_t)t * p.ld_first + e]; }
    return v;
}
template <typename ST, bool NORM> __device__ void gqa_prep_heads(const pi_gqa_prep & p, int t, int b) {      // NORM: q_norm and k_norm are given
    const int head = b * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63, half = p.rot_dim / 2;
    if (head >= p.n_head + p.n_kv) return;
    const bool key = head >= p.n_head;
    const int g = head - p.n_head;
    const float * z = p.z + (size_t)t * p.ldz, * src = key ? z + p.off_k + g * p.dim : z + head * p.dim;
    const float * w = key ? p.k_norm : p.q_norm;             // (pairs i, i + half of the rotation's dimensions)
    const float2 * cs = (const float2 *)p.cs + (size_t)t * half;
    ST * row = key ? (ST *)p.cache + ((size_t)p.cell[t] * p.n_kv + g) * 2 * p.hd : (ST *)p.q + ((size_t)t * p.n_head + head) * p.hd;
    constexpr int J = kGqaMaxDim / 64;
    float x[J], y[J];                                    // the lane's values and what each is paired with (no guard around a load)
    float2 c[J];
    float ss = 0.0f;
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int e = min(lane + 64 * j, p.dim - 1), o = e >= 2 * half ? e : e < half ? e + half : e - half;
        x[j] = src[e]; y[j] = src[o];
        c[j] = cs[min(e < half ? e : e - half, max(half - 1, 0))];
    }
#pragma unroll
    for (int j = 0; j < J; ++j) {
        if (lane + 64 * j >= p.dim) x[j] = 0.0f;
        ss = fmaf(x[j], x[j], ss);
    }
    float sc = 1.0f;
    if constexpr (NORM) {
        sc = pi_inv_sqrt(pi_wave_sum(ss) / (float)p.dim + p.eps);
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const int e = min(lane + 64 * j, p.dim - 1), o = e >= 2 * half ? e : e < half ? e + half : e - half;
            x[j] *= w[e]; y[j] *= w[o];
        }
    }
    ss = 0.0f;
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int e = lane + 64 * j;
        if (e < 2 * half) x[j] = e >= half ? x[j] * c[j].x + y[j] * c[j].y : x[j] * c[j].x - y[j] * c[j].y;
        ss = fmaf(x[j], x[j], ss);
    }
    if (p.unit) sc = pi_inv_sqrt(pi_wave_sum(ss) / (float)p.dim + p.eps);
    if (!key && p.temp) sc *= p.temp[head];
#pragma unroll
    for (int j = 0; j < J; ++j) { const int e = lane + 64 * j; if (e < p.hd) row[e] = to_st<ST>(x[j] * sc); }      // (zeros behind dim)
    if (key) {
        const float * v = z + p.off_v + g * p.vdim;
        float sv = 1.0f;
#pragma unroll
        for (int j = 0; j < J; ++j) x[j] = mixed_value(p, v[min(lane + 64 * j, p.vdim - 1)], t, g * p.vdim + min(lane + 64 * j, p.vdim - 1));
        ss = 0.0f;
#pragma unroll
        for (int j = 0; j < J; ++j) { if (lane + 64 * j >= p.vdim) x[j] = 0.0f; ss = fmaf(x[j], x[j], ss); }
        if (p.unit_v) sv = pi_inv_sqrt(pi_wave_sum(ss) / (float)p.vdim + p.eps);
#pragma unroll
        for (int j = 0; j < J; ++j) { const int e = lane + 64 * j; if (e < p.hd) row[p.hd + e] = to_st<ST>(x[j] * sv); }
    }
}
// The same for neighbouring pairs, which one lane holds: pairs lane and lane + 64 of N heads of a wave, 4 N heads a block, everything requested
// together and without guards (past the end of a row: its last values again, not used).  EVEN: no row starts or ends in the middle of a pair.
template <typename ST, int N, bool EVEN> __device__ void gqa_prep_pairs(const pi_gqa_prep & p, int t, int b) {
    const int lane = threadIdx.x & 63, half = p.rot_dim / 2, all = p.n_head + p.n_kv, h0 = (b * 4 + (int)(threadIdx.x >> 6)) * N;
    if (h0 >= all) return;
    const float * z = p.z + (size_t)t * p.ldz, * qn = p.q_norm ? p.q_norm : z, * kn = p.k_norm ? p.k_norm : z;
    const float2 * cs = (const float2 *)p.cs + (size_t)t * half;
    const int cell = p.cell[t];
    constexpr int J = kGqaMaxDim / 128;
    const auto load = [](const float * a, int e, int n) {
        if constexpr (EVEN) return *reinterpret_cast<const float2 *>(a + min(e, n - 2));
        else return make_float2(a[min(e, n - 1)], a[min(e + 1, n - 1)]);
    };
    const auto store = [](ST * o, float a, float b) {
        struct alignas(2 * sizeof(ST)) Pair { ST v[2]; } q{{to_st<ST>(a), to_st<ST>(b)}};
        *reinterpret_cast<Pair *>(o) = q;
    };
    float2 x[N][J], v[N][J], wq[J], wk[J], c[J];
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int e = 2 * (lane + 64 * j);
        wq[j] = load(qn, e, p.dim);
        wk[j] = load(kn, e, p.dim);
        c[j] = cs[min(lane + 64 * j, max(half - 1, 0))];
#pragma unroll
        for (int n = 0; n < N; ++n) {
            const int h = min(h0 + n, all - 1), g = h - p.n_head;
            x[n][j] = load(g >= 0 ? z + p.off_k + g * p.dim : z + h * p.dim, e, p.dim);
        }
    }
    const bool keys = h0 + N > p.n_head;
    if (keys) {
#pragma unroll
        for (int j = 0; j < J; ++j)
#pragma unroll
            for (int n = 0; n < N; ++n) v[n][j] = load(z + p.off_v + max(min(h0 + n, all - 1) - p.n_head, 0) * p.vdim, 2 * (lane + 64 * j), p.vdim);
    }
#pragma unroll
    for (int n = 0; n < N; ++n) {
        const int h = h0 + n, g = h - p.n_head;
        if (h >= all) break;
        const bool key = g >= 0;
        float ss = 0.0f;
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const int e = 2 * (lane + 64 * j);
            if (e >= p.dim) x[n][j].x = 0.0f;
            if (e + 1 >= p.dim) x[n][j].y = 0.0f;
            ss = fmaf(x[n][j].x, x[n][j].x, fmaf(x[n][j].y, x[n][j].y, ss));
        }
        float sc = p.q_norm || p.unit ? pi_inv_sqrt(pi_wave_sum(ss) / (float)p.dim + p.eps) : 1.0f;      // (a rotation changes no sum of squares)
        if (!key && p.temp) sc *= p.temp[h];
        ST * row = key ? (ST *)p.cache + ((size_t)cell * p.n_kv + g) * 2 * p.hd : (ST *)p.q + ((size_t)t * p.n_head + h) * p.hd;
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const int e = 2 * (lane + 64 * j);
            const float2 f = !p.q_norm ? make_float2(1.0f, 1.0f) : key ? wk[j] : wq[j], r = e < p.rot_dim ? c[j] : make_float2(1.0f, 0.0f);
            const float a = x[n][j].x * f.x * sc, o = x[n][j].y * f.y * sc;
            if (e < p.hd) store(row + e, a * r.x - o * r.y, o * r.x + a * r.y);
        }
        if (!key) continue;
        if (p.v_keep || p.v_first) {
#pragma unroll
            for (int j = 0; j < J; ++j) {
                const int e = 2 * (lane + 64 * j);
                if (e < p.vdim) v[n][j].x = mixed_value(p, v[n][j].x, t, g * p.vdim + e);
                if (e + 1 < p.vdim) v[n][j].y = mixed_value(p, v[n][j].y, t, g * p.vdim + e + 1);
            }
        }
        float sv = 0.0f;
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const int e = 2 * (lane + 64 * j);
            if (e >= p.vdim) v[n][j].x = 0.0f;
            if (e + 1 >= p.vdim) v[n][j].y = 0.0f;
            sv = fmaf(v[n][j].x, v[n][j].x, fmaf(v[n][j].y, v[n][j].y, sv));
        }
        const float s2 = p.unit_v ? pi_inv_sqrt(pi_wave_sum(sv) / (float)p.vdim + p.eps) : 1.0f;
#pragma unroll
        for (int j = 0; j < J; ++j) { const int e = 2 * (lane + 64 * j); if (e < p.hd) store(row + p.hd + e, v[n][j].x * s2, v[n][j].y * s2); }
    }
}
// heads of a block: neighbouring pairs of long steps several a wave
constexpr int kGqaPrepHeads = 4;
__host__ __device__ inline int gqa_prep_blocks(const pi_gqa_prep & p) {
    const int per = p.rot_pairs && p.T > 16 ? 4 * kGqaPrepHeads : 4;
    return (p.n_head + p.n_kv + per - 1) / per;
}
template <typename ST, bool PAIRS> __device__ void gqa_prep_block(const pi_gqa_prep & p, int t, int b) {
    const bool even = ((p.dim | p.vdim | p.ldz | p.off_k | p.off_v) & 1) == 0;
    if (!PAIRS && !p.q_norm) gqa_prep_heads<ST, false>(p, t, b);
    else if (!PAIRS) gqa_prep_heads<ST, true>(p, t, b);
    else if (p.T > 16) { if (even) gqa_prep_pairs<ST, kGqaPrepHeads, true>(p, t, b); else gqa_prep_pairs<ST, kGqaPrepHeads, false>(p, t, b); }
    else if (even) gqa_prep_pairs<ST, 1, true>(p, t, b);
    else gqa_prep_pairs<ST, 1, false>(p, t, b);
}
inline bool gqa_prep_ok(int type, const pi_gqa_prep & p) {
    return p.z && p.cs && p.q && p.cache && p.cell && p.T > 0 && p.n_head > 0 && p.n_kv > 0 && p.n_head % p.n_kv == 0 && p.rot_dim >= 0 && p.rot_dim % 2 == 0 && p.rot_dim <= p.dim &&
           p.hd == pi_k_gqa_head_ld(type, p.dim, p.vdim) && p.hd > 0 && p.off_k >= p.n_head * p.dim && p.off_k + p.n_kv * p.dim <= p.ldz && p.off_v >= 0 &&
           p.off_v + p.n_kv * p.vdim <= p.ldz && !p.q_norm == !p.k_norm && !(p.q_norm && p.unit) && (!(p.v_first || p.v_keep) || p.ld_first >= p.n_kv * p.vdim) && (!p.v_first || p.v_mix);
}

// ---- grouped-query attention: the parts of one row of a work item, by one wave (fixed order, the sink in the denominator) -------------
__host__ __device__ inline int gqa_rows(int wide) { return wide ? 128 : 16; }
// vg: the group, or (all_values) the pair of a group and whose values its rows met
__device__ void gqa_merge_row(const pi_gqa_attn & p, int item_index, int vg, int r) {
    const int n_groups = p.all_values ? p.n_kv * p.n_kv : p.n_kv, g = p.all_values ? vg / p.n_kv : vg;
    const int lane = threadIdx.x & 63, per = p.n_head / p.n_kv, R = gqa_rows(p.wide);
    const int4 item = reinterpret_cast<const int4 *>(p.work)[item_index];
    if (r >= item.z) return;
    const size_t srow = ((size_t)item_index * n_groups + vg) * R + r;
    const float * acc = p.scratch + srow * p.n_parts * p.hd;
    const float2 ml = lane < p.n_parts ? reinterpret_cast<const float2 *>(p.scratch + (size_t)p.n_work * n_groups * R * p.n_parts * p.hd)[srow * p.n_parts + lane]
                                       : make_float2(-INFINITY, 0.0f);
    const int rr = item.y + r, head = g * per + rr % per;
    const float sink = p.sinks ? p.sinks[head] : p.sink, m = fmaxf(pi_wave_max(ml.x), sink);
    const float e = ml.x == -INFINITY ? 0.0f : expf(ml.x - m);
    const float l = pi_wave_sum(e * ml.y) + expf(sink - m);
    const float f = e / l * p.out_scale;
    bf16 * out = (bf16 *)p.att + (size_t)(item.x + rr / per) * p.ld_att + head * p.vdim;
    float * all = p.all_values ? (float *)p.att + (((size_t)(item.x + rr / per) * p.n_head + head) * p.n_kv + vg % p.n_kv) * p.vdim : nullptr;
    for (int c0 = 0; c0 < p.vdim; c0 += 64) {            // (every lane stays in the loop: the factors are passed between lanes)
        const int c = min(c0 + lane, p.hd - 1);
        float v = 0.0f;
        for (int s0 = 0; s0 < p.n_parts; s0 += 8) {
            float a[8];
#pragma unroll
            for (int u = 0; u < 8; ++u) a[u] = acc[(size_t)min(s0 + u, p.n_parts - 1) * p.hd + c];
#pragma unroll
            for (int u = 0; u < 8; ++u) {
                const float w = __shfl(f, min(s0 + u, PI_WAVE - 1), PI_WAVE);
                if (s0 + u < p.n_parts) v = fmaf(w, a[u], v);
            }
        }
        if (c0 + lane < p.vdim) { if (all) all[c0 + lane] = v; else out[c0 + lane] = (bf16)v; }
    }
}

// ---- gated norm by a block of 256 threads: of one token, or (heads) of as many of a token's heads as there are groups of lanes in it,
// four values a lane ----------------------------------------------------------------------------------------------------------------------
__host__ __device__ inline int gate_norm_lanes(const pi_gate_norm & p) { const int q = (p.n / p.heads + 3) / 4; return q <= 8 ? 8 : q <= 16 ? 16 : q <= 32 ? 32 : 64; }
__host__ __device__ inline int gate_norm_per_token(const pi_gate_norm & p) { const int per = 256 / gate_norm_lanes(p); return (p.heads + per - 1) / per; }
__host__ __device__ inline int gate_norm_blocks(const pi_gate_norm & p) { return p.heads > 0 ? p.T * gate_norm_per_token(p) : p.T; }
template <typename ST> __device__ void gate_norm_heads(const pi_gate_norm & p, int t, int b) {
    const int vd = p.n / p.heads, lanes = gate_norm_lanes(p), h = min(b * (256 / lanes) + (int)threadIdx.x / lanes, p.heads - 1), c = (int)(threadIdx.x % lanes) * 4;      // (behind the last head: it again)
    const float * o = p.o + (size_t)t * p.n + h * vd, * g = p.z + (size_t)t * p.ldz + p.off_gate + h * vd, * w = p.w + h * vd;
    ST * out = (ST *)p.att + (size_t)t * p.ld_att + h * vd + c;
    const bool quads = ((vd | p.ldz | p.off_gate) & 3) == 0;
    float v[4] = {0.0f, 0.0f, 0.0f, 0.0f}, gv[4], wv[4];
    const float den = p.den ? p.den[(size_t)t * p.heads + h] : 1.0f;
    if (quads) {
        const int e = min(c, vd - 4);
        const float4 a = *reinterpret_cast<const float4 *>(o + e), q = *reinterpret_cast<const float4 *>(g + e), f = *reinterpret_cast<const float4 *>(w + e);
        if (c < vd) { v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; }
        gv[0] = q.x; gv[1] = q.y; gv[2] = q.z; gv[3] = q.w;
        wv[0] = f.x; wv[1] = f.y; wv[2] = f.z; wv[3] = f.w;
    } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int e = min(c + j, vd - 1);
            if (c + j < vd) v[j] = o[e];
            gv[j] = g[e]; wv[j] = w[e];
        }
    }
    const float per = 1.0f / den;
    float ss = 0.0f;
#pragma unroll
    for (int j = 0; j < 4; ++j) { v[j] *= per; ss = fmaf(v[j], v[j], ss); }
    for (int k = 1; k < lanes; k <<= 1) ss += __shfl_xor(ss, k, PI_WAVE);
    const float sc = pi_inv_sqrt(ss / (float)vd + p.eps) * p.scale;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] *= sc * wv[j] * (p.silu ? silu_f32(gv[j]) : sigmoid_f32(gv[j]));
    if (c < vd) store4(out, v, quads && ((uintptr_t)out & (4 * sizeof(ST) - 1)) == 0, vd - c);
}
template <typename ST> __device__ void gate_norm_block(const pi_gate_norm & p, int b, double * red) {
    if (p.heads > 0) { const int per = gate_norm_per_token(p); gate_norm_heads<ST>(p, b / per, b % per); return; }
    const int t = b;
    const float * o = p.o + (size_t)t * p.n, * g = p.z + (size_t)t * p.ldz + p.off_gate;
    ST * out = (ST *)p.att + (size_t)t * p.ld_att;
    constexpr int K = 16;
    const int nt = blockDim.x;
    const auto gate = [&](float z) { return p.silu ? silu_f32(z) : sigmoid_f32(z); };
    if (p.n <= K * nt) {                              // one memory round trip: everything requested together, kept in registers
        float v[K], gv[K], wv[K];
        double s = 0.0;
#pragma unroll
        for (int k = 0; k < K; ++k) {
            const int i = min((int)threadIdx.x + k * nt, p.n - 1);
            v[k] = o[i]; gv[k] = g[i]; wv[k] = p.w[i];
        }
#pragma unroll
        for (int k = 0; k < K; ++k) if ((int)threadIdx.x + k * nt < p.n) s += (double)v[k] * (double)v[k];
        s = block_sum_f64(s, red);
        const float sc = pi_inv_sqrt((float)(s / p.n) + p.eps) * p.scale;
#pragma unroll
        for (int k = 0; k < K; ++k) {
            const int i = threadIdx.x + k * nt;
            if (i < p.n) out[i] = to_st<ST>(v[k] * sc * wv[k] * gate(gv[k]));
        }
        return;
    }
    double s = 0.0;
    for (int i = threadIdx.x; i < p.n; i += nt) s += (double)o[i] * (double)o[i];
    s = block_sum_f64(s, red);
    const float sc = pi_inv_sqrt((float)(s / p.n) + p.eps) * p.scale;
    for (int i = threadIdx.x; i < p.n; i += nt) out[i] = to_st<ST>(o[i] * sc * p.w[i] * gate(g[i]));
}
inline bool gate_norm_ok(const pi_gate_norm & p) {
    return p.o && p.z && p.w && p.att && p.n > 0 && p.T > 0 && p.off_gate >= 0 && p.off_gate + p.n <= p.ldz && p.ld_att >= p.n && p.heads >= 0 &&
           (p.heads == 0 ? !p.den : p.n % p.heads == 0 && p.n / p.heads <= 256);
}

}  // namespace
