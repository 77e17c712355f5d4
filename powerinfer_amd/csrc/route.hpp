// Expert choice of one token by one workgroup, shared by the stand-alone operator and the step kernels.
#pragma once
#include "kernels_common.hpp"

namespace {

// soft: the experts with the largest logits, their weights the soft-max over them; else sigmoid scores, a bias on the choice (optional) and groups,
// weights over their sum or (raw) as they are.
// ldz: values between the tokens' rows of z (0: E)
struct RouteArgs { const float * z; int E, top, G, keep; const float * bias; int32_t * ids; float * weights; int ldz = 0; bool soft = false, raw = false; };

__host__ __device__ inline size_t route_lds_bytes(int E, int G, int top) { return sizeof(float) * (size_t)(2 * ((E + 3) / 4 * 4) + (G > top ? G : top)); }

// every thread of the workgroup; sm (16-byte aligned): route_lds_bytes of LDS - scores, choice scores (padded with -inf to a multiple of
// four), the groups' sums and later the chosen scores.  The lower index wins a tie.
__device__ void route_token(const RouteArgs & r, int t, float * sm) {
    const int E = r.E, E4 = (E + 3) / 4 * 4, G = r.G, tid = threadIdx.x, nt = blockDim.x, size = E / G;
    float * sc = sm, * ch = sm + E4, * gs = sm + 2 * E4;
    const float * z = r.z + (size_t)t * (r.ldz ? r.ldz : E);
    for (int e = tid; e < E4; e += nt) {
        float s = 0.0f, c = -INFINITY;
        if (e < E) {
            s = r.soft ? z[e] : 1.0f / (1.0f + expf(-z[e]));
            c = r.soft || !r.bias ? s : s + r.bias[e];
            if (!(c == c)) c = -INFINITY;                      // not a number: never chosen over a number
        }
        sc[e] = s;
        ch[e] = c;
    }
    __syncthreads();
    if (r.keep < G) {
        for (int g = tid; g < G; g += nt) {
            float a = -INFINITY, b = -INFINITY;
#pragma unroll 4
            for (int k = 0; k < size; ++k) {
                const float v = ch[g * size + k];
                b = fmaxf(b, fminf(a, v));
                a = fmaxf(a, v);
            }
            gs[g] = size > 1 ? a + b : a;
        }
        __syncthreads();
        // a group stays if fewer than `keep` groups come before it (larger sum, or the same sum and a lower index)
        for (int e = tid; e < E; e += nt) {
            const int g = e / size;
            const float mine = gs[g];
            int before = 0;
            for (int o = 0; o < G; ++o) before += (gs[o] > mine || (gs[o] == mine && o < g)) ? 1 : 0;
            if (before >= r.keep) ch[e] = -INFINITY;
        }
        __syncthreads();
    }
    // An expert's rank by comparison with all others (ties by index, so that the ranks are a permutation): reads that all lanes share,
    // no chain of reductions.
    int32_t * ids = r.ids + (size_t)t * r.top;
    for (int e = tid; e < E; e += nt) {
        const float c = ch[e];
        int rank = 0;
#pragma unroll 4
        for (int o = 0; o < E4; o += 4) {
            const float4 v = *reinterpret_cast<const float4 *>(ch + o);
            rank += (v.x > c || (v.x == c && o < e) ? 1 : 0) + (v.y > c || (v.y == c && o + 1 < e) ? 1 : 0) +
                    (v.z > c || (v.z == c && o + 2 < e) ? 1 : 0) + (v.w > c || (v.w == c && o + 3 < e) ? 1 : 0);
        }
        if (rank < r.top) { ids[rank] = e; gs[rank] = sc[e]; }
    }
    __syncthreads();
    float total = 0.0f;
    if (r.soft) {
        const float m = gs[0];                                 // rank 0 holds the largest
        for (int k = 0; k < r.top; ++k) total += expf(gs[k] - m);
        for (int k = tid; k < r.top; k += nt) r.weights[(size_t)t * r.top + k] = expf(gs[k] - m) / total;
        return;
    }
    for (int k = 0; k < r.top; ++k) total += gs[k];
    for (int k = tid; k < r.top; k += nt) r.weights[(size_t)t * r.top + k] = r.raw ? gs[k] : gs[k] / (total + 1e-20f);
}

}  // namespace
