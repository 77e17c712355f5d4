// Expert choice of one token by one wave, shared by the stand-alone operator and the step kernels.
#pragma once
#include "kernels_common.hpp"

namespace {

struct RouteArgs { const float * z; int E, top, G, keep; const float * bias; int32_t * ids; float * weights; };

__device__ __forceinline__ void wave_argmax(float & v, int & i) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
        const float ov = __shfl_xor(v, o, PI_WAVE); const int oi = __shfl_xor(i, o, PI_WAVE);
        if (ov > v || (ov == v && oi < i)) { v = ov; i = oi; }
    }
}
// orders a wave's own LDS accesses (they complete in program order; this keeps the compiler from moving them)
__device__ __forceinline__ void wave_lds_fence() {
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup");
    __builtin_amdgcn_wave_barrier();
}
__host__ __device__ inline size_t route_lds_bytes(int E, int G) { return sizeof(float) * (size_t)(2 * E + G); }

// lanes 0..63 of one wave; sm: route_lds_bytes of LDS (scores, choice scores, the groups' sums).  The lower index wins a tie.
__device__ void route_token(const RouteArgs & r, int t, float * sm) {
    const int E = r.E, G = r.G, lane = threadIdx.x & 63, size = E / G;
    float * sc = sm, * ch = sm + E, * gs = sm + 2 * E;
    for (int e = lane; e < E; e += 64) {
        const float s = 1.0f / (1.0f + expf(-r.z[(size_t)t * E + e]));
        sc[e] = s;
        ch[e] = s + r.bias[e];
    }
    wave_lds_fence();
    if (r.keep < G) {
        for (int g = lane; g < G; g += 64) {
            float a = -INFINITY, b = -INFINITY;
            for (int k = 0; k < size; ++k) {
                const float v = ch[g * size + k];
                if (v > a) { b = a; a = v; } else if (v > b) b = v;
            }
            gs[g] = size > 1 ? a + b : a;
        }
        wave_lds_fence();
        // a group stays if fewer than `keep` groups come before it (larger sum, or the same sum and a lower index)
        for (int g = lane; g < G; g += 64) {
            int before = 0;
            for (int o = 0; o < G; ++o) before += (gs[o] > gs[g] || (gs[o] == gs[g] && o < g)) ? 1 : 0;
            if (before >= r.keep) for (int k = 0; k < size; ++k) ch[g * size + k] = -INFINITY;
        }
        wave_lds_fence();
    }
    float total = 0.0f;
    for (int k = 0; k < r.top; ++k) {
        float v = -INFINITY; int idx = E;
        for (int e = lane; e < E; e += 64) {
            const float c = ch[e];
            if (c > v || (c == v && e < idx)) { v = c; idx = e; }
        }
        wave_argmax(v, idx);
        if (idx >= E) idx = 0;                                 // not-a-number scores: any expert, never an index outside
        const float s = sc[idx];
        total += s;
        if (lane == 0) { r.ids[(size_t)t * r.top + k] = idx; r.weights[(size_t)t * r.top + k] = s; ch[idx] = __int_as_float(0x7fc00000); }      // taken: compares false with everything
        wave_lds_fence();
    }
    if (lane == 0) for (int k = 0; k < r.top; ++k) r.weights[(size_t)t * r.top + k] /= total + 1e-20f;        // lane 0 wrote them, lane 0 reads them back
}

}  // namespace
