// Element types of the operators that exist for bf16 and for fp32 activations: conversions and the matrix-core fragment of each.
#pragma once
#include "kernels_common.hpp"

namespace {

typedef __bf16 bf16;

__device__ __forceinline__ float bf16_to_f32(uint16_t b) { return __uint_as_float((uint32_t)b << 16); }
template <typename ST> __device__ __forceinline__ ST to_st(float v) { return (ST)v; }           // bf16: round to nearest even
template <typename ST> __device__ __forceinline__ float from_st(ST v) { return (float)v; }

// eight consecutive columns of one row of a 16 x 32 operand tile (lane l: row l % 16, columns 8 * (l / 16) ..)
template <typename ST> struct Frag;
template <> struct Frag<bf16> { pi_u32x4 v; };
template <> struct Frag<float> { float v[8]; };

__device__ __forceinline__ Frag<bf16> frag_load(const bf16 * p) { return Frag<bf16>{pi_ld16(p)}; }
__device__ __forceinline__ Frag<float> frag_load(const float * p) {
    Frag<float> f;
    const float4 a = reinterpret_cast<const float4 *>(p)[0], b = reinterpret_cast<const float4 *>(p)[1];
    f.v[0] = a.x; f.v[1] = a.y; f.v[2] = a.z; f.v[3] = a.w; f.v[4] = b.x; f.v[5] = b.y; f.v[6] = b.z; f.v[7] = b.w;
    return f;
}
template <typename ST> __device__ __forceinline__ Frag<ST> frag_weights(const uint16_t * p);      // bf16 weights in the storage's fragment
template <> __device__ __forceinline__ Frag<bf16> frag_weights<bf16>(const uint16_t * p) { return Frag<bf16>{pi_ld16(p)}; }
template <> __device__ __forceinline__ Frag<float> frag_weights<float>(const uint16_t * p) {
    const pi_u32x4 w = pi_ld16(p);
    Frag<float> f;
#pragma unroll
    for (int j = 0; j < 4; ++j) { f.v[2 * j] = __uint_as_float(w[j] << 16); f.v[2 * j + 1] = __uint_as_float(w[j] & 0xffff0000u); }
    return f;
}
__device__ __forceinline__ pi_f4 mfma_bf16(const pi_u32x4 & a, const pi_u32x4 & b, pi_f4 c) {
    return mma16<bf16>(a, b, c);
}
__device__ __forceinline__ void frag_mma(const Frag<bf16> & a, const Frag<bf16> & b, pi_f4 & c) { c = mfma_bf16(a.v, b.v, c); }
// the k index within a step is free as long as both operands agree: instruction j takes columns 8 g + j of the four lane groups
__device__ __forceinline__ void frag_mma(const Frag<float> & a, const Frag<float> & b, pi_f4 & c) {
#pragma unroll
    for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[j], b.v[j], c, 0, 0, 0);
}

}  // namespace
