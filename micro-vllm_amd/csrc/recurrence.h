// Shared by the recurrences whose state rows decay one by one (delta.hip, gla.hip): activation-type stores, gates on the
// hardware's exponential, and the fp32 matrix product.
#pragma once
#include "common.h"

namespace mv {

template <bool F32> struct ActD;
template <> struct ActD<true> {
    typedef float T;
    static __device__ __forceinline__ void st(float* p, float v) { *p = v; }
};
template <> struct ActD<false> {
    typedef uint16_t T;
    static __device__ __forceinline__ void st(uint16_t* p, float v) { *p = (uint16_t)f32_to_bf16_bits(v); }
};

constexpr float kLog2E = 1.4426950408889634f;
// 1 / (1 + e^-v) on the hardware's 2^x and reciprocal (each within one unit in the last place)
__device__ __forceinline__ float sigmoid_d(float v) {
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-v * kLog2E));
}

// exp(neg_a * softplus(raw + bias)).  softplus(v) = max(v, 0) + log(1 + e) with e = exp(-|v|), and
// log(1 + e) = 2 artanh(s), s = e / (2 + e) <= 1/3, by its series to s^15 (the rest is below 2e-9 of the sum): the
// relative precision stays where e is small - a gate next to one, applied a thousand times over.
__device__ __forceinline__ float decay_gate(float raw, float bias, float neg_a) {
    const float v = raw + bias;
    const float e = __builtin_amdgcn_exp2f(-fabsf(v) * kLog2E);
    const float s = e * __builtin_amdgcn_rcpf(2.0f + e), s2 = s * s;
    float c = fmaf(s2, 1.0f / 15.0f, 1.0f / 13.0f);
    c = fmaf(s2, c, 1.0f / 11.0f);
    c = fmaf(s2, c, 1.0f / 9.0f);
    c = fmaf(s2, c, 1.0f / 7.0f);
    c = fmaf(s2, c, 1.0f / 5.0f);
    c = fmaf(s2, c, 1.0f / 3.0f);
    c = fmaf(s2, c, 1.0f);
    const float sp = fmaf(2.0f * s, c, fmaxf(v, 0.f));
    return __builtin_amdgcn_exp2f((neg_a * kLog2E) * sp);
}

// v_mfma_f32_16x16x4_f32 (true fp32): operand A lane (r, g) = A[r][g], B lane (r, g) = B[g][r], result lane (r, g) =
// C[4 g + j][r] (r = lane % 16, g = lane / 16).  The contraction index is a label: in step j of a group of 16, slot g may
// stand for index 4 g + j, so a result can be the next product's operand B where it lies and operand A is a 16-byte read.
#define MV_DMFMA(acc, a_, b_) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a_, b_, acc, 0, 0, 0)

__device__ __forceinline__ int pad16(int v) { return (v + 15) & ~15; }

}  // namespace mv
