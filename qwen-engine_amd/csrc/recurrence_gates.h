// Activations and gates that the kernels of the recurrences apply as they read their operands, all in 32-bit.
#pragma once
#include "common.h"

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
// sigmoid(z) and sigmoid(-z), neither by a difference.  exp(-|z|) from the hardware's exponential of base 2 with the
// rounding of the argument's product put back (a few parts in 10^7; nothing here overflows: the argument is not positive).
__device__ __forceinline__ void sigmoid_both(float z, float& pos, float& neg) {
    const float x = -fabsf(z);
    const float t = x * 1.44269502f;                         // log2(e), high part
    const float lost = fmaf(x, 1.92596303e-8f, fmaf(x, 1.44269502f, -t));
    const float e0 = __builtin_amdgcn_exp2f(t);
    const float e = fmaf(e0 * 0.693147182f, lost, e0);
    const float big = __builtin_amdgcn_rcpf(1.f + e), small = e * big;
    pos = z >= 0.f ? big : small;
    neg = z >= 0.f ? small : big;
}
__device__ __forceinline__ float silu_quick(float z) {
    float p, n;
    sigmoid_both(z, p, n);
    return z * p;
}
// f = l + (1 - l) sigmoid(z) and 1 - f
__device__ __forceinline__ void forget_gate(float z, float l, float& f, float& kf) {
    float p, n;
    sigmoid_both(z, p, n);
    f = fmaf(1.f - l, p, l);
    kf = (1.f - l) * n;
}
