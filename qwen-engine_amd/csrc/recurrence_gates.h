// Activations and gates that the kernels of the recurrences apply as they read their operands, all in 32-bit.
#pragma once
#include "common.h"

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
// f = l + (1 - l) sigmoid(z) and 1 - f, neither by a difference
__device__ __forceinline__ void forget_gate(float z, float l, float& f, float& kf) {
    const float e = expf(-fabsf(z));
    const float big = 1.f / (1.f + e), small = e * big;
    f = fmaf(1.f - l, z >= 0.f ? big : small, l);
    kf = (1.f - l) * (z >= 0.f ? small : big);
}
