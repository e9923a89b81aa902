// The activations of one value that kernels apply, by code: 0 SiLU, 1 GELU in its tanh form
// 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), 2 GELU with the error function, 3 relu(z)^2.
#pragma once
#include "zi_common.h"

#define ZI_ACT_SILU 0
#define ZI_ACT_GELU_TANH 1
#define ZI_ACT_GELU_ERF 2
#define ZI_ACT_RELU2 3

__device__ __forceinline__ float zi_activation(float z, int act) {
    if (act == ZI_ACT_GELU_TANH) return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
    if (act == ZI_ACT_GELU_ERF) return 0.5f * z * (1.f + erff(z * 0.70710678118654752440f));
    return z / (1.f + expf(-z));
}

// The same for a launch of its own and for a product's epilogue (ERF false there: no caller has that code).  The tanh form as
// z / (1 + e^(-2u)), u = sqrt(2 / pi) (z + 0.044715 z^3), which is the same and loses nothing to cancellation; ROUGH, for
// bfloat16 results, by the chip's exponential and reciprocal.
template <bool ROUGH, bool ERF = true>
__device__ __forceinline__ float zi_activate_value(float z, int act) {
    if (act == ZI_ACT_RELU2) {
        const float p = fmaxf(z, 0.f);
        return p * p;
    }
    if (ERF && act == ZI_ACT_GELU_ERF) return zi_activation(z, act);
    const float w = act == ZI_ACT_GELU_TANH ? -2.f * 0.7978845608028654f * z * fmaf(0.044715f * z, z, 1.f) : -z;
    return ROUGH ? z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(w * 1.4426950408889634f)) : z / (1.f + expf(w));
}
