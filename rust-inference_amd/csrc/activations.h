// The activations of feed-forwards without a gate, in float32.
#pragma once
#include "common.h"

#define PN_ACT_GELU_ERF 0
#define PN_ACT_GELU_TANH 1
#define PN_ACT_RELU2 2

__device__ __forceinline__ float pn_activate(float v, int kind) {
    if (kind == PN_ACT_GELU_ERF) return 0.5f * v * (1.f + erff(v * 0.7071067811865476f));
    if (kind == PN_ACT_GELU_TANH) return 0.5f * v * (1.f + tanhf(0.7978845608028654f * (v + 0.044715f * v * v * v)));
    const float r = fmaxf(v, 0.f);
    return r * r;
}
