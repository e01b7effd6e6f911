// Activation formulas that more than one kernel file uses.
#pragma once

#include "common.h"

__device__ __forceinline__ float squared_relu(float x) {
    const float y = fmaxf(x, 0.f);
    return y * y;
}

// gelu in its tanh form, 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), as z * sigmoid(2 sqrt(2 / pi) (z + ...)).
__device__ __forceinline__ float gelu_tanh(float z) {
    constexpr float kTwice = 1.5957691216057308f;  // 2 sqrt(2 / pi)
    return z / (1.0f + expf(-kTwice * fmaf(0.044715f * z * z, z, z)));
}

// A gated unit with bounded inputs: g' = min(g, limit), u' = clamp(u, -limit, limit),
// y = g' * sigmoid(alpha * (g' + cubic * g'^3)) * (u' + offset).  float32.  cubic = 0 is the plain sigmoid gate;
// alpha = 2 sqrt(2 / pi), cubic = 0.044715 is the tanh form of gelu, 0.5 g (1 + tanh(sqrt(2 / pi) (g + 0.044715 g^3))),
// since 0.5 (1 + tanh z) = sigmoid(2 z).
__device__ __forceinline__ float clamped_glu(float g, float u, float limit, float alpha, float offset, float cubic = 0.f) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    const float inner = cubic != 0.f ? fmaf(cubic * g * g, g, g) : g;
    return g / (1.0f + expf(-alpha * inner)) * (u + offset);
}
