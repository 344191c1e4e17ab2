// Activations of gated feed-forwards, shared by the dense and the experts' kernels.
#pragma once
#include "common.h"

// act: 0 silu, 1 relu (max(g, 0)), 2 gelu with the tanh form 0.5 g (1 + tanh(sqrt(2/pi) (g + 0.044715 g^3))),
// 3 g sigmoid(1.702 g).
__device__ __forceinline__ float gate_activation(float g, int act) {
    if (act == 1) return fmaxf(g, 0.f);
    if (act == 3) return g / (1.0f + expf(-1.702f * g));      // g sigmoid(1.702 g)
    if (act == 2) return 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
    return g / (1.0f + expf(-g));
}

// limit > 0: g is cut off above at limit and u is held inside [-limit, limit] first; up_offset is added to u (after
// the limit).
__device__ __forceinline__ float gated_value(float g, float u, int act, float limit, float up_offset) {
    if (limit > 0.f) {
        g = fminf(g, limit);
        u = fminf(fmaxf(u, -limit), limit);
    }
    return gate_activation(g, act) * (u + up_offset);
}
