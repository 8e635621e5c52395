// The gate unit of feed-forwards with clamped halves: gate * sigmoid(alpha * gate) * (up + shift), gate = min(g, limit), up = clamp(u,
// -limit, limit) (limit infinite: unclamped), in 32-bit.
#pragma once

#include "common.h"

struct GateUnit {
    float limit, alpha, shift;
};

__device__ __forceinline__ float gated(float g, float u, const GateUnit& unit) {
    g = fminf(g, unit.limit);
    u = fminf(fmaxf(u, -unit.limit), unit.limit);
    return g / (1.0f + expf(-unit.alpha * g)) * (u + unit.shift);
}
