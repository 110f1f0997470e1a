// Activations of gated feed-forwards.
#pragma once
#include "hm_common.h"

namespace homura {

// act(gate) * up of a gated feed-forward. Silu: silu(g) u. ClampedSigmoid: with g = min(g, limit) and u clamped to
// [-limit, limit], g sigmoid(slope g) (u + 1).
struct GatedAct {
    enum Kind { Silu = 0, ClampedSigmoid = 1 };
    int kind = Silu;
    float limit = 0.f, slope = 1.f;
};
__device__ __forceinline__ float gated_act(const GatedAct &a, float g, float u) {
    if (a.kind == GatedAct::ClampedSigmoid) {
        g = fminf(g, a.limit);
        u = fminf(fmaxf(u, -a.limit), a.limit) + 1.0f;
        return g / (1.0f + expf(-a.slope * g)) * u;
    }
    return g / (1.0f + expf(-g)) * u;
}

}  // namespace homura
