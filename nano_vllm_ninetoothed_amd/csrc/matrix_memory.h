// Gates of the matrix memory (decayed_recurrence.hip): both are logarithms.
#pragma once
#include "mixed_types.h"

namespace mops {

constexpr float kMemoryEps = 1e-6f;      // added to the denominator

__device__ __forceinline__ float capped_gate(float x, float cap) { return cap * tanhf(x / cap); }
__device__ __forceinline__ float log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }

}  // namespace mops
