// What an expert does with its first matrix's rows: the forms that the kernels for few rows and for many share.
#pragma once
#include "common.h"

enum ExpertForm : int { EXPERT_GATED_SILU = 0, EXPERT_GELU = 1, EXPERT_CAPPED = 2, EXPERT_RELU_SQUARED = 3 };

// gated forms have a gate row and an up row for each inner value, plain ones an up row
__host__ __device__ inline bool expert_is_gated(int form) { return form == EXPERT_GATED_SILU || form == EXPERT_CAPPED; }

struct ExpertCap { float limit, slope, shift; };

__device__ inline float expert_silu_gated(float g, float u) { return g / (1.0f + expf(-g)) * u; }
__device__ inline float expert_gelu(float z) { return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f)); }
__device__ inline float expert_relu_squared(float z) { const float p = fmaxf(z, 0.f); return p * p; }
__device__ inline float expert_plain(int form, float z) { return form == EXPERT_GELU ? expert_gelu(z) : expert_relu_squared(z); }
__device__ inline float expert_capped(float gate, float up, const ExpertCap& c) {
    const float g = fminf(gate, c.limit);
    const float u = fminf(fmaxf(up, -c.limit), c.limit);
    return g * (1.0f / (1.0f + expf(-c.slope * g))) * (u + c.shift);
}
