// stream32_epilogue.h -- what follows the sum of a full-precision linear of the f32-stream designs (kernels_stream32.h: LinearF32Params), shared by its forms
// (k_stream32.hip: few rows, tile; k_linear_mfma.hip: matrix cores).
#pragma once

#include "device_utils.h"
#include "kernels_stream32.h"

namespace uzu {
namespace k {

__device__ __forceinline__ float gelu_tanh_f32(float z) { return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))); }

// The matrix-core form unrolls its epilogue over 64 sums per thread: one kernel with every branch inlined 64 times does not fit the instruction cache, so it is
// compiled for what a launch uses.
enum EpilogueKind {
    kEpilogueLean,  // bias, act 0 / 1, scale, residual
    kEpilogueXielu, // ... with act 3
    kEpilogueFull
};
inline EpilogueKind epilogue_kind(const LinearF32Params& p) {
    if (p.soft_cap != 0.0f || p.gate || p.mul_table || p.act == 2) return kEpilogueFull;
    return p.act == 3 ? kEpilogueXielu : kEpilogueLean;
}

// act: 0 none, 1 max(v, 0)^2, 2 gelu (tanh form), 3 a v^2 + v / 2 for v > 0, b (e^v - 1 - v) + v / 2 otherwise
template <int KIND = kEpilogueFull> __device__ __forceinline__ float linear_act(float v, const LinearF32Params& p) {
    if (KIND != kEpilogueXielu && p.act == 1) {
        const float t = fmaxf(v, 0.0f);
        return t * t;
    }
    if (KIND == kEpilogueFull && p.act == 2) return gelu_tanh_f32(v);
    if (KIND == kEpilogueXielu || (KIND == kEpilogueFull && p.act == 3)) {
        const float n = fminf(v, 0.0f);
        const float curve = v > 0.0f ? p.act_a * v * v : p.act_b * (expm1f(n) - n);
        return fmaf(0.5f, v, curve);
    }
    return v;
}

// bias, activation, the product's scale, the cap, a sigmoid gate (per product or per column), a multiplier per (row's token, column) -- everything in front of the
// residual row
template <int KIND = kEpilogueFull> __device__ __forceinline__ float linear_value(float sum, float bias, const LinearF32Params& p, uint32_t row, uint32_t z, uint32_t n) {
    float v = linear_act<KIND>(sum + bias, p);
    if (p.y_scale != 0.0f) v *= p.y_scale;
    if (KIND != kEpilogueFull) return v;
    if (p.soft_cap != 0.0f) v = p.soft_cap * tanhf(v / p.soft_cap);
    if (p.gate) v *= 1.0f / (1.0f + expf(-p.gate[(size_t)row * p.ldgate + (p.gate_batch ? (size_t)z * p.gate_batch + n : z)]));
    if (p.mul_table) {
        uint32_t t = p.mul_tokens[row];
        if (t >= p.mul_vocab) t = 0;
        v *= bf16_to_f32(p.mul_table[(size_t)t * p.mul_ld + p.mul_col0 + n]);
    }
    return v;
}
__device__ __forceinline__ float linear_epilogue(float sum, float bias, const LinearF32Params& p, uint32_t row, uint32_t z, uint32_t n) {
    const float v = linear_value(sum, bias, p, row, z, n);
    return p.residual ? v + p.residual[(size_t)row * p.ldr + n] : v;
}

} // namespace k
} // namespace uzu
