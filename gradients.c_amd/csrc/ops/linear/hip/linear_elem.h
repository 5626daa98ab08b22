/*
 * Element type of the projection kernels.  The kernels are written over gd_elem; a translation unit that defines
 * GD_LINEAR_BF16 before including them (linear_bf16.hip, linear_tile_bf16.hip, linear_wide_bf16.hip) gets BF16
 * operands, every other one F16.  The matrix instructions of the two types have the same shape, rate and operand
 * layout, so nothing else differs, except that the BF16 build
 *   - instantiates only what its callers use: [N,K] weights, no prologue, no rotation epilogue;
 *   - keeps a gated projection in F32 up to the product with the gate (the F16 build rounds value and gate first,
 *     as the reference's separate operators do), and knows further gate functions (GD_HIP_LINEAR_GELU_GATE,
 *     GD_HIP_LINEAR_CLAMPED_GATE) and the square of relu (GD_HIP_LINEAR_SQUARE_RELU);
 *   - can store F32 results (GD_HIP_LINEAR_Y_F32; few-row kernels only).
 */
#ifndef GD_LINEAR_ELEM_H
#define GD_LINEAR_ELEM_H
#include "../../_shared/hip_device.h"

#ifdef GD_LINEAR_BF16
typedef gd_bf16 gd_elem;
typedef gd_bf16x8 gd_elem8;
typedef gd_bf16x4 gd_elem4;
#define GD_MFMA_16X16X32(a, b, c) __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0)
#define GD_MFMA_32X32X16(a, b, c) __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0)
#define GD_LINEAR_FN(name) name##_bf16
#define GD_LINEAR_IS_BF16 1
#else
typedef gd_half gd_elem;
typedef gd_half8 gd_elem8;
typedef gd_half4 gd_elem4;
#define GD_MFMA_16X16X32(a, b, c) __builtin_amdgcn_mfma_f32_16x16x32_f16(a, b, c, 0, 0, 0)
#define GD_MFMA_32X32X16(a, b, c) __builtin_amdgcn_mfma_f32_32x32x16_f16(a, b, c, 0, 0, 0)
#define GD_LINEAR_FN(name) name
#define GD_LINEAR_IS_BF16 0
#endif

#if GD_LINEAR_IS_BF16
/* g sigmoid(alpha g) (v + 1), g = min(gate, limit), v = value kept within +-limit; the result is rounded to 16 bits */
__device__ __forceinline__ float gd_lin_clamped_gate(float value, float gate, float limit, float alpha)
{
    const float g = fminf(gate, limit), v = fminf(fmaxf(value, -limit), limit);
    return g * gd_sigmoid_fast(alpha * g) * (v + 1.0f);
}

/* value * gate function of a gated projection, both still F32 */
__device__ __forceinline__ float gd_lin_gated(float value, float gate, const gd_hip_linear_params &p)
{
    if (p.flags & GD_HIP_LINEAR_CLAMPED_GATE) return gd_lin_clamped_gate(value, gate, p.gate_limit, p.gate_alpha);
    if (p.flags & GD_HIP_LINEAR_GELU_GATE) return value * gd_gelu_tanh_f32(gate);
    return value * gd_silu_f32(gate);
}

/* what becomes of an output that is not gated */
__device__ __forceinline__ float gd_lin_activated(float u, uint32_t flags)
{
    if (flags & GD_HIP_LINEAR_SQUARE_RELU) return u > 0.f ? u * u : 0.f;
    return u;
}
#endif

#endif
