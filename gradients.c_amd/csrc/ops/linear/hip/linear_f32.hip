/*
 * Projections over F32 operands in true 32-bit arithmetic (fused multiply-adds, no reduced-precision matrix mode):
 * y = x w^T [+ bias], optionally gated.  This is the precision reference of the 16-bit kernels, not a speed path: a
 * 64 x 64 output tile per workgroup of 256 threads, 4 x 4 outputs per thread, K in LDS tiles of 16.  Any shape, any
 * 4-byte aligned pitch, [N,K] weights.
 */
#include "../../_shared/hip_device.h"
#include "hip_linear_types.h"

#define GD_F32_TILE 64
#define GD_F32_BK 16

/* GATED: w has 2 * swiglu_cols rows, the gate of output column n in row swiglu_cols + n */
template <bool GATED>
__global__ void __launch_bounds__(256)
gd_linear_f32_kernel(const float *__restrict__ x, const float *__restrict__ w, const float *__restrict__ bias,
                     float *__restrict__ y, gd_hip_linear_params p)
{
    __shared__ float sx[GD_F32_BK][GD_F32_TILE + 4], sw[GATED ? 2 : 1][GD_F32_BK][GD_F32_TILE + 4];
    const uint32_t m0 = blockIdx.y * GD_F32_TILE, n0 = blockIdx.x * GD_F32_TILE;
    const uint32_t tx = threadIdx.x & 15u, ty = threadIdx.x >> 4;
    float acc[GATED ? 2 : 1][4][4] = {};
    for (uint32_t k0 = 0; k0 < p.K; k0 += GD_F32_BK) {
        for (uint32_t i = threadIdx.x; i < GD_F32_TILE * GD_F32_BK; i += 256u) {
            const uint32_t r = i / GD_F32_BK, k = i % GD_F32_BK;
            const bool kok = k0 + k < p.K, nok = kok && n0 + r < p.N;
            sx[k][r] = kok && m0 + r < p.M ? x[(size_t)(m0 + r) * p.ldx + k0 + k] : 0.f;
            sw[0][k][r] = nok ? w[(size_t)(n0 + r) * p.ldw + k0 + k] : 0.f;
            if (GATED) sw[GATED ? 1 : 0][k][r] = nok ? w[(size_t)(p.swiglu_cols + n0 + r) * p.ldw + k0 + k] : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (uint32_t k = 0; k < GD_F32_BK; ++k) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float a = sx[k][ty + 16u * i];
#pragma unroll
                for (int g = 0; g < (GATED ? 2 : 1); ++g)
#pragma unroll
                    for (int j = 0; j < 4; ++j) acc[g][i][j] = fmaf(a, sw[g][k][tx + 16u * j], acc[g][i][j]);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const uint32_t m = m0 + ty + 16u * i, n = n0 + tx + 16u * j;
            if (m >= p.M || n >= p.N) continue;
            float v = acc[0][i][j] + (p.epilogue != GD_HIP_EPI_NONE ? bias[n] : 0.f);
            if (GATED) {
                const float g = acc[GATED ? 1 : 0][i][j] + (p.epilogue != GD_HIP_EPI_NONE ? bias[p.swiglu_cols + n] : 0.f);
                /* the accurate functions: this path is held to 32-bit rounding */
                if (p.flags & GD_HIP_LINEAR_CLAMPED_GATE) {
                    const float c = fminf(g, p.gate_limit);
                    v = c / (1.0f + expf(-p.gate_alpha * c)) * (fminf(fmaxf(v, -p.gate_limit), p.gate_limit) + 1.0f);
                } else if (p.flags & GD_HIP_LINEAR_GELU_GATE)
                    v *= 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
                else v *= g / (1.0f + expf(-g));
            }
            if (!GATED && (p.flags & GD_HIP_LINEAR_SQUARE_RELU)) v = v > 0.f ? v * v : 0.f;
            y[(size_t)m * p.ldy + n] = v;
        }
    }
}

extern "C" int gd_hip_launch_linear_f32(hipStream_t stream, const void *x, const void *w, const void *bias, void *y,
                                        const gd_hip_linear_params *params)
{
    const gd_hip_linear_params &p = *params;
    if (p.M == 0u || p.N == 0u) return (int)hipSuccess;
    const dim3 grid((p.N + GD_F32_TILE - 1u) / GD_F32_TILE, (p.M + GD_F32_TILE - 1u) / GD_F32_TILE);
    if (p.swiglu_cols != 0u)
        gd_linear_f32_kernel<true><<<grid, 256, 0, stream>>>((const float *)x, (const float *)w, (const float *)bias, (float *)y, p);
    else
        gd_linear_f32_kernel<false><<<grid, 256, 0, stream>>>((const float *)x, (const float *)w, (const float *)bias, (float *)y, p);
    return (int)hipGetLastError();
}
