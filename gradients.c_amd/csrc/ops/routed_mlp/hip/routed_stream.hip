/*
 * Projections of few rows per expert (gfx950, BF16): the decode form of a routed feed-forward.  HBM-bound on the weights
 * of the experts that have rows.
 *
 * A workgroup takes one tile of the work list (up to 16 packed rows of one expert) and 16 * NT weight rows; its
 * wavefronts split K and are summed through LDS, like gd_linear_stream_kernel (ops/linear/hip/linear_stream_kernel.h).
 * Both operands of the matrix instruction are fetched with one 16-byte load per lane straight from memory; the loads of
 * the next U steps are requested while the matrix cores work on the current ones.  Gated: half of the column tiles are
 * value rows, the other half the matching gate rows, and a thread that adds up a value finds its gate beside it.
 *
 * MFMA operand layout (v_mfma_f32_16x16x32_bf16): lane l supplies row / column l % 16 and the 8 consecutive k starting
 * at 8 * (l / 16); the result lane holds column l % 16, rows 4 * (l / 16) .. + 3.
 */
#include "../../_shared/hip_device.h"
#include "hip_routed_mlp_types.h"

#define GD_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0)

/* grid (ceil(n / outputs of a workgroup), max_tiles); k % 8 == 0 */
template <int NT, int WAVES, bool GATED>
__global__ void __launch_bounds__(WAVES * 64)
gd_routed_stream_kernel(const gd_bf16 *__restrict__ x, const gd_bf16 *__restrict__ w, gd_bf16 *__restrict__ y,
                        const int32_t *__restrict__ first, const int32_t *__restrict__ tiles, gd_hip_routed_params p)
{
    constexpr int U = NT >= 4 ? 2 : 4;
    constexpr int OT = GATED ? NT / 2 : NT; /* column tiles that produce outputs */
    __shared__ float sm[WAVES][NT][64][4];
    const uint32_t lane = threadIdx.x & 63u, li = lane & 15u, lg = lane >> 4;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t e = (uint32_t)tiles[2u + 2u * blockIdx.y], m0 = (uint32_t)tiles[3u + 2u * blockIdx.y];
    if (blockIdx.y >= (uint32_t)tiles[0]) return; /* (the list has room for max_tiles: what lies behind it is not used) */
    const uint32_t m_end = (uint32_t)first[e + 1u], n0 = blockIdx.x * (16u * OT);
    const gd_bf16 *we = w + (size_t)e * (GATED ? 2u : 1u) * p.n * p.k;
    const gd_bf16 *xr = x + (size_t)min(m0 + li, m_end - 1u) * p.k;
    const gd_bf16 *wr[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) {
        const uint32_t n = min(n0 + 16u * (uint32_t)(j % OT) + li, p.n - 1u);
        wr[j] = we + (size_t)(j >= OT ? p.n + n : n) * p.k;
    }
    const uint32_t steps = (p.k + 31u) / 32u, per = (steps + WAVES - 1u) / WAVES;
    const uint32_t s_begin = wave * per, s_end = min(s_begin + per, steps);
    const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
    gd_float4 acc[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[j] = (gd_float4){0.f, 0.f, 0.f, 0.f};
    gd_bf16x8 xa[2][U], wa[2][U][NT];
    auto load = [&](gd_bf16x8 (&xv)[U], gd_bf16x8 (&wv)[U][NT], uint32_t s0) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const uint32_t k = 32u * (s0 + (uint32_t)u) + 8u * lg;
            const bool ok = s0 + (uint32_t)u < s_end && k < p.k;
            const uint32_t at = ok ? k : 0u; /* a place that exists; the row's fragment is zero instead */
            xv[u] = *reinterpret_cast<const gd_bf16x8 *>(xr + at);
            if (!ok) xv[u] = zero;
#pragma unroll
            for (int j = 0; j < NT; ++j) wv[u][j] = ok ? *reinterpret_cast<const gd_bf16x8 *>(wr[j] + at) : zero;
        }
    };
    auto multiply = [&](const gd_bf16x8 (&xv)[U], const gd_bf16x8 (&wv)[U][NT]) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int j = 0; j < NT; ++j) acc[j] = GD_MFMA(xv[u], wv[u][j], acc[j]);
    };
    if (s_begin < s_end) load(xa[0], wa[0], s_begin);
    for (uint32_t s = s_begin; s < s_end; s += 2u * U) {
        if (s + U < s_end) load(xa[1], wa[1], s + U);
        multiply(xa[0], wa[0]);
        if (s + 2u * U < s_end) load(xa[0], wa[0], s + 2u * U);
        if (s + U < s_end) multiply(xa[1], wa[1]);
    }
#pragma unroll
    for (int j = 0; j < NT; ++j) *reinterpret_cast<gd_float4 *>(&sm[wave][j][lane][0]) = acc[j];
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < OT * 256u; i += WAVES * 64u) {
        const uint32_t j = i >> 8, l = i & 63u, r = (i >> 6) & 3u;
        const uint32_t row = m0 + 4u * (l >> 4) + r, col = n0 + 16u * j + (l & 15u);
        if (row >= m_end || col >= p.n) continue;
        float v = 0.f, g = 0.f;
#pragma unroll
        for (int t = 0; t < WAVES; ++t) {
            v += sm[t][j][l][r];
            if (GATED) g += sm[t][GATED ? j + OT : j][l][r];
        }
        if (GATED) {
            g = fminf(g, p.gate_limit);
            v = g * gd_sigmoid_fast(p.gate_alpha * g) * (fminf(fmaxf(v, -p.gate_limit), p.gate_limit) + 1.0f);
        }
        y[(size_t)row * p.n + col] = (gd_bf16)v;
    }
}

/* The caller has checked: BF16, k % 8 == 0, 16-byte aligned x and w, tiles of 16 rows, max_tiles <= 65535. */
extern "C" int gd_hip_launch_routed_stream(hipStream_t stream, const void *x, const void *w, void *y, const int32_t *first,
                                           const int32_t *tiles, const gd_hip_routed_params *p)
{
    const uint32_t steps = (p->k + 31u) / 32u, outs = p->gated ? 16u : 32u;
    const dim3 grid((p->n + outs - 1u) / outs, p->max_tiles);
#define GD_GO(W, G) gd_routed_stream_kernel<2, W, G><<<grid, W * 64, 0, stream>>>((const gd_bf16 *)x, (const gd_bf16 *)w, (gd_bf16 *)y, first, tiles, *p)
    if (steps <= 16u) { if (p->gated) GD_GO(4, true); else GD_GO(4, false); }
    else { if (p->gated) GD_GO(8, true); else GD_GO(8, false); }
#undef GD_GO
    return (int)hipGetLastError();
}
