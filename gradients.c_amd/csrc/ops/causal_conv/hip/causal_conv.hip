/*
 * Short causal convolution per channel with its activation (gfx950): y[t, c] = silu(bias[c] + sum_k w[c, K-1-k]
 * u[t-k, c]), zeros before position 0.
 *
 * The last inputs of every sequence live in a ring [slots, K, C] whose place p % K holds the input of position p.
 * Positions in front of the packed rows are read there, positions below 0 are zeros, so a slot that is used again
 * needs no clearing, and a decode step (one token per sequence) may store its own input while it reads the K-1
 * places before it: they are never the same.  With more than one token per sequence the places do coincide, so the
 * ring is then written by a second launch behind the first.
 */
#include "../../_shared/hip_device.h"
#include "../../_shared/packed_seqs.h"

template <typename T>
__global__ void __launch_bounds__(256)
gd_causal_conv_silu_kernel(const T *__restrict__ u, uint32_t ldu, const float *__restrict__ w,
                           const float *__restrict__ bias, T *__restrict__ ring, T *__restrict__ out, uint32_t C,
                           uint32_t K, gd_hip_seqs q, int store_ring)
{
    const uint32_t row = blockIdx.x, c = blockIdx.y * 256u + threadIdx.x;
    int32_t s, pos, slot;
    if (c >= C || !gd_seq_of_row(q, row, &s, &pos, &slot)) return;
    const int32_t start = q.start[s];
    T *rg = ring + (size_t)slot * K * C + c;
    const float *wc = w + (size_t)c * K;
    const T now = u[(size_t)row * ldu + c];
    float acc = fmaf(wc[K - 1u], (float)now, bias[c]);
    for (uint32_t k = 1u; k < K; ++k) {
        const int32_t p = pos - (int32_t)k;
        if (p < 0) break;
        const float v = p >= start ? (float)u[(size_t)(row - k) * ldu + c] : (float)rg[(size_t)((uint32_t)p % K) * C];
        acc = fmaf(wc[K - 1u - k], v, acc);
    }
    out[(size_t)row * C + c] = (T)gd_silu_f32(acc);
    if (store_ring) rg[(size_t)((uint32_t)pos % K) * C] = now;
}

/* the last K inputs of every sequence's new rows into its ring */
template <typename T>
__global__ void __launch_bounds__(256)
gd_causal_conv_ring_kernel(const T *__restrict__ u, uint32_t ldu, T *__restrict__ ring, uint32_t C, uint32_t K,
                           gd_hip_seqs q)
{
    const uint32_t c = blockIdx.y * 256u + threadIdx.x;
    int32_t first, n, start, slot;
    if (c >= C || !gd_seq_span(q, blockIdx.x, &first, &n, &start, &slot)) return;
    T *rg = ring + (size_t)slot * K * C + c;
    for (int32_t i = n > (int32_t)K ? n - (int32_t)K : 0; i < n; ++i)
        rg[(size_t)((uint32_t)(start + i) % K) * C] = u[(size_t)(first + i) * ldu + c];
}

extern "C" int gd_hip_launch_causal_conv_silu(hipStream_t stream, const void *u, uint32_t ldu, const float *w,
                                              const float *bias, void *ring, void *out, uint32_t C, uint32_t K,
                                              const gd_hip_seqs *q, int is_f32)
{
    const dim3 grid(q->rows, (C + 255u) / 256u), grid_ring(q->seqs, (C + 255u) / 256u);
    const int single = q->max_new == 1u;
#define GD_GO(T)                                                                                                       \
    do {                                                                                                               \
        gd_causal_conv_silu_kernel<T><<<grid, 256, 0, stream>>>((const T *)u, ldu, w, bias, (T *)ring, (T *)out, C, K, \
                                                                *q, single);                                          \
        if (!single) gd_causal_conv_ring_kernel<T><<<grid_ring, 256, 0, stream>>>((const T *)u, ldu, (T *)ring, C, K, *q); \
    } while (0)
    if (q->rows == 0u || q->seqs == 0u || C == 0u || K == 0u) return (int)hipSuccess;
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}
