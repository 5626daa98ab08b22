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

/* The same for BF16 with 2 to 4 taps and 16-byte aligned rows: a thread carries 8 channels through up to `run` rows with
 * the last K - 1 inputs in registers, so every input is read once and whole cache lines move. */
template <int K>
__global__ void __launch_bounds__(256)
gd_causal_conv_silu_vec_kernel(const gd_bf16 *__restrict__ u, uint32_t ldu, const float *__restrict__ w,
                               const float *__restrict__ bias, gd_bf16 *__restrict__ ring, gd_bf16 *__restrict__ out,
                               uint32_t C, gd_hip_seqs q, uint32_t run, int store_ring)
{
    const uint32_t chunks = C / 8u, idx = blockIdx.x * 256u + threadIdx.x, c = (idx % chunks) * 8u;
    const uint32_t r0 = idx / chunks * run, r1 = min(r0 + run, q.rows);
    if (r0 >= q.rows) return;
    float taps[K][8], b[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        b[e] = bias[c + e];
#pragma unroll
        for (int k = 0; k < K; ++k) taps[k][e] = w[(size_t)(c + e) * K + k];
    }
    gd_bf16x8 win[K]; /* win[k]: input k tokens back; win[0]: the current one */
    int32_t seq = -1;
    for (uint32_t row = r0; row < r1; ++row) {
        int32_t s, pos, slot;
        if (!gd_seq_of_row(q, row, &s, &pos, &slot)) {
            seq = -1;
            continue;
        }
        gd_bf16 *rg = ring + (size_t)slot * K * C + c;
#pragma unroll
        for (int k = K - 1; k > 0; --k) win[k] = win[k - 1];
        if (s != seq) { /* first row of this thread in the sequence: what lies in front of it */
            const int32_t start = q.start[s];
#pragma unroll
            for (int k = 1; k < K; ++k) {
                const int32_t p = pos - k;
                win[k] = (gd_bf16x8)(gd_bf16)0.f;
                if (p >= start) win[k] = *reinterpret_cast<const gd_bf16x8 *>(u + (size_t)(row - (uint32_t)k) * ldu + c);
                else if (p >= 0) win[k] = *reinterpret_cast<const gd_bf16x8 *>(rg + (size_t)((uint32_t)p % K) * C);
            }
            seq = s;
        }
        win[0] = *reinterpret_cast<const gd_bf16x8 *>(u + (size_t)row * ldu + c);
        gd_bf16x8 o;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float acc = fmaf(taps[K - 1][e], (float)win[0][e], b[e]);
#pragma unroll
            for (int k = 1; k < K; ++k) acc = fmaf(taps[K - 1 - k][e], (float)win[k][e], acc);
            o[e] = (gd_bf16)(acc * gd_sigmoid_fast(acc));
        }
        *reinterpret_cast<gd_bf16x8 *>(out + (size_t)row * C + c) = o;
        if (store_ring) *reinterpret_cast<gd_bf16x8 *>(rg + (size_t)((uint32_t)pos % K) * C) = win[0];
    }
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
                                              const gd_hip_seqs *q, int is_f32, int aligned16)
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
    if (!is_f32 && aligned16 && (C % 8u) == 0u && K >= 2u && K <= 4u) {
        const uint32_t run = q->rows >= 512u ? 16u : 1u;
        const uint64_t threads = (uint64_t)(C / 8u) * ((q->rows + run - 1u) / run);
        const unsigned blocks = (unsigned)((threads + 255u) / 256u);
#define GD_VEC(KV) gd_causal_conv_silu_vec_kernel<KV><<<blocks, 256, 0, stream>>>((const gd_bf16 *)u, ldu, w, bias, (gd_bf16 *)ring, (gd_bf16 *)out, C, *q, run, single)
        if (K == 2u) GD_VEC(2);
        else if (K == 3u) GD_VEC(3);
        else GD_VEC(4);
#undef GD_VEC
        if (!single)
            gd_causal_conv_ring_kernel<gd_bf16><<<grid_ring, 256, 0, stream>>>((const gd_bf16 *)u, ldu, (gd_bf16 *)ring, C, K, *q);
        return (int)hipGetLastError();
    }
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}
