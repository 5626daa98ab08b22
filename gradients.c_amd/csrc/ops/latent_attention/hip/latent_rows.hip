/*
 * Row kernels of latent attention (gfx950), any sizes, BF16 and F32:
 *   prepare  per new token: cosines and sines of its position; RMS norm of the query latent; RMS norm of the key/value
 *            latent and rotation of the shared key part, both into the token's cache row
 *   query    per token and head: the unrotated query taken through the key up-projection, so that its product with a
 *            latent is its product with the key (q . (W_uk c) = (W_uk^T q) . c), and the rotated part turned to its
 *            position: one absorbed query row of a cache row's layout
 *   attend   per token and head: softmax over the sequence's cache rows up to the token's own, and the weighted sum of
 *            their latents (scores, weights and sums in F32)
 *   value    per token and head: the value up-projection of that sum, times the sigmoid of the output gate
 * They are the F32 path and the path of sizes outside the matrix-core kernels (latent_decode.hip, latent_prefill.hip).
 */
#include "../../_shared/hip_device.h"
#include "hip_latent_attention_types.h"

template <typename T>
__global__ void __launch_bounds__(256)
gd_latent_prepare_kernel(const T *__restrict__ proj, uint32_t ld, const float *__restrict__ q_norm,
                         const float *__restrict__ kv_norm, const float *__restrict__ freq, float *__restrict__ angles,
                         T *__restrict__ cq, T *__restrict__ cache, gd_hip_latent_params m, gd_hip_seqs q)
{
    __shared__ float red[2][4];
    const uint32_t row = blockIdx.x;
    const T *pq = proj + (size_t)row * ld, *pc = pq + m.q_rank, *pr = pc + m.kv_rank;
    int32_t s, pos, slot;
    const bool live = gd_seq_of_row(q, row, &s, &pos, &slot) && (uint32_t)pos < m.tmax;
    float sq = 0.f, sc = 0.f;
    for (uint32_t c = threadIdx.x; c < m.q_rank; c += 256u) sq = fmaf((float)pq[c], (float)pq[c], sq);
    for (uint32_t c = threadIdx.x; c < m.kv_rank; c += 256u) sc = fmaf((float)pc[c], (float)pc[c], sc);
    sq = gd_block_sum<4>(sq, red[0]);
    sc = gd_block_sum<4>(sc, red[1]);
    const float iq = 1.0f / sqrtf(sq / (float)m.q_rank + m.eps), ic = 1.0f / sqrtf(sc / (float)m.kv_rank + m.eps);
    for (uint32_t c = threadIdx.x; c < m.q_rank; c += 256u) cq[(size_t)row * m.q_rank + c] = (T)((float)pq[c] * iq * q_norm[c]);
    if (!live) return;
    T *dst = cache + ((size_t)slot * m.tmax + (uint32_t)pos) * m.pitch;
    for (uint32_t c = threadIdx.x; c < m.kv_rank; c += 256u) dst[c] = (T)((float)pc[c] * ic * kv_norm[c]);
    const uint32_t half = m.rot_dim / 2u;
    for (uint32_t i = threadIdx.x; i < half; i += 256u) {
        const float u = (float)pr[i], v = (float)pr[half + i];
        float s1, c1;
        sincosf((float)pos * freq[i], &s1, &c1);
        angles[(size_t)row * m.rot_dim + i] = c1;
        angles[(size_t)row * m.rot_dim + half + i] = s1;
        dst[m.kv_rank + i] = (T)(u * c1 - v * s1);
        dst[m.kv_rank + half + i] = (T)(v * c1 + u * s1);
    }
    for (uint32_t c = m.kv_rank + m.rot_dim + threadIdx.x; c < m.pitch; c += 256u) dst[c] = (T)0.f;
}

/* prepare for BF16 rows of q_rank + kv_rank <= 4096 in 16-byte pieces: a wavefront per row, the row in registers */
__global__ void __launch_bounds__(256)
gd_latent_prepare_vec_kernel(const gd_bf16 *__restrict__ proj, uint32_t ld, const float *__restrict__ q_norm,
                             const float *__restrict__ kv_norm, const float *__restrict__ freq, float *__restrict__ angles,
                             gd_bf16 *__restrict__ cq, gd_bf16 *__restrict__ cache, gd_hip_latent_params m, gd_hip_seqs q)
{
    constexpr int KEEP = 8;
    const uint32_t row = blockIdx.x * 4u + (threadIdx.x >> 6), lane = threadIdx.x & 63u;
    if (row >= q.rows) return;
    const gd_bf16 *pr = proj + (size_t)row * ld;
    const uint32_t qc = m.q_rank / 8u, all = qc + m.kv_rank / 8u, half = m.rot_dim / 2u;
    int32_t s, pos, slot;
    const bool live = gd_seq_of_row(q, row, &s, &pos, &slot) && (uint32_t)pos < m.tmax;
    gd_bf16x8 v[KEEP];
    float sq = 0.f, sc = 0.f;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const uint32_t c = lane + 64u * i;
        if (c < all) v[i] = *reinterpret_cast<const gd_bf16x8 *>(pr + c * 8u);
    }
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const uint32_t c = lane + 64u * i;
        if (c >= all) continue;
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf((float)v[i][e], (float)v[i][e], ss);
        if (c < qc) sq += ss;
        else sc += ss;
    }
    sq = gd_wave_sum(sq);
    sc = gd_wave_sum(sc);
    const float iq = 1.0f / sqrtf(sq / (float)m.q_rank + m.eps), ic = 1.0f / sqrtf(sc / (float)m.kv_rank + m.eps);
    gd_bf16 *dst = cache + ((size_t)(live ? slot : 0) * m.tmax + (uint32_t)(live ? pos : 0)) * m.pitch;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const uint32_t c = lane + 64u * i;
        if (c >= all) continue;
        const bool is_q = c < qc;
        const float inv = is_q ? iq : ic, *w = is_q ? q_norm + c * 8u : kv_norm + (c - qc) * 8u;
        gd_bf16x8 o;
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = (gd_bf16)((float)v[i][e] * inv * w[e]);
        if (is_q) *reinterpret_cast<gd_bf16x8 *>(cq + (size_t)row * m.q_rank + c * 8u) = o;
        else if (live) *reinterpret_cast<gd_bf16x8 *>(dst + (c - qc) * 8u) = o;
    }
    if (!live) return;
    const gd_bf16 *rot = pr + m.q_rank + m.kv_rank;
    for (uint32_t i = lane; i < half; i += 64u) {
        const float a = (float)rot[i], b = (float)rot[half + i];
        float s1, c1;
        sincosf((float)pos * freq[i], &s1, &c1);
        angles[(size_t)row * m.rot_dim + i] = c1;
        angles[(size_t)row * m.rot_dim + half + i] = s1;
        dst[m.kv_rank + i] = (gd_bf16)(a * c1 - b * s1);
        dst[m.kv_rank + half + i] = (gd_bf16)(b * c1 + a * s1);
    }
    for (uint32_t c = m.kv_rank + m.rot_dim + lane; c < m.pitch; c += 64u) dst[c] = (gd_bf16)0.f;
}

/* grid (rows, heads); w_ukt [heads, kv_rank, dim]; ql [rows, heads, pitch] */
template <typename T>
__global__ void __launch_bounds__(256)
gd_latent_query_kernel(const T *__restrict__ qv, const T *__restrict__ w_ukt, const float *__restrict__ angles,
                       T *__restrict__ ql, gd_hip_latent_params m)
{
    extern __shared__ float sq[]; /* dim */
    const uint32_t row = blockIdx.x, h = blockIdx.y, half = m.rot_dim / 2u;
    const T *src = qv + ((size_t)row * m.heads + h) * (m.dim + m.rot_dim);
    for (uint32_t d = threadIdx.x; d < m.dim; d += 256u) sq[d] = (float)src[d];
    __syncthreads();
    T *dst = ql + ((size_t)row * m.heads + h) * m.pitch;
    for (uint32_t c = threadIdx.x; c < m.kv_rank; c += 256u) {
        const T *w = w_ukt + ((size_t)h * m.kv_rank + c) * m.dim;
        float a = 0.f;
        for (uint32_t d = 0; d < m.dim; ++d) a = fmaf(sq[d], (float)w[d], a);
        dst[c] = (T)a;
    }
    for (uint32_t i = threadIdx.x; i < half; i += 256u) {
        const float u = (float)src[m.dim + i], v = (float)src[m.dim + half + i];
        const float c1 = angles[(size_t)row * m.rot_dim + i], s1 = angles[(size_t)row * m.rot_dim + half + i];
        dst[m.kv_rank + i] = (T)(u * c1 - v * s1);
        dst[m.kv_rank + half + i] = (T)(v * c1 + u * s1);
    }
    for (uint32_t c = m.kv_rank + m.rot_dim + threadIdx.x; c < m.pitch; c += 256u) dst[c] = (T)0.f;
}

/* grid (rows, heads); o_lat F32 [rows, heads, kv_rank] */
template <typename T>
__global__ void __launch_bounds__(256)
gd_latent_attend_kernel(const T *__restrict__ ql, const T *__restrict__ cache, float *__restrict__ o_lat,
                        gd_hip_latent_params m, gd_hip_seqs q)
{
    extern __shared__ float smem[]; /* query [pitch], sums [kv_rank] */
    __shared__ float sp[256], red[4];
    float *sq = smem, *so = smem + m.pitch;
    const uint32_t row = blockIdx.x, h = blockIdx.y;
    int32_t s, pos, slot;
    if (!gd_seq_of_row(q, row, &s, &pos, &slot)) return;
    const uint32_t keys = min((uint32_t)pos + 1u, m.tmax), used = m.kv_rank + m.rot_dim;
    const T *src = ql + ((size_t)row * m.heads + h) * m.pitch, *rows = cache + (size_t)slot * m.tmax * m.pitch;
    for (uint32_t c = threadIdx.x; c < used; c += 256u) sq[c] = (float)src[c];
    for (uint32_t c = threadIdx.x; c < m.kv_rank; c += 256u) so[c] = 0.f;
    float mx = -INFINITY, total = 0.f;
    for (uint32_t k0 = 0; k0 < keys; k0 += 256u) {
        __syncthreads();
        const uint32_t k = k0 + threadIdx.x;
        float score = -INFINITY;
        if (k < keys) {
            const T *kr = rows + (size_t)k * m.pitch;
            float a = 0.f;
            for (uint32_t c = 0; c < used; ++c) a = fmaf(sq[c], (float)kr[c], a);
            score = a * m.scale;
        }
        /* maximum of the block's scores */
        float t = gd_wave_max(score);
        if ((threadIdx.x & 63u) == 0u) red[threadIdx.x >> 6] = t;
        __syncthreads();
        t = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float nmx = fmaxf(mx, t), keep = expf(mx - nmx);
        const float p = k < keys ? expf(score - nmx) : 0.f;
        sp[threadIdx.x] = p;
        __syncthreads();
        total = total * keep + gd_block_sum<4>(p, red);
        mx = nmx;
        const uint32_t nk = min(keys - k0, 256u);
        for (uint32_t c = threadIdx.x; c < m.kv_rank; c += 256u) {
            float a = so[c] * keep;
            const T *kr = rows + (size_t)k0 * m.pitch + c;
            for (uint32_t j = 0; j < nk; ++j) a = fmaf(sp[j], (float)kr[(size_t)j * m.pitch], a);
            so[c] = a;
        }
    }
    for (uint32_t c = threadIdx.x; c < m.kv_rank; c += 256u)
        o_lat[((size_t)row * m.heads + h) * m.kv_rank + c] = so[c] / total;
}

/* grid (rows, heads); out [rows, heads * vdim] */
template <typename T>
__global__ void __launch_bounds__(256)
gd_latent_value_kernel(const float *__restrict__ o_lat, const T *__restrict__ w_uv, const T *__restrict__ gate,
                       uint32_t ldg, T *__restrict__ out, gd_hip_latent_params m)
{
    extern __shared__ float so[]; /* kv_rank */
    const uint32_t row = blockIdx.x, h = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63u;
    for (uint32_t c = threadIdx.x; c < m.kv_rank; c += 256u) so[c] = o_lat[((size_t)row * m.heads + h) * m.kv_rank + c];
    __syncthreads();
    for (uint32_t v = wave; v < m.vdim; v += 4u) {
        const T *w = w_uv + ((size_t)h * m.vdim + v) * m.kv_rank;
        float a = 0.f;
        for (uint32_t c = lane; c < m.kv_rank; c += 64u) a = fmaf(so[c], (float)w[c], a);
        a = gd_wave_sum(a);
        if (lane == 0u) {
            const float g = (float)gate[(size_t)row * ldg + h * m.vdim + v];
            out[(size_t)row * m.heads * m.vdim + h * m.vdim + v] = (T)(a * gd_sigmoid_f32(g));
        }
    }
}

extern "C" int gd_hip_launch_latent_prepare(hipStream_t stream, const void *proj, uint32_t ld, const float *q_norm,
                                            const float *kv_norm, const float *freq, float *angles, void *cq, void *cache,
                                            const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32, int aligned16)
{
    if (!is_f32 && aligned16 && (m->q_rank % 8u) == 0u && (m->kv_rank % 8u) == 0u && m->q_rank + m->kv_rank <= 4096u) {
        gd_latent_prepare_vec_kernel<<<(q->rows + 3u) / 4u, 256, 0, stream>>>(
            (const gd_bf16 *)proj, ld, q_norm, kv_norm, freq, angles, (gd_bf16 *)cq, (gd_bf16 *)cache, *m, *q);
        return (int)hipGetLastError();
    }
#define GD_GO(T) gd_latent_prepare_kernel<T><<<q->rows, 256, 0, stream>>>((const T *)proj, ld, q_norm, kv_norm, freq, angles, (T *)cq, (T *)cache, *m, *q)
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_latent_query(hipStream_t stream, const void *qv, const void *w_ukt, const float *angles,
                                          void *ql, const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32)
{
    const dim3 grid(q->rows, m->heads);
#define GD_GO(T) gd_latent_query_kernel<T><<<grid, 256, m->dim * sizeof(float), stream>>>((const T *)qv, (const T *)w_ukt, angles, (T *)ql, *m)
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_latent_attend(hipStream_t stream, const void *ql, const void *cache, float *o_lat,
                                           const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32)
{
    const dim3 grid(q->rows, m->heads);
    const size_t lds = (m->pitch + m->kv_rank) * sizeof(float);
    if (q->rows == 0u) return (int)hipSuccess;
    if (lds > 48u * 1024u) return (int)hipErrorInvalidValue;
#define GD_GO(T) gd_latent_attend_kernel<T><<<grid, 256, lds, stream>>>((const T *)ql, (const T *)cache, o_lat, *m, *q)
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_latent_value(hipStream_t stream, const float *o_lat, const void *w_uv, const void *gate,
                                          uint32_t ldg, void *out, uint32_t rows, const gd_hip_latent_params *m, int is_f32)
{
    const dim3 grid(rows, m->heads);
    if (rows == 0u) return (int)hipSuccess;
#define GD_GO(T) gd_latent_value_kernel<T><<<grid, 256, m->kv_rank * sizeof(float), stream>>>(o_lat, (const T *)w_uv, (const T *)gate, ldg, (T *)out, *m)
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}
