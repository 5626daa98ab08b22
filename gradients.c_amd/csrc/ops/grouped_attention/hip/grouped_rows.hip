/*
 * Attention with grouped heads, row kernels (gfx950), any sizes, BF16 and F32:
 *   rotate  queries and keys of the new rows turned to their positions, in place
 *   attend  per new row and query head: softmax over the keys the row sees, the weighted values, the output gate
 *   store   rotated keys and values of the new rows to their places in the caches
 * A row at position p of a sequence whose first new position is s sees the positions from its chunk's first on: those in
 * front of s lie in the caches, the others among the new rows.  With chunks the place of a position is counted from the
 * start of its chunk, so a later chunk overwrites an earlier one: that is why new rows are stored behind the attention,
 * and only those of a sequence's last chunk.
 * They are the F32 path and the path of sizes outside the matrix-core kernels (grouped_decode.hip, grouped_prefill.hip).
 */
#include "../../_shared/hip_device.h"
#include "hip_grouped_attention_types.h"

/* grid rows; a thread per rotation pair of the row's query and key heads */
template <typename T>
__global__ void __launch_bounds__(256)
gd_grouped_rotate_kernel(T *__restrict__ proj, const float *__restrict__ freq, gd_hip_grouped_params m, gd_hip_seqs q)
{
    int32_t seq, pos, slot;
    if (!gd_seq_of_row(q, blockIdx.x, &seq, &pos, &slot)) return;
    T *row = proj + (size_t)blockIdx.x * m.ld;
    const uint32_t pairs = (m.heads + m.kv_heads) * m.half;
    for (uint32_t i = threadIdx.x; i < pairs; i += 256u) {
        const uint32_t h = i / m.half, p = i % m.half; /* the key heads follow the query heads */
        T *at = row + (size_t)h * m.dim + 2u * p;
        float s, c;
        gd_grouped_angle(m, pos, freq[p], &s, &c);
        const float u = (float)at[0], v = (float)at[1];
        at[0] = (T)(u * c - v * s);
        at[1] = (T)(v * c + u * s);
    }
}

/* grid (rows, heads) */
template <typename T>
__global__ void __launch_bounds__(256)
gd_grouped_attend_kernel(const T *__restrict__ proj, const T *__restrict__ k_cache, const T *__restrict__ v_cache,
                         T *__restrict__ out, gd_hip_grouped_params m, gd_hip_seqs q)
{
    extern __shared__ float smem[]; /* query [dim], sums [vdim] */
    __shared__ float sp[256], red[4];
    float *sq = smem, *so = smem + m.dim;
    const uint32_t row = blockIdx.x, h = blockIdx.y, g = h / m.per;
    int32_t seq, pos, slot;
    if (!gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const int32_t start = q.start[seq], first = gd_grouped_first(m, pos), base = gd_grouped_first(m, start);
    const T *src = proj + (size_t)row * m.ld + (size_t)h * m.dim;
    /* position j >= start: packed row row - (pos - j); in front of it: the caches, where first == base */
    const T *kn = proj + m.k_col + (size_t)g * m.dim, *vn = proj + m.v_col + (size_t)g * m.vdim;
    const size_t slab = ((size_t)slot * m.kv_heads + g) * m.places;
    const T *kc = k_cache + slab * m.dim, *vc = v_cache + slab * m.vdim;
    auto key = [&](int32_t j) {
        return j >= start ? kn + (size_t)(row - (uint32_t)(pos - j)) * m.ld : kc + (size_t)min((uint32_t)(j - base), m.places - 1u) * m.dim;
    };
    auto value = [&](int32_t j) {
        return j >= start ? vn + (size_t)(row - (uint32_t)(pos - j)) * m.ld : vc + (size_t)min((uint32_t)(j - base), m.places - 1u) * m.vdim;
    };
    for (uint32_t c = threadIdx.x; c < m.dim; c += 256u) sq[c] = (float)src[c];
    for (uint32_t c = threadIdx.x; c < m.vdim; c += 256u) so[c] = 0.f;
    float mx = -INFINITY, total = 0.f;
    for (int32_t j0 = first; j0 <= pos; j0 += 256) {
        __syncthreads();
        const int32_t j = j0 + (int32_t)threadIdx.x;
        float score = -INFINITY;
        if (j <= pos) {
            const T *kr = key(j);
            float a = 0.f;
            for (uint32_t c = 0; c < m.dim; ++c) a = fmaf(sq[c], (float)kr[c], a);
            score = a * m.scale;
        }
        float t = gd_wave_max(score);
        if ((threadIdx.x & 63u) == 0u) red[threadIdx.x >> 6] = t;
        __syncthreads();
        t = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float nmx = fmaxf(mx, t), keep = expf(mx - nmx);
        const float p = j <= pos ? expf(score - nmx) : 0.f;
        sp[threadIdx.x] = p;
        __syncthreads();
        total = total * keep + gd_block_sum<4>(p, red);
        mx = nmx;
        const int32_t nk = min(pos + 1 - j0, 256);
        for (uint32_t c = threadIdx.x; c < m.vdim; c += 256u) {
            float a = so[c] * keep;
            for (int32_t i = 0; i < nk; ++i) a = fmaf(sp[i], (float)value(j0 + i)[c], a);
            so[c] = a;
        }
    }
    const float gate = (float)proj[(size_t)row * m.ld + m.g_col + h];
    const float mult = (1.0f / (1.0f + expf(-gate))) / total;
    for (uint32_t c = threadIdx.x; c < m.vdim; c += 256u)
        out[((size_t)row * m.heads + h) * m.vdim + c] = (T)(so[c] * mult);
}

/* grid rows */
template <typename T>
__global__ void __launch_bounds__(256)
gd_grouped_store_kernel(const T *__restrict__ proj, T *__restrict__ k_cache, T *__restrict__ v_cache,
                        gd_hip_grouped_params m, gd_hip_seqs q)
{
    const uint32_t row = blockIdx.x;
    int32_t seq, pos, slot;
    if (!gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const int32_t last = q.start[seq] + (q.cu[seq + 1] - q.cu[seq]) - 1, first = gd_grouped_first(m, pos);
    if (gd_grouped_first(m, last) != first) return; /* of a chunk that is over */
    const uint32_t place = (uint32_t)(pos - first);
    if (place >= m.places) return;
    const T *src = proj + (size_t)row * m.ld;
    for (uint32_t c = threadIdx.x; c < m.kv_heads * m.dim; c += 256u)
        k_cache[(((size_t)slot * m.kv_heads + c / m.dim) * m.places + place) * m.dim + c % m.dim] = src[m.k_col + c];
    for (uint32_t c = threadIdx.x; c < m.kv_heads * m.vdim; c += 256u)
        v_cache[(((size_t)slot * m.kv_heads + c / m.vdim) * m.places + place) * m.vdim + c % m.vdim] = src[m.v_col + c];
}

extern "C" int gd_hip_launch_grouped_rotate(hipStream_t stream, void *proj, const float *freq,
                                            const gd_hip_grouped_params *m, const gd_hip_seqs *q, int is_f32)
{
    if (is_f32) gd_grouped_rotate_kernel<float><<<q->rows, 256, 0, stream>>>((float *)proj, freq, *m, *q);
    else gd_grouped_rotate_kernel<gd_bf16><<<q->rows, 256, 0, stream>>>((gd_bf16 *)proj, freq, *m, *q);
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_grouped_attend(hipStream_t stream, const void *proj, const void *k_cache, const void *v_cache,
                                            void *out, const gd_hip_grouped_params *m, const gd_hip_seqs *q, int is_f32)
{
    const dim3 grid(q->rows, m->heads);
    const size_t lds = (m->dim + m->vdim) * sizeof(float);
    if (lds > 48u * 1024u) return (int)hipErrorInvalidValue;
#define GD_GO(T) gd_grouped_attend_kernel<T><<<grid, 256, lds, stream>>>((const T *)proj, (const T *)k_cache, (const T *)v_cache, (T *)out, *m, *q)
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_grouped_store(hipStream_t stream, const void *proj, void *k_cache, void *v_cache,
                                           const gd_hip_grouped_params *m, const gd_hip_seqs *q, int is_f32)
{
#define GD_GO(T) gd_grouped_store_kernel<T><<<q->rows, 256, 0, stream>>>((const T *)proj, (T *)k_cache, (T *)v_cache, *m, *q)
    if (is_f32) GD_GO(float); else GD_GO(gd_bf16);
#undef GD_GO
    return (int)hipGetLastError();
}
