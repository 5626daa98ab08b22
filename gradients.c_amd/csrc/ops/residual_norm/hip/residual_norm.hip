/*
 * F32 residual stream with norms on the sublayers' outputs or in front of the sublayers (gfx950).  HBM-bound row kernels, one workgroup per row:
 *   embed      x = table[id] * scale, and x once more in the type the projections read
 *   norm_add   x += mult * (u * w / rms(u)) for a sublayer's output u, and the copy
 *   add_norm   x += a sublayer's output u and the outputs of the experts a row went through, then h = x * w / rms(x),
 *              which the next sublayer reads, once more for every expert the row goes to
 *   norm_rows  out = x * w / rms(x) of picked rows (the model's last norm in front of the LM head)
 * Sums, norms and the residual itself are F32 whatever the element type.  Rows of up to 8 * 256 * 4 elements on
 * aligned pointers stay in registers between the sum of squares and the update; others are read twice.
 */
#include "../../_shared/hip_device.h"

#define GD_RN_THREADS 256
#define GD_RN_CHUNKS 4 /* 8-element chunks per thread on the register path */

template <typename T>
struct gd_rn_vec;
/* gd_backend_routed_rows; top 0: none */
template <typename T>
struct gd_hip_routed_choice {
    T *at;
    const int32_t *place;
    uint32_t rows, top;
    float weight;
};
template <>
struct gd_rn_vec<gd_bf16> {
    static __device__ __forceinline__ void load(const gd_bf16 *p, float (&v)[8])
    {
        const gd_bf16x8 t = *reinterpret_cast<const gd_bf16x8 *>(p);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = (float)t[e];
    }
    static __device__ __forceinline__ void store(gd_bf16 *p, const float (&v)[8])
    {
        gd_bf16x8 t;
#pragma unroll
        for (int e = 0; e < 8; ++e) t[e] = (gd_bf16)v[e];
        *reinterpret_cast<gd_bf16x8 *>(p) = t;
    }
};
template <>
struct gd_rn_vec<float> {
    static __device__ __forceinline__ void load(const float *p, float (&v)[8])
    {
        const gd_float4 a = reinterpret_cast<const gd_float4 *>(p)[0], b = reinterpret_cast<const gd_float4 *>(p)[1];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            v[e] = a[e];
            v[4 + e] = b[e];
        }
    }
    static __device__ __forceinline__ void store(float *p, const float (&v)[8])
    {
        gd_float4 a, b;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            a[e] = v[e];
            b[e] = v[4 + e];
        }
        reinterpret_cast<gd_float4 *>(p)[0] = a;
        reinterpret_cast<gd_float4 *>(p)[1] = b;
    }
};

template <typename T>
__global__ void __launch_bounds__(GD_RN_THREADS)
gd_residual_embed_kernel(const T *__restrict__ table, const int32_t *__restrict__ ids, float *__restrict__ x,
                         T *__restrict__ copy, uint32_t vocab, uint32_t cols, float scale)
{
    const int32_t id = ids[blockIdx.x];
    const bool ok = id >= 0 && (uint32_t)id < vocab;
    const T *row = table + (size_t)(ok ? id : 0) * cols;
    if (ok && (cols % 8u) == 0u && ((reinterpret_cast<uintptr_t>(table) | reinterpret_cast<uintptr_t>(copy)) & 15u) == 0u) {
        for (uint32_t c = threadIdx.x * 8u; c < cols; c += GD_RN_THREADS * 8u) {
            float v[8];
            gd_rn_vec<T>::load(row + c, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] *= scale;
            gd_rn_vec<float>::store(x + (size_t)blockIdx.x * cols + c, v);
            if (copy != nullptr) gd_rn_vec<T>::store(copy + (size_t)blockIdx.x * cols + c, v);
        }
        return;
    }
    for (uint32_t c = threadIdx.x; c < cols; c += GD_RN_THREADS) {
        const float v = ok ? (float)row[c] * scale : __builtin_nanf("");
        x[(size_t)blockIdx.x * cols + c] = v;
        if (copy != nullptr) copy[(size_t)blockIdx.x * cols + c] = (T)v;
    }
}

template <typename T, bool VEC>
__global__ void __launch_bounds__(GD_RN_THREADS)
gd_residual_norm_add_kernel(const T *__restrict__ u, const float *__restrict__ w, float *__restrict__ x,
                            T *__restrict__ copy, uint32_t cols, float eps, float mult)
{
    __shared__ float red[GD_RN_THREADS / 64];
    const size_t base = (size_t)blockIdx.x * cols;
    float ss = 0.f;
    if (VEC) {
        float uv[GD_RN_CHUNKS][8], xv[GD_RN_CHUNKS][8], wv[GD_RN_CHUNKS][8]; /* all requested in front of the sum */
#pragma unroll
        for (int i = 0; i < GD_RN_CHUNKS; ++i) {
            const uint32_t c = (threadIdx.x + i * GD_RN_THREADS) * 8u;
            if (c >= cols) continue;
            gd_rn_vec<T>::load(u + base + c, uv[i]);
            gd_rn_vec<float>::load(x + base + c, xv[i]);
            gd_rn_vec<float>::load(w + c, wv[i]);
        }
#pragma unroll
        for (int i = 0; i < GD_RN_CHUNKS; ++i) {
            if ((threadIdx.x + i * GD_RN_THREADS) * 8u >= cols) continue;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss = fmaf(uv[i][e], uv[i][e], ss);
        }
        ss = gd_block_sum<GD_RN_THREADS / 64>(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
#pragma unroll
        for (int i = 0; i < GD_RN_CHUNKS; ++i) {
            const uint32_t c = (threadIdx.x + i * GD_RN_THREADS) * 8u;
            if (c >= cols) continue;
#pragma unroll
            for (int e = 0; e < 8; ++e) xv[i][e] += mult * (uv[i][e] * inv * wv[i][e]);
            gd_rn_vec<float>::store(x + base + c, xv[i]);
            if (copy != nullptr) gd_rn_vec<T>::store(copy + base + c, xv[i]);
        }
        return;
    }
    for (uint32_t c = threadIdx.x; c < cols; c += GD_RN_THREADS) {
        const float v = (float)u[base + c];
        ss = fmaf(v, v, ss);
    }
    ss = gd_block_sum<GD_RN_THREADS / 64>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
    for (uint32_t c = threadIdx.x; c < cols; c += GD_RN_THREADS) {
        const float v = x[base + c] + mult * ((float)u[base + c] * inv * w[c]);
        x[base + c] = v;
        if (copy != nullptr) copy[base + c] = (T)v;
    }
}

/* u, w and out may be null; choices of a row: rows place[row * top + k] of the packed rows, negative: none.  LANES
 * threads per row, 256 or 64 (a wavefront: no exchange through LDS, for many short rows).  VEC: rows of up to 8 * LANES * 4
 * elements in 16-byte pieces, in registers between the sum of squares and the stores. */
template <typename T, bool VEC, int LANES>
__global__ void __launch_bounds__(GD_RN_THREADS)
gd_residual_add_norm_kernel(const T *__restrict__ u, gd_hip_routed_choice<T> in, float *__restrict__ x,
                            const float *__restrict__ w, T *__restrict__ out, gd_hip_routed_choice<T> to, uint32_t cols,
                            float eps, uint32_t n_rows)
{
    __shared__ float red[GD_RN_THREADS / 64];
    const uint32_t row = blockIdx.x * (GD_RN_THREADS / LANES) + threadIdx.x / LANES, sub = threadIdx.x % LANES;
    if (LANES < GD_RN_THREADS && row >= n_rows) return;
    const size_t base = (size_t)row * cols;
    float ss = 0.f;
    if (VEC) {
        float uv[GD_RN_CHUNKS][8], xv[GD_RN_CHUNKS][8], wv[GD_RN_CHUNKS][8]; /* all requested in front of the sums */
#pragma unroll
        for (int i = 0; i < GD_RN_CHUNKS; ++i) {
            const uint32_t c = (sub + i * LANES) * 8u;
            if (c >= cols) continue;
            if (u != nullptr) gd_rn_vec<T>::load(u + base + c, uv[i]);
            gd_rn_vec<float>::load(x + base + c, xv[i]);
            if (w != nullptr) gd_rn_vec<float>::load(w + c, wv[i]);
        }
        if (u != nullptr) {
#pragma unroll
            for (int i = 0; i < GD_RN_CHUNKS; ++i) {
                if ((sub + i * LANES) * 8u >= cols) continue;
#pragma unroll
                for (int e = 0; e < 8; ++e) xv[i][e] += uv[i][e];
            }
        }
        for (uint32_t k = 0; k < in.top; ++k) {
            const int32_t at = in.place[row * in.top + k];
            if (at < 0 || (uint32_t)at >= in.rows) continue;
#pragma unroll
            for (int i = 0; i < GD_RN_CHUNKS; ++i) {
                const uint32_t c = (sub + i * LANES) * 8u;
                if (c < cols) gd_rn_vec<T>::load(in.at + (size_t)at * cols + c, uv[i]);
            }
#pragma unroll
            for (int i = 0; i < GD_RN_CHUNKS; ++i) {
                if ((sub + i * LANES) * 8u >= cols) continue;
#pragma unroll
                for (int e = 0; e < 8; ++e) xv[i][e] = fmaf(in.weight, uv[i][e], xv[i][e]);
            }
        }
        const bool changed = u != nullptr || in.top != 0u;
#pragma unroll
        for (int i = 0; i < GD_RN_CHUNKS; ++i) {
            const uint32_t c = (sub + i * LANES) * 8u;
            if (c >= cols) continue;
            if (changed) gd_rn_vec<float>::store(x + base + c, xv[i]);
#pragma unroll
            for (int e = 0; e < 8; ++e) ss = fmaf(xv[i][e], xv[i][e], ss);
        }
        if (w == nullptr) return;
        ss = LANES == 64 ? gd_wave_sum(ss) : gd_block_sum<GD_RN_THREADS / 64>(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
#pragma unroll
        for (int i = 0; i < GD_RN_CHUNKS; ++i) {
            const uint32_t c = (sub + i * LANES) * 8u;
            if (c >= cols) continue;
#pragma unroll
            for (int e = 0; e < 8; ++e) xv[i][e] = xv[i][e] * inv * wv[i][e];
            gd_rn_vec<T>::store(out + base + c, xv[i]);
        }
        for (uint32_t k = 0; k < to.top; ++k) {
            const int32_t at = to.place[row * to.top + k];
            if (at < 0 || (uint32_t)at >= to.rows) continue;
#pragma unroll
            for (int i = 0; i < GD_RN_CHUNKS; ++i) {
                const uint32_t c = (sub + i * LANES) * 8u;
                if (c < cols) gd_rn_vec<T>::store(to.at + (size_t)at * cols + c, xv[i]);
            }
        }
        return;
    }
    for (uint32_t c = threadIdx.x; c < cols; c += GD_RN_THREADS) {
        float v = x[base + c];
        if (u != nullptr) v += (float)u[base + c];
        for (uint32_t k = 0; k < in.top; ++k) {
            const int32_t at = in.place[row * in.top + k];
            if (at >= 0 && (uint32_t)at < in.rows) v = fmaf(in.weight, (float)in.at[(size_t)at * cols + c], v);
        }
        x[base + c] = v;
        ss = fmaf(v, v, ss);
    }
    if (w == nullptr) return;
    ss = gd_block_sum<GD_RN_THREADS / 64>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
    for (uint32_t c = threadIdx.x; c < cols; c += GD_RN_THREADS) { /* the columns this thread has just stored */
        const T h = (T)(x[base + c] * inv * w[c]);
        out[base + c] = h;
        for (uint32_t k = 0; k < to.top; ++k) {
            const int32_t at = to.place[row * to.top + k];
            if (at >= 0 && (uint32_t)at < to.rows) to.at[(size_t)at * cols + c] = h;
        }
    }
}

template <typename T>
__global__ void __launch_bounds__(GD_RN_THREADS)
gd_residual_norm_rows_kernel(const float *__restrict__ x, const int32_t *__restrict__ rows, uint32_t n_rows,
                             const float *__restrict__ w, T *__restrict__ out, uint32_t cols, float eps)
{
    __shared__ float red[GD_RN_THREADS / 64];
    const int32_t src = rows != nullptr ? rows[blockIdx.x] : (int32_t)blockIdx.x;
    if (src < 0 || (uint32_t)src >= n_rows) return;
    const float *xr = x + (size_t)src * cols;
    float ss = 0.f;
    for (uint32_t c = threadIdx.x; c < cols; c += GD_RN_THREADS) ss = fmaf(xr[c], xr[c], ss);
    ss = gd_block_sum<GD_RN_THREADS / 64>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
    for (uint32_t c = threadIdx.x; c < cols; c += GD_RN_THREADS)
        out[(size_t)blockIdx.x * cols + c] = (T)(xr[c] * inv * w[c]);
}

extern "C" int gd_hip_launch_residual_embed(hipStream_t stream, const void *table, const int32_t *ids, float *x,
                                            void *copy, uint32_t n, uint32_t vocab, uint32_t cols, float scale, int is_f32)
{
    if (n == 0u) return (int)hipSuccess;
    if (is_f32)
        gd_residual_embed_kernel<float><<<n, GD_RN_THREADS, 0, stream>>>((const float *)table, ids, x, (float *)copy, vocab, cols, scale);
    else
        gd_residual_embed_kernel<gd_bf16><<<n, GD_RN_THREADS, 0, stream>>>((const gd_bf16 *)table, ids, x, (gd_bf16 *)copy, vocab, cols, scale);
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_residual_norm_add(hipStream_t stream, const void *u, const float *w, float *x, void *copy,
                                               uint32_t rows, uint32_t cols, float eps, float mult, int is_f32,
                                               int aligned16)
{
    if (rows == 0u) return (int)hipSuccess;
    const bool vec = aligned16 && (cols % 8u) == 0u && cols <= 8u * GD_RN_THREADS * GD_RN_CHUNKS;
#define GD_GO(T, V) gd_residual_norm_add_kernel<T, V><<<rows, GD_RN_THREADS, 0, stream>>>((const T *)u, w, x, (T *)copy, cols, eps, mult)
    if (is_f32) { if (vec) GD_GO(float, true); else GD_GO(float, false); }
    else { if (vec) GD_GO(gd_bf16, true); else GD_GO(gd_bf16, false); }
#undef GD_GO
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_residual_add_norm(hipStream_t stream, const void *u, void *in, const int32_t *in_place,
                                               uint32_t in_rows, uint32_t in_top, float in_weight, float *x, const float *w,
                                               void *out, void *to, const int32_t *to_place, uint32_t to_rows,
                                               uint32_t to_top, uint32_t rows, uint32_t cols, float eps, int is_f32,
                                               int aligned16)
{
    if (rows == 0u) return (int)hipSuccess;
    const bool vec = aligned16 && (cols % 8u) == 0u && cols <= 8u * GD_RN_THREADS * GD_RN_CHUNKS;
    /* a wavefront per row where a workgroup would leave half of its threads idle and there are rows enough (1024 columns,
     * 40,796 rows: 155 -> 101 us; at 2048 columns a workgroup is as fast) */
    const bool wave = vec && cols <= 1024u && rows >= 1024u;
#define GD_GO(T, V, L)                                                                                                 \
    gd_residual_add_norm_kernel<T, V, L><<<(rows + GD_RN_THREADS / L - 1u) / (GD_RN_THREADS / L), GD_RN_THREADS, 0, stream>>>( \
        (const T *)u, gd_hip_routed_choice<T>{(T *)in, in_place, in_rows, in_top, in_weight}, x, w, (T *)out,          \
        gd_hip_routed_choice<T>{(T *)to, to_place, to_rows, to_top, 1.0f}, cols, eps, rows)
#define GD_GO_TYPE(T) do { if (wave) GD_GO(T, true, 64); else if (vec) GD_GO(T, true, 256); else GD_GO(T, false, 256); } while (0)
    if (is_f32) GD_GO_TYPE(float);
    else GD_GO_TYPE(gd_bf16);
#undef GD_GO_TYPE
#undef GD_GO
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_residual_norm_rows(hipStream_t stream, const float *x, const int32_t *rows, uint32_t n_rows,
                                                const float *w, void *out, uint32_t n_out, uint32_t cols, float eps,
                                                int is_f32)
{
    if (n_out == 0u) return (int)hipSuccess;
    if (is_f32)
        gd_residual_norm_rows_kernel<float><<<n_out, GD_RN_THREADS, 0, stream>>>(x, rows, n_rows, w, (float *)out, cols, eps);
    else
        gd_residual_norm_rows_kernel<gd_bf16><<<n_out, GD_RN_THREADS, 0, stream>>>(x, rows, n_rows, w, (gd_bf16 *)out, cols, eps);
    return (int)hipGetLastError();
}
