/*
 * Selective state-space recurrence token by token (gfx950):
 *   dt = softplus(dt_raw + dt_bias_h), S <- exp(-exp(a_log_h) dt) S + dt B x^T, y = S^T C + d_h x
 * with S [N, P] per head, in F32 from the first token to the last; B and C are shared by the heads of a group.
 *
 * One workgroup owns a [N, 32] column slice of one head of one sequence and keeps it in registers: thread (r, l) holds
 * rows r, r + 32, ... of columns 4l .. 4l+3, so a state row is read and written in whole 128-byte lines.  Tokens come
 * in batches of GD_SSM_BATCH through LDS; the column sums of S^T C go through wavefront shuffles and one LDS exchange
 * per batch.  This is the decode step (HBM-bound on reading and writing S once), the whole F32 path and the path of
 * short portions; long BF16 prompts take the matrix-core kernel of ssm_scan_chunk.hip.
 *
 * A sequence that starts at position 0 starts from a zero state, whatever its slot holds.
 */
#include "../../_shared/hip_device.h"
#include "hip_ssm_scan_types.h"

#define GD_SSM_BATCH 8
#define GD_SSM_COLS 32
#define GD_SSM_STATE_MAX 512

__device__ __forceinline__ float gd_softplus(float v) { return fmaxf(v, 0.0f) + log1pf(expf(-fabsf(v))); }

/* silu of the causal convolution of channel c at position pos, rounded to T as the separate operator stores it; keep:
 * this workgroup is the one that stores the channel's new input */
template <typename T>
__device__ __forceinline__ float gd_ssm_conv_at(const gd_hip_ssm_conv &cv, const T *__restrict__ u, T *__restrict__ rg,
                                                uint32_t c, int32_t pos, bool keep)
{
    const float *w = cv.taps + (size_t)c * cv.K;
    const T now = u[c];
    float acc = fmaf(w[cv.K - 1u], (float)now, cv.bias[c]);
    if (cv.K <= 4u) { /* the places of the ring in one batch of loads */
        float v[4], wv[4];
#pragma unroll
        for (uint32_t k = 1u; k < 4u; ++k) {
            const bool ok = k < cv.K && (int32_t)k <= pos;
            v[k] = ok ? (float)rg[(size_t)((uint32_t)(pos - (int32_t)k) % cv.K) * cv.C + c] : 0.f;
            wv[k] = ok ? w[cv.K - 1u - k] : 0.f;
        }
#pragma unroll
        for (uint32_t k = 1u; k < 4u; ++k) acc = fmaf(wv[k], v[k], acc);
    } else
    for (uint32_t k = 1u; k < cv.K && (int32_t)k <= pos; ++k)
        acc = fmaf(w[cv.K - 1u - k], (float)rg[(size_t)((uint32_t)(pos - (int32_t)k) % cv.K) * cv.C + c], acc);
    if (keep) rg[(size_t)((uint32_t)pos % cv.K) * cv.C + c] = now;
    return (float)(T)gd_silu_f32(acc);
}

/* CONV: xbc holds the inputs of the convolution (row pitch ld_xbc) and every sequence brings one token: the channels a
 * workgroup needs are convolved here.  B and C are convolved by every workgroup of their group; the places of the
 * ring that are read (positions in front of the token) and written (its own) differ, so they do not race. */
template <typename T, int NR, bool CONV>
__global__ void __launch_bounds__(256)
gd_ssm_scan_kernel(const T *__restrict__ xbc, const T *__restrict__ dt_raw, const float *__restrict__ dt_bias,
                   const float *__restrict__ a_log, const float *__restrict__ d_skip, float *__restrict__ states,
                   T *__restrict__ y, gd_hip_ssm_params m, gd_hip_ssm_conv cv, gd_hip_seqs q)
{
    __shared__ float sb[GD_SSM_BATCH][NR * 32], sc[GD_SSM_BATCH][NR * 32], sx[GD_SSM_BATCH][GD_SSM_COLS];
    __shared__ float part[GD_SSM_BATCH][4][GD_SSM_COLS], sdt[GD_SSM_BATCH], sdec[GD_SSM_BATCH];
    const uint32_t p0 = blockIdx.x * GD_SSM_COLS, h = blockIdx.y;
    const uint32_t l = threadIdx.x & 7u, r = threadIdx.x >> 3, wave = threadIdx.x >> 6;
    const uint32_t N = m.state, P = m.vdim, inner = m.heads * P, g = h / (m.heads / m.groups);
    int32_t first, n, start, slot;
    if (!gd_seq_span(q, blockIdx.z, &first, &n, &start, &slot)) return;
    float *st = states + ((size_t)slot * m.heads + h) * N * P + p0;
    const float rate = expf(a_log[h]), bias = dt_bias[h], skip = d_skip[h];
    const uint32_t cols = min(P - p0, (uint32_t)GD_SSM_COLS);
    const bool vec = (P & 3u) == 0u;
    gd_float4 S[NR];
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const uint32_t row = r + 32u * i;
        S[i] = (gd_float4){0.f, 0.f, 0.f, 0.f};
        if (start > 0 && row < N && 4u * l < cols) {
            if (vec) S[i] = *reinterpret_cast<const gd_float4 *>(st + (size_t)row * P + 4u * l);
            else
                for (uint32_t e = 0; e < 4u && 4u * l + e < cols; ++e) S[i][e] = st[(size_t)row * P + 4u * l + e];
        }
    }
    for (int32_t t0 = 0; t0 < n; t0 += GD_SSM_BATCH) {
        const uint32_t nb = min((uint32_t)(n - t0), (uint32_t)GD_SSM_BATCH);
        const T *rows = xbc + (size_t)(first + t0) * m.ld_xbc;
        if (CONV) {
            T *rg = (T *)cv.ring + (size_t)slot * cv.K * cv.C;
            const bool own = blockIdx.x == 0u && h % (m.heads / m.groups) == 0u; /* of B and C of the group */
            for (uint32_t i = threadIdx.x; i < 2u * NR * 32u + GD_SSM_COLS; i += 256u) {
                const uint32_t k = i % (NR * 32u), part = i / (NR * 32u);
                if (part < 2u) {
                    float *dst = part == 0u ? &sb[0][k] : &sc[0][k];
                    *dst = k < N ? gd_ssm_conv_at<T>(cv, rows, rg, inner + (part * m.groups + g) * N + k, start, own) : 0.f;
                } else {
                    const uint32_t c = i - 2u * NR * 32u;
                    sx[0][c] = c < cols ? gd_ssm_conv_at<T>(cv, rows, rg, h * P + p0 + c, start, true) : 0.f;
                }
            }
        } else {
        for (uint32_t i = threadIdx.x; i < nb * (NR * 32u); i += 256u) {
            const uint32_t t = i / (NR * 32u), k = i % (NR * 32u);
            const T *b = rows + (size_t)t * m.ld_xbc + inner + g * N;
            sb[t][k] = k < N ? (float)b[k] : 0.f;
            sc[t][k] = k < N ? (float)b[m.groups * N + k] : 0.f;
        }
        for (uint32_t i = threadIdx.x; i < nb * GD_SSM_COLS; i += 256u) {
            const uint32_t t = i / GD_SSM_COLS, c = i % GD_SSM_COLS;
            sx[t][c] = c < cols ? (float)rows[(size_t)t * m.ld_xbc + h * P + p0 + c] : 0.f;
        }
        }
        if (threadIdx.x < nb) {
            const float dt = gd_softplus((float)dt_raw[(size_t)(first + t0 + (int32_t)threadIdx.x) * m.ld_dt + h] + bias);
            sdt[threadIdx.x] = dt;
            sdec[threadIdx.x] = expf(-rate * dt);
        }
        __syncthreads();
        for (uint32_t t = 0; t < nb; ++t) {
            const float dec = sdec[t], dt = sdt[t];
            const gd_float4 x4 = *reinterpret_cast<const gd_float4 *>(&sx[t][4u * l]);
            gd_float4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < NR; ++i) {
                const float b = dt * sb[t][r + 32u * i], c = sc[t][r + 32u * i];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    S[i][e] = fmaf(dec, S[i][e], b * x4[e]);
                    acc[e] = fmaf(S[i][e], c, acc[e]);
                }
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                acc[e] += __shfl_xor(acc[e], 8, 64);
                acc[e] += __shfl_xor(acc[e], 16, 64);
                acc[e] += __shfl_xor(acc[e], 32, 64);
            }
            if ((threadIdx.x & 63u) < 8u) *reinterpret_cast<gd_float4 *>(&part[t][wave][4u * l]) = acc;
        }
        __syncthreads();
        for (uint32_t i = threadIdx.x; i < nb * GD_SSM_COLS; i += 256u) {
            const uint32_t t = i / GD_SSM_COLS, c = i % GD_SSM_COLS;
            if (c < cols)
                y[(size_t)(first + t0 + (int32_t)t) * inner + h * P + p0 + c] =
                    (T)(part[t][0][c] + part[t][1][c] + part[t][2][c] + part[t][3][c] + skip * sx[t][c]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < NR; ++i) {
        const uint32_t row = r + 32u * i;
        if (row < N && 4u * l < cols) {
            if (vec) *reinterpret_cast<gd_float4 *>(st + (size_t)row * P + 4u * l) = S[i];
            else
                for (uint32_t e = 0; e < 4u && 4u * l + e < cols; ++e) st[(size_t)row * P + 4u * l + e] = S[i][e];
        }
    }
}

extern "C" int gd_hip_launch_ssm_scan(hipStream_t stream, const void *xbc, const void *dt_raw, const float *dt_bias,
                                      const float *a_log, const float *d_skip, float *states, void *y,
                                      const gd_hip_ssm_params *m, const gd_hip_ssm_conv *cv, const gd_hip_seqs *q,
                                      int is_f32)
{
    const dim3 grid((m->vdim + GD_SSM_COLS - 1u) / GD_SSM_COLS, m->heads, q->seqs);
    if (q->rows == 0u || q->seqs == 0u) return (int)hipSuccess;
    if (m->state > GD_SSM_STATE_MAX) return (int)hipErrorInvalidValue;
    const gd_hip_ssm_conv none = {nullptr, nullptr, nullptr, 0u, 0u};
#define GD_GO(T, NR, CONV) gd_ssm_scan_kernel<T, NR, CONV><<<grid, 256, 0, stream>>>((const T *)xbc, (const T *)dt_raw, dt_bias, a_log, d_skip, states, (T *)y, *m, CONV ? *cv : none, *q)
#define GD_PICK(T, CONV)                              \
    do {                                              \
        if (m->state <= 32u) GD_GO(T, 1, CONV);       \
        else if (m->state <= 64u) GD_GO(T, 2, CONV);  \
        else if (m->state <= 128u) GD_GO(T, 4, CONV); \
        else if (m->state <= 256u) GD_GO(T, 8, CONV); \
        else GD_GO(T, 16, CONV);                      \
    } while (0)
    if (cv != nullptr) {
        if (is_f32) GD_PICK(float, true); else GD_PICK(gd_bf16, true);
    } else {
        if (is_f32) GD_PICK(float, false); else GD_PICK(gd_bf16, false);
    }
#undef GD_PICK
#undef GD_GO
    return (int)hipGetLastError();
}

/* out = weight * v / rms(v over its part) with v = y * silu(z), the row cut into equal parts */
template <typename T>
__global__ void __launch_bounds__(256)
gd_gated_group_norm_kernel(const T *__restrict__ y, const T *__restrict__ z, uint32_t ldz, const float *__restrict__ w,
                           T *__restrict__ out, uint32_t part, uint32_t inner, float eps)
{
    __shared__ float red[4];
    const uint32_t c0 = blockIdx.y * part;
    const T *yr = y + (size_t)blockIdx.x * inner + c0, *zr = z + (size_t)blockIdx.x * ldz + c0;
    constexpr int KEEP = 8;
    float keep[KEEP], ss = 0.f;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const uint32_t c = threadIdx.x + 256u * i;
        keep[i] = c < part ? (float)yr[c] * gd_silu_f32((float)zr[c]) : 0.f;
        ss = fmaf(keep[i], keep[i], ss);
    }
    for (uint32_t c = threadIdx.x + 256u * KEEP; c < part; c += 256u) {
        const float v = (float)yr[c] * gd_silu_f32((float)zr[c]);
        ss = fmaf(v, v, ss);
    }
    ss = gd_block_sum<4>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)part + eps);
    T *o = out + (size_t)blockIdx.x * inner + c0;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const uint32_t c = threadIdx.x + 256u * i;
        if (c < part) o[c] = (T)(keep[i] * inv * w[c0 + c]);
    }
    for (uint32_t c = threadIdx.x + 256u * KEEP; c < part; c += 256u)
        o[c] = (T)((float)yr[c] * gd_silu_f32((float)zr[c]) * inv * w[c0 + c]);
}

/* BF16 with parts of a multiple of 8 up to 8192 and 16-byte aligned rows: the part stays in registers */
__global__ void __launch_bounds__(256)
gd_gated_group_norm_vec_kernel(const gd_bf16 *__restrict__ y, const gd_bf16 *__restrict__ z, uint32_t ldz,
                               const float *__restrict__ w, gd_bf16 *__restrict__ out, uint32_t part, uint32_t inner,
                               float eps)
{
    __shared__ float red[4];
    const uint32_t c0 = blockIdx.y * part;
    const gd_bf16 *yr = y + (size_t)blockIdx.x * inner + c0, *zr = z + (size_t)blockIdx.x * ldz + c0;
    constexpr int KEEP = 4;
    gd_bf16x8 yv[KEEP], zv[KEEP];
    gd_float4 wv[KEEP][2]; /* requested with the rest: behind the sum they would be one more round trip */
    float v[KEEP][8], ss = 0.f;
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const uint32_t c = (threadIdx.x + 256u * i) * 8u;
        if (c >= part) continue;
        yv[i] = *reinterpret_cast<const gd_bf16x8 *>(yr + c);
        zv[i] = *reinterpret_cast<const gd_bf16x8 *>(zr + c);
        wv[i][0] = *reinterpret_cast<const gd_float4 *>(w + c0 + c);
        wv[i][1] = *reinterpret_cast<const gd_float4 *>(w + c0 + c + 4u);
    }
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        if ((threadIdx.x + 256u * i) * 8u >= part) continue;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            v[i][e] = (float)yv[i][e] * (float)zv[i][e] * gd_sigmoid_fast((float)zv[i][e]);
            ss = fmaf(v[i][e], v[i][e], ss);
        }
    }
    ss = gd_block_sum<4>(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)part + eps);
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const uint32_t c = (threadIdx.x + 256u * i) * 8u;
        if (c >= part) continue;
        gd_bf16x8 o;
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = (gd_bf16)(v[i][e] * inv * wv[i][e >> 2][e & 3]);
        *reinterpret_cast<gd_bf16x8 *>(out + (size_t)blockIdx.x * inner + c0 + c) = o;
    }
}

extern "C" int gd_hip_launch_gated_group_norm(hipStream_t stream, const void *y, const void *z, uint32_t ldz,
                                              const float *w, void *out, uint32_t rows, uint32_t inner, uint32_t groups,
                                              float eps, int is_f32, int aligned16)
{
    const dim3 grid(rows, groups);
    if (rows == 0u) return (int)hipSuccess;
    if (!is_f32 && aligned16 && (inner / groups) % 8u == 0u && inner / groups <= 8192u) {
        gd_gated_group_norm_vec_kernel<<<grid, 256, 0, stream>>>((const gd_bf16 *)y, (const gd_bf16 *)z, ldz, w, (gd_bf16 *)out, inner / groups, inner, eps);
        return (int)hipGetLastError();
    }
    if (is_f32)
        gd_gated_group_norm_kernel<float><<<grid, 256, 0, stream>>>((const float *)y, (const float *)z, ldz, w, (float *)out, inner / groups, inner, eps);
    else
        gd_gated_group_norm_kernel<gd_bf16><<<grid, 256, 0, stream>>>((const gd_bf16 *)y, (const gd_bf16 *)z, ldz, w, (gd_bf16 *)out, inner / groups, inner, eps);
    return (int)hipGetLastError();
}
