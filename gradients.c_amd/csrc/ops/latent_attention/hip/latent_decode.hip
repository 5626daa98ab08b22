/*
 * Latent attention of few new tokens per sequence on the matrix cores (gfx950, BF16): the absorbed form, in which all
 * heads of a token share one "key", the cache row, and one "value", its latent part.
 *
 *   absorb  q_lat[h] = W_uk[h]^T q[h] per 16 rows, head and 64 latent columns, and the rotated query part behind it
 *   attend  a workgroup of 4 wavefronts takes 16 heads of one token over a piece of its keys: a cache row is read from
 *           memory once for all of them.  HBM-bound on the cache rows.
 *   value   merges the pieces of 16 tokens and one head, multiplies by the value up-projection and the output gate
 *
 * attend.  Keys advance in tiles of 64 rows that go through registers into LDS (one stage; the loads of the next tile
 * are in flight while the current one is used; two workgroups per compute unit overlap their barriers).  Both products
 * are computed transposed, so that a head lives in one lane column:
 *     S^T = K Q^T    wavefront w: keys 16w .. 16w+15; A = key rows from LDS, B = the query rows, kept in registers
 *     O^T = V^T P^T  wavefront w: a quarter of the latent columns over all 64 keys; A by the transposing LDS read
 * Scores, softmax and sums are F32.  The weights enter the second product as two BF16 numbers, their rounding and the
 * rest, so that they keep 16 bits; a row's maximum is a reference point that moves only when a tile raises it by more
 * than 8 binary orders.
 *
 * MFMA operand layout (v_mfma_f32_16x16x32_bf16): lane l supplies row / column l % 16 and the 8 consecutive k starting
 * at 8 * (l / 16); the result lane holds column l % 16, rows 4 * (l / 16) .. + 3.
 */
#include "../../_shared/hip_device.h"
#include "hip_latent_attention_types.h"

#define GD_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0)
#define GD_LD_TILE 64u

/* grid (ceil(kv_rank / 64), heads, ceil(rows / 16)); dim % 8 == 0, rot_dim % 8 == 0 (16-byte fragments of q) */
__global__ void __launch_bounds__(256)
gd_latent_absorb_kernel(const gd_bf16 *__restrict__ qv, const gd_bf16 *__restrict__ w_ukt,
                        const float *__restrict__ angles, gd_bf16 *__restrict__ ql, gd_hip_latent_params m, uint32_t rows)
{
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, li = lane & 15u, lg = lane >> 4;
    const uint32_t h = blockIdx.y, r0 = blockIdx.z * 16u, hd = m.dim + m.rot_dim;
    const uint32_t c0 = blockIdx.x * 64u + wave * 16u;
    const gd_bf16 *qr = qv + ((size_t)min(r0 + li, rows - 1u) * m.heads + h) * hd;
    if (c0 < m.kv_rank) {
        const gd_bf16 *wr = w_ukt + ((size_t)h * m.kv_rank + min(c0 + li, m.kv_rank - 1u)) * m.dim;
        const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
        gd_float4 acc = {0.f, 0.f, 0.f, 0.f};
        for (uint32_t k = 0; k < m.dim; k += 32u) {
            const uint32_t kk = k + 8u * lg;
            gd_bf16x8 a = zero, b = zero;
            if (kk < m.dim) {
                a = *reinterpret_cast<const gd_bf16x8 *>(qr + kk);
                b = *reinterpret_cast<const gd_bf16x8 *>(wr + kk);
            }
            acc = GD_MFMA(a, b, acc);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t row = r0 + 4u * lg + (uint32_t)r;
            if (row < rows && c0 + li < m.kv_rank)
                ql[((size_t)row * m.heads + h) * m.pitch + c0 + li] = (gd_bf16)acc[r];
        }
    }
    if (blockIdx.x != 0u) return;
    const uint32_t half = m.rot_dim / 2u, tail = m.pitch - m.kv_rank;
    for (uint32_t i = threadIdx.x; i < 16u * tail; i += 256u) {
        const uint32_t row = r0 + i / tail, e = i % tail;
        if (row >= rows) break;
        float v = 0.f;
        if (e < m.rot_dim) {
            const gd_bf16 *src = qv + ((size_t)row * m.heads + h) * hd + m.dim;
            const uint32_t p = e < half ? e : e - half;
            const float c = angles[(size_t)row * m.rot_dim + p], s = angles[(size_t)row * m.rot_dim + half + p];
            const float u = (float)src[p], w = (float)src[half + p];
            v = e < half ? u * c - w * s : w * c + u * s;
        }
        ql[((size_t)row * m.heads + h) * m.pitch + m.kv_rank + e] = (gd_bf16)v;
    }
}

/* STEPS: 32-wide steps that cover a cache row (pitch <= 32 * STEPS).  grid (pieces, ceil(heads / 16), rows).
 * o_part F32 [rows, pieces, heads, kv_rank], ml F32 [rows, pieces, heads, 2] (reference point in the exp2 domain, sum) */
template <int STEPS>
__global__ void __launch_bounds__(256, STEPS <= 20 ? 2 : 1)
gd_latent_attend_mfma_kernel(const gd_bf16 *__restrict__ ql, const gd_bf16 *__restrict__ cache, float *__restrict__ o_part,
                             float *__restrict__ ml, gd_hip_latent_params m, gd_hip_seqs q)
{
    constexpr uint32_t STRIDE = STEPS * 64u + 16u;      /* bytes per key row in LDS: 16 rows of a chunk hit all banks */
    constexpr int CT = (2 * STEPS + 3) / 4;             /* 16-wide latent column tiles per wavefront */
    extern __shared__ __align__(16) unsigned char gd_ld_smem[]; /* [64] key rows */
    __shared__ __align__(16) gd_bf16 s_p[2][16][GD_LD_TILE + 8]; /* weights, high and low parts: [head][key] */
    __shared__ float s_max[4][16], s_sum[4][16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, li = lane & 15u, lg = lane >> 4;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const uint32_t row = blockIdx.z, h0 = blockIdx.y * 16u;
    int32_t seq, pos, slot;
    if (!gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const uint32_t keys = min((uint32_t)pos + 1u, m.tmax);
    const uint32_t k_begin = blockIdx.x * m.piece_keys;
    if (k_begin >= keys) return;
    const uint32_t k_end = min(keys, k_begin + m.piece_keys);
    const uint32_t chunks = m.pitch / 8u;

    /* query fragments of head h0 + li */
    gd_bf16x8 qf[STEPS];
    const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
    {
        const gd_bf16 *qr = ql + ((size_t)row * m.heads + min(h0 + li, m.heads - 1u)) * m.pitch;
#pragma unroll
        for (int s = 0; s < STEPS; ++s) {
            const uint32_t c = 4u * s + lg;
            qf[s] = c < chunks ? *reinterpret_cast<const gd_bf16x8 *>(qr + c * 8u) : zero;
        }
    }
    /* staging: thread t carries chunk t % 4 + 4 * s of key t / 4, s = 0 .. STEPS-1 */
    const uint32_t st_key = tid >> 2, st_c = tid & 3u;
    const gd_bf16 *rows = cache + (size_t)slot * m.tmax * m.pitch;
    gd_bf16x8 stage[STEPS];
    auto request = [&](uint32_t k0) __attribute__((always_inline)) {
        const bool live = k0 + st_key < k_end;
        const gd_bf16 *kr = rows + (size_t)min(k0 + st_key, k_end - 1u) * m.pitch;
#pragma unroll
        for (int s = 0; s < STEPS; ++s) {
            const uint32_t c = st_c + 4u * s;
            stage[s] = live && c < chunks ? *reinterpret_cast<const gd_bf16x8 *>(kr + c * 8u) : zero;
        }
    };
    gd_float4 o[CT];
#pragma unroll
    for (int t = 0; t < CT; ++t) o[t] = (gd_float4){0.f, 0.f, 0.f, 0.f};
    float mref = -INFINITY, sum = 0.f; /* of head h0 + li; sum: this wavefront's keys, its lane group's rows */
    const float scale2 = m.scale * 1.4426950408889634f;

    request(k_begin);
    for (uint32_t k0 = k_begin; k0 < k_end; k0 += GD_LD_TILE) {
        __syncthreads(); /* the tile before is used up */
        {
            unsigned char *dst = gd_ld_smem + st_key * STRIDE + st_c * 16u;
#pragma unroll
            for (int s = 0; s < STEPS; ++s) *reinterpret_cast<gd_bf16x8 *>(dst + s * 64u) = stage[s];
        }
        if (k0 + GD_LD_TILE < k_end) request(k0 + GD_LD_TILE);
        __syncthreads();
        /* scores of this wavefront's 16 keys */
        gd_float4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
        const unsigned char *kf = gd_ld_smem + (wave * 16u + li) * STRIDE + lg * 16u;
#pragma unroll
        for (int s = 0; s < STEPS; ++s) {
            const gd_bf16x8 a = *reinterpret_cast<const gd_bf16x8 *>(kf + s * 64u);
            if (s & 1) s1 = GD_MFMA(a, qf[s], s1);
            else s0 = GD_MFMA(a, qf[s], s0);
        }
        float sc[4], mx = -INFINITY;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t key = k0 + wave * 16u + 4u * lg + (uint32_t)r;
            sc[r] = key < k_end ? (s0[r] + s1[r]) * scale2 : -INFINITY;
            mx = fmaxf(mx, sc[r]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        if (lg == 0u) s_max[wave][li] = mx;
        __syncthreads();
        mx = fmaxf(fmaxf(s_max[0][li], s_max[1][li]), fmaxf(s_max[2][li], s_max[3][li]));
        /* every wavefront sees the same maxima and takes the same decision; the tile holds at least one live key, so
         * mx is finite (or NaN) */
        if (__builtin_amdgcn_ballot_w64(!(mx <= mref + 8.f)) != 0ull) {
            const float next = fmaxf(mref, mx), keep = __builtin_amdgcn_exp2f(mref - next);
            mref = next;
            sum *= keep;
#pragma unroll
            for (int t = 0; t < CT; ++t)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[t][r] *= keep;
        }
        gd_bf16x4 hi, lo;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float p = __builtin_amdgcn_exp2f(sc[r] - mref);
            sum += p;
            hi[r] = (gd_bf16)p;
            lo[r] = (gd_bf16)(p - (float)hi[r]);
        }
        *reinterpret_cast<gd_bf16x4 *>(&s_p[0][li][wave * 16u + 4u * lg]) = hi;
        *reinterpret_cast<gd_bf16x4 *>(&s_p[1][li][wave * 16u + 4u * lg]) = lo;
        __syncthreads();
        /* latents weighted: key steps of 32 */
        typedef short gd_short4 __attribute__((ext_vector_type(4)));
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            const gd_bf16x8 ph = *reinterpret_cast<const gd_bf16x8 *>(&s_p[0][li][32 * ks + 8 * (int)lg]);
            const gd_bf16x8 pl = *reinterpret_cast<const gd_bf16x8 *>(&s_p[1][li][32 * ks + 8 * (int)lg]);
#pragma unroll
            for (int t = 0; t < CT; ++t) {
                const uint32_t col = (wave * (uint32_t)CT + (uint32_t)t) * 16u;
                if (col >= m.kv_rank) continue; /* uniform */
                const unsigned char *src = gd_ld_smem + (32u * ks + 8u * lg + ((lane >> 2) & 3u)) * STRIDE +
                                           (col + (lane & 3u) * 4u) * 2u;
                union { gd_short4 s[2]; gd_bf16x8 v; } u;
                u.s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)src);
                u.s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)(src + 4u * STRIDE));
                o[t] = GD_MFMA(u.v, ph, o[t]);
                o[t] = GD_MFMA(u.v, pl, o[t]);
            }
        }
    }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (lg == 0u) s_sum[wave][li] = sum;
    __syncthreads();
    const uint32_t h = h0 + li;
    if (h >= m.heads) return;
    const size_t part = ((size_t)row * m.pieces + blockIdx.x) * m.heads + h;
    if (wave == 0u && lg == 0u) {
        ml[part * 2u] = mref;
        ml[part * 2u + 1u] = s_sum[0][li] + s_sum[1][li] + s_sum[2][li] + s_sum[3][li];
    }
#pragma unroll
    for (int t = 0; t < CT; ++t) {
        const uint32_t col = (wave * (uint32_t)CT + (uint32_t)t) * 16u + 4u * lg;
        if (col < m.kv_rank) *reinterpret_cast<gd_float4 *>(o_part + part * m.kv_rank + col) = o[t];
    }
}

/* grid (ceil(vdim / 32), heads, ceil(rows / 16)); kv_rank % 16 == 0 */
__global__ void __launch_bounds__(256)
gd_latent_value_mfma_kernel(const float *__restrict__ o_part, const float *__restrict__ ml,
                            const gd_bf16 *__restrict__ w_uv, const gd_bf16 *__restrict__ gate, uint32_t ldg,
                            gd_bf16 *__restrict__ out, gd_hip_latent_params m, gd_hip_seqs q)
{
    extern __shared__ __align__(16) unsigned char gd_lv_smem[]; /* merged latents BF16 [16][kv_rank + 8] */
    __shared__ float s_w[16][64], s_acc[2][64][4];
    __shared__ uint32_t s_live[16];
    gd_bf16 *s_o = reinterpret_cast<gd_bf16 *>(gd_lv_smem);
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, li = lane & 15u, lg = lane >> 4;
    const uint32_t h = blockIdx.y, r0 = blockIdx.z * 16u, stride = m.kv_rank + 8u;
    /* weights of the pieces: exp2(reference - largest reference) / total (m.pieces <= 64) */
    if (tid < 16u) {
        const uint32_t row = r0 + tid;
        int32_t seq, pos, slot;
        uint32_t live = 0u;
        if (row < q.rows && gd_seq_of_row(q, row, &seq, &pos, &slot)) {
            const uint32_t keys = min((uint32_t)pos + 1u, m.tmax);
            const float *v = ml + ((size_t)row * m.pieces * m.heads + h) * 2u;
            const size_t step = (size_t)m.heads * 2u;
            float mx = -INFINITY, total = 0.f;
            live = min((keys + m.piece_keys - 1u) / m.piece_keys, m.pieces);
            for (uint32_t i = 0; i < live; ++i) mx = fmaxf(mx, v[i * step]);
            for (uint32_t i = 0; i < live; ++i) {
                const float w = __builtin_amdgcn_exp2f(v[i * step] - mx);
                s_w[tid][i] = w;
                total = fmaf(w, v[i * step + 1u], total);
            }
            for (uint32_t i = 0; i < live; ++i) s_w[tid][i] /= total;
        }
        s_live[tid] = live;
    }
    __syncthreads();
    const uint32_t quads = m.kv_rank / 4u;
    for (uint32_t i = tid; i < 16u * quads; i += 256u) {
        const uint32_t r = i / quads, c = (i % quads) * 4u, live = s_live[r];
        const float *src = o_part + ((size_t)(r0 + r) * m.pieces * m.heads + h) * m.kv_rank + c;
        gd_float4 a = {0.f, 0.f, 0.f, 0.f};
        for (uint32_t p = 0; p < live; ++p) {
            const gd_float4 v = *reinterpret_cast<const gd_float4 *>(src + (size_t)p * m.heads * m.kv_rank);
#pragma unroll
            for (int e = 0; e < 4; ++e) a[e] = fmaf(s_w[r][p], v[e], a[e]);
        }
        gd_bf16x4 b;
#pragma unroll
        for (int e = 0; e < 4; ++e) b[e] = (gd_bf16)a[e];
        *reinterpret_cast<gd_bf16x4 *>(s_o + r * stride + c) = b;
    }
    __syncthreads();
    /* wavefront: column tile wave % 2, half wave / 2 of the latent columns */
    const uint32_t v0 = blockIdx.x * 32u + (wave & 1u) * 16u, steps = (m.kv_rank + 31u) / 32u;
    const uint32_t s_begin = (wave >> 1) * ((steps + 1u) / 2u), s_end = (wave >> 1) ? steps : (steps + 1u) / 2u;
    const gd_bf16 *wr = w_uv + ((size_t)h * m.vdim + min(v0 + li, m.vdim - 1u)) * m.kv_rank;
    const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
    gd_float4 acc = {0.f, 0.f, 0.f, 0.f};
    for (uint32_t s = s_begin; s < s_end; ++s) {
        const uint32_t c = 32u * s + 8u * lg;
        gd_bf16x8 a = zero, b = zero;
        if (c < m.kv_rank) {
            a = *reinterpret_cast<const gd_bf16x8 *>(s_o + li * stride + c);
            b = *reinterpret_cast<const gd_bf16x8 *>(wr + c);
        }
        acc = GD_MFMA(a, b, acc);
    }
    if (wave >= 2u) *reinterpret_cast<gd_float4 *>(&s_acc[wave & 1u][lane][0]) = acc;
    __syncthreads();
    if (wave >= 2u || v0 + li >= m.vdim) return;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const uint32_t lr = 4u * lg + (uint32_t)r, row = r0 + lr;
        if (row >= q.rows || s_live[lr] == 0u) continue;
        const float g = (float)gate[(size_t)row * ldg + h * m.vdim + v0 + li];
        out[((size_t)row * m.heads + h) * m.vdim + v0 + li] =
            (gd_bf16)((acc[r] + s_acc[wave & 1u][lane][r]) * gd_sigmoid_f32(g));
    }
}

template <int STEPS>
static int launch_attend(hipStream_t stream, const gd_bf16 *ql, const gd_bf16 *cache, float *o_part, float *ml,
                         const gd_hip_latent_params &m, const gd_hip_seqs &q)
{
    constexpr size_t lds = (size_t)GD_LD_TILE * (STEPS * 64u + 16u);
    static bool configured = false;
    if (!configured && lds > 48u * 1024u) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(gd_latent_attend_mfma_kernel<STEPS>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
        configured = true;
    }
    gd_latent_attend_mfma_kernel<STEPS><<<dim3(m.pieces, (m.heads + 15u) / 16u, q.rows), 256, lds, stream>>>(ql, cache, o_part, ml, m, q);
    return (int)hipGetLastError();
}

/* the three launches; the caller has checked: BF16, dim % 8 == 0, rot_dim % 8 == 0, kv_rank % 16 == 0, kv_rank <= 1024
 * (so that the merged latents fit LDS), pitch <= 1088, pieces <= 64, rows <= 65535, 16-byte aligned operands */
extern "C" int gd_hip_launch_latent_decode(hipStream_t stream, const void *qv, const void *w_ukt, const void *w_uv,
                                           const void *gate, uint32_t ldg, const float *angles, const void *cache,
                                           void *ql, float *o_part, float *ml, void *out, const gd_hip_latent_params *mp,
                                           const gd_hip_seqs *qp)
{
    const gd_hip_latent_params &m = *mp;
    const gd_hip_seqs &q = *qp;
    const uint32_t steps = (m.pitch + 31u) / 32u, rt = (q.rows + 15u) / 16u;
    const gd_bf16 *qlp = (const gd_bf16 *)ql, *cp = (const gd_bf16 *)cache;
    int e;
    gd_latent_absorb_kernel<<<dim3((m.kv_rank + 63u) / 64u, m.heads, rt), 256, 0, stream>>>(
        (const gd_bf16 *)qv, (const gd_bf16 *)w_ukt, angles, (gd_bf16 *)ql, m, q.rows);
    e = (int)hipGetLastError();
    if (e != 0) return e;
    if (steps <= 6u) e = launch_attend<6>(stream, qlp, cp, o_part, ml, m, q);
    else if (steps <= 10u) e = launch_attend<10>(stream, qlp, cp, o_part, ml, m, q);
    else if (steps <= 18u) e = launch_attend<18>(stream, qlp, cp, o_part, ml, m, q);
    else if (steps <= 34u) e = launch_attend<34>(stream, qlp, cp, o_part, ml, m, q);
    else return (int)hipErrorInvalidValue;
    if (e != 0) return e;
    gd_latent_value_mfma_kernel<<<dim3((m.vdim + 31u) / 32u, m.heads, rt), 256, 16u * (m.kv_rank + 8u) * 2u, stream>>>(
        o_part, ml, (const gd_bf16 *)w_uv, (const gd_bf16 *)gate, ldg, (gd_bf16 *)out, m, q);
    return (int)hipGetLastError();
}
