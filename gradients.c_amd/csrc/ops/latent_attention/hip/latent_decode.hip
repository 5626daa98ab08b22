/*
 * Latent attention of few new tokens per sequence on the matrix cores (gfx950, BF16): the absorbed form, in which all
 * heads of a token share one "key", the cache row, and one "value", its latent part.
 *
 *   absorb  q_lat[h] = W_uk[h]^T q[h] per 16 rows, head and 64 latent columns, and the rotated query part behind it
 *   attend  a workgroup of 4 wavefronts takes 16 or 32 heads of one token over a piece of its keys: a cache row is read from
 *           memory once for all of them.  HBM-bound on the cache rows.
 *   merge   the pieces of a token and head into one latent vector
 *   value   16 tokens and one head: the value up-projection and the output gate
 *
 * attend.  Keys advance in tiles of 32 rows through two LDS stages filled by global -> LDS loads; two workgroups share a
 * compute unit.  Both products are computed transposed, so that a head lives in one lane column:
 *     S^T = K Q^T    wavefront w: keys 16 (w % 2) .. + 15 over half w / 2 of the row; the query rows stay in registers;
 *                    the halves meet in LDS, where every wavefront picks up the scores of all 32 keys
 *     O^T = V^T P^T  wavefront w: a quarter of the latent columns; A by the transposing LDS read.  The weights a lane
 *                    has computed (keys 4g + r and 16 + 4g + r of lane group g) are its B operand as they are: the
 *                    transposing read supplies the latents of the same keys in the same k slots
 * Scores, softmax and sums are F32.  The weights enter the second product as two BF16 numbers, their rounding and the
 * rest, so that they keep 16 bits; a row's maximum is a reference point that moves only when a tile raises it by more
 * than 8 binary orders.
 *
 * LDS rows hold 4 * STEPS chunks of 16 bytes (a multiple of 8; chunks behind the cache row repeat its first and meet
 * zeros in the query).  Chunk c of key row r sits at c ^ swizzle(r): rows r, r+1 differ by half the banks, and the three
 * bits taken from r >> 1 spread 16 rows of one chunk, and the four rows of a transposing read, over all of them.
 *
 * MFMA operand layout (v_mfma_f32_16x16x32_bf16): lane l supplies row / column l % 16 and the 8 consecutive k starting
 * at 8 * (l / 16); the result lane holds column l % 16, rows 4 * (l / 16) .. + 3.
 */
#include "../../_shared/hip_device.h"
#include "hip_latent_attention_types.h"

#define GD_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0)
#define GD_LD_TILE 32u

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

/* 16 bytes per lane from global memory straight into LDS (lane l's data lands at lds_address + 16*l); the kernel
 * places its own s_waitcnt vmcnt */
__device__ __forceinline__ void gd_ld_load_lds16(const gd_bf16 *lane_address, uint32_t lds_byte_address)
{
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off"
                 :
                 : "s"(lds_byte_address), "v"(lane_address)
                 : "memory");
}

__device__ __forceinline__ uint32_t gd_ld_swizzle(uint32_t r)
{
    return ((r & 2u) << 1) | ((r & 4u) >> 1) | ((r & 8u) >> 3);
}

/* STEPS: 32-wide steps that cover a cache row (pitch <= 32 * STEPS, STEPS even); HG: groups of 16 heads per workgroup,
 * which share every fragment read from LDS.  grid (pieces, ceil(heads / (16 * HG)), rows).
 * o_part F32 [rows, pieces, heads, kv_rank], ml F32 [rows, pieces, heads, 2] (reference point in the exp2 domain, sum) */
template <int STEPS, int HG>
__global__ void __launch_bounds__(256, STEPS <= 18 ? 2 : 1)
gd_latent_attend_mfma_kernel(const gd_bf16 *__restrict__ ql, const gd_bf16 *__restrict__ cache, float *__restrict__ o_part,
                             float *__restrict__ ml, gd_hip_latent_params m, gd_hip_seqs q)
{
    constexpr uint32_t KC = 4u * STEPS, ROW = KC * 16u, STAGE = GD_LD_TILE * ROW; /* chunks, bytes per row; bytes */
    constexpr int NL = STEPS / 2, HS = STEPS / 2; /* wavefront loads per tile; steps of a wavefront's half */
    constexpr int CT = (2 * STEPS + 3) / 4;       /* 16-wide latent column tiles per wavefront */
    extern __shared__ __align__(16) unsigned char gd_ld_smem[]; /* [2][32] key rows */
    __shared__ __align__(16) float s_part[HG][4][64][4];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, li = lane & 15u, lg = lane >> 4;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const uint32_t row = blockIdx.z, h0 = blockIdx.y * (16u * HG), kg = wave & 1u, hf = wave >> 1;
    int32_t seq, pos, slot;
    if (!gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const uint32_t keys = min((uint32_t)pos + 1u, m.tmax);
    const uint32_t k_begin = blockIdx.x * m.piece_keys;
    if (k_begin >= keys) return;
    const uint32_t k_end = min(keys, k_begin + m.piece_keys);
    const uint32_t chunks = m.pitch / 8u;

    /* load t of this wavefront fills chunks (wave * NL + t) * 64 + lane of a tile */
    const gd_bf16 *rows = cache + (size_t)slot * m.tmax * m.pitch;
    const uint32_t lds_base = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) unsigned char *)gd_ld_smem;
    uint32_t ld_row[NL], ld_off[NL];
#pragma unroll
    for (int t = 0; t < NL; ++t) {
        const uint32_t g = (wave * (uint32_t)NL + (uint32_t)t) * 64u + lane, r = g / KC, c = (g % KC) ^ gd_ld_swizzle(r);
        ld_row[t] = r;
        ld_off[t] = c < chunks ? c * 8u : 0u;
    }
    auto issue = [&](uint32_t k0, uint32_t stage) __attribute__((always_inline)) {
#pragma unroll
        for (int t = 0; t < NL; ++t)
            gd_ld_load_lds16(rows + (size_t)min(k0 + ld_row[t], k_end - 1u) * m.pitch + ld_off[t],
                             lds_base + stage * STAGE + (wave * (uint32_t)NL + (uint32_t)t) * 1024u);
    };
    /* query fragments of heads h0 + 16 n + li, this wavefront's half of the row */
    gd_bf16x8 qf[HG][HS];
    const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
#pragma unroll
    for (int n = 0; n < HG; ++n) {
        const gd_bf16 *qr = ql + ((size_t)row * m.heads + min(h0 + 16u * (uint32_t)n + li, m.heads - 1u)) * m.pitch;
#pragma unroll
        for (int s = 0; s < HS; ++s) {
            const uint32_t c = 4u * (hf * (uint32_t)HS + (uint32_t)s) + lg;
            qf[n][s] = *reinterpret_cast<const gd_bf16x8 *>(qr + (c < chunks ? c * 8u : 0u));
        }
    }
    gd_float4 o[HG][CT];
    float mref[HG], sum[HG]; /* of head h0 + 16 n + li; sum: the keys of this lane group */
#pragma unroll
    for (int n = 0; n < HG; ++n) {
        mref[n] = -INFINITY;
        sum[n] = 0.f;
#pragma unroll
        for (int t = 0; t < CT; ++t) o[n][t] = (gd_float4){0.f, 0.f, 0.f, 0.f};
    }
    const float scale2 = m.scale * 1.4426950408889634f;
    const uint32_t k_row = 16u * kg + li, k_swz = gd_ld_swizzle(k_row);
    const uint32_t tr_q = lane & 3u, tr_e = (lane >> 2) & 3u, v_row = 4u * lg + tr_e;
    const uint32_t v_swz0 = gd_ld_swizzle(v_row), v_swz1 = gd_ld_swizzle(16u + v_row);
    typedef short gd_short4 __attribute__((ext_vector_type(4)));

    issue(k_begin, 0u);
    if (k_begin + GD_LD_TILE < k_end) issue(k_begin + GD_LD_TILE, 1u);
    /* The query rows are complete from here on.  Without this use of them the compiler, which does not count the loads
     * into LDS, would wait for all memory at their first use in every pass of the loop: right behind the request for
     * the next tile. */
#pragma unroll
    for (int n = 0; n < HG; ++n)
#pragma unroll
        for (int s = 0; s < HS; ++s) {
            qf[n][s] = 4u * (hf * (uint32_t)HS + (uint32_t)s) + lg < chunks ? qf[n][s] : zero;
            asm volatile("" : "+v"(qf[n][s]));
        }
    uint32_t it = 0u;
    for (uint32_t k0 = k_begin; k0 < k_end; k0 += GD_LD_TILE, ++it) {
        const unsigned char *tile = gd_ld_smem + (it & 1u) * STAGE;
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); /* this wavefront's share of the tile is in LDS */
        __syncthreads(); /* everyone's share is, and the other stage is no longer read */
        if (it != 0u && k0 + GD_LD_TILE < k_end) issue(k0 + GD_LD_TILE, (it + 1u) & 1u);
        gd_float4 sp[HG];
#pragma unroll
        for (int n = 0; n < HG; ++n) sp[n] = (gd_float4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < HS; ++s) {
            const uint32_t c = 4u * (hf * (uint32_t)HS + (uint32_t)s) + lg;
            const gd_bf16x8 a = *reinterpret_cast<const gd_bf16x8 *>(tile + k_row * ROW + (c ^ k_swz) * 16u);
#pragma unroll
            for (int n = 0; n < HG; ++n) sp[n] = GD_MFMA(a, qf[n][s], sp[n]);
        }
#pragma unroll
        for (int n = 0; n < HG; ++n) *reinterpret_cast<gd_float4 *>(&s_part[n][wave][lane][0]) = sp[n];
        __syncthreads();
        gd_bf16x8 ph[HG], pl[HG];
#pragma unroll
        for (int n = 0; n < HG; ++n) {
            float sc[8], mx = -INFINITY; /* keys 4 lg + r and 16 + 4 lg + r */
#pragma unroll
            for (int g = 0; g < 2; ++g) {
                const gd_float4 a = *reinterpret_cast<const gd_float4 *>(&s_part[n][g][lane][0]);
                const gd_float4 b = *reinterpret_cast<const gd_float4 *>(&s_part[n][2 + g][lane][0]);
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const uint32_t key = k0 + 16u * (uint32_t)g + 4u * lg + (uint32_t)r;
                    sc[4 * g + r] = key < k_end ? (a[r] + b[r]) * scale2 : -INFINITY;
                    mx = fmaxf(mx, sc[4 * g + r]);
                }
            }
            mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
            /* the tile holds at least one live key, so mx is finite (or NaN) */
            if (__builtin_amdgcn_ballot_w64(!(mx <= mref[n] + 8.f)) != 0ull) {
                const float next = fmaxf(mref[n], mx), keep = __builtin_amdgcn_exp2f(mref[n] - next);
                mref[n] = next;
                sum[n] *= keep;
#pragma unroll
                for (int t = 0; t < CT; ++t)
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[n][t][r] *= keep;
            }
#pragma unroll
            for (int r = 0; r < 8; ++r) {
                const float p = __builtin_amdgcn_exp2f(sc[r] - mref[n]);
                sum[n] += p;
                ph[n][r] = (gd_bf16)p;
                pl[n][r] = (gd_bf16)(p - (float)ph[n][r]);
            }
        }
#pragma unroll
        for (int t = 0; t < CT; ++t) {
            const uint32_t col = (wave * (uint32_t)CT + (uint32_t)t) * 16u;
            if (col >= m.kv_rank) continue; /* uniform */
            const uint32_t c = col / 8u + (tr_q >> 1), w8 = (tr_q & 1u) * 8u;
            union { gd_short4 s[2]; gd_bf16x8 v; } u;
            u.s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)(
                tile + v_row * ROW + (c ^ v_swz0) * 16u + w8));
            u.s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)(
                tile + (16u + v_row) * ROW + (c ^ v_swz1) * 16u + w8));
#pragma unroll
            for (int n = 0; n < HG; ++n) {
                o[n][t] = GD_MFMA(u.v, ph[n], o[n][t]);
                o[n][t] = GD_MFMA(u.v, pl[n], o[n][t]);
            }
        }
    }
#pragma unroll
    for (int n = 0; n < HG; ++n) {
        sum[n] += __shfl_xor(sum[n], 16, 64);
        sum[n] += __shfl_xor(sum[n], 32, 64);
        const uint32_t h = h0 + 16u * (uint32_t)n + li;
        if (h >= m.heads) continue;
        const size_t part = ((size_t)row * m.pieces + blockIdx.x) * m.heads + h;
        if (wave == 0u && lg == 0u) {
            ml[part * 2u] = mref[n];
            ml[part * 2u + 1u] = sum[n];
        }
#pragma unroll
        for (int t = 0; t < CT; ++t) {
            const uint32_t col = (wave * (uint32_t)CT + (uint32_t)t) * 16u + 4u * lg;
            if (col < m.kv_rank) *reinterpret_cast<gd_float4 *>(o_part + part * m.kv_rank + col) = o[n][t];
        }
    }
}

/* grid (rows, heads); merged BF16 [rows, heads, kv_rank]; pieces <= 64, kv_rank % 4 == 0 */
__global__ void __launch_bounds__(256)
gd_latent_merge_kernel(const float *__restrict__ o_part, const float *__restrict__ ml, gd_bf16 *__restrict__ merged,
                       gd_hip_latent_params m, gd_hip_seqs q)
{
    __shared__ float s_w[64];
    __shared__ gd_float4 s_half[128];
    const uint32_t row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63u;
    int32_t seq, pos, slot;
    if (!gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const uint32_t keys = min((uint32_t)pos + 1u, m.tmax);
    const uint32_t live = min((keys + m.piece_keys - 1u) / m.piece_keys, m.pieces);
    if (threadIdx.x < 64u) { /* a lane per piece: exp2(reference - largest reference) / total */
        const float *v = ml + (((size_t)row * m.pieces + min(lane, live - 1u)) * m.heads + h) * 2u;
        const float ref = lane < live ? v[0] : -INFINITY, part = v[1];
        const float top = gd_wave_max(ref); /* by all lanes: an exchange inside a condition would lose some */
        const float w = lane < live ? __builtin_amdgcn_exp2f(ref - top) : 0.f;
        s_w[lane] = w / gd_wave_sum(w * part);
    }
    __syncthreads();
    /* 128 threads take four columns each, the two halves of the workgroup every other piece */
    const uint32_t quads = m.kv_rank / 4u, side = threadIdx.x >> 7;
    for (uint32_t c0 = 0; c0 < quads; c0 += 128u) {
        const uint32_t c = c0 + (threadIdx.x & 127u);
        gd_float4 a = {0.f, 0.f, 0.f, 0.f};
        if (c < quads) {
            const float *src = o_part + ((size_t)row * m.pieces * m.heads + h) * m.kv_rank + c * 4u;
#pragma unroll 4
            for (uint32_t p = side; p < live; p += 2u) {
                const gd_float4 v = *reinterpret_cast<const gd_float4 *>(src + (size_t)p * m.heads * m.kv_rank);
#pragma unroll
                for (int e = 0; e < 4; ++e) a[e] = fmaf(s_w[p], v[e], a[e]);
            }
        }
        if (side != 0u) s_half[threadIdx.x & 127u] = a;
        __syncthreads();
        if (side == 0u && c < quads) {
            const gd_float4 v = s_half[threadIdx.x];
            gd_bf16x4 b;
#pragma unroll
            for (int e = 0; e < 4; ++e) b[e] = (gd_bf16)(a[e] + v[e]);
            *reinterpret_cast<gd_bf16x4 *>(merged + ((size_t)row * m.heads + h) * m.kv_rank + c * 4u) = b;
        }
        __syncthreads();
    }
}

/* grid (ceil(vdim / 32), heads, ceil(rows / 16)); kv_rank % 16 == 0 */
__global__ void __launch_bounds__(256)
gd_latent_value_mfma_kernel(const gd_bf16 *__restrict__ merged, const gd_bf16 *__restrict__ w_uv,
                            const gd_bf16 *__restrict__ gate, uint32_t ldg, gd_bf16 *__restrict__ out,
                            gd_hip_latent_params m, uint32_t rows)
{
    __shared__ float s_acc[2][64][4];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, li = lane & 15u, lg = lane >> 4;
    const uint32_t h = blockIdx.y, r0 = blockIdx.z * 16u;
    /* wavefront: column tile wave % 2, half wave / 2 of the latent columns */
    const uint32_t v0 = blockIdx.x * 32u + (wave & 1u) * 16u, steps = (m.kv_rank + 31u) / 32u;
    const uint32_t s_begin = (wave >> 1) * ((steps + 1u) / 2u), s_end = (wave >> 1) ? steps : (steps + 1u) / 2u;
    const gd_bf16 *wr = w_uv + ((size_t)h * m.vdim + min(v0 + li, m.vdim - 1u)) * m.kv_rank;
    const gd_bf16 *mr = merged + ((size_t)min(r0 + li, rows - 1u) * m.heads + h) * m.kv_rank;
    const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
    float g[4];
#pragma unroll
    for (int r = 0; r < 4; ++r)
        g[r] = (float)gate[(size_t)min(r0 + 4u * lg + (uint32_t)r, rows - 1u) * ldg + h * m.vdim + min(v0 + li, m.vdim - 1u)];
    gd_float4 acc = {0.f, 0.f, 0.f, 0.f};
    for (uint32_t s = s_begin; s < s_end; s += 4u) { /* the loads of four steps together */
        gd_bf16x8 a[4], b[4];
#pragma unroll
        for (uint32_t t = 0; t < 4u; ++t) {
            const uint32_t c = 32u * (s + t) + 8u * lg;
            const bool ok = s + t < s_end && c < m.kv_rank;
            a[t] = ok ? *reinterpret_cast<const gd_bf16x8 *>(mr + c) : zero;
            b[t] = ok ? *reinterpret_cast<const gd_bf16x8 *>(wr + c) : zero;
        }
#pragma unroll
        for (int t = 0; t < 4; ++t) acc = GD_MFMA(a[t], b[t], acc);
    }
    if (wave >= 2u) *reinterpret_cast<gd_float4 *>(&s_acc[wave & 1u][lane][0]) = acc;
    __syncthreads();
    if (wave >= 2u || v0 + li >= m.vdim) return;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const uint32_t row = r0 + 4u * lg + (uint32_t)r;
        if (row < rows)
            out[((size_t)row * m.heads + h) * m.vdim + v0 + li] =
                (gd_bf16)((acc[r] + s_acc[wave & 1u][lane][r]) * gd_sigmoid_f32(g[r]));
    }
}

template <int STEPS, int HG>
static int launch_attend(hipStream_t stream, const gd_bf16 *ql, const gd_bf16 *cache, float *o_part, float *ml,
                         const gd_hip_latent_params &m, const gd_hip_seqs &q)
{
    constexpr size_t lds = (size_t)2u * GD_LD_TILE * STEPS * 64u;
    static bool configured = false;
    if (!configured && lds > 48u * 1024u) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(gd_latent_attend_mfma_kernel<STEPS, HG>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
        configured = true;
    }
    gd_latent_attend_mfma_kernel<STEPS, HG><<<dim3(m.pieces, (m.heads + 16u * HG - 1u) / (16u * HG), q.rows), 256, lds, stream>>>(ql, cache, o_part, ml, m, q);
    return (int)hipGetLastError();
}

/* the four launches (the absorbed queries' place takes the merged latents); the caller has checked: BF16, dim % 8 == 0, rot_dim % 8 == 0, kv_rank % 16 == 0, pitch <= 1088, pieces <= 64, rows <= 65535, 16-byte aligned operands */
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
#define GD_GO(S) e = m.heads > 16u ? launch_attend<S, 2>(stream, qlp, cp, o_part, ml, m, q) : launch_attend<S, 1>(stream, qlp, cp, o_part, ml, m, q)
    if (steps <= 6u) GD_GO(6);
    else if (steps <= 10u) GD_GO(10);
    else if (steps <= 18u) GD_GO(18);
    else if (steps <= 34u) e = launch_attend<34, 1>(stream, qlp, cp, o_part, ml, m, q);
    else return (int)hipErrorInvalidValue;
#undef GD_GO
    if (e != 0) return e;
    /* the queries are used up: their place takes the merged latents (kv_rank <= pitch) */
    gd_latent_merge_kernel<<<dim3(q.rows, m.heads), 256, 0, stream>>>(o_part, ml, (gd_bf16 *)ql, m, q);
    e = (int)hipGetLastError();
    if (e != 0) return e;
    gd_latent_value_mfma_kernel<<<dim3((m.vdim + 31u) / 32u, m.heads, rt), 256, 0, stream>>>(
        qlp, (const gd_bf16 *)w_uv, (const gd_bf16 *)gate, ldg, (gd_bf16 *)out, m, q.rows);
    return (int)hipGetLastError();
}
