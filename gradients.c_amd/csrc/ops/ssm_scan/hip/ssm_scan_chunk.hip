/*
 * Selective state-space recurrence of prompts on the matrix cores (gfx950, BF16 x, B and C; F32 decays and state).
 *
 * In chunks of 64 tokens with running sums cs_i of the decays' logarithms a_i = -exp(a_log) dt_i, the recurrence of a
 * head is (S the state in front of the chunk, i, j places in it):
 *   y_i = sum_{j <= i} (C_i . B_j) exp(cs_i - cs_j) dt_j x_j + exp(cs_i) S^T C_i + d x_i
 *   S  <- exp(cs_63) S + sum_j exp(cs_63 - cs_j) dt_j B_j x_j^T
 * four small matrix products.  A workgroup of 4 wavefronts owns a [N, PT] column slice of one head of one sequence and
 * walks its chunks with the state in the F32 accumulators of the last product; nothing but x, B, C, dt is read and
 * nothing but y is written per chunk.
 *
 * Exactness: x, B and C are BF16 as the convolution leaves them.  Whatever else enters a product - the decayed,
 * step-weighted C B^T, the decayed B, the state - is F32 and enters as two BF16 numbers, its rounding and the rest (16
 * bits), each with a matrix instruction of its own; sums are F32.
 *
 * All products by v_mfma_f32_32x32x16_bf16: lane l supplies row / column l % 32 and the 8 consecutive k starting at
 * 8 * (l / 32); the result lane holds column l % 32, register 4q + r row 8q + 4 * (l / 32) + r.
 *   G = C B^T        wavefront w: 32 x 32 quadrant (w / 2, w % 2); the one above the diagonal is skipped
 *   Y = M X + E C S  wavefront w: row block w / 2, columns 32 * (w % 2) .. (PT = 64)
 *   S = B'^T X       32 x 32 tiles of the [NP, PT] state dealt out to the wavefronts
 * Tokens behind a sequence's end enter with dt = 0 and zero rows: they neither decay nor add.
 */
#include "../../_shared/hip_device.h"
#include "hip_ssm_scan_types.h"

#define GD_SC_L 64u
#define GD_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0)
typedef short gd_sc_short4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ void gd_sc_split(float v, gd_bf16 *hi, gd_bf16 *lo)
{
    *hi = (gd_bf16)v;
    *lo = (gd_bf16)(v - (float)*hi);
}

/* 8 consecutive k (rows k0 .. k0+7 of an LDS tile [k][column], `stride` bytes per row) of column col0 + l % 32, for the
 * lane's half k0 = ... + 8 * (l / 32): two transposing reads of four rows each */
__device__ __forceinline__ gd_bf16x8 gd_sc_turned(const unsigned char *tile, uint32_t stride, uint32_t k0, uint32_t col0,
                                                  uint32_t lane)
{
    const uint32_t q = lane & 3u, e = (lane >> 2) & 3u, g1 = (lane >> 4) & 1u;
    const unsigned char *src = tile + (k0 + 8u * (lane >> 5) + e) * stride + (col0 + 16u * g1 + 4u * q) * 2u;
    union { gd_sc_short4 s[2]; gd_bf16x8 v; } u;
    u.s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_sc_short4 *)src);
    u.s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_sc_short4 *)(src + 4u * stride));
    return u.v;
}

template <int NP>
struct gd_sc_layout {
    static constexpr uint32_t PT = 64u;
    static constexpr uint32_t BC = NP * 2u + 16u; /* bytes per token row of B and C; per column row of S^T */
    static constexpr uint32_t XS = PT * 2u + 16u; /* per token row of X */
    static constexpr uint32_t MS = GD_SC_L * 2u + 16u;
    /* M takes the place of C, which is used up when M is written */
    static constexpr uint32_t CM = BC > 2u * MS ? GD_SC_L * BC : GD_SC_L * 2u * MS;
    static constexpr uint32_t b = 0u, c = b + GD_SC_L * BC, mh = c, ml = mh + GD_SC_L * MS, x = c + CM, sh = x + GD_SC_L * XS,
                              sl = sh + PT * BC, end = sl + PT * BC;
};

template <int NP>
__global__ void __launch_bounds__(256, NP <= 128 ? 2 : 1)
gd_ssm_scan_chunk_kernel(const gd_bf16 *__restrict__ xbc, const gd_bf16 *__restrict__ dt_raw,
                         const float *__restrict__ dt_bias, const float *__restrict__ a_log,
                         const float *__restrict__ d_skip, float *__restrict__ states, gd_bf16 *__restrict__ y,
                         gd_hip_ssm_params m, gd_hip_seqs q)
{
    using L = gd_sc_layout<NP>;
    constexpr int TILES = NP / 32 * 2, TPW = (TILES + 3) / 4; /* 32 x 32 tiles of the state, per wavefront */
    constexpr int NCH = NP / 8;                               /* 16-byte chunks per token of B and C */
    extern __shared__ __align__(16) unsigned char sm[];
    __shared__ __align__(16) float s_cs[GD_SC_L], s_dt[GD_SC_L], s_w[GD_SC_L]; /* cs in the exp2 domain */
    const uint32_t tid = threadIdx.x, lane = tid & 63u, lc = lane & 31u, hh = lane >> 5;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const uint32_t p0 = blockIdx.x * L::PT, h = blockIdx.y, N = m.state, P = m.vdim, inner = m.heads * P;
    const uint32_t g = h / (m.heads / m.groups), cols = min(P - p0, L::PT);
    int32_t first, n, start, slot;
    if (!gd_seq_span(q, blockIdx.z, &first, &n, &start, &slot)) return;
    float *st = states + ((size_t)slot * m.heads + h) * N * P + p0;
    const float rate = expf(a_log[h]) * 1.4426950408889634f, bias = dt_bias[h], skip = d_skip[h];

    /* the state: tile t of this wavefront covers rows 32 * nb, columns 32 * pb */
    gd_float16 S[TPW];
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
        const uint32_t ti = wave * (uint32_t)TPW + (uint32_t)t, nb = ti / 2u, pb = ti % 2u, col = 32u * pb + lc;
#pragma unroll
        for (int e = 0; e < 16; ++e) {
            const uint32_t row = 32u * nb + 8u * (uint32_t)(e >> 2) + 4u * hh + (uint32_t)(e & 3);
            S[t][e] = start > 0 && ti < (uint32_t)TILES && row < N && col < cols ? st[(size_t)row * P + col] : 0.f;
        }
    }

    /* staging registers of the next chunk: 16-byte pieces of B, C (64 x NCH each) and X (64 x 8) */
    constexpr int BCL = (int)(GD_SC_L * NCH / 256u), XL = 2;
    gd_bf16x8 rb[BCL], rc[BCL], rx[XL];
    float r_dt = 0.f;
    const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
    auto request = [&](int32_t t0) __attribute__((always_inline)) {
        const gd_bf16 *rows = xbc + (size_t)(first + t0) * m.ld_xbc;
        const uint32_t nt = (uint32_t)(n - t0);
#pragma unroll
        for (int i = 0; i < BCL; ++i) {
            const uint32_t idx = tid + 256u * (uint32_t)i, t = idx / NCH, c = idx % NCH;
            const gd_bf16 *src = rows + (size_t)min(t, nt - 1u) * m.ld_xbc + inner + g * N + c * 8u;
            const bool ok = t < nt && c * 8u < N;
            rb[i] = ok ? *reinterpret_cast<const gd_bf16x8 *>(src) : zero;
            rc[i] = ok ? *reinterpret_cast<const gd_bf16x8 *>(src + m.groups * N) : zero;
        }
#pragma unroll
        for (int i = 0; i < XL; ++i) {
            const uint32_t idx = tid + 256u * (uint32_t)i, t = idx / 8u, c = idx % 8u;
            rx[i] = t < nt && c * 8u < cols
                        ? *reinterpret_cast<const gd_bf16x8 *>(rows + (size_t)t * m.ld_xbc + h * P + p0 + c * 8u) : zero;
        }
        if (tid < GD_SC_L) r_dt = tid < nt ? (float)dt_raw[(size_t)(first + t0 + (int32_t)tid) * m.ld_dt + h] : 0.f;
    };
    request(0);
    for (int32_t t0 = 0; t0 < n; t0 += (int32_t)GD_SC_L) {
        const uint32_t nt = min((uint32_t)(n - t0), GD_SC_L);
        __syncthreads(); /* the chunk before is used up */
#pragma unroll
        for (int i = 0; i < BCL; ++i) {
            const uint32_t idx = tid + 256u * (uint32_t)i, t = idx / NCH, c = idx % NCH;
            *reinterpret_cast<gd_bf16x8 *>(sm + L::b + t * L::BC + c * 16u) = rb[i];
            *reinterpret_cast<gd_bf16x8 *>(sm + L::c + t * L::BC + c * 16u) = rc[i];
        }
#pragma unroll
        for (int i = 0; i < XL; ++i) {
            const uint32_t idx = tid + 256u * (uint32_t)i, t = idx / 8u, c = idx % 8u;
            *reinterpret_cast<gd_bf16x8 *>(sm + L::x + t * L::XS + c * 16u) = rx[i];
        }
        if (wave == 0u) { /* running sums of the decays' logarithms */
            const float raw = r_dt + bias;
            const float dt = tid < nt ? fmaxf(raw, 0.0f) + log1pf(expf(-fabsf(raw))) : 0.f;
            float cs = -rate * dt;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) {
                const float up = __shfl_up(cs, off, 64);
                if ((int)lane >= off) cs += up;
            }
            s_cs[lane] = cs;
            s_dt[lane] = dt;
            s_w[lane] = __builtin_amdgcn_exp2f(__shfl(cs, 63, 64) - cs) * dt;
        }
        /* the state in front of the chunk as S^T, in two parts */
#pragma unroll
        for (int t = 0; t < TPW; ++t) {
            const uint32_t ti = wave * (uint32_t)TPW + (uint32_t)t, nb = ti / 2u, pb = ti % 2u;
            if (ti >= (uint32_t)TILES) continue;
#pragma unroll
            for (int a = 0; a < 4; ++a) {
                gd_bf16x4 vh, vl;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    gd_bf16 hi, lo;
                    gd_sc_split(S[t][4 * a + r], &hi, &lo);
                    vh[r] = hi;
                    vl[r] = lo;
                }
                const uint32_t at = (32u * pb + lc) * L::BC + (32u * nb + 8u * (uint32_t)a + 4u * hh) * 2u;
                *reinterpret_cast<gd_bf16x4 *>(sm + L::sh + at) = vh;
                *reinterpret_cast<gd_bf16x4 *>(sm + L::sl + at) = vl;
            }
        }
        if (t0 + (int32_t)GD_SC_L < n) request(t0 + (int32_t)GD_SC_L);
        __syncthreads();

        /* G^T = B C^T keeps a lane's registers along j, four consecutive ones per store of M[i][j]; Y^T: rows p (columns
         * 32 * pb of the slice), columns i (row block ib): a lane holds one token */
        const uint32_t ib = wave >> 1, jb = wave & 1u, pb = jb, i = 32u * ib + lc;
        gd_float16 gm, ys;
#pragma unroll
        for (int e = 0; e < 16; ++e) gm[e] = ys[e] = 0.f;
#pragma unroll
        for (int ks = 0; ks < NP / 16; ++ks) {
            const uint32_t c = (16u * ks + 8u * hh) * 2u;
            const gd_bf16x8 cv = *reinterpret_cast<const gd_bf16x8 *>(sm + L::c + i * L::BC + c);
            const gd_bf16x8 ah = *reinterpret_cast<const gd_bf16x8 *>(sm + L::sh + (32u * pb + lc) * L::BC + c);
            const gd_bf16x8 al = *reinterpret_cast<const gd_bf16x8 *>(sm + L::sl + (32u * pb + lc) * L::BC + c);
            if (jb <= ib) {
                const gd_bf16x8 bv = *reinterpret_cast<const gd_bf16x8 *>(sm + L::b + (32u * jb + lc) * L::BC + c);
                gm = GD_MFMA(bv, cv, gm);
            }
            ys = GD_MFMA(ah, cv, ys);
            ys = GD_MFMA(al, cv, ys);
        }
        const float ci = s_cs[i];
        __syncthreads(); /* C is used up: M takes its place */
        if (jb <= ib) {
#pragma unroll
            for (int a = 0; a < 4; ++a) {
                const uint32_t j0 = 32u * jb + 8u * (uint32_t)a + 4u * hh;
                const gd_float4 cj = *reinterpret_cast<const gd_float4 *>(&s_cs[j0]);
                const gd_float4 dj = *reinterpret_cast<const gd_float4 *>(&s_dt[j0]);
                gd_bf16x4 vh, vl;
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float v = j0 + (uint32_t)r <= i ? gm[4 * a + r] * __builtin_amdgcn_exp2f(ci - cj[r]) * dj[r] : 0.f;
                    gd_bf16 hi, lo;
                    gd_sc_split(v, &hi, &lo);
                    vh[r] = hi;
                    vl[r] = lo;
                }
                *reinterpret_cast<gd_bf16x4 *>(sm + L::mh + i * L::MS + j0 * 2u) = vh;
                *reinterpret_cast<gd_bf16x4 *>(sm + L::ml + i * L::MS + j0 * 2u) = vl;
            }
        }
        __syncthreads();
        {
            const float ei = __builtin_amdgcn_exp2f(ci);
#pragma unroll
            for (int e = 0; e < 16; ++e) ys[e] *= ei;
#pragma unroll
            for (int ks = 0; ks < 4; ++ks) { /* X^T M^T over j <= i: the second half only for the lower rows */
                if (16u * ks >= 32u * (ib + 1u)) continue;
                const uint32_t j = (16u * ks + 8u * hh) * 2u;
                const gd_bf16x8 xv = gd_sc_turned(sm + L::x, L::XS, 16u * (uint32_t)ks, 32u * pb, lane);
                const gd_bf16x8 mh = *reinterpret_cast<const gd_bf16x8 *>(sm + L::mh + i * L::MS + j);
                const gd_bf16x8 ml = *reinterpret_cast<const gd_bf16x8 *>(sm + L::ml + i * L::MS + j);
                ys = GD_MFMA(xv, mh, ys);
                ys = GD_MFMA(xv, ml, ys);
            }
            if (i < nt) {
                gd_bf16 *yr = y + (size_t)(first + t0 + (int32_t)i) * inner + h * P + p0 + 32u * pb;
#pragma unroll
                for (int a = 0; a < 4; ++a) {
                    const uint32_t p = 8u * (uint32_t)a + 4u * hh;
                    if (32u * pb + p >= cols) continue;
                    const gd_bf16x4 xv = *reinterpret_cast<const gd_bf16x4 *>(sm + L::x + i * L::XS + (32u * pb + p) * 2u);
                    gd_bf16x4 o;
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[r] = (gd_bf16)(ys[4 * a + r] + skip * (float)xv[r]);
                    *reinterpret_cast<gd_bf16x4 *>(yr + p) = o;
                }
            }
        }
        /* state behind the chunk */
        const float decay = __builtin_amdgcn_exp2f(s_cs[GD_SC_L - 1u]);
        constexpr int PB = TPW < 2 ? TPW : 2; /* tiles of one row block that lie with this wavefront */
#pragma unroll
        for (int t = 0; t < TPW; ++t)
#pragma unroll
            for (int e = 0; e < 16; ++e) S[t][e] *= decay;
#pragma unroll
        for (int tb = 0; tb < TPW; tb += PB) {
            const uint32_t ti = wave * (uint32_t)TPW + (uint32_t)tb, nb = ti / 2u;
            if (ti >= (uint32_t)TILES) continue;
#pragma unroll
            for (int ks = 0; ks < 4; ++ks) {
                const gd_bf16x8 bv = gd_sc_turned(sm + L::b, L::BC, 16u * (uint32_t)ks, 32u * nb, lane);
                const gd_float4 w0 = *reinterpret_cast<const gd_float4 *>(&s_w[16 * ks + 8 * (int)hh]);
                const gd_float4 w1 = *reinterpret_cast<const gd_float4 *>(&s_w[16 * ks + 8 * (int)hh + 4]);
                gd_bf16x8 bh, bl;
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    gd_bf16 hi, lo;
                    gd_sc_split((float)bv[e] * (e < 4 ? w0[e & 3] : w1[e & 3]), &hi, &lo);
                    bh[e] = hi;
                    bl[e] = lo;
                }
#pragma unroll
                for (int u = 0; u < PB; ++u) {
                    const gd_bf16x8 xv = gd_sc_turned(sm + L::x, L::XS, 16u * (uint32_t)ks, 32u * ((ti + (uint32_t)u) % 2u), lane);
                    S[tb + u] = GD_MFMA(bh, xv, S[tb + u]);
                    S[tb + u] = GD_MFMA(bl, xv, S[tb + u]);
                }
            }
        }
    }
#pragma unroll
    for (int t = 0; t < TPW; ++t) {
        const uint32_t ti = wave * (uint32_t)TPW + (uint32_t)t, nb = ti / 2u, pb = ti % 2u, col = 32u * pb + lc;
#pragma unroll
        for (int e = 0; e < 16; ++e) {
            const uint32_t row = 32u * nb + 8u * (uint32_t)(e >> 2) + 4u * hh + (uint32_t)(e & 3);
            if (ti < (uint32_t)TILES && row < N && col < cols) st[(size_t)row * P + col] = S[t][e];
        }
    }
}

template <int NP>
static int launch_chunk(hipStream_t stream, const gd_bf16 *xbc, const gd_bf16 *dt_raw, const float *dt_bias,
                        const float *a_log, const float *d_skip, float *states, gd_bf16 *y, const gd_hip_ssm_params &m,
                        const gd_hip_seqs &q)
{
    constexpr size_t lds = gd_sc_layout<NP>::end;
    static bool configured = false;
    if (!configured) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(gd_ssm_scan_chunk_kernel<NP>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
        configured = true;
    }
    gd_ssm_scan_chunk_kernel<NP><<<dim3((m.vdim + 63u) / 64u, m.heads, q.seqs), 256, lds, stream>>>(
        xbc, dt_raw, dt_bias, a_log, d_skip, states, y, m, q);
    return (int)hipGetLastError();
}

/* The caller has checked: BF16, state, vdim and row pitch of xbc multiples of 8, state <= 256, 16-byte aligned xbc and
 * y */
extern "C" int gd_hip_launch_ssm_scan_chunk(hipStream_t stream, const void *xbc, const void *dt_raw, const float *dt_bias,
                                            const float *a_log, const float *d_skip, float *states, void *y,
                                            const gd_hip_ssm_params *m, const gd_hip_seqs *q)
{
#define GD_GO(NP) return launch_chunk<NP>(stream, (const gd_bf16 *)xbc, (const gd_bf16 *)dt_raw, dt_bias, a_log, d_skip, states, (gd_bf16 *)y, *m, *q)
    if (m->state <= 32u) GD_GO(32);
    if (m->state <= 64u) GD_GO(64);
    if (m->state <= 128u) GD_GO(128);
    GD_GO(256);
#undef GD_GO
}
