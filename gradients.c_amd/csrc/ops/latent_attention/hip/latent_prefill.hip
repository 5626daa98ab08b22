/*
 * Latent attention of prompts and long portions on the matrix cores (gfx950, BF16): the expanded form.  The latents of
 * all tokens a sequence holds are gathered (gather kernel), taken through the stacked key and value up-projections by
 * the projection kernel, and attended over like ordinary keys and values; the rotated key part, shared by the heads,
 * is read from the gathered cache rows.
 *
 * The attention kernel follows gd_sdpa_varlen_mfma_kernel (ops/sdpa_varlen/hip/sdpa_varlen_mfma.hip): a workgroup of 4
 * wavefronts owns 128 consecutive new rows of one sequence and one head, keys advance in blocks of 64 through two LDS
 * stages filled by global -> LDS loads, both products transposed (S^T = K Q^T, O^T = V^T P^T) so that a query row
 * lives in one lane.  What is different here:
 *   - query and value sizes differ (dim + rot_dim padded to 16 * KSTEPS with zeros in the query, vdim to 32 * DTILES
 *     with columns that are not stored), and a key row comes from two places;
 *   - new rows sit behind the tokens of earlier portions: row i of a sequence has position start + i and sees the keys
 *     up to it;
 *   - the query's rotated part is turned to its position while it is loaded;
 *   - the weights enter the second product as two BF16 numbers (rounding and rest: 16 bits);
 *   - the output gate is applied in F32 before the one rounding.
 */
#include "../../_shared/hip_device.h"
#include "hip_latent_attention_types.h"

#define GD_LP_NEG_INF (-__builtin_inff())

/* cache rows [slot, 0 .. start + n) of every sequence, packed, 16 rows per workgroup; kv_cu [seqs + 1] */
__global__ void __launch_bounds__(256)
gd_latent_gather_kernel(const gd_bf16 *__restrict__ cache, const int32_t *__restrict__ kv_cu, gd_bf16 *__restrict__ packed,
                        uint32_t total, gd_hip_latent_params m, gd_hip_seqs q)
{
    __shared__ long long s_src[16]; /* first element of the cache row; -1: none */
    const uint32_t r0 = blockIdx.x * 16u, chunks = m.pitch / 8u;
    if (threadIdx.x < 16u) {
        const uint32_t r = r0 + threadIdx.x;
        long long src = -1;
        if (r < total) {
            uint32_t lo = 0u, hi = q.seqs; /* the sequence whose range holds r */
            while (hi - lo > 1u) {
                const uint32_t mid = (lo + hi) / 2u;
                if ((uint32_t)kv_cu[mid] <= r) lo = mid;
                else hi = mid;
            }
            const int32_t slot = q.slot[lo];
            const uint32_t at = r - (uint32_t)kv_cu[lo];
            if (slot >= 0 && (uint32_t)slot < q.slots && at < m.tmax) src = (long long)(((size_t)slot * m.tmax + at) * m.pitch);
        }
        s_src[threadIdx.x] = src;
    }
    __syncthreads();
    for (uint32_t i = threadIdx.x; i < 16u * chunks; i += 256u) {
        const uint32_t r = i / chunks, c = i % chunks;
        const long long src = s_src[r];
        if (src >= 0)
            reinterpret_cast<gd_bf16x8 *>(packed + (size_t)(r0 + r) * m.pitch)[c] =
                reinterpret_cast<const gd_bf16x8 *>(cache + src)[c];
    }
}

/* 16 bytes per lane from global memory straight into LDS (lane l's data lands at lds_address + 16*l); the kernel
 * places its own s_waitcnt vmcnt */
__device__ __forceinline__ void gd_lp_load_lds16(const gd_bf16 *lane_address, uint32_t lds_byte_address)
{
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off"
                 :
                 : "s"(lds_byte_address), "v"(lane_address)
                 : "memory");
}

template <int KSTEPS, int DTILES>
__global__ void __launch_bounds__(256, 2)
gd_latent_prefill_kernel(const gd_bf16 *__restrict__ q_rows, const gd_bf16 *__restrict__ kv, const gd_bf16 *__restrict__ packed,
                         const float *__restrict__ angles, const gd_bf16 *__restrict__ gate, uint32_t ldg,
                         const int32_t *__restrict__ kv_cu, uint32_t kv_total, gd_bf16 *__restrict__ out,
                         gd_hip_latent_params m, gd_hip_seqs sq)
{
    constexpr uint32_t BQ = 128u, BKEYS = 64u;
    constexpr uint32_t KC = 2u * KSTEPS, VC = 4u * DTILES; /* 16-byte chunks per key / value row in LDS */
    constexpr int KL = (int)(BKEYS * KC / 256u), VL = (int)(BKEYS * VC / 256u); /* wavefront loads per block */
    constexpr uint32_t STAGE = BKEYS * (KC + VC) * 16u;
    typedef short gd_short4 __attribute__((ext_vector_type(4)));
    extern __shared__ __align__(16) unsigned char gd_lp_smem[]; /* [2 stages][K block, V block] */
    const uint32_t tid = threadIdx.x, lane = tid & 63u;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const uint32_t lq = lane & 31u, hh = lane >> 5;
    const uint32_t head = blockIdx.x % m.heads, pair = blockIdx.x / m.heads;

    /* (sequence, 128-row block) number `pair`, 64 sequences at a time across the lanes */
    uint32_t seen = 0u, b = sq.seqs;
    int first = 0, end = 0;
    for (uint32_t b0 = 0u; b0 < sq.seqs; b0 += 64u) {
        const uint32_t bl = b0 + lane;
        int s0 = 0, e0 = 0;
        if (bl < sq.seqs) {
            s0 = sq.cu[bl];
            e0 = sq.cu[bl + 1u];
        }
        const uint32_t nb = e0 > s0 ? ((uint32_t)(e0 - s0) + BQ - 1u) / BQ : 0u;
        uint32_t incl = nb;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const uint32_t up = (uint32_t)__shfl_up((int)incl, off, 64);
            if ((int)lane >= off) incl += up;
        }
        const unsigned long long hit = __builtin_amdgcn_ballot_w64(seen + incl > pair);
        if (hit != 0ull) {
            const int src = __builtin_ctzll(hit);
            b = b0 + (uint32_t)src;
            first = __shfl(s0, src, 64);
            end = __shfl(e0, src, 64);
            seen += (uint32_t)__shfl((int)(incl - nb), src, 64);
            break;
        }
        seen += (uint32_t)__shfl((int)incl, 63, 64);
    }
    if (b == sq.seqs || first < 0 || end > (int)sq.rows) return;
    const int start = sq.start[b], slot = sq.slot[b], kv0 = kv_cu[b], kv1 = kv_cu[b + 1u];
    const int n = end - first, n_kv = start + n;
    if (start < 0 || slot < 0 || (uint32_t)slot >= sq.slots || kv0 < 0 || kv1 > (int)kv_total || kv1 - kv0 < n_kv) return;
    const int i0 = (int)((pair - seen) * BQ);
    const int kend = min(n_kv, start + min(i0 + (int)BQ, n)); /* keys of the block's last row */
    const int wi0 = i0 + (int)wave * 32, i = wi0 + (int)lq;
    const bool row_live = i < n;
    const uint32_t qd = m.dim + m.rot_dim, half = m.rot_dim / 2u;
    const size_t qrow = (size_t)(first + min(i, n - 1));

    gd_bf16x8 qf[KSTEPS];
    {
        const gd_bf16 *qp = q_rows + (qrow * m.heads + head) * qd;
        const float *ang = angles + qrow * m.rot_dim;
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ++ks) {
            const uint32_t e0 = 16u * ks + 8u * hh;
            qf[ks] = *reinterpret_cast<const gd_bf16x8 *>(qp + (e0 < qd ? e0 : 0u)); /* rows behind the end: the last */
        }
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ++ks) {
            const uint32_t e0 = 16u * ks + 8u * hh;
            if (e0 >= qd) {
                qf[ks] = (gd_bf16x8)(gd_bf16)0.f;
            } else if (e0 >= m.dim && half % 8u == 0u) { /* the 8 elements lie in one half */
                const uint32_t r0 = e0 - m.dim, p0 = r0 < half ? r0 : r0 - half;
                const gd_bf16x8 other = *reinterpret_cast<const gd_bf16x8 *>(qp + m.dim + (r0 < half ? r0 + half : p0));
                const gd_float4 c4[2] = {*reinterpret_cast<const gd_float4 *>(ang + p0),
                                         *reinterpret_cast<const gd_float4 *>(ang + p0 + 4u)};
                const gd_float4 s4[2] = {*reinterpret_cast<const gd_float4 *>(ang + half + p0),
                                         *reinterpret_cast<const gd_float4 *>(ang + half + p0 + 4u)};
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const float c = c4[e >> 2][e & 3], s = s4[e >> 2][e & 3], own = (float)qf[ks][e], far = (float)other[e];
                    qf[ks][e] = (gd_bf16)(r0 < half ? own * c - far * s : own * c + far * s);
                }
            } else if (e0 >= m.dim) {
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const uint32_t r = e0 + (uint32_t)e - m.dim, p = r < half ? r : r - half;
                    const float c = ang[p], s = ang[half + p], own = (float)qf[ks][e];
                    const float other = (float)qp[m.dim + (r < half ? r + half : r - half)];
                    qf[ks][e] = (gd_bf16)(r < half ? own * c - other * s : own * c + other * s);
                }
            }
        }
    }

    /* staging: load t of this wavefront fills LDS chunks (wave * KL + t) * 64 + lane of the K block (V likewise); chunk
     * g is chunk g % KC of key g / KC, taken from the place the swizzle names */
    const uint32_t ldkv = m.heads * (m.dim + m.vdim);
    const uint32_t k_chunks = m.dim / 8u, all_chunks = qd / 8u, v_chunks = m.vdim / 8u;
    const uint32_t lds_base = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) unsigned char *)gd_lp_smem;
    const gd_bf16 *k_src[KL], *v_src[VL];
    uint32_t k_pitch[KL], k_row[KL], v_row[VL];
#pragma unroll
    for (int t = 0; t < KL; ++t) {
        const uint32_t g = (wave * (uint32_t)KL + (uint32_t)t) * 64u + lane, r = g / KC, pos = g % KC;
        const uint32_t c = pos ^ (KC % 16u == 0u ? (r & 15u) : ((r >> 1) & 7u));
        const bool rot = c >= k_chunks && c < all_chunks;
        k_row[t] = r;
        k_pitch[t] = rot ? m.pitch : ldkv;
        k_src[t] = rot ? packed + m.kv_rank + (c - k_chunks) * 8u : kv + head * m.dim + (c < k_chunks ? c * 8u : 0u);
    }
#pragma unroll
    for (int t = 0; t < VL; ++t) {
        const uint32_t g = (wave * (uint32_t)VL + (uint32_t)t) * 64u + lane, r = g / VC, pos = g % VC;
        const uint32_t c = pos ^ (DTILES == 4 ? ((r & 3u) << 2) : (((r >> 1) & 1u) << 2));
        v_row[t] = r;
        v_src[t] = kv + m.heads * m.dim + head * m.vdim + (c < v_chunks ? c * 8u : 0u);
    }
    auto issue_block = [&](int jb, uint32_t stage) __attribute__((always_inline)) {
        const uint32_t base = lds_base + stage * STAGE;
#pragma unroll
        for (int t = 0; t < KL; ++t) {
            const uint32_t row = (uint32_t)kv0 + min((uint32_t)jb + k_row[t], (uint32_t)n_kv - 1u);
            gd_lp_load_lds16(k_src[t] + (size_t)row * k_pitch[t], base + (wave * (uint32_t)KL + (uint32_t)t) * 1024u);
        }
#pragma unroll
        for (int t = 0; t < VL; ++t) {
            const uint32_t row = (uint32_t)kv0 + min((uint32_t)jb + v_row[t], (uint32_t)n_kv - 1u);
            gd_lp_load_lds16(v_src[t] + (size_t)row * ldkv,
                             base + BKEYS * KC * 16u + (wave * (uint32_t)VL + (uint32_t)t) * 1024u);
        }
    };

    gd_float16 o[DTILES];
#pragma unroll
    for (int t = 0; t < DTILES; ++t)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[t][e] = 0.f;
    float mref = GD_LP_NEG_INF, l = 0.f;
    const float scale2 = m.scale * 1.4426950408889634f;
    const int jmax = start + min(i, n - 1); /* last visible key of this lane's row */
    const int wave_first = start + wi0;     /* position of the wavefront's first row */
    const uint32_t tr_q = lane & 3u, tr_e = (lane >> 2) & 3u, tr_g1 = (lane >> 4) & 1u;

    issue_block(0, 0u);
    uint32_t it = 0u;
    for (int jb = 0; jb < kend; jb += (int)BKEYS, ++it) {
        const uint32_t stage = it & 1u;
        __builtin_amdgcn_s_waitcnt(0x0F70); /* vmcnt(0): this wavefront's share of block jb is in LDS */
        __syncthreads();                    /* everyone's share is, and the other stage is no longer read */
        if (jb + (int)BKEYS < kend) issue_block(jb + (int)BKEYS, stage ^ 1u);
        const unsigned char *sK = gd_lp_smem + (size_t)stage * STAGE;
        const unsigned char *sV = sK + BKEYS * KC * 16u;
        if (jb > wave_first + 31) continue; /* every row of the wavefront precedes the block */

        gd_float16 st[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
#pragma unroll
            for (int e = 0; e < 16; ++e) st[t][e] = 0.f;
            const uint32_t r = 32u * t + lq, swz = KC % 16u == 0u ? (r & 15u) : ((r >> 1) & 7u);
#pragma unroll
            for (int ks = 0; ks < KSTEPS; ++ks) {
                const gd_bf16x8 kf = *reinterpret_cast<const gd_bf16x8 *>(sK + (r * KC + ((2u * ks + hh) ^ swz)) * 16u);
                st[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[ks], st[t], 0, 0, 0);
            }
        }
        /* raw scores; the scale rides in the multiply-add in front of the exp2, so the mask and the maximum follow its
         * sign */
        float mloc = GD_LP_NEG_INF;
        const bool full = jb + 63 <= wave_first;
#pragma unroll
        for (int t = 0; t < 2; ++t) {
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const int j = jb + 32 * t + 8 * (e >> 2) + 4 * (int)hh + (e & 3);
                st[t][e] = full || j <= jmax ? st[t][e] * scale2 : GD_LP_NEG_INF;
                mloc = fmaxf(mloc, st[t][e]);
            }
        }
        mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
        const bool moves = mloc > mref + 8.f || (mref == GD_LP_NEG_INF && mloc != GD_LP_NEG_INF);
        if (__builtin_amdgcn_ballot_w64(moves) != 0ull) {
            const float next = fmaxf(mref, mloc), safe = next == GD_LP_NEG_INF ? 0.f : next;
            const float corr = __builtin_amdgcn_exp2f(mref - safe);
            l *= corr;
            mref = next;
#pragma unroll
            for (int t = 0; t < DTILES; ++t)
#pragma unroll
                for (int e = 0; e < 16; ++e) o[t][e] *= corr;
        }
        const float msafe = mref == GD_LP_NEG_INF ? 0.f : mref;
        gd_bf16x8 ph[4], pl[4];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const float pe = __builtin_amdgcn_exp2f(st[t][e] - msafe);
                l += pe;
                const gd_bf16 hi = (gd_bf16)pe;
                ph[2 * t + (e >> 3)][e & 7] = hi;
                pl[2 * t + (e >> 3)][e & 7] = (gd_bf16)(pe - (float)hi);
            }
        }
        /* rows of V behind the last key are copies of the last row (clamped loads): finite, and their weights are 0 */
#pragma unroll
        for (int ts = 0; ts < 4; ++ts) {
#pragma unroll
            for (int dt = 0; dt < DTILES; ++dt) {
                const uint32_t chunk = 4u * dt + 2u * tr_g1 + (tr_q >> 1);
                const uint32_t r_lo = 16u * ts + 4u * hh + tr_e; /* second read: + 8; both have r & 3 == tr_e */
                const uint32_t swz_lo = DTILES == 4 ? (tr_e << 2) : (((r_lo >> 1) & 1u) << 2);
                const uint32_t swz_hi = DTILES == 4 ? (tr_e << 2) : ((((r_lo + 8u) >> 1) & 1u) << 2);
                union { gd_short4 s[2]; gd_bf16x8 v; } u;
                u.s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)(
                    sV + (r_lo * VC + (chunk ^ swz_lo)) * 16u + (tr_q & 1u) * 8u));
                u.s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)(
                    sV + ((r_lo + 8u) * VC + (chunk ^ swz_hi)) * 16u + (tr_q & 1u) * 8u));
                o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(u.v, ph[ts], o[dt], 0, 0, 0);
                o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(u.v, pl[ts], o[dt], 0, 0, 0);
            }
        }
    }

    /* normalise and gate in registers, then through LDS so that rows leave in whole pieces */
    const gd_bf16 *gr = gate + qrow * ldg + head * m.vdim;
    gd_bf16x4 gv[DTILES][4]; /* requested together */
    if (((reinterpret_cast<uintptr_t>(gate) | (ldg * 2u)) & 7u) == 0u) {
#pragma unroll
        for (int dt = 0; dt < DTILES; ++dt)
#pragma unroll
            for (int a = 0; a < 4; ++a) {
                const uint32_t c = 32u * dt + 8u * a + 4u * hh;
                gv[dt][a] = *reinterpret_cast<const gd_bf16x4 *>(gr + (c < m.vdim ? c : 0u));
            }
    } else {
#pragma unroll
        for (int dt = 0; dt < DTILES; ++dt)
#pragma unroll
            for (int a = 0; a < 4; ++a)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const uint32_t c = 32u * dt + 8u * a + 4u * hh;
                    gv[dt][a][r] = gr[(c < m.vdim ? c : 0u) + (uint32_t)r];
                }
    }
    l += __shfl_xor(l, 32, 64);
    const float inv = l > 0.f ? 1.f / l : 0.f;
    constexpr uint32_t OS = 32u * DTILES + 8u; /* elements per row of the LDS block */
    __syncthreads(); /* all fragment reads of the last block are done */
    gd_bf16 *sO = reinterpret_cast<gd_bf16 *>(gd_lp_smem) + (size_t)wave * 32u * OS;
#pragma unroll
    for (int dt = 0; dt < DTILES; ++dt) {
#pragma unroll
        for (int a = 0; a < 4; ++a) {
            const uint32_t c = 32u * dt + 8u * a + 4u * hh;
            gd_bf16x4 hv;
#pragma unroll
            for (int r = 0; r < 4; ++r) hv[r] = (gd_bf16)(o[dt][4 * a + r] * inv * gd_sigmoid_fast((float)gv[dt][a][r]));
            *reinterpret_cast<gd_bf16x4 *>(sO + lq * OS + c) = hv;
        }
    }
    __syncthreads();
    for (uint32_t c = lane; c < 32u * v_chunks; c += 64u) {
        const uint32_t r = c / v_chunks, cc = c % v_chunks;
        const int ri = wi0 + (int)r;
        if (ri < n)
            *reinterpret_cast<gd_bf16x8 *>(out + ((size_t)(first + ri) * m.heads + head) * m.vdim + cc * 8u) =
                *reinterpret_cast<const gd_bf16x8 *>(sO + r * OS + cc * 8u);
    }
}

extern "C" int gd_hip_launch_latent_gather(hipStream_t stream, const void *cache, const int32_t *kv_cu, void *packed,
                                           uint32_t total, const gd_hip_latent_params *m, const gd_hip_seqs *q)
{
    gd_latent_gather_kernel<<<(total + 15u) / 16u, 256, 0, stream>>>((const gd_bf16 *)cache, kv_cu, (gd_bf16 *)packed, total, *m, *q);
    return (int)hipGetLastError();
}

template <int KSTEPS, int DTILES>
static int launch_prefill(hipStream_t stream, const void *q_rows, const void *kv, const void *packed, const float *angles,
                          const void *gate, uint32_t ldg, const int32_t *kv_cu, uint32_t kv_total, void *out,
                          const gd_hip_latent_params &m, const gd_hip_seqs &q, unsigned blocks)
{
    constexpr size_t stages = 2u * 64u * (2u * KSTEPS + 4u * DTILES) * 16u, rows = 128u * (32u * DTILES + 8u) * 2u;
    constexpr size_t lds = stages > rows ? stages : rows;
    static bool configured = false;
    if (!configured) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(gd_latent_prefill_kernel<KSTEPS, DTILES>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
        configured = true;
    }
    gd_latent_prefill_kernel<KSTEPS, DTILES><<<blocks, 256, lds, stream>>>(
        (const gd_bf16 *)q_rows, (const gd_bf16 *)kv, (const gd_bf16 *)packed, angles, (const gd_bf16 *)gate, ldg, kv_cu,
        kv_total, (gd_bf16 *)out, m, q);
    return (int)hipGetLastError();
}

/* kv [kv_total, heads * (dim + vdim)]: the expanded keys of all heads, then the values.  The caller has checked: BF16,
 * dim, rot_dim and vdim multiples of 8, dim + rot_dim <= 256, vdim <= 128, kv_rank % 8 == 0, 16-byte aligned operands */
extern "C" int gd_hip_launch_latent_prefill(hipStream_t stream, const void *q_rows, const void *kv, const void *packed,
                                            const float *angles, const void *gate, uint32_t ldg, const int32_t *kv_cu,
                                            uint32_t kv_total, void *out, const gd_hip_latent_params *m,
                                            const gd_hip_seqs *q)
{
    const uint64_t pairs = (uint64_t)(q->rows + 127u) / 128u + q->seqs, blocks = pairs * m->heads;
    const uint32_t qd = m->dim + m->rot_dim;
    if (blocks > 0x7fffffffull) return (int)hipErrorInvalidValue;
#define GD_GO(KS, DT) return launch_prefill<KS, DT>(stream, q_rows, kv, packed, angles, gate, ldg, kv_cu, kv_total, out, *m, *q, (unsigned)blocks)
    if (m->vdim <= 64u) {
        if (qd <= 64u) GD_GO(4, 2);
        if (qd <= 128u) GD_GO(8, 2);
        if (qd <= 192u) GD_GO(12, 2);
        GD_GO(16, 2);
    }
    if (qd <= 128u) GD_GO(8, 4);
    if (qd <= 192u) GD_GO(12, 4);
    GD_GO(16, 4);
#undef GD_GO
}
