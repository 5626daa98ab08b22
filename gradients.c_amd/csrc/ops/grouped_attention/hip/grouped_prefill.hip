/*
 * Attention with grouped heads of prompts and portions on the matrix cores (gfx950, BF16), and the row kernels around it:
 *   rotate  queries and keys of the new rows turned to their positions, in place, 16-byte pieces
 *   attend  below
 *   store   rotated keys and values of the rows that later rows can see to their places in the caches
 *
 * The attention kernel follows gd_sdpa_varlen_mfma_kernel (ops/sdpa_varlen/hip/sdpa_varlen_mfma.hip): a workgroup of 4
 * wavefronts owns 128 consecutive new rows of one sequence and one head, keys advance in blocks of 64 positions through
 * two LDS stages filled by global -> LDS loads, both products transposed (S^T = K Q^T, O^T = V^T P^T) so that a query row
 * lives in one lane.  What is different here:
 *   - keys and values are read where the projection left them (positions of this call) or from the caches (positions of
 *     the current chunk in front of it); the choice is made per key row while a block is requested;
 *   - blocks start at the first position that the workgroup's first row sees, and a row is masked on both sides: by its
 *     own position and by the start of its chunk;
 *   - key and value sizes differ (dim padded to 16 * KSTEPS with zeros in the query, vdim to 32 * DTILES with columns
 *     that are not stored);
 *   - the weights enter the second product as two BF16 numbers (rounding and rest: 16 bits);
 *   - the head's output gate is applied in F32 before the one rounding;
 *   - workgroups that the dispatcher deals to one XCD take neighbouring heads, which share keys and values in its L2.
 */
#include "../../_shared/hip_device.h"
#include "hip_grouped_attention_types.h"

#define GD_GP_NEG_INF (-__builtin_inff())

/* 16 rows per workgroup; a thread turns the same 8 dimensions of every query and key head of its row */
__global__ void __launch_bounds__(256)
gd_grouped_rotate_vec_kernel(gd_bf16 *__restrict__ proj, const float *__restrict__ freq, gd_hip_grouped_params m,
                             gd_hip_seqs q, uint32_t lanes)
{
    const uint32_t per_block = 256u / lanes, sub = threadIdx.x % lanes, row = blockIdx.x * per_block + threadIdx.x / lanes;
    int32_t seq, pos, slot;
    if (threadIdx.x / lanes >= per_block || row >= q.rows || !gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const uint32_t heads = m.heads + m.kv_heads;
    for (uint32_t c = sub; c < m.half / 4u; c += lanes) {
        float cs[4], sn[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) gd_grouped_angle(m, pos, freq[4u * c + (uint32_t)i], &sn[i], &cs[i]);
        gd_bf16 *at = proj + (size_t)row * m.ld + c * 8u;
        for (uint32_t h0 = 0; h0 < heads; h0 += 4u) { /* the loads of four heads together */
            gd_bf16x8 v[4];
#pragma unroll
            for (uint32_t t = 0; t < 4u; ++t) v[t] = *reinterpret_cast<const gd_bf16x8 *>(at + (size_t)min(h0 + t, heads - 1u) * m.dim);
#pragma unroll
            for (uint32_t t = 0; t < 4u; ++t) {
                if (h0 + t >= heads) break;
                gd_bf16x8 o;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float a = (float)v[t][2 * i], b = (float)v[t][2 * i + 1];
                    o[2 * i] = (gd_bf16)(a * cs[i] - b * sn[i]);
                    o[2 * i + 1] = (gd_bf16)(b * cs[i] + a * sn[i]);
                }
                *reinterpret_cast<gd_bf16x8 *>(at + (size_t)(h0 + t) * m.dim) = o;
            }
        }
    }
}

/* 4 rows per workgroup, a wavefront each */
__global__ void __launch_bounds__(256)
gd_grouped_store_vec_kernel(const gd_bf16 *__restrict__ proj, gd_bf16 *__restrict__ k_cache, gd_bf16 *__restrict__ v_cache,
                            gd_hip_grouped_params m, gd_hip_seqs q)
{
    const uint32_t row = blockIdx.x * 4u + (threadIdx.x >> 6), lane = threadIdx.x & 63u;
    int32_t seq, pos, slot;
    if (row >= q.rows || !gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const int32_t last = q.start[seq] + (q.cu[seq + 1] - q.cu[seq]) - 1, first = gd_grouped_first(m, pos);
    if (gd_grouped_first(m, last) != first) return; /* of a chunk that is over */
    const uint32_t place = (uint32_t)(pos - first), kch = m.dim / 8u, vch = m.vdim / 8u;
    if (place >= m.places) return;
    const gd_bf16 *src = proj + (size_t)row * m.ld;
    const size_t slab = (size_t)slot * m.kv_heads;
    for (uint32_t c = lane; c < m.kv_heads * kch; c += 64u)
        *reinterpret_cast<gd_bf16x8 *>(k_cache + ((slab + c / kch) * m.places + place) * m.dim + (c % kch) * 8u) =
            *reinterpret_cast<const gd_bf16x8 *>(src + m.k_col + c * 8u);
    for (uint32_t c = lane; c < m.kv_heads * vch; c += 64u)
        *reinterpret_cast<gd_bf16x8 *>(v_cache + ((slab + c / vch) * m.places + place) * m.vdim + (c % vch) * 8u) =
            *reinterpret_cast<const gd_bf16x8 *>(src + m.v_col + c * 8u);
}

/* 16 bytes per lane from global memory straight into LDS (lane l's data lands at lds_address + 16*l); the kernel
 * places its own s_waitcnt vmcnt */
__device__ __forceinline__ void gd_gp_load_lds16(const gd_bf16 *lane_address, uint32_t lds_byte_address)
{
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off"
                 :
                 : "s"(lds_byte_address), "v"(lane_address)
                 : "memory");
}

template <int KSTEPS, int DTILES>
__global__ void __launch_bounds__(256, 2)
gd_grouped_prefill_kernel(const gd_bf16 *__restrict__ proj, const gd_bf16 *__restrict__ k_cache,
                          const gd_bf16 *__restrict__ v_cache, gd_bf16 *__restrict__ out, gd_hip_grouped_params m,
                          gd_hip_seqs sq)
{
    constexpr uint32_t BQ = 128u, BKEYS = 64u;
    constexpr uint32_t KC = 2u * KSTEPS, VC = 4u * DTILES; /* 16-byte chunks per key / value row in LDS */
    constexpr int KL = (int)(BKEYS * KC / 256u), VL = (int)(BKEYS * VC / 256u); /* wavefront loads per block */
    constexpr uint32_t STAGE = BKEYS * (KC + VC) * 16u;
    typedef short gd_short4 __attribute__((ext_vector_type(4)));
    extern __shared__ __align__(16) unsigned char gd_gp_smem[]; /* [2 stages][K block, V block] */
    const uint32_t tid = threadIdx.x, lane = tid & 63u;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const uint32_t lq = lane & 31u, hh = lane >> 5;
    uint32_t head = blockIdx.x % m.heads;
    const uint32_t pair = blockIdx.x / m.heads;
    /* workgroup ids are dealt round-robin to the 8 XCDs: runs of neighbouring heads stay on one */
    if ((m.heads & 7u) == 0u) head = (head & 7u) * (m.heads >> 3) + (head >> 3);
    const uint32_t g = head / m.per;

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
    const int start = __builtin_amdgcn_readfirstlane(sq.start[b]), slot = __builtin_amdgcn_readfirstlane(sq.slot[b]);
    if (start < 0 || slot < 0 || (uint32_t)slot >= sq.slots) return;
    first = __builtin_amdgcn_readfirstlane(first);
    const int n = __builtin_amdgcn_readfirstlane(end) - first, n_kv = start + n;
    const int i0 = (int)((pair - seen) * BQ);
    const int kend = min(n_kv, start + min(i0 + (int)BQ, n)); /* one behind the position of the block's last row */
    const int base = gd_grouped_first(m, start);              /* position of place 0 of the caches */
    const int jb0 = gd_grouped_first(m, start + i0);          /* the first position the block's first row sees */
    const int wi0 = i0 + (int)wave * 32, i = wi0 + (int)lq;
    const size_t qrow = (size_t)(first + min(i, n - 1));
    if (jb0 < start && start - base > (int)m.places) return; /* (positions the caches cannot hold) */

    gd_bf16x8 qf[KSTEPS];
    {
        const gd_bf16 *qp = proj + qrow * m.ld + (size_t)head * m.dim;
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ++ks) {
            const uint32_t e0 = 16u * ks + 8u * hh;
            qf[ks] = *reinterpret_cast<const gd_bf16x8 *>(qp + (e0 < m.dim ? e0 : 0u)); /* rows behind the end: the last */
        }
#pragma unroll
        for (int ks = 0; ks < KSTEPS; ++ks) {
            if (16u * ks + 8u * hh >= m.dim) qf[ks] = (gd_bf16x8)(gd_bf16)0.f;
        }
    }
    const float gate = (float)proj[qrow * m.ld + m.g_col + head];

    /* staging: load t of this wavefront fills LDS chunks (wave * KL + t) * 64 + lane of the K block (V likewise); chunk
     * c of key r lies at the place the swizzle names.  Bases are those of position 0: position p of this call is packed
     * row first + p - start, position p in front of it cache row p - base */
    const uint32_t k_chunks = m.dim / 8u, v_chunks = m.vdim / 8u;
    const uint32_t lds_base = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) unsigned char *)gd_gp_smem;
    const size_t slab = ((size_t)slot * m.kv_heads + g) * m.places;
    const gd_bf16 *k_new = proj + m.k_col + g * m.dim, *v_new = proj + m.v_col + g * m.vdim;
    const gd_bf16 *k_old = k_cache + slab * m.dim, *v_old = v_cache + slab * m.vdim;
    uint32_t k_row[KL], k_off[KL], v_row[VL], v_off[VL];
#pragma unroll
    for (int t = 0; t < KL; ++t) {
        const uint32_t x = (wave * (uint32_t)KL + (uint32_t)t) * 64u + lane, r = x / KC, at = x % KC;
        const uint32_t c = at ^ (KC % 16u == 0u ? (r & 15u) : ((r >> 1) & 7u));
        k_row[t] = r;
        k_off[t] = c < k_chunks ? c * 8u : 0u;
    }
#pragma unroll
    for (int t = 0; t < VL; ++t) {
        const uint32_t x = (wave * (uint32_t)VL + (uint32_t)t) * 64u + lane, r = x / VC, at = x % VC;
        const uint32_t c = at ^ (DTILES == 4 ? ((r & 3u) << 2) : (((r >> 1) & 1u) << 2));
        v_row[t] = r;
        v_off[t] = c < v_chunks ? c * 8u : 0u;
    }
    auto issue_block = [&](int jb, uint32_t stage) __attribute__((always_inline)) {
        const uint32_t at = lds_base + stage * STAGE;
        const bool all_new = jb >= start; /* uniform */
#pragma unroll
        for (int t = 0; t < KL; ++t) {
            const int j = min(jb + (int)k_row[t], n_kv - 1);
            const gd_bf16 *src = k_new + (size_t)(first + j - start) * m.ld;
            if (!all_new && j < start) src = k_old + (size_t)(j - base) * m.dim;
            gd_gp_load_lds16(src + k_off[t], at + (wave * (uint32_t)KL + (uint32_t)t) * 1024u);
        }
#pragma unroll
        for (int t = 0; t < VL; ++t) {
            const int j = min(jb + (int)v_row[t], n_kv - 1);
            const gd_bf16 *src = v_new + (size_t)(first + j - start) * m.ld;
            if (!all_new && j < start) src = v_old + (size_t)(j - base) * m.vdim;
            gd_gp_load_lds16(src + v_off[t], at + BKEYS * KC * 16u + (wave * (uint32_t)VL + (uint32_t)t) * 1024u);
        }
    };

    gd_float16 o[DTILES];
#pragma unroll
    for (int t = 0; t < DTILES; ++t)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[t][e] = 0.f;
    float mref = GD_GP_NEG_INF, l = 0.f;
    const float scale2 = m.scale * 1.4426950408889634f;
    /* visible positions of this lane's row, and of the wavefront's rows together */
    const int jmax = start + min(i, n - 1), jmin = gd_grouped_first(m, jmax);
    const int wave_first = start + wi0, wave_last = wi0 < n ? start + min(wi0 + 31, n - 1) : -1;
    const int wave_jmin = gd_grouped_first(m, min(wave_first, n_kv - 1)), wave_jfull = gd_grouped_first(m, max(wave_last, 0));
    const uint32_t tr_q = lane & 3u, tr_e = (lane >> 2) & 3u, tr_g1 = (lane >> 4) & 1u;

    issue_block(jb0, 0u);
    uint32_t it = 0u;
    for (int jb = jb0; jb < kend; jb += (int)BKEYS, ++it) {
        const uint32_t stage = it & 1u;
        __builtin_amdgcn_s_waitcnt(0x0F70); /* vmcnt(0): this wavefront's share of block jb is in LDS */
        __syncthreads();                    /* everyone's share is, and the other stage is no longer read */
        if (jb + (int)BKEYS < kend) issue_block(jb + (int)BKEYS, stage ^ 1u);
        const unsigned char *sK = gd_gp_smem + (size_t)stage * STAGE;
        const unsigned char *sV = sK + BKEYS * KC * 16u;
        if (jb > wave_last || jb + (int)BKEYS <= wave_jmin) continue; /* no row of the wavefront sees the block */

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
        float mloc = GD_GP_NEG_INF;
        const bool full = jb + 63 <= wave_first && jb >= wave_jfull;
#pragma unroll
        for (int t = 0; t < 2; ++t) {
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const int j = jb + 32 * t + 8 * (e >> 2) + 4 * (int)hh + (e & 3);
                st[t][e] = full || (j <= jmax && j >= jmin) ? st[t][e] * scale2 : GD_GP_NEG_INF;
                mloc = fmaxf(mloc, st[t][e]);
            }
        }
        mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
        const bool moves = mloc > mref + 8.f || (mref == GD_GP_NEG_INF && mloc != GD_GP_NEG_INF);
        if (__builtin_amdgcn_ballot_w64(moves) != 0ull) {
            const float next = fmaxf(mref, mloc), safe = next == GD_GP_NEG_INF ? 0.f : next;
            const float corr = __builtin_amdgcn_exp2f(mref - safe);
            l *= corr;
            mref = next;
#pragma unroll
            for (int t = 0; t < DTILES; ++t)
#pragma unroll
                for (int e = 0; e < 16; ++e) o[t][e] *= corr;
        }
        const float msafe = mref == GD_GP_NEG_INF ? 0.f : mref;
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
    l += __shfl_xor(l, 32, 64);
    const float mult = l > 0.f ? gd_sigmoid_f32(gate) / l : 0.f;
    constexpr uint32_t OS = 32u * DTILES + 8u; /* elements per row of the LDS block */
    __syncthreads(); /* all fragment reads of the last block are done */
    gd_bf16 *sO = reinterpret_cast<gd_bf16 *>(gd_gp_smem) + (size_t)wave * 32u * OS;
#pragma unroll
    for (int dt = 0; dt < DTILES; ++dt) {
#pragma unroll
        for (int a = 0; a < 4; ++a) {
            gd_bf16x4 hv;
#pragma unroll
            for (int r = 0; r < 4; ++r) hv[r] = (gd_bf16)(o[dt][4 * a + r] * mult);
            *reinterpret_cast<gd_bf16x4 *>(sO + lq * OS + 32u * dt + 8u * a + 4u * hh) = hv;
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

template <int KSTEPS, int DTILES>
static int launch_prefill(hipStream_t stream, const gd_bf16 *proj, const gd_bf16 *k_cache, const gd_bf16 *v_cache, gd_bf16 *out,
                          const gd_hip_grouped_params &m, const gd_hip_seqs &q, unsigned blocks)
{
    constexpr size_t stages = 2u * 64u * (2u * KSTEPS + 4u * DTILES) * 16u, rows = 128u * (32u * DTILES + 8u) * 2u;
    constexpr size_t lds = stages > rows ? stages : rows;
    static bool configured = false;
    if (!configured) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(gd_grouped_prefill_kernel<KSTEPS, DTILES>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
        configured = true;
    }
    gd_grouped_prefill_kernel<KSTEPS, DTILES><<<blocks, 256, lds, stream>>>(proj, k_cache, v_cache, out, m, q);
    return (int)hipGetLastError();
}

/* rotate, attend, store.  The caller has checked: BF16, dim and vdim multiples of 8, dim <= 256, vdim <= 128, rot_dims a
 * multiple of 8, 16-byte aligned rows everywhere */
extern "C" int gd_hip_launch_grouped_prefill(hipStream_t stream, void *proj, const float *freq, void *k_cache, void *v_cache,
                                             void *out, const gd_hip_grouped_params *mp, const gd_hip_seqs *qp)
{
    const gd_hip_grouped_params &m = *mp;
    const gd_hip_seqs &q = *qp;
    const uint64_t pairs = (uint64_t)(q.rows + 127u) / 128u + q.seqs, blocks = pairs * m.heads;
    int e = 0;
    if (blocks > 0x7fffffffull) return (int)hipErrorInvalidValue;
    if (m.half != 0u) {
        const uint32_t lanes = m.half / 4u < 64u ? m.half / 4u : 64u, per_block = 256u / lanes;
        gd_grouped_rotate_vec_kernel<<<(q.rows + per_block - 1u) / per_block, 256, 0, stream>>>((gd_bf16 *)proj, freq, m, q, lanes);
        e = (int)hipGetLastError();
        if (e != 0) return e;
    }
#define GD_GO(KS, DT) e = launch_prefill<KS, DT>(stream, (const gd_bf16 *)proj, (const gd_bf16 *)k_cache, (const gd_bf16 *)v_cache, (gd_bf16 *)out, m, q, (unsigned)blocks)
    if (m.vdim <= 64u) {
        if (m.dim <= 64u) GD_GO(4, 2);
        else if (m.dim <= 128u) GD_GO(8, 2);
        else if (m.dim <= 192u) GD_GO(12, 2);
        else GD_GO(16, 2);
    } else {
        if (m.dim <= 64u) GD_GO(4, 4);
        else if (m.dim <= 128u) GD_GO(8, 4);
        else if (m.dim <= 192u) GD_GO(12, 4);
        else GD_GO(16, 4);
    }
#undef GD_GO
    if (e != 0) return e;
    gd_grouped_store_vec_kernel<<<(q.rows + 3u) / 4u, 256, 0, stream>>>((const gd_bf16 *)proj, (gd_bf16 *)k_cache,
                                                                       (gd_bf16 *)v_cache, m, q);
    return (int)hipGetLastError();
}
