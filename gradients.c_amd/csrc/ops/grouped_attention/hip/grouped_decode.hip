/*
 * Attention with grouped heads of one new token per sequence on the matrix cores (gfx950, BF16): rotation, cache update,
 * attention and output gate in one launch (and one more that merges pieces, where a sequence's keys are cut).
 *
 * A workgroup of 4 wavefronts takes up to 16 query heads of one key/value head over a piece of the keys: a cache row is
 * read from memory once for all of them.  HBM-bound on the cache rows.  The wavefronts share nothing inside the loop:
 * each takes every fourth tile of 32 keys through its own two LDS stages, filled by global -> LDS loads that it counts
 * itself, and keeps its own softmax; the four results meet in LDS behind the loop.  Both products are transposed, so
 * that a head lives in one lane column:
 *     S^T = K Q^T    16 keys per instruction, the query rows stay in registers
 *     O^T = V^T P^T  A by the transposing LDS read.  The weights a lane has computed (keys 4g + r and 16 + 4g + r of lane
 *                    group g) are its B operand as they are: the transposing read supplies the values of the same keys in
 *                    the same k slots
 * The new token's own key and value come from the projection: the wavefront whose tile holds them rotates the key, puts
 * both into the tile and, behind the loop, into the caches.
 * Scores, softmax and sums are F32.  The weights enter the second product as two BF16 numbers, their rounding and the
 * rest, so that they keep 16 bits; a row's maximum is a reference point that moves only when a tile raises it by more
 * than 8 binary orders.
 *
 * LDS rows hold a multiple of 8 chunks of 16 bytes (chunks behind the row repeat its first: keys meet zeros in the
 * query there, values are not stored).  Chunk c of row r sits at c ^ swizzle(r), which spreads 16 rows of one chunk, and
 * the four rows of a transposing read, over all banks.
 *
 * MFMA operand layout (v_mfma_f32_16x16x32_bf16): lane l supplies row / column l % 16 and the 8 consecutive k starting
 * at 8 * (l / 16); the result lane holds column l % 16, rows 4 * (l / 16) .. + 3.
 */
#include "../../_shared/hip_device.h"
#include "hip_grouped_attention_types.h"

#define GD_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0)
#define GD_GD_TILE 32u

/* 16 bytes per lane from global memory straight into LDS (lane l's data lands at lds_address + 16*l); the kernel
 * places its own s_waitcnt vmcnt */
__device__ __forceinline__ void gd_gd_load_lds16(const gd_bf16 *lane_address, uint32_t lds_byte_address)
{
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off"
                 :
                 : "s"(lds_byte_address), "v"(lane_address)
                 : "memory");
}

__device__ __forceinline__ uint32_t gd_gd_swizzle(uint32_t r)
{
    return ((r & 2u) << 1) | ((r & 4u) >> 1) | ((r & 8u) >> 3);
}

/* eight consecutive elements turned: four pairs with their cosines and sines */
__device__ __forceinline__ gd_bf16x8 gd_gd_turn(gd_bf16x8 v, gd_float4 c, gd_float4 s)
{
    gd_bf16x8 o;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float a = (float)v[2 * i], b = (float)v[2 * i + 1];
        o[2 * i] = (gd_bf16)(a * c[i] - b * s[i]);
        o[2 * i + 1] = (gd_bf16)(b * c[i] + a * s[i]);
    }
    return o;
}

/* STEPS: 32-wide steps that cover dim, even; VT: 16-wide tiles that cover vdim.  grid (pieces, kv_heads * groups of 16
 * query heads, rows).  o_part F32 [rows, pieces, heads, vdim], ml F32 [rows, pieces, heads, 2] (reference point in the
 * exp2 domain, sum); both unused with one piece, when out is written */
template <int STEPS, int VT>
__global__ void __launch_bounds__(256)
gd_grouped_decode_kernel(const gd_bf16 *__restrict__ proj, const float *__restrict__ freq, gd_bf16 *__restrict__ k_cache,
                         gd_bf16 *__restrict__ v_cache, gd_bf16 *__restrict__ out, float *__restrict__ o_part,
                         float *__restrict__ ml, gd_hip_grouped_params m, gd_hip_seqs q)
{
    constexpr uint32_t KC = 4u * STEPS, VC = 2u * VT, KROW = KC * 16u, VROW = VC * 16u; /* chunks and bytes of an LDS row */
    constexpr uint32_t K_BYTES = GD_GD_TILE * KROW, STAGE = K_BYTES + GD_GD_TILE * VROW;
    constexpr int KL = (int)(GD_GD_TILE * KC / 64u), VL = (int)(GD_GD_TILE * VC / 64u); /* wavefront loads of a tile */
    constexpr uint32_t OS = 16u * VT + 4u;                                              /* floats of a row of results */
    extern __shared__ __align__(16) unsigned char gd_gd_smem[]; /* [4 wavefronts][2 stages][keys, values] */
    __shared__ __align__(16) float s_cos[STEPS * 16], s_sin[STEPS * 16];
    __shared__ float s_ref[4][16], s_sum[4][16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, li = lane & 15u, lg = lane >> 4;
    const uint32_t wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const uint32_t row = blockIdx.z, groups = (m.per + 15u) / 16u, g = blockIdx.y / groups, hg = blockIdx.y % groups;
    const uint32_t h0 = g * m.per + 16u * hg, n_heads = min(m.per - 16u * hg, 16u);
    const uint32_t kch = m.dim / 8u, vch = m.vdim / 8u, half = m.half;
    int32_t seq, pos, slot;
    const bool live = gd_seq_of_row(q, row, &seq, &pos, &slot);

    /* requested together with the position: query rows, the new key and value, a frequency */
    const gd_bf16 *pr = proj + (size_t)row * m.ld;
    const gd_bf16x8 zero = (gd_bf16x8)(gd_bf16)0.f;
    gd_bf16x8 qf[STEPS];
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
        const uint32_t c = 4u * (uint32_t)s + lg;
        qf[s] = *reinterpret_cast<const gd_bf16x8 *>(pr + (size_t)(h0 + min(li, n_heads - 1u)) * m.dim + (c < kch ? c * 8u : 0u));
    }
    gd_bf16x8 k_new = *reinterpret_cast<const gd_bf16x8 *>(pr + m.k_col + g * m.dim + (lane < kch ? lane * 8u : 0u));
    gd_bf16x8 v_new = *reinterpret_cast<const gd_bf16x8 *>(pr + m.v_col + g * m.vdim + (lane < vch ? lane * 8u : 0u));
    float f = tid < half ? freq[tid] : 0.f;
    if (!live) return;
    const uint32_t keys = (uint32_t)(pos - gd_grouped_first(m, pos)) + 1u; /* the last of them is the row's own */
    const uint32_t k_begin = blockIdx.x * m.piece_keys;
    if (k_begin >= keys || keys > m.places) return;
    const uint32_t k_end = min(keys, k_begin + m.piece_keys), tiles = (k_end - k_begin + GD_GD_TILE - 1u) / GD_GD_TILE;
    const bool holds_new = k_end == keys;
#pragma unroll
    for (int s = 0; s < STEPS; ++s) asm volatile("" : "+v"(qf[s])); /* complete before the tiles are requested: the */
    asm volatile("" : "+v"(k_new), "+v"(v_new), "+v"(f));           /* compiler does not count the loads into LDS */

    const size_t slab = ((size_t)slot * m.kv_heads + g) * m.places;
    gd_bf16 *kc = k_cache + slab * m.dim, *vc = v_cache + slab * m.vdim;
    unsigned char *const own = gd_gd_smem + wave * (2u * STAGE);
    const uint32_t lds_base = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) unsigned char *)own;
    auto issue = [&](uint32_t k0, uint32_t stage) __attribute__((always_inline)) {
#pragma unroll
        for (int t = 0; t < KL; ++t) {
            const uint32_t i = (uint32_t)t * 64u + lane, r = i / KC, c = (i % KC) ^ gd_gd_swizzle(r);
            gd_gd_load_lds16(kc + (size_t)min(k0 + r, k_end - 1u) * m.dim + (c < kch ? c * 8u : 0u),
                             lds_base + stage * STAGE + (uint32_t)t * 1024u);
        }
#pragma unroll
        for (int t = 0; t < VL; ++t) {
            const uint32_t i = (uint32_t)t * 64u + lane, r = i / VC, c = (i % VC) ^ gd_gd_swizzle(r);
            gd_gd_load_lds16(vc + (size_t)min(k0 + r, k_end - 1u) * m.vdim + (c < vch ? c * 8u : 0u),
                             lds_base + stage * STAGE + K_BYTES + (uint32_t)t * 1024u);
        }
    };
    if (wave < tiles) issue(k_begin + wave * GD_GD_TILE, 0u);
    if (wave + 4u < tiles) issue(k_begin + (wave + 4u) * GD_GD_TILE, 1u);

    /* the angles of the position, while the first tiles are on their way */
    if (tid < STEPS * 16u) {
        float sn = 0.f, cs = 1.f;
        if (tid < half) gd_grouped_angle(m, pos, f, &sn, &cs);
        s_cos[tid] = cs;
        s_sin[tid] = sn;
    }
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
        const uint32_t c = 4u * (uint32_t)s + lg;
        qf[s] = c < kch ? gd_gd_turn(qf[s], *reinterpret_cast<const gd_float4 *>(s_cos + 4u * c),
                                     *reinterpret_cast<const gd_float4 *>(s_sin + 4u * c))
                        : zero;
        asm volatile("" : "+v"(qf[s]));
    }
    {
        const uint32_t c = min(lane, KC - 1u);
        k_new = gd_gd_turn(k_new, *reinterpret_cast<const gd_float4 *>(s_cos + 4u * c),
                           *reinterpret_cast<const gd_float4 *>(s_sin + 4u * c));
    }

    gd_float4 o[VT];
    float mref = -INFINITY, sum = 0.f; /* of head h0 + li; sum: the keys of this lane group */
#pragma unroll
    for (int t = 0; t < VT; ++t) o[t] = (gd_float4){0.f, 0.f, 0.f, 0.f};
    const float scale2 = m.scale * 1.4426950408889634f;
    const uint32_t k_swz = gd_gd_swizzle(li); /* rows li and 16 + li */
    const uint32_t tr_q = lane & 3u, tr_e = (lane >> 2) & 3u, v_row = 4u * lg + tr_e, v_swz = gd_gd_swizzle(v_row);
    typedef short gd_short4 __attribute__((ext_vector_type(4)));

    uint32_t stage = 0u;
    for (uint32_t t = wave; t < tiles; t += 4u, stage ^= 1u) {
        const uint32_t k0 = k_begin + t * GD_GD_TILE;
        unsigned char *const sk = own + stage * STAGE, *const sv = sk + K_BYTES;
        /* loads return in order: this tile is complete once only the next one's are outstanding */
        if (t + 4u < tiles) asm volatile("s_waitcnt vmcnt(%0)" ::"i"(KL + VL) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        if (holds_new && t + 1u == tiles) {
            const uint32_t r = keys - 1u - k0; /* the new key's row; behind it zeros: their weights are 0 */
            if (lane < kch) *reinterpret_cast<gd_bf16x8 *>(sk + r * KROW + (lane ^ gd_gd_swizzle(r)) * 16u) = k_new;
            if (lane < vch) *reinterpret_cast<gd_bf16x8 *>(sv + r * VROW + (lane ^ gd_gd_swizzle(r)) * 16u) = v_new;
            for (uint32_t i = (r + 1u) * VC + lane; i < GD_GD_TILE * VC; i += 64u) *reinterpret_cast<gd_bf16x8 *>(sv + i * 16u) = zero;
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        }
        gd_float4 sp[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int s = 0; s < STEPS; ++s) {
            const uint32_t c = 4u * (uint32_t)s + lg;
#pragma unroll
            for (int n = 0; n < 2; ++n) {
                const gd_bf16x8 a = *reinterpret_cast<const gd_bf16x8 *>(sk + (16u * (uint32_t)n + li) * KROW + (c ^ k_swz) * 16u);
                sp[n] = GD_MFMA(a, qf[s], sp[n]);
            }
        }
        float sc[8], mx = -INFINITY; /* keys 4 lg + r and 16 + 4 lg + r */
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const uint32_t key = k0 + 16u * (uint32_t)(e >> 2) + 4u * lg + (uint32_t)(e & 3);
            sc[e] = key < k_end ? sp[e >> 2][e & 3] * scale2 : -INFINITY;
            mx = fmaxf(mx, sc[e]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        /* the tile holds at least one live key, so mx is finite (or NaN) */
        if (__builtin_amdgcn_ballot_w64(!(mx <= mref + 8.f)) != 0ull) {
            const float next = fmaxf(mref, mx), keep = __builtin_amdgcn_exp2f(mref - next);
            mref = next;
            sum *= keep;
#pragma unroll
            for (int v = 0; v < VT; ++v)
#pragma unroll
                for (int r = 0; r < 4; ++r) o[v][r] *= keep;
        }
        gd_bf16x8 ph, pl;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float p = __builtin_amdgcn_exp2f(sc[e] - mref);
            sum += p;
            ph[e] = (gd_bf16)p;
            pl[e] = (gd_bf16)(p - (float)ph[e]);
        }
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            const uint32_t c = 2u * (uint32_t)v + (tr_q >> 1), w8 = (tr_q & 1u) * 8u;
            union { gd_short4 s[2]; gd_bf16x8 v; } u;
            u.s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)(
                sv + v_row * VROW + (c ^ v_swz) * 16u + w8));
            u.s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) gd_short4 *)(
                sv + (16u + v_row) * VROW + (c ^ v_swz) * 16u + w8));
            o[v] = GD_MFMA(u.v, ph, o[v]);
            o[v] = GD_MFMA(u.v, pl, o[v]);
        }
        if (t + 8u < tiles) {
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); /* the stage is no longer read */
            issue(k0 + 8u * GD_GD_TILE, stage);
        }
    }

    /* the four wavefronts' results, in the memory of the tiles */
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (lg == 0u) {
        s_ref[wave][li] = mref;
        s_sum[wave][li] = sum;
    }
    __syncthreads();
    float *so = reinterpret_cast<float *>(gd_gd_smem) + wave * (16u * OS);
#pragma unroll
    for (int v = 0; v < VT; ++v) *reinterpret_cast<gd_float4 *>(so + li * OS + 16u * (uint32_t)v + 4u * lg) = o[v];
    __syncthreads();
    const float *all = reinterpret_cast<const float *>(gd_gd_smem);
    const uint32_t quads = m.vdim / 4u;
    for (uint32_t i = tid; i < n_heads * quads; i += 256u) {
        const uint32_t h = i / quads, c = (i % quads) * 4u;
        const float top = fmaxf(fmaxf(s_ref[0][h], s_ref[1][h]), fmaxf(s_ref[2][h], s_ref[3][h]));
        gd_float4 a = {0.f, 0.f, 0.f, 0.f};
        float l = 0.f;
#pragma unroll
        for (uint32_t w = 0; w < 4u; ++w) {
            const float k = __builtin_amdgcn_exp2f(s_ref[w][h] - top); /* a wavefront without a tile: 0 */
            const gd_float4 v = *reinterpret_cast<const gd_float4 *>(all + w * (16u * OS) + h * OS + c);
            l = fmaf(k, s_sum[w][h], l);
#pragma unroll
            for (int e = 0; e < 4; ++e) a[e] = fmaf(k, v[e], a[e]);
        }
        if (m.pieces == 1u) {
            const float mult = gd_sigmoid_f32((float)pr[m.g_col + h0 + h]) / l;
            gd_bf16x4 b;
#pragma unroll
            for (int e = 0; e < 4; ++e) b[e] = (gd_bf16)(a[e] * mult);
            *reinterpret_cast<gd_bf16x4 *>(out + ((size_t)row * m.heads + h0 + h) * m.vdim + c) = b;
        } else {
            const size_t part = ((size_t)row * m.pieces + blockIdx.x) * m.heads + h0 + h;
            *reinterpret_cast<gd_float4 *>(o_part + part * m.vdim + c) = a;
            if (c == 0u) {
                ml[part * 2u] = top;
                ml[part * 2u + 1u] = l;
            }
        }
    }
    if (holds_new && hg == 0u && wave == 0u) {
        if (lane < kch) *reinterpret_cast<gd_bf16x8 *>(kc + (size_t)(keys - 1u) * m.dim + lane * 8u) = k_new;
        if (lane < vch) *reinterpret_cast<gd_bf16x8 *>(vc + (size_t)(keys - 1u) * m.vdim + lane * 8u) = v_new;
    }
}

/* grid (rows, ceil(heads / 4)); a wavefront per row and head; pieces <= 64, vdim % 4 == 0, vdim <= 256 */
__global__ void __launch_bounds__(256)
gd_grouped_merge_kernel(const float *__restrict__ o_part, const float *__restrict__ ml, const gd_bf16 *__restrict__ proj,
                        gd_bf16 *__restrict__ out, gd_hip_grouped_params m, gd_hip_seqs q)
{
    const uint32_t row = blockIdx.x, h = blockIdx.y * 4u + (threadIdx.x >> 6), lane = threadIdx.x & 63u;
    int32_t seq, pos, slot;
    if (h >= m.heads || !gd_seq_of_row(q, row, &seq, &pos, &slot)) return;
    const uint32_t keys = (uint32_t)(pos - gd_grouped_first(m, pos)) + 1u;
    if (keys > m.places) return;
    const uint32_t live = min((keys + m.piece_keys - 1u) / m.piece_keys, m.pieces);
    const size_t first = (size_t)row * m.pieces * m.heads + h;
    /* a lane per piece: exp2(reference - largest reference) / total */
    const float *v = ml + (first + (size_t)min(lane, live - 1u) * m.heads) * 2u;
    const float ref = lane < live ? v[0] : -INFINITY, part = v[1], gate = (float)proj[(size_t)row * m.ld + m.g_col + h];
    const float top = gd_wave_max(ref); /* by all lanes: an exchange inside a condition would lose some */
    const float w = lane < live ? __builtin_amdgcn_exp2f(ref - top) : 0.f;
    const float mine = w * (gd_sigmoid_f32(gate) / gd_wave_sum(w * part));
    gd_float4 a = {0.f, 0.f, 0.f, 0.f};
    const float *src = o_part + first * m.vdim + min(lane * 4u, m.vdim - 4u);
#pragma unroll 8
    for (uint32_t p = 0; p < live; ++p) {
        const gd_float4 t = *reinterpret_cast<const gd_float4 *>(src + (size_t)p * m.heads * m.vdim);
        const float k = __shfl(mine, (int)p, 64);
#pragma unroll
        for (int e = 0; e < 4; ++e) a[e] = fmaf(k, t[e], a[e]);
    }
    if (lane * 4u >= m.vdim) return;
    gd_bf16x4 b;
#pragma unroll
    for (int e = 0; e < 4; ++e) b[e] = (gd_bf16)a[e];
    *reinterpret_cast<gd_bf16x4 *>(out + ((size_t)row * m.heads + h) * m.vdim + lane * 4u) = b;
}

template <int STEPS, int VT>
static int launch_decode(hipStream_t stream, const gd_bf16 *proj, const float *freq, gd_bf16 *k_cache, gd_bf16 *v_cache,
                         gd_bf16 *out, float *o_part, float *ml, const gd_hip_grouped_params &m, const gd_hip_seqs &q)
{
    constexpr size_t stages = (size_t)4u * 2u * GD_GD_TILE * (4u * STEPS + 2u * VT) * 16u, rows = (size_t)4u * 16u * (16u * VT + 4u) * 4u;
    constexpr size_t lds = stages > rows ? stages : rows;
    static bool configured = false;
    if (!configured) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(gd_grouped_decode_kernel<STEPS, VT>),
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return (int)e;
        configured = true;
    }
    gd_grouped_decode_kernel<STEPS, VT><<<dim3(m.pieces, m.kv_heads * ((m.per + 15u) / 16u), q.rows), 256, lds, stream>>>(
        proj, freq, k_cache, v_cache, out, o_part, ml, m, q);
    return (int)hipGetLastError();
}

/* The caller has checked: BF16, one row per sequence, dim, vdim and rot_dims multiples of 8, both up to 128, pieces <=
 * 64, pieces of a multiple of 32 keys, rows <= 65535, 16-byte aligned rows everywhere. */
extern "C" int gd_hip_launch_grouped_decode(hipStream_t stream, const void *proj, const float *freq, void *k_cache,
                                            void *v_cache, void *out, float *o_part, float *ml,
                                            const gd_hip_grouped_params *mp, const gd_hip_seqs *qp)
{
    const gd_hip_grouped_params &m = *mp;
    const gd_hip_seqs &q = *qp;
    int e;
#define GD_GO(S, V) e = launch_decode<S, V>(stream, (const gd_bf16 *)proj, freq, (gd_bf16 *)k_cache, (gd_bf16 *)v_cache, (gd_bf16 *)out, o_part, ml, m, q)
    if (m.dim <= 64u) { if (m.vdim <= 64u) GD_GO(2, 4); else GD_GO(2, 8); }
    else { if (m.vdim <= 64u) GD_GO(4, 4); else GD_GO(4, 8); }
#undef GD_GO
    if (e != 0 || m.pieces == 1u) return e;
    gd_grouped_merge_kernel<<<dim3(q.rows, (m.heads + 3u) / 4u), 256, 0, stream>>>(o_part, ml, (const gd_bf16 *)proj,
                                                                                  (gd_bf16 *)out, m, q);
    return (int)hipGetLastError();
}
