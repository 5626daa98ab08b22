/*
 * Routed feed-forward (gfx950): the tables of a step and the projections for any sizes.
 *   route    one workgroup per table: packs the choices of the step's rows by expert and writes the work list
 *   project  64 x 64 output tiles of one expert, F32 arithmetic; the F32 path and the path of sizes outside the
 *            matrix-core kernels (routed_stream.hip, routed_tile.hip)
 */
#include "../../_shared/hip_device.h"
#include "hip_routed_mlp_types.h"

#define GD_ROUTE_THREADS 1024u
#define GD_ROUTE_MAX_EXPERTS 4096u
#define GD_ROUTE_BATCH 8u /* choices a thread looks up together */

/* exclusive sums of v over the workgroup's threads; total receives the sum */
__device__ __forceinline__ uint32_t gd_route_scan(uint32_t v, uint32_t *smem, uint32_t *total)
{
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6;
    uint32_t incl = v;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const uint32_t up = (uint32_t)__shfl_up((int)incl, off, 64);
        if ((int)lane >= off) incl += up;
    }
    __syncthreads();
    if (lane == 63u) smem[wave] = incl;
    __syncthreads();
    uint32_t before = 0u, all = 0u;
    for (uint32_t w = 0; w < GD_ROUTE_THREADS / 64u; ++w) {
        if (w < wave) before += smem[w];
        all += smem[w];
    }
    *total = all;
    return before + incl - v;
}

__global__ void __launch_bounds__(GD_ROUTE_THREADS)
gd_route_kernel(gd_hip_route_jobs jobs, const int32_t *__restrict__ ids, uint32_t rows)
{
    __shared__ uint32_t s_count[GD_ROUTE_MAX_EXPERTS], s_first[GD_ROUTE_MAX_EXPERTS], s_scan[GD_ROUTE_THREADS / 64u];
    const gd_hip_route_job j = jobs.job[blockIdx.x];
    const uint32_t pairs = rows * j.top, tid = threadIdx.x;
    for (uint32_t e = tid; e < j.experts; e += GD_ROUTE_THREADS) s_count[e] = 0u;
    __syncthreads();
    /* the experts of BATCH choices of this thread, p, p + threads, ..: all ids requested together, then all entries */
    auto experts_of = [&](uint32_t p, int32_t (&e)[GD_ROUTE_BATCH]) __attribute__((always_inline)) {
        int32_t id[GD_ROUTE_BATCH];
#pragma unroll
        for (uint32_t i = 0; i < GD_ROUTE_BATCH; ++i) {
            const uint32_t at = p + i * GD_ROUTE_THREADS;
            id[i] = at < pairs ? ids[at / j.top] : -1;
        }
#pragma unroll
        for (uint32_t i = 0; i < GD_ROUTE_BATCH; ++i) {
            const uint32_t at = p + i * GD_ROUTE_THREADS;
            e[i] = id[i] >= 0 && (uint32_t)id[i] < j.vocab ? j.table[(size_t)id[i] * j.top + at % j.top] : -1;
        }
#pragma unroll
        for (uint32_t i = 0; i < GD_ROUTE_BATCH; ++i) e[i] = (uint32_t)e[i] < j.experts ? e[i] : -1;
    };
    /* the choice's rank among those of its expert waits in place */
    for (uint32_t p = tid; p < pairs; p += GD_ROUTE_BATCH * GD_ROUTE_THREADS) {
        int32_t e[GD_ROUTE_BATCH];
        experts_of(p, e);
#pragma unroll
        for (uint32_t i = 0; i < GD_ROUTE_BATCH; ++i) {
            if (p + i * GD_ROUTE_THREADS < pairs)
                j.place[p + i * GD_ROUTE_THREADS] = e[i] >= 0 ? (int32_t)atomicAdd(&s_count[e[i]], 1u) : -1;
        }
    }
    __syncthreads();
    /* four neighbouring experts per thread */
    uint32_t n[4], tiles[4], sum = 0u, tile_sum = 0u, total, tile_total;
#pragma unroll
    for (uint32_t i = 0; i < 4u; ++i) {
        const uint32_t e = tid * 4u + i;
        n[i] = e < j.experts ? s_count[e] : 0u;
        tiles[i] = (n[i] + j.tile_rows - 1u) / j.tile_rows;
        sum += n[i];
        tile_sum += tiles[i];
    }
    uint32_t at = gd_route_scan(sum, s_scan, &total), tile_at = gd_route_scan(tile_sum, s_scan, &tile_total);
    if (tid == 0u) {
        j.tiles[0] = (int32_t)tile_total;
        j.first[j.experts] = (int32_t)total;
    }
#pragma unroll
    for (uint32_t i = 0; i < 4u; ++i) {
        const uint32_t e = tid * 4u + i;
        if (e >= j.experts) break;
        s_first[e] = at;
        j.first[e] = (int32_t)at;
        for (uint32_t t = 0; t < tiles[i]; ++t, ++tile_at) {
            j.tiles[2u + 2u * tile_at] = (int32_t)e;
            j.tiles[3u + 2u * tile_at] = (int32_t)(at + t * j.tile_rows);
        }
        at += n[i];
    }
    __syncthreads();
    for (uint32_t p = tid; p < pairs; p += GD_ROUTE_BATCH * GD_ROUTE_THREADS) {
        int32_t e[GD_ROUTE_BATCH], rank[GD_ROUTE_BATCH];
#pragma unroll
        for (uint32_t i = 0; i < GD_ROUTE_BATCH; ++i)
            rank[i] = p + i * GD_ROUTE_THREADS < pairs ? j.place[p + i * GD_ROUTE_THREADS] : -1;
        experts_of(p, e);
#pragma unroll
        for (uint32_t i = 0; i < GD_ROUTE_BATCH; ++i) {
            if (e[i] >= 0 && rank[i] >= 0) j.place[p + i * GD_ROUTE_THREADS] = rank[i] + (int32_t)s_first[e[i]];
        }
    }
}

#define GD_RR_TILE 64u
#define GD_RR_BK 16u

/* grid (ceil(n / 64), max_tiles); tile_rows = 64 */
template <typename T, bool GATED>
__global__ void __launch_bounds__(256)
gd_routed_project_kernel(const T *__restrict__ x, const T *__restrict__ w, T *__restrict__ y,
                         const int32_t *__restrict__ first, const int32_t *__restrict__ tiles, gd_hip_routed_params p)
{
    __shared__ float sx[GD_RR_BK][GD_RR_TILE + 4], sw[GATED ? 2 : 1][GD_RR_BK][GD_RR_TILE + 4];
    if (blockIdx.y >= (uint32_t)tiles[0]) return;
    const uint32_t e = (uint32_t)tiles[2u + 2u * blockIdx.y], m0 = (uint32_t)tiles[3u + 2u * blockIdx.y];
    const uint32_t m_end = (uint32_t)first[e + 1u], n0 = blockIdx.x * GD_RR_TILE;
    const T *we = w + (size_t)e * (GATED ? 2u : 1u) * p.n * p.k;
    const uint32_t tx = threadIdx.x & 15u, ty = threadIdx.x >> 4;
    float acc[GATED ? 2 : 1][4][4] = {};
    for (uint32_t k0 = 0; k0 < p.k; k0 += GD_RR_BK) {
        for (uint32_t i = threadIdx.x; i < GD_RR_TILE * GD_RR_BK; i += 256u) {
            const uint32_t r = i / GD_RR_BK, k = i % GD_RR_BK;
            const bool kok = k0 + k < p.k, nok = kok && n0 + r < p.n;
            sx[k][r] = kok && m0 + r < m_end ? (float)x[(size_t)(m0 + r) * p.k + k0 + k] : 0.f;
            sw[0][k][r] = nok ? (float)we[(size_t)(n0 + r) * p.k + k0 + k] : 0.f;
            if (GATED) sw[GATED ? 1 : 0][k][r] = nok ? (float)we[(size_t)(p.n + n0 + r) * p.k + k0 + k] : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (uint32_t k = 0; k < GD_RR_BK; ++k) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float a = sx[k][ty + 16u * i];
#pragma unroll
                for (int g = 0; g < (GATED ? 2 : 1); ++g)
#pragma unroll
                    for (int c = 0; c < 4; ++c) acc[g][i][c] = fmaf(a, sw[g][k][tx + 16u * c], acc[g][i][c]);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const uint32_t m = m0 + ty + 16u * i, n = n0 + tx + 16u * c;
            if (m >= m_end || n >= p.n) continue;
            float v = acc[0][i][c];
            if (GATED) {
                const float g = fminf(acc[GATED ? 1 : 0][i][c], p.gate_limit);
                v = g / (1.0f + expf(-p.gate_alpha * g)) * (fminf(fmaxf(v, -p.gate_limit), p.gate_limit) + 1.0f);
            }
            y[(size_t)m * p.n + n] = (T)v;
        }
    }
}

extern "C" int gd_hip_launch_route(hipStream_t stream, const gd_hip_route_jobs *jobs, uint32_t n_jobs, const int32_t *ids,
                                   uint32_t rows)
{
    gd_route_kernel<<<n_jobs, GD_ROUTE_THREADS, 0, stream>>>(*jobs, ids, rows);
    return (int)hipGetLastError();
}

extern "C" int gd_hip_launch_routed_project(hipStream_t stream, const void *x, const void *w, void *y, const int32_t *first,
                                            const int32_t *tiles, const gd_hip_routed_params *p, int is_f32)
{
    const dim3 grid((p->n + GD_RR_TILE - 1u) / GD_RR_TILE, p->max_tiles);
#define GD_GO(T, G) gd_routed_project_kernel<T, G><<<grid, 256, 0, stream>>>((const T *)x, (const T *)w, (T *)y, first, tiles, *p)
    if (is_f32) { if (p->gated) GD_GO(float, true); else GD_GO(float, false); }
    else { if (p->gated) GD_GO(gd_bf16, true); else GD_GO(gd_bf16, false); }
#undef GD_GO
    return (int)hipGetLastError();
}
