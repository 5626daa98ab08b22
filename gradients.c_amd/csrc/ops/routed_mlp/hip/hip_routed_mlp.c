/* Host dispatch of gd_backend_route_by_tables and gd_backend_routed_mlp. */
#include <string.h>

#include "../../_shared/packed_seqs_host.h"
#include "../../linear/hip/hip_linear_types.h"
#include "hip_routed_mlp_types.h"

int gd_hip_launch_route(hipStream_t stream, const gd_hip_route_jobs *jobs, uint32_t n_jobs, const int32_t *ids, uint32_t rows);
int gd_hip_launch_routed_project(hipStream_t stream, const void *x, const void *w, void *y, const int32_t *first,
                                 const int32_t *tiles, const gd_hip_routed_params *p, int is_f32);

int gd_hip_launch_routed_stream(hipStream_t stream, const void *x, const void *w, void *y, const int32_t *first,
                                const int32_t *tiles, const gd_hip_routed_params *p);
int gd_hip_launch_linear_tile_grouped_bf16(hipStream_t stream, const void *x, const void *w, void *y,
                                           const gd_hip_linear_params *p, const int32_t *first, const int32_t *tiles,
                                           uint32_t w_rows, uint32_t max_tiles, int big_tiles, int compute_units);

/* the kernels that walk the work list, by the rows of its tiles */
#define GD_ROUTED_STREAM_ROWS 16u /* few rows per expert, BF16 */
#define GD_ROUTED_ANY_ROWS 64u    /* any sizes and types */
#define GD_ROUTED_TILE_ROWS 128u  /* many rows per expert, BF16 */
#define GD_ROUTED_WIDE_ROWS 256u  /* very many */

static bool args_ok(const gd_backend_routed_args *a)
{
    return a != NULL && a->experts != 0u && a->experts <= GD_BACKEND_ROUTED_MAX_EXPERTS && a->top != 0u &&
           a->top <= a->experts && a->width != 0u && a->ff != 0u && a->width <= 0x7fffffffu / 2u && a->ff <= 0x7fffffffu / 4u;
}

static uint32_t tile_rows_of(const gd_backend_routed_args *a, uint32_t rows, uint32_t dtype)
{
    const uint64_t per_expert = (uint64_t)rows * a->top / a->experts;
    if (dtype != GD_BACKEND_DTYPE_BF16 || (a->width % 8u) != 0u || (a->ff % 8u) != 0u) return GD_ROUTED_ANY_ROWS;
    if (per_expert >= 768u) return GD_ROUTED_WIDE_ROWS;
    return per_expert >= 24u ? GD_ROUTED_TILE_ROWS : GD_ROUTED_STREAM_ROWS;
}

/* every expert with rows has at most one tile that is not full */
uint32_t gd_backend_route_tiles(const gd_backend_routed_args *args, uint32_t rows, uint32_t tile_rows)
{
    const uint64_t pairs = (uint64_t)rows * args->top;
    const uint64_t n = pairs / tile_rows + (pairs < args->experts ? pairs : args->experts);
    return n > 0x3fffffffu ? 0x3fffffffu : (uint32_t)(n < pairs ? n : pairs);
}

gd_status gd_backend_route_by_tables(gd_backend *backend, const gd_backend_route_job *jobs, uint32_t n_jobs,
                                     const gd_backend_tensor_view *ids, uint32_t dtype)
{
    uint32_t done, i;
    int e = 0;
    if (backend == NULL || (jobs == NULL && n_jobs != 0u) || !gd_hip_view_ok(ids) || ids->count > 0x7fffffffu ||
        !gd_hip_i32_vector(ids, ids->count) || !gd_hip_layer_dtype(dtype))
        return GD_ERR_INVALID_ARGUMENT;
    for (i = 0u; i < n_jobs; ++i) {
        const gd_backend_route_job *j = &jobs[i];
        const uint64_t pairs = args_ok(j->args) ? (uint64_t)ids->count * j->args->top : UINT64_MAX;
        if (pairs > 0x3fffffffu || !gd_hip_view_ok(j->table) || j->table->rank != 2u || j->table->dtype != GD_BACKEND_DTYPE_I32 ||
            j->table->shape[1] != (int64_t)j->args->top || j->table->shape[0] > 0x7fffffff || (j->table->offset & 3u) != 0u ||
            !gd_hip_i32_vector(j->place, pairs) || !gd_hip_i32_vector(j->first, (uint64_t)j->args->experts + 1u) ||
            !gd_hip_view_ok(j->tiles) || !gd_hip_i32_vector(j->tiles, j->tiles->count) ||
            j->tiles->count < 2u + 2u * (size_t)gd_backend_route_tiles(j->args, (uint32_t)ids->count, 1u))
            return GD_ERR_INVALID_ARGUMENT;
    }
    for (done = 0u; done < n_jobs && e == 0; done += i) {
        gd_hip_route_jobs batch;
        for (i = 0u; i < GD_HIP_ROUTE_JOBS && done + i < n_jobs; ++i) {
            const gd_backend_route_job *j = &jobs[done + i];
            batch.job[i].table = (const int32_t *)gd_hip_view_ptr(j->table);
            batch.job[i].place = (int32_t *)gd_hip_view_ptr(j->place);
            batch.job[i].first = (int32_t *)gd_hip_view_ptr(j->first);
            batch.job[i].tiles = (int32_t *)gd_hip_view_ptr(j->tiles);
            batch.job[i].vocab = (uint32_t)j->table->shape[0];
            batch.job[i].top = j->args->top;
            batch.job[i].experts = j->args->experts;
            batch.job[i].tile_rows = tile_rows_of(j->args, (uint32_t)ids->count, dtype);
        }
        e = gd_hip_launch_route(backend->stream, &batch, i, (const int32_t *)gd_hip_view_ptr(ids), (uint32_t)ids->count);
    }
    return gd_hip_finish_op(backend, e);
}

static bool packed_ok(const gd_backend_tensor_view *v, uint64_t packed, uint32_t cols)
{
    return gd_hip_view_ok(v) && v->rank == 2u && v->shape[0] >= (int64_t)(packed + GD_BACKEND_ROUTED_PAD) &&
           v->shape[1] == (int64_t)cols && (v->offset & 15u) == 0u;
}

static bool weight_ok(const gd_backend_tensor_view *v, uint64_t rows, uint32_t cols)
{
    return gd_hip_view_ok(v) && v->rank == 2u && v->shape[0] == (int64_t)rows && v->shape[1] == (int64_t)cols &&
           (v->offset & 15u) == 0u;
}

/* y [packed, n] = x [packed, k] times the experts' weights */
static int project(gd_backend *backend, const gd_backend_tensor_view *x, const gd_backend_tensor_view *w,
                   const gd_backend_tensor_view *y, const int32_t *first, const int32_t *tiles, const gd_hip_routed_params *p,
                   uint32_t dtype)
{
    const void *xp = gd_hip_view_ptr(x), *wp = gd_hip_view_ptr(w);
    void *yp = gd_hip_view_ptr(y);
    gd_hip_linear_params l;
    if (p->tile_rows == GD_ROUTED_ANY_ROWS)
        return gd_hip_launch_routed_project(backend->stream, xp, wp, yp, first, tiles, p, dtype == GD_BACKEND_DTYPE_F32);
    if (p->tile_rows == GD_ROUTED_STREAM_ROWS)
        return gd_hip_launch_routed_stream(backend->stream, xp, wp, yp, first, tiles, p);
    memset(&l, 0, sizeof(l));
    l.M = p->packed;
    l.N = l.ldy = p->n;
    l.K = l.ldx = l.ldw = p->k;
    l.w_is_nk = 1u;
    if (p->gated) {
        l.swiglu_cols = p->n;
        l.flags = GD_HIP_LINEAR_CLAMPED_GATE;
        l.gate_limit = p->gate_limit;
        l.gate_alpha = p->gate_alpha;
    }
    return gd_hip_launch_linear_tile_grouped_bf16(backend->stream, xp, wp, yp, &l, first, tiles, p->n * (p->gated ? 2u : 1u),
                                                  p->max_tiles, p->tile_rows == GD_ROUTED_WIDE_ROWS, backend->compute_units);
}

gd_status gd_backend_routed_mlp(gd_backend *backend, const gd_backend_tensor_view *rows,
                                const gd_backend_tensor_view *w_upgate, const gd_backend_tensor_view *w_down,
                                const gd_backend_tensor_view *act, const gd_backend_tensor_view *out,
                                const gd_backend_routes *routes, const gd_backend_routed_args *args)
{
    gd_hip_routed_params up, down;
    uint64_t packed;
    uint32_t dtype, tile_rows;
    const int32_t *first, *tiles;
    int e;
    if (backend == NULL || !args_ok(args) || routes == NULL || routes->rows == 0u || !gd_hip_view_ok(rows))
        return GD_ERR_INVALID_ARGUMENT;
    packed = (uint64_t)routes->rows * args->top;
    dtype = rows->dtype;
    if (packed > 0x3fffffffu || !packed_ok(rows, packed, args->width) || !packed_ok(act, packed, args->ff) ||
        !packed_ok(out, packed, args->width) || !weight_ok(w_upgate, 2u * (uint64_t)args->experts * args->ff, args->width) ||
        !weight_ok(w_down, (uint64_t)args->experts * args->width, args->ff) ||
        !gd_hip_i32_vector(routes->first, (uint64_t)args->experts + 1u) || !gd_hip_view_ok(routes->tiles) ||
        !gd_hip_i32_vector(routes->tiles, routes->tiles->count) ||
        routes->tiles->count < 2u + 2u * (size_t)gd_backend_route_tiles(args, routes->rows, 1u))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(dtype) || act->dtype != dtype || out->dtype != dtype || w_upgate->dtype != dtype ||
        w_down->dtype != dtype)
        return GD_ERR_UNSUPPORTED;
    tile_rows = tile_rows_of(args, routes->rows, dtype);
    first = (const int32_t *)gd_hip_view_ptr(routes->first);
    tiles = (const int32_t *)gd_hip_view_ptr(routes->tiles);
    up.n = args->ff;
    up.k = args->width;
    up.experts = args->experts;
    up.packed = (uint32_t)packed;
    up.max_tiles = gd_backend_route_tiles(args, routes->rows, tile_rows);
    up.tile_rows = tile_rows;
    up.gated = 1u;
    up.gate_limit = args->gate_limit;
    up.gate_alpha = args->gate_alpha;
    down = up;
    down.n = args->width;
    down.k = args->ff;
    down.gated = 0u;
    if (up.max_tiles > 65535u) return GD_ERR_UNSUPPORTED;
    e = project(backend, rows, w_upgate, act, first, tiles, &up, dtype);
    if (e == 0) e = project(backend, act, w_down, out, first, tiles, &down, dtype);
    return gd_hip_finish_op(backend, e);
}
