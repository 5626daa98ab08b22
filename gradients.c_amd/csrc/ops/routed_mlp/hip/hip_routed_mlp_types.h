#ifndef GD_HIP_ROUTED_MLP_TYPES_H
#define GD_HIP_ROUTED_MLP_TYPES_H
#include <stdint.h>

/* one table of a routing launch; the work list `tiles` starts with the number of its tiles and an unused word, then
 * (expert, first packed row) per tile of tile_rows rows of one expert */
typedef struct gd_hip_route_job {
    const int32_t *table;
    int32_t *place, *first, *tiles;
    uint32_t vocab, top, experts, tile_rows;
} gd_hip_route_job;

#define GD_HIP_ROUTE_JOBS 32
typedef struct gd_hip_route_jobs {
    gd_hip_route_job job[GD_HIP_ROUTE_JOBS];
} gd_hip_route_jobs;

/* one of the two projections of the packed rows: y [packed, n] = x [packed, k] w[expert]^T, w [experts, rows_w, k] with
 * rows_w = n, or gated 2 n: n value rows, then n gate rows */
typedef struct gd_hip_routed_params {
    uint32_t n, k, experts, packed, max_tiles, tile_rows, gated;
    float gate_limit, gate_alpha;
} gd_hip_routed_params;

#endif
