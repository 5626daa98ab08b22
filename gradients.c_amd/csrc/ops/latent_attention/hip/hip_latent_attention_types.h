#ifndef GD_HIP_LATENT_ATTENTION_TYPES_H
#define GD_HIP_LATENT_ATTENTION_TYPES_H
#include "../../_shared/packed_seqs.h"

/* sizes of a latent attention layer; a cache row is [kv_rank latent values | rot_dim rotated key values | padding] */
typedef struct gd_hip_latent_params {
    uint32_t heads, dim, rot_dim, vdim, q_rank, kv_rank;
    uint32_t pitch; /* elements per cache row and per absorbed query row: kv_rank + rot_dim rounded up to 8 */
    uint32_t tmax;  /* cache rows per slot */
    float scale, eps;
    /* matrix-core decode form: keys per piece and pieces per row (piece results [rows, pieces, heads]) */
    uint32_t piece_keys, pieces;
} gd_hip_latent_params;
#endif
