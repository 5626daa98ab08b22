#ifndef GD_HIP_GROUPED_ATTENTION_TYPES_H
#define GD_HIP_GROUPED_ATTENTION_TYPES_H
#include <stdint.h>

#include "../../_shared/packed_seqs.h"

typedef struct gd_hip_grouped_params {
    uint32_t heads, kv_heads, per, dim, vdim, half; /* per: query heads of a key/value head; half: rotation pairs of a head */
    uint32_t chunk;                                 /* 0: every earlier position is seen */
    uint32_t places;                                /* rows of a slot and head in the caches */
    uint32_t ld;                                    /* distance of the rows of proj, elements */
    uint32_t k_col, v_col, g_col;                   /* first column of the keys, values and gates */
    uint32_t piece_keys, pieces;                    /* decode form */
    float scale, rot_mult;
} gd_hip_grouped_params;

#ifdef __HIPCC__
/* first position that a row at position pos sees, and the place of a position in the caches */
__device__ __forceinline__ int32_t gd_grouped_first(const gd_hip_grouped_params &m, int32_t pos)
{
    return m.chunk != 0u ? pos - pos % (int32_t)m.chunk : 0;
}

/* sine and cosine of pos * freq, times rot_mult.  What the product loses to rounding (for large angles more than the
 * functions do) is put back to first order. */
__device__ __forceinline__ void gd_grouped_angle(const gd_hip_grouped_params &m, int32_t pos, float freq, float *s, float *c)
{
    const float at = (float)pos, angle = at * freq, rest = fmaf(at, freq, -angle);
    float sn, cs;
    sincosf(angle, &sn, &cs);
    *s = fmaf(cs, rest, sn) * m.rot_mult;
    *c = fmaf(-sn, rest, cs) * m.rot_mult;
}
#endif
#endif
