#ifndef GD_HIP_SSM_SCAN_TYPES_H
#define GD_HIP_SSM_SCAN_TYPES_H
#include "../../_shared/packed_seqs.h"

typedef struct gd_hip_ssm_params {
    uint32_t heads, vdim, state, groups; /* H, P, N, G; head h reads group h / (H / G) */
    uint32_t ld_xbc, ld_dt;              /* row pitches in elements */
} gd_hip_ssm_params;
#endif
