#ifndef GD_HIP_SSM_SCAN_TYPES_H
#define GD_HIP_SSM_SCAN_TYPES_H
#include "../../_shared/packed_seqs.h"

typedef struct gd_hip_ssm_params {
    uint32_t heads, vdim, state, groups; /* H, P, N, G; head h reads group h / (H / G) */
    uint32_t ld_xbc, ld_dt;              /* row pitches in elements */
} gd_hip_ssm_params;

/* the convolution in front of a decode step's recurrence: taps F32 [C,K], bias F32 [C], ring [slots,K,C] */
typedef struct gd_hip_ssm_conv {
    const float *taps, *bias;
    void *ring;
    uint32_t C, K;
} gd_hip_ssm_conv;
#endif
