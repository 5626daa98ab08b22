/*
 * The packed new tokens of several sequences as the kernels with per-sequence state see them (device pointers of
 * gd_backend_packed_seqs).  Row r belongs to sequence row_seq[r], whose rows are cu[s] .. cu[s+1]; its position is
 * start[s] + r - cu[s]; its cache or state lies in slot[s].  A sequence with a negative start or a slot outside
 * [0, slots) is skipped.  The tables come from the caller, so every index is checked against its bound on the device.
 */
#ifndef GD_PACKED_SEQS_H
#define GD_PACKED_SEQS_H
#include <stdint.h>

typedef struct gd_hip_seqs {
    const int32_t *row_seq, *cu, *slot, *start;
    uint32_t rows, seqs, max_new, slots;
} gd_hip_seqs;

#ifdef __HIPCC__
/* sequence of row r and what belongs to it; false: skip the row */
__device__ __forceinline__ bool gd_seq_of_row(const gd_hip_seqs &q, uint32_t row, int32_t *seq, int32_t *pos,
                                              int32_t *slot)
{
    if (q.max_new == 1u && q.rows == q.seqs) { /* one row each, in order: one round trip to memory less */
        const int32_t st = q.start[row], sl = q.slot[row];
        *seq = (int32_t)row;
        *slot = sl;
        *pos = st;
        return st >= 0 && sl >= 0 && (uint32_t)sl < q.slots;
    }
    const int32_t s = q.row_seq[row];
    if (s < 0 || (uint32_t)s >= q.seqs) return false;
    const int32_t st = q.start[s], sl = q.slot[s], first = q.cu[s];
    if (st < 0 || sl < 0 || (uint32_t)sl >= q.slots || first < 0 || (uint32_t)first > row) return false;
    *seq = s;
    *slot = sl;
    *pos = st + (int32_t)(row - (uint32_t)first);
    return true;
}

/* rows [first, first + n) of sequence s, clamped to the packed rows; false: nothing to do */
__device__ __forceinline__ bool gd_seq_span(const gd_hip_seqs &q, uint32_t s, int32_t *first, int32_t *n, int32_t *start,
                                            int32_t *slot)
{
    const int32_t a = q.cu[s], b = q.cu[s + 1u];
    *start = q.start[s];
    *slot = q.slot[s];
    if (a < 0 || b <= a || (uint32_t)b > q.rows || *start < 0 || *slot < 0 || (uint32_t)*slot >= q.slots) return false;
    *first = a;
    *n = b - a;
    return true;
}
#endif
#endif
