/* Host side of gd_backend_packed_seqs: checks and device pointers.  N = rows of the packed operands, slots = places of
 * the state tensor. */
#ifndef GD_PACKED_SEQS_HOST_H
#define GD_PACKED_SEQS_HOST_H
#include "../../backends/hip/backend_hip_internal.h"
#include "packed_seqs.h"

static inline bool gd_hip_i32_vector(const gd_backend_tensor_view *v, uint64_t n)
{
    return gd_hip_view_ok(v) && v->dtype == GD_BACKEND_DTYPE_I32 && v->count == (size_t)n && (v->offset & 3u) == 0u;
}

static inline bool gd_hip_f32_view(const gd_backend_tensor_view *v, uint64_t n)
{
    return gd_hip_view_ok(v) && v->dtype == GD_BACKEND_DTYPE_F32 && v->count == (size_t)n && (v->offset & 15u) == 0u;
}

/* element type of the stateful layers */
static inline bool gd_hip_layer_dtype(uint32_t dtype)
{
    return dtype == GD_BACKEND_DTYPE_BF16 || dtype == GD_BACKEND_DTYPE_F32;
}

static inline bool gd_hip_packed_seqs(const gd_backend_packed_seqs *s, uint64_t rows, uint64_t slots, gd_hip_seqs *out)
{
    uint64_t seqs;
    if (s == NULL || !gd_hip_view_ok(s->slot) || s->slot->rank != 1u || rows == 0u || rows > 0x7fffffffu || slots == 0u ||
        slots > 0x7fffffffu || s->max_new == 0u)
        return false;
    seqs = s->slot->count;
    if (seqs == 0u || seqs > 65535u || !gd_hip_i32_vector(s->slot, seqs) || !gd_hip_i32_vector(s->start, seqs) ||
        !gd_hip_i32_vector(s->cu, seqs + 1u) || !gd_hip_i32_vector(s->row_seq, rows) || rows < s->max_new)
        return false;
    out->row_seq = (const int32_t *)gd_hip_view_ptr(s->row_seq);
    out->cu = (const int32_t *)gd_hip_view_ptr(s->cu);
    out->slot = (const int32_t *)gd_hip_view_ptr(s->slot);
    out->start = (const int32_t *)gd_hip_view_ptr(s->start);
    out->rows = (uint32_t)rows;
    out->seqs = (uint32_t)seqs;
    out->max_new = s->max_new;
    out->slots = (uint32_t)slots;
    return true;
}
#endif
