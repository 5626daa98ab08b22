/* Host dispatch of gd_backend_causal_conv_silu. */
#include "../../_shared/packed_seqs_host.h"

int gd_hip_launch_causal_conv_silu(hipStream_t stream, const void *u, uint32_t ldu, const float *w, const float *bias,
                                   void *ring, void *out, uint32_t C, uint32_t K, const gd_hip_seqs *q, int is_f32,
                                   int aligned16);

gd_status gd_backend_causal_conv_silu(gd_backend *backend, const gd_backend_matrix_view *x,
                                      const gd_backend_tensor_view *taps, const gd_backend_tensor_view *bias,
                                      const gd_backend_tensor_view *ring, const gd_backend_tensor_view *out,
                                      const gd_backend_packed_seqs *seqs)
{
    gd_hip_seqs q;
    if (backend == NULL || !gd_hip_matrix_ok(x) || !gd_hip_view_ok(taps) || taps->rank != 2u || !gd_hip_view_ok(ring) ||
        ring->rank != 3u || !gd_hip_view_ok(out) || out->rank != 2u || taps->shape[0] != (int64_t)x->cols ||
        taps->shape[1] > 4096 || !gd_hip_f32_view(taps, taps->count) || !gd_hip_f32_view(bias, x->cols) ||
        ring->shape[1] != taps->shape[1] || ring->shape[2] != taps->shape[0] || out->shape[0] != (int64_t)x->rows ||
        out->shape[1] != (int64_t)x->cols || !gd_hip_packed_seqs(seqs, x->rows, (uint64_t)ring->shape[0], &q) ||
        (x->cols + 255u) / 256u > 65535u)
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(x->dtype) || ring->dtype != x->dtype || out->dtype != x->dtype) return GD_ERR_UNSUPPORTED;
    return gd_hip_finish_op(backend, gd_hip_launch_causal_conv_silu(
        backend->stream, gd_hip_matrix_ptr(x), (uint32_t)(x->row_bytes / gd_hip_dtype_size(x->dtype)),
        (const float *)gd_hip_view_ptr(taps), (const float *)gd_hip_view_ptr(bias), gd_hip_view_ptr(ring),
        gd_hip_view_ptr(out), x->cols, (uint32_t)taps->shape[1], &q, x->dtype == GD_BACKEND_DTYPE_F32,
        ((x->offset | x->row_bytes | ring->offset | out->offset) & 15u) == 0u));
}
