/* Host dispatch of gd_backend_ssm_scan and gd_backend_gated_group_norm. */
#include "../../_shared/packed_seqs_host.h"
#include "hip_ssm_scan_types.h"

int gd_hip_launch_ssm_scan(hipStream_t stream, const void *xbc, const void *dt_raw, const float *dt_bias,
                           const float *a_log, const float *d_skip, float *states, void *y, const gd_hip_ssm_params *m,
                           const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_ssm_scan_chunk(hipStream_t stream, const void *xbc, const void *dt_raw, const float *dt_bias,
                                 const float *a_log, const float *d_skip, float *states, void *y,
                                 const gd_hip_ssm_params *m, const gd_hip_seqs *q);
int gd_hip_launch_gated_group_norm(hipStream_t stream, const void *y, const void *z, uint32_t ldz, const float *w,
                                   void *out, uint32_t rows, uint32_t inner, uint32_t groups, float eps, int is_f32,
                                   int aligned16);

/* new rows of a sequence from which the chunked matrix-core form is taken */
#define GD_HIP_SSM_CHUNK_FROM 17u

gd_status gd_backend_ssm_scan(gd_backend *backend, const gd_backend_tensor_view *xbc, const gd_backend_matrix_view *dt,
                              const gd_backend_tensor_view *dt_bias, const gd_backend_tensor_view *a_log,
                              const gd_backend_tensor_view *d_skip, const gd_backend_tensor_view *states,
                              const gd_backend_tensor_view *y, const gd_backend_packed_seqs *seqs,
                              const gd_backend_ssm_args *args)
{
    gd_hip_ssm_params m;
    gd_hip_seqs q;
    uint64_t inner, cols;
    if (backend == NULL || args == NULL || !gd_hip_view_ok(xbc) || xbc->rank != 2u || !gd_hip_matrix_ok(dt) ||
        !gd_hip_view_ok(states) || states->rank != 4u || !gd_hip_view_ok(y) || y->rank != 2u || args->heads == 0u ||
        args->vdim == 0u || args->state == 0u || args->groups == 0u || (args->heads % args->groups) != 0u)
        return GD_ERR_INVALID_ARGUMENT;
    inner = (uint64_t)args->heads * args->vdim;
    cols = inner + 2u * (uint64_t)args->groups * args->state;
    if (cols > 0x7fffffffu || xbc->shape[1] != (int64_t)cols || dt->rows != (uint64_t)xbc->shape[0] ||
        dt->cols != args->heads || y->shape[0] != xbc->shape[0] || y->shape[1] != (int64_t)inner ||
        states->shape[1] != (int64_t)args->heads || states->shape[2] != (int64_t)args->state ||
        states->shape[3] != (int64_t)args->vdim || !gd_hip_f32_view(states, states->count) ||
        !gd_hip_f32_view(dt_bias, args->heads) || !gd_hip_f32_view(a_log, args->heads) ||
        !gd_hip_f32_view(d_skip, args->heads) ||
        !gd_hip_packed_seqs(seqs, (uint64_t)xbc->shape[0], (uint64_t)states->shape[0], &q) || args->heads > 65535u)
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(xbc->dtype) || dt->dtype != xbc->dtype || y->dtype != xbc->dtype || args->state > 512u)
        return GD_ERR_UNSUPPORTED;
    m.heads = args->heads;
    m.vdim = args->vdim;
    m.state = args->state;
    m.groups = args->groups;
    m.ld_xbc = (uint32_t)cols;
    m.ld_dt = (uint32_t)(dt->row_bytes / gd_hip_dtype_size(dt->dtype));
    if (xbc->dtype == GD_BACKEND_DTYPE_BF16 && q.max_new >= GD_HIP_SSM_CHUNK_FROM && (m.state % 8u) == 0u &&
        m.state <= 256u && (m.vdim % 8u) == 0u && ((xbc->offset | y->offset) & 15u) == 0u)
        return gd_hip_finish_op(backend, gd_hip_launch_ssm_scan_chunk(
            backend->stream, gd_hip_view_ptr(xbc), gd_hip_matrix_ptr(dt), (const float *)gd_hip_view_ptr(dt_bias),
            (const float *)gd_hip_view_ptr(a_log), (const float *)gd_hip_view_ptr(d_skip), (float *)gd_hip_view_ptr(states),
            gd_hip_view_ptr(y), &m, &q));
    return gd_hip_finish_op(backend, gd_hip_launch_ssm_scan(
        backend->stream, gd_hip_view_ptr(xbc), gd_hip_matrix_ptr(dt), (const float *)gd_hip_view_ptr(dt_bias),
        (const float *)gd_hip_view_ptr(a_log), (const float *)gd_hip_view_ptr(d_skip), (float *)gd_hip_view_ptr(states),
        gd_hip_view_ptr(y), &m, &q, xbc->dtype == GD_BACKEND_DTYPE_F32));
}

gd_status gd_backend_gated_group_norm(gd_backend *backend, const gd_backend_tensor_view *y,
                                      const gd_backend_matrix_view *z, const gd_backend_tensor_view *weight,
                                      const gd_backend_tensor_view *out, uint32_t parts, float eps)
{
    if (backend == NULL || !gd_hip_view_ok(y) || y->rank != 2u || !gd_hip_matrix_ok(z) || !gd_hip_view_ok(out) ||
        out->rank != 2u || z->rows != (uint64_t)y->shape[0] || z->cols != (uint64_t)y->shape[1] ||
        out->shape[0] != y->shape[0] || out->shape[1] != y->shape[1] || !gd_hip_f32_view(weight, z->cols) ||
        parts == 0u || parts > 65535u || (z->cols % parts) != 0u || !(eps >= 0.0f))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(y->dtype) || z->dtype != y->dtype || out->dtype != y->dtype) return GD_ERR_UNSUPPORTED;
    return gd_hip_finish_op(backend, gd_hip_launch_gated_group_norm(
        backend->stream, gd_hip_view_ptr(y), gd_hip_matrix_ptr(z), (uint32_t)(z->row_bytes / gd_hip_dtype_size(z->dtype)),
        (const float *)gd_hip_view_ptr(weight), gd_hip_view_ptr(out), z->rows, z->cols, parts, eps,
        y->dtype == GD_BACKEND_DTYPE_F32, ((y->offset | z->offset | z->row_bytes | out->offset) & 15u) == 0u));
}
