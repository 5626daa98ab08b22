/* Host dispatch of gd_backend_ssm_scan and gd_backend_gated_group_norm. */
#include "../../_shared/packed_seqs_host.h"
#include "hip_ssm_scan_types.h"

int gd_hip_launch_ssm_scan(hipStream_t stream, const void *xbc, const void *dt_raw, const float *dt_bias,
                           const float *a_log, const float *d_skip, float *states, void *y, const gd_hip_ssm_params *m,
                           const gd_hip_ssm_conv *cv, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_ssm_scan_chunk(hipStream_t stream, const void *xbc, const void *dt_raw, const float *dt_bias,
                                 const float *a_log, const float *d_skip, float *states, void *y,
                                 const gd_hip_ssm_params *m, const gd_hip_seqs *q);
int gd_hip_launch_gated_group_norm(hipStream_t stream, const void *y, const void *z, uint32_t ldz, const float *w,
                                   void *out, uint32_t rows, uint32_t inner, uint32_t groups, float eps, int is_f32,
                                   int aligned16);

/* new rows of a sequence from which the chunked matrix-core form is taken */
#define GD_HIP_SSM_CHUNK_FROM 17u

/* checks shared by the two entry points; rows: packed rows of the inputs */
static gd_status ssm_params(const gd_backend_matrix_view *dt, const gd_backend_tensor_view *dt_bias,
                            const gd_backend_tensor_view *a_log, const gd_backend_tensor_view *d_skip,
                            const gd_backend_tensor_view *states, const gd_backend_tensor_view *y,
                            const gd_backend_packed_seqs *seqs, const gd_backend_ssm_args *args, uint64_t rows,
                            uint32_t dtype, gd_hip_ssm_params *m, gd_hip_seqs *q)
{
    uint64_t inner, cols;
    if (args == NULL || !gd_hip_matrix_ok(dt) || !gd_hip_view_ok(states) || states->rank != 4u || !gd_hip_view_ok(y) ||
        y->rank != 2u || args->heads == 0u || args->vdim == 0u || args->state == 0u || args->groups == 0u ||
        (args->heads % args->groups) != 0u)
        return GD_ERR_INVALID_ARGUMENT;
    inner = (uint64_t)args->heads * args->vdim;
    cols = inner + 2u * (uint64_t)args->groups * args->state;
    if (cols > 0x7fffffffu || dt->rows != rows || dt->cols != args->heads || y->shape[0] != (int64_t)rows ||
        y->shape[1] != (int64_t)inner || states->shape[1] != (int64_t)args->heads ||
        states->shape[2] != (int64_t)args->state || states->shape[3] != (int64_t)args->vdim ||
        !gd_hip_f32_view(states, states->count) || !gd_hip_f32_view(dt_bias, args->heads) ||
        !gd_hip_f32_view(a_log, args->heads) || !gd_hip_f32_view(d_skip, args->heads) ||
        !gd_hip_packed_seqs(seqs, rows, (uint64_t)states->shape[0], q) || args->heads > 65535u)
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(dtype) || dt->dtype != dtype || y->dtype != dtype || args->state > 512u)
        return GD_ERR_UNSUPPORTED;
    m->heads = args->heads;
    m->vdim = args->vdim;
    m->state = args->state;
    m->groups = args->groups;
    m->ld_xbc = (uint32_t)cols;
    m->ld_dt = (uint32_t)(dt->row_bytes / gd_hip_dtype_size(dtype));
    return GD_OK;
}

gd_status gd_backend_ssm_scan(gd_backend *backend, const gd_backend_tensor_view *xbc, const gd_backend_matrix_view *dt,
                              const gd_backend_tensor_view *dt_bias, const gd_backend_tensor_view *a_log,
                              const gd_backend_tensor_view *d_skip, const gd_backend_tensor_view *states,
                              const gd_backend_tensor_view *y, const gd_backend_packed_seqs *seqs,
                              const gd_backend_ssm_args *args)
{
    gd_hip_ssm_params m;
    gd_hip_seqs q;
    gd_status st;
    if (backend == NULL || !gd_hip_view_ok(xbc) || xbc->rank != 2u) return GD_ERR_INVALID_ARGUMENT;
    st = ssm_params(dt, dt_bias, a_log, d_skip, states, y, seqs, args, (uint64_t)xbc->shape[0], xbc->dtype, &m, &q);
    if (st != GD_OK) return st;
    if (xbc->shape[1] != (int64_t)m.ld_xbc) return GD_ERR_INVALID_ARGUMENT;
    if (xbc->dtype == GD_BACKEND_DTYPE_BF16 && q.max_new >= GD_HIP_SSM_CHUNK_FROM && (m.state % 8u) == 0u &&
        m.state <= 256u && (m.vdim % 8u) == 0u && ((xbc->offset | y->offset) & 15u) == 0u)
        return gd_hip_finish_op(backend, gd_hip_launch_ssm_scan_chunk(
            backend->stream, gd_hip_view_ptr(xbc), gd_hip_matrix_ptr(dt), (const float *)gd_hip_view_ptr(dt_bias),
            (const float *)gd_hip_view_ptr(a_log), (const float *)gd_hip_view_ptr(d_skip), (float *)gd_hip_view_ptr(states),
            gd_hip_view_ptr(y), &m, &q));
    return gd_hip_finish_op(backend, gd_hip_launch_ssm_scan(
        backend->stream, gd_hip_view_ptr(xbc), gd_hip_matrix_ptr(dt), (const float *)gd_hip_view_ptr(dt_bias),
        (const float *)gd_hip_view_ptr(a_log), (const float *)gd_hip_view_ptr(d_skip), (float *)gd_hip_view_ptr(states),
        gd_hip_view_ptr(y), &m, NULL, &q, xbc->dtype == GD_BACKEND_DTYPE_F32));
}

gd_status gd_backend_conv_ssm_step(gd_backend *backend, const gd_backend_matrix_view *x, const gd_backend_tensor_view *taps,
                                   const gd_backend_tensor_view *bias, const gd_backend_tensor_view *ring,
                                   const gd_backend_matrix_view *dt, const gd_backend_tensor_view *dt_bias,
                                   const gd_backend_tensor_view *a_log, const gd_backend_tensor_view *d_skip,
                                   const gd_backend_tensor_view *states, const gd_backend_tensor_view *y,
                                   const gd_backend_packed_seqs *seqs, const gd_backend_ssm_args *args)
{
    gd_hip_ssm_params m;
    gd_hip_ssm_conv cv;
    gd_hip_seqs q;
    gd_status st;
    if (backend == NULL || !gd_hip_matrix_ok(x) || !gd_hip_view_ok(taps) || taps->rank != 2u || !gd_hip_view_ok(ring) ||
        ring->rank != 3u)
        return GD_ERR_INVALID_ARGUMENT;
    st = ssm_params(dt, dt_bias, a_log, d_skip, states, y, seqs, args, x->rows, x->dtype, &m, &q);
    if (st != GD_OK) return st;
    if (x->cols != m.ld_xbc || taps->shape[0] != (int64_t)x->cols || taps->shape[1] > 4096 ||
        !gd_hip_f32_view(taps, taps->count) || !gd_hip_f32_view(bias, x->cols) || ring->shape[0] != states->shape[0] ||
        ring->shape[1] != taps->shape[1] || ring->shape[2] != taps->shape[0] || q.max_new != 1u)
        return GD_ERR_INVALID_ARGUMENT;
    if (ring->dtype != x->dtype) return GD_ERR_UNSUPPORTED;
    m.ld_xbc = (uint32_t)(x->row_bytes / gd_hip_dtype_size(x->dtype));
    cv.taps = (const float *)gd_hip_view_ptr(taps);
    cv.bias = (const float *)gd_hip_view_ptr(bias);
    cv.ring = gd_hip_view_ptr(ring);
    cv.C = x->cols;
    cv.K = (uint32_t)taps->shape[1];
    return gd_hip_finish_op(backend, gd_hip_launch_ssm_scan(
        backend->stream, gd_hip_matrix_ptr(x), gd_hip_matrix_ptr(dt), (const float *)gd_hip_view_ptr(dt_bias),
        (const float *)gd_hip_view_ptr(a_log), (const float *)gd_hip_view_ptr(d_skip), (float *)gd_hip_view_ptr(states),
        gd_hip_view_ptr(y), &m, &cv, &q, x->dtype == GD_BACKEND_DTYPE_F32));
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
