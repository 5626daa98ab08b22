/* Host dispatch of gd_backend_residual_embed / _norm_add / _add_norm / _norm_rows. */
#include "../../_shared/packed_seqs_host.h"

int gd_hip_launch_residual_embed(hipStream_t stream, const void *table, const int32_t *ids, float *x, void *copy,
                                 uint32_t n, uint32_t vocab, uint32_t cols, float scale, int is_f32);
int gd_hip_launch_residual_norm_add(hipStream_t stream, const void *u, const float *w, float *x, void *copy,
                                    uint32_t rows, uint32_t cols, float eps, float mult, int is_f32, int aligned16);
int gd_hip_launch_residual_add_norm(hipStream_t stream, const void *u, void *in, const int32_t *in_place, uint32_t in_rows,
                                    uint32_t in_top, float in_weight, float *x, const float *w, void *out, void *to,
                                    const int32_t *to_place, uint32_t to_rows, uint32_t to_top, uint32_t rows,
                                    uint32_t cols, float eps, int is_f32, int aligned16);
int gd_hip_launch_residual_norm_rows(hipStream_t stream, const float *x, const int32_t *rows, uint32_t n_rows,
                                     const float *w, void *out, uint32_t n_out, uint32_t cols, float eps, int is_f32);

static bool residual_ok(const gd_backend_tensor_view *x)
{
    return gd_hip_view_ok(x) && x->rank == 2u && gd_hip_f32_view(x, x->count) && x->shape[0] <= 0x7fffffff &&
           x->shape[1] <= 0x7fffffff;
}

static bool same_shape(const gd_backend_tensor_view *a, const gd_backend_tensor_view *x)
{
    return gd_hip_view_ok(a) && a->rank == 2u && a->shape[0] == x->shape[0] && a->shape[1] == x->shape[1];
}

gd_status gd_backend_residual_embed(gd_backend *backend, const gd_backend_tensor_view *table,
                                    const gd_backend_tensor_view *ids, const gd_backend_tensor_view *residual,
                                    const gd_backend_tensor_view *copy, float scale)
{
    if (backend == NULL || !gd_hip_view_ok(table) || table->rank != 2u || !residual_ok(residual) ||
        (copy != NULL && !same_shape(copy, residual)))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(table->dtype) || (copy != NULL && copy->dtype != table->dtype)) return GD_ERR_UNSUPPORTED;
    if (table->shape[1] != residual->shape[1] || table->shape[0] > 0x7fffffff ||
        !gd_hip_i32_vector(ids, (uint64_t)residual->shape[0]))
        return GD_ERR_INVALID_ARGUMENT;
    return gd_hip_finish_op(backend, gd_hip_launch_residual_embed(
        backend->stream, gd_hip_view_ptr(table), (const int32_t *)gd_hip_view_ptr(ids), (float *)gd_hip_view_ptr(residual),
        copy != NULL ? gd_hip_view_ptr(copy) : NULL, (uint32_t)residual->shape[0], (uint32_t)table->shape[0],
        (uint32_t)table->shape[1], scale, table->dtype == GD_BACKEND_DTYPE_F32));
}

gd_status gd_backend_residual_norm_add(gd_backend *backend, const gd_backend_tensor_view *branch,
                                       const gd_backend_tensor_view *weight, const gd_backend_tensor_view *residual,
                                       const gd_backend_tensor_view *copy, float eps, float mult)
{
    if (backend == NULL || !residual_ok(residual) || !same_shape(branch, residual) ||
        !gd_hip_f32_view(weight, (uint64_t)residual->shape[1]) || (copy != NULL && !same_shape(copy, residual)) ||
        !(eps >= 0.0f))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(branch->dtype) || (copy != NULL && copy->dtype != branch->dtype)) return GD_ERR_UNSUPPORTED;
    return gd_hip_finish_op(backend, gd_hip_launch_residual_norm_add(
        backend->stream, gd_hip_view_ptr(branch), (const float *)gd_hip_view_ptr(weight), (float *)gd_hip_view_ptr(residual),
        copy != NULL ? gd_hip_view_ptr(copy) : NULL, (uint32_t)residual->shape[0], (uint32_t)residual->shape[1], eps, mult,
        branch->dtype == GD_BACKEND_DTYPE_F32, ((branch->offset | (copy != NULL ? copy->offset : 0u)) & 15u) == 0u));
}

static bool routed_ok(const gd_backend_routed_rows *r, const gd_backend_tensor_view *x, uint32_t dtype)
{
    return gd_hip_view_ok(r->rows) && r->rows->rank == 2u && r->rows->shape[1] == x->shape[1] && r->rows->dtype == dtype &&
           r->rows->shape[0] <= 0x7fffffff && r->top != 0u && (uint64_t)x->shape[0] * r->top <= 0x7fffffffu &&
           gd_hip_i32_vector(r->place, (uint64_t)x->shape[0] * r->top);
}

gd_status gd_backend_residual_add_norm(gd_backend *backend, const gd_backend_tensor_view *branch,
                                       const gd_backend_routed_rows *added, const gd_backend_tensor_view *residual,
                                       const gd_backend_tensor_view *weight, const gd_backend_tensor_view *out,
                                       const gd_backend_routed_rows *packed, float eps)
{
    uint32_t dtype;
    uint64_t offsets;
    if (backend == NULL || !residual_ok(residual) || (weight != NULL) != (out != NULL) || (packed != NULL && out == NULL) ||
        (branch == NULL && added == NULL && out == NULL) || (branch != NULL && !same_shape(branch, residual)) ||
        (out != NULL && (!same_shape(out, residual) || !gd_hip_f32_view(weight, (uint64_t)residual->shape[1]))) || !(eps >= 0.0f))
        return GD_ERR_INVALID_ARGUMENT;
    if (branch != NULL) dtype = branch->dtype;
    else if (out != NULL) dtype = out->dtype;
    else dtype = added->rows != NULL ? added->rows->dtype : 0u;
    if (!gd_hip_layer_dtype(dtype) || (out != NULL && out->dtype != dtype)) return GD_ERR_UNSUPPORTED;
    if ((added != NULL && !routed_ok(added, residual, dtype)) || (packed != NULL && !routed_ok(packed, residual, dtype)))
        return GD_ERR_INVALID_ARGUMENT;
    offsets = (branch != NULL ? branch->offset : 0u) | (out != NULL ? out->offset : 0u) |
              (added != NULL ? added->rows->offset : 0u) | (packed != NULL ? packed->rows->offset : 0u);
    return gd_hip_finish_op(backend, gd_hip_launch_residual_add_norm(
        backend->stream, branch != NULL ? gd_hip_view_ptr(branch) : NULL, added != NULL ? gd_hip_view_ptr(added->rows) : NULL,
        added != NULL ? (const int32_t *)gd_hip_view_ptr(added->place) : NULL,
        added != NULL ? (uint32_t)added->rows->shape[0] : 0u, added != NULL ? added->top : 0u,
        added != NULL ? added->weight : 0.0f, (float *)gd_hip_view_ptr(residual),
        weight != NULL ? (const float *)gd_hip_view_ptr(weight) : NULL, out != NULL ? gd_hip_view_ptr(out) : NULL,
        packed != NULL ? gd_hip_view_ptr(packed->rows) : NULL,
        packed != NULL ? (const int32_t *)gd_hip_view_ptr(packed->place) : NULL,
        packed != NULL ? (uint32_t)packed->rows->shape[0] : 0u, packed != NULL ? packed->top : 0u,
        (uint32_t)residual->shape[0], (uint32_t)residual->shape[1], eps, dtype == GD_BACKEND_DTYPE_F32, (offsets & 15u) == 0u));
}

gd_status gd_backend_residual_norm_rows(gd_backend *backend, const gd_backend_tensor_view *residual,
                                        const gd_backend_tensor_view *rows, const gd_backend_tensor_view *weight,
                                        const gd_backend_tensor_view *out, float eps)
{
    if (backend == NULL || !residual_ok(residual) || !gd_hip_view_ok(out) || out->rank != 2u ||
        out->shape[1] != residual->shape[1] || out->shape[0] > 0x7fffffff || !(eps >= 0.0f) ||
        !gd_hip_f32_view(weight, (uint64_t)residual->shape[1]) ||
        (rows != NULL ? !gd_hip_i32_vector(rows, (uint64_t)out->shape[0]) : out->shape[0] > residual->shape[0]))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(out->dtype)) return GD_ERR_UNSUPPORTED;
    return gd_hip_finish_op(backend, gd_hip_launch_residual_norm_rows(
        backend->stream, (const float *)gd_hip_view_ptr(residual), rows != NULL ? (const int32_t *)gd_hip_view_ptr(rows) : NULL,
        (uint32_t)residual->shape[0], (const float *)gd_hip_view_ptr(weight), gd_hip_view_ptr(out),
        (uint32_t)out->shape[0], (uint32_t)out->shape[1], eps, out->dtype == GD_BACKEND_DTYPE_F32));
}
