/* Host dispatch of gd_backend_grouped_attend. */
#include "../../_shared/packed_seqs_host.h"
#include "hip_grouped_attention_types.h"

int gd_hip_launch_grouped_rotate(hipStream_t stream, void *proj, const float *freq, const gd_hip_grouped_params *m,
                                 const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_grouped_attend(hipStream_t stream, const void *proj, const void *k_cache, const void *v_cache, void *out,
                                 const gd_hip_grouped_params *m, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_grouped_store(hipStream_t stream, const void *proj, void *k_cache, void *v_cache,
                                const gd_hip_grouped_params *m, const gd_hip_seqs *q, int is_f32);

static bool params(const gd_backend_grouped_args *a, uint64_t places, gd_hip_grouped_params *m)
{
    if (a == NULL || a->heads == 0u || a->heads > 65535u || a->kv_heads == 0u || a->heads % a->kv_heads != 0u ||
        a->dim == 0u || a->dim > 4096u || a->vdim == 0u || a->vdim > 4096u || a->rot_dims > a->dim ||
        (a->rot_dims & 1u) != 0u || a->chunk > 0x7fffffffu || places == 0u || places > 0x7fffffffu)
        return false;
    m->heads = a->heads;
    m->kv_heads = a->kv_heads;
    m->per = a->heads / a->kv_heads;
    m->dim = a->dim;
    m->vdim = a->vdim;
    m->half = a->rot_dims / 2u;
    m->chunk = a->chunk;
    m->places = (uint32_t)places;
    m->ld = 0u;
    m->k_col = m->heads * m->dim;
    m->v_col = m->k_col + m->kv_heads * m->dim;
    m->g_col = m->v_col + m->kv_heads * m->vdim;
    m->piece_keys = m->pieces = 1u;
    m->scale = a->scale;
    m->rot_mult = a->rot_mult;
    return true;
}

size_t gd_backend_grouped_work_bytes(const gd_backend *backend, const gd_backend_grouped_args *args, uint32_t rows,
                                     uint32_t max_new, uint32_t cache_rows, uint32_t dtype)
{
    (void)backend;
    (void)args;
    (void)rows;
    (void)max_new;
    (void)cache_rows;
    (void)dtype;
    return 256u;
}

static bool cache_ok(const gd_backend_tensor_view *c, uint32_t kv_heads, uint32_t dim)
{
    return gd_hip_view_ok(c) && c->rank == 4u && c->shape[1] == (int64_t)kv_heads && c->shape[3] == (int64_t)dim &&
           (c->offset & 15u) == 0u;
}

gd_status gd_backend_grouped_attend(gd_backend *backend, const gd_backend_matrix_view *proj,
                                    const gd_backend_tensor_view *freq, const gd_backend_tensor_view *k_cache,
                                    const gd_backend_tensor_view *v_cache, const gd_backend_tensor_view *work,
                                    const gd_backend_tensor_view *out, const gd_backend_packed_seqs *seqs,
                                    const gd_backend_grouped_args *args)
{
    gd_hip_grouped_params m;
    gd_hip_seqs q;
    uint32_t dtype;
    int f32, e = 0;
    if (backend == NULL || args == NULL || !gd_hip_matrix_ok(proj) || !cache_ok(k_cache, args->kv_heads, args->dim) ||
        !cache_ok(v_cache, args->kv_heads, args->vdim) || k_cache->shape[0] != v_cache->shape[0] ||
        k_cache->shape[2] != v_cache->shape[2] || !params(args, (uint64_t)k_cache->shape[2], &m) ||
        proj->cols < m.g_col + m.heads || (m.half != 0u && !gd_hip_f32_view(freq, m.half)) || !gd_hip_view_ok(out) ||
        out->rank != 2u || out->shape[0] != (int64_t)proj->rows || out->shape[1] != (int64_t)m.heads * m.vdim ||
        !gd_hip_view_ok(work) || !gd_hip_packed_seqs(seqs, proj->rows, (uint64_t)k_cache->shape[0], &q))
        return GD_ERR_INVALID_ARGUMENT;
    dtype = proj->dtype;
    if (!gd_hip_layer_dtype(dtype) || k_cache->dtype != dtype || v_cache->dtype != dtype || out->dtype != dtype ||
        work->dtype != GD_BACKEND_DTYPE_U8)
        return GD_ERR_UNSUPPORTED;
    if (work->count < gd_backend_grouped_work_bytes(backend, args, proj->rows, q.max_new, m.places, dtype) ||
        (work->offset & 255u) != 0u)
        return GD_ERR_INVALID_ARGUMENT;
    f32 = dtype == GD_BACKEND_DTYPE_F32;
    m.ld = (uint32_t)(proj->row_bytes / gd_hip_dtype_size(dtype));
    if (m.half != 0u)
        e = gd_hip_launch_grouped_rotate(backend->stream, gd_hip_matrix_ptr(proj), (const float *)gd_hip_view_ptr(freq), &m, &q, f32);
    if (e == 0)
        e = gd_hip_launch_grouped_attend(backend->stream, gd_hip_matrix_ptr(proj), gd_hip_view_ptr(k_cache),
                                         gd_hip_view_ptr(v_cache), gd_hip_view_ptr(out), &m, &q, f32);
    if (e == 0)
        e = gd_hip_launch_grouped_store(backend->stream, gd_hip_matrix_ptr(proj), gd_hip_view_ptr(k_cache),
                                        gd_hip_view_ptr(v_cache), &m, &q, f32);
    return gd_hip_finish_op(backend, e);
}
