/* Host dispatch of gd_backend_latent_*. */
#include "../../_shared/packed_seqs_host.h"
#include "hip_latent_attention_types.h"

int gd_hip_launch_latent_prepare(hipStream_t stream, const void *proj, uint32_t ld, const float *q_norm,
                                 const float *kv_norm, const float *freq, void *cq, void *cache,
                                 const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_latent_query(hipStream_t stream, const void *qv, const void *w_uk, const float *freq, void *ql,
                               const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_latent_attend(hipStream_t stream, const void *ql, const void *cache, float *o_lat,
                                const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_latent_value(hipStream_t stream, const float *o_lat, const void *w_uv, const void *gate, uint32_t ldg,
                               void *out, uint32_t rows, const gd_hip_latent_params *m, int is_f32);

#define GD_HIP_LATENT_RANK_MAX 2048u

uint32_t gd_backend_latent_pitch(uint32_t kv_rank, uint32_t rot_dim) { return (kv_rank + rot_dim + 7u) & ~7u; }

static size_t pad256(size_t n) { return (n + 255u) & ~(size_t)255u; }

static bool params(const gd_backend_latent_args *a, gd_hip_latent_params *m)
{
    if (a == NULL || a->heads == 0u || a->heads > 65535u || a->dim == 0u || a->rot_dim == 0u || (a->rot_dim & 1u) != 0u ||
        a->vdim == 0u || a->q_rank == 0u || a->kv_rank == 0u || a->dim > 4096u || a->vdim > 4096u || a->rot_dim > 4096u ||
        !(a->eps >= 0.0f))
        return false;
    m->heads = a->heads;
    m->dim = a->dim;
    m->rot_dim = a->rot_dim;
    m->vdim = a->vdim;
    m->q_rank = a->q_rank;
    m->kv_rank = a->kv_rank;
    m->pitch = gd_backend_latent_pitch(a->kv_rank, a->rot_dim);
    m->tmax = 0u;
    m->scale = a->scale;
    m->eps = a->eps;
    return true;
}

static bool cache_fits(const gd_backend_tensor_view *cache, gd_hip_latent_params *m)
{
    if (!gd_hip_view_ok(cache) || cache->rank != 3u || cache->shape[2] != (int64_t)m->pitch ||
        cache->shape[1] > 0x7fffffff || (cache->offset & 15u) != 0u)
        return false;
    m->tmax = (uint32_t)cache->shape[1];
    return true;
}

size_t gd_backend_latent_work_bytes(const gd_backend *backend, const gd_backend_latent_args *args, uint32_t rows,
                                    uint32_t tmax, uint32_t dtype)
{
    gd_hip_latent_params m;
    (void)backend;
    (void)tmax;
    if (!params(args, &m)) return 0u;
    return pad256((size_t)rows * m.heads * m.pitch * gd_hip_dtype_size(dtype)) +
           pad256((size_t)rows * m.heads * m.kv_rank * sizeof(float));
}

gd_status gd_backend_latent_prepare(gd_backend *backend, const gd_backend_matrix_view *proj,
                                    const gd_backend_tensor_view *q_norm, const gd_backend_tensor_view *kv_norm,
                                    const gd_backend_tensor_view *freq, const gd_backend_tensor_view *cq,
                                    const gd_backend_tensor_view *cache, const gd_backend_packed_seqs *seqs,
                                    const gd_backend_latent_args *args)
{
    gd_hip_latent_params m;
    gd_hip_seqs q;
    if (backend == NULL || !gd_hip_matrix_ok(proj) || !params(args, &m) || !cache_fits(cache, &m) ||
        (uint64_t)proj->cols < (uint64_t)m.q_rank + m.kv_rank + m.rot_dim || !gd_hip_f32_view(q_norm, m.q_rank) ||
        !gd_hip_f32_view(kv_norm, m.kv_rank) || !gd_hip_f32_view(freq, m.rot_dim / 2u) || !gd_hip_view_ok(cq) ||
        cq->rank != 2u || cq->shape[0] != (int64_t)proj->rows || cq->shape[1] != (int64_t)m.q_rank ||
        !gd_hip_packed_seqs(seqs, proj->rows, (uint64_t)cache->shape[0], &q))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(proj->dtype) || cq->dtype != proj->dtype || cache->dtype != proj->dtype)
        return GD_ERR_UNSUPPORTED;
    return gd_hip_finish_op(backend, gd_hip_launch_latent_prepare(
        backend->stream, gd_hip_matrix_ptr(proj), (uint32_t)(proj->row_bytes / gd_hip_dtype_size(proj->dtype)),
        (const float *)gd_hip_view_ptr(q_norm), (const float *)gd_hip_view_ptr(kv_norm), (const float *)gd_hip_view_ptr(freq),
        gd_hip_view_ptr(cq), gd_hip_view_ptr(cache), &m, &q, proj->dtype == GD_BACKEND_DTYPE_F32));
}

gd_status gd_backend_latent_attend(gd_backend *backend, const gd_backend_tensor_view *qv,
                                   const gd_backend_tensor_view *w_uk, const gd_backend_tensor_view *w_uv,
                                   const gd_backend_matrix_view *gate, const gd_backend_tensor_view *freq,
                                   const gd_backend_tensor_view *cache, const gd_backend_tensor_view *work,
                                   const gd_backend_tensor_view *out, const gd_backend_packed_seqs *seqs,
                                   const gd_backend_latent_args *args)
{
    gd_hip_latent_params m;
    gd_hip_seqs q;
    uint64_t rows;
    size_t need;
    unsigned char *ql;
    float *o_lat;
    int f32, e;
    if (backend == NULL || !params(args, &m) || !cache_fits(cache, &m) || !gd_hip_view_ok(qv) || qv->rank != 2u ||
        !gd_hip_view_ok(w_uk) || w_uk->rank != 2u || !gd_hip_view_ok(w_uv) || w_uv->rank != 2u || !gd_hip_matrix_ok(gate) ||
        !gd_hip_view_ok(out) || out->rank != 2u || !gd_hip_view_ok(work) || !gd_hip_f32_view(freq, m.rot_dim / 2u))
        return GD_ERR_INVALID_ARGUMENT;
    rows = (uint64_t)qv->shape[0];
    if (qv->shape[1] != (int64_t)m.heads * (m.dim + m.rot_dim) || w_uk->shape[0] != (int64_t)m.heads * m.dim ||
        w_uk->shape[1] != (int64_t)m.kv_rank || w_uv->shape[0] != (int64_t)m.heads * m.vdim ||
        w_uv->shape[1] != (int64_t)m.kv_rank || gate->rows != rows || gate->cols != m.heads * m.vdim ||
        out->shape[0] != (int64_t)rows || out->shape[1] != (int64_t)m.heads * m.vdim ||
        !gd_hip_packed_seqs(seqs, rows, (uint64_t)cache->shape[0], &q))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(qv->dtype) || w_uk->dtype != qv->dtype || w_uv->dtype != qv->dtype ||
        gate->dtype != qv->dtype || out->dtype != qv->dtype || cache->dtype != qv->dtype ||
        work->dtype != GD_BACKEND_DTYPE_U8 || m.kv_rank > GD_HIP_LATENT_RANK_MAX)
        return GD_ERR_UNSUPPORTED;
    need = gd_backend_latent_work_bytes(backend, args, (uint32_t)rows, m.tmax, qv->dtype);
    if (work->count < need || (work->offset & 255u) != 0u) return GD_ERR_INVALID_ARGUMENT;
    f32 = qv->dtype == GD_BACKEND_DTYPE_F32;
    ql = (unsigned char *)gd_hip_view_ptr(work);
    o_lat = (float *)(ql + pad256((size_t)rows * m.heads * m.pitch * gd_hip_dtype_size(qv->dtype)));
    e = gd_hip_launch_latent_query(backend->stream, gd_hip_view_ptr(qv), gd_hip_view_ptr(w_uk),
                                   (const float *)gd_hip_view_ptr(freq), ql, &m, &q, f32);
    if (e == 0) e = gd_hip_launch_latent_attend(backend->stream, ql, gd_hip_view_ptr(cache), o_lat, &m, &q, f32);
    if (e == 0)
        e = gd_hip_launch_latent_value(backend->stream, o_lat, gd_hip_view_ptr(w_uv), gd_hip_matrix_ptr(gate),
                                       (uint32_t)(gate->row_bytes / gd_hip_dtype_size(gate->dtype)), gd_hip_view_ptr(out),
                                       (uint32_t)rows, &m, f32);
    return gd_hip_finish_op(backend, e);
}
