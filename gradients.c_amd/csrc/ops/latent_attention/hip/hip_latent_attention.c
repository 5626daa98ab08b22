/* Host dispatch of gd_backend_latent_*. */
#include "../../_shared/packed_seqs_host.h"
#include "hip_latent_attention_types.h"

int gd_hip_launch_latent_prepare(hipStream_t stream, const void *proj, uint32_t ld, const float *q_norm,
                                 const float *kv_norm, const float *freq, float *angles, void *cq, void *cache,
                                 const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32, int aligned16);
int gd_hip_launch_latent_query(hipStream_t stream, const void *qv, const void *w_ukt, const float *angles, void *ql,
                               const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_latent_attend(hipStream_t stream, const void *ql, const void *cache, float *o_lat,
                                const gd_hip_latent_params *m, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_latent_value(hipStream_t stream, const float *o_lat, const void *w_uv, const void *gate, uint32_t ldg,
                               void *out, uint32_t rows, const gd_hip_latent_params *m, int is_f32);

int gd_hip_launch_latent_decode(hipStream_t stream, const void *qv, const void *w_ukt, const void *w_uv, const void *gate,
                                uint32_t ldg, const float *angles, const void *cache, void *ql, float *o_part, float *ml,
                                void *out, const gd_hip_latent_params *m, const gd_hip_seqs *q);
int gd_hip_launch_latent_gather(hipStream_t stream, const void *cache, const int32_t *kv_cu, void *packed, uint32_t total,
                                const gd_hip_latent_params *m, const gd_hip_seqs *q);
int gd_hip_launch_latent_prefill(hipStream_t stream, const void *q_rows, const void *kv, const void *packed,
                                 const float *angles, const void *gate, uint32_t ldg, const int32_t *kv_cu,
                                 uint32_t kv_total, void *out, const gd_hip_latent_params *m, const gd_hip_seqs *q);

#define GD_HIP_LATENT_RANK_MAX 2048u
#define GD_HIP_LATENT_PIECES_MAX 64u
/* new tokens per sequence up to which the absorbed form is taken */
#define GD_HIP_LATENT_FEW 32u

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
    m->piece_keys = m->pieces = 1u;
    return true;
}

/* the matrix-core forms */
static bool decode_sizes(const gd_hip_latent_params *m, uint32_t dtype)
{
    return dtype == GD_BACKEND_DTYPE_BF16 && (m->dim % 8u) == 0u && (m->rot_dim % 8u) == 0u && (m->kv_rank % 16u) == 0u &&
           m->pitch <= 1088u;
}

static bool prefill_sizes(const gd_hip_latent_params *m, uint32_t dtype)
{
    return dtype == GD_BACKEND_DTYPE_BF16 && (m->dim % 8u) == 0u && (m->rot_dim % 8u) == 0u && (m->vdim % 8u) == 0u &&
           (m->kv_rank % 8u) == 0u && m->dim + m->rot_dim <= 256u && m->vdim <= 128u;
}

/* keys per piece of the decode form: two workgroups (of up to 32 heads) per compute unit over the longest sequences, whole tiles of 64,
 * pieces of at least 128 keys */
static void cut(gd_hip_latent_params *m, uint32_t rows, uint32_t units)
{
    const uint64_t groups = (uint64_t)rows * ((m->pitch > 576u ? (m->heads + 15u) / 16u : (m->heads + 31u) / 32u));
    uint64_t want = (2u * (uint64_t)units + groups - 1u) / groups, len;
    if (want > GD_HIP_LATENT_PIECES_MAX) want = GD_HIP_LATENT_PIECES_MAX;
    len = ((m->tmax + want - 1u) / want + 63u) & ~63ull;
    if (len < 128u) len = 128u;
    m->piece_keys = (uint32_t)len;
    m->pieces = (uint32_t)((m->tmax + len - 1u) / len);
}

static bool cache_fits(const gd_backend_tensor_view *cache, gd_hip_latent_params *m)
{
    if (!gd_hip_view_ok(cache) || cache->rank != 3u || cache->shape[2] != (int64_t)m->pitch ||
        cache->shape[1] > 0x7fffffff || (cache->offset & 15u) != 0u)
        return false;
    m->tmax = (uint32_t)cache->shape[1];
    return true;
}

/* Layout of the work area, by form:
 *   row kernels   absorbed queries T [rows, heads, pitch], sums F32 [rows, heads, kv_rank]
 *   decode        absorbed queries, piece results F32 [rows, pieces, heads, kv_rank] and [rows, pieces, heads, 2]
 *   prefill       gathered cache rows [kv_total, pitch], expanded keys and values [kv_total, heads * (dim + vdim)] */
typedef struct work_layout {
    size_t ql, sums, ml, total;
} work_layout;

static work_layout absorbed_layout(const gd_hip_latent_params *m, uint32_t rows, uint32_t dtype)
{
    const size_t RH = (size_t)rows * m->heads, P = decode_sizes(m, dtype) ? m->pieces : 1u;
    work_layout w;
    w.ql = 0u;
    w.sums = pad256(RH * m->pitch * gd_hip_dtype_size(dtype));
    w.ml = w.sums + pad256(RH * P * m->kv_rank * sizeof(float));
    w.total = w.ml + pad256(RH * P * 2u * sizeof(float));
    return w;
}

static size_t expanded_bytes(const gd_hip_latent_params *m, uint64_t kv_total)
{
    return pad256((size_t)kv_total * m->pitch * 2u) + pad256((size_t)kv_total * m->heads * (m->dim + m->vdim) * 2u);
}

size_t gd_backend_latent_work_bytes(const gd_backend *backend, const gd_backend_latent_args *args, uint32_t rows,
                                    uint32_t max_new, uint32_t kv_total, uint32_t tmax, uint32_t dtype)
{
    const uint32_t units = backend != NULL ? (uint32_t)backend->compute_units : 256u;
    gd_hip_latent_params m;
    if (!params(args, &m) || rows == 0u || tmax == 0u) return 0u;
    m.tmax = tmax;
    if (prefill_sizes(&m, dtype) && kv_total != 0u && max_new > GD_HIP_LATENT_FEW) return expanded_bytes(&m, kv_total);
    cut(&m, rows, units);
    return absorbed_layout(&m, rows, dtype).total;
}

gd_status gd_backend_latent_prepare(gd_backend *backend, const gd_backend_matrix_view *proj,
                                    const gd_backend_tensor_view *q_norm, const gd_backend_tensor_view *kv_norm,
                                    const gd_backend_tensor_view *freq, const gd_backend_tensor_view *angles,
                                    const gd_backend_tensor_view *cq, const gd_backend_tensor_view *cache,
                                    const gd_backend_packed_seqs *seqs,
                                    const gd_backend_latent_args *args)
{
    gd_hip_latent_params m;
    gd_hip_seqs q;
    if (backend == NULL || !gd_hip_matrix_ok(proj) || !params(args, &m) || !cache_fits(cache, &m) ||
        (uint64_t)proj->cols < (uint64_t)m.q_rank + m.kv_rank + m.rot_dim || !gd_hip_f32_view(q_norm, m.q_rank) ||
        !gd_hip_f32_view(kv_norm, m.kv_rank) || !gd_hip_f32_view(freq, m.rot_dim / 2u) ||
        !gd_hip_f32_view(angles, (uint64_t)proj->rows * m.rot_dim) || !gd_hip_view_ok(cq) || cq->rank != 2u || cq->shape[0] != (int64_t)proj->rows || cq->shape[1] != (int64_t)m.q_rank ||
        !gd_hip_packed_seqs(seqs, proj->rows, (uint64_t)cache->shape[0], &q))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(proj->dtype) || cq->dtype != proj->dtype || cache->dtype != proj->dtype)
        return GD_ERR_UNSUPPORTED;
    return gd_hip_finish_op(backend, gd_hip_launch_latent_prepare(
        backend->stream, gd_hip_matrix_ptr(proj), (uint32_t)(proj->row_bytes / gd_hip_dtype_size(proj->dtype)),
        (const float *)gd_hip_view_ptr(q_norm), (const float *)gd_hip_view_ptr(kv_norm), (const float *)gd_hip_view_ptr(freq),
        (float *)gd_hip_view_ptr(angles), gd_hip_view_ptr(cq), gd_hip_view_ptr(cache), &m, &q, proj->dtype == GD_BACKEND_DTYPE_F32,
        ((proj->offset | proj->row_bytes | cq->offset | cache->offset) & 15u) == 0u));
}

static bool aligned16(const gd_backend_tensor_view *a, const gd_backend_tensor_view *b, const gd_backend_tensor_view *c)
{
    return ((a->offset | b->offset | c->offset) & 15u) == 0u;
}

gd_status gd_backend_latent_attend(gd_backend *backend, const gd_backend_tensor_view *qv,
                                   const gd_backend_tensor_view *w_ukt, const gd_backend_tensor_view *w_ukv,
                                   const gd_backend_matrix_view *gate, const gd_backend_tensor_view *angles,
                                   const gd_backend_tensor_view *cache, const gd_backend_tensor_view *work,
                                   const gd_backend_tensor_view *out, const gd_backend_packed_seqs *seqs,
                                   const gd_backend_latent_args *args)
{
    gd_hip_latent_params m;
    gd_hip_seqs q;
    gd_backend_tensor_view w_uv;
    const float *ang;
    uint64_t rows;
    size_t need;
    unsigned char *wp;
    uint32_t ldg, dtype;
    int e;
    if (backend == NULL || !params(args, &m) || !cache_fits(cache, &m) || !gd_hip_view_ok(qv) || qv->rank != 2u ||
        !gd_hip_view_ok(w_ukt) || w_ukt->rank != 2u || !gd_hip_view_ok(w_ukv) || w_ukv->rank != 2u ||
        !gd_hip_matrix_ok(gate) || !gd_hip_view_ok(out) || out->rank != 2u || !gd_hip_view_ok(work))
        return GD_ERR_INVALID_ARGUMENT;
    rows = (uint64_t)qv->shape[0];
    dtype = qv->dtype;
    if (qv->shape[1] != (int64_t)m.heads * (m.dim + m.rot_dim) || w_ukt->shape[0] != (int64_t)m.heads * m.kv_rank ||
        w_ukt->shape[1] != (int64_t)m.dim || w_ukv->shape[0] != (int64_t)m.heads * (m.dim + m.vdim) ||
        w_ukv->shape[1] != (int64_t)m.kv_rank || gate->rows != rows || gate->cols != m.heads * m.vdim ||
        out->shape[0] != (int64_t)rows || out->shape[1] != (int64_t)m.heads * m.vdim ||
        !gd_hip_f32_view(angles, rows * m.rot_dim) || !gd_hip_packed_seqs(seqs, rows, (uint64_t)cache->shape[0], &q) ||
        (seqs->kv_cu != NULL && !gd_hip_i32_vector(seqs->kv_cu, (uint64_t)q.seqs + 1u)))
        return GD_ERR_INVALID_ARGUMENT;
    if (!gd_hip_layer_dtype(dtype) || w_ukt->dtype != dtype || w_ukv->dtype != dtype || gate->dtype != dtype ||
        out->dtype != dtype || cache->dtype != dtype || work->dtype != GD_BACKEND_DTYPE_U8 ||
        m.kv_rank > GD_HIP_LATENT_RANK_MAX)
        return GD_ERR_UNSUPPORTED;
    need = gd_backend_latent_work_bytes(backend, args, (uint32_t)rows, q.max_new, seqs->kv_cu != NULL ? seqs->kv_total : 0u,
                                        m.tmax, dtype);
    if (work->count < need || (work->offset & 255u) != 0u) return GD_ERR_INVALID_ARGUMENT;
    wp = (unsigned char *)gd_hip_view_ptr(work);
    ang = (const float *)gd_hip_view_ptr(angles);
    ldg = (uint32_t)(gate->row_bytes / gd_hip_dtype_size(dtype));
    if (prefill_sizes(&m, dtype) && seqs->kv_cu != NULL && seqs->kv_total != 0u && q.max_new > GD_HIP_LATENT_FEW) {
        /* expanded: all latents the sequences hold through the stacked up-projections, then ordinary attention */
        unsigned char *kv = wp + pad256((size_t)seqs->kv_total * m.pitch * 2u);
        const int32_t *kv_cu = (const int32_t *)gd_hip_view_ptr(seqs->kv_cu);
        gd_backend_matrix_view xm, wm, ym;
        gd_status st;
        if (!aligned16(qv, cache, out) || (w_ukv->offset & 15u) != 0u) return GD_ERR_INVALID_ARGUMENT;
        e = gd_hip_launch_latent_gather(backend->stream, gd_hip_view_ptr(cache), kv_cu, wp, seqs->kv_total, &m, &q);
        if (e != 0) return gd_hip_finish_op(backend, e);
        xm.buffer = ym.buffer = work->buffer;
        xm.offset = work->offset;
        xm.rows = ym.rows = seqs->kv_total;
        xm.cols = m.kv_rank;
        xm.row_bytes = (size_t)m.pitch * 2u;
        xm.dtype = wm.dtype = ym.dtype = dtype;
        wm.buffer = w_ukv->buffer;
        wm.offset = w_ukv->offset;
        wm.rows = ym.cols = m.heads * (m.dim + m.vdim);
        wm.cols = m.kv_rank;
        wm.row_bytes = (size_t)m.kv_rank * 2u;
        ym.offset = work->offset + (size_t)(kv - wp);
        ym.row_bytes = (size_t)ym.cols * 2u;
        st = gd_backend_matmul_nt(backend, &xm, &wm, &ym);
        if (st != GD_OK) return st;
        return gd_hip_finish_op(backend, gd_hip_launch_latent_prefill(
            backend->stream, gd_hip_view_ptr(qv), kv, wp, ang, gd_hip_matrix_ptr(gate), ldg, kv_cu, seqs->kv_total,
            gd_hip_view_ptr(out), &m, &q));
    }
    {
        work_layout w;
        w_uv = *w_ukv;
        w_uv.offset += (size_t)m.heads * m.dim * m.kv_rank * gd_hip_dtype_size(dtype);
        cut(&m, (uint32_t)rows, (uint32_t)backend->compute_units);
        w = absorbed_layout(&m, (uint32_t)rows, dtype);
        if (decode_sizes(&m, dtype) && rows <= 65535u && aligned16(qv, w_ukt, &w_uv))
            return gd_hip_finish_op(backend, gd_hip_launch_latent_decode(
                backend->stream, gd_hip_view_ptr(qv), gd_hip_view_ptr(w_ukt), gd_hip_view_ptr(&w_uv),
                gd_hip_matrix_ptr(gate), ldg, ang, gd_hip_view_ptr(cache), wp + w.ql, (float *)(wp + w.sums),
                (float *)(wp + w.ml), gd_hip_view_ptr(out), &m, &q));
        e = gd_hip_launch_latent_query(backend->stream, gd_hip_view_ptr(qv), gd_hip_view_ptr(w_ukt), ang, wp + w.ql, &m, &q,
                                       dtype == GD_BACKEND_DTYPE_F32);
        if (e == 0)
            e = gd_hip_launch_latent_attend(backend->stream, wp + w.ql, gd_hip_view_ptr(cache), (float *)(wp + w.sums), &m,
                                            &q, dtype == GD_BACKEND_DTYPE_F32);
        if (e == 0)
            e = gd_hip_launch_latent_value(backend->stream, (float *)(wp + w.sums), gd_hip_view_ptr(&w_uv),
                                           gd_hip_matrix_ptr(gate), ldg, gd_hip_view_ptr(out), (uint32_t)rows, &m,
                                           dtype == GD_BACKEND_DTYPE_F32);
        return gd_hip_finish_op(backend, e);
    }
}
