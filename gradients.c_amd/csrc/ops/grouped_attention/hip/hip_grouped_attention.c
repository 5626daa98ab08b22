/* Host dispatch of gd_backend_grouped_attend. */
#include "../../_shared/packed_seqs_host.h"
#include "hip_grouped_attention_types.h"

int gd_hip_launch_grouped_rotate(hipStream_t stream, void *proj, const float *freq, const gd_hip_grouped_params *m,
                                 const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_grouped_attend(hipStream_t stream, const void *proj, const void *k_cache, const void *v_cache, void *out,
                                 const gd_hip_grouped_params *m, const gd_hip_seqs *q, int is_f32);
int gd_hip_launch_grouped_store(hipStream_t stream, const void *proj, void *k_cache, void *v_cache,
                                const gd_hip_grouped_params *m, const gd_hip_seqs *q, int is_f32);

int gd_hip_launch_grouped_decode(hipStream_t stream, const void *proj, const float *freq, void *k_cache, void *v_cache,
                                 void *out, float *o_part, float *ml, const gd_hip_grouped_params *m, const gd_hip_seqs *q);
int gd_hip_launch_grouped_prefill(hipStream_t stream, void *proj, const float *freq, void *k_cache, void *v_cache, void *out,
                                  const gd_hip_grouped_params *m, const gd_hip_seqs *q);

/* most pieces a row's keys are cut into: the merge kernel holds one per lane */
#define GD_HIP_GROUPED_PIECES_MAX 64u

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

/* the matrix-core forms: one new row per sequence, or any number */
static bool decode_sizes(const gd_hip_grouped_params *m, uint32_t dtype)
{
    return dtype == GD_BACKEND_DTYPE_BF16 && (m->dim % 8u) == 0u && (m->vdim % 8u) == 0u && (m->half % 4u) == 0u &&
           m->dim <= 128u && m->vdim <= 128u;
}

static bool prefill_sizes(const gd_hip_grouped_params *m, uint32_t dtype)
{
    return dtype == GD_BACKEND_DTYPE_BF16 && (m->dim % 8u) == 0u && (m->vdim % 8u) == 0u && (m->half % 4u) == 0u &&
           m->dim <= 256u && m->vdim <= 128u;
}

/* keys per piece of the decode form: a workgroup (of up to 16 heads) per compute unit over the most keys a row can see,
 * whole tiles of 32 for each of the four wavefronts */
static void cut(gd_hip_grouped_params *m, uint32_t rows, uint32_t units)
{
    const uint64_t keys = m->chunk != 0u && m->chunk < m->places ? m->chunk : m->places;
    const uint64_t groups = (uint64_t)rows * m->kv_heads * ((m->per + 15u) / 16u);
    uint64_t want = (units + groups - 1u) / groups, len;
    if (want > GD_HIP_GROUPED_PIECES_MAX) want = GD_HIP_GROUPED_PIECES_MAX;
    len = ((keys + want - 1u) / want + 127u) & ~127ull;
    m->piece_keys = (uint32_t)len;
    m->pieces = (uint32_t)((keys + len - 1u) / len);
}

static size_t pad256(size_t n) { return (n + 255u) & ~(size_t)255u; }

/* work area of the decode form: piece results F32 [rows, pieces, heads, vdim], then [rows, pieces, heads, 2] */
static size_t sums_bytes(const gd_hip_grouped_params *m, uint32_t rows)
{
    return pad256((size_t)rows * m->pieces * m->heads * m->vdim * sizeof(float));
}

size_t gd_backend_grouped_work_bytes(const gd_backend *backend, const gd_backend_grouped_args *args, uint32_t rows,
                                     uint32_t max_new, uint32_t cache_rows, uint32_t dtype)
{
    const uint32_t units = backend != NULL ? (uint32_t)backend->compute_units : 256u;
    gd_hip_grouped_params m;
    if (!params(args, cache_rows, &m) || rows == 0u) return 0u;
    if (max_new != 1u || !decode_sizes(&m, dtype)) return 256u;
    cut(&m, rows, units);
    /* nothing is stored with one piece; what few rows need with theirs is asked for all the same, so that a work area for
     * many rows serves fewer */
    if (m.pieces == 1u && rows > 2u * units) rows = 2u * units;
    return sums_bytes(&m, rows) + pad256((size_t)rows * m.pieces * m.heads * 2u * sizeof(float));
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
    const float *fp;
    void *pp, *kp, *vp, *op;
    bool aligned;
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
    fp = m.half != 0u ? (const float *)gd_hip_view_ptr(freq) : NULL;
    pp = gd_hip_matrix_ptr(proj);
    kp = gd_hip_view_ptr(k_cache);
    vp = gd_hip_view_ptr(v_cache);
    op = gd_hip_view_ptr(out);
    aligned = ((proj->offset | proj->row_bytes | out->offset) & 15u) == 0u;
    if (q.max_new == 1u && decode_sizes(&m, dtype) && aligned && q.rows <= 65535u) {
        unsigned char *wp = (unsigned char *)gd_hip_view_ptr(work);
        cut(&m, q.rows, (uint32_t)backend->compute_units);
        return gd_hip_finish_op(backend, gd_hip_launch_grouped_decode(backend->stream, pp, fp, kp, vp, op, (float *)wp,
                                                                      (float *)(wp + sums_bytes(&m, q.rows)), &m, &q));
    }
    if (prefill_sizes(&m, dtype) && aligned)
        return gd_hip_finish_op(backend, gd_hip_launch_grouped_prefill(backend->stream, pp, fp, kp, vp, op, &m, &q));
    if (m.half != 0u) e = gd_hip_launch_grouped_rotate(backend->stream, pp, fp, &m, &q, f32);
    if (e == 0) e = gd_hip_launch_grouped_attend(backend->stream, pp, kp, vp, op, &m, &q, f32);
    if (e == 0) e = gd_hip_launch_grouped_store(backend->stream, pp, kp, vp, &m, &q, f32);
    return gd_hip_finish_op(backend, e);
}
