/*
 * The decoder whose layers are listed in a configuration (layer_list.h): weights, caches and states, and one forward
 * over packed new tokens that serves prompts, portions of prompts and decode steps alike.
 *
 * Per layer, with an F32 residual stream x and its copy h in the projections' type:
 *   mixer   mamba2            in -> causal conv + silu -> recurrence -> gate, group norm -> out
 *           latent_attention  [dq | dkv | g] -> norms, rotation, cache append -> uq -> attention, output gate -> out
 *   x += m * norm1(mixer(h));  h = x
 *   feed-forward  gelu(gate) * up with biases -> down;  x += m * norm2(ff(h));  h = x
 * Projections that read the same input are one weight matrix.  What a sequence keeps: the convolution's last inputs and
 * the recurrent state (mamba2), the latent and the rotated key part of every token (latent_attention), each in the
 * place of its slot; positions decide what of it is read, so nothing is cleared when a slot is used again.
 */
#include <math.h>
#include <stdio.h>

#include "layer_list.h"

#define MAX_PIECES 3

typedef struct layer_weights {
    gd_tensor norm1, norm2;
    gd_tensor in, conv, conv_b, dt_bias, a_log, d_skip, gnorm; /* mamba2; in: also [dq | dkv | g] of latent attention */
    gd_tensor dq_norm, dkv_norm, uq, ukv, ukt, freq; /* latent attention; ukv: [uk | uv]; ukt: uk turned per head */
    gd_tensor out;
    gd_tensor upgate, upgate_b, down, down_b; /* feed-forward; upgate: [up | gate] */
    gd_tensor ring, states, cache;            /* per slot */
} layer_weights;

struct layer_list {
    layer_list_config c;
    gd_dtype type; /* of projections and activations */
    int32_t max_step_tokens;
    int32_t kv_rows; /* tokens whose keys and values a step may expand at once (latent attention) */
    gd_tensor embed, final_norm;
    layer_weights *layers;
    gd_tensor rows_dev, cu_dev; /* 0 .. batch-1 and 0 .. batch: the tables of a decode step over every slot */
};

static int64_t conv_channels(const layer_config *l)
{
    return (int64_t)l->ssm.heads * l->ssm.vdim + 2 * (int64_t)l->ssm.groups * l->ssm.state;
}
static int64_t inner_size(const layer_config *l) { return (int64_t)l->ssm.heads * l->ssm.vdim; }
static int64_t mixer_in(const layer_config *l)
{
    if (l->mixer == MIXER_MAMBA2) return inner_size(l) + conv_channels(l) + l->ssm.heads;
    return (int64_t)l->latent.q_rank + l->latent.kv_rank + l->latent.rot_dim + (int64_t)l->latent.heads * l->latent.vdim;
}
static int64_t mixer_out(const layer_config *l)
{
    return l->mixer == MIXER_MAMBA2 ? inner_size(l) : (int64_t)l->latent.heads * l->latent.vdim;
}
static int64_t query_size(const layer_config *l)
{
    return (int64_t)l->latent.heads * (l->latent.dim + l->latent.rot_dim);
}

/* ---- weights ------------------------------------------------------------------------------------- */

/* One weight of the decoder: where it goes, its type and shape, the tensors of the file that are stacked in it, and the
 * range of random weights. */
typedef struct weight {
    gd_tensor *dst;
    gd_dtype type;
    int64_t rows, cols; /* cols 0: a vector */
    const char *piece[MAX_PIECES];
    int64_t piece_rows[MAX_PIECES];
    float lo, hi;
} weight;

typedef gd_status (*weight_fn)(void *user, const weight *w, int32_t layer);

/* calls fn for every weight, the layers' in order (layer -1: the model's own); ll->layers NULL: destinations are NULL */
static gd_status each_weight(const layer_list_config *c, gd_dtype type, struct layer_list *ll, weight_fn fn, void *user)
{
    int32_t i;
#define AT(field) (ll != NULL ? &ll->field : NULL)
#define ONE(dst_, type_, rows_, cols_, name_, lo_, hi_)                                                         \
    do {                                                                                                        \
        const weight w_ = {dst_, type_, rows_, cols_, {name_, NULL, NULL}, {rows_, 0, 0}, lo_, hi_};            \
        TRY(fn(user, &w_, i));                                                                                  \
    } while (0)
    i = -1;
    ONE(AT(embed), type, c->vocab, c->width, "embed", -0.05f, 0.05f);
    ONE(AT(final_norm), GD_DTYPE_F32, c->width, 0, "final.norm", 1.0f, 1.0f);
    for (i = 0; i < c->n_layers; ++i) {
        const layer_config *l = &c->layers[i];
        const float wide = 1.7f / sqrtf((float)c->width); /* uniform range whose products keep unit variance */
        ONE(AT(layers[i].norm1), GD_DTYPE_F32, c->width, 0, "norm1", 1.0f, 1.0f);
        if (l->mixer == MIXER_MAMBA2) {
            const int64_t ch = conv_channels(l), H = l->ssm.heads;
            ONE(AT(layers[i].in), type, mixer_in(l), c->width, "mix.in", -wide, wide);
            ONE(AT(layers[i].conv), GD_DTYPE_F32, ch, l->taps, "mix.conv", -0.5f, 0.5f);
            ONE(AT(layers[i].conv_b), GD_DTYPE_F32, ch, 0, "mix.conv.b", -0.1f, 0.1f);
            ONE(AT(layers[i].dt_bias), GD_DTYPE_F32, H, 0, "mix.dt_bias", -4.6f, -2.3f);
            ONE(AT(layers[i].a_log), GD_DTYPE_F32, H, 0, "mix.A_log", 0.0f, 2.7f);
            ONE(AT(layers[i].d_skip), GD_DTYPE_F32, H, 0, "mix.D", 0.5f, 1.5f);
            ONE(AT(layers[i].gnorm), GD_DTYPE_F32, inner_size(l), 0, "mix.norm", 1.0f, 1.0f);
        } else {
            const gd_backend_latent_args *a = &l->latent;
            const int64_t H = a->heads;
            const float qr = 1.7f / sqrtf((float)a->q_rank), kr = 1.7f / sqrtf((float)a->kv_rank);
            const weight in = {AT(layers[i].in), type, mixer_in(l), c->width, {"mix.dq", "mix.dkv", "mix.g"},
                               {a->q_rank, (int64_t)a->kv_rank + a->rot_dim, H * a->vdim}, -wide, wide};
            const weight ukv = {AT(layers[i].ukv), type, H * ((int64_t)a->dim + a->vdim), a->kv_rank,
                                {"mix.uk", "mix.uv", NULL}, {H * a->dim, H * a->vdim, 0}, -kr, kr};
            TRY(fn(user, &in, i));
            ONE(AT(layers[i].dq_norm), GD_DTYPE_F32, a->q_rank, 0, "mix.dq.norm", 1.0f, 1.0f);
            ONE(AT(layers[i].dkv_norm), GD_DTYPE_F32, a->kv_rank, 0, "mix.dkv.norm", 1.0f, 1.0f);
            ONE(AT(layers[i].uq), type, query_size(l), a->q_rank, "mix.uq", -qr, qr);
            TRY(fn(user, &ukv, i));
            ONE(AT(layers[i].ukt), type, H * a->kv_rank, a->dim, NULL, 0.0f, 0.0f); /* from ukv */
            ONE(AT(layers[i].freq), GD_DTYPE_F32, a->rot_dim / 2, 0, NULL, 0.0f, 0.0f); /* computed, not stored */
        }
        ONE(AT(layers[i].out), type, c->width, mixer_out(l), "mix.o", -wide, wide);
        if (l->ff > 0) {
            const weight ug = {AT(layers[i].upgate), type, 2 * (int64_t)l->ff, c->width, {"mlp.up", "mlp.gate", NULL},
                               {l->ff, l->ff, 0}, -wide, wide};
            const weight ugb = {AT(layers[i].upgate_b), type, 2 * (int64_t)l->ff, 0, {"mlp.up.b", "mlp.gate.b", NULL},
                                {l->ff, l->ff, 0}, -0.1f, 0.1f};
            const float fr = 1.7f / sqrtf((float)l->ff);
            TRY(fn(user, &ug, i));
            TRY(fn(user, &ugb, i));
            ONE(AT(layers[i].down), type, c->width, l->ff, "mlp.down", -fr, fr);
            ONE(AT(layers[i].down_b), type, c->width, 0, "mlp.down.b", -0.1f, 0.1f);
            ONE(AT(layers[i].norm2), GD_DTYPE_F32, c->width, 0, "norm2", 1.0f, 1.0f);
        }
    }
#undef ONE
#undef AT
    return GD_OK;
}

static int64_t weight_count(const weight *w) { return w->rows * (w->cols > 0 ? w->cols : 1); }

static gd_status add_bytes(void *user, const weight *w, int32_t layer)
{
    (void)layer;
    *(size_t *)user += gd_pad256((size_t)weight_count(w) * gd_dtype_size(w->type));
    return GD_OK;
}

typedef struct weight_load {
    gd_context *ctx;
    const layer_list_config *c;
    gd_safetensors *file;
    uint64_t seed;
    unsigned char *raw, *turned; /* host staging of the largest weight */
    gd_tensor *ukv;              /* the layer's, already filled */
} weight_load;

static gd_status allocate_weight(void *user, const weight *w, int32_t layer)
{
    const weight_load *wl = (const weight_load *)user;
    int64_t dims[2] = {w->rows, w->cols};
    (void)layer;
    return gd_tensor_empty(wl->ctx, GD_ARENA_PARAMS, w->type, gd_shape_make(w->cols > 0 ? 2U : 1U, dims), 256U, w->dst);
}

static float bf16_value(uint16_t bits)
{
    const uint32_t u = (uint32_t)bits << 16;
    float f;
    memcpy(&f, &u, sizeof(f));
    return f;
}

static uint16_t bf16_bits(float f) /* to nearest, ties to even */
{
    uint32_t u;
    memcpy(&u, &f, sizeof(u));
    if ((u & 0x7fffffffU) > 0x7f800000U) return (uint16_t)((u >> 16) | 0x40U); /* NaN stays NaN */
    return (uint16_t)((u + 0x7fffU + ((u >> 16) & 1U)) >> 16);
}

/* n values of a file tensor into dst as type `to` */
static void convert(const unsigned char *src, gd_dtype from, unsigned char *dst, gd_dtype to, int64_t n)
{
    int64_t i;
    if (from == to) {
        memcpy(dst, src, (size_t)n * gd_dtype_size(to));
        return;
    }
#pragma omp parallel for schedule(static) if (n > 65536)
    for (i = 0; i < n; ++i) {
        const float f = from == GD_DTYPE_F32 ? ((const float *)src)[i] : bf16_value(((const uint16_t *)src)[i]);
        if (to == GD_DTYPE_F32) ((float *)dst)[i] = f;
        else ((uint16_t *)dst)[i] = bf16_bits(f);
    }
}

static void tensor_name(char *out, size_t size, const char *piece, int32_t layer)
{
    if (layer < 0) (void)snprintf(out, size, "%s", piece);
    else (void)snprintf(out, size, "l%d.%s", (int)layer, piece);
}

/* the file holds the piece in the right shape and a type that converts */
static gd_status check_weight(void *user, const weight *w, int32_t layer)
{
    weight_load *wl = (weight_load *)user;
    int p;
    for (p = 0; p < MAX_PIECES && w->piece[p] != NULL; ++p) {
        char name[64];
        const gd_safetensor *t;
        tensor_name(name, sizeof(name), w->piece[p], layer);
        t = gd_safetensors_find(wl->file, name);
        if (t == NULL || t->rank != (w->cols > 0 ? 2U : 1U) || t->shape[0] != w->piece_rows[p] ||
            (w->cols > 0 && t->shape[1] != w->cols))
            return GD_ERR_BAD_STATE;
        if (t->dtype != GD_DTYPE_BF16 && t->dtype != GD_DTYPE_F32) return GD_ERR_UNSUPPORTED;
    }
    return GD_OK;
}

static gd_status fill_weight(void *user, const weight *w, int32_t layer)
{
    weight_load *wl = (weight_load *)user;
    const int64_t n = weight_count(w);
    int64_t done = 0;
    int p;
    if (w->piece[0] == NULL && w->cols > 0) { /* ukt [heads, kv_rank, dim] from the first part of ukv [heads, dim, kv_rank] */
        const gd_backend_latent_args *a = &wl->c->layers[layer].latent;
        const size_t es = gd_dtype_size(w->type);
        const int64_t D = a->dim, R = a->kv_rank;
        gd_tensor uk;
        TRY(gd_tensor_slice(wl->ctx, wl->ukv, 0U, 0, (int64_t)a->heads * D, &uk));
        TRY(gd_tensor_read(wl->ctx, &uk, wl->raw, (size_t)n * es));
#pragma omp parallel for schedule(static)
        for (done = 0; done < n; ++done) {
            const int64_t h = done / (R * D), r = done / D % R, d = done % D;
            memcpy(wl->turned + (size_t)done * es, wl->raw + (size_t)((h * D + d) * R + r) * es, es);
        }
        return gd_tensor_write(wl->ctx, w->dst, wl->turned, (size_t)n * es);
    }
    if (w->piece[0] != NULL && !strcmp(w->piece[0], "mix.uk")) wl->ukv = w->dst;
    if (w->piece[0] == NULL) { /* rotation frequencies: base^(-2i/dims), in double, rounded once */
        const layer_config *l = &wl->c->layers[layer];
        float *f = (float *)wl->turned;
        for (done = 0; done < n; ++done)
            f[done] = (float)pow(l->rot_base, -2.0 * (double)done / (double)l->latent.rot_dim);
        return gd_tensor_write(wl->ctx, w->dst, f, (size_t)n * sizeof(float));
    }
    if (wl->file == NULL) {
        wl->seed = gd_splitmix64(wl->seed);
        return gd_backend_rand_uniform(gd_context_backend(wl->ctx), (gd_backend_buffer *)w->dst->storage.buffer,
                                       w->dst->storage.offset, (size_t)n, (uint32_t)w->type, wl->seed, w->lo, w->hi);
    }
    for (p = 0; p < MAX_PIECES && w->piece[p] != NULL; ++p) {
        const int64_t m = w->piece_rows[p] * (w->cols > 0 ? w->cols : 1);
        char name[64];
        const gd_safetensor *t;
        tensor_name(name, sizeof(name), w->piece[p], layer);
        t = gd_safetensors_find(wl->file, name);
        TRY(gd_safetensors_read(wl->file, t, wl->raw));
        convert(wl->raw, t->dtype, wl->turned + (size_t)done * gd_dtype_size(w->type), w->type, m);
        done += m;
    }
    return gd_tensor_write(wl->ctx, w->dst, wl->turned, (size_t)n * gd_dtype_size(w->type));
}

static gd_status largest_weight(void *user, const weight *w, int32_t layer)
{
    int64_t *most = (int64_t *)user;
    (void)layer;
    if (weight_count(w) > *most) *most = weight_count(w);
    return GD_OK;
}

static gd_status load_weights(gd_context *ctx, struct layer_list *ll, gd_safetensors *file, uint64_t seed)
{
    weight_load wl = {ctx, &ll->c, file, seed, NULL, NULL, NULL};
    int64_t most = 0;
    gd_status st;
    if (file != NULL) TRY(each_weight(&ll->c, ll->type, ll, check_weight, &wl)); /* before the first byte is written */
    TRY(each_weight(&ll->c, ll->type, ll, allocate_weight, &wl));
    TRY(each_weight(&ll->c, ll->type, ll, largest_weight, &most));
    wl.raw = (unsigned char *)malloc((size_t)most * 4U);
    wl.turned = (unsigned char *)malloc((size_t)most * 4U);
    st = wl.raw == NULL || wl.turned == NULL ? GD_ERR_OUT_OF_MEMORY : each_weight(&ll->c, ll->type, ll, fill_weight, &wl);
    free(wl.raw);
    free(wl.turned);
    return st;
}

/* ---- caches and states ----------------------------------------------------------------------------- */

static void state_dims(const layer_config *l, int64_t slots, int64_t max_seq, int64_t ring[3], int64_t states[4],
                       int64_t cache[3])
{
    ring[0] = states[0] = cache[0] = slots;
    ring[1] = l->taps;
    ring[2] = conv_channels(l);
    states[1] = l->ssm.heads;
    states[2] = l->ssm.state;
    states[3] = l->ssm.vdim;
    cache[1] = max_seq;
    cache[2] = gd_backend_latent_pitch(l->latent.kv_rank, l->latent.rot_dim);
}

static size_t state_bytes(const layer_list_config *c, gd_dtype type, int64_t slots, int64_t max_seq)
{
    const size_t es = gd_dtype_size(type);
    size_t total = 0U;
    int32_t i;
    for (i = 0; i < c->n_layers; ++i) {
        int64_t r[3], s[4], k[3];
        state_dims(&c->layers[i], slots, max_seq, r, s, k);
        if (c->layers[i].mixer == MIXER_MAMBA2)
            total += gd_pad256((size_t)(r[0] * r[1] * r[2]) * es) + gd_pad256((size_t)(s[0] * s[1] * s[2] * s[3]) * 4U);
        else total += gd_pad256((size_t)(k[0] * k[1] * k[2]) * es);
    }
    return total + 2U * gd_pad256((size_t)(slots + 1) * 4U);
}

static gd_status allocate_states(gd_context *ctx, struct layer_list *ll, int64_t slots, int64_t max_seq)
{
    int64_t bdim[1] = {slots}, cdim[1] = {slots + 1};
    int32_t *iota = (int32_t *)malloc((size_t)(slots + 1) * sizeof(int32_t));
    gd_status st = iota == NULL ? GD_ERR_OUT_OF_MEMORY : GD_OK;
    int32_t i;
    for (i = 0; i < ll->c.n_layers && st == GD_OK; ++i) {
        int64_t r[3], s[4], k[3];
        state_dims(&ll->c.layers[i], slots, max_seq, r, s, k);
        if (ll->c.layers[i].mixer == MIXER_MAMBA2) {
            st = gd_tensor_zeros(ctx, GD_ARENA_STATE, ll->type, gd_shape_make(3U, r), 256U, &ll->layers[i].ring);
            if (st == GD_OK)
                st = gd_tensor_zeros(ctx, GD_ARENA_STATE, GD_DTYPE_F32, gd_shape_make(4U, s), 256U, &ll->layers[i].states);
        } else {
            st = gd_tensor_zeros(ctx, GD_ARENA_STATE, ll->type, gd_shape_make(3U, k), 256U, &ll->layers[i].cache);
        }
    }
    if (st == GD_OK) st = gd_tensor_empty(ctx, GD_ARENA_STATE, GD_DTYPE_I32, gd_shape_make(1U, bdim), 256U, &ll->rows_dev);
    if (st == GD_OK) st = gd_tensor_empty(ctx, GD_ARENA_STATE, GD_DTYPE_I32, gd_shape_make(1U, cdim), 256U, &ll->cu_dev);
    if (st == GD_OK) {
        for (i = 0; i <= (int32_t)slots; ++i) iota[i] = i;
        st = gd_tensor_write(ctx, &ll->rows_dev, iota, (size_t)slots * sizeof(int32_t));
        if (st == GD_OK) st = gd_tensor_write(ctx, &ll->cu_dev, iota, (size_t)(slots + 1) * sizeof(int32_t));
    }
    free(iota);
    return st;
}

/* ---- forward ----------------------------------------------------------------------------------------- */

/* Scratch of one forward, shared by its layers (they run one after the other): the residual stream, its copy, and four
 * buffers whose largest use decides their size. */
typedef struct scratch_sizes {
    int64_t proj, a, b, branch; /* elements per row */
    int64_t angles;             /* F32 values per row */
    size_t work;                /* bytes for the whole step */
} scratch_sizes;

static int64_t max64(int64_t a, int64_t b) { return a > b ? a : b; }

static scratch_sizes sizes_of(const layer_list_config *c, gd_dtype type, int64_t rows, int64_t max_new, int64_t kv_total,
                              int64_t max_seq)
{
    scratch_sizes s = {0, c->width, 1, c->width, 1, 256U};
    int32_t i;
    for (i = 0; i < c->n_layers; ++i) {
        const layer_config *l = &c->layers[i];
        s.proj = max64(s.proj, mixer_in(l));
        if (l->mixer == MIXER_MAMBA2) {
            s.a = max64(s.a, max64(conv_channels(l), inner_size(l)));
            s.b = max64(s.b, inner_size(l));
        } else {
            const size_t w = gd_backend_latent_work_bytes(NULL, &l->latent, (uint32_t)rows, (uint32_t)max_new, (uint32_t)kv_total,
                                                          (uint32_t)max_seq, (uint32_t)type);
            s.angles = max64(s.angles, l->latent.rot_dim);
            s.a = max64(s.a, max64(l->latent.q_rank, mixer_out(l)));
            s.b = max64(s.b, query_size(l));
            if (w > s.work) s.work = w;
        }
        s.a = max64(s.a, l->ff);
    }
    return s;
}

static size_t forward_bytes(const layer_list_config *c, const scratch_sizes *s, gd_dtype type, int64_t rows)
{
    const size_t es = gd_dtype_size(type), R = (size_t)rows;
    return gd_pad256(R * (size_t)c->width * 4U) + gd_pad256(R * (size_t)c->width * es) + gd_pad256(R * (size_t)s->proj * es) +
           gd_pad256(R * (size_t)s->a * es) + gd_pad256(R * (size_t)s->b * es) + gd_pad256(R * (size_t)s->branch * es) +
           gd_pad256(R * (size_t)s->angles * 4U) + gd_pad256(s->work);
}

typedef struct forward {
    gd_gpt_decoder *d;
    gd_backend *be;
    struct layer_list *ll;
    uint32_t type;
    int64_t rows;
    gd_backend_packed_seqs seqs;
    gd_backend_tensor_view row_seq, cu, slot, start, kv_cu, ids;
    gd_tensor x, h, proj, a, b, branch, angles, work; /* h: the copy of x, or x itself when the projections are F32 */
} forward;

static void view2(const gd_tensor *t, uint32_t dtype, int64_t d0, int64_t d1, gd_backend_tensor_view *v)
{
    memset(v, 0, sizeof(*v));
    v->buffer = (gd_backend_buffer *)t->storage.buffer;
    v->offset = t->storage.offset + t->view_offset;
    v->dtype = dtype;
    v->rank = 2U;
    v->shape[0] = d0;
    v->shape[1] = d1;
    v->strides[0] = d1;
    v->strides[1] = 1;
    v->count = (size_t)(d0 * d1);
}

/* columns [col, col + cols) of a buffer of rows of `pitch` elements */
static void columns(const gd_tensor *t, uint32_t dtype, int64_t rows, int64_t pitch, int64_t col, int64_t cols,
                    gd_backend_matrix_view *m)
{
    const size_t es = gd_dtype_size((gd_dtype)dtype);
    m->buffer = (gd_backend_buffer *)t->storage.buffer;
    m->offset = t->storage.offset + t->view_offset + (size_t)col * es;
    m->rows = (uint32_t)rows;
    m->cols = (uint32_t)cols;
    m->row_bytes = (size_t)pitch * es;
    m->dtype = dtype;
}

static gd_status scratch(gd_context *ctx, gd_dtype type, int64_t rows, int64_t cols, gd_tensor *out)
{
    int64_t dims[2] = {rows, cols};
    return gd_tensor_empty(ctx, GD_ARENA_SCRATCH, type, gd_shape_make(2U, dims), 256U, out);
}

/* kv_total 0: the tokens the sequences hold are not expanded */
static gd_status forward_begin(forward *f, gd_gpt_decoder *d, int64_t rows, int64_t max_new, int64_t kv_total)
{
    struct layer_list *ll = d->layers;
    const scratch_sizes s = sizes_of(&ll->c, ll->type, rows, max_new, kv_total, d->cfg.max_seq);
    int64_t wdim[1] = {(int64_t)s.work};
    f->d = d;
    f->be = gd_context_backend(d->ctx);
    f->ll = ll;
    f->type = (uint32_t)ll->type;
    f->rows = rows;
    f->seqs.row_seq = &f->row_seq;
    f->seqs.cu = &f->cu;
    f->seqs.slot = &f->slot;
    f->seqs.start = &f->start;
    f->seqs.max_new = (uint32_t)max_new;
    f->seqs.kv_cu = kv_total > 0 ? &f->kv_cu : NULL;
    f->seqs.kv_total = (uint32_t)kv_total;
    TRY(scratch(d->ctx, GD_DTYPE_F32, rows, ll->c.width, &f->x));
    if (ll->type == GD_DTYPE_F32) f->h = f->x;
    else TRY(scratch(d->ctx, ll->type, rows, ll->c.width, &f->h));
    TRY(scratch(d->ctx, ll->type, rows, s.proj, &f->proj));
    TRY(scratch(d->ctx, ll->type, rows, s.a, &f->a));
    TRY(scratch(d->ctx, ll->type, rows, s.b, &f->b));
    TRY(scratch(d->ctx, GD_DTYPE_F32, rows, s.angles, &f->angles));
    TRY(scratch(d->ctx, ll->type, rows, s.branch, &f->branch));
    return gd_tensor_empty(d->ctx, GD_ARENA_SCRATCH, GD_DTYPE_U8, gd_shape_make(1U, wdim), 256U, &f->work);
}

/* y [rows, w rows] = x [rows, w cols] w^T (+ bias), buffers holding packed rows */
static gd_status project(forward *f, const gd_tensor *x, const gd_tensor *w, const gd_tensor *bias, uint32_t epilogue,
                         gd_tensor *y)
{
    const gd_backend_fused_linear_args args = {1U, bias != NULL ? 1U : 0U, 0U, 0.0f, epilogue};
    const int64_t outs = epilogue != 0U ? w->shape[0] / 2 : w->shape[0];
    gd_backend_matrix_view xm, wm, ym;
    gd_backend_vector_view bv;
    columns(x, f->type, f->rows, w->shape[1], 0, w->shape[1], &xm);
    mview(w, w->shape[0], w->shape[1], &wm);
    columns(y, f->type, f->rows, outs, 0, outs, &ym);
    if (bias != NULL) vview(bias, &bv);
    return gd_backend_fused_linear(f->be, &xm, &wm, bias != NULL ? &bv : NULL, NULL, NULL, &ym, &args);
}

/* x += m * norm(branch), h = x */
static gd_status add_branch(forward *f, const gd_tensor *norm)
{
    const int64_t W = f->ll->c.width;
    gd_backend_tensor_view vb, vn, vx, vh;
    view2(&f->branch, f->type, f->rows, W, &vb);
    tview(norm, &vn);
    view2(&f->x, GD_BACKEND_DTYPE_F32, f->rows, W, &vx);
    view2(&f->h, f->type, f->rows, W, &vh);
    return gd_backend_residual_norm_add(f->be, &vb, &vn, &vx, f->ll->type == GD_DTYPE_F32 ? NULL : &vh, f->ll->c.eps,
                                        f->ll->c.residual_mult);
}

static gd_status mamba2(forward *f, const layer_config *l, layer_weights *w)
{
    const int64_t inner = inner_size(l), ch = conv_channels(l), P = mixer_in(l);
    gd_backend_matrix_view z, u, dt;
    gd_backend_tensor_view taps, cb, ring, conv, dtb, al, dk, st, y, gn, out;
    TRY(project(f, &f->h, &w->in, NULL, 0U, &f->proj));
    columns(&f->proj, f->type, f->rows, P, 0, inner, &z);
    columns(&f->proj, f->type, f->rows, P, inner, ch, &u);
    columns(&f->proj, f->type, f->rows, P, inner + ch, l->ssm.heads, &dt);
    tview(&w->conv, &taps);
    tview(&w->conv_b, &cb);
    tview(&w->ring, &ring);
    tview(&w->dt_bias, &dtb);
    tview(&w->a_log, &al);
    tview(&w->d_skip, &dk);
    tview(&w->states, &st);
    view2(&f->b, f->type, f->rows, inner, &y);
    if (f->seqs.max_new == 1U) {
        TRY(gd_backend_conv_ssm_step(f->be, &u, &taps, &cb, &ring, &dt, &dtb, &al, &dk, &st, &y, &f->seqs, &l->ssm));
    } else {
        view2(&f->a, f->type, f->rows, ch, &conv);
        TRY(gd_backend_causal_conv_silu(f->be, &u, &taps, &cb, &ring, &conv, &f->seqs));
        TRY(gd_backend_ssm_scan(f->be, &conv, &dt, &dtb, &al, &dk, &st, &y, &f->seqs, &l->ssm));
    }
    tview(&w->gnorm, &gn);
    view2(&f->a, f->type, f->rows, inner, &out);
    TRY(gd_backend_gated_group_norm(f->be, &y, &z, &gn, &out, (uint32_t)l->norm_groups, f->ll->c.eps));
    return project(f, &f->a, &w->out, NULL, 0U, &f->branch);
}

static gd_status latent_attention(forward *f, const layer_config *l, layer_weights *w)
{
    const gd_backend_latent_args *a = &l->latent;
    const int64_t P = mixer_in(l), gate_col = P - mixer_out(l);
    gd_backend_matrix_view pm, gate;
    gd_backend_tensor_view qn, kn, freq, ang, cq, cache, q, ukt, ukv, work, out;
    TRY(project(f, &f->h, &w->in, NULL, 0U, &f->proj));
    columns(&f->proj, f->type, f->rows, P, 0, gate_col, &pm);
    columns(&f->proj, f->type, f->rows, P, gate_col, mixer_out(l), &gate);
    tview(&w->dq_norm, &qn);
    tview(&w->dkv_norm, &kn);
    tview(&w->freq, &freq);
    tview(&w->cache, &cache);
    view2(&f->a, f->type, f->rows, a->q_rank, &cq);
    view2(&f->angles, GD_BACKEND_DTYPE_F32, f->rows, a->rot_dim, &ang);
    TRY(gd_backend_latent_prepare(f->be, &pm, &qn, &kn, &freq, &ang, &cq, &cache, &f->seqs, a));
    TRY(project(f, &f->a, &w->uq, NULL, 0U, &f->b));
    view2(&f->b, f->type, f->rows, query_size(l), &q);
    tview(&w->ukt, &ukt);
    tview(&w->ukv, &ukv);
    tview(&f->work, &work);
    view2(&f->a, f->type, f->rows, mixer_out(l), &out);
    TRY(gd_backend_latent_attend(f->be, &q, &ukt, &ukv, &gate, &ang, &cache, &work, &out, &f->seqs, a));
    return project(f, &f->a, &w->out, NULL, 0U, &f->branch);
}

/* every layer over the rows of f, from the token ids to the residual stream in f->x */
static gd_status run_layers(forward *f)
{
    const int64_t W = f->ll->c.width;
    gd_backend_tensor_view ve, vx, vh;
    int32_t i;
    tview(&f->ll->embed, &ve);
    view2(&f->x, GD_BACKEND_DTYPE_F32, f->rows, W, &vx);
    view2(&f->h, f->type, f->rows, W, &vh);
    TRY(gd_backend_residual_embed(f->be, &ve, &f->ids, &vx, f->ll->type == GD_DTYPE_F32 ? NULL : &vh,
                                  f->ll->c.embedding_scale));
    for (i = 0; i < f->ll->c.n_layers; ++i) {
        const layer_config *l = &f->ll->c.layers[i];
        layer_weights *w = &f->ll->layers[i];
        if (l->mixer == MIXER_MAMBA2) TRY(mamba2(f, l, w));
        else TRY(latent_attention(f, l, w));
        TRY(add_branch(f, &w->norm1));
        if (l->ff > 0) {
            TRY(project(f, &f->h, &w->upgate, &w->upgate_b, 2U, &f->a));
            TRY(project(f, &f->a, &w->down, &w->down_b, 0U, &f->branch));
            TRY(add_branch(f, &w->norm2));
        }
    }
    return GD_OK;
}

/* F32 logits of the picked rows (NULL: of all rows) */
static gd_status head(forward *f, const gd_backend_tensor_view *rows, int64_t n, gd_tensor *logits)
{
    const layer_list_config *c = &f->ll->c;
    gd_backend_tensor_view vx, vn, vo;
    gd_backend_matrix_view xm, wm, ym;
    gd_tensor normed;
    TRY(scratch(f->d->ctx, f->ll->type, n, c->width, &normed));
    TRY(scratch(f->d->ctx, GD_DTYPE_F32, n, c->vocab, logits));
    view2(&f->x, GD_BACKEND_DTYPE_F32, f->rows, c->width, &vx);
    tview(&f->ll->final_norm, &vn);
    tview(&normed, &vo);
    TRY(gd_backend_residual_norm_rows(f->be, &vx, rows, &vn, &vo, c->eps));
    mview(&normed, n, c->width, &xm);
    mview(&f->ll->embed, c->vocab, c->width, &wm);
    mview(logits, n, c->vocab, &ym);
    return gd_backend_matmul_nt(f->be, &xm, &wm, &ym);
}

static gd_status layer_list_step(gd_gpt_decoder *d, const gd_tensor *ids, const gd_tensor *positions, bool fused,
                                 gd_tensor *logits)
{
    forward f;
    (void)fused; /* one form: its launches are fused as far as they go */
    TRY(forward_begin(&f, d, d->cfg.batch, 1, 0));
    view1(ids, &f.ids);
    view1(&d->layers->rows_dev, &f.row_seq);
    view1(&d->layers->rows_dev, &f.slot);
    view1(&d->layers->cu_dev, &f.cu);
    view1(positions, &f.start);
    TRY(run_layers(&f));
    return head(&f, NULL, f.rows, logits);
}

static gd_status layer_list_extend(gd_gpt_decoder *d, const gd_extend_rows *e, gd_tensor *logits)
{
    enum { IDS, ROW_SEQ, CU, SLOT, START, KV_CU, WANT, PARTS };
    const int64_t N = e->rows, S = e->n_seqs;
    const int64_t len[PARTS] = {N, N, S + 1, S, S, S + 1, e->n_want};
    int64_t at[PARTS + 1], kv_total = 0;
    forward f;
    gd_tensor tables, part[PARTS];
    gd_backend_tensor_view want;
    int32_t *host;
    int32_t s, r;
    gd_status st;
    if (N > d->layers->max_step_tokens) return GD_ERR_INVALID_ARGUMENT;
    at[0] = 0;
    for (r = 0; r < PARTS; ++r) at[r + 1] = at[r] + len[r];
    host = (int32_t *)malloc((size_t)at[PARTS] * sizeof(int32_t));
    if (host == NULL) return GD_ERR_OUT_OF_MEMORY;
    /* one upload for all tables of the step */
    memcpy(host + at[IDS], e->ids, (size_t)N * sizeof(int32_t));
    memcpy(host + at[CU], e->cu, (size_t)(S + 1) * sizeof(int32_t));
    memcpy(host + at[SLOT], e->slots, (size_t)S * sizeof(int32_t));
    memcpy(host + at[START], e->start, (size_t)S * sizeof(int32_t));
    if (e->n_want > 0) memcpy(host + at[WANT], e->want, (size_t)e->n_want * sizeof(int32_t));
    host[at[KV_CU]] = 0;
    for (s = 0; s < S; ++s) {
        for (r = e->cu[s]; r < e->cu[s + 1]; ++r) host[at[ROW_SEQ] + r] = s;
        kv_total += e->start[s] + (e->cu[s + 1] - e->cu[s]);
        host[at[KV_CU] + s + 1] = kv_total <= INT32_MAX ? (int32_t)kv_total : INT32_MAX;
    }
    if (kv_total > d->layers->kv_rows) kv_total = 0; /* too many tokens to expand at once: the absorbed form */
    st = data_i32(d->ctx, host, at[PARTS], &tables);
    free(host);
    for (r = 0; r < PARTS && st == GD_OK; ++r) {
        if (len[r] > 0) st = gd_tensor_slice(d->ctx, &tables, 0U, at[r], len[r], &part[r]);
    }
    if (st != GD_OK) return st;
    TRY(forward_begin(&f, d, N, e->max_new, kv_total));
    view1(&part[IDS], &f.ids);
    view1(&part[ROW_SEQ], &f.row_seq);
    view1(&part[CU], &f.cu);
    view1(&part[SLOT], &f.slot);
    view1(&part[START], &f.start);
    view1(&part[KV_CU], &f.kv_cu);
    TRY(run_layers(&f));
    if (e->n_want == 0) return GD_OK;
    view1(&part[WANT], &want);
    return head(&f, &want, e->n_want, logits);
}

static gd_status layer_list_prefill(gd_gpt_decoder *d, const int32_t *ids, const int32_t *cu, gd_tensor *logits)
{
    const int32_t B = d->cfg.batch;
    int32_t *t = (int32_t *)calloc((size_t)B * 3U, sizeof(int32_t));
    gd_extend_rows e;
    gd_status st;
    int32_t b;
    if (t == NULL) return GD_ERR_OUT_OF_MEMORY;
    memset(&e, 0, sizeof(e));
    for (b = 0; b < B; ++b) {
        t[b] = b;                    /* slots */
        t[2 * B + b] = cu[b + 1] - 1; /* last rows; t[B ..]: starts, all 0 */
        if (cu[b + 1] - cu[b] > e.max_new) e.max_new = cu[b + 1] - cu[b];
    }
    e.n_seqs = B;
    e.rows = cu[B];
    e.slots = t;
    e.ids = ids;
    e.cu = cu;
    e.start = t + B;
    e.want = t + 2 * B;
    e.n_want = B;
    st = layer_list_extend(d, &e, logits);
    free(t);
    return st;
}

/* ---- creation ------------------------------------------------------------------------------------------ */

static bool layer_list_can_fuse(const gd_gpt_decoder *d)
{
    (void)d;
    return true;
}

static bool layer_list_feeds_x0(const gd_gpt_decoder *d)
{
    (void)d; /* the embedding is scaled into an F32 residual: gathered at the start of the step */
    return false;
}

static gd_tensor *layer_list_tensor(gd_gpt_decoder *d, const char *name, int32_t layer)
{
    struct layer_list *ll = d->layers;
    layer_weights *w;
    if (!strcmp(name, "embed")) return &ll->embed;
    if (!strcmp(name, "final_norm")) return &ll->final_norm;
    if (layer < 0 || layer >= ll->c.n_layers) return NULL;
    w = &ll->layers[layer];
    if (!strcmp(name, "cache") && ll->c.layers[layer].mixer == MIXER_LATENT_ATTENTION) return &w->cache;
    if (!strcmp(name, "states") && ll->c.layers[layer].mixer == MIXER_MAMBA2) return &w->states;
    if (!strcmp(name, "conv_ring") && ll->c.layers[layer].mixer == MIXER_MAMBA2) return &w->ring;
    return NULL;
}

static void layer_list_destroy(gd_gpt_decoder *d)
{
    if (d->layers == NULL) return;
    gd_layer_list_config_free(&d->layers->c);
    free(d->layers->layers);
    free(d->layers);
}

static const gd_decoder_model layer_list_model = {"Girirax", layer_list_prefill, layer_list_step, layer_list_extend,
                                                  layer_list_can_fuse, layer_list_feeds_x0, layer_list_tensor,
                                                  layer_list_destroy};

/* the options with their defaults filled in, and what the session keeps of the configuration */
static gd_status settle(const layer_list_config *c, const gd_model_options *in, gd_model_options *o, gd_gpt_config *g)
{
    *o = *in;
    if (o->batch == 0) o->batch = 1;
    if (o->compute == GD_DTYPE_INVALID) o->compute = GD_DTYPE_BF16;
    if (o->max_seq <= 0 || o->batch < 0 || o->max_step_tokens < 0) return GD_ERR_INVALID_ARGUMENT;
    if (o->compute != GD_DTYPE_BF16 && o->compute != GD_DTYPE_F32) return GD_ERR_UNSUPPORTED;
    if (o->max_step_tokens == 0 || o->max_step_tokens > (int64_t)o->batch * o->max_seq) {
        const int64_t all = (int64_t)o->batch * o->max_seq;
        o->max_step_tokens = all > INT32_MAX ? INT32_MAX : (int32_t)all;
    }
    if (o->max_step_tokens < o->batch) o->max_step_tokens = o->batch;
    memset(g, 0, sizeof(*g));
    g->vocab = c->vocab;
    g->d_model = c->width;
    g->n_layers = c->n_layers;
    g->max_seq = o->max_seq;
    g->batch = o->batch;
    g->tie_lm_head = 1;
    return GD_OK;
}

/* tokens whose keys and values a step may expand: a step of new prompts, and one long sequence continued */
static int32_t kv_rows(const gd_model_options *o)
{
    const int64_t n = (int64_t)o->max_step_tokens + o->max_seq;
    return n > INT32_MAX ? INT32_MAX : (int32_t)n;
}

gd_status gd_layer_list_memory(const layer_list_config *c, const gd_model_options *in, gd_memory_config *out)
{
    gd_model_options o;
    gd_gpt_config g;
    size_t params = 0U, rows, logit_rows, step;
    scratch_sizes s;
    TRY(settle(c, in, &o, &g));
    TRY(each_weight(c, o.compute, NULL, add_bytes, &params));
    rows = (size_t)o.max_step_tokens;
    logit_rows = ((size_t)1 << 30) / ((size_t)c->vocab * 4U);
    if (logit_rows > rows) logit_rows = rows;
    *out = gd_memory_config_default();
    out->params_bytes = params + 4096U;
    out->state_bytes = state_bytes(c, o.compute, o.batch, o.max_seq) + gd_decoder_session_bytes(&g, GD_DTYPE_F32, false) + 4096U;
    /* a resident session holds an eager step and a captured one, its records besides; logits of every row of a step,
     * up to 1 GiB of them */
    /* the largest step: every form attention may take with that many rows */
    s = sizes_of(c, o.compute, (int64_t)rows, 1, 0, o.max_seq);
    step = forward_bytes(c, &s, o.compute, (int64_t)rows);
    s = sizes_of(c, o.compute, (int64_t)rows, (int64_t)rows, kv_rows(&o), o.max_seq);
    step = step > forward_bytes(c, &s, o.compute, (int64_t)rows) ? step : forward_bytes(c, &s, o.compute, (int64_t)rows);
    /* few rows are cut into more pieces per row; a resident session has an eager and a captured step */
    s = sizes_of(c, o.compute, 512, 1, 0, o.max_seq);
    step += 2U * s.work;
    s = sizes_of(c, o.compute, o.batch, 1, 0, o.max_seq);
    out->scratch_slot_bytes = step + 2U * forward_bytes(c, &s, o.compute, o.batch) +
                              logit_rows * (size_t)c->vocab * 4U + rows * (size_t)c->width * 4U +
                              2U * gd_pad256((size_t)o.batch * (size_t)c->vocab * 4U) +
                              (size_t)o.batch * (size_t)o.max_seq * 8U + ((size_t)16 << 20);
    out->data_slot_bytes = rows * 16U + (size_t)o.batch * 64U + ((size_t)1 << 20);
    out->scratch_slots = 2U;
    out->data_slots = 2U;
    return GD_OK;
}

static gd_status copy_config(const layer_list_config *c, layer_list_config *out)
{
    *out = *c;
    out->layers = (layer_config *)malloc((size_t)c->n_layers * sizeof(layer_config));
    if (out->layers == NULL) return GD_ERR_OUT_OF_MEMORY;
    memcpy(out->layers, c->layers, (size_t)c->n_layers * sizeof(layer_config));
    return GD_OK;
}

gd_status gd_layer_list_create(gd_context *ctx, const layer_list_config *c, const gd_model_options *in,
                               gd_safetensors *weights, uint64_t seed, gd_gpt_decoder **out)
{
    gd_model_options o;
    gd_gpt_config g;
    gd_gpt_decoder *d;
    struct layer_list *ll;
    gd_status st;
    *out = NULL;
    TRY(settle(c, in, &o, &g));
    TRY(gd_decoder_session_create(ctx, &layer_list_model, &g, &d));
    d->layers = ll = (struct layer_list *)calloc(1, sizeof(*ll));
    st = ll == NULL ? GD_ERR_OUT_OF_MEMORY : copy_config(c, &ll->c);
    if (st == GD_OK) {
        ll->type = o.compute;
        ll->max_step_tokens = o.max_step_tokens;
        ll->kv_rows = kv_rows(&o);
        ll->layers = (layer_weights *)calloc((size_t)c->n_layers, sizeof(layer_weights));
        if (ll->layers == NULL) st = GD_ERR_OUT_OF_MEMORY;
    }
    if (st == GD_OK) st = load_weights(ctx, ll, weights, seed);
    if (st == GD_OK) st = allocate_states(ctx, ll, o.batch, o.max_seq);
    if (st == GD_OK) st = gd_decoder_session_allocate(d, GD_DTYPE_F32, false);
    if (st != GD_OK) {
        gd_gpt_decoder_destroy(d);
        return st;
    }
    d->token_embedding = ll->embed;
    *out = d;
    return GD_OK;
}
