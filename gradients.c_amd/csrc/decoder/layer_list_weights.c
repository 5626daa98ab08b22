/* The weights of a layer-list decoder: which ones a configuration asks for, and filling them from a file or a seed. */
#include <math.h>
#include <stdio.h>

#include "layer_list_internal.h"

#define MAX_PIECES 4

/* What a weight that is not a stack of file tensors is made from */
typedef enum weight_source { FROM_FILE, TURNED_UK, FREQUENCIES, EXPERT_TABLE } weight_source;

/* One weight of the decoder: where it goes, its type and shape, the tensors of the file that are stacked in it, and the
 * range of random weights. */
typedef struct weight {
    gd_tensor *dst;
    gd_dtype type;
    int64_t rows, cols; /* cols 0: a vector */
    const char *piece[MAX_PIECES];
    int64_t piece_rows[MAX_PIECES];
    float lo, hi;
    int32_t copies; /* > 0: the pieces once for every number below it, written into their names */
    float offset;   /* added to the file's values */
    weight_source source;
} weight;

typedef gd_status (*weight_fn)(void *user, const weight *w, int32_t layer);

/* calls fn for every weight, the layers' in order (layer -1: the model's own); ll NULL: destinations are NULL */
static gd_status each_weight(const layer_list_config *c, gd_dtype type, struct layer_list *ll, weight_fn fn, void *user)
{
    const float one = 1.0f, off = c->norm_offset;
    int32_t i;
#define AT(field) (ll != NULL ? &ll->field : NULL)
#define ADD(...)                         \
    do {                                 \
        const weight w_ = {__VA_ARGS__}; \
        TRY(fn(user, &w_, i));           \
    } while (0)
#define ONE(dst_, type_, rows_, cols_, name_, lo_, hi_) ADD(dst_, type_, rows_, cols_, {name_}, {rows_}, lo_, hi_, 0, 0.0f, FROM_FILE)
#define NORM(dst_, name_) ADD(dst_, GD_DTYPE_F32, c->width, 0, {name_}, {c->width}, one, one, 0, off, FROM_FILE)
    i = -1;
    ONE(AT(embed), type, c->vocab, c->width, "embed", -0.05f, 0.05f);
    if (c->own_head) ONE(AT(head), type, c->vocab, c->width, "head", -0.05f, 0.05f);
    NORM(AT(final_norm), "final.norm");
    for (i = 0; i < c->n_layers; ++i) {
        const layer_config *l = &c->layers[i];
        const float wide = 1.7f / sqrtf((float)c->width); /* uniform range whose products keep unit variance */
        const float fr = 1.7f / sqrtf((float)(l->ff > 0 ? l->ff : 1));
        if (l->weights_of != i) continue;
        NORM(AT(layers[i].norm1), "norm1");
        if (l->mixer == MIXER_MAMBA2) {
            const int64_t ch = conv_channels(l), H = l->ssm.heads;
            ONE(AT(layers[i].in), type, mixer_in(l), c->width, "mix.in", -wide, wide);
            ONE(AT(layers[i].conv), GD_DTYPE_F32, ch, l->taps, "mix.conv", -0.5f, 0.5f);
            ONE(AT(layers[i].conv_b), GD_DTYPE_F32, ch, 0, "mix.conv.b", -0.1f, 0.1f);
            ONE(AT(layers[i].dt_bias), GD_DTYPE_F32, H, 0, "mix.dt_bias", -4.6f, -2.3f);
            ONE(AT(layers[i].a_log), GD_DTYPE_F32, H, 0, "mix.A_log", 0.0f, 2.7f);
            ONE(AT(layers[i].d_skip), GD_DTYPE_F32, H, 0, "mix.D", 0.5f, 1.5f);
            ONE(AT(layers[i].gnorm), GD_DTYPE_F32, inner_size(l), 0, "mix.norm", 1.0f, 1.0f);
        } else if (l->mixer == MIXER_LATENT_ATTENTION) {
            const gd_backend_latent_args *a = &l->latent;
            const int64_t H = a->heads;
            const float qr = 1.7f / sqrtf((float)a->q_rank), kr = 1.7f / sqrtf((float)a->kv_rank);
            ADD(AT(layers[i].in), type, mixer_in(l), c->width, {"mix.dq", "mix.dkv", "mix.g"},
                {a->q_rank, (int64_t)a->kv_rank + a->rot_dim, H * a->vdim}, -wide, wide, 0, 0.0f, FROM_FILE);
            ONE(AT(layers[i].dq_norm), GD_DTYPE_F32, a->q_rank, 0, "mix.dq.norm", 1.0f, 1.0f);
            ONE(AT(layers[i].dkv_norm), GD_DTYPE_F32, a->kv_rank, 0, "mix.dkv.norm", 1.0f, 1.0f);
            ONE(AT(layers[i].uq), type, query_size(l), a->q_rank, "mix.uq", -qr, qr);
            ADD(AT(layers[i].ukv), type, H * ((int64_t)a->dim + a->vdim), a->kv_rank, {"mix.uk", "mix.uv"},
                {H * a->dim, H * a->vdim}, -kr, kr, 0, 0.0f, FROM_FILE);
            ADD(AT(layers[i].ukt), type, H * a->kv_rank, a->dim, {NULL}, {0}, 0.0f, 0.0f, 0, 0.0f, TURNED_UK);
            ADD(AT(layers[i].freq), GD_DTYPE_F32, a->rot_dim / 2, 0, {NULL}, {0}, 0.0f, 0.0f, 0, 0.0f, FREQUENCIES);
        } else {
            const gd_backend_grouped_args *a = &l->grouped;
            const int64_t H = a->heads, G = a->kv_heads;
            ADD(AT(layers[i].in), type, mixer_in(l), c->width, {"mix.q", "mix.k", "mix.v", "mix.g"},
                {H * a->dim, G * a->dim, G * a->vdim, H}, -wide, wide, 0, 0.0f, FROM_FILE);
            ADD(AT(layers[i].freq), GD_DTYPE_F32, a->rot_dims / 2, 0, {NULL}, {0}, 0.0f, 0.0f, 0, 0.0f, FREQUENCIES);
        }
        ONE(AT(layers[i].out), type, c->width, mixer_out(l), "mix.o", -wide, wide);
        if (l->mlp == MLP_NONE) continue;
        NORM(AT(layers[i].norm2), "norm2");
        if (l->mlp == MLP_GELU_GATED) {
            ADD(AT(layers[i].upgate), type, 2 * (int64_t)l->ff, c->width, {"mlp.up", "mlp.gate"}, {l->ff, l->ff}, -wide, wide, 0, 0.0f, FROM_FILE);
            ADD(AT(layers[i].upgate_b), type, 2 * (int64_t)l->ff, 0, {"mlp.up.b", "mlp.gate.b"}, {l->ff, l->ff}, -0.1f, 0.1f, 0, 0.0f, FROM_FILE);
            ONE(AT(layers[i].down), type, c->width, l->ff, "mlp.down", -fr, fr);
            ONE(AT(layers[i].down_b), type, c->width, 0, "mlp.down.b", -0.1f, 0.1f);
        } else if (l->mlp == MLP_SQUARE_RELU) {
            ONE(AT(layers[i].upgate), type, l->ff, c->width, "mlp.up", -wide, wide);
            ONE(AT(layers[i].down), type, c->width, l->ff, "mlp.down", -fr, fr);
        } else {
            const gd_backend_routed_args *a = &l->routed;
            const int64_t E = a->experts, F = a->ff, S = l->shared_ff;
            const float er = 1.7f / sqrtf((float)F), sr = 1.7f / sqrtf((float)(S > 0 ? S : 1));
            ADD(AT(layers[i].table), GD_DTYPE_I32, c->vocab, a->top, {"mlp.table"}, {c->vocab}, 0.0f, 0.0f, 0, 0.0f, EXPERT_TABLE);
            ADD(AT(layers[i].expert_upgate), type, E * 2 * F, c->width, {"mlp.e%d.up", "mlp.e%d.gate"}, {F, F}, -wide, wide, (int32_t)E, 0.0f, FROM_FILE);
            ADD(AT(layers[i].expert_down), type, E * c->width, F, {"mlp.e%d.down"}, {c->width}, -er, er, (int32_t)E, 0.0f, FROM_FILE);
            if (S > 0) {
                ADD(AT(layers[i].upgate), type, 2 * S, c->width, {"mlp.shared.up", "mlp.shared.gate"}, {S, S}, -wide, wide, 0, 0.0f, FROM_FILE);
                ONE(AT(layers[i].down), type, c->width, S, "mlp.shared.down", -sr, sr);
            }
        }
    }
#undef NORM
#undef ONE
#undef ADD
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

size_t gd_layer_list_weight_bytes(const layer_list_config *c, gd_dtype type)
{
    size_t bytes = 0U;
    (void)each_weight(c, type, NULL, add_bytes, &bytes);
    return bytes;
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

/* n values of a file tensor, plus offset, into dst as type `to` */
static void convert(const unsigned char *src, gd_dtype from, unsigned char *dst, gd_dtype to, int64_t n, float offset)
{
    int64_t i;
    if (from == to && offset == 0.0f) {
        memcpy(dst, src, (size_t)n * gd_dtype_size(to));
        return;
    }
#pragma omp parallel for schedule(static) if (n > 65536)
    for (i = 0; i < n; ++i) {
        const float f = offset + (from == GD_DTYPE_F32 ? ((const float *)src)[i] : bf16_value(((const uint16_t *)src)[i]));
        if (to == GD_DTYPE_F32) ((float *)dst)[i] = f;
        else ((uint16_t *)dst)[i] = bf16_bits(f);
    }
}

static const gd_safetensor *piece_of(gd_safetensors *file, const char *piece, int32_t copy, int32_t layer)
{
    char part[64], name[96];
    const char *hole = strstr(piece, "%d");
    if (hole != NULL)
        (void)snprintf(part, sizeof(part), "%.*s%d%s", (int)(hole - piece), piece, (int)copy, hole + 2);
    else (void)snprintf(part, sizeof(part), "%s", piece);
    if (layer < 0) (void)snprintf(name, sizeof(name), "%s", part);
    else (void)snprintf(name, sizeof(name), "l%d.%s", (int)layer, part);
    return gd_safetensors_find(file, name);
}

static int32_t copies_of(const weight *w) { return w->copies > 0 ? w->copies : 1; }

/* the file holds the pieces in the right shape and a type that converts */
static gd_status check_weight(void *user, const weight *w, int32_t layer)
{
    weight_load *wl = (weight_load *)user;
    int32_t copy;
    int p;
    for (copy = 0; copy < copies_of(w); ++copy) {
        for (p = 0; p < MAX_PIECES && w->piece[p] != NULL; ++p) {
            const gd_safetensor *t = piece_of(wl->file, w->piece[p], copy, layer);
            if (t == NULL || t->rank != (w->cols > 0 ? 2U : 1U) || t->shape[0] != w->piece_rows[p] ||
                (w->cols > 0 && t->shape[1] != w->cols))
                return GD_ERR_BAD_STATE;
            if (w->type == GD_DTYPE_I32 ? t->dtype != GD_DTYPE_I32 : t->dtype != GD_DTYPE_BF16 && t->dtype != GD_DTYPE_F32)
                return GD_ERR_UNSUPPORTED;
        }
    }
    return GD_OK;
}

/* ukt [heads, kv_rank, dim] from the first part of ukv [heads, dim, kv_rank] */
static gd_status fill_turned_uk(weight_load *wl, const weight *w, const layer_config *l)
{
    const int64_t n = weight_count(w), D = l->latent.dim, R = l->latent.kv_rank;
    const size_t es = gd_dtype_size(w->type);
    gd_tensor uk;
    int64_t i;
    TRY(gd_tensor_slice(wl->ctx, wl->ukv, 0U, 0, (int64_t)l->latent.heads * D, &uk));
    TRY(gd_tensor_read(wl->ctx, &uk, wl->raw, (size_t)n * es));
#pragma omp parallel for schedule(static)
    for (i = 0; i < n; ++i) {
        const int64_t h = i / (R * D), r = i / D % R, d = i % D;
        memcpy(wl->turned + (size_t)i * es, wl->raw + (size_t)((h * D + d) * R + r) * es, es);
    }
    return gd_tensor_write(wl->ctx, w->dst, wl->turned, (size_t)n * es);
}

/* Frequency of rotation pair i of `dims` rotated dimensions: base^(-2i/dims), and with YaRN scaling divided by `factor`
 * for the pairs that turn slowly: the pair that turns t times over `original` positions is number
 * dims ln(original / (2 pi t)) / (2 ln base); pairs up to the one of t = fast stay, those from the one of t = slow on
 * are scaled, the ones between are mixed linearly. */
static double frequency(int64_t i, int64_t dims, double base, const rot_scaling *s)
{
    const double f = pow(base, -2.0 * (double)i / (double)dims), pi = 3.14159265358979323846;
    double lo, hi, ramp, span;
    if (s->factor == 0.0) return f;
    lo = floor((double)dims * log(s->original / (2.0 * pi * s->fast)) / (2.0 * log(base)));
    hi = ceil((double)dims * log(s->original / (2.0 * pi * s->slow)) / (2.0 * log(base)));
    if (lo < 0.0) lo = 0.0;
    if (hi > (double)(dims - 1)) hi = (double)(dims - 1);
    span = hi - lo > 0.001 ? hi - lo : 0.001;
    ramp = ((double)i - lo) / span;
    ramp = ramp < 0.0 ? 0.0 : ramp > 1.0 ? 1.0 : ramp;
    return f / s->factor * ramp + f * (1.0 - ramp);
}

/* in double, rounded once */
static gd_status fill_frequencies(weight_load *wl, const weight *w, const layer_config *l)
{
    const int64_t n = weight_count(w);
    float *f = (float *)wl->turned;
    int64_t i;
    for (i = 0; i < n; ++i) f[i] = (float)frequency(i, 2 * n, l->rot_base, &l->scaling);
    return gd_tensor_write(wl->ctx, w->dst, f, (size_t)n * sizeof(float));
}

/* the experts of every token id: in range and different from each other, which the kernels rely on */
static gd_status fill_table(weight_load *wl, const weight *w, const layer_config *l, int32_t layer)
{
    const int64_t V = w->rows, K = w->cols, E = l->routed.experts;
    int32_t *t = (int32_t *)wl->raw;
    int64_t v, a, b;
    if (wl->file != NULL) {
        TRY(gd_safetensors_read(wl->file, piece_of(wl->file, w->piece[0], 0, layer), t));
    } else {
        for (v = 0; v < V; ++v) { /* neighbours on a circle of the experts, at a random place */
            wl->seed = gd_splitmix64(wl->seed);
            for (a = 0; a < K; ++a) t[v * K + a] = (int32_t)((wl->seed % (uint64_t)E + (uint64_t)(a * (E / K))) % (uint64_t)E);
        }
    }
    for (v = 0; v < V; ++v) {
        for (a = 0; a < K; ++a) {
            if (t[v * K + a] < 0 || t[v * K + a] >= E) return GD_ERR_BAD_STATE;
            for (b = 0; b < a; ++b) {
                if (t[v * K + a] == t[v * K + b]) return GD_ERR_BAD_STATE;
            }
        }
    }
    return gd_tensor_write(wl->ctx, w->dst, t, (size_t)(V * K) * sizeof(int32_t));
}

static gd_status fill_weight(void *user, const weight *w, int32_t layer)
{
    weight_load *wl = (weight_load *)user;
    const layer_config *l = layer >= 0 ? &wl->c->layers[layer] : NULL;
    const int64_t n = weight_count(w);
    int64_t done = 0;
    int32_t copy;
    int p;
    if (w->source == TURNED_UK) return fill_turned_uk(wl, w, l);
    if (w->source == FREQUENCIES) return fill_frequencies(wl, w, l);
    if (w->source == EXPERT_TABLE) return fill_table(wl, w, l, layer);
    if (!strcmp(w->piece[0], "mix.uk")) wl->ukv = w->dst;
    if (wl->file == NULL) {
        wl->seed = gd_splitmix64(wl->seed);
        return gd_backend_rand_uniform(gd_context_backend(wl->ctx), (gd_backend_buffer *)w->dst->storage.buffer,
                                       w->dst->storage.offset, (size_t)n, (uint32_t)w->type, wl->seed, w->lo, w->hi);
    }
    for (copy = 0; copy < copies_of(w); ++copy) {
        for (p = 0; p < MAX_PIECES && w->piece[p] != NULL; ++p) {
            const int64_t m = w->piece_rows[p] * (w->cols > 0 ? w->cols : 1);
            const gd_safetensor *t = piece_of(wl->file, w->piece[p], copy, layer);
            TRY(gd_safetensors_read(wl->file, t, wl->raw));
            convert(wl->raw, t->dtype, wl->turned + (size_t)done * gd_dtype_size(w->type), w->type, m, w->offset);
            done += m;
        }
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

gd_status gd_layer_list_load(gd_context *ctx, struct layer_list *ll, gd_safetensors *file, uint64_t seed)
{
    weight_load wl = {ctx, &ll->c, file, seed, NULL, NULL, NULL};
    int64_t most = 0;
    int32_t i;
    gd_status st;
    if (file != NULL) TRY(each_weight(&ll->c, ll->type, ll, check_weight, &wl)); /* before the first byte is written */
    TRY(each_weight(&ll->c, ll->type, ll, allocate_weight, &wl));
    TRY(each_weight(&ll->c, ll->type, ll, largest_weight, &most));
    wl.raw = (unsigned char *)malloc((size_t)most * 4U);
    wl.turned = (unsigned char *)malloc((size_t)most * 4U);
    st = wl.raw == NULL || wl.turned == NULL ? GD_ERR_OUT_OF_MEMORY : each_weight(&ll->c, ll->type, ll, fill_weight, &wl);
    free(wl.raw);
    free(wl.turned);
    for (i = 0; i < ll->c.n_layers && st == GD_OK; ++i) {
        if (ll->c.layers[i].weights_of != i) ll->layers[i] = ll->layers[ll->c.layers[i].weights_of];
    }
    return st;
}
