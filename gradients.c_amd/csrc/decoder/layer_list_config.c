/* config.json of a layer-list decoder -> layer_list_config, every size and constant checked. */
#include <math.h>
#include <stdarg.h>
#include <stdio.h>

#include "layer_list.h"

#define SIZE_MAX_I32 (1 << 28)
#define BONATAR_GATE_ALPHA 1.702f /* steepness of the experts' gate */

typedef struct parse {
    char *message;
    size_t size;
    gd_status st; /* the first failure */
} parse;

static void fail(parse *p, gd_status st, const char *fmt, ...)
{
    va_list ap;
    if (p->st != GD_OK) return;
    p->st = st;
    if (p->message == NULL || p->size == 0U) return;
    va_start(ap, fmt);
    (void)vsnprintf(p->message, p->size, fmt, ap);
    va_end(ap);
}

static int32_t size_of(parse *p, const gd_json *o, const char *where, const char *key)
{
    int64_t v = 0;
    if (!gd_json_int(gd_json_get(o, key), &v) || v <= 0 || v > SIZE_MAX_I32) {
        fail(p, GD_ERR_BAD_STATE, "%s.%s must be a positive whole number", where, key);
        return 1;
    }
    return (int32_t)v;
}

static double real_of(parse *p, const gd_json *o, const char *where, const char *key)
{
    const gd_json *v = gd_json_get(o, key);
    if (v == NULL || v->type != GD_JSON_NUMBER || !isfinite(v->number)) {
        fail(p, GD_ERR_BAD_STATE, "%s.%s must be a number", where, key);
        return 1.0;
    }
    return v->number;
}

static void parse_mamba2(parse *p, const gd_json *m, const char *where, layer_config *l)
{
    l->mixer = MIXER_MAMBA2;
    l->ssm.heads = (uint32_t)size_of(p, m, where, "heads");
    l->ssm.vdim = (uint32_t)size_of(p, m, where, "vdim");
    l->ssm.state = (uint32_t)size_of(p, m, where, "state");
    l->ssm.groups = (uint32_t)size_of(p, m, where, "groups");
    l->norm_groups = size_of(p, m, where, "norm_groups");
    l->taps = size_of(p, m, where, "conv");
    if (l->ssm.heads % l->ssm.groups != 0U) fail(p, GD_ERR_BAD_STATE, "%s: heads is not a multiple of groups", where);
    if ((int64_t)l->ssm.heads * l->ssm.vdim % l->norm_groups != 0)
        fail(p, GD_ERR_BAD_STATE, "%s: heads * vdim is not a multiple of norm_groups", where);
}

/* rotated dimensions of an attention mixer and their base */
static uint32_t parse_rot(parse *p, const gd_json *m, const char *where, layer_config *l)
{
    const gd_json *rot = gd_json_get(m, "rot");
    const uint32_t dims = (uint32_t)size_of(p, rot, where, "dims");
    l->rot_base = real_of(p, rot, where, "base");
    if (!(l->rot_base > 0.0)) fail(p, GD_ERR_BAD_STATE, "%s.rot.base must be positive", where);
    if (dims % 2U != 0U) fail(p, GD_ERR_BAD_STATE, "%s.rot.dims must be even", where);
    return dims;
}

static void parse_latent(parse *p, const gd_json *m, const char *where, layer_config *l, float eps)
{
    l->mixer = MIXER_LATENT_ATTENTION;
    l->latent.heads = (uint32_t)size_of(p, m, where, "heads");
    l->latent.dim = (uint32_t)size_of(p, m, where, "dim");
    l->latent.rot_dim = (uint32_t)size_of(p, m, where, "rot_dim");
    l->latent.vdim = (uint32_t)size_of(p, m, where, "vdim");
    l->latent.q_rank = (uint32_t)size_of(p, m, where, "q_rank");
    l->latent.kv_rank = (uint32_t)size_of(p, m, where, "kv_rank");
    l->latent.scale = (float)real_of(p, m, where, "scale");
    l->latent.eps = eps;
    if (parse_rot(p, m, where, l) != l->latent.rot_dim) fail(p, GD_ERR_BAD_STATE, "%s: rot.dims must be rot_dim", where);
}

/* query heads in groups that share keys and values; without "mask" every earlier position is seen */
static void parse_grouped(parse *p, const gd_json *m, const char *where, layer_config *l)
{
    const gd_json *scaling = gd_json_get(gd_json_get(m, "rot"), "scaling"), *mask = gd_json_get(m, "mask");
    gd_backend_grouped_args *a = &l->grouped;
    l->mixer = MIXER_GROUPED_ATTENTION;
    a->heads = (uint32_t)size_of(p, m, where, "heads");
    a->kv_heads = (uint32_t)size_of(p, m, where, "kv_heads");
    a->dim = (uint32_t)size_of(p, m, where, "dim");
    a->vdim = (uint32_t)size_of(p, m, where, "vdim");
    a->scale = (float)real_of(p, m, where, "scale");
    a->rot_dims = parse_rot(p, m, where, l);
    a->rot_mult = 1.0f;
    if (mask != NULL && mask->type != GD_JSON_NULL) a->chunk = (uint32_t)size_of(p, mask, where, "size");
    if (a->heads % a->kv_heads != 0U) fail(p, GD_ERR_BAD_STATE, "%s: heads is not a multiple of kv_heads", where);
    if (a->rot_dims > a->dim) fail(p, GD_ERR_BAD_STATE, "%s: rot.dims is more than dim", where);
    if (scaling == NULL || scaling->type == GD_JSON_NULL) return;
    l->scaling.factor = real_of(p, scaling, where, "factor");
    l->scaling.original = real_of(p, scaling, where, "original");
    l->scaling.fast = real_of(p, scaling, where, "fast");
    l->scaling.slow = real_of(p, scaling, where, "slow");
    if (!(l->scaling.factor > 0.0 && l->scaling.original > 0.0 && l->scaling.fast > 0.0 && l->scaling.slow > 0.0) ||
        l->rot_base == 1.0)
        fail(p, GD_ERR_BAD_STATE, "%s.rot.scaling must hold positive numbers", where);
    else a->rot_mult = (float)(0.1 * log(l->scaling.factor) + 1.0);
}

/* "kind": dense, or moe: experts chosen by a table over token ids, with or without a shared expert */
static void parse_square_relu_or_routed(parse *p, const gd_json *mlp, const char *where, int32_t width, layer_config *l)
{
    const gd_json *kind = gd_json_get(mlp, "kind"), *expert, *router, *shared;
    gd_backend_routed_args *a = &l->routed;
    if (kind != NULL && kind->type == GD_JSON_STRING && !strcmp(kind->string, "dense")) {
        l->mlp = MLP_SQUARE_RELU;
        l->ff = size_of(p, mlp, where, "ff");
        return;
    }
    if (kind == NULL || kind->type != GD_JSON_STRING || strcmp(kind->string, "moe") != 0) {
        fail(p, GD_ERR_UNSUPPORTED, "%s.kind must be dense or moe", where);
        return;
    }
    l->mlp = MLP_ROUTED;
    expert = gd_json_get(mlp, "expert");
    router = gd_json_get(mlp, "router");
    shared = gd_json_get(mlp, "shared");
    a->experts = (uint32_t)size_of(p, router, where, "experts");
    a->top = (uint32_t)size_of(p, router, where, "top");
    a->width = (uint32_t)width;
    a->ff = (uint32_t)size_of(p, expert, where, "ff");
    a->gate_limit = (float)real_of(p, expert, where, "limit");
    a->gate_alpha = BONATAR_GATE_ALPHA;
    a->weight = 1.0f / (float)a->top;
    if (a->top > a->experts) fail(p, GD_ERR_BAD_STATE, "%s: top is more than experts", where);
    if (a->experts > GD_BACKEND_ROUTED_MAX_EXPERTS)
        fail(p, GD_ERR_UNSUPPORTED, "%s: more than %u experts", where, GD_BACKEND_ROUTED_MAX_EXPERTS);
    if (shared == NULL || shared->type == GD_JSON_NULL) return;
    l->shared_ff = size_of(p, shared, where, "ff");
    l->shared_limit = (float)real_of(p, shared, where, "limit");
}

/* what every architecture has; the layers are allocated and empty behind it */
static bool parse_model(parse *p, const gd_json *root, layer_list_config *c)
{
    const gd_json *layers = gd_json_get(root, "layers");
    memset(c, 0, sizeof(*c));
    c->vocab = size_of(p, root, "config", "vocab");
    c->width = size_of(p, root, "config", "width");
    c->eps = (float)real_of(p, gd_json_get(root, "norm"), "norm", "eps");
    c->residual_mult = 1.0f;
    c->embedding_scale = (float)real_of(p, gd_json_get(root, "embedding"), "embedding", "scale");
    if (!(c->eps >= 0.0f)) fail(p, GD_ERR_BAD_STATE, "norm.eps must not be negative");
    if (layers == NULL || layers->type != GD_JSON_ARRAY || layers->count == 0U || layers->count > 4096U) {
        fail(p, GD_ERR_BAD_STATE, "layers must be a list");
        return false;
    }
    c->n_layers = (int32_t)layers->count;
    c->layers = (layer_config *)calloc(layers->count, sizeof(layer_config));
    if (c->layers == NULL) fail(p, GD_ERR_OUT_OF_MEMORY, "out of memory");
    return c->layers != NULL;
}

static const char *layer_type(parse *p, const gd_json *v, int32_t i)
{
    const gd_json *type = gd_json_get(v, "type");
    if (type != NULL && type->type == GD_JSON_STRING) return type->string;
    fail(p, GD_ERR_BAD_STATE, "layers[%d].type must be a name", (int)i);
    return "";
}

static gd_status parsed(parse *p, layer_list_config *c)
{
    if (p->st != GD_OK) gd_layer_list_config_free(c);
    return p->st;
}

gd_status gd_layer_list_parse_girirax(const gd_json *root, layer_list_config *c, char *message, size_t message_size)
{
    parse p = {message, message_size, GD_OK};
    const gd_json *v;
    int32_t i = 0;
    if (!parse_model(&p, root, c)) return p.st;
    c->architecture = "Girirax";
    c->residual_mult = (float)real_of(&p, root, "config", "residual_mult");
    for (v = gd_json_get(root, "layers")->child; v != NULL; v = v->next, ++i) {
        const gd_json *mlp = gd_json_get(v, "mlp"), *kind = gd_json_get(mlp, "kind");
        const char *type = layer_type(&p, v, i);
        char where[48];
        layer_config *l = &c->layers[i];
        (void)snprintf(where, sizeof(where), "layers[%d].mixer", (int)i);
        l->weights_of = i;
        if (!strcmp(type, "mamba2")) parse_mamba2(&p, gd_json_get(v, "mixer"), where, l);
        else if (!strcmp(type, "latent_attention")) parse_latent(&p, gd_json_get(v, "mixer"), where, l, c->eps);
        else fail(&p, GD_ERR_UNSUPPORTED, "layers[%d]: no mixer '%s'", (int)i, type);
        if (mlp == NULL || mlp->type == GD_JSON_NULL) continue;
        if (kind == NULL || kind->type != GD_JSON_STRING || strcmp(kind->string, "dense") != 0)
            fail(&p, GD_ERR_UNSUPPORTED, "layers[%d].mlp.kind must be dense", (int)i);
        (void)snprintf(where, sizeof(where), "layers[%d].mlp", (int)i);
        l->mlp = MLP_GELU_GATED;
        l->ff = size_of(&p, mlp, where, "ff");
    }
    return parsed(&p, c);
}

/* layers that use another layer's weights: each is given the one that owns them, and must be of its sizes */
static void resolve_weights(parse *p, layer_list_config *c)
{
    int32_t i, hops;
    for (i = 0; i < c->n_layers; ++i) {
        layer_config a, b;
        int32_t j = i;
        for (hops = 0; c->layers[j].weights_of != j && hops <= c->n_layers; ++hops) j = c->layers[j].weights_of;
        if (c->layers[j].weights_of != j) {
            fail(p, GD_ERR_BAD_STATE, "layers[%d].weights_of leads to no layer with weights", (int)i);
            return;
        }
        memcpy(&a, &c->layers[i], sizeof(a)); /* the whole of both, padding included: they come zeroed */
        memcpy(&b, &c->layers[j], sizeof(b));
        a.weights_of = b.weights_of;
        if (memcmp(&a, &b, sizeof(a)) != 0)
            fail(p, GD_ERR_BAD_STATE, "layers[%d].weights_of names a layer of other sizes", (int)i);
    }
    for (i = 0; i < c->n_layers; ++i) {
        int32_t j = i;
        while (p->st == GD_OK && c->layers[j].weights_of != j) j = c->layers[j].weights_of;
        c->layers[i].weights_of = j;
    }
}

gd_status gd_layer_list_parse_bonatar(const gd_json *root, layer_list_config *c, char *message, size_t message_size)
{
    parse p = {message, message_size, GD_OK};
    const gd_json *v;
    int32_t i = 0;
    if (!parse_model(&p, root, c)) return p.st;
    c->architecture = "Bonatar";
    c->norms_first = true;
    c->norm_offset = 1.0f;
    c->own_head = true;
    for (v = gd_json_get(root, "layers")->child; v != NULL; v = v->next, ++i) {
        const gd_json *mlp = gd_json_get(v, "mlp"), *shares = gd_json_get(v, "weights_of");
        const char *type = layer_type(&p, v, i);
        char where[48];
        int64_t j = i;
        layer_config *l = &c->layers[i];
        (void)snprintf(where, sizeof(where), "layers[%d].mixer", (int)i);
        if (!strcmp(type, "attention")) parse_grouped(&p, gd_json_get(v, "mixer"), where, l);
        else fail(&p, GD_ERR_UNSUPPORTED, "layers[%d]: no mixer '%s'", (int)i, type);
        (void)snprintf(where, sizeof(where), "layers[%d].mlp", (int)i);
        if (mlp != NULL && mlp->type != GD_JSON_NULL) parse_square_relu_or_routed(&p, mlp, where, c->width, l);
        if (shares != NULL && shares->type != GD_JSON_NULL && (!gd_json_int(shares, &j) || j < 0 || j >= c->n_layers)) {
            fail(&p, GD_ERR_BAD_STATE, "layers[%d].weights_of must be the number of a layer", (int)i);
            j = i;
        }
        l->weights_of = (int32_t)j;
    }
    resolve_weights(&p, c);
    return parsed(&p, c);
}

void gd_layer_list_config_free(layer_list_config *c)
{
    free(c->layers);
    c->layers = NULL;
}
