/* config.json of a layer-list decoder -> layer_list_config, every size and constant checked. */
#include <math.h>
#include <stdarg.h>
#include <stdio.h>

#include "layer_list.h"

#define SIZE_MAX_I32 (1 << 28)

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

static void parse_latent(parse *p, const gd_json *m, const char *where, layer_config *l, float eps)
{
    const gd_json *rot = gd_json_get(m, "rot");
    l->mixer = MIXER_LATENT_ATTENTION;
    l->latent.heads = (uint32_t)size_of(p, m, where, "heads");
    l->latent.dim = (uint32_t)size_of(p, m, where, "dim");
    l->latent.rot_dim = (uint32_t)size_of(p, m, where, "rot_dim");
    l->latent.vdim = (uint32_t)size_of(p, m, where, "vdim");
    l->latent.q_rank = (uint32_t)size_of(p, m, where, "q_rank");
    l->latent.kv_rank = (uint32_t)size_of(p, m, where, "kv_rank");
    l->latent.scale = (float)real_of(p, m, where, "scale");
    l->latent.eps = eps;
    l->rot_base = real_of(p, rot, where, "base");
    if (!(l->rot_base > 0.0)) fail(p, GD_ERR_BAD_STATE, "%s.rot.base must be positive", where);
    if ((uint32_t)size_of(p, rot, where, "dims") != l->latent.rot_dim || l->latent.rot_dim % 2U != 0U)
        fail(p, GD_ERR_BAD_STATE, "%s: rot.dims must be rot_dim, an even number", where);
}

gd_status gd_layer_list_parse(const gd_json *root, layer_list_config *c, char *message, size_t message_size)
{
    parse p = {message, message_size, GD_OK};
    const gd_json *layers = gd_json_get(root, "layers"), *v;
    int32_t i = 0;
    memset(c, 0, sizeof(*c));
    c->vocab = size_of(&p, root, "config", "vocab");
    c->width = size_of(&p, root, "config", "width");
    c->eps = (float)real_of(&p, gd_json_get(root, "norm"), "norm", "eps");
    c->residual_mult = (float)real_of(&p, root, "config", "residual_mult");
    c->embedding_scale = (float)real_of(&p, gd_json_get(root, "embedding"), "embedding", "scale");
    if (!(c->eps >= 0.0f)) fail(&p, GD_ERR_BAD_STATE, "norm.eps must not be negative");
    if (layers == NULL || layers->type != GD_JSON_ARRAY || layers->count == 0U || layers->count > 4096U) {
        fail(&p, GD_ERR_BAD_STATE, "layers must be a list");
        return p.st;
    }
    c->n_layers = (int32_t)layers->count;
    c->layers = (layer_config *)calloc(layers->count, sizeof(layer_config));
    if (c->layers == NULL) return GD_ERR_OUT_OF_MEMORY;
    for (v = layers->child; v != NULL; v = v->next, ++i) {
        const gd_json *type = gd_json_get(v, "type"), *mlp = gd_json_get(v, "mlp"), *kind = gd_json_get(mlp, "kind");
        char where[48];
        layer_config *l = &c->layers[i];
        (void)snprintf(where, sizeof(where), "layers[%d].mixer", (int)i);
        if (type == NULL || type->type != GD_JSON_STRING) {
            fail(&p, GD_ERR_BAD_STATE, "layers[%d].type must be a name", (int)i);
            continue;
        }
        if (!strcmp(type->string, "mamba2")) parse_mamba2(&p, gd_json_get(v, "mixer"), where, l);
        else if (!strcmp(type->string, "latent_attention")) parse_latent(&p, gd_json_get(v, "mixer"), where, l, c->eps);
        else fail(&p, GD_ERR_UNSUPPORTED, "layers[%d]: no mixer '%s'", (int)i, type->string);
        if (mlp == NULL || mlp->type == GD_JSON_NULL) continue;
        if (kind == NULL || kind->type != GD_JSON_STRING || strcmp(kind->string, "dense") != 0)
            fail(&p, GD_ERR_UNSUPPORTED, "layers[%d].mlp.kind must be dense", (int)i);
        (void)snprintf(where, sizeof(where), "layers[%d].mlp", (int)i);
        l->ff = size_of(&p, mlp, where, "ff");
    }
    if (p.st != GD_OK) gd_layer_list_config_free(c);
    return p.st;
}

void gd_layer_list_config_free(layer_list_config *c)
{
    free(c->layers);
    c->layers = NULL;
}
