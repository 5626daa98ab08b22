/* The architectures this library serves and how each is opened (gd_model.h). */
#include <stdio.h>
#include <sys/stat.h>

#include "gd_checkpoint.h"
#include "layer_list.h"

typedef struct architecture architecture;

struct gd_model {
    const architecture *arch;
    /* gpt_lm */
    char *path;
    gd_gpt_config gpt;
    /* layer lists */
    layer_list_config layers;
    gd_safetensors *weights; /* NULL: drawn from seed */
    uint64_t seed;
};

struct architecture {
    const char *name;
    gd_status (*configure)(gd_model *m, const gd_json *root, char *message, size_t size); /* folders only */
    gd_status (*memory)(const gd_model *m, const gd_model_options *o, gd_memory_config *out);
    gd_status (*create)(gd_context *ctx, gd_model *m, const gd_model_options *o, gd_gpt_decoder **out);
};

/* ---- gpt_lm: a checkpoint of the reference's example --------------------------------------------- */

static void gpt_options(const gd_model *m, const gd_model_options *o, gd_gpt_config *c)
{
    *c = m->gpt;
    if (o->max_seq > 0) c->max_seq = o->max_seq;
    c->batch = o->batch > 0 ? o->batch : 1;
}

static gd_status gpt_config(const gd_model *m, const gd_model_options *o, gd_gpt_config *c)
{
    gpt_options(m, o, c);
    if (o->heads > 0) { /* the file may not say: read it once more with the caller's value */
        c->n_heads = o->heads;
        c->head_dim = 0;
    }
    TRY(gd_gpt_config_from_checkpoint(m->path, c));
    return c->max_seq > 0 ? GD_OK : GD_ERR_INVALID_ARGUMENT;
}

static gd_status gpt_memory(const gd_model *m, const gd_model_options *o, gd_memory_config *out)
{
    gd_gpt_config c;
    int64_t rows;
    TRY(gpt_config(m, o, &c));
    rows = o->max_step_tokens > 0 ? o->max_step_tokens : (int64_t)c.batch * c.max_seq;
    if (rows > INT32_MAX) rows = INT32_MAX;
    *out = gd_memory_config_default();
    out->params_bytes = gd_gpt_params_bytes(&c);
    out->state_bytes = gd_gpt_state_bytes(&c);
    out->scratch_slot_bytes = gd_gpt_scratch_bytes(&c, (int32_t)rows);
    out->data_slot_bytes = (size_t)(16 * rows) + ((size_t)1 << 20);
    return GD_OK;
}

static gd_status gpt_create(gd_context *ctx, gd_model *m, const gd_model_options *o, gd_gpt_decoder **out)
{
    gd_gpt_config c;
    gd_status st;
    TRY(gpt_config(m, o, &c));
    TRY(gd_gpt_decoder_create(ctx, &c, out));
    st = gd_gpt_decoder_load_checkpoint(*out, m->path, 1);
    if (st == GD_OK) return GD_OK;
    gd_gpt_decoder_destroy(*out);
    *out = NULL;
    return st;
}

/* ---- layer lists ------------------------------------------------------------------------------------- */

static gd_status girirax_configure(gd_model *m, const gd_json *root, char *message, size_t size)
{
    return gd_layer_list_parse_girirax(root, &m->layers, message, size);
}

static gd_status bonatar_configure(gd_model *m, const gd_json *root, char *message, size_t size)
{
    return gd_layer_list_parse_bonatar(root, &m->layers, message, size);
}

static gd_status layers_memory(const gd_model *m, const gd_model_options *o, gd_memory_config *out)
{
    return gd_layer_list_memory(&m->layers, o, out);
}

static gd_status layers_create(gd_context *ctx, gd_model *m, const gd_model_options *o, gd_gpt_decoder **out)
{
    return gd_layer_list_create(ctx, &m->layers, o, m->weights, m->seed, out);
}

static const architecture architectures[] = {
    {"gpt_lm", NULL, gpt_memory, gpt_create},
    {"Girirax", girirax_configure, layers_memory, layers_create},
    {"Bonatar", bonatar_configure, layers_memory, layers_create},
};

/* ---- opening ------------------------------------------------------------------------------------------- */

static void say(char *message, size_t size, const char *text)
{
    if (message != NULL && size > 0U) (void)snprintf(message, size, "%s", text);
}

static gd_status configure(gd_model *m, const char *text, size_t len, char *message, size_t size)
{
    gd_json_doc doc;
    const gd_json *name;
    gd_status st = GD_ERR_UNSUPPORTED;
    size_t i;
    if (!gd_json_parse(text, len, &doc)) {
        say(message, size, "config.json is not JSON");
        return GD_ERR_BAD_STATE;
    }
    name = gd_json_get(doc.root, "architecture");
    if (name == NULL || name->type != GD_JSON_STRING) {
        say(message, size, "config.json has no architecture");
        st = GD_ERR_BAD_STATE;
    } else {
        for (i = 0; i < sizeof(architectures) / sizeof(architectures[0]); ++i) {
            if (architectures[i].configure != NULL && !strcmp(architectures[i].name, name->string))
                m->arch = &architectures[i];
        }
        if (m->arch == NULL) say(message, size, "config.json names an architecture this library does not have");
        else st = m->arch->configure(m, doc.root, message, size);
    }
    gd_json_free(&doc);
    return st;
}

static gd_status open_folder(gd_model *m, const char *path, char *message, size_t size)
{
    const size_t n = strlen(path) + 32U;
    char *file = (char *)malloc(n), *text = NULL;
    FILE *f;
    long len;
    gd_status st = GD_ERR_IO;
    if (file == NULL) return GD_ERR_OUT_OF_MEMORY;
    (void)snprintf(file, n, "%s/config.json", path);
    f = fopen(file, "rb");
    if (f != NULL && fseek(f, 0, SEEK_END) == 0 && (len = ftell(f)) >= 0 && len < (64 << 20)) {
        rewind(f);
        text = (char *)malloc((size_t)len + 1U);
        if (text != NULL && fread(text, 1, (size_t)len, f) == (size_t)len) st = configure(m, text, (size_t)len, message, size);
    }
    if (st == GD_ERR_IO) say(message, size, "config.json cannot be read");
    if (f != NULL) fclose(f);
    free(text);
    if (st == GD_OK) {
        (void)snprintf(file, n, "%s/model.safetensors", path);
        st = gd_safetensors_open(file, &m->weights);
        if (st != GD_OK) say(message, size, "model.safetensors cannot be read");
    }
    free(file);
    return st;
}

gd_status gd_model_open(const char *path, gd_model **out, char *message, size_t message_size)
{
    struct stat info;
    gd_model *m;
    gd_status st;
    if (message != NULL && message_size > 0U) message[0] = '\0';
    if (out != NULL) *out = NULL;
    if (path == NULL || out == NULL) return GD_ERR_INVALID_ARGUMENT;
    if (stat(path, &info) != 0) {
        say(message, message_size, "no such file or folder");
        return GD_ERR_IO;
    }
    m = (gd_model *)calloc(1, sizeof(*m));
    if (m == NULL) return GD_ERR_OUT_OF_MEMORY;
    if (S_ISDIR(info.st_mode)) {
        st = open_folder(m, path, message, message_size);
    } else {
        m->arch = &architectures[0];
        m->path = strdup(path);
        m->gpt.batch = 1;
        m->gpt.rms_eps = 1.0e-5f;
        m->gpt.rope_theta = 10000.0f;
        st = m->path == NULL ? GD_ERR_OUT_OF_MEMORY : gd_gpt_config_from_checkpoint(path, &m->gpt);
        /* a checkpoint that does not tell its heads is opened all the same: options.heads completes it */
        if (st == GD_ERR_BAD_STATE && m->gpt.d_model > 0 && m->gpt.n_heads <= 0) st = GD_OK;
        if (st != GD_OK) say(message, message_size, "not a checkpoint of the gpt_lm example");
    }
    if (st != GD_OK) {
        gd_model_close(m);
        return st;
    }
    *out = m;
    return GD_OK;
}

gd_status gd_model_open_config(const char *config_json, uint64_t seed, gd_model **out, char *message,
                               size_t message_size)
{
    gd_model *m;
    gd_status st;
    if (message != NULL && message_size > 0U) message[0] = '\0';
    if (out != NULL) *out = NULL;
    if (config_json == NULL || out == NULL) return GD_ERR_INVALID_ARGUMENT;
    m = (gd_model *)calloc(1, sizeof(*m));
    if (m == NULL) return GD_ERR_OUT_OF_MEMORY;
    m->seed = seed;
    st = configure(m, config_json, strlen(config_json), message, message_size);
    if (st != GD_OK) {
        gd_model_close(m);
        return st;
    }
    *out = m;
    return GD_OK;
}

void gd_model_close(gd_model *m)
{
    if (m == NULL) return;
    gd_safetensors_close(m->weights);
    gd_layer_list_config_free(&m->layers);
    free(m->path);
    free(m);
}

const char *gd_model_architecture(const gd_model *m) { return m != NULL ? m->arch->name : NULL; }
int32_t gd_model_vocab(const gd_model *m) { return m == NULL ? 0 : m->path != NULL ? m->gpt.vocab : m->layers.vocab; }
int32_t gd_model_layers(const gd_model *m)
{
    return m == NULL ? 0 : m->path != NULL ? m->gpt.n_layers : m->layers.n_layers;
}

gd_status gd_model_memory(const gd_model *m, const gd_model_options *options, gd_memory_config *out)
{
    if (m == NULL || options == NULL || out == NULL) return GD_ERR_INVALID_ARGUMENT;
    return m->arch->memory(m, options, out);
}

gd_status gd_model_create_decoder(gd_context *ctx, gd_model *m, const gd_model_options *options, gd_gpt_decoder **out)
{
    if (out != NULL) *out = NULL;
    if (ctx == NULL || m == NULL || options == NULL || out == NULL) return GD_ERR_INVALID_ARGUMENT;
    return m->arch->create(ctx, m, options, out);
}
