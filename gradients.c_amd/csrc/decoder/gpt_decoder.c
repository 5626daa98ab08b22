/*
 * Decoder-only language model of the reference's example, inference part, with run-time
 * dimensions.  The operator order, residual wiring and cache bookkeeping restate
 * examples/gpt_lm/gpt_lm_shared.c of the reference: gpt_block_decode_cached (:961-1071),
 * gpt_lm_decode_logits (:1204-1246), gpt_block_prefill_cached (:825-959),
 * gpt_lm_prefill_last_logits (:1174-1202), gpt_kv_cache_init (:480-538) and the weight
 * initialisation (:196-218, 290-402).  Everything goes through the public gd_* operators.
 */
#include <math.h>
#include <stdlib.h>
#include <string.h>

#include <stdio.h>

#include "gd_checkpoint.h"
#include "decoder_internal.h"

typedef struct gpt_linear {
    gd_tensor weight, bias;
    bool transposed; /* weight stored [out, in] */
} gpt_linear;

typedef struct gpt_block {
    gd_tensor attn_norm_w, mlp_norm_w;
    gpt_linear qkv_proj, attn_proj, up_gate, down_proj;
    /* the down projection's weight once more as [d_model, hidden] (the reference keeps it [hidden, d_model]): with
     * few rows the projection streams the weight once, and rows that are contiguous along the summed dimension
     * come in whole cache lines per workgroup; a 16-column slice of the [K,N] layout uses a quarter of every line */
    gd_tensor down_t;
} gpt_block;

/* ---- deterministic initialisation (reference :32-48, 196-218) ----------------------- */

/* Draw number n (1-based) of the stream started at `seed`: the state advances by a constant, so any draw
 * is addressable and the fill below can run in parallel and still equal the reference's sequential loop. */
static double uniform_open_closed_at(uint64_t seed, uint64_t n)
{
    return ((double)(gd_mix64(seed + n * UINT64_C(0x9e3779b97f4a7c15)) >> 11) + 1.0) * (1.0 / 9007199254740992.0);
}

/* twin != NULL: t is [rows, cols]; the same values also go to twin as [cols, rows] */
static gd_status init_normal_twin(gd_context *ctx, gd_tensor *t, uint64_t seed, float stddev, gd_tensor *twin,
                                  int64_t rows, int64_t cols)
{
    int64_t n, pairs, pi;
    float *values;
    gd_status st;
    TRY(gd_tensor_numel(t, &n));
    values = (float *)malloc((size_t)n * sizeof(float));
    if (values == NULL) return GD_ERR_OUT_OF_MEMORY;
    pairs = (n + 1) / 2;
#pragma omp parallel for schedule(static)
    for (pi = 0; pi < pairs; ++pi) {
        const double u1 = uniform_open_closed_at(seed, 2U * (uint64_t)pi + 1U);
        const double u2 = uniform_open_closed_at(seed, 2U * (uint64_t)pi + 2U);
        const double radius = sqrt(-2.0 * log(u1)), angle = 6.283185307179586476925286766559 * u2;
        values[2 * pi] = (float)(radius * cos(angle) * (double)stddev);
        if (2 * pi + 1 < n) values[2 * pi + 1] = (float)(radius * sin(angle) * (double)stddev);
    }
    st = gd_tensor_write_f32(ctx, t, values, (size_t)n);
    if (st == GD_OK && twin != NULL) {
        float *turned = (float *)malloc((size_t)n * sizeof(float));
        int64_t r;
        if (turned == NULL) {
            free(values);
            return GD_ERR_OUT_OF_MEMORY;
        }
#pragma omp parallel for schedule(static)
        for (r = 0; r < cols; ++r) {
            int64_t c;
            for (c = 0; c < rows; ++c) turned[r * rows + c] = values[c * cols + r];
        }
        st = gd_tensor_write_f32(ctx, twin, turned, (size_t)n);
        free(turned);
    }
    free(values);
    return st;
}

static gd_status init_normal(gd_context *ctx, gd_tensor *t, uint64_t seed, float stddev)
{
    return init_normal_twin(ctx, t, seed, stddev, NULL, 0, 0);
}

static gd_status param(gd_context *ctx, gd_dtype dtype, uint32_t rank, int64_t d0, int64_t d1, gd_tensor *out)
{
    int64_t dims[2] = {d0, d1};
    return gd_tensor_empty(ctx, GD_ARENA_PARAMS, dtype, gd_shape_make(rank, dims), 256U, out);
}

static gd_status linear_init(gd_context *ctx, gpt_linear *l, int64_t in, int64_t out, bool transposed, uint64_t seed,
                             float stddev)
{
    l->transposed = transposed;
    TRY(param(ctx, GD_DTYPE_F16, 2U, transposed ? out : in, transposed ? in : out, &l->weight));
    TRY(init_normal(ctx, &l->weight, seed, stddev));
    TRY(param(ctx, GD_DTYPE_F16, 1U, out, 0, &l->bias));
    return gd_tensor_zero_(ctx, &l->bias);
}

static gd_status ones_param(gd_context *ctx, int64_t n, gd_tensor *out)
{
    int64_t dims[1] = {n};
    return gd_tensor_ones(ctx, GD_ARENA_PARAMS, GD_DTYPE_F16, gd_shape_make(1U, dims), 256U, out);
}

size_t gd_gpt_params_bytes(const gd_gpt_config *c)
{
    const size_t Dm = (size_t)c->d_model, Hm = (size_t)c->mlp_hidden, V = (size_t)c->vocab;
    size_t per_layer = 2U * gd_pad256(Dm * 2U) + gd_pad256(3U * Dm * Dm * 2U) + gd_pad256(3U * Dm * 2U) + gd_pad256(Dm * Dm * 2U) +
                       gd_pad256(Dm * 2U) + gd_pad256(2U * Hm * Dm * 2U) + gd_pad256(2U * Hm * 2U) + 2U * gd_pad256(Hm * Dm * 2U) +
                       gd_pad256(Dm * 2U);
    size_t total = gd_pad256(V * Dm * 2U) * (c->tie_lm_head ? 1U : 2U) + gd_pad256(V * 2U) + gd_pad256(Dm * 2U);
    return total + per_layer * (size_t)c->n_layers + 4096U;
}

size_t gd_gpt_state_bytes(const gd_gpt_config *c)
{
    const size_t cache = gd_pad256((size_t)c->batch * (size_t)c->max_seq * (size_t)c->n_heads * (size_t)c->head_dim * 2U);
    return cache * 2U * (size_t)c->n_layers + gd_decoder_session_bytes(c, GD_DTYPE_F16, true) + 4096U;
}

size_t gd_gpt_scratch_bytes(const gd_gpt_config *c, int32_t max_prefill_tokens)
{
    /* every operator output of every layer lives until the step ends (bump allocation): 13 d_model-wide and one
     * 2 x hidden-wide F16 tensor per layer and row, each padded to 256 bytes; 10 % slack; one transient activation of
     * the many-row swiglu path; logits, picks and records; 64 MiB for everything small */
    const size_t rows = (size_t)(max_prefill_tokens > c->batch ? max_prefill_tokens : c->batch);
    const size_t picked = c->m3_block_size > 0 ? (size_t)c->n_heads * 16U * 4U + 256U : 0U; /* block ids of a row */
    const size_t per_row = 2U * (13U * (size_t)c->d_model + 2U * (size_t)c->mlp_hidden) + 14U * 256U + picked;
    const size_t layers = rows * per_row * (size_t)c->n_layers;
    const size_t angles = (rows + 32U) * ((size_t)c->head_dim * 4U + 4U) + 3U * 256U; /* cos, sin and cache row per prompt row */
    return layers + layers / 10U + rows * ((size_t)c->d_model * 4U + (size_t)c->mlp_hidden * 2U) + angles +
           (size_t)c->batch * (size_t)c->vocab * 4U + ((size_t)64 << 20);
}

static const gd_decoder_model gpt_model;

gd_status gd_gpt_decoder_create(gd_context *ctx, const gd_gpt_config *cfg, gd_gpt_decoder **out)
{
    gd_gpt_decoder *d;
    const float std = 0.02f;
    float resid;
    int32_t l;
    int64_t cache_dims[4];
    gd_status st = GD_OK;
    if (out != NULL) *out = NULL;
    if (ctx == NULL || cfg == NULL || out == NULL || cfg->vocab <= 0 || cfg->d_model <= 0 || cfg->n_layers <= 0 ||
        cfg->n_heads <= 0 || cfg->head_dim <= 0 || cfg->mlp_hidden <= 0 || cfg->max_seq <= 0 || cfg->batch <= 0 ||
        cfg->n_heads * cfg->head_dim != cfg->d_model || cfg->sdpa_window < 0 || cfg->m3_block_size < 0 ||
        cfg->m3_block_size > 128 || cfg->m3_topk_blocks < 0 || cfg->m3_topk_blocks > 16 || cfg->m3_init_blocks < 0 ||
        cfg->m3_local_blocks < 0 || (cfg->m3_block_size > 0 && cfg->head_dim > 64))
        return GD_ERR_INVALID_ARGUMENT;
    TRY(gd_decoder_session_create(ctx, &gpt_model, cfg, &d));
    if (!(d->cfg.rms_eps > 0.0f)) d->cfg.rms_eps = 1.0e-5f;
    if (!(d->cfg.rope_theta > 0.0f)) d->cfg.rope_theta = 10000.0f;
    d->blocks = (gpt_block *)calloc((size_t)cfg->n_layers, sizeof(gpt_block));
    d->k_cache = (gd_tensor *)calloc((size_t)cfg->n_layers, sizeof(gd_tensor));
    d->v_cache = (gd_tensor *)calloc((size_t)cfg->n_layers, sizeof(gd_tensor));
    if (d->blocks == NULL || d->k_cache == NULL || d->v_cache == NULL) {
        gd_gpt_decoder_destroy(d);
        return GD_ERR_OUT_OF_MEMORY;
    }
    resid = std / sqrtf(2.0f * (float)cfg->n_layers);
#define STEP(expr) do { if (st == GD_OK) st = (expr); } while (0)
    STEP(param(ctx, GD_DTYPE_F16, 2U, cfg->vocab, cfg->d_model, &d->token_embedding));
    STEP(init_normal(ctx, &d->token_embedding, gd_splitmix64(cfg->seed ^ UINT64_C(0xabc001)), std));
    if (cfg->tie_lm_head) {
        d->lm_head = d->token_embedding;
    } else {
        STEP(param(ctx, GD_DTYPE_F16, 2U, cfg->vocab, cfg->d_model, &d->lm_head));
        STEP(init_normal(ctx, &d->lm_head, gd_splitmix64(cfg->seed ^ UINT64_C(0xabc002)), std));
    }
    STEP(param(ctx, GD_DTYPE_F16, 1U, cfg->vocab, 0, &d->lm_head_bias));
    STEP(gd_tensor_zero_(ctx, &d->lm_head_bias));
    STEP(ones_param(ctx, cfg->d_model, &d->final_norm_w));
    cache_dims[0] = cfg->batch;
    cache_dims[1] = cfg->max_seq;
    cache_dims[2] = cfg->n_heads;
    cache_dims[3] = cfg->head_dim;
    for (l = 0; l < cfg->n_layers && st == GD_OK; ++l) {
        gpt_block *b = &d->blocks[l];
        const uint64_t bs = cfg->seed ^ ((uint64_t)l << 8);
        STEP(ones_param(ctx, cfg->d_model, &b->attn_norm_w));
        STEP(ones_param(ctx, cfg->d_model, &b->mlp_norm_w));
        STEP(linear_init(ctx, &b->qkv_proj, cfg->d_model, 3 * (int64_t)cfg->d_model, true, gd_splitmix64(bs ^ 1U), std));
        STEP(linear_init(ctx, &b->attn_proj, cfg->d_model, cfg->d_model, true, gd_splitmix64(bs ^ 2U), resid));
        STEP(linear_init(ctx, &b->up_gate, cfg->d_model, 2 * (int64_t)cfg->mlp_hidden, true, gd_splitmix64(bs ^ 3U), std));
        b->down_proj.transposed = false;
        STEP(param(ctx, GD_DTYPE_F16, 2U, cfg->mlp_hidden, cfg->d_model, &b->down_proj.weight));
        STEP(param(ctx, GD_DTYPE_F16, 2U, cfg->d_model, cfg->mlp_hidden, &b->down_t));
        STEP(init_normal_twin(ctx, &b->down_proj.weight, gd_splitmix64(bs ^ 4U), resid, &b->down_t, cfg->mlp_hidden,
                              cfg->d_model));
        STEP(param(ctx, GD_DTYPE_F16, 1U, cfg->d_model, 0, &b->down_proj.bias));
        STEP(gd_tensor_zero_(ctx, &b->down_proj.bias));
        STEP(gd_tensor_zeros(ctx, GD_ARENA_STATE, GD_DTYPE_F16, gd_shape_make(4U, cache_dims), 256U, &d->k_cache[l]));
        STEP(gd_tensor_zeros(ctx, GD_ARENA_STATE, GD_DTYPE_F16, gd_shape_make(4U, cache_dims), 256U, &d->v_cache[l]));
    }
    STEP(gd_decoder_session_allocate(d, GD_DTYPE_F16, true));
#undef STEP
    if (st != GD_OK) {
        gd_gpt_decoder_destroy(d);
        return st;
    }
    *out = d;
    return GD_OK;
}

static void gpt_destroy(gd_gpt_decoder *d)
{
    free(d->blocks);
    free(d->k_cache);
    free(d->v_cache);
}

static gd_tensor *gpt_tensor(gd_gpt_decoder *d, const char *name, int32_t layer)
{
    gpt_block *b;
    if (!strcmp(name, "embed")) return &d->token_embedding;
    if (!strcmp(name, "lm_head")) return &d->lm_head;
    if (!strcmp(name, "lm_bias")) return &d->lm_head_bias;
    if (!strcmp(name, "final_norm")) return &d->final_norm_w;
    if (layer < 0 || layer >= d->cfg.n_layers) return NULL;
    b = &d->blocks[layer];
    if (!strcmp(name, "attn_norm")) return &b->attn_norm_w;
    if (!strcmp(name, "mlp_norm")) return &b->mlp_norm_w;
    if (!strcmp(name, "w_qkv")) return &b->qkv_proj.weight;
    if (!strcmp(name, "b_qkv")) return &b->qkv_proj.bias;
    if (!strcmp(name, "w_attn")) return &b->attn_proj.weight;
    if (!strcmp(name, "b_attn")) return &b->attn_proj.bias;
    if (!strcmp(name, "w_upgate")) return &b->up_gate.weight;
    if (!strcmp(name, "b_upgate")) return &b->up_gate.bias;
    if (!strcmp(name, "w_down")) return &b->down_proj.weight;
    if (!strcmp(name, "w_down_t")) return &b->down_t;
    if (!strcmp(name, "b_down")) return &b->down_proj.bias;
    if (!strcmp(name, "k_cache")) return &d->k_cache[layer];
    if (!strcmp(name, "v_cache")) return &d->v_cache[layer];
    return NULL;
}

/* ---- weights from a checkpoint of the reference ------------------------------------------ */

typedef struct ckpt_slot {
    char path[GD_CHECKPOINT_PATH_MAX];
    gd_tensor *dst, *second; /* second: another tensor that receives the same values (untied LM head) */
    gd_tensor *turned;       /* [cols, rows] copy of a [rows, cols] weight */
    const gd_checkpoint_entry *entry;
} ckpt_slot;

static void slot_set(ckpt_slot *s, gd_tensor *dst, const char *fmt, int32_t layer)
{
    memset(s, 0, sizeof(*s));
    (void)snprintf(s->path, sizeof(s->path), fmt, (int)layer);
    s->dst = dst;
}

/* same test as the reference's gd_ckpt_file_entry_matches_tensor (src/nn/module_io.c:809-824) */
static bool entry_fits(const gd_checkpoint_entry *e, const gd_tensor *t)
{
    size_t nbytes = 0U;
    uint32_t i;
    if (gd_tensor_logical_nbytes(t, &nbytes) != GD_OK || e->dtype != t->dtype || e->rank != t->rank ||
        e->nbytes != (uint64_t)nbytes)
        return false;
    for (i = 0U; i < t->rank; ++i) {
        if (e->shape[i] != t->shape[i]) return false;
    }
    return true;
}

gd_status gd_gpt_decoder_load_checkpoint(gd_gpt_decoder *d, const char *path, int32_t strict)
{
    gd_checkpoint *ck = NULL;
    ckpt_slot *slots;
    unsigned char *bytes = NULL, *flipped = NULL;
    size_t n_slots, capacity = 0U, si;
    uint32_t fi;
    int32_t l;
    gd_status st;
    if (d == NULL || path == NULL || path[0] == '\0' || d->model != &gpt_model) return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BUSY;
    /* the names gpt_lm_init gives its parameters (gpt_lm_shared.c:272-279, 303-338, 382-413) */
    n_slots = 3U + 10U * (size_t)d->cfg.n_layers;
    slots = (ckpt_slot *)calloc(n_slots, sizeof(*slots));
    if (slots == NULL) return GD_ERR_OUT_OF_MEMORY;
    slot_set(&slots[0], &d->token_embedding, "gpt_lm.token_embedding", 0);
    if (!d->cfg.tie_lm_head) slots[0].second = &d->lm_head; /* the reference's head is the embedding table */
    slot_set(&slots[1], &d->lm_head_bias, "gpt_lm.lm_head_bias", 0);
    slot_set(&slots[2], &d->final_norm_w, "gpt_lm.final_norm_w", 0);
    for (l = 0; l < d->cfg.n_layers; ++l) {
        gpt_block *b = &d->blocks[l];
        ckpt_slot *s = &slots[3U + 10U * (size_t)l];
        slot_set(&s[0], &b->attn_norm_w, "gpt_lm.blocks.%d.attn_norm_w", l);
        slot_set(&s[1], &b->mlp_norm_w, "gpt_lm.blocks.%d.mlp_norm_w", l);
        slot_set(&s[2], &b->qkv_proj.weight, "gpt_lm.blocks.%d.qkv_proj.weight", l);
        slot_set(&s[3], &b->qkv_proj.bias, "gpt_lm.blocks.%d.qkv_proj.bias", l);
        slot_set(&s[4], &b->attn_proj.weight, "gpt_lm.blocks.%d.attn_proj.weight", l);
        slot_set(&s[5], &b->attn_proj.bias, "gpt_lm.blocks.%d.attn_proj.bias", l);
        slot_set(&s[6], &b->up_gate.weight, "gpt_lm.blocks.%d.up_gate.weight", l);
        slot_set(&s[7], &b->up_gate.bias, "gpt_lm.blocks.%d.up_gate.bias", l);
        slot_set(&s[8], &b->down_proj.weight, "gpt_lm.blocks.%d.down_proj.weight", l);
        s[8].turned = &b->down_t;
        slot_set(&s[9], &b->down_proj.bias, "gpt_lm.blocks.%d.down_proj.bias", l);
    }
    st = gd_checkpoint_open(path, &ck);
    /* everything is checked before the first byte is written (module_io.c:868-899): a refused file leaves the
     * decoder's weights as they were */
    for (fi = 0U; st == GD_OK && fi < gd_checkpoint_count(ck); ++fi) {
        const gd_checkpoint_entry *e = gd_checkpoint_entry_at(ck, fi);
        ckpt_slot *hit = NULL;
        if (e->flags == GD_CHECKPOINT_ENTRY_BUFFER) continue; /* the decoder registers no buffers */
        for (si = 0U; si < n_slots; ++si) {
            if (strcmp(slots[si].path, e->path) == 0) {
                hit = &slots[si];
                break;
            }
        }
        if (hit == NULL) {
            if (strict) st = GD_ERR_BAD_STATE; /* unexpected tensor */
            continue;
        }
        if (!entry_fits(e, hit->dst)) {
            st = GD_ERR_BAD_STATE; /* dtype, rank, shape or size differ */
            break;
        }
        hit->entry = e;
        if ((size_t)e->nbytes > capacity) capacity = (size_t)e->nbytes;
    }
    for (si = 0U; st == GD_OK && strict && si < n_slots; ++si) {
        if (slots[si].entry == NULL) st = GD_ERR_BAD_STATE; /* missing tensor */
    }
    if (st == GD_OK && capacity > 0U) {
        bytes = (unsigned char *)malloc(capacity);
        flipped = (unsigned char *)malloc(capacity);
        if (bytes == NULL || flipped == NULL) st = GD_ERR_OUT_OF_MEMORY;
    }
    for (si = 0U; st == GD_OK && si < n_slots; ++si) {
        const ckpt_slot *s = &slots[si];
        size_t nbytes;
        if (s->entry == NULL) continue;
        nbytes = (size_t)s->entry->nbytes;
        st = gd_checkpoint_read(ck, s->entry, 0U, bytes, nbytes);
        if (st == GD_OK) st = gd_tensor_write(d->ctx, s->dst, bytes, nbytes);
        if (st == GD_OK && s->second != NULL) st = gd_tensor_write(d->ctx, s->second, bytes, nbytes);
        if (st == GD_OK && s->turned != NULL) {
            const int64_t rows = s->dst->shape[0], cols = s->dst->shape[1];
            const uint16_t *src = (const uint16_t *)bytes;
            uint16_t *out = (uint16_t *)flipped;
            int64_t c;
#pragma omp parallel for schedule(static)
            for (c = 0; c < cols; ++c) {
                int64_t r;
                for (r = 0; r < rows; ++r) out[c * rows + r] = src[r * cols + c];
            }
            st = gd_tensor_write(d->ctx, s->turned, flipped, nbytes);
        }
    }
    free(bytes);
    free(flipped);
    gd_checkpoint_close(ck);
    free(slots);
    return st;
}

/* value of "key=value" on a line of its own in the metadata blob, as the reference's inference programs look it
 * up (examples/gpt_lm/infer.c:344-376); false if absent or not a whole non-negative number that fits an int32 */
static bool metadata_i32(const char *blob, size_t len, const char *key, int32_t *out)
{
    const size_t key_len = strlen(key);
    size_t at = 0U;
    while (at < len) {
        size_t end = at;
        while (end < len && blob[end] != '\n') ++end;
        if (end > at + key_len && strncmp(blob + at, key, key_len) == 0 && blob[at + key_len] == '=') {
            int64_t v = 0;
            size_t i = at + key_len + 1U;
            if (i == end) return false;
            for (; i < end; ++i) {
                if (blob[i] < '0' || blob[i] > '9') return false;
                v = v * 10 + (blob[i] - '0');
                if (v > INT32_MAX) return false;
            }
            *out = (int32_t)v;
            return true;
        }
        at = end < len ? end + 1U : end;
    }
    return false;
}

gd_status gd_gpt_config_from_checkpoint(const char *path, gd_gpt_config *cfg)
{
    gd_checkpoint *ck = NULL;
    const gd_checkpoint_entry *embed, *down;
    char *blob = NULL;
    size_t blob_len = 0U;
    int32_t layers = 0, v;
    uint32_t i;
    gd_status st;
    if (path == NULL || cfg == NULL) return GD_ERR_INVALID_ARGUMENT;
    st = gd_checkpoint_open(path, &ck);
    if (st != GD_OK) return st;
    /* the directory fixes vocabulary, width, MLP width and depth */
    embed = gd_checkpoint_find(ck, "gpt_lm.token_embedding");
    down = gd_checkpoint_find(ck, "gpt_lm.blocks.0.down_proj.weight");
    for (i = 0U; i < gd_checkpoint_count(ck); ++i) {
        const char *p = gd_checkpoint_entry_at(ck, i)->path;
        int n = -1, used = 0;
        if (sscanf(p, "gpt_lm.blocks.%d.attn_norm_w%n", &n, &used) == 1 && used > 0 && p[used] == '\0' && n >= layers)
            layers = n + 1;
    }
    if (embed == NULL || down == NULL || embed->rank != 2U || down->rank != 2U || layers <= 0 ||
        embed->shape[0] > INT32_MAX || embed->shape[1] > INT32_MAX || down->shape[0] > INT32_MAX ||
        down->shape[1] != embed->shape[1]) {
        gd_checkpoint_close(ck);
        return GD_ERR_BAD_STATE;
    }
    cfg->vocab = (int32_t)embed->shape[0];
    cfg->d_model = (int32_t)embed->shape[1];
    cfg->mlp_hidden = (int32_t)down->shape[0];
    cfg->n_layers = layers;
    gd_checkpoint_close(ck); /* embed and down point into ck: nothing reads them past this line */
    cfg->tie_lm_head = 1;
    /* the metadata the reference's trainer writes (examples/gpt_lm/main.c:1836-1864) carries what shapes cannot
     * tell; where it repeats what the directory fixes, the two must agree */
    st = gd_checkpoint_read_metadata(path, &blob, &blob_len);
    if (st != GD_OK) return st;
    if ((metadata_i32(blob, blob_len, "vocab_size", &v) && v != cfg->vocab) ||
        (metadata_i32(blob, blob_len, "d_model", &v) && v != cfg->d_model) ||
        (metadata_i32(blob, blob_len, "mlp_hidden", &v) && v != cfg->mlp_hidden) ||
        (metadata_i32(blob, blob_len, "n_layers", &v) && v != cfg->n_layers)) {
        free(blob);
        return GD_ERR_BAD_STATE;
    }
    if (metadata_i32(blob, blob_len, "n_heads", &v)) cfg->n_heads = v;
    if (metadata_i32(blob, blob_len, "head_dim", &v)) cfg->head_dim = v;
    if (metadata_i32(blob, blob_len, "sdpa_window", &v)) cfg->sdpa_window = v;
    if (cfg->max_seq <= 0 && metadata_i32(blob, blob_len, "context_length", &v)) cfg->max_seq = v;
    /* "architecture=minimax_m3" switches the packed prefill to picked blocks (the reference's inference programs
     * read the same keys, infer.c:407-421); the other lines give the block size and counts */
    {
        static const char key[] = "architecture=minimax_m3";
        size_t at = 0U;
        bool m3 = false;
        while (at < blob_len && !m3) {
            size_t end = at;
            while (end < blob_len && blob[end] != '\n') ++end;
            m3 = end - at == sizeof(key) - 1U && strncmp(blob + at, key, sizeof(key) - 1U) == 0;
            at = end < blob_len ? end + 1U : end;
        }
        if (m3) {
            cfg->m3_block_size = metadata_i32(blob, blob_len, "minimax_m3_block_size", &v) && v > 0 ? v : 128;
            cfg->m3_topk_blocks = metadata_i32(blob, blob_len, "minimax_m3_topk_blocks", &v) && v > 0 ? v : 3;
            cfg->m3_init_blocks = metadata_i32(blob, blob_len, "minimax_m3_init_blocks", &v) ? v : 1;
            cfg->m3_local_blocks = metadata_i32(blob, blob_len, "minimax_m3_local_blocks", &v) ? v : 1;
        }
    }
    free(blob);
    if (cfg->n_heads > 0 && cfg->head_dim <= 0 && cfg->d_model % cfg->n_heads == 0) cfg->head_dim = cfg->d_model / cfg->n_heads;
    if (cfg->head_dim > 0 && cfg->n_heads <= 0 && cfg->d_model % cfg->head_dim == 0) cfg->n_heads = cfg->d_model / cfg->head_dim;
    if (cfg->n_heads <= 0 || cfg->head_dim <= 0 || (int64_t)cfg->n_heads * cfg->head_dim != cfg->d_model)
        return GD_ERR_BAD_STATE;
    return GD_OK;
}

/* ---- forward pieces -------------------------------------------------------------------- */

/* reference src/nn/module.c:1012-1028 */
static gd_status linear_forward(gd_context *ctx, const gpt_linear *l, const gd_tensor *x, gd_tensor *out)
{
    if (l->transposed) return gd_linear_transposed_weight(ctx, x, &l->weight, &l->bias, out);
    return gd_linear(ctx, x, &l->weight, &l->bias, out);
}

static gd_status fused_project_rows(gd_gpt_decoder *d, int64_t B, const gd_tensor *x, int64_t x_cols,
                                    const gpt_linear *lin, const gd_tensor *w_override, const gd_tensor *bias,
                                    const gd_tensor *residual, const gd_tensor *norm_w, uint32_t prologue,
                                    uint32_t epilogue, int64_t n_out, gd_tensor *y);

/* attention input -> block output of the packed prefill: the two residual additions ride in the epilogues of the
 * projections in front of them (same F16 rounding points as the separate gd_add), everything else as block_tail */
static gd_status block_tail_prefill(gd_gpt_decoder *d, const gpt_block *b, const gd_tensor *residual,
                                    const gd_tensor *attn_flat, gd_tensor *out)
{
    gd_context *ctx = d->ctx;
    const int64_t rows = attn_flat->shape[0], Dm = d->cfg.d_model, Hm = d->cfg.mlp_hidden;
    gd_tensor attn_resid, mlp_normed, up_gate, gated;
    TRY(fused_project_rows(d, rows, attn_flat, Dm, &b->attn_proj, NULL, &b->attn_proj.bias, residual, NULL, 0U, 0U, Dm,
                           &attn_resid));
    TRY(gd_rms_norm(ctx, &attn_resid, &b->mlp_norm_w, d->cfg.rms_eps, &mlp_normed));
    if (b->up_gate.transposed && (Dm % 8) == 0) {
        /* swiglu in the epilogue of the up/gate projection: the [rows, 2H] intermediate is never written */
        TRY(fused_project_rows(d, rows, &mlp_normed, Dm, &b->up_gate, NULL, &b->up_gate.bias, NULL, NULL, 0U, 1U, Hm,
                               &gated));
    } else {
        TRY(linear_forward(ctx, &b->up_gate, &mlp_normed, &up_gate));
        TRY(gd_swiglu_split(ctx, &up_gate, &gated));
    }
    /* through the [N,K] twin of the down projection's [K,N] weight, as the decode step does: the same products and
     * sums, and the kernel's small tiles (the rows of the last, partly filled round) are a third faster on [N,K] */
    return fused_project_rows(d, rows, &gated, Hm, &b->down_proj, &b->down_t, &b->down_proj.bias, &attn_resid, NULL, 0U,
                              0U, Dm, out);
}

/* attention input -> block output, shared by decode and prefill (reference :1052-1070, 941-958) */
static gd_status block_tail(gd_gpt_decoder *d, const gpt_block *b, const gd_tensor *residual, const gd_tensor *attn_flat,
                            gd_tensor *out)
{
    gd_context *ctx = d->ctx;
    gd_tensor attn_proj, attn_resid, mlp_normed, up_gate, mlp_proj;
    TRY(linear_forward(ctx, &b->attn_proj, attn_flat, &attn_proj));
    TRY(gd_add(ctx, residual, &attn_proj, &attn_resid));
    TRY(gd_rms_norm(ctx, &attn_resid, &b->mlp_norm_w, d->cfg.rms_eps, &mlp_normed));
    TRY(linear_forward(ctx, &b->up_gate, &mlp_normed, &up_gate));
    TRY(gd_swiglu_split_linear(ctx, &up_gate, &b->down_proj.weight, &b->down_proj.bias, &mlp_proj));
    return gd_add(ctx, &attn_resid, &mlp_proj, out);
}

static gd_status block_decode(gd_gpt_decoder *d, int32_t l, const gd_tensor *x, const gd_tensor *positions,
                              const gd_tensor *cache_positions, gd_tensor *out)
{
    gd_context *ctx = d->ctx;
    const gpt_block *b = &d->blocks[l];
    const gd_gpt_config *c = &d->cfg;
    const gd_rope_config rope = {c->rope_theta, c->head_dim, false};
    const gd_sdpa_decode_config sdpa = {0.0f, c->sdpa_window, 0};
    gd_tensor normed, qkv, q3, k3, v3, q, k, v, attn, attn_flat;
    int64_t q_shape[4] = {x->shape[0], 1, c->n_heads, c->head_dim};
    int64_t flat_shape[2] = {x->shape[0], c->d_model};
    TRY(gd_rms_norm(ctx, x, &b->attn_norm_w, c->rms_eps, &normed));
    TRY(linear_forward(ctx, &b->qkv_proj, &normed, &qkv));
    TRY(gd_qkv_split_rope(ctx, &qkv, positions, c->n_heads, c->head_dim, &rope, &q3, &k3, &v3));
    TRY(gd_reshape(ctx, &q3, gd_shape_make(4U, q_shape), &q));
    TRY(gd_reshape(ctx, &k3, gd_shape_make(4U, q_shape), &k));
    TRY(gd_reshape(ctx, &v3, gd_shape_make(4U, q_shape), &v));
    TRY(gd_kv_cache_append_positions(ctx, &d->k_cache[l], &d->v_cache[l], cache_positions, &k, &v));
    TRY(gd_sdpa_decode_positions(ctx, &q, &d->k_cache[l], &d->v_cache[l], cache_positions, &sdpa, &attn));
    TRY(gd_reshape(ctx, &attn, gd_shape_make(2U, flat_shape), &attn_flat));
    return block_tail(d, b, x, &attn_flat, out);
}

/* angles and cache rows of the packed prompt rows (gd_backend_rope_table_packed), shared by the layers of a prefill */
typedef struct prefill_rope_rows {
    gd_tensor cos_rows, sin_rows, cache_rows;
} prefill_rope_rows;

static gd_status scratch_f16(gd_context *ctx, int64_t rows, int64_t cols, gd_tensor *out);

/* the qkv projection can carry rotation, split and cache append in its epilogue (gd_backend_linear_qkv_rope_packed) */
static bool prefill_rope_in_projection(const gd_gpt_decoder *d)
{
    const gd_gpt_config *c = &d->cfg;
    const bool m3 = c->m3_block_size > 0 && c->m3_topk_blocks > 0 &&
                    (int64_t)c->max_seq > (int64_t)c->m3_block_size * 8 &&
                    (int64_t)c->m3_block_size * c->m3_topk_blocks * 2 < (int64_t)c->max_seq;
    return !m3 && (c->head_dim == 64 || c->head_dim == 128) && (c->d_model % 256) == 0 &&
           d->blocks[0].qkv_proj.transposed && d->blocks[0].qkv_proj.weight.dtype == GD_DTYPE_F16 &&
           (uint64_t)c->batch * (uint64_t)c->max_seq * (uint64_t)c->d_model * 2U < 0xffffffffULL;
}

static gd_status block_prefill(gd_gpt_decoder *d, int32_t l, const gd_tensor *x, const gd_tensor *positions,
                               const gd_tensor *cu, const gd_tensor *cache_positions, const prefill_rope_rows *rows,
                               gd_tensor *out)
{
    gd_context *ctx = d->ctx;
    const gpt_block *b = &d->blocks[l];
    const gd_gpt_config *c = &d->cfg;
    const gd_rope_config rope = {c->rope_theta, c->head_dim, false};
    const gd_sdpa_varlen_config sdpa = {0.0f, true, c->sdpa_window, 0, c->max_seq};
    const bool m3 = c->m3_block_size > 0 && c->m3_topk_blocks > 0 &&
                    (int64_t)c->max_seq > (int64_t)c->m3_block_size * 8 &&
                    (int64_t)c->m3_block_size * c->m3_topk_blocks * 2 < (int64_t)c->max_seq;
    /* the prefill appends every sequence at cache position 0 (gd_gpt_decoder_prefill), so the attention can read the
     * keys and values of a sequence where the append has just put them, and the packed k / v are never written */
    const bool from_caches = !m3 && (c->head_dim == 64 || c->head_dim == 128) &&
                             (uint64_t)c->batch * (uint64_t)c->max_seq * (uint64_t)c->n_heads * (uint64_t)c->head_dim * 2U <
                                 0xffffffffULL;
    gd_tensor normed, qkv, q, k, v, attn, attn_flat;
    int64_t flat_shape[2] = {x->shape[0], c->d_model};
    bool attended = false;
    TRY(gd_rms_norm(ctx, x, &b->attn_norm_w, c->rms_eps, &normed));
    if (rows != NULL && from_caches && x->shape[0] >= 256) {
        /* rotation, split and cache append in the epilogue of the projection's tiles; attention from the caches */
        const gd_backend_sdpa_varlen_args va = {(float)(1.0 / sqrt((double)c->head_dim)), 1U, (uint32_t)c->sdpa_window, 0U,
                                                (uint32_t)c->max_seq, 0U};
        const int64_t N = x->shape[0];
        int64_t dims[3] = {N, c->n_heads, c->head_dim};
        gd_backend_matrix_view xm, wm, workm;
        gd_backend_vector_view bv;
        gd_backend_tensor_view vcos, vsin, vrows, vq, vkc, vvc, vcu, vo;
        gd_status st;
        TRY(gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F16, gd_shape_make(3U, dims), 256U, &q));
        TRY(scratch_f16(ctx, N, 3 * (int64_t)c->d_model, &qkv));
        mview(&normed, N, c->d_model, &xm);
        mview(&b->qkv_proj.weight, b->qkv_proj.weight.shape[0], b->qkv_proj.weight.shape[1], &wm);
        mview(&qkv, N, 3 * (int64_t)c->d_model, &workm);
        vview(&b->qkv_proj.bias, &bv);
        tview(&rows->cos_rows, &vcos);
        tview(&rows->sin_rows, &vsin);
        tview(&rows->cache_rows, &vrows);
        tview(&q, &vq);
        tview(&d->k_cache[l], &vkc);
        tview(&d->v_cache[l], &vvc);
        tview(cu, &vcu);
        /* bias mode 2: gd_linear_transposed_weight is matmul_nt + add, two roundings */
        st = gd_backend_linear_qkv_rope_packed(gd_context_backend(ctx), &xm, &wm, &bv, &vcos, &vsin, &vrows, &vq, &vkc, &vvc,
                                               &workm, (uint32_t)c->n_heads, (uint32_t)c->head_dim, 2U);
        if (st == GD_OK) {
            TRY(gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F16, gd_shape_make(3U, dims), 256U, &attn));
            tview(&attn, &vo);
            TRY(gd_backend_sdpa_varlen_cached(gd_context_backend(ctx), &vq, &vkc, &vvc, &vcu, &vo, &va));
            TRY(gd_reshape(ctx, &attn, gd_shape_make(2U, flat_shape), &attn_flat));
            return block_tail_prefill(d, b, x, &attn_flat, out);
        }
        if (st != GD_ERR_UNSUPPORTED) return st;
    }
    TRY(linear_forward(ctx, &b->qkv_proj, &normed, &qkv));
    if ((c->head_dim % 16) == 0 && qkv.dtype == GD_DTYPE_F16) {
        /* rotation, split and cache append in one pass over the projection: the appended rows are not read back */
        const gd_backend_rope_args ra = {c->rope_theta, (uint32_t)c->head_dim, 0U};
        int64_t dims[3] = {x->shape[0], c->n_heads, c->head_dim};
        gd_backend_tensor_view vqkv, vpos, vcp, vcu, vq, vk, vv, vkc, vvc;
        TRY(gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F16, gd_shape_make(3U, dims), 256U, &q));
        if (!from_caches) {
            TRY(gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F16, gd_shape_make(3U, dims), 256U, &k));
            TRY(gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F16, gd_shape_make(3U, dims), 256U, &v));
            tview(&k, &vk);
            tview(&v, &vv);
        }
        tview(&qkv, &vqkv);
        tview(positions, &vpos);
        tview(cache_positions, &vcp);
        tview(cu, &vcu);
        tview(&q, &vq);
        tview(&d->k_cache[l], &vkc);
        tview(&d->v_cache[l], &vvc);
        TRY(gd_backend_qkv_rope_append_packed(gd_context_backend(ctx), &vqkv, &vpos, &vcp, &vcu, &vq,
                                              from_caches ? NULL : &vk, from_caches ? NULL : &vv, &vkc, &vvc,
                                              (uint32_t)c->n_heads, (uint32_t)c->head_dim, &ra));
        if (from_caches) {
            const gd_backend_sdpa_varlen_args va = {(float)(1.0 / sqrt((double)c->head_dim)), 1U, (uint32_t)c->sdpa_window,
                                                    0U, (uint32_t)c->max_seq, 0U};
            gd_backend_tensor_view vo;
            TRY(gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F16, gd_shape_make(3U, dims), 256U, &attn));
            tview(&attn, &vo);
            TRY(gd_backend_sdpa_varlen_cached(gd_context_backend(ctx), &vq, &vkc, &vvc, &vcu, &vo, &va));
            attended = true;
        }
    } else {
        TRY(gd_qkv_split_rope(ctx, &qkv, positions, c->n_heads, c->head_dim, &rope, &q, &k, &v));
        TRY(gd_kv_cache_append_packed(ctx, &d->k_cache[l], &d->v_cache[l], cache_positions, cu, &k, &v));
    }
    /* MiniMax-M3: picked blocks when the context is long enough for that to matter (reference :588-600, 918-933) */
    if (attended) {
        /* done above, from the caches */
    } else if (m3) {
        const gd_minimax_m3_sparse_config m3 = {0.0f, c->m3_block_size, c->m3_topk_blocks, c->m3_init_blocks,
                                                c->m3_local_blocks, c->max_seq};
        gd_tensor picked;
        TRY(gd_minimax_m3_index_topk(ctx, &q, &k, cu, &m3, &picked));
        TRY(gd_minimax_m3_sparse_attention(ctx, &q, &k, &v, cu, &picked, &m3, &attn));
    } else {
        TRY(gd_sdpa_varlen(ctx, &q, &k, &v, cu, &sdpa, &attn));
    }
    TRY(gd_reshape(ctx, &attn, gd_shape_make(2U, flat_shape), &attn_flat));
    if (x->shape[0] >= 128) return block_tail_prefill(d, b, x, &attn_flat, out);
    return block_tail(d, b, x, &attn_flat, out);
}

static gd_status head(gd_gpt_decoder *d, const gd_tensor *x, gd_tensor *logits)
{
    gd_tensor normed;
    TRY(gd_rms_norm(d->ctx, x, &d->final_norm_w, d->cfg.rms_eps, &normed));
    return gd_linear_transposed_weight(d->ctx, &normed, &d->lm_head, &d->lm_head_bias, logits);
}

static gd_status gpt_prefill(gd_gpt_decoder *d, const int32_t *ids, const int32_t *cu, gd_tensor *logits)
{
    gd_context *ctx = d->ctx;
    gd_tensor t_ids, t_pos, t_cu, t_cache_pos, t_last, x, y, last_hidden;
    prefill_rope_rows rope_rows;
    bool have_rows = false;
    gd_status st = GD_OK;
    int32_t *positions, *zero, *last_rows;
    const int32_t B = d->cfg.batch, N = cu[B];
    int32_t b, r, l;
    positions = (int32_t *)malloc((size_t)N * sizeof(int32_t));
    zero = (int32_t *)calloc((size_t)B, sizeof(int32_t));
    last_rows = (int32_t *)malloc((size_t)B * sizeof(int32_t));
    if (positions == NULL || zero == NULL || last_rows == NULL) st = GD_ERR_OUT_OF_MEMORY;
    for (b = 0; b < B && st == GD_OK; ++b) {
        for (r = cu[b]; r < cu[b + 1]; ++r) positions[r] = r - cu[b];
        last_rows[b] = cu[b + 1] - 1;
    }
    if (st == GD_OK) st = data_i32(ctx, ids, N, &t_ids);
    if (st == GD_OK) st = data_i32(ctx, positions, N, &t_pos);
    if (st == GD_OK) st = data_i32(ctx, cu, (int64_t)B + 1, &t_cu);
    if (st == GD_OK) st = data_i32(ctx, zero, B, &t_cache_pos);
    if (st == GD_OK) st = data_i32(ctx, last_rows, B, &t_last);
    free(positions);
    free(zero);
    free(last_rows);
    if (st == GD_OK) st = gd_embedding(ctx, &d->token_embedding, &t_ids, &x);
    if (st == GD_OK && N >= 256 && prefill_rope_in_projection(d)) {
        /* once for all layers: the angles of every row's position and the cache row its k and v go to */
        const gd_backend_rope_args ra = {d->cfg.rope_theta, (uint32_t)d->cfg.head_dim, 0U};
        int64_t tdims[2] = {((int64_t)N + 31) / 32 * 32, d->cfg.head_dim / 2}, rdims[1] = {N};
        gd_backend_tensor_view vpos, vcp, vcu, vcos, vsin, vrows;
        st = gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F32, gd_shape_make(2U, tdims), 256U, &rope_rows.cos_rows);
        if (st == GD_OK)
            st = gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F32, gd_shape_make(2U, tdims), 256U, &rope_rows.sin_rows);
        if (st == GD_OK)
            st = gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_I32, gd_shape_make(1U, rdims), 256U, &rope_rows.cache_rows);
        if (st == GD_OK) {
            tview(&t_pos, &vpos);
            tview(&t_cache_pos, &vcp);
            tview(&t_cu, &vcu);
            tview(&rope_rows.cos_rows, &vcos);
            tview(&rope_rows.sin_rows, &vsin);
            tview(&rope_rows.cache_rows, &vrows);
            st = gd_backend_rope_table_packed(gd_context_backend(ctx), &vpos, &vcp, &vcu, &vcos, &vsin, &vrows,
                                              (uint32_t)d->cfg.head_dim, (uint32_t)d->cfg.max_seq, &ra);
            have_rows = st == GD_OK;
            if (st == GD_ERR_UNSUPPORTED) st = GD_OK;
        }
    }
    for (l = 0; l < d->cfg.n_layers && st == GD_OK; ++l) {
        st = block_prefill(d, l, &x, &t_pos, &t_cu, &t_cache_pos, have_rows ? &rope_rows : NULL, &y);
        x = y;
    }
    if (st == GD_OK) st = gd_gather_rows(ctx, &x, &t_last, &last_hidden);
    return st == GD_OK ? head(d, &last_hidden, logits) : st;
}

/* ---- device-resident decode -------------------------------------------------------------- */

static gd_status scratch_f16(gd_context *ctx, int64_t rows, int64_t cols, gd_tensor *out)
{
    int64_t dims[2] = {rows, cols};
    return gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F16, gd_shape_make(2U, dims), 256U, out);
}

/* y = [residual +] bias_mode(prologue(x) @ w) through gd_backend_fused_linear */
static gd_status fused_project_rows(gd_gpt_decoder *d, int64_t B, const gd_tensor *x, int64_t x_cols,
                                    const gpt_linear *lin, const gd_tensor *w_override, const gd_tensor *bias,
                                    const gd_tensor *residual, const gd_tensor *norm_w, uint32_t prologue,
                                    uint32_t epilogue, int64_t n_out, gd_tensor *y)
{
    gd_backend_matrix_view xm, wm, rm, ym;
    gd_backend_vector_view bv, nv;
    gd_backend_fused_linear_args a;
    const gd_tensor *w = w_override != NULL ? w_override : &lin->weight;
    gd_status st;
    TRY(scratch_f16(d->ctx, B, n_out, y));
    mview(x, B, x_cols, &xm);
    mview(w, w->shape[0], w->shape[1], &wm);
    mview(y, B, n_out, &ym);
    if (residual != NULL) mview(residual, B, n_out, &rm);
    if (norm_w != NULL) vview(norm_w, &nv);
    vview(bias, &bv);
    a.w_is_nk = (lin->transposed || w_override != NULL) ? 1U : 0U; /* an override is the [N,K] twin of a [K,N] weight */
    a.bias_mode = lin->transposed ? 2U : 1U; /* gd_linear_transposed_weight: matmul_nt + add (two roundings);
                                                gd_linear: F32 bias in front of the single rounding */
    a.prologue = prologue;
    a.eps = d->cfg.rms_eps;
    a.epilogue = epilogue;
    st = gd_backend_fused_linear(gd_context_backend(d->ctx), &xm, &wm, &bv, residual != NULL ? &rm : NULL,
                                 norm_w != NULL ? &nv : NULL, &ym, &a);
    return st;
}

static gd_status fused_project(gd_gpt_decoder *d, const gd_tensor *x, int64_t x_cols, const gpt_linear *lin,
                               const gd_tensor *w_override, const gd_tensor *bias, const gd_tensor *residual,
                               const gd_tensor *norm_w, uint32_t prologue, uint32_t epilogue, int64_t n_out, gd_tensor *y)
{
    return fused_project_rows(d, d->cfg.batch, x, x_cols, lin, w_override, bias, residual, norm_w, prologue, epilogue,
                              n_out, y);
}

/* The decode step with the fused backend entry points: same operators, same rounding points as
 * block_decode, 6 launches per layer. */
static gd_status enqueue_fused_step(gd_gpt_decoder *d, gd_tensor *logits)
{
    gd_context *ctx = d->ctx;
    gd_backend *be = gd_context_backend(ctx);
    const gd_gpt_config *c = &d->cfg;
    const gd_backend_rope_args rope = {c->rope_theta, (uint32_t)c->head_dim, 0U};
    const gd_sdpa_decode_config sdpa = {0.0f, c->sdpa_window, 0};
    const int64_t B = c->batch, Dm = c->d_model, Hm = c->mlp_hidden;
    gd_tensor x, qkv, q, q4, attn, x1, ug, x2;
    gd_backend_tensor_view vqkv, vpos, vq, vk, vv;
    int64_t q_shape[4] = {B, 1, c->n_heads, c->head_dim};
    int32_t l;
    if (d->resident_x0) x = d->x0_dev;
    else TRY(gd_embedding(ctx, &d->token_embedding, &d->ids_dev, &x));
    for (l = 0; l < c->n_layers; ++l) {
        const gpt_block *b = &d->blocks[l];
        TRY(scratch_f16(ctx, B, Dm, &q));
        tview(&d->pos_dev, &vpos);
        tview(&d->k_cache[l], &vk);
        tview(&d->v_cache[l], &vv);
        memset(&vq, 0, sizeof(vq));
        vq.buffer = (gd_backend_buffer *)q.storage.buffer;
        vq.offset = q.storage.offset;
        vq.count = (size_t)(B * Dm);
        vq.dtype = (uint32_t)GD_DTYPE_F16;
        vq.rank = 3U;
        vq.shape[0] = B; vq.shape[1] = c->n_heads; vq.shape[2] = c->head_dim;
        vq.strides[0] = Dm; vq.strides[1] = c->head_dim; vq.strides[2] = 1;
        if (B < 128 && (c->head_dim % 32) == 0) {
            /* qkv projection with rotation and cache append in its epilogue: the [B,3Dm] intermediate is never stored */
            gd_backend_matrix_view xm, wm;
            gd_backend_vector_view bv, nv;
            gd_backend_fused_linear_args fa;
            mview(&x, B, Dm, &xm);
            mview(&b->qkv_proj.weight, 3 * Dm, Dm, &wm);
            vview(&b->qkv_proj.bias, &bv);
            vview(&b->attn_norm_w, &nv);
            fa.w_is_nk = 1U;
            fa.bias_mode = 2U;
            fa.prologue = 2U;
            fa.eps = c->rms_eps;
            fa.epilogue = 0U;
            TRY(gd_backend_fused_qkv_rope_append(be, &xm, &wm, &bv, &nv, &vpos, &vpos, &vq, &vk, &vv, (uint32_t)c->n_heads,
                                                 (uint32_t)c->head_dim, &rope, &fa));
        } else {
            TRY(fused_project(d, &x, Dm, &b->qkv_proj, NULL, &b->qkv_proj.bias, NULL, &b->attn_norm_w, 2U, 0U, 3 * Dm, &qkv));
            tview(&qkv, &vqkv);
            TRY(gd_backend_qkv_rope_append(be, &vqkv, &vpos, &vpos, &vq, &vk, &vv, (uint32_t)c->n_heads,
                                           (uint32_t)c->head_dim, &rope));
        }
        TRY(gd_reshape(ctx, &q, gd_shape_make(4U, q_shape), &q4));
        TRY(gd_sdpa_decode_positions(ctx, &q4, &d->k_cache[l], &d->v_cache[l], &d->pos_dev, &sdpa, &attn));
        TRY(fused_project(d, &attn, Dm, &b->attn_proj, NULL, &b->attn_proj.bias, &x, NULL, 0U, 0U, Dm, &x1));
        if (B < 128) {
            /* the gate is applied in the up/gate projection's epilogue: the [B,2Hm] intermediate is never stored */
            TRY(fused_project(d, &x1, Dm, &b->up_gate, NULL, &b->up_gate.bias, NULL, &b->mlp_norm_w, 2U, 1U, Hm, &ug));
            TRY(fused_project(d, &ug, Hm, &b->down_proj, &b->down_t, &b->down_proj.bias, &x1, NULL, 0U, 0U, Dm, &x2));
        } else {
            TRY(fused_project(d, &x1, Dm, &b->up_gate, NULL, &b->up_gate.bias, NULL, &b->mlp_norm_w, 2U, 0U, 2 * Hm, &ug));
            TRY(fused_project(d, &ug, 2 * Hm, &b->down_proj, &b->down_t, &b->down_proj.bias, &x1, NULL, 1U, 0U, Dm, &x2));
        }
        x = x2;
    }
    {
        gpt_linear head_lin;
        head_lin.weight = d->lm_head;
        head_lin.bias = d->lm_head_bias;
        head_lin.transposed = true;
        TRY(fused_project(d, &x, Dm, &head_lin, NULL, &d->lm_head_bias, NULL, &d->final_norm_w, 2U, 0U, c->vocab, logits));
    }
    return GD_OK;
}

static gd_status gpt_step(gd_gpt_decoder *d, const gd_tensor *ids, const gd_tensor *positions, bool fused,
                          gd_tensor *logits)
{
    gd_tensor x, y;
    int32_t l;
    if (fused) return enqueue_fused_step(d, logits);
    TRY(gd_embedding(d->ctx, &d->token_embedding, ids, &x));
    for (l = 0; l < d->cfg.n_layers; ++l) {
        TRY(block_decode(d, l, &x, positions, positions, &y));
        x = y;
    }
    return head(d, &x, logits);
}

/* the fused rope + append kernel needs NeoX pairs of a head size that is a multiple of 16 */
static bool gpt_can_fuse(const gd_gpt_decoder *d) { return (d->cfg.head_dim % 16) == 0; }
static bool gpt_feeds_x0(const gd_gpt_decoder *d) { return (d->cfg.d_model % 8) == 0; }

static const gd_decoder_model gpt_model = {"gpt_lm", gpt_prefill, gpt_step, NULL, gpt_can_fuse, gpt_feeds_x0,
                                           gpt_tensor, gpt_destroy};
