/*
 * What the parts of the decoder share: the decoder object, the table of functions a model fills in, and small view
 * helpers.  session.c holds everything that does not depend on the model (step scopes, resident sessions, sampling,
 * generation, portions of prompts, slots); gpt_decoder.c is the reference example's model, layer_list.c the model whose
 * layers are listed in a configuration file; model_registry.c finds the model of a path.
 */
#ifndef GD_DECODER_INTERNAL_H
#define GD_DECODER_INTERNAL_H

#include <stdlib.h>
#include <string.h>

#include "gd_gpt_decoder.h"
#include "gd_model.h"

#define TRY(expr)                       \
    do {                                \
        gd_status st__ = (expr);        \
        if (st__ != GD_OK) return st__; \
    } while (0)

/* new tokens of some sequences, packed; see gd_gpt_decoder_extend */
typedef struct gd_extend_rows {
    int32_t n_seqs, rows, max_new; /* sequences, packed rows, largest number of new rows of a sequence */
    const int32_t *slots;          /* [n_seqs] */
    const int32_t *ids, *cu;       /* [rows], [n_seqs + 1] */
    const int32_t *start;          /* [n_seqs]: position of every sequence's first new row */
    const int32_t *want;           /* [n_want]: packed rows whose logits are asked for */
    int32_t n_want;
} gd_extend_rows;

/* A model behind a decoder.  All of these enqueue inside an open step scope and leave logits [rows, vocab] of the
 * decoder's logits type in scratch. */
typedef struct gd_decoder_model {
    const char *architecture;
    /* packed prompts of every batch row from position 0: logits of each row's last token */
    gd_status (*prefill)(gd_gpt_decoder *d, const int32_t *ids, const int32_t *cu, gd_tensor *logits);
    /* one token per batch row; ids and positions I32 [batch] on the device.  fused: the form with fused entry points,
     * which may start from the embedding rows in x0_dev (feeds_x0) */
    gd_status (*step)(gd_gpt_decoder *d, const gd_tensor *ids, const gd_tensor *positions, bool fused, gd_tensor *logits);
    /* new tokens of any sequences behind what they already hold; NULL: the model cannot continue a prompt */
    gd_status (*extend)(gd_gpt_decoder *d, const gd_extend_rows *e, gd_tensor *logits);
    bool (*can_fuse)(const gd_gpt_decoder *d);
    bool (*feeds_x0)(const gd_gpt_decoder *d);
    gd_tensor *(*tensor)(gd_gpt_decoder *d, const char *name, int32_t layer);
    void (*destroy)(gd_gpt_decoder *d);
} gd_decoder_model;

struct gd_gpt_decoder {
    gd_context *ctx;
    const gd_decoder_model *model;
    gd_gpt_config cfg; /* vocab, d_model, n_layers, max_seq and batch of any model; the rest: gpt_decoder.c */
    int32_t *pos;      /* host copy of the live lengths */
    bool *slot_taken;  /* [batch]: gd_gpt_decoder_acquire */
    /* gpt_decoder.c */
    gd_tensor token_embedding, lm_head, lm_head_bias, final_norm_w;
    struct gpt_block *blocks;
    gd_tensor *k_cache, *v_cache;
    /* layer_list.c */
    struct layer_list *layers;
    /* device-resident decode state (state arena) */
    gd_tensor ids_dev, pos_dev, step_dev, step_rows_dev; /* step counters: one for the whole batch / one per row */
    gd_tensor x0_dev;     /* [B, Dm]: embedding rows of the tokens the fused resident step starts from */
    bool resident_x0;     /* x0_dev is kept current by the greedy-pick kernel */
    /* open resident session */
    bool resident_open;
    int32_t resident_max_steps, resident_steps, resident_hold, resident_unfused, resident_keep_logits;
    gd_backend_graph *resident_graph;
    gd_tensor resident_out_ids, resident_out_gaps;
    /* sampling front end (state arena): what the reference's generation loop keeps on the host */
    gd_tensor last_logits;                 /* [B, V] F16 or F32: logits of the last packed prefill */
    gd_tensor history, hist_len, finished; /* [B, max_seq], [B], [B] I32 */
    gd_tensor sample_state, sample_work;   /* generator + per-row records; [B*V] F32 */
    bool resident_sampling;
    gd_gpt_sampling sampling;
};

/* session.c: the model-independent part of a decoder.  create: the object with ctx, model and cfg set and nothing on
 * the device; allocate: its tensors in the state arena, logits of the given type, x0 rows only if a model feeds them. */
gd_status gd_decoder_session_create(gd_context *ctx, const gd_decoder_model *model, const gd_gpt_config *cfg,
                                    gd_gpt_decoder **out);
gd_status gd_decoder_session_allocate(gd_gpt_decoder *d, gd_dtype logits_dtype, bool x0_rows);
size_t gd_decoder_session_bytes(const gd_gpt_config *cfg, gd_dtype logits_dtype, bool x0_rows);

static inline size_t gd_pad256(size_t n) { return (n + 255U) & ~(size_t)255U; }

static inline uint64_t gd_mix64(uint64_t x)
{
    x = (x ^ (x >> 30)) * UINT64_C(0xbf58476d1ce4e5b9);
    x = (x ^ (x >> 27)) * UINT64_C(0x94d049bb133111eb);
    return x ^ (x >> 31);
}

static inline uint64_t gd_splitmix64(uint64_t x) { return gd_mix64(x + UINT64_C(0x9e3779b97f4a7c15)); }

/* views of contiguous tensors */
static inline void tview(const gd_tensor *t, gd_backend_tensor_view *v)
{
    int64_t stride = 1;
    uint32_t i;
    memset(v, 0, sizeof(*v));
    v->buffer = (gd_backend_buffer *)t->storage.buffer;
    v->offset = t->storage.offset + t->view_offset;
    v->dtype = (uint32_t)t->dtype;
    v->rank = t->rank;
    for (i = t->rank; i > 0U; --i) {
        v->shape[i - 1U] = t->shape[i - 1U];
        v->strides[i - 1U] = stride;
        stride *= t->shape[i - 1U];
    }
    v->count = (size_t)stride;
}

static inline void view1(const gd_tensor *t, gd_backend_tensor_view *v)
{
    memset(v, 0, sizeof(*v));
    v->buffer = (gd_backend_buffer *)t->storage.buffer;
    v->offset = t->storage.offset + t->view_offset;
    v->count = (size_t)t->shape[0];
    v->dtype = (uint32_t)t->dtype;
    v->rank = 1U;
    v->shape[0] = t->shape[0];
    v->strides[0] = 1;
}

static inline bool mview(const gd_tensor *t, int64_t rows, int64_t cols, gd_backend_matrix_view *m)
{
    m->buffer = (gd_backend_buffer *)t->storage.buffer;
    m->offset = t->storage.offset + t->view_offset;
    m->rows = (uint32_t)rows;
    m->cols = (uint32_t)cols;
    m->row_bytes = (size_t)cols * gd_dtype_size(t->dtype);
    m->dtype = (uint32_t)t->dtype;
    return m->buffer != NULL;
}

static inline void vview(const gd_tensor *t, gd_backend_vector_view *v)
{
    v->buffer = (gd_backend_buffer *)t->storage.buffer;
    v->offset = t->storage.offset + t->view_offset;
    v->length = (uint32_t)t->shape[0];
    v->dtype = (uint32_t)t->dtype;
}

static inline gd_status data_i32(gd_context *ctx, const int32_t *values, int64_t n, gd_tensor *out)
{
    int64_t dims[1] = {n};
    TRY(gd_tensor_empty(ctx, GD_ARENA_DATA, GD_DTYPE_I32, gd_shape_make(1U, dims), 256U, out));
    return gd_tensor_write(ctx, out, values, (size_t)n * sizeof(int32_t));
}

#endif
