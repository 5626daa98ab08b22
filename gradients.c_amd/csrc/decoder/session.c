/*
 * The model-independent part of a decoder: step scopes, the device-resident greedy or sampled session, generation
 * (examples/gpt_lm/gpt_lm_shared.c:1322-1442, 1444-1700 of the reference), portions of prompts and the slots they live
 * in.  What a step computes comes from the model's table of functions (decoder_internal.h).
 */
#include <stdio.h>

#include "../core/core_internal.h" /* F16 bits of F32 logits */
#include "decoder_internal.h"

gd_status gd_decoder_session_create(gd_context *ctx, const gd_decoder_model *model, const gd_gpt_config *cfg,
                                    gd_gpt_decoder **out)
{
    gd_gpt_decoder *d = (gd_gpt_decoder *)calloc(1, sizeof(*d));
    *out = NULL;
    if (d == NULL) return GD_ERR_OUT_OF_MEMORY;
    d->ctx = ctx;
    d->model = model;
    d->cfg = *cfg;
    d->pos = (int32_t *)calloc((size_t)cfg->batch, sizeof(int32_t));
    d->slot_taken = (bool *)calloc((size_t)cfg->batch, sizeof(bool));
    if (d->pos == NULL || d->slot_taken == NULL) {
        gd_gpt_decoder_destroy(d);
        return GD_ERR_OUT_OF_MEMORY;
    }
    *out = d;
    return GD_OK;
}

size_t gd_decoder_session_bytes(const gd_gpt_config *c, gd_dtype logits_dtype, bool x0_rows)
{
    const size_t B = (size_t)c->batch, V = (size_t)c->vocab;
    return gd_pad256(B * V * gd_dtype_size(logits_dtype)) +
           gd_pad256(gd_backend_sample_work_count((uint32_t)B, (uint32_t)V) * 4U) +
           gd_pad256(B * (size_t)c->max_seq * 4U) + 2U * gd_pad256(B * 4U) +
           gd_pad256(gd_backend_sample_state_count((uint32_t)B) * 4U) + 4U * gd_pad256(B * 4U) +
           (x0_rows ? gd_pad256(B * (size_t)c->d_model * 2U) : 0U);
}

gd_status gd_decoder_session_allocate(gd_gpt_decoder *d, gd_dtype logits_dtype, bool x0_rows)
{
    gd_context *ctx = d->ctx;
    const gd_gpt_config *c = &d->cfg;
    int64_t bdim[1] = {c->batch}, one[1] = {1}, xdim[2] = {c->batch, c->d_model};
    int64_t ldim[2] = {c->batch, c->vocab}, hdim[2] = {c->batch, c->max_seq};
    int64_t sdim[1] = {(int64_t)gd_backend_sample_state_count((uint32_t)c->batch)};
    int64_t wdim[1] = {(int64_t)gd_backend_sample_work_count((uint32_t)c->batch, (uint32_t)c->vocab)};
#define STATE(dtype, rank, dims, t) TRY(gd_tensor_zeros(ctx, GD_ARENA_STATE, (dtype), gd_shape_make((rank), (dims)), 256U, (t)))
    STATE(GD_DTYPE_I32, 1U, bdim, &d->ids_dev);
    STATE(GD_DTYPE_I32, 1U, bdim, &d->pos_dev);
    STATE(GD_DTYPE_I32, 1U, one, &d->step_dev);
    STATE(GD_DTYPE_I32, 1U, bdim, &d->step_rows_dev);
    if (x0_rows) STATE(GD_DTYPE_F16, 2U, xdim, &d->x0_dev);
    STATE(logits_dtype, 2U, ldim, &d->last_logits);
    STATE(GD_DTYPE_I32, 2U, hdim, &d->history);
    STATE(GD_DTYPE_I32, 1U, bdim, &d->hist_len);
    STATE(GD_DTYPE_I32, 1U, bdim, &d->finished);
    STATE(GD_DTYPE_I32, 1U, sdim, &d->sample_state);
    STATE(GD_DTYPE_F32, 1U, wdim, &d->sample_work);
#undef STATE
    return GD_OK;
}

void gd_gpt_decoder_destroy(gd_gpt_decoder *d)
{
    if (d == NULL) return;
    d->model->destroy(d);
    free(d->pos);
    free(d->slot_taken);
    free(d);
}

int32_t *gd_gpt_decoder_positions(gd_gpt_decoder *d) { return d != NULL ? d->pos : NULL; }

gd_tensor *gd_gpt_decoder_tensor(gd_gpt_decoder *d, const char *name, int32_t layer)
{
    if (d == NULL || name == NULL) return NULL;
    if (!strcmp(name, "last_logits")) return &d->last_logits;
    return d->model->tensor(d, name, layer);
}

/* ---- one step with host tokens ---------------------------------------------------------------- */

static gd_status fetch(gd_gpt_decoder *d, const gd_tensor *logits, const gd_tensor *ids, const gd_tensor *gaps,
                       int32_t *next_ids, float *out_gaps, uint16_t *out_logits)
{
    const size_t B = (size_t)d->cfg.batch, n = B * (size_t)d->cfg.vocab;
    if (next_ids != NULL) TRY(gd_tensor_read(d->ctx, ids, next_ids, B * sizeof(int32_t)));
    if (out_gaps != NULL) TRY(gd_tensor_read(d->ctx, gaps, out_gaps, B * sizeof(float)));
    if (out_logits != NULL && logits->dtype == GD_DTYPE_F32) {
        float *wide = (float *)malloc(n * sizeof(float));
        gd_status st = wide == NULL ? GD_ERR_OUT_OF_MEMORY : gd_tensor_read(d->ctx, logits, wide, n * sizeof(float));
        size_t i;
        for (i = 0U; st == GD_OK && i < n; ++i) out_logits[i] = gd_f32_to_f16_bits(wide[i]);
        free(wide);
        return st;
    }
    if (out_logits != NULL) TRY(gd_tensor_read(d->ctx, logits, out_logits, n * 2U));
    return GD_OK;
}

gd_status gd_gpt_decoder_step(gd_gpt_decoder *d, const int32_t *ids, int32_t *next_ids, float *gaps, uint16_t *logits)
{
    gd_context *ctx;
    gd_tensor t_ids, t_pos, t_logits, t_next, t_gaps;
    gd_status st;
    int32_t b;
    if (d == NULL || ids == NULL) return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BUSY;
    ctx = d->ctx;
    TRY(gd_begin_step(ctx, GD_SCOPE_INFER, gd_batch_empty()));
    st = data_i32(ctx, ids, d->cfg.batch, &t_ids);
    if (st == GD_OK) st = data_i32(ctx, d->pos, d->cfg.batch, &t_pos);
    if (st == GD_OK) st = d->model->step(d, &t_ids, &t_pos, false, &t_logits);
    if (st == GD_OK) st = gd_argmax_rows(ctx, &t_logits, &t_next, &t_gaps);
    if (st != GD_OK) {
        (void)gd_end_step(ctx);
        return st;
    }
    for (b = 0; b < d->cfg.batch; ++b) d->pos[b] += 1;
    TRY(gd_end_step(ctx));
    return fetch(d, &t_logits, &t_next, &t_gaps, next_ids, gaps, logits);
}

static gd_status keep_logits(gd_gpt_decoder *d, const gd_tensor *logits);

gd_status gd_gpt_decoder_prefill(gd_gpt_decoder *d, const int32_t *ids, const int32_t *cu, int32_t *next_ids,
                                 float *gaps, uint16_t *logits)
{
    gd_context *ctx;
    gd_tensor t_logits, t_next, t_gaps;
    gd_status st;
    int32_t B, b;
    if (d == NULL || ids == NULL || cu == NULL) return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BUSY;
    ctx = d->ctx;
    B = d->cfg.batch;
    if (cu[0] != 0 || cu[B] <= 0) return GD_ERR_INVALID_ARGUMENT;
    for (b = 0; b < B; ++b) {
        if (cu[b + 1] <= cu[b] || cu[b + 1] - cu[b] > d->cfg.max_seq) return GD_ERR_INVALID_ARGUMENT;
    }
    TRY(gd_begin_step(ctx, GD_SCOPE_INFER, gd_batch_empty()));
    st = d->model->prefill(d, ids, cu, &t_logits);
    if (st == GD_OK) st = gd_argmax_rows(ctx, &t_logits, &t_next, &t_gaps);
    /* the sampling front end starts from these logits without a round trip through the host */
    if (st == GD_OK) st = keep_logits(d, &t_logits);
    if (st != GD_OK) {
        (void)gd_end_step(ctx);
        return st;
    }
    for (b = 0; b < B; ++b) d->pos[b] = cu[b + 1] - cu[b];
    TRY(gd_end_step(ctx));
    return fetch(d, &t_logits, &t_next, &t_gaps, next_ids, gaps, logits);
}

/* ---- portions of prompts, slots ----------------------------------------------------------------- */

gd_status gd_gpt_decoder_acquire(gd_gpt_decoder *d, int32_t *slot)
{
    int32_t b;
    if (d == NULL || slot == NULL) return GD_ERR_INVALID_ARGUMENT;
    for (b = 0; b < d->cfg.batch; ++b) {
        if (d->slot_taken[b]) continue;
        d->slot_taken[b] = true;
        d->pos[b] = 0;
        *slot = b;
        return GD_OK;
    }
    return GD_ERR_BUSY;
}

gd_status gd_gpt_decoder_release(gd_gpt_decoder *d, int32_t slot)
{
    if (d == NULL || slot < 0 || slot >= d->cfg.batch || !d->slot_taken[slot]) return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BUSY;
    d->slot_taken[slot] = false;
    d->pos[slot] = 0;
    return GD_OK;
}

gd_status gd_gpt_decoder_extend(gd_gpt_decoder *d, const int32_t *slots, int32_t n_seqs, const int32_t *ids,
                                const int32_t *cu, const int32_t *want, int32_t n_want, float *logits)
{
    gd_extend_rows e;
    gd_tensor t_logits;
    int32_t *start;
    gd_status st = GD_OK;
    int32_t s, i;
    if (d == NULL || slots == NULL || ids == NULL || cu == NULL || n_seqs <= 0 || n_seqs > d->cfg.batch || n_want < 0 ||
        (n_want > 0 && (want == NULL || logits == NULL)) || cu[0] != 0)
        return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BUSY;
    if (d->model->extend == NULL) return GD_ERR_UNSUPPORTED;
    e.max_new = 0;
    for (s = 0; s < n_seqs; ++s) {
        const int32_t n = cu[s + 1] - cu[s];
        if (n <= 0 || slots[s] < 0 || slots[s] >= d->cfg.batch || n > d->cfg.max_seq - d->pos[slots[s]])
            return GD_ERR_INVALID_ARGUMENT;
        for (i = 0; i < s; ++i) {
            if (slots[i] == slots[s]) return GD_ERR_INVALID_ARGUMENT;
        }
        if (n > e.max_new) e.max_new = n;
    }
    for (i = 0; i < n_want; ++i) {
        if (want[i] < 0 || want[i] >= cu[n_seqs]) return GD_ERR_INVALID_ARGUMENT;
    }
    start = (int32_t *)malloc((size_t)n_seqs * sizeof(int32_t));
    if (start == NULL) return GD_ERR_OUT_OF_MEMORY;
    for (s = 0; s < n_seqs; ++s) start[s] = d->pos[slots[s]];
    e.n_seqs = n_seqs;
    e.rows = cu[n_seqs];
    e.slots = slots;
    e.ids = ids;
    e.cu = cu;
    e.start = start;
    e.want = want;
    e.n_want = n_want;
    st = gd_begin_step(d->ctx, GD_SCOPE_INFER, gd_batch_empty());
    if (st == GD_OK) {
        gd_status end;
        st = d->model->extend(d, &e, &t_logits);
        end = gd_end_step(d->ctx);
        if (st == GD_OK) st = end;
    }
    free(start);
    if (st != GD_OK) return st;
    for (s = 0; s < n_seqs; ++s) d->pos[slots[s]] += cu[s + 1] - cu[s];
    if (n_want > 0) return gd_tensor_read_f32(d->ctx, &t_logits, logits, (size_t)n_want * (size_t)d->cfg.vocab);
    return gd_synchronize(d->ctx);
}

/* ---- device-resident decode -------------------------------------------------------------------- */

/* sampled pick instead of the greedy one: token, history, finished flags, feedback and records in two launches */
static gd_status enqueue_sample(gd_gpt_decoder *d, const gd_tensor *logits, int32_t pos_delta)
{
    gd_backend_tensor_view vl, vh, vhl, vf, vst, vw, vi, vp, vs, vo, vt, vx;
    gd_backend_sample_tensors t;
    gd_backend_sample_args a;
    tview(logits, &vl);
    tview(&d->history, &vh);
    view1(&d->hist_len, &vhl);
    view1(&d->finished, &vf);
    view1(&d->sample_state, &vst);
    view1(&d->sample_work, &vw);
    view1(&d->ids_dev, &vi);
    view1(&d->pos_dev, &vp);
    view1(&d->step_rows_dev, &vs);
    view1(&d->resident_out_ids, &vo);
    memset(&t, 0, sizeof(t));
    t.history = &vh;
    t.hist_len = &vhl;
    t.finished = &vf;
    t.state = &vst;
    t.work = &vw;
    t.ids = &vi;
    t.positions = &vp;
    t.step_counters = &vs;
    t.out_ids = &vo;
    if (d->resident_x0) {
        tview(&d->token_embedding, &vt);
        tview(&d->x0_dev, &vx);
        t.table = &vt;
        t.next_x = &vx;
    }
    a.temperature = d->sampling.temperature;
    a.min_p = d->sampling.min_p;
    a.repetition_penalty = d->sampling.repetition_penalty;
    a.logits_softcap = d->sampling.logits_softcap;
    a.stop_token = d->sampling.stop_token;
    a.pos_delta = pos_delta;
    return gd_backend_sample_advance(gd_context_backend(d->ctx), &vl, &t, &a);
}

/* GD_GPT_RESIDENT_KEEP_LOGITS: the step's logits into the state tensor that outlives the step scope */
static gd_status keep_logits(gd_gpt_decoder *d, const gd_tensor *logits)
{
    return gd_backend_copy(gd_context_backend(d->ctx), (gd_backend_buffer *)d->last_logits.storage.buffer,
                           d->last_logits.storage.offset + d->last_logits.view_offset,
                           (gd_backend_buffer *)logits->storage.buffer, logits->storage.offset + logits->view_offset,
                           (size_t)d->cfg.batch * (size_t)d->cfg.vocab * gd_dtype_size(logits->dtype));
}

static gd_status enqueue_resident_step(gd_gpt_decoder *d)
{
    gd_context *ctx = d->ctx;
    gd_tensor logits, next, gaps;
    gd_backend_tensor_view vl, vn, vg, vi, vp, vs, vo, vog, vt, vx;
    const int32_t delta = d->resident_hold ? 0 : 1;
    TRY(d->model->step(d, &d->ids_dev, &d->pos_dev, d->resident_unfused == 0, &logits));
    if (d->resident_sampling) return enqueue_sample(d, &logits, delta);
    if (d->resident_keep_logits) TRY(keep_logits(d, &logits));
    view1(&d->ids_dev, &vi);
    view1(&d->pos_dev, &vp);
    view1(&d->resident_out_ids, &vo);
    view1(&d->resident_out_gaps, &vog);
    if (!d->resident_unfused) {
        /* greedy pick, token feedback, position and record keeping in one launch */
        tview(&logits, &vl);
        view1(&d->step_rows_dev, &vs);
        if (d->resident_x0) {
            tview(&d->token_embedding, &vt);
            tview(&d->x0_dev, &vx);
        }
        return gd_backend_argmax_advance(gd_context_backend(ctx), &vl, &vi, &vp, &vs, &vo, &vog, delta,
                                         d->resident_x0 ? &vt : NULL, d->resident_x0 ? &vx : NULL);
    }
    TRY(gd_argmax_rows(ctx, &logits, &next, &gaps));
    view1(&next, &vn);
    view1(&gaps, &vg);
    view1(&d->step_dev, &vs);
    return gd_backend_decode_advance(gd_context_backend(ctx), &vn, &vg, &vi, &vp, &vs, &vo, &vog, delta);
}

static void resident_abort(gd_gpt_decoder *d)
{
    (void)gd_end_step(d->ctx);
    if (d->resident_graph != NULL) gd_backend_graph_destroy(d->resident_graph);
    d->resident_graph = NULL;
    d->resident_open = false;
    d->resident_sampling = false;
}

/* sampling == NULL: greedy session that starts from first_ids.  Otherwise: the session starts from the logits the
 * last prefill left in last_logits; max_steps counts picks (the one on those logits included), so at most
 * max_steps - 1 decode steps run; history / hist_len / finished / sample_state were set by the caller. */
static gd_status resident_begin_impl(gd_gpt_decoder *d, const int32_t *first_ids, int32_t max_steps, int32_t flags,
                                     const gd_gpt_sampling *sampling)
{
    const int32_t hold_positions = flags & GD_GPT_RESIDENT_HOLD_POSITIONS;
    gd_context *ctx;
    gd_backend *be;
    gd_status st;
    int64_t dims[1];
    int32_t b, zero = 0;
    if (d == NULL || (first_ids == NULL && sampling == NULL) || max_steps <= 0) return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BUSY;
    ctx = d->ctx;
    be = gd_context_backend(ctx);
    for (b = 0; b < d->cfg.batch; ++b) {
        /* a sampled session may run past the end of a cache: such rows have ended (their history is full), their
         * appends are skipped and their results ignored, as in the reference's loop */
        if (d->pos[b] < 0 || (sampling == NULL && d->pos[b] + (hold_positions ? 1 : max_steps) > d->cfg.max_seq))
            return GD_ERR_INVALID_ARGUMENT;
    }
    if (sampling == NULL) TRY(gd_tensor_write(ctx, &d->ids_dev, first_ids, (size_t)d->cfg.batch * sizeof(int32_t)));
    TRY(gd_tensor_write(ctx, &d->pos_dev, d->pos, (size_t)d->cfg.batch * sizeof(int32_t)));
    TRY(gd_tensor_write(ctx, &d->step_dev, &zero, sizeof(zero)));
    TRY(gd_tensor_zero_(ctx, &d->step_rows_dev));
    TRY(gd_begin_step(ctx, GD_SCOPE_INFER, gd_batch_empty()));
    d->resident_open = true;
    d->resident_graph = NULL;
    d->resident_max_steps = max_steps;
    d->resident_steps = 0;
    d->resident_hold = hold_positions != 0;
    d->resident_sampling = sampling != NULL;
    if (sampling != NULL) d->sampling = *sampling;
    d->resident_unfused = (flags & GD_GPT_RESIDENT_UNFUSED) != 0 || !d->model->can_fuse(d);
    d->resident_keep_logits = sampling == NULL && (flags & GD_GPT_RESIDENT_KEEP_LOGITS) != 0;
    dims[0] = (int64_t)max_steps * d->cfg.batch;
    st = gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_I32, gd_shape_make(1U, dims), 256U, &d->resident_out_ids);
    if (st == GD_OK) st = gd_tensor_empty(ctx, GD_ARENA_SCRATCH, GD_DTYPE_F32, gd_shape_make(1U, dims), 256U, &d->resident_out_gaps);
    /* fused step: the pick kernel leaves the next input rows in x0_dev; the first ones are gathered here */
    d->resident_x0 = !d->resident_unfused && d->model->feeds_x0(d);
    if (sampling != NULL) {
        /* pick number 0, on the prefill's logits: positions stay, the token becomes the first step's input */
        if (st == GD_OK) st = enqueue_sample(d, &d->last_logits, 0);
        max_steps -= 1; /* decode steps from here on */
    } else if (st == GD_OK && d->resident_x0) {
        gd_backend_tensor_view vt, vi, vx;
        gd_backend_embedding_args ea;
        tview(&d->token_embedding, &vt);
        tview(&d->ids_dev, &vi);
        tview(&d->x0_dev, &vx);
        ea.ids_count = (uint64_t)d->cfg.batch;
        ea.vocab = (uint64_t)d->cfg.vocab;
        ea.dim = (uint64_t)d->cfg.d_model;
        st = gd_backend_embedding_forward(be, &vt, &vi, &vx, &ea);
    }
    /* the first step runs eagerly (it also sizes the attention workspace); later steps replay a graph */
    if (st == GD_OK && max_steps > 0) {
        st = enqueue_resident_step(d);
        if (st == GD_OK) d->resident_steps = 1;
    }
    if (st == GD_OK && max_steps > 1) {
        st = gd_backend_graph_begin_capture(be);
        if (st == GD_OK) {
            st = enqueue_resident_step(d);
            if (st == GD_OK) st = gd_backend_graph_end_capture(be, &d->resident_graph);
            else (void)gd_backend_graph_end_capture(be, &d->resident_graph);
        }
    }
    if (st != GD_OK) resident_abort(d);
    return st;
}

gd_status gd_gpt_decoder_resident_begin(gd_gpt_decoder *d, const int32_t *first_ids, int32_t max_steps,
                                        int32_t flags)
{
    if (first_ids == NULL) return GD_ERR_INVALID_ARGUMENT;
    return resident_begin_impl(d, first_ids, max_steps, flags, NULL);
}

gd_status gd_gpt_decoder_resident_run(gd_gpt_decoder *d, int32_t n_steps)
{
    gd_backend *be;
    int32_t s;
    if (d == NULL || n_steps < 0) return GD_ERR_INVALID_ARGUMENT;
    if (!d->resident_open) return GD_ERR_BAD_STATE;
    if (d->resident_steps + n_steps > d->resident_max_steps - (d->resident_sampling ? 1 : 0)) return GD_ERR_INVALID_ARGUMENT;
    if (n_steps > 0 && d->resident_graph == NULL) return GD_ERR_BAD_STATE;
    be = gd_context_backend(d->ctx);
    for (s = 0; s < n_steps; ++s) {
        TRY(gd_backend_graph_launch(be, d->resident_graph));
        d->resident_steps += 1;
    }
    return GD_OK;
}

gd_status gd_gpt_decoder_resident_sync(gd_gpt_decoder *d)
{
    if (d == NULL) return GD_ERR_INVALID_ARGUMENT;
    return gd_synchronize(d->ctx);
}

gd_status gd_gpt_decoder_resident_end(gd_gpt_decoder *d, int32_t *out_ids, float *out_gaps, int32_t *steps_done)
{
    gd_context *ctx;
    gd_status st;
    gd_tensor ids_view, gaps_view;
    int32_t b, records;
    if (d == NULL) return GD_ERR_INVALID_ARGUMENT;
    if (!d->resident_open) return GD_ERR_BAD_STATE;
    ctx = d->ctx;
    st = gd_end_step(ctx);
    /* a sampled session has one record more than decode steps: the pick on the prefill's logits */
    records = d->resident_steps + (d->resident_sampling ? 1 : 0);
    if (st == GD_OK && out_ids != NULL) {
        st = gd_tensor_slice(ctx, &d->resident_out_ids, 0U, 0, (int64_t)records * d->cfg.batch, &ids_view);
        if (st == GD_OK) st = gd_tensor_read(ctx, &ids_view, out_ids, (size_t)records * (size_t)d->cfg.batch * sizeof(int32_t));
    }
    if (st == GD_OK && out_gaps != NULL && !d->resident_sampling) {
        st = gd_tensor_slice(ctx, &d->resident_out_gaps, 0U, 0, (int64_t)d->resident_steps * d->cfg.batch, &gaps_view);
        if (st == GD_OK) st = gd_tensor_read(ctx, &gaps_view, out_gaps, (size_t)d->resident_steps * (size_t)d->cfg.batch * sizeof(float));
    }
    if (d->resident_graph != NULL) gd_backend_graph_destroy(d->resident_graph);
    d->resident_graph = NULL;
    d->resident_open = false;
    d->resident_sampling = false;
    if (steps_done != NULL) *steps_done = records;
    if (st == GD_OK && !d->resident_hold) {
        for (b = 0; b < d->cfg.batch; ++b) d->pos[b] += d->resident_steps;
    }
    return st;
}

gd_status gd_gpt_decoder_resident_begin_sampled(gd_gpt_decoder *d, const int32_t *ids, const int32_t *cu,
                                                int32_t max_picks, int32_t flags, const gd_gpt_sampling *sampling)
{
    gd_context *ctx;
    gd_tensor head_words;
    int32_t *hist, *lens;
    int32_t state_words[8];
    int32_t B, b;
    gd_status st;
    if (d == NULL || ids == NULL || cu == NULL || sampling == NULL || max_picks <= 0 || cu[0] != 0 ||
        sampling->stop_token >= d->cfg.vocab)
        return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BAD_STATE;
    ctx = d->ctx;
    B = d->cfg.batch;
    if (B <= 0) return GD_ERR_BAD_STATE;
    for (b = 0; b < B; ++b) {
        if (cu[b + 1] < cu[b] || cu[b + 1] - cu[b] > d->cfg.max_seq) return GD_ERR_INVALID_ARGUMENT;
    }
    hist = (int32_t *)calloc((size_t)B * (size_t)d->cfg.max_seq, sizeof(int32_t));
    lens = (int32_t *)calloc((size_t)B, sizeof(int32_t));
    if (hist == NULL || lens == NULL) {
        free(hist); free(lens);
        return GD_ERR_OUT_OF_MEMORY;
    }
    for (b = 0; b < B; ++b) {
        lens[b] = cu[b + 1] - cu[b];
        memcpy(hist + (size_t)b * (size_t)d->cfg.max_seq, ids + cu[b], (size_t)lens[b] * sizeof(int32_t));
    }
    memset(state_words, 0, sizeof(state_words));
    memcpy(&state_words[0], &sampling->rng_state, sizeof(uint64_t));
    memcpy(&state_words[2], &sampling->rng_state, sizeof(uint64_t));
    st = gd_tensor_slice(ctx, &d->sample_state, 0U, 0, 8, &head_words);
    if (st == GD_OK) st = gd_tensor_write(ctx, &head_words, state_words, sizeof(state_words));
    if (st == GD_OK) st = gd_tensor_write(ctx, &d->history, hist, (size_t)B * (size_t)d->cfg.max_seq * sizeof(int32_t));
    if (st == GD_OK) st = gd_tensor_write(ctx, &d->hist_len, lens, (size_t)B * sizeof(int32_t));
    if (st == GD_OK) st = gd_tensor_zero_(ctx, &d->finished);
    free(hist); free(lens);
    if (st != GD_OK) return st;
    return resident_begin_impl(d, NULL, max_picks, flags, sampling);
}

/* ---- generation with the sampling front end ---------------------------------------------- */

uint64_t gd_gpt_generation_rng(uint64_t seed, int32_t n_prompts, uint64_t step)
{
    return gd_splitmix64(seed ^ UINT64_C(0xdec0de1234567890) ^ (uint64_t)n_prompts ^ step);
}

gd_status gd_gpt_decoder_generate(gd_gpt_decoder *d, const int32_t *ids, const int32_t *cu, int32_t max_new,
                                  const gd_gpt_sampling *sampling, int32_t *out_tokens, int32_t *out_counts)
{
    const int32_t check_every = 32; /* decode steps between two looks at the finished flags */
    gd_context *ctx;
    int32_t *packed = NULL, *pcu = NULL, *lens = NULL, *records = NULL, *flags = NULL;
    int32_t B, ctx_len, room, b, total = 0, done = 0, decode_steps;
    gd_status st;
    if (d == NULL || ids == NULL || cu == NULL || sampling == NULL || out_tokens == NULL || out_counts == NULL ||
        max_new <= 0)
        return GD_ERR_INVALID_ARGUMENT;
    if (d->resident_open) return GD_ERR_BUSY;
    ctx = d->ctx;
    B = d->cfg.batch;
    ctx_len = d->cfg.max_seq;
    if (sampling->stop_token >= d->cfg.vocab || cu[0] != 0) return GD_ERR_INVALID_ARGUMENT;
    /* reference :1514-1518: the prompt may use what the new tokens leave of the context, at least one row short of it */
    room = max_new >= ctx_len ? ctx_len - 1 : ctx_len - max_new;
    if (room <= 0) return GD_ERR_INVALID_ARGUMENT;
    for (b = 0; b < B; ++b) {
        if (cu[b + 1] <= cu[b]) return GD_ERR_INVALID_ARGUMENT; /* empty prompt (:1520-1522) */
    }
    pcu = (int32_t *)calloc((size_t)B + 1U, sizeof(int32_t));
    lens = (int32_t *)calloc((size_t)B, sizeof(int32_t));
    flags = (int32_t *)calloc((size_t)B, sizeof(int32_t));
    records = (int32_t *)malloc((size_t)max_new * (size_t)B * sizeof(int32_t));
    if (pcu == NULL || lens == NULL || flags == NULL || records == NULL) {
        st = GD_ERR_OUT_OF_MEMORY;
        goto out;
    }
    /* a prompt longer than the room keeps its last tokens (:1523-1533) */
    for (b = 0; b < B; ++b) {
        const int32_t n = cu[b + 1] - cu[b];
        lens[b] = n > room ? room : n;
        pcu[b + 1] = pcu[b] + lens[b];
    }
    total = pcu[B];
    packed = (int32_t *)malloc((size_t)total * sizeof(int32_t));
    if (packed == NULL) {
        st = GD_ERR_OUT_OF_MEMORY;
        goto out;
    }
    for (b = 0; b < B; ++b) {
        const int32_t *src = ids + cu[b + 1] - lens[b];
        memcpy(packed + pcu[b], src, (size_t)lens[b] * sizeof(int32_t));
    }
    st = gd_gpt_decoder_prefill(d, packed, pcu, NULL, NULL, NULL); /* leaves the logits in last_logits */
    if (st == GD_OK) st = gd_gpt_decoder_resident_begin_sampled(d, packed, pcu, max_new, 0, sampling);
    if (st != GD_OK) goto out;
    /* the reference leaves its loop when every row has ended (:1607, 1634-1636): look at the flags now and then */
    decode_steps = max_new - 1;
    while (d->resident_steps < decode_steps) {
        int32_t n = decode_steps - d->resident_steps, alive = 0;
        if (n > check_every) n = check_every;
        st = gd_gpt_decoder_resident_run(d, n);
        if (st == GD_OK && d->resident_steps < decode_steps) {
            st = gd_tensor_read(ctx, &d->finished, flags, (size_t)B * sizeof(int32_t));
            for (b = 0; b < B; ++b) alive += flags[b] == 0;
        } else {
            alive = 1;
        }
        if (st != GD_OK) {
            resident_abort(d);
            goto out;
        }
        if (alive == 0) break;
    }
    st = gd_gpt_decoder_resident_end(d, records, NULL, &done);
    if (st != GD_OK) goto out;
    for (b = 0; b < B; ++b) {
        int32_t s, n = 0;
        for (s = 0; s < done; ++s) {
            const int32_t token = records[(size_t)s * (size_t)B + (size_t)b];
            if (token >= 0) out_tokens[(size_t)b * (size_t)max_new + (size_t)n++] = token;
        }
        out_counts[b] = n;
    }
out:
    free(packed); free(pcu); free(lens); free(records); free(flags);
    return st;
}

gd_status gd_gpt_decoder_run_resident(gd_gpt_decoder *d, const int32_t *first_ids, int32_t n_steps, int32_t *out_ids,
                                      float *out_gaps, float *step_ms)
{
    gd_backend_timer *timer = NULL;
    gd_status st;
    float ms = 0.0f;
    if (d == NULL || n_steps <= 0 || out_ids == NULL) return GD_ERR_INVALID_ARGUMENT;
    TRY(gd_gpt_decoder_resident_begin(d, first_ids, n_steps, 0));
    st = GD_OK;
    if (step_ms != NULL) st = gd_backend_timer_create(gd_context_backend(d->ctx), &timer);
    if (st == GD_OK && timer != NULL) st = gd_backend_timer_start(timer);
    if (st == GD_OK) st = gd_gpt_decoder_resident_run(d, n_steps - 1);
    if (st == GD_OK && timer != NULL) st = gd_backend_timer_stop(timer);
    if (st != GD_OK) {
        resident_abort(d);
    } else {
        st = gd_gpt_decoder_resident_end(d, out_ids, out_gaps, NULL);
        if (st == GD_OK && timer != NULL) st = gd_backend_timer_elapsed_ms(timer, &ms);
    }
    if (timer != NULL) gd_backend_timer_destroy(timer);
    if (step_ms != NULL) *step_ms = n_steps > 1 ? ms / (float)(n_steps - 1) : 0.0f;
    return st;
}
