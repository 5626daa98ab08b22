/*
 * The decoder whose layers are listed in a configuration (layer_list.h): caches, states, and one forward over packed new
 * tokens that serves prompts, portions of prompts and decode steps alike.
 *
 * The residual stream x is F32; h is what a sublayer reads, in the projections' type.
 *   mixer   mamba2              in -> causal conv + silu -> recurrence -> gate, group norm -> out
 *           latent_attention    [dq | dkv | g] -> norms, rotation, cache append -> uq -> attention, output gate -> out
 *           grouped attention   [q | k | v | g] -> rotation, attention, output gate, cache append -> out
 *   feed-forward  gelu(gate) * up with biases -> down;  relu(up)^2 -> down;  routed experts and a shared one
 * Norms on the outputs:  x += m * norm1(mixer(h)), h = x;  x += m * norm2(ff(h)), h = x.
 * Norms first:  h = norm1(x), x += mixer(h);  h = norm2(x), x += ff(h): a sublayer's result is added together with the norm in
 * front of the next one, so that the stream is read and written once per sublayer.
 * Projections that read the same input are one weight matrix.  What a sequence keeps: the convolution's last inputs and
 * the recurrent state (mamba2), the latent and the rotated key part of every token (latent_attention), rotated keys and
 * values of every token, or with chunks of the current chunk's (grouped attention), each in the place of its slot;
 * positions decide what of it is read, so nothing is cleared when a slot is used again.
 */
#include <math.h>
#include <stdio.h>

#include "layer_list_internal.h"

/* ---- caches and states ----------------------------------------------------------------------------- */

/* what a layer keeps: mamba2 its ring and states, latent attention its cache, grouped attention keys and values */
typedef struct state_shapes {
    int64_t ring[3], states[4], cache[3], k[4], v[4];
} state_shapes;

static state_shapes state_dims(const layer_config *l, int64_t slots, int64_t max_seq)
{
    state_shapes s;
    memset(&s, 0, sizeof(s));
    s.ring[0] = s.states[0] = s.cache[0] = s.k[0] = s.v[0] = slots;
    s.ring[1] = l->taps;
    s.ring[2] = conv_channels(l);
    s.states[1] = l->ssm.heads;
    s.states[2] = l->ssm.state;
    s.states[3] = l->ssm.vdim;
    s.cache[1] = max_seq;
    s.cache[2] = gd_backend_latent_pitch(l->latent.kv_rank, l->latent.rot_dim);
    s.k[1] = s.v[1] = l->grouped.kv_heads;
    s.k[2] = s.v[2] = l->grouped.chunk > 0U && l->grouped.chunk < max_seq ? l->grouped.chunk : max_seq;
    s.k[3] = l->grouped.dim;
    s.v[3] = l->grouped.vdim;
    return s;
}

static size_t dims_bytes(const int64_t *dims, int rank, size_t es)
{
    int i;
    for (i = 0; i < rank; ++i) es *= (size_t)dims[i];
    return gd_pad256(es);
}

/* the tables of a routed layer for steps of up to `rows` tokens: place, first, tiles */
static void route_dims(const layer_config *l, int64_t rows, int64_t dims[3])
{
    dims[0] = rows * l->routed.top;
    dims[1] = (int64_t)l->routed.experts + 1;
    dims[2] = 2 + 2 * (int64_t)gd_backend_route_tiles(&l->routed, (uint32_t)rows, 1U);
}

static size_t state_bytes(const layer_list_config *c, gd_dtype type, int64_t slots, int64_t max_seq, int64_t step_tokens)
{
    const size_t es = gd_dtype_size(type);
    size_t total = 0U;
    int32_t i, t;
    for (i = 0; i < c->n_layers; ++i) {
        const layer_config *l = &c->layers[i];
        const state_shapes s = state_dims(l, slots, max_seq);
        if (l->mixer == MIXER_MAMBA2) total += dims_bytes(s.ring, 3, es) + dims_bytes(s.states, 4, 4U);
        else if (l->mixer == MIXER_LATENT_ATTENTION) total += dims_bytes(s.cache, 3, es);
        else total += dims_bytes(s.k, 4, es) + dims_bytes(s.v, 4, es);
        if (l->mlp == MLP_ROUTED && l->weights_of == i) {
            int64_t r[3];
            route_dims(l, step_tokens, r);
            for (t = 0; t < 3; ++t) total += dims_bytes(&r[t], 1, 4U);
        }
    }
    return total + 2U * gd_pad256((size_t)(slots + 1) * 4U);
}

static gd_status state_zeros(gd_context *ctx, gd_dtype type, uint32_t rank, int64_t *dims, gd_tensor *out)
{
    return gd_tensor_zeros(ctx, GD_ARENA_STATE, type, gd_shape_make(rank, dims), 256U, out);
}

static gd_status allocate_layer_state(gd_context *ctx, struct layer_list *ll, int32_t i, int64_t slots, int64_t max_seq)
{
    const layer_config *l = &ll->c.layers[i];
    layer_weights *w = &ll->layers[i];
    state_shapes s = state_dims(l, slots, max_seq);
    if (l->mixer == MIXER_MAMBA2) {
        TRY(state_zeros(ctx, ll->type, 3U, s.ring, &w->ring));
        TRY(state_zeros(ctx, GD_DTYPE_F32, 4U, s.states, &w->states));
    } else if (l->mixer == MIXER_LATENT_ATTENTION) {
        TRY(state_zeros(ctx, ll->type, 3U, s.cache, &w->cache));
    } else {
        TRY(state_zeros(ctx, ll->type, 4U, s.k, &w->k_cache));
        TRY(state_zeros(ctx, ll->type, 4U, s.v, &w->v_cache));
    }
    if (l->mlp == MLP_ROUTED && l->weights_of == i) {
        int64_t r[3];
        route_dims(l, ll->max_step_tokens, r);
        TRY(state_zeros(ctx, GD_DTYPE_I32, 1U, &r[0], &w->place));
        TRY(state_zeros(ctx, GD_DTYPE_I32, 1U, &r[1], &w->first));
        TRY(state_zeros(ctx, GD_DTYPE_I32, 1U, &r[2], &w->tiles));
    }
    return GD_OK;
}

static gd_status allocate_states(gd_context *ctx, struct layer_list *ll, int64_t slots, int64_t max_seq)
{
    int64_t bdim[1] = {slots}, cdim[1] = {slots + 1};
    int32_t *iota = (int32_t *)malloc((size_t)(slots + 1) * sizeof(int32_t));
    gd_status st = iota == NULL ? GD_ERR_OUT_OF_MEMORY : GD_OK;
    int32_t i;
    for (i = 0; i < ll->c.n_layers && st == GD_OK; ++i) st = allocate_layer_state(ctx, ll, i, slots, max_seq);
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
    int64_t packed, packed_ff;  /* elements for the whole step: packed rows of the routed experts, and their activations */
} scratch_sizes;

static int64_t max64(int64_t a, int64_t b) { return a > b ? a : b; }

static scratch_sizes sizes_of(const layer_list_config *c, gd_dtype type, int64_t rows, int64_t max_new, int64_t kv_total,
                              int64_t max_seq)
{
    scratch_sizes s = {0, c->width, 1, c->width, 1, 256U, 1, 1};
    int32_t i;
    for (i = 0; i < c->n_layers; ++i) {
        const layer_config *l = &c->layers[i];
        s.proj = max64(s.proj, mixer_pitch(l));
        if (l->mixer == MIXER_MAMBA2) {
            s.a = max64(s.a, max64(conv_channels(l), inner_size(l)));
            s.b = max64(s.b, inner_size(l));
        } else if (l->mixer == MIXER_GROUPED_ATTENTION) {
            const size_t w = gd_backend_grouped_work_bytes(NULL, &l->grouped, (uint32_t)rows, (uint32_t)max_new,
                                                           (uint32_t)max_seq, (uint32_t)type);
            s.a = max64(s.a, mixer_out(l));
            if (w > s.work) s.work = w;
        } else {
            const size_t w = gd_backend_latent_work_bytes(NULL, &l->latent, (uint32_t)rows, (uint32_t)max_new, (uint32_t)kv_total,
                                                          (uint32_t)max_seq, (uint32_t)type);
            s.angles = max64(s.angles, l->latent.rot_dim);
            s.a = max64(s.a, max64(l->latent.q_rank, mixer_out(l)));
            s.b = max64(s.b, query_size(l));
            if (w > s.work) s.work = w;
        }
        s.a = max64(s.a, max64(l->ff, l->shared_ff));
        if (l->mlp == MLP_ROUTED) {
            const int64_t packed = rows * l->routed.top + GD_BACKEND_ROUTED_PAD;
            s.packed = max64(s.packed, packed * c->width);
            s.packed_ff = max64(s.packed_ff, packed * l->routed.ff);
        }
    }
    return s;
}

static size_t forward_bytes(const layer_list_config *c, const scratch_sizes *s, gd_dtype type, int64_t rows)
{
    const size_t es = gd_dtype_size(type), R = (size_t)rows;
    return gd_pad256(R * (size_t)c->width * 4U) + gd_pad256(R * (size_t)c->width * es) + gd_pad256(R * (size_t)s->proj * es) +
           gd_pad256(R * (size_t)s->a * es) + gd_pad256(R * (size_t)s->b * es) + gd_pad256(R * (size_t)s->branch * es) +
           gd_pad256(R * (size_t)s->angles * 4U) + gd_pad256(s->work) + 2U * gd_pad256((size_t)s->packed * es) +
           gd_pad256((size_t)s->packed_ff * es);
}

typedef struct forward {
    gd_gpt_decoder *d;
    gd_backend *be;
    struct layer_list *ll;
    uint32_t type;
    int64_t rows;
    gd_backend_packed_seqs seqs;
    gd_backend_tensor_view row_seq, cu, slot, start, kv_cu, ids;
    gd_tensor x, h, proj, a, b, branch, angles, work; /* h: what a sublayer reads; x itself when that is an F32 copy */
    gd_tensor packed, packed_act, packed_out;         /* of the routed experts */
    /* norms first: what waits to be added to the stream */
    bool branch_waits;
    layer_weights *routed_waits;
    const layer_config *routed_config;
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
    if (ll->type == GD_DTYPE_F32 && !ll->c.norms_first) f->h = f->x;
    else TRY(scratch(d->ctx, ll->type, rows, ll->c.width, &f->h));
    TRY(scratch(d->ctx, ll->type, rows, s.proj, &f->proj));
    TRY(scratch(d->ctx, ll->type, rows, s.a, &f->a));
    TRY(scratch(d->ctx, ll->type, rows, s.b, &f->b));
    TRY(scratch(d->ctx, GD_DTYPE_F32, rows, s.angles, &f->angles));
    TRY(scratch(d->ctx, ll->type, rows, s.branch, &f->branch));
    TRY(scratch(d->ctx, ll->type, 1, s.packed, &f->packed));
    TRY(scratch(d->ctx, ll->type, 1, s.packed_ff, &f->packed_act));
    TRY(scratch(d->ctx, ll->type, 1, s.packed, &f->packed_out));
    f->branch_waits = false;
    f->routed_waits = NULL;
    return gd_tensor_empty(d->ctx, GD_ARENA_SCRATCH, GD_DTYPE_U8, gd_shape_make(1U, wdim), 256U, &f->work);
}

static bool epilogue_gated(uint32_t epilogue)
{
    return epilogue != 0U && epilogue != GD_BACKEND_EPILOGUE_SQUARE_RELU;
}

/* y [rows, outputs] = x [rows, w cols] w^T (+ bias) with the epilogue of args, buffers holding rows `pitch` apart
 * (0: packed) */
static gd_status project_as(forward *f, const gd_tensor *x, const gd_tensor *w, const gd_tensor *bias,
                            gd_backend_fused_linear_args args, int64_t pitch, gd_tensor *y)
{
    const int64_t outs = epilogue_gated(args.epilogue) ? w->shape[0] / 2 : w->shape[0];
    gd_backend_matrix_view xm, wm, ym;
    gd_backend_vector_view bv;
    args.w_is_nk = 1U;
    args.bias_mode = bias != NULL ? 1U : 0U;
    columns(x, f->type, f->rows, w->shape[1], 0, w->shape[1], &xm);
    mview(w, w->shape[0], w->shape[1], &wm);
    columns(y, f->type, f->rows, pitch > 0 ? pitch : outs, 0, outs, &ym);
    if (bias != NULL) vview(bias, &bv);
    return gd_backend_fused_linear(f->be, &xm, &wm, bias != NULL ? &bv : NULL, NULL, NULL, &ym, &args);
}

static gd_status project(forward *f, const gd_tensor *x, const gd_tensor *w, const gd_tensor *bias, uint32_t epilogue,
                         gd_tensor *y)
{
    gd_backend_fused_linear_args args;
    memset(&args, 0, sizeof(args));
    args.epilogue = epilogue;
    return project_as(f, x, w, bias, args, 0, y);
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

static gd_status grouped_attention(forward *f, const layer_config *l, layer_weights *w)
{
    const gd_backend_fused_linear_args plain = {0U, 0U, 0U, 0.0f, 0U, 0.0f, 0.0f};
    gd_backend_matrix_view pm;
    gd_backend_tensor_view freq, kc, vc, work, out;
    TRY(project_as(f, &f->h, &w->in, NULL, plain, mixer_pitch(l), &f->proj));
    columns(&f->proj, f->type, f->rows, mixer_pitch(l), 0, mixer_in(l), &pm);
    tview(&w->freq, &freq);
    tview(&w->k_cache, &kc);
    tview(&w->v_cache, &vc);
    tview(&f->work, &work);
    view2(&f->a, f->type, f->rows, mixer_out(l), &out);
    TRY(gd_backend_grouped_attend(f->be, &pm, &freq, &kc, &vc, &work, &out, &f->seqs, &l->grouped));
    return project(f, &f->a, &w->out, NULL, 0U, &f->branch);
}

static gd_status mixer(forward *f, const layer_config *l, layer_weights *w)
{
    if (l->mixer == MIXER_MAMBA2) return mamba2(f, l, w);
    if (l->mixer == MIXER_LATENT_ATTENTION) return latent_attention(f, l, w);
    return grouped_attention(f, l, w);
}

/* the step's tables of a routed layer (its weights' owner holds them) and, packed by expert, a buffer's rows */
static void routes_of(const forward *f, const layer_config *l, const layer_weights *w, gd_backend_tensor_view *place,
                      gd_backend_tensor_view *first, gd_backend_tensor_view *tiles)
{
    tview(&w->place, place);
    tview(&w->first, first);
    tview(&w->tiles, tiles);
    place->shape[0] = f->rows * l->routed.top;
    place->count = (size_t)place->shape[0];
}

static void packed_rows(const forward *f, const layer_config *l, const gd_tensor *t, int64_t cols, gd_backend_tensor_view *v)
{
    view2(t, f->type, f->rows * l->routed.top + GD_BACKEND_ROUTED_PAD, cols, v);
}

/* which rows go to which expert, for every table of the model: the token ids alone decide */
static gd_status route(forward *f)
{
    enum { BATCH = 64 };
    gd_backend_route_job jobs[BATCH];
    gd_backend_tensor_view table[BATCH], place[BATCH], first[BATCH], tiles[BATCH];
    uint32_t n = 0U;
    int32_t i;
    for (i = 0; i < f->ll->c.n_layers; ++i) {
        const layer_config *l = &f->ll->c.layers[i];
        layer_weights *w = &f->ll->layers[i];
        if (l->mlp != MLP_ROUTED || l->weights_of != i) continue;
        tview(&w->table, &table[n]);
        routes_of(f, l, w, &place[n], &first[n], &tiles[n]);
        jobs[n].table = &table[n];
        jobs[n].place = &place[n];
        jobs[n].first = &first[n];
        jobs[n].tiles = &tiles[n];
        jobs[n].args = &l->routed;
        if (++n < BATCH) continue;
        TRY(gd_backend_route_by_tables(f->be, jobs, n, &f->ids, f->type));
        n = 0U;
    }
    return n > 0U ? gd_backend_route_by_tables(f->be, jobs, n, &f->ids, f->type) : GD_OK;
}

/* x += what waits;  h = norm(x) * weight (NULL: only the sum);  rows of a routed feed-forward that follows are packed */
static gd_status settle_stream(forward *f, const gd_tensor *norm, const layer_config *next, layer_weights *next_w,
                               gd_tensor *h)
{
    const int64_t W = f->ll->c.width;
    gd_backend_tensor_view vb, vn, vx, vh, place_in, place_out, first, tiles, rows_in, rows_out;
    gd_backend_routed_rows in, out;
    view2(&f->branch, f->type, f->rows, W, &vb);
    view2(&f->x, GD_BACKEND_DTYPE_F32, f->rows, W, &vx);
    view2(h, f->type, f->rows, W, &vh);
    if (norm != NULL) tview(norm, &vn);
    if (f->routed_waits != NULL) {
        routes_of(f, f->routed_config, f->routed_waits, &place_in, &first, &tiles);
        packed_rows(f, f->routed_config, &f->packed_out, W, &rows_in);
        in.rows = &rows_in;
        in.place = &place_in;
        in.top = f->routed_config->routed.top;
        in.weight = f->routed_config->routed.weight;
    }
    if (next != NULL) {
        routes_of(f, next, next_w, &place_out, &first, &tiles);
        packed_rows(f, next, &f->packed, W, &rows_out);
        out.rows = &rows_out;
        out.place = &place_out;
        out.top = next->routed.top;
        out.weight = 1.0f;
    }
    TRY(gd_backend_residual_add_norm(f->be, f->branch_waits ? &vb : NULL, f->routed_waits != NULL ? &in : NULL, &vx,
                                     norm != NULL ? &vn : NULL, norm != NULL ? &vh : NULL, next != NULL ? &out : NULL,
                                     f->ll->c.eps));
    f->branch_waits = false;
    f->routed_waits = NULL;
    return GD_OK;
}

static gd_status square_relu(forward *f, layer_weights *w)
{
    TRY(project(f, &f->h, &w->upgate, NULL, GD_BACKEND_EPILOGUE_SQUARE_RELU, &f->a));
    f->branch_waits = true;
    return project(f, &f->a, &w->down, NULL, 0U, &f->branch);
}

/* the packed rows (settle_stream) through their experts, and all rows through the shared one */
static gd_status routed(forward *f, const layer_config *l, layer_weights *w)
{
    gd_backend_tensor_view rows, act, out, up, down, place, first, tiles;
    gd_backend_routes routes;
    routes_of(f, l, w, &place, &first, &tiles);
    packed_rows(f, l, &f->packed, l->routed.width, &rows);
    packed_rows(f, l, &f->packed_act, l->routed.ff, &act);
    packed_rows(f, l, &f->packed_out, l->routed.width, &out);
    tview(&w->expert_upgate, &up);
    tview(&w->expert_down, &down);
    routes.first = &first;
    routes.tiles = &tiles;
    routes.rows = (uint32_t)f->rows;
    TRY(gd_backend_routed_mlp(f->be, &rows, &up, &down, &act, &out, &routes, &l->routed));
    f->routed_waits = w;
    f->routed_config = l;
    if (l->shared_ff > 0) {
        const gd_backend_fused_linear_args gate = {0U, 0U, 0U, 0.0f, GD_BACKEND_EPILOGUE_CLAMPED_GATE, l->shared_limit,
                                                   l->routed.gate_alpha};
        TRY(project_as(f, &f->h, &w->upgate, NULL, gate, 0, &f->a));
        TRY(project(f, &f->a, &w->down, NULL, 0U, &f->branch));
        f->branch_waits = true;
    }
    return GD_OK;
}

/* Norms in front of the sublayers.  all_normed: the last norm of every row is left in f->h; otherwise only the stream
 * is complete. */
static gd_status run_norms_first(forward *f, bool all_normed)
{
    const layer_list_config *c = &f->ll->c;
    int32_t i;
    TRY(route(f));
    TRY(settle_stream(f, &f->ll->layers[0].norm1, NULL, NULL, &f->h));
    for (i = 0; i < c->n_layers; ++i) {
        const layer_config *l = &c->layers[i];
        layer_weights *w = &f->ll->layers[i], *owner = &f->ll->layers[l->weights_of];
        const bool last = i + 1 == c->n_layers;
        TRY(mixer(f, l, w));
        f->branch_waits = true;
        if (l->mlp != MLP_NONE) {
            TRY(settle_stream(f, &w->norm2, l->mlp == MLP_ROUTED ? l : NULL, owner, &f->h));
            if (l->mlp == MLP_ROUTED) TRY(routed(f, l, owner));
            else TRY(square_relu(f, w));
        }
        TRY(settle_stream(f, !last ? &f->ll->layers[i + 1].norm1 : all_normed ? &f->ll->final_norm : NULL, NULL, NULL, &f->h));
    }
    return GD_OK;
}

static gd_status run_norms_behind(forward *f)
{
    int32_t i;
    for (i = 0; i < f->ll->c.n_layers; ++i) {
        const layer_config *l = &f->ll->c.layers[i];
        layer_weights *w = &f->ll->layers[i];
        TRY(mixer(f, l, w));
        TRY(add_branch(f, &w->norm1));
        if (l->mlp == MLP_GELU_GATED) {
            TRY(project(f, &f->h, &w->upgate, &w->upgate_b, GD_BACKEND_EPILOGUE_GELU_GATE, &f->a));
            TRY(project(f, &f->a, &w->down, &w->down_b, 0U, &f->branch));
            TRY(add_branch(f, &w->norm2));
        }
    }
    return GD_OK;
}

/* every layer over the rows of f, from the token ids to the residual stream in f->x (see run_norms_first) */
static gd_status run_layers(forward *f, bool all_normed)
{
    const int64_t W = f->ll->c.width;
    const bool copy = !f->ll->c.norms_first && f->ll->type != GD_DTYPE_F32;
    gd_backend_tensor_view ve, vx, vh;
    tview(&f->ll->embed, &ve);
    view2(&f->x, GD_BACKEND_DTYPE_F32, f->rows, W, &vx);
    view2(&f->h, f->type, f->rows, W, &vh);
    TRY(gd_backend_residual_embed(f->be, &ve, &f->ids, &vx, copy ? &vh : NULL, f->ll->c.embedding_scale));
    return f->ll->c.norms_first ? run_norms_first(f, all_normed) : run_norms_behind(f);
}

/* F32 logits of the picked rows (NULL: of all rows, whose last norm may already be in f->h) */
static gd_status head(forward *f, const gd_backend_tensor_view *rows, int64_t n, bool normed, gd_tensor *logits)
{
    const layer_list_config *c = &f->ll->c;
    const gd_tensor *weight = c->own_head ? &f->ll->head : &f->ll->embed;
    gd_backend_tensor_view vx, vn, vo;
    gd_backend_matrix_view xm, wm, ym;
    gd_tensor last = f->h;
    TRY(scratch(f->d->ctx, GD_DTYPE_F32, n, c->vocab, logits));
    if (!normed) {
        TRY(scratch(f->d->ctx, f->ll->type, n, c->width, &last));
        view2(&f->x, GD_BACKEND_DTYPE_F32, f->rows, c->width, &vx);
        tview(&f->ll->final_norm, &vn);
        tview(&last, &vo);
        TRY(gd_backend_residual_norm_rows(f->be, &vx, rows, &vn, &vo, c->eps));
    }
    mview(&last, n, c->width, &xm);
    mview(weight, c->vocab, c->width, &wm);
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
    TRY(run_layers(&f, true));
    return head(&f, NULL, f.rows, d->layers->c.norms_first, logits);
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
    TRY(run_layers(&f, false));
    if (e->n_want == 0) return GD_OK;
    view1(&part[WANT], &want);
    return head(&f, &want, e->n_want, false, logits);
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
    if (!strcmp(name, "head") && ll->c.own_head) return &ll->head;
    if (!strcmp(name, "final_norm")) return &ll->final_norm;
    if (layer < 0 || layer >= ll->c.n_layers) return NULL;
    w = &ll->layers[layer];
    if (!strcmp(name, "cache") && ll->c.layers[layer].mixer == MIXER_LATENT_ATTENTION) return &w->cache;
    if (ll->c.layers[layer].mixer == MIXER_GROUPED_ATTENTION) {
        if (!strcmp(name, "k_cache")) return &w->k_cache;
        if (!strcmp(name, "v_cache")) return &w->v_cache;
    }
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

#define LAYER_LIST_MODEL(name)                                                                                         \
    {name, layer_list_prefill, layer_list_step, layer_list_extend, layer_list_can_fuse, layer_list_feeds_x0,           \
     layer_list_tensor, layer_list_destroy}
static const gd_decoder_model layer_list_models[] = {LAYER_LIST_MODEL("Girirax"), LAYER_LIST_MODEL("Bonatar")};

static const gd_decoder_model *model_of(const layer_list_config *c)
{
    size_t i;
    for (i = 0U; i < sizeof(layer_list_models) / sizeof(layer_list_models[0]); ++i) {
        if (!strcmp(layer_list_models[i].architecture, c->architecture)) return &layer_list_models[i];
    }
    return NULL;
}

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
    g->tie_lm_head = c->own_head ? 0 : 1;
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
    size_t rows, logit_rows, step;
    scratch_sizes s;
    TRY(settle(c, in, &o, &g));
    rows = (size_t)o.max_step_tokens;
    logit_rows = ((size_t)1 << 30) / ((size_t)c->vocab * 4U);
    if (logit_rows > rows) logit_rows = rows;
    *out = gd_memory_config_default();
    out->params_bytes = gd_layer_list_weight_bytes(c, o.compute) + 4096U;
    out->state_bytes = state_bytes(c, o.compute, o.batch, o.max_seq, o.max_step_tokens) + gd_decoder_session_bytes(&g, GD_DTYPE_F32, false) + 4096U;
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
    if (model_of(c) == NULL) return GD_ERR_UNSUPPORTED;
    TRY(gd_decoder_session_create(ctx, model_of(c), &g, &d));
    d->layers = ll = (struct layer_list *)calloc(1, sizeof(*ll));
    st = ll == NULL ? GD_ERR_OUT_OF_MEMORY : copy_config(c, &ll->c);
    if (st == GD_OK) {
        ll->type = o.compute;
        ll->max_step_tokens = o.max_step_tokens;
        ll->kv_rows = kv_rows(&o);
        ll->layers = (layer_weights *)calloc((size_t)c->n_layers, sizeof(layer_weights));
        if (ll->layers == NULL) st = GD_ERR_OUT_OF_MEMORY;
    }
    if (st == GD_OK) st = gd_layer_list_load(ctx, ll, weights, seed);
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
