/* What the parts of the layer-list decoder share: layer_list.c (caches, states and the forward pass) and
 * layer_list_weights.c (which weights a configuration has, and where they come from). */
#ifndef GD_LAYER_LIST_INTERNAL_H
#define GD_LAYER_LIST_INTERNAL_H

#include "layer_list.h"

typedef struct layer_weights {
    gd_tensor norm1, norm2;
    gd_tensor in, conv, conv_b, dt_bias, a_log, d_skip, gnorm; /* in: every projection of the mixer's input, stacked:
                                                                  mamba2's own, latent [dq | dkv | g], grouped [q | k | v | g] */
    gd_tensor dq_norm, dkv_norm, uq, ukv, ukt, freq; /* attention; ukv: [uk | uv]; ukt: uk turned per head */
    gd_tensor out;
    gd_tensor upgate, upgate_b, down, down_b;    /* feed-forward; upgate: [up | gate]; a routed one: its shared expert */
    gd_tensor expert_upgate, expert_down, table; /* experts one behind the other; I32 [vocab, top] */
    gd_tensor place, first, tiles;               /* the step's routes (gd_backend_route_by_tables) */
    /* per slot, every layer's own */
    gd_tensor ring, states, cache, k_cache, v_cache;
} layer_weights;

struct layer_list {
    layer_list_config c;
    gd_dtype type; /* of projections and activations */
    int32_t max_step_tokens;
    int32_t kv_rows; /* tokens whose keys and values a step may expand at once (latent attention) */
    gd_tensor embed, head, final_norm;
    layer_weights *layers;
    gd_tensor rows_dev, cu_dev; /* 0 .. batch-1 and 0 .. batch: the tables of a decode step over every slot */
};

static inline int64_t conv_channels(const layer_config *l)
{
    return (int64_t)l->ssm.heads * l->ssm.vdim + 2 * (int64_t)l->ssm.groups * l->ssm.state;
}
static inline int64_t inner_size(const layer_config *l) { return (int64_t)l->ssm.heads * l->ssm.vdim; }
/* columns of the stacked input projection */
static inline int64_t mixer_in(const layer_config *l)
{
    if (l->mixer == MIXER_MAMBA2) return inner_size(l) + conv_channels(l) + l->ssm.heads;
    if (l->mixer == MIXER_GROUPED_ATTENTION)
        return (int64_t)l->grouped.heads * (l->grouped.dim + 1) + (int64_t)l->grouped.kv_heads * (l->grouped.dim + l->grouped.vdim);
    return (int64_t)l->latent.q_rank + l->latent.kv_rank + l->latent.rot_dim + (int64_t)l->latent.heads * l->latent.vdim;
}
/* distance of its rows: 16-byte pieces for the attention that reads them where they lie */
static inline int64_t mixer_pitch(const layer_config *l)
{
    return l->mixer == MIXER_GROUPED_ATTENTION ? (mixer_in(l) + 7) / 8 * 8 : mixer_in(l);
}
static inline int64_t mixer_out(const layer_config *l)
{
    if (l->mixer == MIXER_MAMBA2) return inner_size(l);
    if (l->mixer == MIXER_GROUPED_ATTENTION) return (int64_t)l->grouped.heads * l->grouped.vdim;
    return (int64_t)l->latent.heads * l->latent.vdim;
}
static inline int64_t query_size(const layer_config *l)
{
    return (int64_t)l->latent.heads * (l->latent.dim + l->latent.rot_dim);
}

size_t gd_layer_list_weight_bytes(const layer_list_config *c, gd_dtype type);
/* allocates every weight in the parameter arena and fills it */
gd_status gd_layer_list_load(gd_context *ctx, struct layer_list *ll, gd_safetensors *file, uint64_t seed);

#endif
