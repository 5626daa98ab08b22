/*
 * Decoders whose layers are listed one by one in a configuration: every layer has a mixer (a state-space recurrence,
 * latent attention or attention with grouped heads, each with its own sizes) and possibly a feed-forward (gated, square
 * relu, or experts chosen by token id).  Architectures "Girirax" and "Bonatar": they differ in what a layer may hold and
 * in where its norms stand.
 */
#ifndef GD_LAYER_LIST_H
#define GD_LAYER_LIST_H

#include "decoder_internal.h"
#include "json.h"
#include "safetensors.h"

typedef enum layer_mixer { MIXER_MAMBA2, MIXER_LATENT_ATTENTION, MIXER_GROUPED_ATTENTION } layer_mixer;
typedef enum layer_mlp { MLP_NONE, MLP_GELU_GATED, MLP_SQUARE_RELU, MLP_ROUTED } layer_mlp;

/* YaRN: see gd_yarn_frequency */
typedef struct rot_scaling {
    double factor, original, fast, slow; /* factor 0: none */
} rot_scaling;

typedef struct layer_config {
    layer_mixer mixer;
    /* mamba2 */
    gd_backend_ssm_args ssm;
    int32_t norm_groups, taps;
    /* latent_attention */
    gd_backend_latent_args latent;
    /* grouped attention */
    gd_backend_grouped_args grouped;
    double rot_base; /* both kinds of attention */
    rot_scaling scaling;
    layer_mlp mlp;
    int32_t ff; /* of a feed-forward that is not routed */
    /* MLP_ROUTED: experts chosen by a table, and a shared expert with sizes of its own (shared_ff 0: none) */
    gd_backend_routed_args routed;
    int32_t shared_ff;
    float shared_limit;
    int32_t weights_of; /* the layer whose weights it uses: another one, or itself */
} layer_config;

typedef struct layer_list_config {
    const char *architecture;
    int32_t vocab, width, n_layers;
    float eps, residual_mult, embedding_scale;
    bool norms_first;  /* norms in front of the sublayers (otherwise on their outputs) */
    float norm_offset; /* added to the stored norm weights */
    bool own_head;     /* logits from a matrix of their own (otherwise from the embedding table) */
    layer_config *layers;
} layer_list_config;

/* message receives one line on failure */
gd_status gd_layer_list_parse_girirax(const gd_json *root, layer_list_config *out, char *message, size_t message_size);
gd_status gd_layer_list_parse_bonatar(const gd_json *root, layer_list_config *out, char *message, size_t message_size);
void gd_layer_list_config_free(layer_list_config *c);

gd_status gd_layer_list_memory(const layer_list_config *c, const gd_model_options *o, gd_memory_config *out);
/* weights: the file to load from; NULL: drawn from `seed` */
gd_status gd_layer_list_create(gd_context *ctx, const layer_list_config *c, const gd_model_options *o,
                               gd_safetensors *weights, uint64_t seed, gd_gpt_decoder **out);

#endif
