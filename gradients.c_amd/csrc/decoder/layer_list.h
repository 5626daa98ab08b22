/*
 * Decoders whose layers are listed one by one in a configuration: every layer has a mixer (a state-space recurrence or
 * latent attention, each with its own sizes) and possibly a feed-forward.  Architecture "Girirax".
 */
#ifndef GD_LAYER_LIST_H
#define GD_LAYER_LIST_H

#include "decoder_internal.h"
#include "json.h"
#include "safetensors.h"

typedef enum layer_mixer { MIXER_MAMBA2, MIXER_LATENT_ATTENTION } layer_mixer;

typedef struct layer_config {
    layer_mixer mixer;
    /* mamba2 */
    gd_backend_ssm_args ssm;
    int32_t norm_groups, taps;
    /* latent_attention */
    gd_backend_latent_args latent;
    double rot_base;
    int32_t ff; /* 0: no feed-forward */
} layer_config;

typedef struct layer_list_config {
    int32_t vocab, width, n_layers;
    float eps, residual_mult, embedding_scale;
    layer_config *layers;
} layer_list_config;

/* message receives one line on failure */
gd_status gd_layer_list_parse(const gd_json *root, layer_list_config *out, char *message, size_t message_size);
void gd_layer_list_config_free(layer_list_config *c);

gd_status gd_layer_list_memory(const layer_list_config *c, const gd_model_options *o, gd_memory_config *out);
/* weights: the file to load from; NULL: drawn from `seed` */
gd_status gd_layer_list_create(gd_context *ctx, const layer_list_config *c, const gd_model_options *o,
                               gd_safetensors *weights, uint64_t seed, gd_gpt_decoder **out);

#endif
