/*
 * gd_model.h - opening a stored model without knowing which one it is: a registry of the architectures this
 * library serves.  A path is either
 *   - a ".gdckpt" file of the reference's gpt_lm example (gd_checkpoint.h): "gpt_lm", or
 *   - a folder with config.json and model.safetensors, whose "architecture" names the model: "Girirax" or "Bonatar".
 * The decoder made from it is the one of gd_gpt_decoder.h: prefill, step, resident sessions, sampling and generation
 * are the same calls for every architecture.
 *
 * Configuration of the layer-list decoders: vocab, width, norm.eps, embedding.scale and layers[], every entry with its
 * "type" and "mixer" sizes and its "mlp" (or null).
 * "Girirax": also residual_mult; mlp {"kind": "dense", "ff"}; types
 *   "mamba2"            heads, vdim, state, groups, norm_groups, conv (taps)
 *   "latent_attention"  heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot.base, rot.dims (= rot_dim)
 * "Bonatar": a layer may name in "weights_of" another layer of the same sizes whose weights it uses; type
 *   "attention"         heads, kv_heads, dim, vdim, scale, rot.base, rot.dims, rot.scaling {factor, original, fast, slow}
 *                       (or none), mask.size (positions of a chunk; without mask: all)
 *   mlp {"kind": "dense", "ff"}, or {"kind": "moe", "router": {experts, top}, "expert": {ff, limit},
 *   "shared": {ff, limit} or null}
 */
#ifndef GD_MODEL_H
#define GD_MODEL_H

#include "gd_gpt_decoder.h"

#ifdef __cplusplus
extern "C" {
#endif
#pragma GCC visibility push(default) /* the library is built with hidden visibility: only these are exported */

typedef struct gd_model gd_model;

typedef struct gd_model_options {
    int32_t max_seq;         /* positions per sequence; 0: what the file says (gpt_lm) */
    int32_t batch;           /* sequences held at the same time; 0: 1 */
    int32_t max_step_tokens; /* most tokens of one prefill or extend call; 0: batch * max_seq */
    gd_dtype compute;        /* projections and activations of a layer-list decoder: GD_DTYPE_BF16 (0: this) or
                                GD_DTYPE_F32; gpt_lm always computes in F16 */
    int32_t heads;           /* gpt_lm files that do not say (0: they must) */
} gd_model_options;

/* Reads and checks the description.  GD_ERR_IO: a file is missing or ends early; GD_ERR_UNSUPPORTED: an architecture,
 * layer type or form this library does not have; GD_ERR_BAD_STATE: a malformed or contradictory description.
 * message (may be NULL) receives one line about a failure. */
gd_status gd_model_open(const char *path, gd_model **out, char *message, size_t message_size);
void gd_model_close(gd_model *model);
const char *gd_model_architecture(const gd_model *model);
int32_t gd_model_vocab(const gd_model *model);
int32_t gd_model_layers(const gd_model *model);

/* Arena sizes a context needs for a decoder of this model (gd_context_create). */
gd_status gd_model_memory(const gd_model *model, const gd_model_options *options, gd_memory_config *out);
/* Allocates the decoder in the context's arenas and loads the weights.  The model may be closed afterwards. */
gd_status gd_model_create_decoder(gd_context *ctx, gd_model *model, const gd_model_options *options,
                                  gd_gpt_decoder **out);

/* A layer-list decoder without a weight file, for measurements: config_json is the text of a config.json, the weights
 * are drawn from a generator with the given seed. */
gd_status gd_model_open_config(const char *config_json, uint64_t seed, gd_model **out, char *message,
                               size_t message_size);

#pragma GCC visibility pop
#ifdef __cplusplus
}
#endif

#endif /* GD_MODEL_H */
