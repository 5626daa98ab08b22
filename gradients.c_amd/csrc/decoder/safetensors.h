/*
 * Reader of safetensors files: an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape,
 * data_offsets), then the data.  Host only, like checkpoint.c; the directory is checked completely when the file is
 * opened (byte counts, ranges inside the file, repeated names).
 */
#ifndef GD_SAFETENSORS_H
#define GD_SAFETENSORS_H

#include "gradients_infer.h"

typedef struct gd_safetensor {
    const char *name;
    gd_dtype dtype; /* BF16, F16, F32, I32 */
    uint32_t rank;
    int64_t shape[GD_MAX_DIMS];
    uint64_t offset, nbytes; /* offset from the start of the file */
} gd_safetensor;

typedef struct gd_safetensors gd_safetensors;

gd_status gd_safetensors_open(const char *path, gd_safetensors **out);
void gd_safetensors_close(gd_safetensors *file);
uint32_t gd_safetensors_count(const gd_safetensors *file);
const gd_safetensor *gd_safetensors_find(const gd_safetensors *file, const char *name); /* NULL: absent */
gd_status gd_safetensors_read(gd_safetensors *file, const gd_safetensor *t, void *dst); /* all bytes of t */

#endif
