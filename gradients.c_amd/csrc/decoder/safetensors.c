#include "safetensors.h"

#include <stdio.h>
#include <stdlib.h>
#include <string.h>

#include "json.h"

#define HEADER_MAX ((uint64_t)100 << 20)

struct gd_safetensors {
    FILE *f;
    gd_json_doc doc;
    gd_safetensor *entries; /* sorted by name */
    uint32_t count;
};

static int by_name(const void *a, const void *b)
{
    return strcmp(((const gd_safetensor *)a)->name, ((const gd_safetensor *)b)->name);
}

static gd_dtype dtype_of(const char *s)
{
    if (!strcmp(s, "BF16")) return GD_DTYPE_BF16;
    if (!strcmp(s, "F16")) return GD_DTYPE_F16;
    if (!strcmp(s, "F32")) return GD_DTYPE_F32;
    if (!strcmp(s, "I32")) return GD_DTYPE_I32;
    return GD_DTYPE_INVALID;
}

static gd_status read_entry(const gd_json *node, uint64_t data_start, uint64_t file_size, gd_safetensor *t)
{
    const gd_json *dtype = gd_json_get(node, "dtype"), *shape = gd_json_get(node, "shape"), *v;
    const gd_json *offsets = gd_json_get(node, "data_offsets");
    int64_t lo, hi, n = 1;
    t->name = node->key;
    if (dtype == NULL || dtype->type != GD_JSON_STRING || shape == NULL || shape->type != GD_JSON_ARRAY ||
        shape->count > GD_MAX_DIMS || offsets == NULL || offsets->type != GD_JSON_ARRAY || offsets->count != 2U ||
        !gd_json_int(offsets->child, &lo) || !gd_json_int(offsets->child->next, &hi) || lo < 0 || hi < lo)
        return GD_ERR_BAD_STATE;
    t->dtype = dtype_of(dtype->string);
    if (t->dtype == GD_DTYPE_INVALID) return GD_ERR_UNSUPPORTED;
    for (v = shape->child; v != NULL; v = v->next) {
        if (!gd_json_int(v, &t->shape[t->rank]) || t->shape[t->rank] <= 0 || n > INT64_MAX / 8 / t->shape[t->rank])
            return GD_ERR_BAD_STATE;
        n *= t->shape[t->rank++];
    }
    t->nbytes = (uint64_t)n * gd_dtype_size(t->dtype);
    t->offset = data_start + (uint64_t)lo;
    if (t->nbytes != (uint64_t)(hi - lo)) return GD_ERR_BAD_STATE;
    if ((uint64_t)hi > file_size - data_start) return GD_ERR_IO;
    return GD_OK;
}

gd_status gd_safetensors_open(const char *path, gd_safetensors **out)
{
    gd_safetensors *s = (gd_safetensors *)calloc(1, sizeof(*s));
    unsigned char len_bytes[8];
    uint64_t len = 0U, size;
    char *text = NULL;
    const gd_json *v;
    gd_status st = GD_ERR_IO;
    int i;
    *out = NULL;
    if (s == NULL) return GD_ERR_OUT_OF_MEMORY;
    s->f = fopen(path, "rb");
    if (s->f == NULL || fseek(s->f, 0, SEEK_END) != 0) goto fail;
    size = (uint64_t)ftell(s->f);
    rewind(s->f);
    if (fread(len_bytes, 1, 8, s->f) != 8U) goto fail;
    for (i = 7; i >= 0; --i) len = (len << 8) | len_bytes[i];
    if (len > HEADER_MAX || len > size - 8U) goto fail;
    text = (char *)malloc((size_t)len + 1U);
    if (text == NULL) {
        st = GD_ERR_OUT_OF_MEMORY;
        goto fail;
    }
    if (fread(text, 1, (size_t)len, s->f) != (size_t)len) goto fail;
    st = GD_ERR_BAD_STATE;
    if (!gd_json_parse(text, (size_t)len, &s->doc) || s->doc.root->type != GD_JSON_OBJECT) goto fail;
    s->entries = (gd_safetensor *)calloc(s->doc.root->count + 1U, sizeof(gd_safetensor));
    if (s->entries == NULL) {
        st = GD_ERR_OUT_OF_MEMORY;
        goto fail;
    }
    for (v = s->doc.root->child; v != NULL; v = v->next) {
        if (!strcmp(v->key, "__metadata__")) continue;
        st = read_entry(v, 8U + len, size, &s->entries[s->count]);
        if (st != GD_OK) goto fail;
        s->count += 1U;
    }
    qsort(s->entries, s->count, sizeof(gd_safetensor), by_name);
    st = GD_ERR_BAD_STATE;
    for (i = 1; i < (int)s->count; ++i) {
        if (by_name(&s->entries[i - 1], &s->entries[i]) == 0) goto fail;
    }
    free(text);
    *out = s;
    return GD_OK;
fail:
    free(text);
    gd_safetensors_close(s);
    return st;
}

void gd_safetensors_close(gd_safetensors *s)
{
    if (s == NULL) return;
    if (s->f != NULL) fclose(s->f);
    gd_json_free(&s->doc);
    free(s->entries);
    free(s);
}

uint32_t gd_safetensors_count(const gd_safetensors *s) { return s->count; }

const gd_safetensor *gd_safetensors_find(const gd_safetensors *s, const char *name)
{
    gd_safetensor key;
    memset(&key, 0, sizeof(key));
    key.name = name;
    return (const gd_safetensor *)bsearch(&key, s->entries, s->count, sizeof(gd_safetensor), by_name);
}

gd_status gd_safetensors_read(gd_safetensors *s, const gd_safetensor *t, void *dst)
{
    if (fseek(s->f, (long)t->offset, SEEK_SET) != 0 || fread(dst, 1, (size_t)t->nbytes, s->f) != (size_t)t->nbytes)
        return GD_ERR_IO;
    return GD_OK;
}
