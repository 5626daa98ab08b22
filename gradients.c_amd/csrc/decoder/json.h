/*
 * A small JSON reader (RFC 8259) for configuration files, safetensors headers and step lines: the whole text becomes a
 * tree of nodes in one allocation chain, freed at once.  Objects keep their order; a repeated key gives its first value.
 */
#ifndef GD_JSON_H
#define GD_JSON_H

#include <stdbool.h>
#include <stddef.h>
#include <stdint.h>

typedef enum gd_json_type { GD_JSON_NULL, GD_JSON_BOOL, GD_JSON_NUMBER, GD_JSON_STRING, GD_JSON_ARRAY, GD_JSON_OBJECT } gd_json_type;

typedef struct gd_json gd_json;
struct gd_json {
    gd_json_type type;
    bool boolean;
    double number;
    char *string;      /* STRING: NUL-terminated UTF-8 */
    char *key;         /* inside an object */
    gd_json *child;    /* ARRAY, OBJECT: first element */
    gd_json *next;     /* next element of the same parent */
    size_t count;      /* ARRAY, OBJECT */
};

typedef struct gd_json_doc {
    gd_json *root;
    void *blocks;
} gd_json_doc;

/* false: malformed (or out of memory); nothing to free then */
bool gd_json_parse(const char *text, size_t len, gd_json_doc *doc);
void gd_json_free(gd_json_doc *doc);
const gd_json *gd_json_get(const gd_json *object, const char *key); /* NULL: absent or not an object */
bool gd_json_int(const gd_json *node, int64_t *out);                /* a whole number */

#endif
