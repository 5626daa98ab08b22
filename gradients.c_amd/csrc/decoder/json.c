#include "json.h"

#include <math.h>
#include <stdlib.h>
#include <string.h>

#define MAX_DEPTH 64
#define BLOCK_BYTES 65536U

typedef struct block {
    struct block *next;
    size_t used, size;
    _Alignas(16) char data[];
} block;

typedef struct reader {
    const char *p, *end;
    block *blocks;
    int depth;
} reader;

static void *take(reader *r, size_t n)
{
    void *out;
    n = (n + 15U) & ~(size_t)15U;
    if (r->blocks == NULL || r->blocks->size - r->blocks->used < n) {
        const size_t size = n > BLOCK_BYTES ? n : BLOCK_BYTES;
        block *b = (block *)malloc(sizeof(block) + size);
        if (b == NULL) return NULL;
        b->next = r->blocks;
        b->used = 0U;
        b->size = size;
        r->blocks = b;
    }
    out = r->blocks->data + r->blocks->used;
    r->blocks->used += n;
    memset(out, 0, n);
    return out;
}

static void space(reader *r)
{
    while (r->p < r->end && (*r->p == ' ' || *r->p == '\t' || *r->p == '\n' || *r->p == '\r')) ++r->p;
}

static bool word(reader *r, const char *w)
{
    const size_t n = strlen(w);
    if ((size_t)(r->end - r->p) < n || memcmp(r->p, w, n) != 0) return false;
    r->p += n;
    return true;
}

static bool hex4(reader *r, uint32_t *out)
{
    uint32_t v = 0U;
    int i;
    if (r->end - r->p < 4) return false;
    for (i = 0; i < 4; ++i) {
        const char c = *r->p++;
        if (c >= '0' && c <= '9') v = v * 16U + (uint32_t)(c - '0');
        else if (c >= 'a' && c <= 'f') v = v * 16U + (uint32_t)(c - 'a') + 10U;
        else if (c >= 'A' && c <= 'F') v = v * 16U + (uint32_t)(c - 'A') + 10U;
        else return false;
    }
    *out = v;
    return true;
}

/* behind the opening quote */
static char *string(reader *r)
{
    const char *scan = r->p;
    char *out, *w;
    while (scan < r->end && *scan != '"') scan += *scan == '\\' ? 2 : 1;
    if (scan >= r->end) return NULL;
    out = w = (char *)take(r, (size_t)(scan - r->p) + 1U); /* escapes only shrink */
    if (out == NULL) return NULL;
    while (r->p < r->end && *r->p != '"') {
        uint32_t c = (unsigned char)*r->p++;
        if (c < 0x20U) return NULL;
        if (c != '\\') {
            *w++ = (char)c;
            continue;
        }
        if (r->p >= r->end) return NULL;
        switch (*r->p++) {
        case '"': *w++ = '"'; break;
        case '\\': *w++ = '\\'; break;
        case '/': *w++ = '/'; break;
        case 'b': *w++ = '\b'; break;
        case 'f': *w++ = '\f'; break;
        case 'n': *w++ = '\n'; break;
        case 'r': *w++ = '\r'; break;
        case 't': *w++ = '\t'; break;
        case 'u':
            if (!hex4(r, &c)) return NULL;
            if (c >= 0xd800U && c < 0xdc00U) {
                uint32_t lo;
                if (!word(r, "\\u") || !hex4(r, &lo) || lo < 0xdc00U || lo >= 0xe000U) return NULL;
                c = 0x10000U + ((c - 0xd800U) << 10) + (lo - 0xdc00U);
            }
            if (c < 0x80U) {
                *w++ = (char)c;
            } else if (c < 0x800U) {
                *w++ = (char)(0xc0U | (c >> 6));
                *w++ = (char)(0x80U | (c & 0x3fU));
            } else if (c < 0x10000U) {
                *w++ = (char)(0xe0U | (c >> 12));
                *w++ = (char)(0x80U | ((c >> 6) & 0x3fU));
                *w++ = (char)(0x80U | (c & 0x3fU));
            } else {
                *w++ = (char)(0xf0U | (c >> 18));
                *w++ = (char)(0x80U | ((c >> 12) & 0x3fU));
                *w++ = (char)(0x80U | ((c >> 6) & 0x3fU));
                *w++ = (char)(0x80U | (c & 0x3fU));
            }
            break;
        default: return NULL;
        }
    }
    if (r->p >= r->end) return NULL;
    ++r->p;
    *w = '\0';
    return out;
}

static bool number(reader *r, double *out)
{
    char text[64], *stop;
    size_t n = 0U;
    const char *p = r->p;
    while (p < r->end && n + 1U < sizeof(text) &&
           ((*p >= '0' && *p <= '9') || *p == '-' || *p == '+' || *p == '.' || *p == 'e' || *p == 'E'))
        text[n++] = *p++;
    text[n] = '\0';
    if (n == 0U || text[0] == '+' || text[0] == '.') return false;
    *out = strtod(text, &stop);
    if (*stop != '\0') return false;
    r->p = p;
    return true;
}

static gd_json *value(reader *r);

static bool elements(reader *r, gd_json *parent, char close)
{
    gd_json **link = &parent->child;
    space(r);
    if (r->p < r->end && *r->p == close) {
        ++r->p;
        return true;
    }
    for (;;) {
        char *key = NULL;
        gd_json *v;
        space(r);
        if (close == '}') {
            if (r->p >= r->end || *r->p++ != '"' || (key = string(r)) == NULL) return false;
            space(r);
            if (r->p >= r->end || *r->p++ != ':') return false;
        }
        v = value(r);
        if (v == NULL) return false;
        v->key = key;
        *link = v;
        link = &v->next;
        parent->count += 1U;
        space(r);
        if (r->p >= r->end) return false;
        if (*r->p == close) {
            ++r->p;
            return true;
        }
        if (*r->p++ != ',') return false;
    }
}

static gd_json *value(reader *r)
{
    gd_json *v;
    bool ok = false;
    space(r);
    if (r->p >= r->end || r->depth >= MAX_DEPTH) return NULL;
    v = (gd_json *)take(r, sizeof(gd_json));
    if (v == NULL) return NULL;
    r->depth += 1;
    switch (*r->p) {
    case '{':
    case '[':
        v->type = *r->p == '{' ? GD_JSON_OBJECT : GD_JSON_ARRAY;
        ++r->p;
        ok = elements(r, v, v->type == GD_JSON_OBJECT ? '}' : ']');
        break;
    case '"':
        ++r->p;
        v->type = GD_JSON_STRING;
        v->string = string(r);
        ok = v->string != NULL;
        break;
    case 't':
        v->type = GD_JSON_BOOL;
        v->boolean = true;
        ok = word(r, "true");
        break;
    case 'f':
        v->type = GD_JSON_BOOL;
        ok = word(r, "false");
        break;
    case 'n': ok = word(r, "null"); break;
    default:
        v->type = GD_JSON_NUMBER;
        ok = number(r, &v->number);
        break;
    }
    r->depth -= 1;
    return ok ? v : NULL;
}

static void free_blocks(block *b)
{
    while (b != NULL) {
        block *next = b->next;
        free(b);
        b = next;
    }
}

bool gd_json_parse(const char *text, size_t len, gd_json_doc *doc)
{
    reader r = {text, text + len, NULL, 0};
    doc->root = value(&r);
    space(&r);
    if (doc->root == NULL || r.p != r.end) {
        free_blocks(r.blocks);
        doc->root = NULL;
        doc->blocks = NULL;
        return false;
    }
    doc->blocks = r.blocks;
    return true;
}

void gd_json_free(gd_json_doc *doc)
{
    free_blocks((block *)doc->blocks);
    doc->root = NULL;
    doc->blocks = NULL;
}

const gd_json *gd_json_get(const gd_json *object, const char *key)
{
    const gd_json *v;
    if (object == NULL || object->type != GD_JSON_OBJECT) return NULL;
    for (v = object->child; v != NULL; v = v->next) {
        if (strcmp(v->key, key) == 0) return v;
    }
    return NULL;
}

bool gd_json_int(const gd_json *node, int64_t *out)
{
    if (node == NULL || node->type != GD_JSON_NUMBER || node->number != floor(node->number) ||
        fabs(node->number) > 9007199254740992.0)
        return false;
    *out = (int64_t)node->number;
    return true;
}
