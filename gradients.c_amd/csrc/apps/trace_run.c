/*
 * Replays token ids through a model, step by step, and writes the logits that are asked for; it samples nothing.
 * Steps are lines of JSON on standard input:
 *   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
 * entries: the next tokens of each request and the places among them whose logits are wanted; end: requests whose
 * slots are given back after the step.  For a step with wanted places DIR/<step>.f32 receives the logits, in the order
 * of the entries, as 32-bit floats; after every step a line "done <step>" is printed.
 *
 * The model, its caches and states, and every kernel are the library's own (gd_model.h, gd_gpt_decoder_extend).
 */
#include <errno.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>
#include <unistd.h>

#include "gd_model.h"
#include "json.h"

#define SLOTS 4

typedef struct request {
    char *id; /* NULL: the slot is free */
    int32_t slot;
} request;

static int complain(const char *what, const char *why)
{
    fprintf(stderr, "trace_run: %s: %s\n", what, why);
    return 1;
}

static int usage(void)
{
    fprintf(stderr, "usage: trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N\n"
                    "replays steps from standard input; see the head of apps/trace_run.c for their form\n");
    return 2;
}

static request *find(request *live, const char *id)
{
    int i;
    for (i = 0; i < SLOTS; ++i) {
        if (live[i].id != NULL && !strcmp(live[i].id, id)) return &live[i];
    }
    return NULL;
}

static gd_status admit(gd_gpt_decoder *dec, request *live, const char *id, request **out)
{
    int i;
    for (i = 0; i < SLOTS; ++i) {
        gd_status st;
        if (live[i].id != NULL) continue;
        st = gd_gpt_decoder_acquire(dec, &live[i].slot);
        if (st != GD_OK) return st;
        live[i].id = strdup(id);
        *out = &live[i];
        return live[i].id != NULL ? GD_OK : GD_ERR_OUT_OF_MEMORY;
    }
    return GD_ERR_BUSY;
}

static int write_logits(const char *dir, long long step, const float *values, size_t n)
{
    const size_t len = strlen(dir) + 40U;
    char *path = (char *)malloc(len);
    FILE *f;
    int ok;
    if (path == NULL) return complain("writing logits", "out of memory");
    (void)snprintf(path, len, "%s/%lld.f32", dir, step);
    f = fopen(path, "wb");
    ok = f != NULL && fwrite(values, sizeof(float), n, f) == n;
    if (f != NULL && fclose(f) != 0) ok = 0;
    if (!ok) (void)complain(path, strerror(errno));
    free(path);
    return ok ? 0 : 1;
}

static int run_step(gd_gpt_decoder *dec, request *live, const char *dir, int32_t vocab, const gd_json *line)
{
    const gd_json *entries = gd_json_get(line, "entries"), *end = gd_json_get(line, "end"), *e, *v;
    int64_t step, value;
    int32_t slots[SLOTS], cu[SLOTS + 1], n_seqs = 0, n_ids = 0, n_want = 0;
    int32_t *ids = NULL, *want = NULL;
    float *logits = NULL;
    size_t all_ids = 0U, all_want = 0U;
    gd_status st = GD_OK;
    int rc = 1;
    if (!gd_json_int(gd_json_get(line, "step"), &step) || entries == NULL || entries->type != GD_JSON_ARRAY)
        return complain("step", "malformed line");
    for (e = entries->child; e != NULL; e = e->next) {
        const gd_json *t = gd_json_get(e, "tokens"), *w = gd_json_get(e, "want");
        if (gd_json_get(e, "id") == NULL || gd_json_get(e, "id")->type != GD_JSON_STRING || t == NULL ||
            t->type != GD_JSON_ARRAY || (w != NULL && w->type != GD_JSON_ARRAY))
            return complain("step", "malformed entry");
        all_ids += t->count;
        all_want += w != NULL ? w->count : 0U;
    }
    ids = (int32_t *)malloc((all_ids + 1U) * sizeof(int32_t));
    want = (int32_t *)malloc((all_want + 1U) * sizeof(int32_t));
    logits = (float *)malloc((all_want * (size_t)vocab + 1U) * sizeof(float));
    if (ids == NULL || want == NULL || logits == NULL) {
        (void)complain("step", "out of memory");
        goto out;
    }
    cu[0] = 0;
    for (e = entries->child; e != NULL; e = e->next) {
        const gd_json *t = gd_json_get(e, "tokens"), *w = gd_json_get(e, "want");
        const char *id = gd_json_get(e, "id")->string;
        request *r = find(live, id);
        if (t->count == 0U) continue;
        if (n_seqs == SLOTS) st = GD_ERR_BUSY;
        if (st == GD_OK && r == NULL) st = admit(dec, live, id, &r);
        if (st != GD_OK) {
            (void)complain("taking a slot", gd_status_string(st));
            goto out;
        }
        for (v = w != NULL ? w->child : NULL; v != NULL; v = v->next) {
            if (!gd_json_int(v, &value) || value < 0 || value >= (int64_t)t->count) {
                (void)complain("step", "a wanted place outside the entry");
                goto out;
            }
            want[n_want++] = n_ids + (int32_t)value;
        }
        for (v = t->child; v != NULL; v = v->next) {
            if (!gd_json_int(v, &value) || value < 0 || value >= vocab) {
                (void)complain("step", "a token outside the vocabulary");
                goto out;
            }
            ids[n_ids++] = (int32_t)value;
        }
        slots[n_seqs++] = r->slot;
        cu[n_seqs] = n_ids;
    }
    if (n_seqs > 0) st = gd_gpt_decoder_extend(dec, slots, n_seqs, ids, cu, want, n_want, logits);
    if (st != GD_OK) {
        (void)complain("gd_gpt_decoder_extend", gd_status_string(st));
        goto out;
    }
    if (n_want > 0 && write_logits(dir, (long long)step, logits, (size_t)n_want * (size_t)vocab) != 0) goto out;
    for (v = end != NULL ? end->child : NULL; v != NULL; v = v->next) {
        request *r = v->type == GD_JSON_STRING ? find(live, v->string) : NULL;
        if (r == NULL) continue;
        (void)gd_gpt_decoder_release(dec, r->slot);
        free(r->id);
        r->id = NULL;
    }
    printf("done %lld\n", (long long)step);
    fflush(stdout);
    rc = 0;
out:
    free(ids);
    free(want);
    free(logits);
    return rc;
}

int main(int argc, char **argv)
{
    const char *model_dir = NULL, *dtype = NULL, *out_dir = NULL;
    long max_tokens = 0;
    char message[256], *text = NULL;
    size_t text_size = 0U;
    ssize_t got;
    request live[SLOTS];
    gd_model_options options;
    gd_memory_config mem;
    gd_model *model = NULL;
    gd_context *ctx = NULL;
    gd_gpt_decoder *dec = NULL;
    int32_t vocab;
    gd_status st;
    int i, rc = 0;
    for (i = 1; i < argc; ++i) {
        const char *v = i + 1 < argc ? argv[i + 1] : NULL;
        if (v == NULL) return usage();
        if (!strcmp(argv[i], "--model")) model_dir = v;
        else if (!strcmp(argv[i], "--dtype")) dtype = v;
        else if (!strcmp(argv[i], "--out")) out_dir = v;
        else if (!strcmp(argv[i], "--max-tokens")) max_tokens = strtol(v, NULL, 10);
        else return usage();
        ++i;
    }
    if (model_dir == NULL || dtype == NULL || out_dir == NULL || max_tokens <= 0 || max_tokens > (1L << 30)) return usage();
    memset(live, 0, sizeof(live));
    memset(&options, 0, sizeof(options));
    options.max_seq = (int32_t)max_tokens;
    options.max_step_tokens = (int32_t)max_tokens;
    options.batch = SLOTS;
    if (!strcmp(dtype, "bfloat16")) options.compute = GD_DTYPE_BF16;
    else if (!strcmp(dtype, "float32")) options.compute = GD_DTYPE_F32;
    else return usage();
    st = gd_model_open(model_dir, &model, message, sizeof(message));
    if (st != GD_OK) return complain(model_dir, message[0] != '\0' ? message : gd_status_string(st));
    vocab = gd_model_vocab(model);
    st = gd_model_memory(model, &options, &mem);
    if (st == GD_OK) st = gd_context_create(&mem, &ctx);
    if (st != GD_OK) return complain("gd_context_create", gd_status_string(st));
    st = gd_model_create_decoder(ctx, model, &options, &dec);
    gd_model_close(model);
    if (st != GD_OK) return complain("gd_model_create_decoder", gd_status_string(st));
    while (rc == 0 && (got = getline(&text, &text_size, stdin)) > 0) {
        gd_json_doc doc;
        if (strspn(text, " \t\r\n") == (size_t)got) continue;
        if (!gd_json_parse(text, (size_t)got, &doc)) {
            rc = complain("step", "not JSON");
            break;
        }
        rc = run_step(dec, live, out_dir, vocab, doc.root);
        gd_json_free(&doc);
    }
    free(text);
    gd_gpt_decoder_destroy(dec);
    gd_context_destroy(ctx);
    fflush(stdout);
    fflush(stderr);
    _exit(rc); /* what the HIP runtime does in its exit handlers is skipped */
}
