/*
 * wr_mix_model.c — reads a mixer-stack model: config.json decides every size and
 * constant, model.safetensors holds bfloat16 weights.  Weights are rearranged
 * here into the operands the device steps take: feature counts padded to
 * multiples of 32 with zeros, products of the same input stacked, the per-head
 * key matrices transposed (they are applied to queries), gate and up outputs
 * interleaved by tiles of 16.
 */
#define _GNU_SOURCE
#include "wr_mix.h"
#include "wr_json.h"
#include "wr_safetensors.h"

#include <math.h>
#include <stdarg.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>

static uint32_t p32(uint32_t n) { return (n + 31) / 32 * 32; }
static uint32_t p16(uint32_t n) { return (n + 15) / 16 * 16; }

/* What tells the designs of this family apart. */
typedef enum { DESIGN_BIPOTAR = 1, DESIGN_TAREDRA = 2, DESIGN_FEDIRAX = 4, DESIGN_MAROSUN = 8 } design_bit;
typedef struct wrh_mix_design {
    const char *arch;
    design_bit  bit;
    uint8_t post_norms;                   /* a sublayer's output is normed before it joins the residual */
    uint8_t norms_around_zero;            /* stored w means 1 + w */
    uint8_t embed_norm;                   /* the embedding is normed; else multiplied by embedding.scale, */
    uint8_t embed_plain;                  /* or taken as it is */
    uint8_t joint;                        /* one norm per layer: mixers and feed-forward read the same rows */
    uint8_t tied_head;                    /* the head is the embedding table */
    uint8_t gelu;                         /* dense feed-forwards gate with the tanh form of GELU, else SiLU */
} wrh_mix_design;

static const wrh_mix_design designs[] = {
    {.arch = "Bipotar", .bit = DESIGN_BIPOTAR, .post_norms = 1, .embed_norm = 1},
    {.arch = "Taredra", .bit = DESIGN_TAREDRA, .norms_around_zero = 1, .tied_head = 1, .gelu = 1},
    {.arch = "Fedirax", .bit = DESIGN_FEDIRAX, .norms_around_zero = 1},
    {.arch = "Marosun", .bit = DESIGN_MAROSUN, .norms_around_zero = 1, .embed_plain = 1, .joint = 1},
};

/* One of the matrices that a product of a layer's input is stacked from: where its outputs lie, and its bias if any. */
typedef struct in_part {
    const char *name;
    uint32_t    rows, *col;
    const char *bias;
} in_part;

#define PARTS_MAX 12

/* Everything the reading functions share; `st` keeps the first failure. */
typedef struct loader {
    wr_engine            *e;
    const wrh_mix_design *design;
    struct wrh_mix_model *mm;
    wrh_safetensors       f;
    float                *vec;            /* host copy of the vector block being gathered */
    size_t                vec_n, vec_cap;
    in_part               parts[PARTS_MAX];   /* of the joint layer being read */
    size_t                n_parts;
    wr_status             st;
} loader;

static void fail(loader *l, wr_status st, const char *fmt, ...)
{
    if (l->st != WR_OK) return;
    char buf[256];
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(buf, sizeof buf, fmt, ap);
    va_end(ap);
    l->st = st;
    wrh_logf(l->e, 0, "loader: %s", buf);
}

/* ---------------------------------------------------------------- config -- */

static uint32_t need_u32(loader *l, const wrh_json *o, const char *key, uint32_t lo, uint32_t hi)
{
    uint32_t v = 0;
    if (!wrh_json_u32(o, key, &v)) fail(l, WR_ERR_FORMAT, "config: '%s' missing or not a whole number", key);
    else if (v < lo || v > hi) fail(l, WR_ERR_LIMIT, "config: '%s' = %u outside [%u, %u]", key, v, lo, hi);
    return v;
}

static double need_num(loader *l, const wrh_json *o, const char *key)
{
    double v = 0;
    if (!wrh_json_num(o, key, &v)) fail(l, WR_ERR_FORMAT, "config: '%s' missing or not a number", key);
    return v;
}

static const wrh_json *need_obj(loader *l, const wrh_json *o, const char *key)
{
    const wrh_json *v = wrh_json_get(o, key);
    if (!v || v->type != WRH_JSON_OBJECT) {
        fail(l, WR_ERR_FORMAT, "config: '%s' missing or not an object", key);
        return NULL;
    }
    return v;
}

/* A key that may be absent or null. */
static const wrh_json *given(const wrh_json *o, const char *key)
{
    const wrh_json *v = wrh_json_get(o, key);
    return v && v->type != WRH_JSON_NULL ? v : NULL;
}

static const char *need_str(loader *l, const wrh_json *o, const char *key)
{
    const wrh_json *v = wrh_json_get(o, key);
    if (!v || v->type != WRH_JSON_STRING) {
        fail(l, WR_ERR_FORMAT, "config: '%s' missing or not a string", key);
        return "";
    }
    return v->text;
}

#define DIM_MAX   (1u << 20)
#define HEADS_MAX 4096u

/* ---------------------------------------------------------------- tensors -- */

static const uint16_t *tensor(loader *l, const char *name, uint32_t rows, uint32_t cols)
{
    if (l->st != WR_OK) return NULL;
    const wrh_tensor *t = wrh_safetensors_find(&l->f, name);
    if (!t) {
        fail(l, WR_ERR_FORMAT, "required tensor %s is missing", name);
        return NULL;
    }
    if (t->dtype != WRH_ST_BF16) {
        fail(l, WR_ERR_UNSUPPORTED, "tensor %s is not bfloat16", name);
        return NULL;
    }
    const int ok = cols ? (t->n_dims == 2 && t->shape[0] == rows && t->shape[1] == cols)
                        : (t->n_dims == 1 && t->shape[0] == rows);
    if (!ok) {
        fail(l, WR_ERR_FORMAT, "tensor %s does not have the shape the configuration gives it (%u x %u)", name, rows, cols);
        return NULL;
    }
    if (((uintptr_t)t->data & 1) != 0) {
        fail(l, WR_ERR_FORMAT, "tensor %s is not aligned in the file", name);
        return NULL;
    }
    return (const uint16_t *)t->data;
}

/* Rows of a matrix whose height only its shape tells; 0 after a failure. */
static uint32_t tensor_rows(loader *l, uint32_t i, const char *name, uint32_t hi)
{
    char nb[128];
    snprintf(nb, sizeof nb, "l%u.%s", i, name);
    if (l->st != WR_OK) return 0;
    const wrh_tensor *t = wrh_safetensors_find(&l->f, nb);
    if (!t || t->n_dims != 2) {
        fail(l, WR_ERR_FORMAT, "required matrix %s is missing", nb);
        return 0;
    }
    if (t->shape[0] < 1 || t->shape[0] > hi) {
        fail(l, WR_ERR_LIMIT, "tensor %s has too many rows", nb);
        return 0;
    }
    return (uint32_t)t->shape[0];
}

/* layer tensor "l<i>.<name>" */
static const uint16_t *ltensor(loader *l, uint32_t i, const char *name, uint32_t rows, uint32_t cols)
{
    char nb[128];
    snprintf(nb, sizeof nb, "l%u.%s", i, name);
    return tensor(l, nb, rows, cols);
}

/* Reserves n floats (padded to 32, zeros) in the vector block; the returned
 * index becomes a device pointer once the block is uploaded. */
static float *vec_take(loader *l, uint32_t n, size_t *at)
{
    const size_t np = p32(n);
    if (l->vec_n + np > l->vec_cap) {
        const size_t cap = (l->vec_n + np) * 2;
        float *v = realloc(l->vec, cap * sizeof *v);
        if (!v) {
            fail(l, WR_ERR_NOMEM, "out of memory");
            return NULL;
        }
        l->vec = v;
        l->vec_cap = cap;
    }
    *at = l->vec_n;
    memset(l->vec + l->vec_n, 0, np * sizeof(float));
    l->vec_n += np;
    return l->vec + *at;
}

static float widen(uint16_t b)
{
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}

/* Until the block is on the device a vector "pointer" is its index + 1. */
static const float *vec_put(loader *l, const uint16_t *src, uint32_t n)
{
    size_t at = 0;
    float *v = src ? vec_take(l, n, &at) : NULL;
    if (!v) return NULL;
    for (uint32_t i = 0; i < n; i++) v[i] = widen(src[i]);
    return (const float *)(uintptr_t)(at + 1);
}

/* a norm's weights, as factors */
static const float *norm_put(loader *l, const uint16_t *src, uint32_t n)
{
    const float *at = vec_put(l, src, n);
    if (at && l->design->norms_around_zero)
        for (uint32_t i = 0; i < n; i++) l->vec[(uintptr_t)at - 1 + i] += 1.0f;
    return at;
}

static void vec_fix(const struct wrh_mix_model *mm, const float **p)
{
    if (*p) *p = mm->vecs + ((uintptr_t)*p - 1);
}

/* A host operand being put together: `batch` matrices [rows][cols], zeros. */
typedef struct operand {
    uint16_t *w;
    uint32_t  batch, rows, cols;
} operand;

static operand operand_new(loader *l, uint32_t batch, uint32_t rows, uint32_t cols)
{
    operand o = {NULL, batch, rows, cols};
    if (l->st == WR_OK) {
        o.w = calloc((size_t)batch * rows * cols, 2);
        if (!o.w) fail(l, WR_ERR_NOMEM, "out of memory");
    }
    return o;
}

static uint16_t *operand_row(const operand *o, uint32_t z, uint32_t row)
{
    return o->w + ((size_t)z * o->rows + row) * o->cols;
}

/* rows of src [n][cols] to rows at, at + 1, ... of matrix z */
static void operand_put(loader *l, operand *o, uint32_t z, uint32_t at, const uint16_t *src, uint32_t n, uint32_t cols)
{
    if (l->st != WR_OK || !src) return;
    for (uint32_t i = 0; i < n; i++)
        memcpy(operand_row(o, z, at + i), src + (size_t)i * cols, (size_t)cols * 2);
}

static wr_hip_mat *operand_up(loader *l, operand *o)
{
    wr_hip_mat *w = NULL;
    if (l->st == WR_OK) {
        const int rc = wr_hip_mix_mat_create(o->batch, o->rows, o->cols, o->w, &w);
        if (rc != WR_HIP_OK) fail(l, rc == WR_HIP_ERR_NOMEM ? WR_ERR_NOMEM : (wr_status)rc, "weight upload failed (rc=%d)", rc);
    }
    free(o->w);
    o->w = NULL;
    return w;
}

/* one matrix as it stands, both sides padded */
static wr_hip_mat *plain(loader *l, const uint16_t *src, uint32_t rows, uint32_t cols, uint32_t rows_p)
{
    operand o = operand_new(l, 1, rows_p, p32(cols));
    operand_put(l, &o, 0, 0, src, rows, cols);
    return operand_up(l, &o);
}

/* ----------------------------------------------------------------- layers -- */

static void read_lightning(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const uint32_t W = l->mm->width, Wp = l->mm->width_p;
    L->kind = WRH_MIXER_LIGHTNING;
    L->heads = need_u32(l, c, "heads", 1, HEADS_MAX);
    L->dim = need_u32(l, c, "dim", 1, WR_HIP_MIX_MAX_STATE_DIM);
    L->vdim = need_u32(l, c, "vdim", 1, DIM_MAX);
    const wrh_json *d = wrh_json_get(c, "decay");
    if (l->st == WR_OK && (!d || d->type != WRH_JSON_ARRAY || d->count != L->heads))
        fail(l, WR_ERR_FORMAT, "config: layer %u: 'decay' does not have one number per head", i);
    if (l->st != WR_OK) return;
    if ((uint64_t)L->heads * L->dim > DIM_MAX || (uint64_t)L->heads * L->vdim > DIM_MAX) {
        fail(l, WR_ERR_LIMIT, "config: layer %u is too wide", i);
        return;
    }
    size_t at = 0;
    float *dv = vec_take(l, L->heads, &at);
    if (!dv) return;
    for (const wrh_json *x = d->first; x; x = x->next) {
        if (x->type != WRH_JSON_NUMBER) {
            fail(l, WR_ERR_FORMAT, "config: layer %u: 'decay' holds something that is not a number", i);
            return;
        }
        *dv++ = (float)x->num;
    }
    L->decay = (const float *)(uintptr_t)(at + 1);
    const uint32_t hq = L->heads * L->dim, hv = L->heads * L->vdim;
    L->qk_p = p32(hq);
    L->v_p = p32(hv);
    operand o = operand_new(l, 1, 2 * L->qk_p + 2 * L->v_p, Wp);
    operand_put(l, &o, 0, 0, ltensor(l, i, "mix.q", hq, W), hq, W);
    operand_put(l, &o, 0, L->qk_p, ltensor(l, i, "mix.k", hq, W), hq, W);
    operand_put(l, &o, 0, 2 * L->qk_p, ltensor(l, i, "mix.v", hv, W), hv, W);
    operand_put(l, &o, 0, 2 * L->qk_p + L->v_p, ltensor(l, i, "mix.g", hv, W), hv, W);
    L->w_qkvg = operand_up(l, &o);
    L->w_o = plain(l, ltensor(l, i, "mix.o", W, hv), W, hv, Wp);
    L->mix_norm = vec_put(l, ltensor(l, i, "mix.norm", hv, 0), hv);
}

/* The model's table of this rotation.  `scaling`: what slows its far pairs down (factor, original, fast, slow), or NULL. */
static uint32_t rope_index(loader *l, double base, uint32_t dims, const wrh_json *scaling)
{
    struct wrh_mix_model *mm = l->mm;
    uint32_t k = 0;
    wrh_mix_rope q = {.base = base, .dims = dims, .gain = 1.0f};
    if (scaling) {
        q.factor = need_num(l, scaling, "factor");
        q.original = need_num(l, scaling, "original");
        q.fast = need_num(l, scaling, "fast");
        q.slow = need_num(l, scaling, "slow");
        if (l->st == WR_OK && (q.factor <= 0 || q.original <= 0 || q.fast <= 0 || q.slow <= 0 || base == 1.0))
            fail(l, WR_ERR_FORMAT, "config: rotation of base %g scaled by %g over %g, between %g and %g turns", base, q.factor,
                 q.original, q.fast, q.slow);
        if (l->st != WR_OK) return 0;
        q.gain = (float)(0.1 * log(q.factor) + 1.0);
    }
    for (; k < mm->n_ropes; k++) {
        const wrh_mix_rope *o = &mm->ropes[k];
        if (o->base == base && o->dims == dims && o->factor == q.factor && o->original == q.original && o->fast == q.fast &&
            o->slow == q.slow)
            break;
    }
    if (k == WRH_MAX_LAYERS) {
        fail(l, WR_ERR_LIMIT, "config: more than %u different rotations", WRH_MAX_LAYERS);
        return 0;
    }
    if (k == mm->n_ropes) mm->ropes[mm->n_ropes++] = q;
    return k;
}

/* Frequency of pair i of a rotation: a pair that turns more than `fast` times over the original length keeps its own, one
 * that turns less than `slow` times has it divided by the factor, with a ramp over the pairs between. */
static double rope_freq(const wrh_mix_rope *q, uint32_t i)
{
    const double f = pow(q->base, -2.0 * i / q->dims), two_pi = 6.283185307179586477;
    if (q->factor == 0) return f;
    const double fast = q->dims * log(q->original / (two_pi * q->fast)) / (2.0 * log(q->base));
    const double slow = q->dims * log(q->original / (two_pi * q->slow)) / (2.0 * log(q->base));
    const double lo = fmax(floor(fast), 0.0), hi = fmin(ceil(slow), q->dims - 1.0);
    const double ramp = fmin(fmax((i - lo) / fmax(hi - lo, 0.001), 0.0), 1.0);
    return f / q->factor * ramp + f * (1.0 - ramp);
}

/* The output matrix over heads whose inputs are padded one by one: [Wp][H * vp], zeros between.  `at`: its first
 * input inside a wider matrix. */
static void put_heads_out(loader *l, operand *o, const uint16_t *wo, uint32_t at, uint32_t H, uint32_t v, uint32_t vp)
{
    if (l->st != WR_OK || !wo) return;
    for (uint32_t r = 0; r < l->mm->width; r++)
        for (uint32_t h = 0; h < H; h++)
            memcpy(operand_row(o, 0, r) + at + (size_t)h * vp, wo + ((size_t)r * H + h) * v, (size_t)v * 2);
}

static void read_latent(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    struct wrh_mix_model *mm = l->mm;
    const uint32_t W = mm->width, Wp = mm->width_p;
    L->kind = WRH_MIXER_LATENT;
    const uint32_t H = L->heads = need_u32(l, c, "heads", 1, HEADS_MAX);
    L->dim = need_u32(l, c, "dim", 1, DIM_MAX);
    L->vdim = need_u32(l, c, "vdim", 1, DIM_MAX);
    L->q_rank = need_u32(l, c, "q_rank", 1, DIM_MAX);
    L->kv_rank = need_u32(l, c, "kv_rank", 1, 4096);
    L->rot_dim = need_u32(l, c, "rot_dim", 0, 4096);
    const double scale = need_num(l, c, "scale");
    const wrh_json *rot = need_obj(l, c, "rot"), *mask = need_obj(l, c, "mask");
    if (l->st != WR_OK) return;
    const double base = need_num(l, rot, "base");
    const uint32_t dims = need_u32(l, rot, "dims", 0, L->rot_dim);
    const uint32_t window = need_u32(l, mask, "size", 1, 0xFFFFFFFFu);
    if (l->st == WR_OK && (dims % 2 || base <= 0)) fail(l, WR_ERR_FORMAT, "config: layer %u: rotation of %u dimensions, base %g", i, dims, base);
    if (l->st != WR_OK) return;
    if ((uint64_t)H * (p32(L->dim) + p32(L->rot_dim)) > DIM_MAX || (uint64_t)H * p32(L->vdim) > DIM_MAX) {
        fail(l, WR_ERR_LIMIT, "config: layer %u is too wide", i);
        return;
    }
    L->q_rank_p = p32(L->q_rank);
    L->dim_p = p32(L->dim);
    L->vdim_p = p32(L->vdim);
    wr_hip_mix_latent *g = &L->geo;
    g->heads = H;
    g->rank = L->kv_rank;
    g->rank_pad = wr_hip_mix_latent_rank_pad(L->kv_rank);
    g->rot = L->rot_dim;
    g->rot_pad = p32(L->rot_dim);
    g->rot_half = dims / 2;
    g->window = window;
    g->scale = (float)scale;
    L->rope = rope_index(l, base, dims, NULL);
    if (l->st != WR_OK) return;

    const uint32_t kp = p32(L->kv_rank), rp = p32(L->rot_dim);
    operand o = operand_new(l, 1, L->q_rank_p + kp + rp, Wp);
    operand_put(l, &o, 0, 0, ltensor(l, i, "mix.dq", L->q_rank, W), L->q_rank, W);
    const uint16_t *dkv = ltensor(l, i, "mix.dkv", L->kv_rank + L->rot_dim, W);
    operand_put(l, &o, 0, L->q_rank_p, dkv, L->kv_rank, W);
    operand_put(l, &o, 0, L->q_rank_p + kp, dkv ? dkv + (size_t)L->kv_rank * W : NULL, L->rot_dim, W);
    L->w_d = operand_up(l, &o);
    L->dq_norm = vec_put(l, ltensor(l, i, "mix.dq.norm", L->q_rank, 0), L->q_rank);
    L->dkv_norm = vec_put(l, ltensor(l, i, "mix.dkv.norm", L->kv_rank, 0), L->kv_rank);

    /* queries: every head's unrotated part first (padded), then the rotated parts */
    const uint32_t hq = L->dim + L->rot_dim;
    const uint16_t *uq = ltensor(l, i, "mix.uq", H * hq, L->q_rank);
    o = operand_new(l, 1, H * L->dim_p + p32(H * L->rot_dim), L->q_rank_p);
    for (uint32_t h = 0; h < H && uq; h++) {
        const uint16_t *src = uq + (size_t)h * hq * L->q_rank;
        operand_put(l, &o, 0, h * L->dim_p, src, L->dim, L->q_rank);
        operand_put(l, &o, 0, H * L->dim_p + h * L->rot_dim, src + (size_t)L->dim * L->q_rank, L->rot_dim, L->q_rank);
    }
    L->w_uq = operand_up(l, &o);

    /* the key matrix of a head maps its query into the latent: transposed */
    const uint16_t *uk = ltensor(l, i, "mix.uk", H * L->dim, L->kv_rank);
    o = operand_new(l, H, g->rank_pad, L->dim_p);
    if (l->st == WR_OK)
        for (uint32_t h = 0; h < H; h++)
            for (uint32_t d = 0; d < L->dim; d++)
                for (uint32_t k = 0; k < L->kv_rank; k++)
                    operand_row(&o, h, k)[d] = uk[((size_t)h * L->dim + d) * L->kv_rank + k];
    L->w_uk = operand_up(l, &o);
    const uint16_t *uv = ltensor(l, i, "mix.uv", H * L->vdim, L->kv_rank);
    o = operand_new(l, H, L->vdim_p, g->rank_pad);
    for (uint32_t h = 0; h < H && uv; h++) operand_put(l, &o, h, 0, uv + (size_t)h * L->vdim * L->kv_rank, L->vdim, L->kv_rank);
    L->w_uv = operand_up(l, &o);

    o = operand_new(l, 1, Wp, H * L->vdim_p);
    put_heads_out(l, &o, ltensor(l, i, "mix.o", W, H * L->vdim), 0, H, L->vdim, L->vdim_p);
    L->w_o = operand_up(l, &o);
}

/* What the recurrences share: sizes, decay and norm; tensor names behind `prefix`. */
static void read_recur(loader *l, uint32_t i, const char *prefix, const wrh_json *c, wrh_mix_recur *q)
{
    char nb[64];
#define NAME(n) (snprintf(nb, sizeof nb, "%s%s", prefix, n), nb)
    q->heads = need_u32(l, c, "heads", 1, HEADS_MAX);
    q->dim = need_u32(l, c, "dim", 1, WR_HIP_MIX_MAX_RECUR_DIM);
    const uint32_t rank = tensor_rows(l, i, NAME("w1"), DIM_MAX);
    if (l->st != WR_OK) return;
    const uint32_t hd = q->heads * q->dim;
    q->hd_p = p32(hd);
    q->rank_p = p32(rank);
    q->w_decay = plain(l, ltensor(l, i, NAME("w2"), hd, rank), hd, rank, q->hd_p);
    q->w0 = vec_put(l, ltensor(l, i, NAME("w0"), hd, 0), hd);
    q->norm = vec_put(l, ltensor(l, i, NAME("norm"), hd, 0), hd);
#undef NAME
}

static void read_wkv(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    struct wrh_mix_model *mm = l->mm;
    const uint32_t W = mm->width, Wp = mm->width_p;
    wrh_mix_recur *q = &L->rec;
    L->kind = WRH_MIXER_WKV;
    read_recur(l, i, "mix.", c, q);
    if (l->st != WR_OK) return;
    const uint32_t hd = q->heads * q->dim;
    L->heads = q->heads;
    L->dim = L->vdim = q->dim;
    q->u = vec_put(l, ltensor(l, i, "mix.u", q->heads, q->dim), hd);
    static const char *const mus[] = {"mix.mu.r", "mix.mu.k", "mix.mu.v", "mix.mu.g", "mix.mu.w"};
    for (uint32_t k = 0; k < 5; k++) {                     /* one after the other: each takes the padded width */
        const float *m = vec_put(l, ltensor(l, i, mus[k], W, 0), W);
        if (k == 0) L->mu = m;
    }
    static const char *const ins[] = {"mix.r", "mix.k", "mix.v", "mix.g"};
    operand o = operand_new(l, 4, q->hd_p, Wp);
    for (uint32_t k = 0; k < 4; k++) operand_put(l, &o, k, 0, ltensor(l, i, ins[k], hd, W), hd, W);
    L->w_rkvg = operand_up(l, &o);
    const uint32_t rank = tensor_rows(l, i, "mix.w1", DIM_MAX);
    L->w_low = plain(l, ltensor(l, i, "mix.w1", rank, W), rank, W, q->rank_p);
    L->w_o = plain(l, ltensor(l, i, "mix.o", W, hd), W, hd, Wp);
    mm->has_shift = 1;
}

static void read_parallel(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    struct wrh_mix_model *mm = l->mm;
    const uint32_t W = mm->width, Wp = mm->width_p;
    L->kind = WRH_MIXER_PARALLEL;
    const wrh_json *left = need_obj(l, c, "left"), *right = need_obj(l, c, "right");
    const double ls = need_num(l, c, "left_scale"), rs = need_num(l, c, "right_scale");
    if (l->st != WR_OK) return;
    wr_hip_mix_window *g = &L->win;
    const uint32_t H = g->heads = L->heads = need_u32(l, left, "heads", 1, HEADS_MAX);
    const uint32_t G = g->kv_heads = need_u32(l, left, "kv_heads", 1, HEADS_MAX);
    const uint32_t D = g->dim = L->dim = need_u32(l, left, "dim", 1, 4096);
    const uint32_t V = g->vdim = L->vdim = need_u32(l, left, "vdim", 1, 4096);
    const wrh_json *rot = need_obj(l, left, "rot"), *mask = need_obj(l, left, "mask");
    g->scale = (float)need_num(l, left, "scale");
    if (l->st != WR_OK) return;
    const double base = need_num(l, rot, "base");
    const uint32_t dims = need_u32(l, rot, "dims", 0, D);
    g->window = need_u32(l, mask, "size", 1, 0xFFFFFFFFu);
    if (l->st == WR_OK && (dims % 2 || base <= 0)) fail(l, WR_ERR_FORMAT, "config: layer %u: rotation of %u dimensions, base %g", i, dims, base);
    if (l->st == WR_OK && H % G) fail(l, WR_ERR_FORMAT, "config: layer %u: %u heads over %u key/value heads", i, H, G);
    if (l->st != WR_OK) return;
    g->dim_pad = wr_hip_mix_window_pad(D);
    g->vdim_pad = wr_hip_mix_window_pad(V);
    g->rot_half = dims / 2;
    g->out_scale = (float)ls;
    g->norm_values = 1;
    g->eps = mm->eps;
    g->maps = 1;
    L->right_scale = (float)rs;
    if ((uint64_t)H * g->dim_pad > DIM_MAX || (uint64_t)H * g->vdim_pad > DIM_MAX) {
        fail(l, WR_ERR_LIMIT, "config: layer %u is too wide", i);
        return;
    }
    L->rope = rope_index(l, base, dims, NULL);
    wrh_mix_recur *q = &L->rec;
    read_recur(l, i, "mix.right.", right, q);
    if (l->st != WR_OK) return;
    const uint32_t hd = q->heads * q->dim;
    q->a_bias = vec_put(l, ltensor(l, i, "mix.right.a.b", hd, 0), hd);
    L->sink = vec_put(l, ltensor(l, i, "mix.left.sink", H, 0), H);

    /* one product of the layer's input: the decay's low-rank part first, then 32-bit rows */
    const uint32_t rank = tensor_rows(l, i, "mix.right.w1", DIM_MAX);
    const struct {
        const char *name;
        uint32_t rows, *col;
    } parts[] = {{"mix.left.q", H * D, &L->col_q},  {"mix.left.k", G * D, &L->col_k},  {"mix.left.v", G * V, &L->col_v},
                 {"mix.right.r", hd, &L->col_rr},   {"mix.right.k", hd, &L->col_rk},   {"mix.right.v", hd, &L->col_rv},
                 {"mix.right.g", hd, &L->col_rg},   {"mix.right.a", hd, &L->col_ra}};
    const size_t n = sizeof parts / sizeof *parts;
    L->ld_in = 0;
    for (size_t k = 0; k < n; k++) {
        *parts[k].col = L->ld_in;
        L->ld_in += p32(parts[k].rows);
    }
    operand o = operand_new(l, 1, q->rank_p + L->ld_in, Wp);
    operand_put(l, &o, 0, 0, ltensor(l, i, "mix.right.w1", rank, W), rank, W);
    for (size_t k = 0; k < n; k++)
        operand_put(l, &o, 0, q->rank_p + *parts[k].col, ltensor(l, i, parts[k].name, parts[k].rows, W), parts[k].rows, W);
    L->w_in = operand_up(l, &o);

    /* one product over both halves' outputs, which arrive scaled */
    o = operand_new(l, 1, Wp, H * g->vdim_pad + q->hd_p);
    put_heads_out(l, &o, ltensor(l, i, "mix.left.o", W, H * V), 0, H, V, g->vdim_pad);
    put_heads_out(l, &o, ltensor(l, i, "mix.right.o", W, hd), H * g->vdim_pad, 1, hd, q->hd_p);
    L->w_o = operand_up(l, &o);
}

/* What attention mixers over grouped keys and values share: sizes and scale. */
static int read_heads(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L, uint32_t maps)
{
    wr_hip_mix_window *g = &L->win;
    const uint32_t H = g->heads = L->heads = need_u32(l, c, "heads", 1, HEADS_MAX);
    const uint32_t G = g->kv_heads = need_u32(l, c, "kv_heads", 1, HEADS_MAX);
    g->dim = L->dim = need_u32(l, c, "dim", 1, 4096);
    g->vdim = L->vdim = need_u32(l, c, "vdim", 1, 4096);
    g->scale = (float)need_num(l, c, "scale");
    if (l->st == WR_OK && H % G) fail(l, WR_ERR_FORMAT, "config: layer %u: %u heads over %u key/value heads", i, H, G);
    if (l->st != WR_OK) return 0;
    g->dim_pad = wr_hip_mix_window_pad(g->dim);
    g->vdim_pad = wr_hip_mix_window_pad(g->vdim);
    g->neighbours = 1;
    g->maps = maps;
    g->out_scale = 1.0f;
    g->eps = l->mm->eps;
    if ((uint64_t)H * maps * g->dim_pad > DIM_MAX || (uint64_t)H * g->vdim_pad > DIM_MAX) {
        fail(l, WR_ERR_LIMIT, "config: layer %u is too wide", i);
        return 0;
    }
    return 1;
}

/* The rotation of queries and keys; returns its base. */
static double read_rotation(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const wrh_json *rot = need_obj(l, c, "rot");
    if (l->st != WR_OK) return 0;
    const double base = need_num(l, rot, "base");
    const uint32_t dims = need_u32(l, rot, "dims", 0, L->win.dim);
    if (l->st == WR_OK && (dims % 2 || base <= 0)) fail(l, WR_ERR_FORMAT, "config: layer %u: rotation of %u dimensions, base %g", i, dims, base);
    if (l->st != WR_OK) return 0;
    L->win.rot_half = dims / 2;
    L->rope = rope_index(l, base, dims, given(rot, "scaling"));
    return base;
}

/* What windowed attention mixers of their own share: sizes, rotation of neighbours, window, scale. */
static int read_window_sizes(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L, uint32_t maps)
{
    L->kind = WRH_MIXER_WINDOW;
    L->kv_from = -1;
    if (!read_heads(l, i, c, L, maps)) return 0;
    (void)read_rotation(l, i, c, L);
    const wrh_json *mask = need_obj(l, c, "mask");
    if (l->st == WR_OK) L->win.window = need_u32(l, mask, "size", 1, 0xFFFFFFFFu);
    return l->st == WR_OK;
}

/* How far apart the rows of n outputs are kept: rows a multiple of 4 KiB apart share too few memory channels. */
static uint32_t row_stride(uint32_t n) { return n % 1024 ? n : n + 32; }

/* One product of a layer's input out of several matrices: where each one's outputs lie, then the operand, with `more`
 * rows behind theirs. */
static operand stack_inputs(loader *l, uint32_t i, const in_part *parts, size_t n, uint32_t *ld, uint32_t more)
{
    *ld = 0;
    for (size_t k = 0; k < n; k++) {
        *parts[k].col = *ld;
        *ld += p32(parts[k].rows);
    }
    operand o = operand_new(l, 1, *ld + more, l->mm->width_p);
    for (size_t k = 0; k < n; k++)
        operand_put(l, &o, 0, *parts[k].col, ltensor(l, i, parts[k].name, parts[k].rows, l->mm->width), parts[k].rows, l->mm->width);
    return o;
}

/* Their biases, and zeros for those that have none and for `more` outputs behind. */
static const float *stack_biases(loader *l, uint32_t i, const in_part *parts, size_t n, uint32_t ld, uint32_t more)
{
    size_t at = 0;
    float *b = l->st == WR_OK ? vec_take(l, ld + more, &at) : NULL;
    for (size_t k = 0; k < n && b; k++) {
        const uint16_t *src = parts[k].bias ? ltensor(l, i, parts[k].bias, parts[k].rows, 0) : NULL;
        for (uint32_t j = 0; src && j < parts[k].rows; j++) b[*parts[k].col + j] = widen(src[j]);
    }
    return b ? (const float *)(uintptr_t)(at + 1) : NULL;
}

static void read_window_out(loader *l, uint32_t i, wrh_mix_layer *L)
{
    const wr_hip_mix_window *g = &L->win;
    operand o = operand_new(l, 1, l->mm->width_p, g->heads * g->vdim_pad);
    put_heads_out(l, &o, ltensor(l, i, "mix.o", l->mm->width, g->heads * g->vdim), 0, g->heads, g->vdim, g->vdim_pad);
    L->w_o = operand_up(l, &o);
}

/* Values that are the keys ahead of their rotation, biases, capped scores, sinks, a gate per head. */
static void read_window_keys(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    if (!read_window_sizes(l, i, c, L, 1)) return;
    wr_hip_mix_window *g = &L->win;
    const uint32_t hq = g->heads * g->dim, hk = g->kv_heads * g->dim;
    if (given(c, "softcap")) g->softcap = (float)need_num(l, c, "softcap");
    if (l->st == WR_OK && (g->vdim != g->dim || g->softcap < 0))
        fail(l, WR_ERR_FORMAT, "config: layer %u: values of %u from keys of %u, scores capped at %g", i, g->vdim, g->dim, g->softcap);
    const in_part parts[] = {{"mix.q", hq, &L->col_q, "mix.q.b"}, {"mix.k", hk, &L->col_k, "mix.k.b"}, {"mix.g", g->heads, &L->col_rg, NULL}};
    const size_t n = sizeof parts / sizeof *parts;
    operand o = stack_inputs(l, i, parts, n, &L->ld_in, 0);
    L->w_in = operand_up(l, &o);
    L->b_in = stack_biases(l, i, parts, n, L->ld_in, 0);
    L->ld_in = row_stride(L->ld_in);
    L->col_v = L->col_k;
    L->has_gate = 1;
    L->sink = vec_put(l, ltensor(l, i, "mix.sink", g->heads, 0), g->heads);
    read_window_out(l, i, L);
}

static double dot_of(loader *l, uint32_t i, const char *a, const char *b, uint32_t n)
{
    const uint16_t *x = ltensor(l, i, a, n, 0), *y = ltensor(l, i, b, n, 0);
    double s = 0;
    for (uint32_t k = 0; x && y && k < n; k++) s += (double)widen(x[k]) * widen(y[k]);
    return s;
}

/* Two maps per head over the same values, normed queries and keys; possibly over another layer's keys and values. */
static void read_window_difference(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    if (!read_window_sizes(l, i, c, L, 2)) return;
    wr_hip_mix_window *g = &L->win;
    const double diff = need_num(l, c, "diff");
    if (given(c, "kv_from")) L->kv_from = (int32_t)need_u32(l, c, "kv_from", 0, 0x7FFFFFFFu);
    if (l->st != WR_OK) return;
    if (L->kv_from >= 0) {
        const wrh_mix_layer *S = (uint32_t)L->kv_from < i ? &l->mm->layers[L->kv_from] : NULL;
        if (!S || S->kind != WRH_MIXER_WINDOW || S->win.maps != 2 || S->kv_from >= 0 || S->win.kv_heads != g->kv_heads ||
            S->win.dim != g->dim || S->win.vdim != g->vdim) {
            fail(l, WR_ERR_FORMAT, "config: layer %u cannot use the keys and values of layer %d", i, L->kv_from);
            return;
        }
    }
    const double lambda = exp(dot_of(l, i, "mix.lq1", "mix.lk1", g->dim)) - exp(dot_of(l, i, "mix.lq2", "mix.lk2", g->dim)) + diff;
    g->diff = (float)lambda;
    g->out_scale = (float)(1.0 - diff);
    const in_part parts[] = {{"mix.q", g->heads * 2 * g->dim, &L->col_q, NULL}, {"mix.k", g->kv_heads * 2 * g->dim, &L->col_k, NULL},
                             {"mix.v", g->kv_heads * g->vdim, &L->col_v, NULL}};
    operand o = stack_inputs(l, i, parts, L->kv_from >= 0 ? 1 : sizeof parts / sizeof *parts, &L->ld_in, 0);
    L->w_in = operand_up(l, &o);
    L->ld_in = row_stride(L->ld_in);
    g->q_norm = vec_put(l, ltensor(l, i, "mix.q.norm", g->dim, 0), g->dim);
    if (L->kv_from < 0) g->k_norm = vec_put(l, ltensor(l, i, "mix.k.norm", g->dim, 0), g->dim);
    else L->col_k = L->col_v = WR_HIP_MIX_NO_KEYS;
    read_window_out(l, i, L);
}

/* gate and up [rows][cols] to rows at, at + 1, ... of matrix z, interleaved by tiles of 16 */
static void put_gated(loader *l, operand *o, uint32_t z, uint32_t at, const uint16_t *gate, const uint16_t *up, uint32_t rows,
                      uint32_t cols)
{
    for (uint32_t r = 0; r < rows && l->st == WR_OK; r++) {
        operand_put(l, o, z, at + r / 16 * 32 + r % 16, gate + (size_t)r * cols, 1, cols);
        operand_put(l, o, z, at + r / 16 * 32 + 16 + r % 16, up + (size_t)r * cols, 1, cols);
    }
}

static void read_dense(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const uint32_t W = l->mm->width, Wp = l->mm->width_p;
    L->mlp = WRH_MLP_DENSE;
    L->gelu = l->design->gelu;
    L->ff = need_u32(l, c, "ff", 1, DIM_MAX);
    if (l->st != WR_OK) return;
    L->ff_p = p32(L->ff);
    const uint16_t *gate = ltensor(l, i, "mlp.gate", L->ff, W), *up = ltensor(l, i, "mlp.up", L->ff, W);
    operand o = operand_new(l, 1, 2 * L->ff_p, Wp);
    put_gated(l, &o, 0, 0, gate, up, L->ff, W);
    L->w_gu = operand_up(l, &o);
    L->w_down = plain(l, ltensor(l, i, "mlp.down", W, L->ff), W, L->ff, Wp);
}

static void read_moe(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const uint32_t W = l->mm->width, Wp = l->mm->width_p;
    L->mlp = WRH_MLP_MOE;
    const wrh_json *ex = need_obj(l, c, "expert"), *ro = need_obj(l, c, "router");
    if (l->st != WR_OK) return;
    L->ff = need_u32(l, ex, "ff", 1, DIM_MAX);
    wr_hip_mix_router *q = &L->router;
    q->experts = need_u32(l, ro, "experts", 1, WR_HIP_MIX_MAX_EXPERTS);
    q->top = need_u32(l, ro, "top", 1, WR_HIP_MIX_MAX_TOP);
    if (l->st == WR_OK && q->top > q->experts) fail(l, WR_ERR_FORMAT, "config: layer %u: more experts per token than experts", i);
    if (l->st != WR_OK) return;
    L->ff_p = p32(L->ff);
    L->router_p = p16(q->experts);
    L->w_router = plain(l, ltensor(l, i, "mlp.router", q->experts, W), q->experts, W, L->router_p);
    operand up = operand_new(l, q->experts, L->ff_p, Wp), down = operand_new(l, q->experts, Wp, L->ff_p);
    for (uint32_t x = 0; x < q->experts && l->st == WR_OK; x++) {
        char nb[64];
        snprintf(nb, sizeof nb, "mlp.e%u.up", x);
        operand_put(l, &up, x, 0, ltensor(l, i, nb, L->ff, W), L->ff, W);
        snprintf(nb, sizeof nb, "mlp.e%u.down", x);
        operand_put(l, &down, x, 0, ltensor(l, i, nb, W, L->ff), W, L->ff);
    }
    L->w_eup = operand_up(l, &up);
    L->w_edown = operand_up(l, &down);
}

/* Experts of gated units: gate and up interleaved, down. */
static void read_gated_experts(loader *l, uint32_t i, wrh_mix_layer *L)
{
    const uint32_t W = l->mm->width, Wp = l->mm->width_p;
    const wr_hip_mix_router *q = &L->router;
    operand up = operand_new(l, q->experts, 2 * L->ff_p, Wp), down = operand_new(l, q->experts, Wp, L->ff_p);
    for (uint32_t x = 0; x < q->experts && l->st == WR_OK; x++) {
        char nb[3][64];
        static const char *const ends[] = {"gate", "up", "down"};
        for (uint32_t k = 0; k < 3; k++) snprintf(nb[k], sizeof nb[k], "mlp.e%u.%s", x, ends[k]);
        const uint16_t *g = ltensor(l, i, nb[0], L->ff, W), *u = ltensor(l, i, nb[1], L->ff, W);
        put_gated(l, &up, x, 0, g, u, L->ff, W);
        operand_put(l, &down, x, 0, ltensor(l, i, nb[2], W, L->ff), W, L->ff);
    }
    L->w_eup = operand_up(l, &up);
    L->w_edown = operand_up(l, &down);
}

/* Clamped gated experts behind a corrected softmax router with groups and outputs that pass the input on; a shared
 * expert with a gate of its own. */
static void read_grouped_moe(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const uint32_t W = l->mm->width, Wp = l->mm->width_p;
    L->mlp = WRH_MLP_MOE;
    const wrh_json *ex = need_obj(l, c, "expert"), *ro = need_obj(l, c, "router"), *sh = given(c, "shared");
    if (l->st != WR_OK) return;
    wr_hip_mix_router *q = &L->router;
    L->ff = need_u32(l, ex, "ff", 1, DIM_MAX);
    L->limit = (float)need_num(l, ex, "limit");
    q->experts = need_u32(l, ro, "experts", 1, WR_HIP_MIX_MAX_EXPERTS);
    q->top = need_u32(l, ro, "top", 1, WR_HIP_MIX_MAX_TOP);
    q->identity = given(ro, "identity") ? need_u32(l, ro, "identity", 0, WR_HIP_MIX_MAX_EXPERTS) : 0;
    q->scale = (float)need_num(l, ro, "scale");
    q->softmax_all = 1;
    const uint32_t outputs = q->experts + q->identity;
    if (l->st == WR_OK && outputs > WR_HIP_MIX_MAX_EXPERTS) fail(l, WR_ERR_LIMIT, "config: layer %u: %u router outputs", i, outputs);
    const wrh_json *groups = given(ro, "groups");
    if (groups) {
        q->groups = need_u32(l, groups, "count", 1, WR_HIP_MIX_MAX_GROUPS);
        q->keep = need_u32(l, groups, "keep", 1, q->groups);
        if (l->st == WR_OK && outputs % q->groups)
            fail(l, WR_ERR_FORMAT, "config: layer %u: %u router outputs in %u groups", i, outputs, q->groups);
    }
    uint32_t shared = 0;
    if (sh) {
        shared = need_u32(l, sh, "ff", 1, DIM_MAX);
        L->shared_limit = (float)need_num(l, sh, "limit");
        q->shared_gate = 1;
    }
    if (l->st != WR_OK) return;
    if (q->top > (q->groups ? outputs / q->groups * q->keep : outputs) || L->limit <= 0 || (sh && L->shared_limit <= 0)) {
        fail(l, WR_ERR_FORMAT, "config: layer %u: %u of %u router outputs, limits %g and %g", i, q->top, outputs, L->limit, L->shared_limit);
        return;
    }
    L->ff_p = p32(L->ff);
    L->shared_p = p32(shared);
    L->router_p = p32(outputs + q->shared_gate);
    operand o = operand_new(l, 1, L->router_p + 2 * L->shared_p, Wp);
    operand_put(l, &o, 0, 0, ltensor(l, i, "mlp.router", outputs, W), outputs, W);
    if (sh) {
        operand_put(l, &o, 0, outputs, ltensor(l, i, "mlp.shared.sg", 1, W), 1, W);
        const uint16_t *gate = ltensor(l, i, "mlp.shared.gate", shared, W), *up = ltensor(l, i, "mlp.shared.up", shared, W);
        put_gated(l, &o, 0, L->router_p, gate, up, shared, W);
        L->w_down = plain(l, ltensor(l, i, "mlp.shared.down", W, shared), W, shared, Wp);
    }
    L->w_router = operand_up(l, &o);
    q->correction = vec_put(l, ltensor(l, i, "mlp.correction", outputs, 0), outputs);
    read_gated_experts(l, i, L);
}

/* ---- joint layers: the mixer's and the feed-forward's readers gather, finish_joint makes the products ---- */

static void joint_part(loader *l, const char *name, uint32_t rows, uint32_t *col, const char *bias)
{
    if (l->n_parts < PARTS_MAX) l->parts[l->n_parts++] = (in_part){name, rows, col, bias};
    else fail(l, WR_ERR_INTERNAL, "too many input products in a layer");
}

static int read_joint_attention(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    L->kind = WRH_MIXER_JOINT;
    L->kv_from = L->turn = -1;
    L->win.window = 0xFFFFFFFFu;
    return c && read_heads(l, i, c, L, 1);
}

/* Biases, normed and rotated queries and keys, a sink per head, values turned with their position. */
static void read_joint_turned(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    if (!read_joint_attention(l, i, c, L)) return;
    wr_hip_mix_window *g = &L->win;
    const double base = read_rotation(l, i, c, L);
    if (l->st == WR_OK && g->vdim % 2) fail(l, WR_ERR_FORMAT, "config: layer %u: values of %u elements turn in pairs", i, g->vdim);
    if (l->st != WR_OK) return;
    L->turn = (int32_t)rope_index(l, base, g->vdim, NULL);
    joint_part(l, "mix.q", g->heads * g->dim, &L->col_q, "mix.q.b");
    joint_part(l, "mix.k", g->kv_heads * g->dim, &L->col_k, "mix.k.b");
    joint_part(l, "mix.v", g->kv_heads * g->vdim, &L->col_v, "mix.v.b");
    g->q_norm = vec_put(l, ltensor(l, i, "mix.q.norm", g->dim, 0), g->dim);
    g->k_norm = vec_put(l, ltensor(l, i, "mix.k.norm", g->dim, 0), g->dim);
    L->sink = vec_put(l, ltensor(l, i, "mix.sink", g->heads, 0), g->heads);
    L->b_o = vec_put(l, ltensor(l, i, "mix.o.b", l->mm->width, 0), l->mm->width);
}

/* Attention in chunks with sinks and a gate per output element, beside the recurrence whose forget gate makes the keys. */
static void read_joint_chunks(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const wrh_json *left = need_obj(l, c, "left"), *right = need_obj(l, c, "right");
    if (!read_joint_attention(l, i, left, L)) return;
    wr_hip_mix_window *g = &L->win;
    wrh_mix_recur *q = &L->rec;
    const wrh_json *mask = need_obj(l, left, "mask");
    if (l->st != WR_OK) return;
    g->chunk = need_u32(l, mask, "size", 1, 0xFFFFFFFFu);
    g->out_scale = (float)need_num(l, c, "left_scale");
    L->right_scale = (float)need_num(l, c, "right_scale");
    q->heads = need_u32(l, right, "heads", 1, HEADS_MAX);
    q->dim = need_u32(l, right, "dim", 1, WR_HIP_MIX_MAX_RECUR_DIM);
    q->vdim = need_u32(l, right, "vdim", 1, WR_HIP_MIX_MAX_RECUR_DIM);
    if (l->st != WR_OK) return;
    const uint32_t hd = q->heads * q->dim;
    L->beside = WRH_BESIDE_FORGET;
    q->hd_p = p32(hd);
    q->hv_p = p32(q->heads * q->vdim);
    L->has_gate = 1;
    g->gate_wide = 1;
    joint_part(l, "mix.right.q", hd, &L->col_rr, NULL);    /* first: it leaves the product through SiLU */
    L->silu_end = q->hd_p;
    joint_part(l, "mix.right.f", hd, &L->col_rk, NULL);    /* (its bias is the recurrence's) */
    joint_part(l, "mix.right.v", q->heads * q->vdim, &L->col_rv, NULL);
    joint_part(l, "mix.left.q", g->heads * g->dim, &L->col_q, NULL);
    joint_part(l, "mix.left.k", g->kv_heads * g->dim, &L->col_k, NULL);
    joint_part(l, "mix.left.v", g->kv_heads * g->vdim, &L->col_v, NULL);
    joint_part(l, "mix.left.g", g->heads * g->vdim, &L->col_rg, NULL);
    q->w0 = vec_put(l, ltensor(l, i, "mix.right.f.b", hd, 0), hd);
    q->lower = vec_put(l, ltensor(l, i, "mix.right.lower", hd, 0), hd);
    q->norm = vec_put(l, ltensor(l, i, "mix.right.norm", q->vdim, 0), q->vdim);
    L->sink = vec_put(l, ltensor(l, i, "mix.left.sink", g->heads, 0), g->heads);
}

/* Attention with one added to the softmax's denominator beside a gated recurrence, each output normed, and their mean. */
static void read_joint_averaged(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const wrh_json *left = need_obj(l, c, "left"), *right = need_obj(l, c, "right");
    if (!read_joint_attention(l, i, left, L)) return;
    wr_hip_mix_window *g = &L->win;
    const uint32_t W = l->mm->width;
    (void)read_rotation(l, i, left, L);
    L->gru = need_u32(l, right, "width", 1, DIM_MAX);
    if (l->st != WR_OK) return;
    L->beside = WRH_BESIDE_GRU;
    L->gru_p = p32(L->gru);
    joint_part(l, "mix.left.q", g->heads * g->dim, &L->col_q, "mix.left.q.b");
    joint_part(l, "mix.left.k", g->kv_heads * g->dim, &L->col_k, "mix.left.k.b");
    joint_part(l, "mix.left.v", g->kv_heads * g->vdim, &L->col_v, "mix.left.v.b");
    joint_part(l, "mix.right.z", L->gru, &L->col_rr, "mix.right.z.b");
    joint_part(l, "mix.right.x", L->gru, &L->col_rk, "mix.right.x.b");
    joint_part(l, "mix.right.g", L->gru, &L->col_rv, NULL);
    g->q_norm = vec_put(l, ltensor(l, i, "mix.left.q.norm", g->dim, 0), g->dim);
    g->k_norm = vec_put(l, ltensor(l, i, "mix.left.k.norm", g->dim, 0), g->dim);
    size_t at = 0;
    if (vec_take(l, g->heads, &at)) L->sink = (const float *)(uintptr_t)(at + 1);      /* scores of zero */
    L->b_o = vec_put(l, ltensor(l, i, "mix.left.o.b", W, 0), W);
    static const char *const outs[] = {"mix.left.out", "mix.right.out"};
    for (uint32_t k = 0; k < 2; k++) {
        L->out_norm[k] = vec_put(l, ltensor(l, i, outs[k], W, 0), W);
        for (uint32_t j = 0; j < W && L->out_norm[k]; j++) l->vec[(uintptr_t)L->out_norm[k] - 1 + j] *= 0.5f;
    }
}

/* Clamped gated units. */
static void read_joint_dense(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    L->mlp = WRH_MLP_DENSE;
    L->ff = need_u32(l, c, "ff", 1, DIM_MAX);
    L->limit = (float)need_num(l, c, "limit");
    if (l->st == WR_OK && !(L->limit > 0)) fail(l, WR_ERR_FORMAT, "config: layer %u: units clamped at %g", i, L->limit);
    L->ff_p = p32(L->ff);
}

/* Gated experts behind a logistic router, whose weights multiply the experts' input. */
static void read_joint_moe(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    L->mlp = WRH_MLP_MOE;
    const wrh_json *ex = need_obj(l, c, "expert"), *ro = need_obj(l, c, "router");
    if (l->st != WR_OK) return;
    wr_hip_mix_router *q = &L->router;
    L->ff = need_u32(l, ex, "ff", 1, DIM_MAX);
    q->experts = need_u32(l, ro, "experts", 1, WR_HIP_MIX_MAX_EXPERTS);
    q->top = need_u32(l, ro, "top", 1, WR_HIP_MIX_MAX_TOP);
    if (l->st == WR_OK && q->top > q->experts) fail(l, WR_ERR_FORMAT, "config: layer %u: more experts per token than experts", i);
    if (l->st != WR_OK) return;
    q->logistic = 1;
    L->gated = L->weigh_input = 1;
    L->ff_p = p32(L->ff);
    L->router_p = p32(q->experts);
    joint_part(l, "mlp.router", q->experts, &L->col_router, NULL);
    read_gated_experts(l, i, L);
}

static void finish_joint(loader *l, uint32_t i, wrh_mix_layer *L)
{
    const uint32_t W = l->mm->width, Wp = l->mm->width_p, ff = L->mlp == WRH_MLP_DENSE ? L->ff_p : 0;
    const wr_hip_mix_window *g = &L->win;
    const uint32_t heads = g->heads * g->vdim_pad, beside = L->beside == WRH_BESIDE_FORGET ? L->rec.hv_p : L->gru_p;
    if (l->st != WR_OK) return;
    int biased = 0;
    for (size_t k = 0; k < l->n_parts; k++) biased |= l->parts[k].bias != NULL;
    operand o = stack_inputs(l, i, l->parts, l->n_parts, &L->n_in, 2 * ff);
    L->ld_in = row_stride(L->n_in);
    const uint16_t *wd = NULL;
    if (ff) {
        const uint16_t *gate = ltensor(l, i, "mlp.gate", L->ff, W), *up = ltensor(l, i, "mlp.up", L->ff, W);
        put_gated(l, &o, 0, L->n_in, gate, up, L->ff, W);
        wd = ltensor(l, i, "mlp.down", W, L->ff);
    }
    L->w_in = operand_up(l, &o);
    if (biased) L->b_in = stack_biases(l, i, l->parts, l->n_parts, L->n_in, 2 * ff);
    const char *first = L->beside ? "mix.left.o" : "mix.o";
    const uint16_t *wo = ltensor(l, i, first, W, g->heads * g->vdim), *wo2 = NULL;
    const uint32_t n2 = L->beside == WRH_BESIDE_FORGET ? L->rec.heads * L->rec.vdim : L->gru;
    if (L->beside) wo2 = ltensor(l, i, "mix.right.o", W, n2);
    const int apart = L->out_norm[0] != NULL;
    o = operand_new(l, 1, Wp, apart ? heads : heads + beside + ff);
    put_heads_out(l, &o, wo, 0, g->heads, g->vdim, g->vdim_pad);
    if (apart) {
        L->w_o = operand_up(l, &o);
        L->w_o2 = plain(l, wo2, W, n2, Wp);
        if (ff) L->w_down = plain(l, wd, W, L->ff, Wp);
        return;
    }
    put_heads_out(l, &o, wo2, heads, 1, n2, beside);
    put_heads_out(l, &o, wd, heads + beside, 1, L->ff, ff);
    L->w_o = operand_up(l, &o);
}

static void read_layer(loader *l, uint32_t i, const wrh_json *c, wrh_mix_layer *L)
{
    const uint32_t W = l->mm->width;
    const char *type = need_str(l, c, "type");
    const wrh_json *mixer = need_obj(l, c, "mixer");
    if (l->st != WR_OK) return;
    static const struct {
        const char *name;
        void (*read)(loader *, uint32_t, const wrh_json *, wrh_mix_layer *);
        unsigned designs;
    } mixers[] = {{"lightning", read_lightning, DESIGN_BIPOTAR},
                  {"latent_attention", read_latent, DESIGN_BIPOTAR},
                  {"wkv", read_wkv, DESIGN_TAREDRA},
                  {"parallel", read_parallel, DESIGN_TAREDRA},
                  {"attention", read_window_keys, DESIGN_FEDIRAX},
                  {"attention_2", read_window_difference, DESIGN_FEDIRAX},
                  {"attention", read_joint_turned, DESIGN_MAROSUN},
                  {"parallel", read_joint_chunks, DESIGN_MAROSUN},
                  {"parallel_2", read_joint_averaged, DESIGN_MAROSUN}},
      mlps[] = {{"dense", read_dense, DESIGN_BIPOTAR | DESIGN_TAREDRA},
                {"moe", read_moe, DESIGN_BIPOTAR},
                {"moe", read_grouped_moe, DESIGN_FEDIRAX},
                {"dense", read_joint_dense, DESIGN_MAROSUN},
                {"moe", read_joint_moe, DESIGN_MAROSUN}};
    const size_t n_mixers = sizeof mixers / sizeof *mixers, n_mlps = sizeof mlps / sizeof *mlps;
    const wrh_mix_design *d = l->design;
    size_t k = 0;
    while (k < n_mixers && (strcmp(type, mixers[k].name) || !(mixers[k].designs & d->bit))) k++;
    if (k == n_mixers) {
        fail(l, WR_ERR_UNSUPPORTED, "layer %u: mixer '%s' is not served by this engine", i, type);
        return;
    }
    l->n_parts = 0;
    mixers[k].read(l, i, mixer, L);
    L->norm1 = norm_put(l, ltensor(l, i, "norm1", W, 0), W);
    if (d->post_norms) L->norm1b = norm_put(l, ltensor(l, i, "norm1b", W, 0), W);
    const wrh_json *mlp = wrh_json_get(c, "mlp");
    if (!mlp || mlp->type == WRH_JSON_NULL) {
        if (d->joint) finish_joint(l, i, L);
        return;
    }
    const char *kind = need_str(l, mlp, "kind");
    if (l->st != WR_OK) return;
    for (k = 0; k < n_mlps && (strcmp(kind, mlps[k].name) || !(mlps[k].designs & d->bit)); k++) {}
    if (k == n_mlps) {
        fail(l, WR_ERR_UNSUPPORTED, "layer %u: feed-forward '%s' is not served by this engine", i, kind);
        return;
    }
    mlps[k].read(l, i, mlp, L);
    if (d->joint) {
        finish_joint(l, i, L);
        return;
    }
    L->norm2 = norm_put(l, ltensor(l, i, "norm2", W, 0), W);
    if (d->post_norms) L->norm2b = norm_put(l, ltensor(l, i, "norm2b", W, 0), W);
}

/* ------------------------------------------------------------------ model -- */

/* The order layers run in, and each run's own pages or state. */
static void plan_runs(loader *l, const wrh_json *cfg)
{
    struct wrh_mix_model *mm = l->mm;
    uint32_t start = 0, stop = 0, times = 1;
    const wrh_json *loop = wrh_json_get(cfg, "loop");
    if (loop && loop->type != WRH_JSON_NULL) {
        start = need_u32(l, loop, "start", 0, mm->n_layers);
        stop = need_u32(l, loop, "stop", start, mm->n_layers);
        times = need_u32(l, loop, "times", 1, 1024);
    }
    if (l->st != WR_OK) return;
    mm->looped = times > 1 && stop > start;
    mm->n_runs = mm->n_layers + (times - 1) * (stop - start);
    mm->runs = calloc(mm->n_runs, sizeof *mm->runs);
    mm->latent_dim = calloc(mm->n_runs, sizeof *mm->latent_dim);
    mm->state_elems = calloc((size_t)2 * mm->n_runs, sizeof *mm->state_elems);
    if (!mm->runs || !mm->latent_dim || !mm->state_elems) {
        fail(l, WR_ERR_NOMEM, "out of memory");
        return;
    }
    uint32_t n = 0;
    for (uint32_t i = 0; i < start; i++) mm->runs[n++].layer = i;
    for (uint32_t t = 0; t < times; t++)
        for (uint32_t i = start; i < stop; i++) {
            mm->runs[n].layer = i;
            mm->runs[n++].add_embedding = (uint8_t)(t > 0 && i == start);
        }
    for (uint32_t i = stop; i < mm->n_layers; i++) mm->runs[n++].layer = i;
    for (uint32_t r = 0; r < n; r++) {
        const wrh_mix_layer *L = &mm->layers[mm->runs[r].layer];
        const uint64_t matrix = (uint64_t)L->rec.heads * L->rec.dim * L->rec.dim;
        switch (L->kind) {
        case WRH_MIXER_LATENT:
            mm->runs[r].store = mm->n_latent;
            mm->latent_dim[mm->n_latent++] = L->geo.rank_pad + L->geo.rot_pad;
            break;
        case WRH_MIXER_LIGHTNING:
            mm->runs[r].store = mm->n_state;
            mm->state_elems[mm->n_state++] = (uint64_t)L->heads * L->dim * L->vdim;
            break;
        case WRH_MIXER_WKV:
            mm->runs[r].store = mm->n_state;
            mm->state_elems[mm->n_state++] = matrix;
            mm->runs[r].store2 = mm->n_state;
            mm->state_elems[mm->n_state++] = mm->width_p;
            break;
        case WRH_MIXER_PARALLEL:
            mm->runs[r].store = mm->n_latent;
            mm->latent_dim[mm->n_latent++] = L->win.kv_heads * (L->win.dim_pad + L->win.vdim_pad);
            mm->runs[r].store2 = mm->n_state;
            mm->state_elems[mm->n_state++] = matrix;
            break;
        case WRH_MIXER_WINDOW:
            if (L->kv_from >= 0) {                         /* the pages of that layer's last run before this one */
                for (uint32_t k = 0; k < r; k++)
                    if (mm->runs[k].layer == (uint32_t)L->kv_from) mm->runs[r].store = mm->runs[k].store;
                break;
            }
            mm->runs[r].store = mm->n_latent;
            mm->latent_dim[mm->n_latent++] = L->win.kv_heads * (L->win.maps * L->win.dim_pad + L->win.vdim_pad);
            break;
        case WRH_MIXER_JOINT:
            mm->runs[r].store = mm->n_latent;
            mm->latent_dim[mm->n_latent++] = L->win.kv_heads * (L->win.dim_pad + L->win.vdim_pad);
            if (L->beside == WRH_BESIDE_NOTHING) break;
            mm->runs[r].store2 = mm->n_state;
            mm->state_elems[mm->n_state++] = L->beside == WRH_BESIDE_GRU ? L->gru_p
                                                                         : (uint64_t)L->rec.heads * L->rec.dim * L->rec.vdim;
            break;
        }
    }
}

static void upload_small(loader *l)
{
    struct wrh_mix_model *mm = l->mm;
    if (l->st != WR_OK) return;
    mm->vecs = wr_hip_attn_dev_alloc(l->vec_n * sizeof(float));
    if (!mm->vecs || wr_hip_attn_h2d(mm->vecs, l->vec, l->vec_n * sizeof(float)) != WR_HIP_OK) {
        fail(l, WR_ERR_NOMEM, "upload of the norm vectors failed");
        return;
    }
    vec_fix(mm, &mm->embed_norm);
    vec_fix(mm, &mm->final_norm);
    for (uint32_t i = 0; i < mm->n_layers; i++) {
        wrh_mix_layer *L = &mm->layers[i];
        const float **p[] = {&L->decay, &L->mix_norm, &L->dq_norm, &L->dkv_norm, &L->norm1, &L->norm1b, &L->norm2, &L->norm2b,
                             &L->mu, &L->sink, &L->rec.w0, &L->rec.u, &L->rec.a_bias, &L->rec.norm, &L->b_in, &L->win.q_norm,
                             &L->win.k_norm, &L->router.correction, &L->rec.lower, &L->b_o, &L->out_norm[0],
                             &L->out_norm[1]};
        for (size_t k = 0; k < sizeof p / sizeof *p; k++) vec_fix(mm, p[k]);
    }
    for (uint32_t r = 0; r < mm->n_ropes && l->st == WR_OK; r++) {
        wrh_mix_rope *R = &mm->ropes[r];
        if (R->dims == 0) continue;
        const size_t bytes = R->dims / 2 * sizeof(double);
        double *f = malloc(bytes);
        R->freq_dev = wr_hip_attn_dev_alloc(bytes);
        if (f)
            for (uint32_t i = 0; i < R->dims / 2; i++) f[i] = rope_freq(R, i);
        if (!f || !R->freq_dev || wr_hip_attn_h2d(R->freq_dev, f, bytes) != WR_HIP_OK)
            fail(l, WR_ERR_NOMEM, "upload of the rotary frequencies failed");
        free(f);
    }
}

void wrh_mix_free(struct wrh_mix_model *mm)
{
    if (!mm) return;
    for (uint32_t i = 0; mm->layers && i < mm->n_layers; i++) {
        wrh_mix_layer *L = &mm->layers[i];
        wr_hip_mat *w[] = {L->w_qkvg, L->w_o, L->w_d, L->w_uq, L->w_uk, L->w_uv, L->w_gu, L->w_down, L->w_router, L->w_eup,
                           L->w_edown, L->w_rkvg, L->w_low, L->w_in, L->rec.w_decay, L->w_o2};
        for (size_t k = 0; k < sizeof w / sizeof *w; k++) wr_hip_mix_mat_destroy(w[k]);
    }
    for (uint32_t r = 0; mm->ropes && r < mm->n_ropes; r++) wr_hip_attn_dev_free(mm->ropes[r].freq_dev);
    wr_hip_mix_mat_destroy(mm->head);
    wr_hip_attn_dev_free(mm->embed_dev);
    wr_hip_attn_dev_free(mm->vecs);
    wr_hip_attn_dev_free(mm->scratch);
    wr_hip_attn_dev_free(mm->logits_dev);
    wr_hip_attn_host_free(mm->logits_host);
    wr_hip_mix_step_destroy(mm->step);
    wr_hip_mix_pool_destroy(mm->pool);
    free(mm->layers);
    free(mm->runs);
    free(mm->ropes);
    free(mm->latent_dim);
    free(mm->state_elems);
    free(mm->free_pages);
    free(mm->free_slots);
    pthread_mutex_destroy(&mm->lock);
    free(mm);
}

wr_status wrh_mix_load(wr_engine *e, const char *dir, const char *arch, const wrh_json *cfg, const wr_model_params *p,
                       wr_model *m)
{
    if (!wr_hip_mix_available()) {
        wrh_logf(e, 0, "loader: architecture '%s' needs the device steps of mixer-stack models, which this device library "
                      "does not have", arch);
        return WR_ERR_UNSUPPORTED;
    }
    struct wrh_mix_model *mm = calloc(1, sizeof *mm);
    if (!mm) return WR_ERR_NOMEM;
    pthread_mutex_init(&mm->lock, NULL);
    const wrh_mix_design *design = designs;
    while (strcmp(design->arch, arch)) design++;           /* (the registry holds no other name) */
    loader l = {.e = e, .design = design, .mm = mm, .st = WR_OK};
    const wrh_json *layers = wrh_json_get(cfg, "layers");
    if (!layers || layers->type != WRH_JSON_ARRAY || layers->count == 0)
        fail(&l, WR_ERR_FORMAT, "config: 'layers' missing or empty");
    mm->f32 = p->keep_quantized == WR_QUANT_F32;
    mm->width = need_u32(&l, cfg, "width", 1, 1u << 16);
    mm->vocab = need_u32(&l, cfg, "vocab", 1, 1u << 24);
    mm->width_p = p32(mm->width);
    mm->vocab_p = p16(mm->vocab);
    const wrh_json *norm = need_obj(&l, cfg, "norm");
    if (norm) mm->eps = (float)need_num(&l, norm, "eps");
    double scale = 1.0;
    if (wrh_json_get(cfg, "logit_scale")) scale = need_num(&l, cfg, "logit_scale");
    mm->logit_scale = (float)scale;
    if (design->embed_plain) {
        mm->embed_scale = 1.0f;
    } else if (!design->embed_norm) {
        const wrh_json *emb = need_obj(&l, cfg, "embedding");
        if (emb) mm->embed_scale = (float)need_num(&l, emb, "scale");
    }
    if (l.st == WR_OK) {
        mm->n_layers = layers->count;
        mm->layers = calloc(mm->n_layers, sizeof *mm->layers);
        mm->ropes = calloc((size_t)2 * mm->n_layers, sizeof *mm->ropes);
        if (!mm->layers || !mm->ropes) fail(&l, WR_ERR_NOMEM, "out of memory");
    }
    if (l.st == WR_OK) {
        char path[4096];
        if ((size_t)snprintf(path, sizeof path, "%s/model.safetensors", dir) >= sizeof path)
            fail(&l, WR_ERR_INVAL, "path too long");
        else {
            const int rc = wrh_safetensors_open(&l.f, path);
            if (rc != WRH_ST_OK) fail(&l, (wr_status)rc, "cannot read %s", path);
        }
    }
    if (l.st == WR_OK) {
        const wrh_json *c = layers->first;
        for (uint32_t i = 0; i < mm->n_layers && l.st == WR_OK; i++, c = c->next) read_layer(&l, i, c, &mm->layers[i]);
        const uint16_t *emb = tensor(&l, "embed", mm->vocab, mm->width);
        if (design->embed_norm) mm->embed_norm = norm_put(&l, tensor(&l, "embed.norm", mm->width, 0), mm->width);
        mm->final_norm = norm_put(&l, tensor(&l, "final.norm", mm->width, 0), mm->width);
        mm->head = plain(&l, design->tied_head ? emb : tensor(&l, "head", mm->vocab, mm->width), mm->vocab, mm->width, mm->vocab_p);
        if (l.st == WR_OK) {
            const size_t bytes = (size_t)mm->vocab * mm->width * 2;
            mm->embed_dev = wr_hip_attn_dev_alloc(bytes);
            if (!mm->embed_dev || wr_hip_attn_h2d(mm->embed_dev, emb, bytes) != WR_HIP_OK)
                fail(&l, WR_ERR_NOMEM, "upload of the embedding failed");
        }
    }
    if (l.st == WR_OK) plan_runs(&l, cfg);
    upload_small(&l);
    if (l.st == WR_OK && wr_hip_attn_sync() != WR_HIP_OK) fail(&l, WR_ERR_INTERNAL, "device error during upload");
    free(l.vec);
    wrh_safetensors_close(&l.f);
    if (l.st != WR_OK) {
        wrh_mix_free(mm);
        return l.st;
    }
    snprintf(m->arch, sizeof m->arch, "%s", arch);
    m->mix = mm;
    m->n_layers = mm->n_runs;
    m->hidden = mm->width;
    m->vocab = mm->vocab;
    m->rms_eps = mm->eps;
    m->tied_head = design->tied_head;
    for (uint32_t i = 0; i < mm->n_layers; i++) {
        const wrh_mix_layer *L = &mm->layers[i];
        if (L->heads > m->n_q) m->n_q = L->heads;
        if (L->dim > m->head_dim) m->head_dim = L->dim;
        if (L->ff > m->ffn) m->ffn = L->ff;
        if (L->kind == WRH_MIXER_LATENT) {
            m->has_swa = 1;
            m->n_kv = 1;                                   /* one latent row per position, shared by the heads */
            if (L->geo.window > m->sliding_window) m->sliding_window = L->geo.window;
            m->rope_base = (float)mm->ropes[L->rope].base;
        }
        if (L->kind == WRH_MIXER_PARALLEL || L->kind == WRH_MIXER_WINDOW) {
            m->has_swa = 1;
            if (L->win.kv_heads > m->n_kv) m->n_kv = L->win.kv_heads;
            if (L->win.window > m->sliding_window) m->sliding_window = L->win.window;
            m->rope_base = (float)mm->ropes[L->rope].base;
        }
        if (L->kind == WRH_MIXER_JOINT) {
            if (L->win.kv_heads > m->n_kv) m->n_kv = L->win.kv_heads;
            if (L->win.chunk) m->has_swa = 1;
            if (L->win.chunk > m->sliding_window) m->sliding_window = L->win.chunk;
            if (L->win.rot_half) m->rope_base = (float)mm->ropes[L->rope].base;
        }
    }
    m->max_context = p->max_context ? p->max_context : WRH_DEFAULT_CTX;
    return WR_OK;
}
