/*
 * wr_mix.c — cache pool and layer walk of mixer-stack models (wr_mix.h).
 *
 * A session of such a model owns nothing on the device: its cached positions live
 * in pages of 64 that it takes from the model's pool as it grows, its recurrent
 * state in one of the pool's slots (two buffers: a step reads the current one and
 * writes the other, and the session moves to it only when the step succeeded).
 * wr_step, wr_prefill and wr_batch_step are special cases of one mixed step over
 * portions of several sessions; a step of more rows than the device scratch takes
 * runs in passes, which is the same as cutting the portions.
 */
#define _POSIX_C_SOURCE 200809L
#include "wr_mix.h"

#include <stdlib.h>
#include <string.h>

static uint32_t p32(uint32_t n) { return (n + 31) / 32 * 32; }

/* ------------------------------------------------------------------- pool -- */

wr_status wr_model_set_cache_pool(wr_model *m, uint32_t tokens, uint32_t sessions)
{
    if (!m) return WR_ERR_INVAL;
    if (!m->mix) return WR_ERR_UNSUPPORTED;
    struct wrh_mix_model *mm = m->mix;
    wr_status st = WR_OK;
    pthread_mutex_lock(&mm->lock);
    if (mm->pool) {
        st = WR_ERR_STATE;                             /* the first session fixed it */
    } else {
        mm->pool_tokens = tokens;
        mm->pool_slots = sessions;
    }
    pthread_mutex_unlock(&mm->lock);
    return st;
}

static wr_status pool_ready(wr_model *m)
{
    struct wrh_mix_model *mm = m->mix;
    if (mm->pool) return WR_OK;
    const uint32_t slots = mm->pool_slots ? mm->pool_slots : WR_BATCH_MAX;
    const uint64_t tokens = mm->pool_tokens ? mm->pool_tokens
                                            : (uint64_t)((m->max_context + WR_HIP_MIX_PAGE - 1) / WR_HIP_MIX_PAGE) *
                                                  WR_HIP_MIX_PAGE * slots;
    const uint64_t pages = (tokens + WR_HIP_MIX_PAGE - 1) / WR_HIP_MIX_PAGE;
    if (pages > 0x7FFFFFFFu) return WR_ERR_LIMIT;
    mm->free_pages = malloc((size_t)pages * sizeof *mm->free_pages);
    mm->free_slots = malloc((size_t)slots * sizeof *mm->free_slots);
    int rc = (mm->free_pages && mm->free_slots) ? WR_HIP_OK : WR_HIP_ERR_NOMEM;
    if (rc == WR_HIP_OK)
        rc = wr_hip_mix_pool_create(mm->f32, mm->n_latent, mm->latent_dim, (uint32_t)pages, mm->n_state, mm->state_elems,
                                    slots, &mm->pool);
    if (rc == WR_HIP_OK) rc = wr_hip_mix_step_create((uint32_t)pages, &mm->step);
    if (rc != WR_HIP_OK) {
        wrh_logf(m->engine, 0, "session: cache pool of %u pages and %u slots could not be made (rc=%d)", (uint32_t)pages,
                slots, rc);
        wr_hip_mix_pool_destroy(mm->pool);
        mm->pool = NULL;
        free(mm->free_pages);
        free(mm->free_slots);
        mm->free_pages = mm->free_slots = NULL;
        return (wr_status)rc;
    }
    mm->n_pages = mm->n_free_pages = (uint32_t)pages;
    mm->n_slots = mm->n_free_slots = slots;
    /* taken from the end: the lowest numbers first */
    for (uint32_t i = 0; i < mm->n_pages; i++) mm->free_pages[i] = mm->n_pages - 1 - i;
    for (uint32_t i = 0; i < slots; i++) mm->free_slots[i] = slots - 1 - i;
    wrh_logf(m->engine, 2, "cache pool: %u pages of %u positions, %u state slots, %.1f MiB", mm->n_pages, WR_HIP_MIX_PAGE,
            slots, (double)wr_hip_mix_pool_bytes(mm->pool) / 1048576.0);
    return WR_OK;
}

wr_status wrh_mix_session_create(wr_model *m, wr_session *s)
{
    struct wrh_mix_model *mm = m->mix;
    wrh_mix_session *ms = calloc(1, sizeof *ms);
    if (!ms) return WR_ERR_NOMEM;
    ms->pages = malloc(((size_t)s->max_context + WR_HIP_MIX_PAGE - 1) / WR_HIP_MIX_PAGE * sizeof *ms->pages);
    if (!ms->pages) {
        free(ms);
        return WR_ERR_NOMEM;
    }
    pthread_mutex_lock(&mm->lock);
    wr_status st = pool_ready(m);
    if (st == WR_OK && mm->n_free_slots == 0) {
        wrh_logf(m->engine, 1, "session: all %u state slots are taken", mm->n_slots);
        st = WR_ERR_BUSY;
    }
    if (st == WR_OK) ms->slot = mm->free_slots[--mm->n_free_slots];
    pthread_mutex_unlock(&mm->lock);
    if (st != WR_OK) {
        free(ms->pages);
        free(ms);
        return st;
    }
    s->mix = ms;
    return WR_OK;
}

void wrh_mix_session_destroy(wr_session *s)
{
    struct wrh_mix_model *mm = s->model->mix;
    pthread_mutex_lock(&mm->lock);
    for (uint32_t i = s->mix->n_pages; i > 0; i--) mm->free_pages[mm->n_free_pages++] = s->mix->pages[i - 1];
    mm->free_slots[mm->n_free_slots++] = s->mix->slot;
    pthread_mutex_unlock(&mm->lock);
    free(s->mix->pages);
    free(s->mix);
    s->mix = NULL;
}

/* ---------------------------------------------------------------- scratch -- */

/* Bump allocation inside the scratch block; with a NULL block it only measures. */
typedef struct bump {
    uint8_t *base;
    size_t   at;
} bump;

static void *take(bump *b, size_t bytes)
{
    uint8_t *p = b->base ? b->base + b->at : NULL;
    b->at += (bytes + 255) & ~(size_t)255;
    return p;
}

/* Rows shared by every layer. */
typedef struct walk {
    float *x, *x0, *y;                     /* [R][width_p]: residual, embedding output, a sublayer's output */
    float *x_next;                         /* the residual's other buffer: a token shift moves it there */
    void  *h;                              /* frag: a sublayer's input */
    float *rope[WRH_MAX_LAYERS];           /* rotary tables (one per distinct rotation) */
} walk;

typedef struct lightning_rows {
    void  *qkvg;
    float *o;
    void  *oh;
} lightning_rows;

typedef struct latent_rows {
    float *d;
    void  *cq, *qu;
    float *qr;
    void  *q, *oc, *ov;
} latent_rows;

typedef struct wkv_rows {
    void  *mix, *low, *oh;
    float *in, *z;
} wkv_rows;

typedef struct parallel_rows {
    void  *low, *q, *oh;
    float *in, *z;
} parallel_rows;

typedef struct window_rows {
    float *in;
    void  *q, *oh;
} window_rows;

/* Where a joint layer's parts of the output product's input lie: buffers of their own with out_norm, else one. */
typedef struct joint_rows {
    float *in;
    void  *q, *attn, *beside, *act;
    uint32_t attn_kt, beside_kt, beside_col, act_kt, act_kt0;
    float *y_attn, *y_beside;
} joint_rows;

typedef struct moe_rows {
    float    *z, *gate, *side, *slot_weight, *ys, *shared;
    uint32_t *slot, *perm;
    int32_t  *group_expert;
    void     *xs, *act, *shared_act;
    uint32_t  groups, tile_groups;
} moe_rows;

/* R rounded up to whole fragment groups */
static size_t r16(size_t rows) { return (rows + 15) / 16 * 16; }

static walk take_walk(bump *b, const struct wrh_mix_model *mm, size_t R)
{
    walk w;
    memset(&w, 0, sizeof w);
    const size_t e = mm->f32 ? 4 : 2;
    w.x = take(b, R * mm->width_p * 4);
    w.x0 = mm->looped ? take(b, R * mm->width_p * 4) : NULL;
    w.x_next = mm->has_shift ? take(b, R * mm->width_p * 4) : NULL;
    w.y = take(b, R * mm->width_p * 4);
    w.h = take(b, r16(R) * mm->width_p * e);
    for (uint32_t i = 0; i < mm->n_ropes; i++) w.rope[i] = take(b, R * mm->ropes[i].dims * 4 + 4);
    return w;
}

static lightning_rows take_lightning(bump *b, const wrh_mix_layer *L, size_t R, size_t e)
{
    lightning_rows r;
    r.qkvg = take(b, r16(R) * (2 * L->qk_p + 2 * L->v_p) * e);
    r.o = take(b, R * L->v_p * 4);
    r.oh = take(b, r16(R) * L->v_p * e);
    return r;
}

static latent_rows take_latent(bump *b, const wrh_mix_layer *L, size_t R, size_t e)
{
    latent_rows r;
    const size_t H = L->heads;
    r.d = take(b, R * (L->q_rank_p + p32(L->kv_rank) + p32(L->rot_dim)) * 4);
    r.cq = take(b, r16(R) * L->q_rank_p * e);
    r.qu = take(b, r16(R) * H * L->dim_p * e);
    r.qr = take(b, R * p32(L->heads * L->rot_dim) * 4 + 4);
    r.q = take(b, r16(R) * H * (L->geo.rank_pad + L->geo.rot_pad) * e);
    r.oc = take(b, r16(R) * H * L->geo.rank_pad * e);
    r.ov = take(b, r16(R) * H * L->vdim_p * e);
    return r;
}

static wkv_rows take_wkv(bump *b, const struct wrh_mix_model *mm, const wrh_mix_layer *L, size_t R)
{
    wkv_rows r;
    const size_t e = mm->f32 ? 4 : 2;
    r.mix = take(b, r16(R) * 5 * mm->width_p * e);
    r.low = take(b, r16(R) * L->rec.rank_p * e);
    r.in = take(b, R * 4 * L->rec.hd_p * 4);
    r.z = take(b, R * L->rec.hd_p * 4);
    r.oh = take(b, r16(R) * L->rec.hd_p * e);
    return r;
}

/* Inputs of the layer's output product: the attention's heads, padded one by one, then the recurrence's. */
static uint32_t parallel_out(const wrh_mix_layer *L) { return L->heads * L->win.vdim_pad + L->rec.hd_p; }

static parallel_rows take_parallel(bump *b, const wrh_mix_layer *L, size_t R, size_t e)
{
    parallel_rows r;
    r.low = take(b, r16(R) * L->rec.rank_p * e);
    r.in = take(b, R * L->ld_in * 4);
    r.z = take(b, R * L->rec.hd_p * 4);
    r.q = take(b, r16(R) * L->heads * L->win.dim_pad * e);
    r.oh = take(b, r16(R) * parallel_out(L) * e);
    return r;
}

static window_rows take_window(bump *b, const wrh_mix_layer *L, size_t R, size_t e)
{
    window_rows r;
    r.in = take(b, R * L->ld_in * 4);
    r.q = take(b, r16(R) * L->heads * L->win.maps * L->win.dim_pad * e);
    r.oh = take(b, r16(R) * L->heads * L->win.vdim_pad * e);
    return r;
}

static uint32_t beside_out(const wrh_mix_layer *L)
{
    return L->beside == WRH_BESIDE_FORGET ? L->rec.hv_p : L->beside == WRH_BESIDE_GRU ? L->gru_p : 0;
}

static joint_rows take_joint(bump *b, const struct wrh_mix_model *mm, const wrh_mix_layer *L, size_t R)
{
    joint_rows r;
    memset(&r, 0, sizeof r);
    const size_t e = mm->f32 ? 4 : 2;
    const uint32_t heads = L->heads * L->win.vdim_pad, beside = beside_out(L), ff = L->mlp == WRH_MLP_DENSE ? L->ff_p : 0;
    r.in = take(b, R * L->ld_in * 4);
    r.q = take(b, r16(R) * L->heads * L->win.dim_pad * e);
    if (L->out_norm[0]) {
        r.attn = take(b, r16(R) * heads * e);
        r.beside = take(b, r16(R) * beside * e);
        r.act = take(b, r16(R) * ff * e);
        r.attn_kt = heads / 32;
        r.beside_kt = beside / 32;
        r.act_kt = ff / 32;
        r.y_attn = take(b, R * mm->width_p * 4);
        r.y_beside = take(b, R * mm->width_p * 4);
        return r;
    }
    r.attn = r.beside = r.act = take(b, r16(R) * (heads + beside + ff) * e);
    r.attn_kt = r.beside_kt = r.act_kt = (heads + beside + ff) / 32;
    r.beside_col = heads;
    r.act_kt0 = (heads + beside) / 32;
    return r;
}

/* Experts whose rows fill whole tiles take the prompt-sized product. */
static uint32_t moe_tile(const struct wrh_mix_model *mm, const wrh_mix_layer *L, size_t R)
{
    return (!mm->f32 && R * L->router.top >= (size_t)L->router.experts * 32) ? 8 : 1;
}

static moe_rows take_moe(bump *b, const struct wrh_mix_model *mm, const wrh_mix_layer *L, size_t R, uint32_t tile)
{
    moe_rows r;
    const size_t e = mm->f32 ? 4 : 2;
    r.tile_groups = tile;
    r.groups = wr_hip_mix_route_groups((uint32_t)R, L->router.experts, L->router.top, tile);
    const size_t slots = (size_t)r.groups * 16;
    r.z = take(b, R * L->router_p * 4);
    r.gate = take(b, R * L->router.top * 4);
    r.side = take(b, R * 2 * 4);
    r.slot = take(b, R * L->router.top * 4);
    r.perm = take(b, slots * 4);
    r.group_expert = take(b, (size_t)r.groups * 4);
    r.slot_weight = L->weigh_input ? take(b, slots * 4) : NULL;
    r.xs = take(b, slots * mm->width_p * e);
    r.act = take(b, slots * L->ff_p * e);
    r.ys = take(b, slots * mm->width_p * 4);
    r.shared_act = L->shared_p ? take(b, r16(R) * L->shared_p * e) : NULL;
    r.shared = L->shared_p ? take(b, R * mm->width_p * 4) : NULL;
    return r;
}

/* Bytes of scratch R rows need: what all layers share, and the most any layer needs beside it.
 * Everything grows with the rows, so what R rows need is enough for fewer. */
static size_t scratch_bytes(const struct wrh_mix_model *mm, size_t R)
{
    const size_t e = mm->f32 ? 4 : 2;
    bump all = {NULL, 0};
    (void)take_walk(&all, mm, R);
    size_t most = 0;
    for (uint32_t i = 0; i < mm->n_layers; i++) {
        const wrh_mix_layer *L = &mm->layers[i];
        bump b = {NULL, 0};
        switch (L->kind) {
        case WRH_MIXER_LIGHTNING: (void)take_lightning(&b, L, R, e); break;
        case WRH_MIXER_LATENT: (void)take_latent(&b, L, R, e); break;
        case WRH_MIXER_WKV: (void)take_wkv(&b, mm, L, R); break;
        case WRH_MIXER_PARALLEL: (void)take_parallel(&b, L, R, e); break;
        case WRH_MIXER_WINDOW: (void)take_window(&b, L, R, e); break;
        case WRH_MIXER_JOINT:
            (void)take_joint(&b, mm, L, R);
            if (L->mlp == WRH_MLP_MOE) (void)take_moe(&b, mm, L, R, 8);
            break;
        }
        if (b.at > most) most = b.at;
        if (L->kind == WRH_MIXER_JOINT) continue;
        bump f = {NULL, 0};
        if (L->mlp == WRH_MLP_DENSE) (void)take(&f, r16(R) * L->ff_p * e);
        if (L->mlp == WRH_MLP_MOE) (void)take_moe(&f, mm, L, R, 8);      /* the larger of the two forms */
        if (f.at > most) most = f.at;
    }
    return all.at + most;
}

static wr_status scratch_ready(wr_model *m, uint32_t rows)
{
    struct wrh_mix_model *mm = m->mix;
    if (!mm->logits_host) {
        const size_t bytes = (size_t)WRH_MIX_LOGIT_ROWS * mm->vocab_p * sizeof(float);
        if (!mm->logits_dev) mm->logits_dev = wr_hip_attn_dev_alloc(bytes);
        mm->logits_host = wr_hip_attn_host_alloc(bytes);
        if (!mm->logits_dev || !mm->logits_host) return WR_ERR_NOMEM;
    }
    if (rows <= mm->rows_cap) return WR_OK;
    uint32_t cap = 64;
    while (cap < rows) cap *= 2;
    wr_hip_attn_dev_free(mm->scratch);
    mm->rows_cap = 0;
    mm->scratch_bytes = scratch_bytes(mm, cap);
    mm->scratch = wr_hip_attn_dev_alloc(mm->scratch_bytes);
    if (!mm->scratch) return WR_ERR_NOMEM;
    mm->rows_cap = cap;
    return WR_OK;
}

static int g_poison;

void wrh_debug_poison_scratch(int on) { g_poison = on; }

static wr_status poison(struct wrh_mix_model *mm)
{
    if (!g_poison) return WR_OK;
    uint8_t *ff = malloc(mm->scratch_bytes);
    if (!ff) return WR_ERR_NOMEM;
    memset(ff, 0xFF, mm->scratch_bytes);
    const int rc = wr_hip_attn_h2d(mm->scratch, ff, mm->scratch_bytes);
    free(ff);
    return rc == WR_HIP_OK ? WR_OK : WR_ERR_INTERNAL;
}

/* ------------------------------------------------------------------- walk -- */

static wr_status op_fail(wr_model *m, const char *what, uint32_t run, int rc)
{
    wrh_logf(m->engine, 0, "session: %s failed at layer run %u (rc=%d)", what, run, rc);
    return (rc < 0) ? (wr_status)rc : WR_ERR_INTERNAL;
}

#define TRY(call, what)                                        \
    do {                                                       \
        const int rc_ = (call);                                \
        if (rc_ != WR_HIP_OK) return op_fail(m, what, r, rc_); \
    } while (0)

static wr_status walk_lightning(wr_model *m, const wrh_mix_layer *L, uint32_t r, const walk *w, bump b, uint32_t R)
{
    struct wrh_mix_model *mm = m->mix;
    const lightning_rows t = take_lightning(&b, L, R, mm->f32 ? 4 : 2);
    const uint32_t ld = 2 * L->qk_p + 2 * L->v_p, col_g = 2 * L->qk_p + L->v_p;
    const wr_hip_mix_gemm in = {.w = L->w_qkvg, .x = w->h, .x_kt = mm->width_p / 32, .rows = R, .out = WR_HIP_MIX_OUT_ROWS,
                                .y_act = t.qkvg, .ldy = ld, .silu_end = col_g, .sigmoid_end = ld};
    TRY(wr_hip_mix_gemm_run(mm->f32, &in), "q/k/v/gate projection");
    TRY(wr_hip_mix_lightning(mm->step, mm->pool, mm->runs[r].store, mm->f32, L->heads, L->dim, L->vdim, L->decay, t.qkvg,
                             ld, L->qk_p, 2 * L->qk_p, t.o, L->v_p), "linear attention");
    const uint8_t *g = (const uint8_t *)t.qkvg + (size_t)col_g * (mm->f32 ? 4 : 2);
    TRY(wr_hip_mix_gate_norm(mm->step, mm->f32, t.o, L->v_p, L->heads * L->vdim, g, ld, L->mix_norm, mm->eps, t.oh),
        "gated norm");
    const wr_hip_mix_gemm out = {.w = L->w_o, .x = t.oh, .x_kt = L->v_p / 32, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                 .y_f32 = w->y, .ldy = mm->width_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &out), "output projection");
    return WR_OK;
}

static wr_status walk_latent(wr_model *m, const wrh_mix_layer *L, uint32_t r, const walk *w, bump b, uint32_t R)
{
    struct wrh_mix_model *mm = m->mix;
    const latent_rows t = take_latent(&b, L, R, mm->f32 ? 4 : 2);
    const wr_hip_mix_latent *g = &L->geo;
    const uint32_t H = L->heads, ldd = L->q_rank_p + p32(L->kv_rank) + p32(L->rot_dim), ldq = p32(H * L->rot_dim);
    const uint32_t kd = (g->rank_pad + g->rot_pad) / 32, store = mm->runs[r].store;
    const wr_hip_mix_gemm down = {.w = L->w_d, .x = w->h, .x_kt = mm->width_p / 32, .rows = R,
                                  .out = WR_HIP_MIX_OUT_ROWS_F32, .y_f32 = t.d, .ldy = ldd};
    TRY(wr_hip_mix_gemm_run(mm->f32, &down), "latent projections");
    TRY(wr_hip_mix_latent_append(mm->step, mm->pool, store, mm->f32, g, t.d, ldd, L->q_rank, L->dq_norm, L->dkv_norm,
                                 mm->eps, w->rope[L->rope], t.cq), "latent norms + cache append");
    const wr_hip_mix_gemm uq = {.w = L->w_uq, .x = t.cq, .x_kt = L->q_rank_p / 32, .rows = R, .out = WR_HIP_MIX_OUT_SPLIT,
                                .h = t.qu, .h_kt = H * L->dim_p / 32, .n_split = H * L->dim_p,
                                .y_f32 = t.qr, .ldy = ldq};
    TRY(wr_hip_mix_gemm_run(mm->f32, &uq), "query projection");
    const wr_hip_mix_gemm uk = {.w = L->w_uk, .x = t.qu, .x_kt = H * L->dim_p / 32, .x_kt_z = L->dim_p / 32, .rows = R,
                                .out = WR_HIP_MIX_OUT_FRAG, .h = t.q, .h_kt = H * kd, .col_z = kd * 32};
    TRY(wr_hip_mix_gemm_run(mm->f32, &uk), "queries into the latent");
    TRY(wr_hip_mix_latent_qrope(mm->step, mm->f32, g, t.qr, ldq, w->rope[L->rope], t.q), "query rotation");
    TRY(wr_hip_mix_latent_attend(mm->step, mm->pool, store, mm->f32, g, t.q, t.oc), "latent attention");
    const wr_hip_mix_gemm uv = {.w = L->w_uv, .x = t.oc, .x_kt = H * g->rank_pad / 32, .x_kt_z = g->rank_pad / 32, .rows = R,
                                .out = WR_HIP_MIX_OUT_FRAG, .h = t.ov, .h_kt = H * L->vdim_p / 32,
                                .col_z = L->vdim_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &uv), "values out of the latent");
    const wr_hip_mix_gemm out = {.w = L->w_o, .x = t.ov, .x_kt = H * L->vdim_p / 32, .rows = R,
                                 .out = WR_HIP_MIX_OUT_ROWS_F32, .y_f32 = w->y, .ldy = mm->width_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &out), "output projection");
    return WR_OK;
}

/* The recurrence, the decay's second product included; `rec` has the rest filled in. */
static wr_status walk_recur(wr_model *m, const wrh_mix_recur *q, uint32_t r, uint32_t store, const void *low, float *z,
                            wr_hip_mix_recurrence *rec)
{
    struct wrh_mix_model *mm = m->mix;
    rec->heads = q->heads;
    rec->dim = q->dim;
    rec->eps = mm->eps;
    rec->w0 = q->w0;
    rec->norm = q->norm;
    rec->w_decay = q->w_decay;
    rec->low = low;
    rec->z = z;
    TRY(wr_hip_mix_recur(mm->step, mm->pool, store, mm->f32, rec), "matrix-state recurrence");
    return WR_OK;
}

/* Takes the residual from w->x and the sublayer output `y` waiting to join it (or NULL) to w->x_next. */
static wr_status walk_wkv(wr_model *m, const wrh_mix_layer *L, uint32_t r, walk *w, bump b, uint32_t R, const float *y)
{
    struct wrh_mix_model *mm = m->mix;
    const wkv_rows t = take_wkv(&b, mm, L, R);
    const wrh_mix_recur *q = &L->rec;
    const uint32_t wkt = mm->width_p / 32, hd = q->hd_p;
    TRY(wr_hip_mix_shift(mm->step, mm->pool, mm->runs[r].store2, mm->f32, mm->width, mm->eps, w->x, y, w->x_next, L->norm1, 5,
                         L->mu, t.mix), "token shift");
    if (y) {
        float *x = w->x;
        w->x = w->x_next;
        w->x_next = x;
    }
    const wr_hip_mix_gemm in = {.w = L->w_rkvg, .x = t.mix, .x_kt = 5 * wkt, .x_kt_z = wkt, .rows = R,
                                .out = WR_HIP_MIX_OUT_ROWS_F32, .y_f32 = t.in, .ldy = 4 * hd, .col_z = hd};
    TRY(wr_hip_mix_gemm_run(mm->f32, &in), "r/k/v/gate projection");
    const wr_hip_mix_gemm low = {.w = L->w_low, .x = t.mix, .x_kt = 5 * wkt, .x_kt0 = 4 * wkt, .rows = R, .out = WR_HIP_MIX_OUT_FRAG,
                                 .h = t.low, .h_kt = q->rank_p / 32, .tanh_end = q->rank_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &low), "decay's low-rank product");
    wr_hip_mix_recurrence rec = {.rule = WR_HIP_MIX_RULE_BONUS, .out_scale = 1.0f, .gate_silu = 1, .u = q->u, .in = t.in,
                                 .ld = 4 * hd, .col_k = hd, .col_v = 2 * hd, .col_g = 3 * hd, .h = t.oh, .h_kt = hd / 32};
    const wr_status st = walk_recur(m, q, r, mm->runs[r].store, t.low, t.z, &rec);
    if (st != WR_OK) return st;
    const wr_hip_mix_gemm out = {.w = L->w_o, .x = t.oh, .x_kt = hd / 32, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                 .y_f32 = w->y, .ldy = mm->width_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &out), "output projection");
    return WR_OK;
}

static wr_status walk_parallel(wr_model *m, const wrh_mix_layer *L, uint32_t r, const walk *w, bump b, uint32_t R)
{
    struct wrh_mix_model *mm = m->mix;
    const parallel_rows t = take_parallel(&b, L, R, mm->f32 ? 4 : 2);
    const wrh_mix_recur *q = &L->rec;
    const uint32_t kt_o = parallel_out(L) / 32, store = mm->runs[r].store;
    const wr_hip_mix_gemm in = {.w = L->w_in, .x = w->h, .x_kt = mm->width_p / 32, .rows = R, .out = WR_HIP_MIX_OUT_SPLIT,
                                .h = t.low, .h_kt = q->rank_p / 32, .n_split = q->rank_p, .tanh_end = q->rank_p,
                                .y_f32 = t.in, .ldy = L->ld_in};
    TRY(wr_hip_mix_gemm_run(mm->f32, &in), "both halves' projections");
    TRY(wr_hip_mix_window_append(mm->step, mm->pool, store, mm->f32, &L->win, t.in, L->ld_in, L->col_q, L->col_k, L->col_v,
                                 w->rope[L->rope], t.q), "rotation + cache append");
    TRY(wr_hip_mix_window_attend(mm->step, mm->pool, store, mm->f32, &L->win, t.q, L->sink, NULL, 0, t.oh, kt_o),
        "windowed attention");
    wr_hip_mix_recurrence rec = {.rule = WR_HIP_MIX_RULE_DELTA, .gain = WRH_DELTA_GAIN, .unit_eps = WRH_DELTA_UNIT_EPS,
                                 .out_scale = L->right_scale, .a_bias = q->a_bias, .in = t.in, .ld = L->ld_in,
                                 .col_r = L->col_rr, .col_k = L->col_rk, .col_v = L->col_rv, .col_a = L->col_ra,
                                 .col_g = L->col_rg, .h = t.oh, .h_kt = kt_o, .col_h = L->heads * L->win.vdim_pad};
    const wr_status st = walk_recur(m, q, r, mm->runs[r].store2, t.low, t.z, &rec);
    if (st != WR_OK) return st;
    const wr_hip_mix_gemm out = {.w = L->w_o, .x = t.oh, .x_kt = kt_o, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                 .y_f32 = w->y, .ldy = mm->width_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &out), "output projection");
    return WR_OK;
}

static wr_status walk_window(wr_model *m, const wrh_mix_layer *L, uint32_t r, const walk *w, bump b, uint32_t R)
{
    struct wrh_mix_model *mm = m->mix;
    const window_rows t = take_window(&b, L, R, mm->f32 ? 4 : 2);
    const uint32_t kt_o = L->heads * L->win.vdim_pad / 32, store = mm->runs[r].store;
    const wr_hip_mix_gemm in = {.w = L->w_in, .x = w->h, .x_kt = mm->width_p / 32, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                .y_f32 = t.in, .ldy = L->ld_in, .bias = L->b_in};
    TRY(wr_hip_mix_gemm_run(mm->f32, &in), "q/k/v projection");
    TRY(wr_hip_mix_window_append(mm->step, mm->pool, store, mm->f32, &L->win, t.in, L->ld_in, L->col_q, L->col_k, L->col_v,
                                 w->rope[L->rope], t.q), "rotation + cache append");
    TRY(wr_hip_mix_window_attend(mm->step, mm->pool, store, mm->f32, &L->win, t.q, L->sink, L->has_gate ? t.in + L->col_rg : NULL,
                                 L->ld_in, t.oh, kt_o), "windowed attention");
    const wr_hip_mix_gemm out = {.w = L->w_o, .x = t.oh, .x_kt = kt_o, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                 .y_f32 = w->y, .ldy = mm->width_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &out), "output projection");
    return WR_OK;
}

/* The experts: the router's logits `z` (row stride ldz) to expert rows that `res` is told to combine. */
static wr_status walk_experts(wr_model *m, const wrh_mix_layer *L, uint32_t r, const walk *w, const moe_rows *t, const float *z,
                              uint32_t ldz, wr_hip_mix_resid *res)
{
    struct wrh_mix_model *mm = m->mix;
    const uint32_t wkt = mm->width_p / 32;
    TRY(wr_hip_mix_route(mm->step, z, ldz, &L->router, t->tile_groups, t->gate, t->side, t->slot_weight, t->slot, t->perm,
                         t->group_expert), "routing");
    wr_hip_mix_gemm up = {.w = L->w_eup, .x = t->xs, .x_kt = wkt, .rows = t->groups * 16, .group_expert = t->group_expert,
                          .tile_groups = t->tile_groups, .out = WR_HIP_MIX_OUT_FRAG, .h = t->act, .h_kt = L->ff_p / 32,
                          .x_scale = t->slot_weight};
    if (t->tile_groups == 1) {                             /* few rows: the product fetches them where they are */
        up.x = w->h;
        up.x_perm = t->perm;
    } else {
        TRY(wr_hip_mix_route_gather(mm->step, mm->f32, w->h, wkt, t->groups, t->perm, t->group_expert, t->xs), "expert rows");
    }
    if (L->gated || L->limit > 0) up.out = WR_HIP_MIX_OUT_GATED;
    else up.relu2 = 1;
    if (L->limit > 0) {
        up.limit = L->limit;
        up.slope = WRH_CLAMPED_SLOPE;
        up.up_bias = WRH_CLAMPED_UP_BIAS;
    }
    TRY(wr_hip_mix_gemm_run(mm->f32, &up), "experts' up projection");
    const wr_hip_mix_gemm down = {.w = L->w_edown, .x = t->act, .x_kt = L->ff_p / 32, .rows = t->groups * 16,
                                  .group_expert = t->group_expert, .tile_groups = t->tile_groups,
                                  .out = WR_HIP_MIX_OUT_ROWS_F32, .y_f32 = t->ys, .ldy = mm->width_p};
    TRY(wr_hip_mix_gemm_run(mm->f32, &down), "experts' down projection");
    res->y = t->ys;
    res->gate = L->weigh_input ? NULL : t->gate;
    res->slot = t->slot;
    res->top = L->router.top;
    return WR_OK;
}

/* A whole joint layer: mixers and feed-forward from the rows in w->h; `res` is told what joins the residual. */
static wr_status walk_joint(wr_model *m, const wrh_mix_layer *L, uint32_t r, const walk *w, bump b, uint32_t R, wr_hip_mix_resid *res)
{
    struct wrh_mix_model *mm = m->mix;
    const joint_rows t = take_joint(&b, mm, L, R);
    const uint32_t store = mm->runs[r].store, store2 = mm->runs[r].store2;
    const int dense = L->mlp == WRH_MLP_DENSE, apart = L->out_norm[0] != NULL;
    wr_hip_mix_gemm in = {.w = L->w_in, .x = w->h, .x_kt = mm->width_p / 32, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                          .y_f32 = t.in, .ldy = L->ld_in, .bias = L->b_in, .silu_end = L->silu_end};
    if (dense) {
        in.out = WR_HIP_MIX_OUT_SPLIT_GATED;
        in.n_split = L->n_in;
        in.h = t.act;
        in.h_kt = t.act_kt;
        in.h_kt0 = t.act_kt0;
        in.limit = L->limit;
        in.slope = WRH_CLAMPED_SLOPE;
        in.up_bias = WRH_CLAMPED_UP_BIAS;
    }
    TRY(wr_hip_mix_gemm_run(mm->f32, &in), "layer's input projections");
    wr_hip_mix_window g = L->win;
    g.turn_values = L->turn >= 0 ? w->rope[L->turn] : NULL;
    TRY(wr_hip_mix_window_append(mm->step, mm->pool, store, mm->f32, &g, t.in, L->ld_in, L->col_q, L->col_k, L->col_v,
                                 w->rope[L->rope], t.q), "rotation + cache append");
    TRY(wr_hip_mix_window_attend(mm->step, mm->pool, store, mm->f32, &g, t.q, L->sink, L->has_gate ? t.in + L->col_rg : NULL,
                                 L->ld_in, t.attn, t.attn_kt), "attention");
    if (L->beside == WRH_BESIDE_FORGET) {
        const wr_hip_mix_recurrence rec = {.heads = L->rec.heads, .dim = L->rec.dim, .vdim = L->rec.vdim,
                                           .rule = WR_HIP_MIX_RULE_FORGET, .eps = mm->eps, .out_scale = L->right_scale,
                                           .w0 = L->rec.w0, .lower = L->rec.lower, .norm = L->rec.norm, .in = t.in,
                                           .ld = L->ld_in, .col_r = L->col_rr, .col_k = L->col_rk, .col_v = L->col_rv,
                                           .h = t.beside, .h_kt = t.beside_kt, .col_h = t.beside_col};
        TRY(wr_hip_mix_recur(mm->step, mm->pool, store2, mm->f32, &rec), "matrix-state recurrence");
    } else if (L->beside == WRH_BESIDE_GRU) {
        const wr_hip_mix_gru gru = {.width = L->gru, .in = t.in, .ld = L->ld_in, .col_z = L->col_rr, .col_x = L->col_rk,
                                    .col_g = L->col_rv, .h = t.beside, .h_kt = t.beside_kt, .col_h = t.beside_col};
        TRY(wr_hip_mix_min_gru(mm->step, mm->pool, store2, mm->f32, &gru), "gated recurrence");
    }
    wr_hip_mix_gemm out = {.w = L->w_o, .x = t.attn, .x_kt = t.attn_kt, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                           .y_f32 = apart ? t.y_attn : w->y, .ldy = mm->width_p, .bias = L->b_o};
    TRY(wr_hip_mix_gemm_run(mm->f32, &out), "output projection");
    if (apart) {
        out = (wr_hip_mix_gemm){.w = L->w_o2, .x = t.beside, .x_kt = t.beside_kt, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                .y_f32 = t.y_beside, .ldy = mm->width_p};
        TRY(wr_hip_mix_gemm_run(mm->f32, &out), "second output projection");
        res->pair_y[0] = t.y_attn;
        res->pair_y[1] = t.y_beside;
        for (int k = 0; k < 2; k++) res->pair_post[k] = L->out_norm[k];
        if (dense) {
            out = (wr_hip_mix_gemm){.w = L->w_down, .x = t.act, .x_kt = t.act_kt, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                    .y_f32 = w->y, .ldy = mm->width_p};
            TRY(wr_hip_mix_gemm_run(mm->f32, &out), "down projection");
        }
    }
    if (dense || !apart) res->y = w->y;
    if (L->mlp == WRH_MLP_MOE) {
        const moe_rows x = take_moe(&b, mm, L, R, moe_tile(mm, L, R));
        res->add = res->y;
        return walk_experts(m, L, r, w, &x, t.in + L->col_router, L->ld_in, res);
    }
    return WR_OK;
}

/* The feed-forward's output: plain rows in w->y, or expert rows that `res` is told to combine. */
static wr_status walk_mlp(wr_model *m, const wrh_mix_layer *L, uint32_t r, const walk *w, bump b, uint32_t R,
                          wr_hip_mix_resid *res)
{
    struct wrh_mix_model *mm = m->mix;
    const uint32_t wkt = mm->width_p / 32;
    if (L->mlp == WRH_MLP_DENSE) {
        void *act = take(&b, r16(R) * L->ff_p * (mm->f32 ? 4 : 2));
        const wr_hip_mix_gemm gu = {.w = L->w_gu, .x = w->h, .x_kt = wkt, .rows = R, .out = WR_HIP_MIX_OUT_GATED, .h = act,
                                    .h_kt = L->ff_p / 32, .gelu = L->gelu};
        TRY(wr_hip_mix_gemm_run(mm->f32, &gu), "gate/up projection");
        const wr_hip_mix_gemm down = {.w = L->w_down, .x = act, .x_kt = L->ff_p / 32, .rows = R,
                                      .out = WR_HIP_MIX_OUT_ROWS_F32, .y_f32 = w->y, .ldy = mm->width_p};
        TRY(wr_hip_mix_gemm_run(mm->f32, &down), "down projection");
        res->y = w->y;
        return WR_OK;
    }
    const moe_rows t = take_moe(&b, mm, L, R, moe_tile(mm, L, R));
    wr_hip_mix_gemm router = {.w = L->w_router, .x = w->h, .x_kt = wkt, .rows = R, .out = WR_HIP_MIX_OUT_ROWS_F32,
                              .y_f32 = t.z, .ldy = L->router_p};
    if (L->shared_p) {                                     /* the shared expert's gate and up ride along */
        router.out = WR_HIP_MIX_OUT_SPLIT_GATED;
        router.n_split = L->router_p;
        router.h = t.shared_act;
        router.h_kt = L->shared_p / 32;
        router.limit = L->shared_limit;
        router.slope = WRH_CLAMPED_SLOPE;
        router.up_bias = WRH_CLAMPED_UP_BIAS;
    }
    TRY(wr_hip_mix_gemm_run(mm->f32, &router), "router");
    const wr_status st = walk_experts(m, L, r, w, &t, t.z, L->router_p, res);
    if (st != WR_OK) return st;
    if (L->shared_p) {
        const wr_hip_mix_gemm sh = {.w = L->w_down, .x = t.shared_act, .x_kt = L->shared_p / 32, .rows = R,
                                    .out = WR_HIP_MIX_OUT_ROWS_F32, .y_f32 = t.shared, .ldy = mm->width_p};
        TRY(wr_hip_mix_gemm_run(mm->f32, &sh), "shared expert's down projection");
    }
    if (L->router.identity || L->shared_p) {
        res->side = t.side;
        res->ident = L->router.identity ? w->h : NULL;
        res->shared = t.shared;
    }
    return WR_OK;
}
static wr_status capture(struct wrh_mix_model *mm, const walk *w, uint32_t R)
{
    const size_t n = (size_t)R * mm->width;
    if (!mm->capture || n > mm->capture_left) return WR_OK;
    for (uint32_t i = 0; i < R; i++)
        if (wr_hip_attn_d2h(mm->capture + (size_t)i * mm->width, w->x + (size_t)i * mm->width_p, mm->width * sizeof(float)))
            return WR_ERR_INTERNAL;
    mm->capture += n;
    mm->capture_left -= n;
    return WR_OK;
}

/* All layers over the rows of mm->step; the residual ends up in w->x. */
static wr_status walk_layers(wr_model *m, walk *w, bump b, uint32_t R, int fail_run)
{
    struct wrh_mix_model *mm = m->mix;
    uint32_t r = 0;
    for (uint32_t i = 0; i < mm->n_ropes; i++)
        if (mm->ropes[i].dims)
            TRY(wr_hip_mix_rope_table(mm->step, mm->ropes[i].freq_dev, mm->ropes[i].dims / 2, mm->ropes[i].gain, w->rope[i]),
                "angles");
    const wrh_mix_layer *next = &mm->layers[mm->runs[0].layer];
    /* a layer behind a token shift makes its input from the residual itself */
    TRY(wr_hip_mix_embed(mm->step, mm->f32, mm->embed_dev, mm->width, mm->embed_norm, mm->embed_scale, mm->eps, w->x, w->x0,
                         next->kind == WRH_MIXER_WKV ? NULL : next->norm1, w->h), "embedding");
    const float *y = NULL;                                 /* a sublayer's output that waits for a token shift */
    for (r = 0; r < mm->n_runs; r++) {
        const wrh_mix_layer *L = next;
        next = r + 1 < mm->n_runs ? &mm->layers[mm->runs[r + 1].layer] : NULL;
        if (fail_run == (int)r) return op_fail(m, "mixer (injected)", r, WR_ERR_INTERNAL);
        wr_status st = WR_ERR_INTERNAL;
        wr_hip_mix_resid res = {.width = mm->width, .eps = mm->eps};
        switch (L->kind) {
        case WRH_MIXER_LIGHTNING: st = walk_lightning(m, L, r, w, b, R); break;
        case WRH_MIXER_LATENT: st = walk_latent(m, L, r, w, b, R); break;
        case WRH_MIXER_WKV: st = walk_wkv(m, L, r, w, b, R, y); break;
        case WRH_MIXER_PARALLEL: st = walk_parallel(m, L, r, w, b, R); break;
        case WRH_MIXER_WINDOW: st = walk_window(m, L, r, w, b, R); break;
        case WRH_MIXER_JOINT: st = walk_joint(m, L, r, w, b, R, &res); break;
        }
        if (st != WR_OK) return st;
        y = NULL;
        res.x = w->x;
        if (L->kind != WRH_MIXER_JOINT) {
            res.y = w->y;
            res.post = L->norm1b;
        }
        if (L->kind != WRH_MIXER_JOINT && L->mlp != WRH_MLP_NONE) {
            /* the mixer's output joins the residual and the feed-forward's input is made */
            res.next = L->norm2;
            res.h = w->h;
            TRY(wr_hip_mix_residual(mm->step, mm->f32, &res), "post-mixer norm + residual");
            res = (wr_hip_mix_resid){.width = mm->width, .eps = mm->eps, .x = w->x, .post = L->norm2b};
            st = walk_mlp(m, L, r, w, b, R, &res);
            if (st != WR_OK) return st;
        }
        /* the layer's output joins the residual and the next layer's input is made */
        if (mm->capture) {
            TRY(wr_hip_mix_residual(mm->step, mm->f32, &res), "post-norm + residual");
            st = capture(mm, w, R);
            if (st != WR_OK) return st;
            res = (wr_hip_mix_resid){.width = mm->width, .eps = mm->eps, .x = w->x};
        }
        if (next) {
            if (mm->runs[r + 1].add_embedding) {
                if (res.add) {                             /* the layer's outputs first */
                    TRY(wr_hip_mix_residual(mm->step, mm->f32, &res), "post-norm + residual");
                    res = (wr_hip_mix_resid){.width = mm->width, .eps = mm->eps, .x = w->x};
                }
                res.add = w->x0;
            }
            if (next->kind != WRH_MIXER_WKV) {
                res.next = next->norm1;
                res.h = w->h;
            } else if (res.y && !res.post && !res.top && !res.add && !res.pair_y[0]) {
                y = res.y;                                 /* the token shift adds it */
                res.y = NULL;
            }
        }
        if (res.y || res.add || res.pair_y[0] || res.next) TRY(wr_hip_mix_residual(mm->step, mm->f32, &res), "post-norm + residual");
    }
    return WR_OK;
}

/* Logits of the step's wanted rows, packed in h's rows after the final norm;
 * row i goes to logits + dest[i] * vocab. */
static wr_status walk_logits(wr_model *m, const walk *w, uint32_t n_want, const uint32_t *dest, float *logits)
{
    struct wrh_mix_model *mm = m->mix;
    const uint32_t r = mm->n_runs, wkt = mm->width_p / 32;
    const size_t e = mm->f32 ? 4 : 2;
    const wr_hip_mix_resid fin = {.width = mm->width, .eps = mm->eps, .x = w->x, .next = mm->final_norm, .wanted = 1, .h = w->h};
    TRY(wr_hip_mix_residual(mm->step, mm->f32, &fin), "final norm");
    for (uint32_t at = 0; at < n_want; at += WRH_MIX_LOGIT_ROWS) {
        const uint32_t n = n_want - at < WRH_MIX_LOGIT_ROWS ? n_want - at : WRH_MIX_LOGIT_ROWS;
        const uint8_t *x = (const uint8_t *)w->h + (size_t)at * mm->width_p * e;      /* whole groups of 16 rows */
        const wr_hip_mix_gemm head = {.w = mm->head, .x = x, .x_kt = wkt, .rows = n, .out = WR_HIP_MIX_OUT_ROWS_F32,
                                      .y_f32 = mm->logits_dev, .ldy = mm->vocab_p, .scale = mm->logit_scale};
        TRY(wr_hip_mix_gemm_run(mm->f32, &head), "head");
        TRY(wr_hip_attn_d2h(mm->logits_host, mm->logits_dev, (size_t)n * mm->vocab_p * sizeof(float)), "logits down");
        for (uint32_t i = 0; i < n; i++)
            memcpy(logits + (size_t)dest[at + i] * m->vocab, mm->logits_host + (size_t)i * mm->vocab_p,
                   (size_t)m->vocab * sizeof(float));
    }
    return WR_OK;
}

void wrh_debug_capture_residual(wr_model *m, float *rows, size_t floats)
{
    if (!m || !m->mix) return;
    pthread_mutex_lock(&m->mix->lock);
    m->mix->capture = rows;
    m->mix->capture_left = rows ? floats : 0;
    pthread_mutex_unlock(&m->mix->lock);
}

/* ------------------------------------------------------------------- step -- */

/* Pages for `tokens` positions; what was taken is noted so that it can be undone. */
static wr_status grow_pages(wr_model *m, wrh_mix_session *ms, uint32_t tokens)
{
    struct wrh_mix_model *mm = m->mix;
    const uint32_t need = (tokens + WR_HIP_MIX_PAGE - 1) / WR_HIP_MIX_PAGE;
    while (ms->n_pages < need) {
        if (mm->n_free_pages == 0) {
            wrh_logf(m->engine, 1, "session: the cache pool's %u pages are all taken", mm->n_pages);
            return WR_ERR_BUSY;
        }
        ms->pages[ms->n_pages++] = mm->free_pages[--mm->n_free_pages];
    }
    return WR_OK;
}

static void shrink_pages(struct wrh_mix_model *mm, wrh_mix_session *ms, uint32_t n_pages)
{
    while (ms->n_pages > n_pages) mm->free_pages[mm->n_free_pages++] = ms->pages[--ms->n_pages];
}

wr_status wrh_mix_step(wr_model *m, const wr_step_entry *entries, uint32_t n, float *logits, int fail_run)
{
    struct wrh_mix_model *mm = m->mix;
    uint32_t done[WR_BATCH_MAX] = {0}, pages_before[WR_BATCH_MAX], longest = 0;
    uint64_t total = 0;
    for (uint32_t i = 0; i < n; i++) {
        const wr_step_entry *q = &entries[i];
        if ((uint64_t)q->session->pos + q->n_tokens > q->session->max_context) return WR_ERR_CTX_FULL;
        for (uint32_t k = 0; k < q->n_tokens; k++)
            if (q->tokens[k] >= m->vocab) return WR_ERR_INVAL;
        for (uint32_t k = 0; k < q->n_want; k++)
            if (q->want[k] >= q->n_tokens) return WR_ERR_INVAL;
        total += q->n_tokens;
    }
    longest = total < WR_HIP_MIX_MAX_ROWS ? (uint32_t)total : WR_HIP_MIX_MAX_ROWS;

    pthread_mutex_lock(&mm->lock);
    for (uint32_t i = 0; i < n; i++) pages_before[i] = entries[i].session->mix->n_pages;
    wr_status st = scratch_ready(m, longest);
    for (uint32_t i = 0; i < n && st == WR_OK; i++)
        st = grow_pages(m, entries[i].session->mix, entries[i].session->pos + entries[i].n_tokens);
    uint32_t *tokens = malloc(((size_t)3 * longest + 1) * sizeof *tokens);
    if (!tokens && st == WR_OK) st = WR_ERR_NOMEM;
    uint32_t *want = tokens ? tokens + longest : NULL, *dest = tokens ? want + longest : NULL;

    uint64_t left = total;
    while (left && st == WR_OK) {
        /* the rows of this pass: as much of each entry as fits, in order */
        wr_hip_mix_seq seqs[WR_BATCH_MAX];
        uint32_t at[WR_BATCH_MAX], n_seq = 0, R = 0, row0 = 0, n_want = 0;
        for (uint32_t i = 0; i < n && R < longest; i++) {
            const wr_step_entry *q = &entries[i];
            wrh_mix_session *ms = q->session->mix;
            uint32_t take_rows = q->n_tokens - done[i];
            if (take_rows == 0) continue;
            if (take_rows > longest - R) take_rows = longest - R;
            memcpy(tokens + R, q->tokens + done[i], (size_t)take_rows * sizeof *tokens);
            /* the call's first pass reads the current buffer; later ones go on in the new one */
            seqs[n_seq] = (wr_hip_mix_seq){take_rows, q->session->pos + done[i], ms->slot,
                                           done[i] ? ms->buf ^ 1u : ms->buf, ms->buf ^ 1u, ms->n_pages, ms->pages};
            at[n_seq++] = i;
            R += take_rows;
        }
        uint32_t base = 0, s = 0;
        int more_than_fit = 0;
        for (uint32_t i = 0; i < n; i++) {
            if (s < n_seq && at[s] == i) {
                for (uint32_t k = 0; k < entries[i].n_want; k++) {
                    const uint32_t p = entries[i].want[k];
                    if (p < done[i] || p >= done[i] + seqs[s].rows) continue;
                    if (n_want == longest) {                   /* the same places asked for again and again */
                        more_than_fit = 1;
                        break;
                    }
                    want[n_want] = row0 + p - done[i];
                    dest[n_want++] = base + k;
                }
                row0 += seqs[s++].rows;
            }
            base += entries[i].n_want;
        }
        if (more_than_fit || n_want > R) {
            st = WR_ERR_LIMIT;
            break;
        }
        if ((st = poison(mm)) != WR_OK) break;
        const int rc = wr_hip_mix_step_set(mm->step, mm->pool, n_seq, seqs, tokens, m->vocab, n_want, want);
        if (rc != WR_HIP_OK) {
            st = op_fail(m, "step", 0, rc);
            break;
        }
        bump b = {mm->scratch, 0};
        walk w = take_walk(&b, mm, R);
        st = walk_layers(m, &w, b, R, fail_run);
        if (st == WR_OK && n_want) st = walk_logits(m, &w, n_want, dest, logits);
        /* the step's descriptors are in page-locked memory: they are free again after the wait */
        const int sync = wr_hip_attn_sync();
        if (st == WR_OK && sync != WR_HIP_OK) st = op_fail(m, "sync", mm->n_runs, sync);
        for (s = 0; s < n_seq; s++) done[at[s]] += seqs[s].rows;
        left -= R;
    }
    free(tokens);
    for (uint32_t i = 0; i < n; i++) {
        wr_session *ss = entries[i].session;
        if (st == WR_OK) {
            ss->mix->buf ^= 1u;
            __atomic_store_n(&ss->pos, ss->pos + entries[i].n_tokens, __ATOMIC_RELEASE);
        } else {
            shrink_pages(mm, ss->mix, pages_before[i]);
        }
    }
    pthread_mutex_unlock(&mm->lock);
    return st;
}
