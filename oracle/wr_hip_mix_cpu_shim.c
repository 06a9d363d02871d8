/*
 * wr_hip_mix_cpu_shim.c — TEST DOUBLE of the device steps of mixer-stack models
 * (include/wr_hip_mix.h).  TEST INFRASTRUCTURE, never shipped: with it the host
 * engine's own logic for these models (reading and rearranging weights, the cache
 * pool, passes, rollback, the mixed step) runs on a machine without a GPU.  Plain
 * loops, 32-bit activations only (f32 = 1); a "frag" buffer is row-major here.
 */
#include <math.h>
#include <stdlib.h>
#include <string.h>

#include "../include/wr_hip_attn.h"
#include "../include/wr_hip_mix.h"

struct wr_hip_mat { uint32_t batch, n_out, n_in; float *w; };
struct wr_hip_mix_pool {
    uint32_t n_pages, n_slots, n_latent, n_state;
    uint32_t *latent_dim;
    uint64_t *state_elems;
    float **latent, **state;
};
struct wr_hip_mix_step {
    uint32_t max_pages, rows, n_seq, n_want;
    uint32_t tokens[WR_HIP_MIX_MAX_ROWS], seq[WR_HIP_MIX_MAX_ROWS], pos[WR_HIP_MIX_MAX_ROWS], want[WR_HIP_MIX_MAX_ROWS];
    wr_hip_mix_seq seqs[WR_HIP_MIX_MAX_SEQS];
    uint32_t row0[WR_HIP_MIX_MAX_SEQS];
};

static int g_late;
/* Test hook: the k-th matrix product from now reports WR_HIP_ERR_INTERNAL (0 disarms). */
void wr_hip_mix_debug_fail_product_in(int k) { g_late = k; }

static float widen(uint16_t b)
{
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}
static uint32_t p32(uint32_t n) { return (n + 31) / 32 * 32; }
static float sig(float z) { return 1.0f / (1.0f + expf(-z)); }

int wr_hip_mix_available(void) { return 1; }

int wr_hip_mix_mat_create(uint32_t batch, uint32_t n_out, uint32_t n_in, const uint16_t *bf16, wr_hip_mat **out)
{
    if (!out || !bf16 || n_out % 16 || n_in % 32) return WR_HIP_ERR_INVAL;
    wr_hip_mat *m = malloc(sizeof *m);
    const size_t n = (size_t)batch * n_out * n_in;
    *m = (wr_hip_mat){batch, n_out, n_in, malloc(n * sizeof(float))};
    for (size_t i = 0; i < n; i++) m->w[i] = widen(bf16[i]);
    *out = m;
    return WR_HIP_OK;
}
void wr_hip_mix_mat_destroy(wr_hip_mat *w)
{
    if (!w) return;
    free(w->w);
    free(w);
}

int wr_hip_mix_pool_create(int f32, uint32_t n_latent, const uint32_t *latent_dim, uint32_t n_pages, uint32_t n_state,
                           const uint64_t *state_elems, uint32_t n_slots, wr_hip_mix_pool **out)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    wr_hip_mix_pool *p = calloc(1, sizeof *p);
    p->n_pages = n_pages;
    p->n_slots = n_slots;
    p->n_latent = n_latent;
    p->n_state = n_state;
    p->latent_dim = calloc(n_latent + 1, 4);
    p->state_elems = calloc(n_state + 1, 8);
    p->latent = calloc(n_latent + 1, sizeof *p->latent);
    p->state = calloc(n_state + 1, sizeof *p->state);
    for (uint32_t i = 0; i < n_latent; i++) {
        p->latent_dim[i] = latent_dim[i];
        const size_t n = (size_t)n_pages * WR_HIP_MIX_PAGE * latent_dim[i];
        p->latent[i] = malloc(n * 4);
        for (size_t k = 0; k < n; k++) p->latent[i][k] = NAN;      /* what was never written must never be read */
    }
    for (uint32_t i = 0; i < n_state; i++) {
        p->state_elems[i] = state_elems[i];
        p->state[i] = malloc((size_t)n_slots * 2 * state_elems[i] * 4);
        for (size_t k = 0; k < (size_t)n_slots * 2 * state_elems[i]; k++) p->state[i][k] = NAN;
    }
    *out = p;
    return WR_HIP_OK;
}
void wr_hip_mix_pool_destroy(wr_hip_mix_pool *p)
{
    if (!p) return;
    for (uint32_t i = 0; i < p->n_latent; i++) free(p->latent[i]);
    for (uint32_t i = 0; i < p->n_state; i++) free(p->state[i]);
    free(p->latent_dim);
    free(p->state_elems);
    free(p->latent);
    free(p->state);
    free(p);
}
uint64_t wr_hip_mix_pool_bytes(const wr_hip_mix_pool *p) { (void)p; return 0; }

int wr_hip_mix_step_create(uint32_t max_pages, wr_hip_mix_step **out)
{
    *out = calloc(1, sizeof **out);
    (*out)->max_pages = max_pages;
    return WR_HIP_OK;
}
void wr_hip_mix_step_destroy(wr_hip_mix_step *s) { free(s); }

int wr_hip_mix_step_set(wr_hip_mix_step *s, const wr_hip_mix_pool *pool, uint32_t n_seq, const wr_hip_mix_seq *seqs,
                        const uint32_t *tokens, uint32_t vocab, uint32_t n_want, const uint32_t *want_rows)
{
    uint32_t rows = 0, pages = 0;
    for (uint32_t i = 0; i < n_seq; i++) {
        const wr_hip_mix_seq *q = &seqs[i];
        if (!q->rows || q->slot >= pool->n_slots || q->n_pages * WR_HIP_MIX_PAGE < q->pos0 + q->rows) return WR_HIP_ERR_INVAL;
        for (uint32_t j = 0; j < q->n_pages; j++)
            if (q->pages[j] >= pool->n_pages) return WR_HIP_ERR_INVAL;
        if (rows + q->rows > WR_HIP_MIX_MAX_ROWS) return WR_HIP_ERR_LIMIT;
        s->seqs[i] = *q;
        s->row0[i] = rows;
        for (uint32_t r = 0; r < q->rows; r++) {
            s->seq[rows + r] = i;
            s->pos[rows + r] = q->pos0 + r;
            if (tokens[rows + r] >= vocab) return WR_HIP_ERR_INVAL;
            s->tokens[rows + r] = tokens[rows + r];
        }
        rows += q->rows;
        pages += q->n_pages;
    }
    if (pages > s->max_pages || n_want > rows) return WR_HIP_ERR_LIMIT;
    for (uint32_t i = 0; i < n_want; i++) s->want[i] = want_rows[i];
    s->rows = rows;
    s->n_seq = n_seq;
    s->n_want = n_want;
    return WR_HIP_OK;
}

static float inv_rms(const float *x, uint32_t n, float eps)
{
    double ss = 0;
    for (uint32_t i = 0; i < n; i++) ss += (double)x[i] * x[i];
    return 1.0f / sqrtf((float)(ss / n) + eps);
}

int wr_hip_mix_embed(wr_hip_mix_step *s, int f32, const uint16_t *table, uint32_t width, const float *norm, float scale,
                     float eps, float *x, float *x0, const float *next, void *h)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t wp = p32(width);
    for (uint32_t r = 0; r < s->rows; r++) {
        float *xr = x + (size_t)r * wp;
        for (uint32_t k = 0; k < wp; k++) xr[k] = k < width ? widen(table[(size_t)s->tokens[r] * width + k]) : 0.0f;
        const float inv = norm ? inv_rms(xr, width, eps) : scale;
        for (uint32_t k = 0; k < wp; k++) xr[k] = xr[k] * inv * (norm ? norm[k] : 1.0f);
        if (x0) memcpy(x0 + (size_t)r * wp, xr, wp * 4);
        if (next) {
            const float i2 = inv_rms(xr, width, eps);
            for (uint32_t k = 0; k < wp; k++) ((float *)h)[(size_t)r * wp + k] = xr[k] * i2 * next[k];
        }
    }
    return WR_HIP_OK;
}

int wr_hip_mix_residual(wr_hip_mix_step *s, int f32, const wr_hip_mix_resid *a)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t wp = p32(a->width), rows = a->wanted ? s->n_want : s->rows;
    float *y = malloc(wp * 4);
    for (uint32_t i = 0; i < rows; i++) {
        const uint32_t r = a->wanted ? s->want[i] : i;
        float *x = a->x + (size_t)r * wp;
        if (a->y) {
            for (uint32_t k = 0; k < wp; k++) {
                y[k] = a->top ? 0.0f : a->y[(size_t)r * wp + k];
                for (uint32_t t = 0; t < a->top; t++) {
                    const uint32_t slot = a->slot[(size_t)r * a->top + t];
                    if (slot != ~0u) y[k] += (a->gate ? a->gate[(size_t)r * a->top + t] : 1.0f) * a->y[(size_t)slot * wp + k];
                }
                if (a->side && a->ident) y[k] += a->side[2 * r] * ((const float *)a->ident)[(size_t)r * wp + k];
                if (a->side && a->shared) y[k] += a->side[2 * r + 1] * a->shared[(size_t)r * wp + k];
            }
            const float inv = a->post ? inv_rms(y, a->width, a->eps) : 1.0f;
            for (uint32_t k = 0; k < wp; k++) x[k] += a->post ? y[k] * inv * a->post[k] : y[k];
        }
        for (int i2 = 0; i2 < 2 && a->pair_y[i2]; i2++) {
            const float *p = a->pair_y[i2] + (size_t)r * wp, inv = inv_rms(p, a->width, a->eps);
            for (uint32_t k = 0; k < wp; k++) x[k] += p[k] * inv * a->pair_post[i2][k];
        }
        if (a->add)
            for (uint32_t k = 0; k < wp; k++) x[k] += a->add[(size_t)r * wp + k];
        if (a->next) {
            const float inv = inv_rms(x, a->width, a->eps);
            for (uint32_t k = 0; k < wp; k++) ((float *)a->h)[(size_t)i * wp + k] = x[k] * inv * a->next[k];
        }
    }
    free(y);
    return WR_HIP_OK;
}

int wr_hip_mix_shift(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, uint32_t width, float eps,
                     const float *x, const float *y, float *x_out, const float *norm, uint32_t n_mix, const float *mu,
                     void *out)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t wp = p32(width);
    float *h = malloc(wp * 4), *p = malloc(wp * 4);
    for (uint32_t i = 0; i < s->n_seq; i++) {
        const wr_hip_mix_seq *q = &s->seqs[i];
        const float *in = pool->state[run] + (size_t)(q->slot * 2 + q->buf_in) * wp;
        for (uint32_t k = 0; k < wp; k++) p[k] = q->pos0 ? in[k] : 0.0f;
        for (uint32_t r = s->row0[i]; r < s->row0[i] + q->rows; r++) {
            for (uint32_t k = 0; k < wp; k++) h[k] = x[(size_t)r * wp + k] + (y ? y[(size_t)r * wp + k] : 0.0f);
            if (y) memcpy(x_out + (size_t)r * wp, h, wp * 4);
            const float inv = inv_rms(h, width, eps);
            for (uint32_t k = 0; k < wp; k++) h[k] *= inv * norm[k];
            for (uint32_t m = 0; m < n_mix; m++)
                for (uint32_t k = 0; k < wp; k++)
                    ((float *)out)[((size_t)r * n_mix + m) * wp + k] = h[k] + (p[k] - h[k]) * mu[m * wp + k];
            memcpy(p, h, wp * 4);
        }
        memcpy(pool->state[run] + (size_t)(q->slot * 2 + q->buf_out) * wp, p, wp * 4);
    }
    free(h);
    free(p);
    return WR_HIP_OK;
}

static float gated_unit(const wr_hip_mix_gemm *a, float g, float u)
{
    if (a->limit > 0) {
        g = fminf(g, a->limit);
        u = fminf(fmaxf(u, -a->limit), a->limit);
        return g * sig(a->slope * g) * (u + a->up_bias);
    }
    return a->gelu ? 0.5f * g * (1.0f + tanhf(0.79788456080286536f * (g + 0.044715f * g * g * g))) * u : g * sig(g) * u;
}

static float row_value(const wr_hip_mix_gemm *a, uint32_t n, float o)
{
    const uint32_t sig_end = a->sigmoid_end > a->silu_end ? a->sigmoid_end : a->silu_end;
    if (a->bias) o += a->bias[n];
    if (n < a->silu_end) return o * sig(o);
    if (n < sig_end) return sig(o);
    if (n < a->tanh_end) return tanhf(o);
    return a->relu2 ? (o > 0 ? o * o : 0) : o;
}

int wr_hip_mix_gemm_run(int f32, const wr_hip_mix_gemm *a)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    if (g_late > 0 && --g_late == 0) return WR_HIP_ERR_INTERNAL;
    const uint32_t N = a->w->n_out, K = a->w->n_in, batch = a->group_expert ? 1 : a->w->batch, ldx = a->x_kt * 32;
    float *v = malloc(N * 4);
    for (uint32_t z = 0; z < batch; z++)
        for (uint32_t r = 0; r < a->rows; r++) {
            uint32_t mat = z;
            if (a->group_expert) {
                if (a->group_expert[r / 16] < 0) continue;
                mat = (uint32_t)a->group_expert[r / 16];
            }
            const uint32_t from = !a->x_perm ? r : a->x_perm[r] == ~0u ? 0 : a->x_perm[r];
            const float *x = (const float *)a->x + (size_t)from * ldx + ((size_t)a->x_kt0 + (size_t)z * a->x_kt_z) * 32;
            const float *w = a->w->w + (size_t)mat * N * K;
            for (uint32_t n = 0; n < N; n++) {
                float acc = 0;
                for (uint32_t k = 0; k < K; k++) acc += w[(size_t)n * K + k] * x[k];
                v[n] = a->x_scale ? acc * a->x_scale[r] : acc;
            }
            float *h = a->h ? (float *)a->h + (size_t)r * a->h_kt * 32 + (size_t)a->h_kt0 * 32 + (size_t)z * a->col_z : NULL;
            if (a->out >= WR_HIP_MIX_OUT_GATED) {
                const uint32_t rows = a->out == WR_HIP_MIX_OUT_SPLIT_GATED ? a->n_split : 0;
                for (uint32_t n = 0; n < rows; n++) a->y_f32[(size_t)r * a->ldy + n] = row_value(a, n, v[n]);
                for (uint32_t n = 0; n < (N - rows) / 2; n++)
                    h[n] = gated_unit(a, v[rows + n / 16 * 32 + n % 16], v[rows + n / 16 * 32 + 16 + n % 16]);
                continue;
            }
            for (uint32_t n = 0; n < N; n++) {
                float o = row_value(a, n, v[n]);
                if (a->scale != 0) o *= a->scale;
                if (a->out == WR_HIP_MIX_OUT_ROWS_F32) a->y_f32[(size_t)r * a->ldy + (size_t)z * a->col_z + n] = o;
                else if (a->out == WR_HIP_MIX_OUT_ROWS) ((float *)a->y_act)[(size_t)r * a->ldy + n] = o;
                else if (a->out == WR_HIP_MIX_OUT_SPLIT && n >= a->n_split) a->y_f32[(size_t)r * a->ldy + n - a->n_split] = o;
                else h[n] = o;
            }
        }
    free(v);
    return WR_HIP_OK;
}

int wr_hip_mix_lightning(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, uint32_t heads, uint32_t dim,
                         uint32_t vdim, const float *decay, const void *qkv, uint32_t ld, uint32_t col_k, uint32_t col_v,
                         float *o, uint32_t ldo)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const size_t all = (size_t)heads * dim * vdim;
    for (uint32_t i = 0; i < s->n_seq; i++) {
        const wr_hip_mix_seq *q = &s->seqs[i];
        float *S = calloc(all, 4);
        if (q->pos0) memcpy(S, pool->state[run] + (size_t)(q->slot * 2 + q->buf_in) * all, all * 4);
        for (uint32_t r = s->row0[i]; r < s->row0[i] + q->rows; r++) {
            const float *row = (const float *)qkv + (size_t)r * ld;
            for (uint32_t h = 0; h < heads; h++)
                for (uint32_t v = 0; v < vdim; v++) {
                    float acc = 0;
                    for (uint32_t d = 0; d < dim; d++) {
                        float *e = &S[((size_t)h * dim + d) * vdim + v];
                        *e = decay[h] * *e + row[col_k + h * dim + d] * row[col_v + h * vdim + v];
                        acc += *e * row[h * dim + d];
                    }
                    o[(size_t)r * ldo + h * vdim + v] = acc;
                }
        }
        memcpy(pool->state[run] + (size_t)(q->slot * 2 + q->buf_out) * all, S, all * 4);
        free(S);
    }
    return WR_HIP_OK;
}

int wr_hip_mix_gate_norm(wr_hip_mix_step *s, int f32, const float *o, uint32_t ldo, uint32_t n, const void *g, uint32_t ldg,
                         const float *norm, float eps, void *h)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t np = p32(n);
    for (uint32_t r = 0; r < s->rows; r++) {
        const float inv = inv_rms(o + (size_t)r * ldo, n, eps);
        for (uint32_t k = 0; k < np; k++)
            ((float *)h)[(size_t)r * np + k] =
                k < n ? o[(size_t)r * ldo + k] * inv * norm[k] * ((const float *)g)[(size_t)r * ldg + k] : 0.0f;
    }
    return WR_HIP_OK;
}

int wr_hip_mix_rope_table(wr_hip_mix_step *s, const double *freq, uint32_t half, float gain, float *table)
{
    for (uint32_t r = 0; r < s->rows; r++)
        for (uint32_t i = 0; i < half; i++) {
            table[2 * ((size_t)r * half + i)] = (float)cos(s->pos[r] * freq[i]) * gain;
            table[2 * ((size_t)r * half + i) + 1] = (float)sin(s->pos[r] * freq[i]) * gain;
        }
    return WR_HIP_OK;
}

/* S <- diag(w) S + (1 - w) v^T, o = S^T r, normed head by head. */
static int recur_forget(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, const wr_hip_mix_recurrence *a)
{
    const uint32_t D = a->dim, V = a->vdim, hv = a->heads * V;
    const size_t all = (size_t)a->heads * D * V;
    if (pool->state_elems[run] != all) return WR_HIP_ERR_INVAL;
    for (uint32_t i = 0; i < s->n_seq; i++) {
        const wr_hip_mix_seq *q = &s->seqs[i];
        float *S = calloc(all, 4), *o = malloc(V * 4);
        if (q->pos0) memcpy(S, pool->state[run] + (size_t)(q->slot * 2 + q->buf_in) * all, all * 4);
        for (uint32_t t = s->row0[i]; t < s->row0[i] + q->rows; t++) {
            const float *row = a->in + (size_t)t * a->ld;
            float *to = (float *)a->h + (size_t)t * a->h_kt * 32 + a->col_h;
            for (uint32_t h = 0; h < a->heads; h++) {
                memset(o, 0, V * 4);
                for (uint32_t d = 0; d < D; d++) {
                    const uint32_t n = h * D + d;
                    const float z = row[a->col_k + n] + a->w0[n], w = a->lower[n] + (1 - a->lower[n]) * sig(z);
                    const float k = (1 - a->lower[n]) * sig(-z);
                    for (uint32_t c = 0; c < V; c++) {
                        float *e = &S[((size_t)h * D + d) * V + c];
                        *e = w * *e + k * row[a->col_v + h * V + c];
                        o[c] += *e * row[a->col_r + n];
                    }
                }
                const float inv = a->out_scale * inv_rms(o, V, a->eps);
                for (uint32_t c = 0; c < V; c++) to[h * V + c] = o[c] * inv * a->norm[c];
            }
            for (uint32_t c = hv; c < p32(hv); c++) to[c] = 0.0f;
        }
        memcpy(pool->state[run] + (size_t)(q->slot * 2 + q->buf_out) * all, S, all * 4);
        free(S);
        free(o);
    }
    return WR_HIP_OK;
}

int wr_hip_mix_min_gru(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, const wr_hip_mix_gru *a)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t wp = p32(a->width);
    if (pool->state_elems[run] != wp) return WR_HIP_ERR_INVAL;
    for (uint32_t i = 0; i < s->n_seq; i++) {
        const wr_hip_mix_seq *q = &s->seqs[i];
        const float *in = pool->state[run] + (size_t)(q->slot * 2 + q->buf_in) * wp;
        float *out = pool->state[run] + (size_t)(q->slot * 2 + q->buf_out) * wp;
        for (uint32_t k = 0; k < wp; k++) {
            float S = q->pos0 ? in[k] : 0.0f;
            for (uint32_t t = s->row0[i]; t < s->row0[i] + q->rows; t++) {
                const float *row = a->in + (size_t)t * a->ld, z = row[a->col_z + k], u = row[a->col_x + k], g = row[a->col_g + k];
                S = sig(-z) * S + sig(z) * (u >= 0 ? u + 0.5f : sig(u));
                ((float *)a->h)[(size_t)t * a->h_kt * 32 + a->col_h + k] = S * g * sig(g);
            }
            out[k] = S;
        }
    }
    return WR_HIP_OK;
}

int wr_hip_mix_recur(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, const wr_hip_mix_recurrence *a)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    if (a->rule == WR_HIP_MIX_RULE_FORGET) return recur_forget(s, pool, run, a);
    const uint32_t D = a->dim, hd = a->heads * D, delta = a->rule == WR_HIP_MIX_RULE_DELTA;
    const size_t all = (size_t)hd * D;
    if (pool->state_elems[run] != all) return WR_HIP_ERR_INVAL;
    const uint32_t ldz = a->w_decay->n_out;
    const wr_hip_mix_gemm decay = {.w = a->w_decay, .x = a->low, .x_kt = a->w_decay->n_in / 32, .rows = s->rows,
                                   .out = WR_HIP_MIX_OUT_ROWS_F32, .y_f32 = a->z, .ldy = ldz};
    const int rc = wr_hip_mix_gemm_run(f32, &decay);
    if (rc != WR_HIP_OK) return rc;
    float w[WR_HIP_MIX_MAX_RECUR_DIM], b[WR_HIP_MIX_MAX_RECUR_DIM], n[WR_HIP_MIX_MAX_RECUR_DIM], o[WR_HIP_MIX_MAX_RECUR_DIM];
    for (uint32_t i = 0; i < s->n_seq; i++) {
        const wr_hip_mix_seq *q = &s->seqs[i];
        float *S = calloc(all, 4);
        if (q->pos0) memcpy(S, pool->state[run] + (size_t)(q->slot * 2 + q->buf_in) * all, all * 4);
        for (uint32_t t = s->row0[i]; t < s->row0[i] + q->rows; t++)
            for (uint32_t h = 0; h < a->heads; h++) {
                const float *row = a->in + (size_t)t * a->ld + h * D, *r = row + a->col_r, *k = row + a->col_k,
                            *v = row + a->col_v, *g = row + a->col_g, *z = a->z + (size_t)t * ldz + h * D;
                float kk = 0, ss = 0;
                for (uint32_t d = 0; d < D; d++) kk += k[d] * k[d];
                for (uint32_t d = 0; d < D; d++) {
                    const float y = z[d] + a->w0[h * D + d];
                    w[d] = expf(a->gain > 0 ? -a->gain * sig(y) : -expf(y));
                    n[d] = k[d] / sqrtf(kk + a->unit_eps);
                    b[d] = delta ? sig(row[a->col_a + d] + a->a_bias[h * D + d]) * n[d] : 0.0f;
                }
                for (uint32_t c = 0; c < D; c++) {
                    float *col = S + (size_t)h * D * D + c, seen = 0, out = 0;
                    for (uint32_t d = 0; d < D; d++) seen += delta ? n[d] * col[d * D] : 0.0f;
                    for (uint32_t d = 0; d < D; d++) {
                        const float old = col[d * D];
                        if (!delta) out += r[d] * (old + a->u[h * D + d] * k[d] * v[c]);
                        col[d * D] = w[d] * old - b[d] * seen + k[d] * v[c];
                        if (delta) out += r[d] * col[d * D];
                    }
                    o[c] = out;
                    ss += out * out;
                }
                const float inv = a->out_scale / sqrtf(ss / D + a->eps);
                float *to = (float *)a->h + (size_t)t * a->h_kt * 32 + a->col_h + h * D;
                for (uint32_t c = 0; c < D; c++) to[c] = o[c] * inv * a->norm[h * D + c] * sig(g[c]) * (a->gate_silu ? g[c] : 1.0f);
                if (h + 1 == a->heads)
                    for (uint32_t c = hd; c < p32(hd); c++) to[c - h * D] = 0.0f;
            }
        memcpy(pool->state[run] + (size_t)(q->slot * 2 + q->buf_out) * all, S, all * 4);
        free(S);
    }
    return WR_HIP_OK;
}

uint32_t wr_hip_mix_latent_rank_pad(uint32_t rank) { return p32(rank); }

static void rotate(const float *x, const float *tab, uint32_t half, uint32_t n, float *out)
{
    for (uint32_t i = 0; i < n; i++) {
        if (i < half) out[i] = x[i] * tab[2 * i] - x[i + half] * tab[2 * i + 1];
        else if (i < 2 * half) out[i] = x[i] * tab[2 * (i - half)] + x[i - half] * tab[2 * (i - half) + 1];
        else out[i] = x[i];
    }
}

int wr_hip_mix_latent_append(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, const wr_hip_mix_latent *g,
                             const float *d, uint32_t ldd, uint32_t q_rank, const float *q_norm, const float *kv_norm,
                             float eps, const float *table, void *cq)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t qp = p32(q_rank), dk = g->rank_pad + g->rot_pad;
    for (uint32_t r = 0; r < s->rows; r++) {
        const float *dr = d + (size_t)r * ldd, *dc = dr + qp;
        const float qi = inv_rms(dr, q_rank, eps), ki = inv_rms(dc, g->rank, eps);
        for (uint32_t k = 0; k < qp; k++) ((float *)cq)[(size_t)r * qp + k] = k < q_rank ? dr[k] * qi * q_norm[k] : 0.0f;
        const wr_hip_mix_seq *q = &s->seqs[s->seq[r]];
        float *row = pool->latent[run] +
                     ((size_t)q->pages[s->pos[r] / WR_HIP_MIX_PAGE] * WR_HIP_MIX_PAGE + s->pos[r] % WR_HIP_MIX_PAGE) * dk;
        memset(row, 0, dk * 4);
        for (uint32_t k = 0; k < g->rank; k++) row[k] = dc[k] * ki * kv_norm[k];
        rotate(dc + p32(g->rank), table + (size_t)r * 2 * g->rot_half, g->rot_half, g->rot, row + g->rank_pad);
    }
    return WR_HIP_OK;
}

int wr_hip_mix_latent_qrope(wr_hip_mix_step *s, int f32, const wr_hip_mix_latent *g, const float *qr, uint32_t ldq,
                            const float *table, void *q)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t dk = g->rank_pad + g->rot_pad;
    for (uint32_t r = 0; r < s->rows; r++)
        for (uint32_t h = 0; h < g->heads; h++) {
            float *out = (float *)q + ((size_t)r * g->heads + h) * dk + g->rank_pad;
            memset(out, 0, g->rot_pad * 4);
            rotate(qr + (size_t)r * ldq + h * g->rot, table + (size_t)r * 2 * g->rot_half, g->rot_half, g->rot, out);
        }
    return WR_HIP_OK;
}

int wr_hip_mix_latent_attend(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, const wr_hip_mix_latent *g,
                             const void *qv, void *ov)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t dk = g->rank_pad + g->rot_pad;
    for (uint32_t r = 0; r < s->rows; r++) {
        const wr_hip_mix_seq *sq = &s->seqs[s->seq[r]];
        const uint32_t pos = s->pos[r], lo = pos + 1 > g->window ? pos + 1 - g->window : 0;
        double *w = malloc(sizeof(double) * (pos - lo + 1));
        for (uint32_t h = 0; h < g->heads; h++) {
            const float *q = (const float *)qv + ((size_t)r * g->heads + h) * dk;
            float *o = (float *)ov + (size_t)r * g->heads * g->rank_pad + (size_t)h * g->rank_pad;
            double mx = -INFINITY, sum = 0;
            for (uint32_t j = lo; j <= pos; j++) {
                const float *row = pool->latent[run] +
                                   ((size_t)sq->pages[j / WR_HIP_MIX_PAGE] * WR_HIP_MIX_PAGE + j % WR_HIP_MIX_PAGE) * dk;
                double a = 0;
                for (uint32_t k = 0; k < dk; k++) a += (double)q[k] * row[k];
                w[j - lo] = a * g->scale;
                if (w[j - lo] > mx) mx = w[j - lo];
            }
            for (uint32_t j = lo; j <= pos; j++) sum += (w[j - lo] = exp(w[j - lo] - mx));
            for (uint32_t k = 0; k < g->rank_pad; k++) {
                double a = 0;
                for (uint32_t j = lo; j <= pos; j++)
                    a += w[j - lo] * pool->latent[run][((size_t)sq->pages[j / WR_HIP_MIX_PAGE] * WR_HIP_MIX_PAGE +
                                                        j % WR_HIP_MIX_PAGE) * dk + k];
                o[k] = (float)(a / sum);
            }
        }
        free(w);
    }
    return WR_HIP_OK;
}

uint32_t wr_hip_mix_window_pad(uint32_t dim) { return p32(dim); }

static float *window_row(wr_hip_mix_pool *pool, uint32_t run, const wr_hip_mix_window *g, const wr_hip_mix_seq *q, uint32_t pos,
                         uint32_t kvh)
{
    const uint32_t per = g->maps * g->dim_pad + g->vdim_pad;
    return pool->latent[run] + (((size_t)q->pages[pos / WR_HIP_MIX_PAGE] * g->kv_heads + kvh) * WR_HIP_MIX_PAGE +
                                pos % WR_HIP_MIX_PAGE) * per;
}

/* One query or key of one map: normed, rotated, padded. */
static void window_turn(const wr_hip_mix_window *g, const float *x, const float *norm, const float *tab, float *out)
{
    float *y = malloc(g->dim * 4);
    const float inv = norm ? inv_rms(x, g->dim, g->eps) : 1.0f;
    for (uint32_t i = 0; i < g->dim; i++) y[i] = norm ? x[i] * inv * norm[i] : x[i];
    memset(out, 0, g->dim_pad * 4);
    if (!g->neighbours) {
        rotate(y, tab, g->rot_half, g->dim, out);
    } else {
        memcpy(out, y, g->dim * 4);
        for (uint32_t i = 0; i < g->rot_half; i++) {
            out[2 * i] = y[2 * i] * tab[2 * i] - y[2 * i + 1] * tab[2 * i + 1];
            out[2 * i + 1] = y[2 * i + 1] * tab[2 * i] + y[2 * i] * tab[2 * i + 1];
        }
    }
    free(y);
}

int wr_hip_mix_window_append(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, const wr_hip_mix_window *g,
                             const float *in, uint32_t ld, uint32_t col_q, uint32_t col_k, uint32_t col_v, const float *table,
                             void *qv)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    for (uint32_t r = 0; r < s->rows; r++) {
        const float *row = in + (size_t)r * ld, *tab = table + (size_t)r * 2 * g->rot_half;
        for (uint32_t h = 0; h < g->heads * g->maps; h++)
            window_turn(g, row + col_q + h * g->dim, g->q_norm, tab, (float *)qv + ((size_t)r * g->heads * g->maps + h) * g->dim_pad);
        for (uint32_t h = 0; h < g->kv_heads && col_k != WR_HIP_MIX_NO_KEYS; h++) {
            float *c = window_row(pool, run, g, &s->seqs[s->seq[r]], s->pos[r], h), *cv = c + g->maps * g->dim_pad;
            for (uint32_t m = 0; m < g->maps; m++)
                window_turn(g, row + col_k + (h * g->maps + m) * g->dim, g->k_norm, tab, c + m * g->dim_pad);
            memset(cv, 0, g->vdim_pad * 4);
            const float *v = row + col_v + h * g->vdim, inv = g->norm_values ? inv_rms(v, g->vdim, g->eps) : 1.0f;
            for (uint32_t k = 0; k < g->vdim; k++) cv[k] = v[k] * inv;
            for (uint32_t k = 0; g->turn_values && k < g->vdim; k += 2) {
                const float *cs = g->turn_values + (size_t)r * g->vdim + k, x = cv[k], y = cv[k + 1];
                cv[k] = x * cs[0] - y * cs[1];
                cv[k + 1] = y * cs[0] + x * cs[1];
            }
        }
    }
    return WR_HIP_OK;
}

int wr_hip_mix_window_attend(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, const wr_hip_mix_window *g,
                             const void *qv, const float *sink, const float *gate, uint32_t ldg, void *ov, uint32_t o_kt)
{
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    const uint32_t V = g->vdim_pad;
    for (uint32_t r = 0; r < s->rows; r++) {
        const wr_hip_mix_seq *sq = &s->seqs[s->seq[r]];
        const uint32_t pos = s->pos[r];
        const uint32_t lo = g->chunk ? pos / g->chunk * g->chunk : pos + 1 > g->window ? pos + 1 - g->window : 0;
        double *w = malloc(sizeof(double) * (pos - lo + 1)), *a2 = malloc(sizeof(double) * 2 * V);
        for (uint32_t h = 0; h < g->heads; h++) {
            const uint32_t kvh = h / (g->heads / g->kv_heads);
            float *o = (float *)ov + (size_t)r * o_kt * 32 + (size_t)h * V;
            for (uint32_t m = 0; m < g->maps; m++) {
                const float *q = (const float *)qv + (((size_t)r * g->heads + h) * g->maps + m) * g->dim_pad;
                double mx = sink ? sink[h] : -INFINITY;
                for (uint32_t j = lo; j <= pos; j++) {
                    const float *c = window_row(pool, run, g, sq, j, kvh) + m * g->dim_pad;
                    double a = 0;
                    for (uint32_t k = 0; k < g->dim_pad; k++) a += (double)q[k] * c[k];
                    a *= g->scale;
                    w[j - lo] = g->softcap > 0 ? g->softcap * tanh(a / g->softcap) : a;
                    if (w[j - lo] > mx) mx = w[j - lo];
                }
                double sum = sink ? exp(sink[h] - mx) : 0;
                for (uint32_t j = lo; j <= pos; j++) sum += (w[j - lo] = exp(w[j - lo] - mx));
                for (uint32_t k = 0; k < V; k++) {
                    double a = 0;
                    for (uint32_t j = lo; j <= pos; j++)
                        a += w[j - lo] * window_row(pool, run, g, sq, j, kvh)[g->maps * g->dim_pad + k];
                    a2[m * V + k] = a / sum;
                }
            }
            double f = gate && !g->gate_wide ? g->out_scale * sig(gate[(size_t)r * ldg + h]) : g->out_scale, ss = 0;
            for (uint32_t k = 0; g->maps == 2 && k < V; k++) {
                a2[k] -= g->diff * a2[V + k];
                ss += a2[k] * a2[k];
            }
            if (g->maps == 2) f /= sqrt(ss / g->vdim + g->eps);
            for (uint32_t k = 0; g->turn_values && k < g->vdim; k += 2) {
                const float *cs = g->turn_values + (size_t)r * g->vdim + k;
                const double x = a2[k], y = a2[k + 1];
                a2[k] = x * cs[0] + y * cs[1];
                a2[k + 1] = y * cs[0] - x * cs[1];
            }
            for (uint32_t k = 0; k < V; k++) o[k] = (float)(a2[k] * f * (g->gate_wide && k < g->vdim ? sig(gate[(size_t)r * ldg + h * g->vdim + k]) : 1.0f));
        }
        free(w);
        free(a2);
    }
    return WR_HIP_OK;
}

uint32_t wr_hip_mix_route_groups(uint32_t rows, uint32_t experts, uint32_t top, uint32_t tile_groups)
{
    const uint32_t pairs = rows * top;
    return (pairs / (tile_groups * 16) + (pairs < experts ? pairs : experts)) * tile_groups;
}

int wr_hip_mix_route(wr_hip_mix_step *s, const float *z, uint32_t ldz, const wr_hip_mix_router *g, uint32_t tile_groups,
                     float *gate, float *side, float *slot_weight, uint32_t *slot, uint32_t *perm, int32_t *group_expert)
{
    const uint32_t experts = g->experts, top = g->top, N = experts + g->identity;
    const uint32_t groups = wr_hip_mix_route_groups(s->rows, experts, top, tile_groups), run = tile_groups * 16;
    if (ldz < N + (g->shared_gate != 0) || (g->groups && N % g->groups)) return WR_HIP_ERR_INVAL;
    float *c = malloc(N * 4), *p = malloc(N * 4), *lead = malloc((g->groups + 1) * 4);
    for (uint32_t r = 0; r < s->rows; r++) {
        const float *zr = z + (size_t)r * ldz;
        float most = zr[0], all = 0;
        for (uint32_t e = 1; e < N; e++) most = fmaxf(most, zr[e]);
        for (uint32_t e = 0; e < N; e++) all += (p[e] = expf(zr[e] - most));
        for (uint32_t e = 0; e < N; e++) c[e] = g->softmax_all ? p[e] / all + (g->correction ? g->correction[e] : 0) : zr[e];
        for (uint32_t k = 0; k < g->groups; k++) {
            lead[k] = -INFINITY;
            for (uint32_t e = k * (N / g->groups); e < (k + 1) * (N / g->groups); e++) lead[k] = fmaxf(lead[k], c[e]);
        }
        for (uint32_t k = 0; k < g->groups; k++) {
            uint32_t ahead = 0;
            for (uint32_t j = 0; j < g->groups; j++) ahead += lead[j] > lead[k] || (lead[j] == lead[k] && j < k);
            for (uint32_t e = 0; ahead >= g->keep && e < N / g->groups; e++) c[k * (N / g->groups) + e] = -INFINITY;
        }
        float sum = 0, own = 0;
        for (uint32_t t = 0; t < top; t++) {
            uint32_t best = 0;
            for (uint32_t e = 1; e < N; e++)
                if (c[e] > c[best]) best = e;
            c[best] = -INFINITY;
            slot[r * top + t] = best;
            sum += gate[r * top + t] = g->logistic ? sig(zr[best]) : g->softmax_all ? p[best] / all : p[best];
        }
        for (uint32_t t = 0; t < top; t++) {
            float *w = &gate[r * top + t];
            if (!g->logistic) *w = g->softmax_all ? *w / (sum + 1e-20f) * g->scale : *w / sum;
            if (slot[r * top + t] >= experts) own += *w;
        }
        if (side) {
            side[2 * r] = own;
            side[2 * r + 1] = g->shared_gate ? sig(zr[N]) : 0;
        }
    }
    free(c);
    free(p);
    free(lead);
    for (uint32_t i = 0; i < groups * 16; i++) perm[i] = ~0u;
    for (uint32_t i = 0; slot_weight && i < groups * 16; i++) slot_weight[i] = 0;
    for (uint32_t i = 0; i < groups; i++) group_expert[i] = -1;
    uint32_t at = 0;
    uint32_t *out = malloc((size_t)s->rows * top * 4);
    memset(out, 0xFF, (size_t)s->rows * top * 4);          /* (the input itself takes no slot) */
    for (uint32_t e = 0; e < experts; e++) {
        const uint32_t begin = at;
        for (uint32_t i = 0; i < s->rows * top; i++)
            if (slot[i] == e) {
                perm[at] = i / top;
                if (slot_weight) slot_weight[at] = gate[i];
                out[i] = at++;
            }
        at = (at + run - 1) / run * run;
        for (uint32_t i = begin / 16; i < at / 16; i++) group_expert[i] = (int32_t)e;
    }
    memcpy(slot, out, (size_t)s->rows * top * 4);
    free(out);
    return WR_HIP_OK;
}

int wr_hip_mix_route_gather(wr_hip_mix_step *s, int f32, const void *h, uint32_t kt, uint32_t n_groups, const uint32_t *perm,
                            const int32_t *group_expert, void *xs)
{
    (void)s;
    if (!f32) return WR_HIP_ERR_UNSUPPORTED;
    for (uint32_t i = 0; i < n_groups * 16; i++) {
        if (group_expert[i / 16] < 0) continue;
        float *to = (float *)xs + (size_t)i * kt * 32;
        if (perm[i] == ~0u) memset(to, 0, (size_t)kt * 128);
        else memcpy(to, (const float *)h + (size_t)perm[i] * kt * 32, (size_t)kt * 128);
    }
    return WR_HIP_OK;
}
