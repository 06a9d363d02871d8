/*
 * wr_hip_mix.h — C ABI of the device steps of mixer-stack models: models whose
 * layers pair a mixer (decayed linear attention, sliding-window attention through
 * a low-rank latent or over grouped keys and values, a matrix-state recurrence
 * with input-made decays, an element-wise gated recurrence) with a feed-forward (dense
 * or a mixture of experts), with norms before and, in some designs, after each, or one
 * norm for both, and bfloat16 weights.
 *
 * Conventions are those of wr_hip_attn.h: plain C, status returns, every call
 * enqueues on the calling thread's stream and returns without waiting unless it
 * says otherwise.  There is no reference interface behind these calls: the
 * reference has no such models.
 *
 * Precision.  Each call takes `f32`: 0 = activations that feed a matrix product
 * are bfloat16 (32-bit accumulation); 1 = they are 32-bit and the products run on
 * the 32-bit matrix instructions.  In both, the residual rows, norms, angles,
 * attention scores and softmax, router logits and the recurrent state are
 * 32-bit.
 *
 * Layouts.  Feature counts are padded to multiples of 32, pads zero.  "rows" is
 * 32-bit row-major [rows][ld].  "frag" is the operand order of the matrix
 * instruction: element (row, k) of a matrix with KT = K/32 input tiles lies at
 * unit ((row/16) * KT + k/32) * 64 + 16 * ((k % 32) / 8) + row % 16, element
 * k % 8 of the unit's eight.
 */
#ifndef WR_HIP_MIX_H
#define WR_HIP_MIX_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define WR_HIP_MIX_PAGE       64u     /* positions per cache page */
#define WR_HIP_MIX_MAX_SEQS   16u     /* requests in one step (WR_HIP_BATCH_MAX) */
#define WR_HIP_MIX_MAX_ROWS   4096u   /* rows in one step */
#define WR_HIP_MIX_MAX_EXPERTS 1024u
#define WR_HIP_MIX_MAX_TOP     64u
#define WR_HIP_MIX_MAX_STATE_DIM 512u /* rows of a recurrent state matrix */
#define WR_HIP_MIX_MAX_RECUR_DIM 256u /* head size of wr_hip_mix_recur */

/* 1 when this build of the library runs mixer-stack models. */
int wr_hip_mix_available(void);

/* ---- weights -------------------------------------------------------------
 * `batch` matrices [n_out][n_in] of bfloat16 (host, row-major, n_out a multiple
 * of 16 and n_in of 32), copied to the device in operand order. Synchronous. */
typedef struct wr_hip_mat wr_hip_mat;
int  wr_hip_mix_mat_create(uint32_t batch, uint32_t n_out, uint32_t n_in,
                           const uint16_t *bf16, wr_hip_mat **out);
void wr_hip_mix_mat_destroy(wr_hip_mat *w);

/* ---- cache pool ----------------------------------------------------------
 * One pool per model, shared by its requests: `n_pages` pages of 64 positions
 * for each of `n_latent` attention layer runs (latent_dim[i] elements per position,
 * a multiple of 32) and `n_slots` state slots for each of `n_state` recurrent
 * layer runs (state_elems[i] floats).  A slot has two buffers: a step reads one
 * and writes the other, so a step that fails has changed nothing. */
typedef struct wr_hip_mix_pool wr_hip_mix_pool;
int  wr_hip_mix_pool_create(int f32, uint32_t n_latent, const uint32_t *latent_dim, uint32_t n_pages,
                            uint32_t n_state, const uint64_t *state_elems, uint32_t n_slots,
                            wr_hip_mix_pool **out);
void wr_hip_mix_pool_destroy(wr_hip_mix_pool *p);
uint64_t wr_hip_mix_pool_bytes(const wr_hip_mix_pool *p);

/* ---- a step's rows --------------------------------------------------------
 * The rows of up to 16 requests, each a run of consecutive positions (a portion
 * of a prompt or a single decoded token). */
typedef struct wr_hip_mix_seq {
    uint32_t rows;             /* how many rows this request brings (> 0) */
    uint32_t pos0;             /* position of the first of them */
    uint32_t slot;             /* its state slot */
    uint32_t buf_in, buf_out;  /* which of the slot's two buffers is read / written (0 or 1) */
    uint32_t n_pages;          /* pages it holds: at least (pos0 + rows) / 64 rounded up */
    const uint32_t *pages;
} wr_hip_mix_seq;

typedef struct wr_hip_mix_step wr_hip_mix_step;
int  wr_hip_mix_step_create(uint32_t max_pages, wr_hip_mix_step **out);
void wr_hip_mix_step_destroy(wr_hip_mix_step *s);
/* Describes the next step.  Checks every count, page and slot against `pool` and
 * every token against `vocab`; nothing is launched when one does not fit.  The
 * previous step of this object must have been waited for. */
int  wr_hip_mix_step_set(wr_hip_mix_step *s, const wr_hip_mix_pool *pool, uint32_t n_seq,
                         const wr_hip_mix_seq *seqs, const uint32_t *tokens, uint32_t vocab,
                         uint32_t n_want, const uint32_t *want_rows);

/* ---- row steps ------------------------------------------------------------
 * x[r] = rmsnorm(table[token r]) * norm, or table[token r] * scale without a norm;
 * x0, if not NULL, receives the same rows; h (frag) = rmsnorm(x[r]) * next, when
 * next is given.  table: device bfloat16 [vocab][width]. */
int wr_hip_mix_embed(wr_hip_mix_step *s, int f32, const uint16_t *table_dev, uint32_t width,
                     const float *norm_dev, float scale, float eps, float *x_dev, float *x0_dev,
                     const float *next_dev, void *h_dev);

/* A sublayer's output joins the residual and the next sublayer's input is made:
 *   x += rmsnorm(y) * post           (when y is given; x += y without `post`; with `top` > 0,
 *                                     row r of y is sum_t gate[r][t] * y[slot[r][t]], the
 *                                     experts' rows, slots of ~0 left out; with `side` as well
 *                                     + side[r][0] * ident[r] + side[r][1] * shared[r])
 *   x += rmsnorm(pair_y[i]) * pair_post[i], i = 0, 1   (when given, both or neither)
 *   x += add                         (when given)
 *   h = rmsnorm(x) * next            (when given; only the step's wanted rows, packed,
 *                                     with `wanted` set)
 * gate may be NULL: ones.  ident: frag rows of the width, may be h itself; shared: 32-bit rows
 * like y; either may be NULL. */
typedef struct wr_hip_mix_resid {
    uint32_t width;
    float eps;
    float *x;
    const float *y, *post, *add, *next;
    const float *gate;
    const uint32_t *slot;
    uint32_t top;
    uint32_t wanted;
    void *h;
    const float *side;
    const void *ident;
    const float *shared;
    const float *pair_y[2], *pair_post[2];
} wr_hip_mix_resid;
int wr_hip_mix_residual(wr_hip_mix_step *s, int f32, const wr_hip_mix_resid *a);
/* Token shift.  x += y first (y may be NULL).  With h[r] = rmsnorm(x[r]) * norm and p[r]
 * the same request's h one position earlier (zeros at position 0, else state `run` of
 * the pool, [width padded to 32] floats, which receives the request's last h):
 * mix i = h + (p - h) * mu[i] goes to out (frag of n_mix * padded width inputs) at input
 * i * padded width.  mu: n_mix vectors of the padded width.  With y the new residual
 * goes to x_out (another buffer than x), which is where x lives from then on. */
int wr_hip_mix_shift(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, uint32_t width,
                     float eps, const float *x_dev, const float *y_dev, float *x_out_dev,
                     const float *norm_dev, uint32_t n_mix, const float *mu_dev, void *out_dev);

/* ---- matrix products -------------------------------------------------------
 * For every matrix z of the batch: outputs = x_z . W_z^T, x_z being the input
 * tiles [x_kt0 + z * x_kt_z, ...) of frag rows with x_kt tiles in all (so x_kt_z = 0
 * shares the input).  With group_expert (see route), group g of 16 rows takes
 * matrix group_expert[g], and groups with a negative entry are skipped.
 * out says where output n of row r goes:
 *   ROWS_F32   y_f32[r][z * col_z + n]     32-bit rows, row stride ldy
 *   ROWS       y_act[r][n]                 activation type, row stride ldy
 *   FRAG       h (frag, h_kt tiles): row r, input h_kt0 * 32 + z * col_z + n
 *   SPLIT      n < n_split: FRAG; else y_f32[r][n - n_split]
 *   GATED      tiles 2j / 2j+1 of W are gate / up: silu(gate) * up to FRAG
 *              (with gelu: 0.5 g (1 + tanh(sqrt(2/pi) (g + 0.044715 g^3))) * up;
 *              with limit > 0: g = min(gate, limit), u = up within [-limit, limit],
 *              g * logistic(slope * g) * (u + up_bias))
 *   SPLIT_GATED n < n_split (a multiple of 32): y_f32[r][n]; the tiles behind as GATED
 * after a factor per row (x_scale, with group_expert), `bias` (a float for each of the n_out
 * outputs, batch 1) and an activation: SiLU for n < silu_end, else the logistic for n <
 * sigmoid_end, else the hyperbolic tangent for n < tanh_end; square of ReLU everywhere with
 * relu2; times `scale` when not 0.  (Gated outputs take the factor alone; `scale` is not for
 * SPLIT_GATED.) */
enum { WR_HIP_MIX_OUT_ROWS_F32 = 0, WR_HIP_MIX_OUT_ROWS = 1, WR_HIP_MIX_OUT_FRAG = 2,
       WR_HIP_MIX_OUT_SPLIT = 3, WR_HIP_MIX_OUT_GATED = 4, WR_HIP_MIX_OUT_SPLIT_GATED = 5 };
typedef struct wr_hip_mix_gemm {
    const wr_hip_mat *w;
    const void *x;
    uint32_t x_kt, x_kt_z;
    uint32_t rows;
    const int32_t *group_expert;
    uint32_t tile_groups;          /* with group_expert: groups that share an expert come in runs of this many (1 or 8) */
    uint32_t out;
    float *y_f32;
    void *y_act;
    uint32_t ldy;
    void *h;
    uint32_t h_kt, col_z;
    uint32_t n_split, silu_end, sigmoid_end, relu2;
    float scale;
    uint32_t tanh_end, gelu;
    uint32_t x_kt0;                /* first input tile of matrix 0 */
    const float *bias;
    float limit, slope, up_bias;
    const uint32_t *x_perm;        /* with group_expert and tile_groups 1: row i is row x_perm[i] of x (any row for ~0) */
    uint32_t h_kt0;                /* input tile of h where its outputs begin */
    const float *x_scale;          /* with group_expert: row i's outputs are those of x_scale[i] times its input */
} wr_hip_mix_gemm;
int wr_hip_mix_gemm_run(int f32, const wr_hip_mix_gemm *a);

/* ---- decayed linear attention ------------------------------------------------
 * Per head S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  qkv: activation-type
 * rows, row stride ld, q at column 0, k at col_k, v at col_v, head by head.
 * o_dev: 32-bit rows, row stride ldo, heads * vdim columns.  State `run` of the
 * pool, [heads][dim][vdim]; a request at position 0 starts from zero. */
int wr_hip_mix_lightning(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32,
                         uint32_t heads, uint32_t dim, uint32_t vdim, const float *decay_dev,
                         const void *qkv_dev, uint32_t ld, uint32_t col_k, uint32_t col_v,
                         float *o_dev, uint32_t ldo);
/* h (frag) = rmsnorm(o) * norm * g; g: activation-type rows. n features. */
int wr_hip_mix_gate_norm(wr_hip_mix_step *s, int f32, const float *o_dev, uint32_t ldo, uint32_t n,
                         const void *g_dev, uint32_t ldg, const float *norm_dev, float eps, void *h_dev);

/* ---- matrix-state recurrence with input-made decays -----------------------------
 * Per head a state S [dim][vdim], key channel by value column, 32-bit.  Every token
 * brings r, k, v and a decay per key channel, w = exp(-exp(z + w0)), or
 * exp(-gain * sigmoid(z + w0)) with `gain` > 0, z = w_decay . low.  Three rules:
 *   BONUS  o = (S + diag(u) k v^T)^T r;  then S <- diag(w) S + k v^T
 *   DELTA  with n = k / sqrt(k . k + unit_eps) and a = sigmoid(za + a_bias):
 *          S <- diag(w) S - (a n) (n^T S) + k v^T (old S on the right);  o = S^T r
 *   FORGET w = lower + (1 - lower) logistic(z + w0) with z the rows at col_k, k = 1 - w:
 *          S <- diag(w) S + k v^T;  o = S^T r    (no low-rank product, no gate; norm is
 *          one of vdim weights that the heads share)
 * vdim is dim but in FORGET.
 * Then each head's o is divided by its root mean square (eps), times norm, times the
 * gate (SiLU or logistic of the rows at col_g), times out_scale, and goes to h (frag,
 * h_kt tiles) at input col_h + head * dim + column; inputs up to the next multiple of
 * 32 are zeros.
 * in: 32-bit rows, stride ld; r, k, v, za, g at their columns, head by head.
 * low: frag rows of w_decay's inputs; z: room for the products, 32-bit rows of w_decay's
 * outputs (used where they are not made in passing).  State `run` of the pool; position 0 starts from zero. */
enum { WR_HIP_MIX_RULE_BONUS = 0, WR_HIP_MIX_RULE_DELTA = 1, WR_HIP_MIX_RULE_FORGET = 2 };
typedef struct wr_hip_mix_recurrence {
    uint32_t heads, dim, rule;
    float gain, unit_eps, eps, out_scale;
    uint32_t gate_silu;                       /* 1: SiLU, 0: logistic */
    const float *w0, *u, *a_bias, *norm;      /* device, heads * dim (u: BONUS, a_bias: DELTA) */
    const float *in;
    uint32_t ld, col_r, col_k, col_v, col_a, col_g;
    const wr_hip_mat *w_decay;                /* [heads * dim padded][rank padded] */
    const void *low;
    float *z;
    void *h;
    uint32_t h_kt, col_h;
    uint32_t vdim;                            /* FORGET */
    const float *lower;                       /* FORGET: device, heads * dim */
} wr_hip_mix_recurrence;
int wr_hip_mix_recur(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32,
                     const wr_hip_mix_recurrence *a);

/* ---- gated recurrence element by element ------------------------------------------
 * z = logistic of the rows at col_z, u the rows at col_x, c = u + 1/2 where u >= 0, else
 * logistic(u):  S <- (1 - z) S + z c, 32-bit;  S times SiLU of the rows at col_g goes to h
 * (frag, h_kt tiles) at input col_h.  `width` elements, padded to 32 (rows, state and
 * operand alike; the rows' pads are zeros).  State `run` of the pool; position 0 starts from zero. */
typedef struct wr_hip_mix_gru {
    uint32_t width;
    const float *in;                          /* 32-bit rows, stride ld */
    uint32_t ld, col_z, col_x, col_g;
    void *h;
    uint32_t h_kt, col_h;
} wr_hip_mix_gru;
int wr_hip_mix_min_gru(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32, const wr_hip_mix_gru *a);

/* ---- windowed attention over grouped keys and values ----------------------------
 * `heads` query heads, `kv_heads` key/value heads (query head h reads h / (heads /
 * kv_heads)), head sizes dim (queries, keys) and vdim (values), padded to dim_pad and
 * vdim_pad (wr_hip_mix_window_pad).  With maps = 2 every head has two queries and every
 * key/value head two keys, one behind the other, and both maps weigh the same values.
 * Queries and keys may be normed (each map's vector over its root mean square, times a
 * weight of dim), then the first 2 * rot_half dimensions are rotated, i with
 * i + rot_half, or with `neighbours` 2i with 2i + 1.
 * With `chunk` a row sees what came before it in its own chunk of that many positions, counted
 * from the request's first.  With turn_values, element 2m of a value is turned with element
 * 2m + 1 by the angles in that table ahead of the cache, and a head's output back by its row's.
 * Cached per position: kv_heads * (maps * dim_pad + vdim_pad) elements. */
typedef struct wr_hip_mix_window {
    uint32_t heads, kv_heads, dim, dim_pad, vdim, vdim_pad, rot_half;
    uint32_t window;               /* keys a row sees, itself included */
    float scale, out_scale;
    uint32_t norm_values;          /* values divided by their root mean square (eps) ahead of the cache */
    float eps;
    uint32_t maps;                 /* 1 or 2 */
    uint32_t neighbours;
    float softcap;                 /* > 0: scores are softcap * tanh(score / softcap) */
    float diff;                    /* maps = 2: how much of the second map's output is taken off */
    const float *q_norm, *k_norm;  /* device, dim floats each, or NULL */
    uint32_t chunk;                /* > 0: in place of the window */
    uint32_t gate_wide;            /* the gate has a logit for every output element */
    const float *turn_values;      /* device, [rows][vdim / 2][2], or NULL */
} wr_hip_mix_window;
/* The padded head size to use: what the matrix kernels take, else a multiple of 32. */
uint32_t wr_hip_mix_window_pad(uint32_t dim);
/* From 32-bit rows (stride ld): queries at col_q, normed and rotated, into q (frag, head h
 * at input h * maps * dim_pad); keys at col_k, normed and rotated, and values at col_v,
 * normed with norm_values, into the cache.  col_v may be col_k.  With col_k =
 * WR_HIP_MIX_NO_KEYS the queries alone: another layer's keys and values serve. */
#define WR_HIP_MIX_NO_KEYS 0xFFFFFFFFu
int wr_hip_mix_window_append(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32,
                             const wr_hip_mix_window *g, const float *in_dev, uint32_t ld, uint32_t col_q,
                             uint32_t col_k, uint32_t col_v, const float *table_dev, void *q_dev);
/* Softmax attention over the cached rows inside the window; with `sink`, a head's weights
 * are exp(score) / (exp(sink[head]) + sum of exp(score)).  With two maps a head's output is
 * first - diff * second, over its root mean square (eps).  Head h's output times out_scale,
 * and times logistic(gate[row * ldg + h]) where `gate` is given (with gate_wide element by
 * element, gate[row * ldg + h * vdim + column]), goes to o (frag, o_kt
 * tiles) at input h * vdim_pad. */
int wr_hip_mix_window_attend(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32,
                             const wr_hip_mix_window *g, const void *q_dev, const float *sink_dev,
                             const float *gate_dev, uint32_t ldg, void *o_dev, uint32_t o_kt);

/* ---- attention through a latent -----------------------------------------------
 * Table of (cos, sin) of position * freq[i], both times gain, for the step's rows, [rows][half][2];
 * freq: device doubles. */
int wr_hip_mix_rope_table(wr_hip_mix_step *s, const double *freq_dev, uint32_t half, float gain, float *table_dev);
/* The geometry of one attention layer.  A cached row is [rank_pad | rot_pad]. */
typedef struct wr_hip_mix_latent {
    uint32_t heads, rank, rank_pad, rot, rot_pad, rot_half;
    uint32_t window;               /* keys a row sees, itself included */
    float scale;
} wr_hip_mix_latent;
/* The rank_pad to use for a latent of `rank` elements: what the matrix kernels take
 * where they take the rank at all, else the next multiple of 32. */
uint32_t wr_hip_mix_latent_rank_pad(uint32_t rank);
/* Splits rows of d = [q latent | (pad32) | kv latent | (pad32) | rotated key part]:
 * the q latent is normed into cq (frag), the kv latent is normed and the key part
 * rotated into the cache of layer run `run`. */
int wr_hip_mix_latent_append(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32,
                             const wr_hip_mix_latent *g, const float *d_dev, uint32_t ldd,
                             uint32_t q_rank, const float *q_norm_dev, const float *kv_norm_dev,
                             float eps, const float *table_dev, void *cq_dev);
/* Rotates the heads' rotated query part (32-bit rows [rows][ldq], head by head)
 * into columns rank_pad .. of each head of q (frag, head h at input h * (rank_pad + rot_pad)). */
int wr_hip_mix_latent_qrope(wr_hip_mix_step *s, int f32, const wr_hip_mix_latent *g, const float *qr_dev,
                            uint32_t ldq, const float *table_dev, void *q_dev);
/* Softmax attention of q (frag, head h at input h * (rank_pad + rot_pad)) over
 * the cached rows of the request inside the window; the weighted latents go to o
 * (frag rows, head h at input h * rank_pad). */
int wr_hip_mix_latent_attend(wr_hip_mix_step *s, wr_hip_mix_pool *pool, uint32_t run, int f32,
                             const wr_hip_mix_latent *g, const void *q_dev, void *o_dev);

/* ---- mixture of experts ---------------------------------------------------------
 * From router logits (32-bit rows, row stride ldz) over `experts` experts and `identity`
 * outputs that pass the layer's input on: the `top` outputs with the largest choice value
 * (lowest index first among equals), their weights, and an order of the (row, choice)
 * pairs by expert: each expert's pairs take runs of tile_groups groups of 16 slots.
 * The choice value is the logit and the weights are the softmax over the chosen, or with
 * logistic their logits' logistic as it is; with
 * softmax_all it is the softmax over all outputs plus `correction`, and the weights are
 * the chosen outputs' softmax over (their sum + 1e-20), times scale.  With groups > 0 the
 * outputs form that many equal groups of neighbours, and only those of the `keep` groups
 * with the largest choice value in them can be chosen.
 * slot[r][t]: the pair's slot, ~0 for an identity output; perm: row of each slot, or ~0;
 * group_expert: expert of each group of 16 slots, or -1; side[r] (may be NULL): the sum of
 * the identity outputs' weights, and, with shared_gate, the logistic of the logit behind
 * the outputs' (else 0).
 * slot_weight (may be NULL): the weight of each slot's pair, 0 for an empty slot.
 * wr_hip_mix_route_groups: how many groups that can take at most. */
typedef struct wr_hip_mix_router {
    uint32_t experts, identity, top;
    uint32_t groups, keep;
    uint32_t softmax_all, shared_gate;
    float scale;
    const float *correction;       /* device, or NULL */
    uint32_t logistic;
} wr_hip_mix_router;
#define WR_HIP_MIX_MAX_GROUPS 64u
uint32_t wr_hip_mix_route_groups(uint32_t rows, uint32_t experts, uint32_t top, uint32_t tile_groups);
int wr_hip_mix_route(wr_hip_mix_step *s, const float *z_dev, uint32_t ldz, const wr_hip_mix_router *g,
                     uint32_t tile_groups, float *gate_dev, float *side_dev, float *slot_weight_dev, uint32_t *slot_dev,
                     uint32_t *perm_dev, int32_t *group_expert_dev);
/* The rows of h in slot order: xs (frag). */
int wr_hip_mix_route_gather(wr_hip_mix_step *s, int f32, const void *h_dev, uint32_t kt, uint32_t n_groups,
                            const uint32_t *perm_dev, const int32_t *group_expert_dev, void *xs_dev);

#ifdef __cplusplus
}
#endif
#endif /* WR_HIP_MIX_H */
