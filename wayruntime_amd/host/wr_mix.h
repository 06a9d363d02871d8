/*
 * wr_mix.h — mixer-stack models: a list of layers, each a mixer (decayed linear
 * attention, windowed attention through a latent, a matrix-state recurrence behind
 * a token shift, windowed grouped-query attention, or that and such a recurrence side
 * by side) and an optional feed-forward (dense or a mixture of experts), with norms
 * before and, in some designs, after each, or one norm whose rows both read, part of
 * the list possibly run several times.  A design (wrh_mix_design) says which of these its models use.  Read from a folder with config.json and
 * model.safetensors.  wr_mix_model.c reads and uploads, wr_mix.c keeps the cache
 * pool and walks the layers.
 */
#ifndef WR_MIX_H
#define WR_MIX_H

#include "wr_host.h"
#include "wr_json.h"
#include "../../include/wr_hip_mix.h"

typedef enum { WRH_MIXER_LIGHTNING, WRH_MIXER_LATENT, WRH_MIXER_WKV, WRH_MIXER_PARALLEL, WRH_MIXER_WINDOW,
               WRH_MIXER_JOINT } wrh_mixer_kind;
/* What stands beside a joint layer's attention. */
typedef enum { WRH_BESIDE_NOTHING, WRH_BESIDE_FORGET, WRH_BESIDE_GRU } wrh_beside_kind;
typedef enum { WRH_MLP_NONE, WRH_MLP_DENSE, WRH_MLP_MOE } wrh_mlp_kind;

/* A matrix-state recurrence: its own part of a layer's products and vectors. */
typedef struct wrh_mix_recur {
    uint32_t heads, dim, hd_p, rank_p;    /* hd = heads * dim; rank of the decay's low-rank product */
    wr_hip_mat *w_decay;                  /* [hd_p][rank_p] */
    const float *w0, *u, *a_bias, *norm;
    uint32_t vdim, hv_p;                  /* a forget gate's: values of their own size */
    const float *lower;
} wrh_mix_recur;

/* Feature counts ending in _p are padded to a multiple of 32. */
typedef struct wrh_mix_layer {
    wrh_mixer_kind kind;
    uint32_t heads, dim, vdim;
    /* lightning: one stacked product [q | k | v | g], then the output product */
    uint32_t qk_p, v_p;
    wr_hip_mat *w_qkvg, *w_o;
    const float *decay, *mix_norm;
    /* latent attention */
    uint32_t q_rank, kv_rank, q_rank_p, dim_p, vdim_p, rot_dim;
    uint32_t rope;                        /* index of the layer's rotary table */
    wr_hip_mix_latent geo;
    wr_hip_mat *w_d, *w_uq, *w_uk, *w_uv;
    const float *dq_norm, *dkv_norm;
    /* wkv: token shift, a batch of four products r, k, v, g, the decay's two; w_o */
    wrh_mix_recur rec;
    wr_hip_mat *w_rkvg, *w_low;
    const float *mu;                      /* five vectors: r, k, v, g, w */
    /* parallel: one stacked product [low | q | k | v | r | k | v | g | a], w_o over both halves' outputs */
    wr_hip_mix_window win;
    float right_scale;
    wr_hip_mat *w_in;
    uint32_t col_q, col_k, col_v, col_rr, col_rk, col_rv, col_rg, col_ra, ld_in;
    const float *sink;
    /* window: one stacked product [q | k | v | gate] (values that are the keys take no part of it), w_o */
    uint8_t has_gate;                     /* a logistic gate per head, its logits at col_rg */
    int32_t kv_from;                      /* layer whose keys and values it reads, or -1 */
    const float *b_in;                    /* a bias for every output of w_in, or NULL */
    /* joint: mixers and feed-forward read one norm.  One stacked product of the mixers' inputs and, behind n_in outputs, a
     * dense feed-forward's gate and up, or the router's logits among the rows; w_o takes out everything, or with
     * out_norm the attention alone (w_o2 what stands beside it, w_down the feed-forward), each mixer's output normed */
    wrh_beside_kind beside;
    int32_t turn;                         /* rotary table of the values, or -1 */
    uint32_t gru, gru_p;                  /* elements of the gated recurrence */
    uint32_t n_in, col_router, silu_end;        /* rows below silu_end leave the product through SiLU */
    wr_hip_mat *w_o2;
    const float *b_o, *out_norm[2];       /* (halved: the outputs are averaged) */
    /* feed-forward */
    wrh_mlp_kind mlp;
    uint8_t gelu;
    uint32_t ff, ff_p;
    wr_hip_mat *w_gu, *w_down, *w_router, *w_eup, *w_edown;
    /* experts: the router's outputs, padded (logit rows); with limit > 0 gated experts, clamped (w_eup: gate and up) */
    wr_hip_mix_router router;
    uint32_t router_p;
    uint8_t gated, weigh_input;           /* gated experts without a clamp; the weights multiply the experts' input */
    float limit;
    /* shared expert: w_router carries its gate's logit and, behind router_p rows, its gate and up; w_down takes it out */
    uint32_t shared_p;                    /* its width, or 0 */
    float shared_limit;
    const float *norm1, *norm1b, *norm2, *norm2b;
} wrh_mix_layer;

/* One run of a layer: a looped layer has several, each with its own cache or state. */
typedef struct wrh_mix_run {
    uint32_t layer;
    uint32_t store;                       /* index of its pages (attention) or state in the pool */
    uint32_t store2;                      /* parallel: state of its recurrence; wkv: the previous token's input */
    uint8_t  add_embedding;               /* the embedding output joins the residual before it */
} wrh_mix_run;

typedef struct wrh_mix_rope {
    double   base;
    uint32_t dims;
    double   factor, original, fast, slow;    /* far pairs slowed down by factor (0: none) */
    float    gain;                            /* of cosine and sine */
    double  *freq_dev;
} wrh_mix_rope;

struct wrh_mix_model {
    int      f32;                         /* 32-bit activations */
    uint32_t width, width_p, vocab, vocab_p, n_layers, n_runs, n_ropes, n_latent, n_state;
    float    eps, logit_scale, embed_scale;
    int      looped, has_shift;
    wrh_mix_layer *layers;
    wrh_mix_run   *runs;
    wrh_mix_rope  *ropes;
    uint32_t *latent_dim;                 /* per latent store */
    uint64_t *state_elems;                /* per state store */
    uint16_t *embed_dev;
    wr_hip_mat *head;
    float   *vecs;                        /* one device block for all vectors */
    const float *embed_norm, *final_norm;

    /* cache pool and scratch, made with the first session */
    pthread_mutex_t lock;                 /* a step at a time; guards everything below */
    uint32_t pool_tokens, pool_slots;     /* as asked for; 0 = default */
    wr_hip_mix_pool *pool;
    wr_hip_mix_step *step;
    uint32_t n_pages, n_free_pages, *free_pages;
    uint32_t n_slots, n_free_slots, *free_slots;
    uint32_t rows_cap;                    /* rows the scratch below is made for */
    uint8_t *scratch;
    size_t   scratch_bytes;
    float   *logits_dev, *logits_host;    /* [WRH_MIX_LOGIT_ROWS][vocab_p] */
    float   *capture;                     /* test hook: the residual rows after every run */
    size_t   capture_left;
};

#define WRH_MIX_LOGIT_ROWS 64

/* The delta rule's own constants: log w = -exp(-1/2) * logistic, unit keys over sqrt(k . k + 1e-6). */
#define WRH_DELTA_GAIN     0.60653065971263342360f
#define WRH_DELTA_UNIT_EPS 1e-6f

/* Clamped gated units: g * logistic(1.702 g) * (u + 1). */
#define WRH_CLAMPED_SLOPE   1.702f
#define WRH_CLAMPED_UP_BIAS 1.0f

typedef struct wrh_mix_session {
    uint32_t slot, buf;                   /* state slot; which of its buffers is current */
    uint32_t n_pages, *pages;
} wrh_mix_session;

wr_status wrh_mix_load(wr_engine *e, const char *dir, const char *arch, const wrh_json *cfg,
                       const wr_model_params *p, wr_model *m);
void      wrh_mix_free(struct wrh_mix_model *mm);

#endif /* WR_MIX_H */
