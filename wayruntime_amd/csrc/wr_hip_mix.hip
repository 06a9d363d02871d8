// C ABI of the mixer-stack steps (include/wr_hip_mix.h): cache pool, a step's row
// descriptors, argument checks and kernel launches.  Shares the library's device,
// thread contexts and streams with wr_hip_attn.hip; there is no CPU path.

#include <hip/hip_runtime.h>

#include <algorithm>
#include <atomic>
#include <cstring>
#include <new>
#include <vector>

#include "../../include/wr_hip_mix.h"
#include "common.hip.h"
#include "runtime.hip.h"
#include "mix_common.hip.h"
#include "kernels_mix_gemm.hip.h"
#include "kernels_mix_rows.hip.h"
#include "kernels_lightning.hip.h"
#include "kernels_latent.hip.h"
#include "kernels_latent_mfma.hip.h"
#include "kernels_recur.hip.h"
#include "kernels_window.hip.h"
#include "kernels_gru.hip.h"

using namespace wr;

static_assert(WR_HIP_MIX_PAGE == kMixPage, "page size");

struct wr_hip_mat {
    uint32_t batch, n_out, n_in;
    void* tiles;
};

struct wr_hip_mix_pool {
    int f32;
    uint32_t n_pages, n_slots;
    std::vector<uint32_t> latent_dim;
    std::vector<uint64_t> state_elems;
    std::vector<uint8_t*> latent;           // [page][64][latent_dim], operand order
    std::vector<float*> state;              // [slot][2][state_elems]
    uint8_t* block = nullptr;
    size_t bytes = 0;
};

namespace {

constexpr uint32_t kMaxRows = WR_HIP_MIX_MAX_ROWS, kMaxSeqs = WR_HIP_MIX_MAX_SEQS;
constexpr uint32_t kMaxChunks = kMaxRows / kMixChunk + kMaxSeqs;
// Requests that bring at most this many rows take the recurrence token by token.
constexpr uint32_t kStepRows = 16;
constexpr size_t kMaxLds = 160 * 1024;

size_t round256(size_t n) { return (n + 255) & ~(size_t)255; }
uint32_t round32(uint32_t n) { return (n + 31) / 32 * 32; }

}  // namespace

// One device block, filled from one pinned block of the same layout by one copy.
struct wr_hip_mix_step {
    uint32_t max_pages;
    uint8_t *host = nullptr, *dev = nullptr;
    size_t o_tokens, o_seq, o_pos, o_want, o_seqs, o_chunks, o_all, o_short, o_long, o_short_rows, o_pages, bytes;
    uint32_t rows = 0, n_seq = 0, n_want = 0, n_chunks = 0, n_short = 0, n_long = 0, n_short_rows = 0;
    uint32_t long_rows[kMaxSeqs];           // rows of each request of the long list
    Buffer chunk_state, state_frag, partial, recur_ops, recur_out, recur_segs;
    template <typename T> T* d(size_t off) const { return reinterpret_cast<T*>(dev + off); }
    template <typename T> T* h(size_t off) const { return reinterpret_cast<T*>(host + off); }
};

#define MIX_LAUNCH(kernel, grid, block, lds, ...)                                          \
    do {                                                                                   \
        kernel<<<grid, block, lds, cx->stream>>>(__VA_ARGS__);                             \
        HIP_TRY(hipGetLastError(), "mixer-stack launch", 0);                               \
    } while (0)

// A kernel that stages more than the 64 KiB it may use without asking: asked once per init.
template <auto Kernel>
static int allow_lds(size_t bytes)
{
    static std::atomic<uint64_t> asked{0};
    if (bytes <= 64 * 1024 || asked.load(std::memory_order_relaxed) == g.generation) return WR_HIP_OK;
    if (bytes > kMaxLds) return WR_HIP_ERR_LIMIT;
    HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(Kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                                (int)kMaxLds), "kernel LDS size", 0);
    asked.store(g.generation, std::memory_order_relaxed);
    return WR_HIP_OK;
}

int wr_hip_mix_available(void) { return 1; }

// ---------------------------------------------------------------- weights --

int wr_hip_mix_mat_create(uint32_t batch, uint32_t n_out, uint32_t n_in, const uint16_t* bf16, wr_hip_mat** out)
{
    if (!out) return WR_HIP_ERR_INVAL;
    *out = nullptr;
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!bf16 || batch == 0 || n_out == 0 || n_in == 0 || n_out % 16 || n_in % 32) return WR_HIP_ERR_INVAL;
    wr_hip_mat* w = new (std::nothrow) wr_hip_mat{batch, n_out, n_in, nullptr};
    if (!w) return WR_HIP_ERR_NOMEM;
    Entered entered_;
    if (!entered_.ok()) {
        delete w;
        return WR_HIP_ERR_NOMEM;
    }
    const size_t bytes = (size_t)batch * n_out * n_in * 2;
    void* rows = nullptr;
    hipError_t e = hipMalloc(&w->tiles, bytes);
    if (e == hipSuccess) e = hipMalloc(&rows, bytes);
    if (e == hipSuccess) e = hipMemcpyAsync(rows, bf16, bytes, hipMemcpyHostToDevice, cx->stream);
    if (e == hipSuccess) {
        const uint64_t units = bytes / 16;
        hipLaunchKernelGGL(mix_pack_kernel, dim3((uint32_t)((units + 255) / 256)), dim3(256), 0, cx->stream,
                           reinterpret_cast<const uint16_t*>(rows), reinterpret_cast<u32x4*>(w->tiles), units, n_in);
        e = hipGetLastError();
    }
    const hipError_t es = hipStreamSynchronize(cx->stream);
    if (e == hipSuccess) e = es;
    if (rows) (void)hipFree(rows);
    if (e != hipSuccess) {
        if (w->tiles) (void)hipFree(w->tiles);
        delete w;
        return hip_fail(e, "weight upload", 0);
    }
    *out = w;
    return WR_HIP_OK;
}

void wr_hip_mix_mat_destroy(wr_hip_mat* w)
{
    if (!w) return;
    wr_hip_attn_dev_free(w->tiles);
    delete w;
}

// ------------------------------------------------------------------- pool --

int wr_hip_mix_pool_create(int f32, uint32_t n_latent, const uint32_t* latent_dim, uint32_t n_pages, uint32_t n_state,
                           const uint64_t* state_elems, uint32_t n_slots, wr_hip_mix_pool** out)
{
    if (!out) return WR_HIP_ERR_INVAL;
    *out = nullptr;
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (n_pages == 0 || n_slots == 0 || (n_latent && !latent_dim) || (n_state && !state_elems)) return WR_HIP_ERR_INVAL;
    for (uint32_t i = 0; i < n_latent; i++)
        if (latent_dim[i] == 0 || latent_dim[i] % 32) return WR_HIP_ERR_INVAL;
    wr_hip_mix_pool* p = new (std::nothrow) wr_hip_mix_pool();
    if (!p) return WR_HIP_ERR_NOMEM;
    p->f32 = f32 != 0;
    p->n_pages = n_pages;
    p->n_slots = n_slots;
    std::vector<size_t> off;
    size_t at = 0;
    for (uint32_t i = 0; i < n_latent; i++) {
        p->latent_dim.push_back(latent_dim[i]);
        off.push_back(at);
        at += round256((size_t)n_pages * kMixPage * latent_dim[i] * (f32 ? 4 : 2));
    }
    for (uint32_t i = 0; i < n_state; i++) {
        p->state_elems.push_back(state_elems[i]);
        off.push_back(at);
        at += round256((size_t)n_slots * 2 * state_elems[i] * 4);
    }
    p->bytes = at ? at : 256;
    Entered entered_;
    hipError_t e = entered_.ok() ? hipMalloc((void**)&p->block, p->bytes) : hipErrorOutOfMemory;
    if (e == hipSuccess) e = hipMemsetAsync(p->block, 0, p->bytes, cx->stream);
    if (e == hipSuccess) e = hipStreamSynchronize(cx->stream);
    if (e != hipSuccess) {
        const size_t want = p->bytes;
        if (p->block) (void)hipFree(p->block);
        delete p;
        logmsg(0, "cache pool: %zu bytes", want);
        return hip_fail(e, "cache pool", 0);
    }
    for (uint32_t i = 0; i < n_latent; i++) p->latent.push_back(p->block + off[i]);
    for (uint32_t i = 0; i < n_state; i++) p->state.push_back(reinterpret_cast<float*>(p->block + off[n_latent + i]));
    *out = p;
    return WR_HIP_OK;
}

void wr_hip_mix_pool_destroy(wr_hip_mix_pool* p)
{
    if (!p) return;
    wr_hip_attn_dev_free(p->block);
    delete p;
}

uint64_t wr_hip_mix_pool_bytes(const wr_hip_mix_pool* p) { return p ? p->bytes : 0; }

// ------------------------------------------------------------------- step --

int wr_hip_mix_step_create(uint32_t max_pages, wr_hip_mix_step** out)
{
    if (!out) return WR_HIP_ERR_INVAL;
    *out = nullptr;
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (max_pages == 0) return WR_HIP_ERR_INVAL;
    wr_hip_mix_step* s = new (std::nothrow) wr_hip_mix_step();
    if (!s) return WR_HIP_ERR_NOMEM;
    s->max_pages = max_pages;
    size_t at = 0;
    auto take = [&](size_t bytes) {
        const size_t o = at;
        at += round256(bytes);
        return o;
    };
    s->o_tokens = take(kMaxRows * 4);
    s->o_seq = take(kMaxRows * 4);
    s->o_pos = take(kMaxRows * 4);
    s->o_want = take(kMaxRows * 4);
    s->o_seqs = take(kMaxSeqs * sizeof(MixSeq));
    s->o_chunks = take(kMaxChunks * sizeof(MixChunk));
    s->o_all = take(kMaxSeqs * 4);
    s->o_short = take(kMaxSeqs * 4);
    s->o_long = take(kMaxSeqs * 4);
    s->o_short_rows = take(kMaxSeqs * kStepRows * sizeof(LatentRow));
    s->o_pages = take((size_t)max_pages * 4);
    s->bytes = at;
    s->host = static_cast<uint8_t*>(wr_hip_attn_host_alloc(at));
    s->dev = static_cast<uint8_t*>(wr_hip_attn_dev_alloc(at));
    if (!s->host || !s->dev) {
        wr_hip_mix_step_destroy(s);
        return WR_HIP_ERR_NOMEM;
    }
    *out = s;
    return WR_HIP_OK;
}

void wr_hip_mix_step_destroy(wr_hip_mix_step* s)
{
    if (!s) return;
    wr_hip_attn_host_free(s->host);
    wr_hip_attn_dev_free(s->dev);
    wr_hip_attn_dev_free(s->chunk_state.p);
    wr_hip_attn_dev_free(s->state_frag.p);
    wr_hip_attn_dev_free(s->partial.p);
    wr_hip_attn_dev_free(s->recur_ops.p);
    wr_hip_attn_dev_free(s->recur_out.p);
    wr_hip_attn_dev_free(s->recur_segs.p);
    delete s;
}

int wr_hip_mix_step_set(wr_hip_mix_step* s, const wr_hip_mix_pool* pool, uint32_t n_seq, const wr_hip_mix_seq* seqs,
                        const uint32_t* tokens, uint32_t vocab, uint32_t n_want, const uint32_t* want_rows)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !pool || !seqs || !tokens || (n_want && !want_rows)) return WR_HIP_ERR_INVAL;
    if (n_seq == 0 || n_seq > kMaxSeqs) return WR_HIP_ERR_LIMIT;
    s->rows = 0;                                           // nothing may be launched on a step that did not check out
    uint64_t rows = 0, pages = 0;
    for (uint32_t i = 0; i < n_seq; i++) {
        const wr_hip_mix_seq& q = seqs[i];
        if (q.rows == 0 || !q.pages || q.slot >= pool->n_slots || q.buf_in > 1 || q.buf_out > 1) return WR_HIP_ERR_INVAL;
        if ((uint64_t)q.pos0 + q.rows > WR_HIP_ATTN_MAX_SEQ) return WR_HIP_ERR_LIMIT;
        if ((uint64_t)q.n_pages * kMixPage < (uint64_t)q.pos0 + q.rows) return WR_HIP_ERR_INVAL;
        for (uint32_t j = 0; j < q.n_pages; j++)
            if (q.pages[j] >= pool->n_pages) return WR_HIP_ERR_INVAL;
        for (uint32_t j = 0; j < i; j++)
            if (seqs[j].slot == q.slot) return WR_HIP_ERR_INVAL;
        rows += q.rows;
        pages += q.n_pages;
    }
    if (rows > kMaxRows || pages > s->max_pages || n_want > rows) return WR_HIP_ERR_LIMIT;
    for (uint64_t r = 0; r < rows; r++)
        if (tokens[r] >= vocab) return WR_HIP_ERR_INVAL;
    for (uint32_t i = 0; i < n_want; i++)
        if (want_rows[i] >= rows) return WR_HIP_ERR_INVAL;
    ENTER();
    uint32_t row = 0, page = 0, chunk = 0, n_short = 0, n_long = 0, short_rows = 0;
    for (uint32_t i = 0; i < n_seq; i++) {
        const wr_hip_mix_seq& q = seqs[i];
        MixSeq m;
        m.row0 = row;
        m.rows = q.rows;
        m.pos0 = q.pos0;
        m.page0 = page;
        m.state_in = q.slot * 2 + q.buf_in;
        m.state_out = q.slot * 2 + q.buf_out;
        m.chunk0 = chunk;
        m.n_chunks = 0;
        if (q.rows > kStepRows) {
            for (uint32_t at = 0; at < q.rows; at += kMixChunk, m.n_chunks++)
                s->h<MixChunk>(s->o_chunks)[chunk++] =
                    MixChunk{i, row + at, std::min(q.rows - at, kMixChunk), (uint32_t)(at == 0 && q.pos0 == 0)};
            s->long_rows[n_long] = q.rows;
            s->h<uint32_t>(s->o_long)[n_long++] = i;
        } else {
            s->h<uint32_t>(s->o_short)[n_short++] = i;
            for (uint32_t r = 0; r < q.rows; r++)
                s->h<LatentRow>(s->o_short_rows)[short_rows++] = LatentRow{row + r, q.pos0 + r, page, 0};
        }
        s->h<uint32_t>(s->o_all)[i] = i;
        s->h<MixSeq>(s->o_seqs)[i] = m;
        for (uint32_t r = 0; r < q.rows; r++) {
            s->h<uint32_t>(s->o_seq)[row + r] = i;
            s->h<uint32_t>(s->o_pos)[row + r] = q.pos0 + r;
        }
        memcpy(s->h<uint32_t>(s->o_pages) + page, q.pages, (size_t)q.n_pages * 4);
        row += q.rows;
        page += q.n_pages;
    }
    memcpy(s->h<uint32_t>(s->o_tokens), tokens, rows * 4);
    if (n_want) memcpy(s->h<uint32_t>(s->o_want), want_rows, (size_t)n_want * 4);
    HIP_TRY(hipMemcpyAsync(s->dev, s->host, s->o_pages + (size_t)page * 4, hipMemcpyHostToDevice, cx->stream),
            "step descriptors", 0);
    s->rows = (uint32_t)rows;
    s->n_seq = n_seq;
    s->n_want = n_want;
    s->n_chunks = chunk;
    s->n_short = n_short;
    s->n_long = n_long;
    s->n_short_rows = short_rows;
    return WR_HIP_OK;
}

// -------------------------------------------------------------- row steps --

static int launch_residual(int f32, bool embed, const MixRowArgs& a)
{
    const bool many = a.rows >= 64, held = a.wpad <= 4096, pair = a.pair_y[0] != nullptr;
    const dim3 g1(a.rows), b1(MixRowShape<1>::kThreads), g4((a.rows + 3) / 4), b4(MixRowShape<4>::kThreads);
#define WR_RESID(F, EMB, PAIR)                                                                   \
    do {                                                                                         \
        if (many && held)                                                                        \
            MIX_LAUNCH((mix_residual_kernel<F, 4, EMB, true, PAIR>), g4, b4, 0, a);              \
        else if (many)                                                                           \
            MIX_LAUNCH((mix_residual_kernel<F, 4, EMB, false, PAIR>), g4, b4, 0, a);             \
        else if (held)                                                                           \
            MIX_LAUNCH((mix_residual_kernel<F, 1, EMB, true, PAIR>), g1, b1, 0, a);              \
        else                                                                                     \
            MIX_LAUNCH((mix_residual_kernel<F, 1, EMB, false, PAIR>), g1, b1, 0, a);             \
    } while (0)
    if (f32 && embed) WR_RESID(true, true, false);
    else if (f32 && pair) WR_RESID(true, false, true);
    else if (f32) WR_RESID(true, false, false);
    else if (embed) WR_RESID(false, true, false);
    else if (pair) WR_RESID(false, false, true);
    else WR_RESID(false, false, false);
#undef WR_RESID
    return WR_HIP_OK;
}

int wr_hip_mix_embed(wr_hip_mix_step* s, int f32, const uint16_t* table_dev, uint32_t width, const float* norm_dev,
                     float scale, float eps, float* x_dev, float* x0_dev, const float* next_dev, void* h_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !table_dev || !width || !x_dev || (next_dev && !h_dev)) return WR_HIP_ERR_INVAL;
    ENTER();
    MixRowArgs a = {};
    a.rows = s->rows;
    a.width = width;
    a.wpad = round32(width);
    a.eps = eps;
    a.x = x_dev;
    a.x0 = x0_dev;
    a.next = next_dev;
    a.h = h_dev;
    a.table = table_dev;
    a.tokens = s->d<uint32_t>(s->o_tokens);
    a.norm = norm_dev;
    a.scale = scale;
    return launch_residual(f32, true, a);
}

int wr_hip_mix_residual(wr_hip_mix_step* s, int f32, const wr_hip_mix_resid* q)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !q || !q->width || !q->x || (q->post && !q->y) || (q->next && !q->h)) return WR_HIP_ERR_INVAL;
    if (q->top && (!q->y || !q->slot)) return WR_HIP_ERR_INVAL;
    const bool pair = q->pair_y[0] != nullptr;
    if (pair != (q->pair_y[1] != nullptr) || (pair && (!q->pair_post[0] || !q->pair_post[1]))) return WR_HIP_ERR_INVAL;
    if (q->side && !q->top) return WR_HIP_ERR_INVAL;
    if (q->wanted && (q->y || q->add || pair || !s->n_want)) return WR_HIP_ERR_INVAL;
    ENTER();
    MixRowArgs a = {};
    a.rows = q->wanted ? s->n_want : s->rows;
    a.width = q->width;
    a.wpad = round32(q->width);
    a.eps = q->eps;
    a.x = q->x;
    a.y = q->y;
    a.post = q->post;
    a.add = q->add;
    a.next = q->next;
    a.h = q->h;
    for (int i = 0; i < 2; i++) {
        a.pair_y[i] = q->pair_y[i];
        a.pair_post[i] = q->pair_post[i];
    }
    a.gate = q->gate;
    a.slot = q->slot;
    a.top = q->top;
    a.side = q->side;
    a.ident = q->ident;
    a.shared = q->shared;
    a.gather = q->wanted ? s->d<uint32_t>(s->o_want) : nullptr;
    return launch_residual(f32, false, a);
}

int wr_hip_mix_shift(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, uint32_t width, float eps,
                     const float* x_dev, const float* y_dev, float* x_out_dev, const float* norm_dev, uint32_t n_mix,
                     const float* mu_dev, void* out_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !pool || run >= pool->state.size() || !width || pool->state_elems[run] != round32(width) || !x_dev ||
        !norm_dev || !n_mix || !mu_dev || !out_dev || (y_dev && (!x_out_dev || x_out_dev == x_dev || x_out_dev == y_dev)))
        return WR_HIP_ERR_INVAL;
    ENTER();
    MixShiftArgs a = {s->d<MixSeq>(s->o_seqs), s->d<uint32_t>(s->o_seq), s->rows, width, round32(width), n_mix, eps, x_dev, y_dev,
                      norm_dev, mu_dev, x_out_dev, pool->state[run], out_dev};
    const bool many = s->rows >= 64, held = a.wpad <= 4096;
    const dim3 g1(s->rows), b1(MixRowShape<1>::kThreads), g4((s->rows + 3) / 4), b4(MixRowShape<4>::kThreads);
    if (f32) {                                             // (not the serving form: two shapes do)
        if (many) MIX_LAUNCH((mix_shift_kernel<true, 4, false>), g4, b4, 0, a);
        else MIX_LAUNCH((mix_shift_kernel<true, 1, false>), g1, b1, 0, a);
    } else if (many) {
        if (held) MIX_LAUNCH((mix_shift_kernel<false, 4, true>), g4, b4, 0, a);
        else MIX_LAUNCH((mix_shift_kernel<false, 4, false>), g4, b4, 0, a);
    } else {
        if (held) MIX_LAUNCH((mix_shift_kernel<false, 1, true>), g1, b1, 0, a);
        else MIX_LAUNCH((mix_shift_kernel<false, 1, false>), g1, b1, 0, a);
    }
    return WR_HIP_OK;
}

// --------------------------------------------------------------- products --

template <bool F32, int NT, int GR>
static int launch_stream(const MixGemmArgs& a, uint32_t batch)
{
    launch_main(mix_gemm_stream_kernel<F32, NT, GR>, dim3((a.ntiles + NT - 1) / NT, (a.groups + GR - 1) / GR, batch),
                dim3(256), a);
    HIP_TRY(hipGetLastError(), "product launch", 0);
    return WR_HIP_OK;
}

template <int GROUPS>
static int launch_lds(const MixGemmArgs& a, uint32_t batch)
{
    int rc = allow_lds<mix_gemm_lds_kernel<GROUPS>>(mix_gemm_lds_bytes<GROUPS>());
    if (rc) return rc;
    const uint32_t nx = (a.ntiles + 7) / 8, share = nx < 8 ? nx : (nx + 7) / 8 * 8;
    launch_main(mix_gemm_lds_kernel<GROUPS>, dim3(share * ((a.groups + 2 * GROUPS - 1) / (2 * GROUPS)), batch), dim3(256), a,
                mix_gemm_lds_bytes<GROUPS>());
    HIP_TRY(hipGetLastError(), "product launch", 0);
    return WR_HIP_OK;
}

int wr_hip_mix_gemm_run(int f32, const wr_hip_mix_gemm* q)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!q || !q->w || !q->x || !q->rows) return WR_HIP_ERR_INVAL;
    const uint32_t ktiles = q->w->n_in / 32, batch = q->group_expert ? 1 : q->w->batch;
    if ((uint64_t)q->x_kt0 + (uint64_t)q->x_kt_z * (batch - 1) + ktiles > q->x_kt) return WR_HIP_ERR_INVAL;
    const bool split_gated = q->out == WR_HIP_MIX_OUT_SPLIT_GATED, gated = q->out == WR_HIP_MIX_OUT_GATED || split_gated;
    const bool frag = q->out == WR_HIP_MIX_OUT_FRAG || q->out == WR_HIP_MIX_OUT_SPLIT || gated;
    if (q->out > WR_HIP_MIX_OUT_SPLIT_GATED || (frag && !q->h)) return WR_HIP_ERR_INVAL;
    if (split_gated && (q->n_split % 32 || q->n_split > q->w->n_out || batch != 1 || q->group_expert)) return WR_HIP_ERR_INVAL;
    const uint32_t n_frag = q->out == WR_HIP_MIX_OUT_SPLIT ? q->n_split
                            : gated ? (q->w->n_out - (split_gated ? q->n_split : 0)) / 2 : q->w->n_out;
    if (frag && ((uint64_t)q->h_kt0 * 32 + (uint64_t)q->col_z * (batch - 1) + n_frag > (uint64_t)q->h_kt * 32)) return WR_HIP_ERR_INVAL;
    if (q->out == WR_HIP_MIX_OUT_SPLIT && (q->n_split % 16 || q->n_split > q->w->n_out)) return WR_HIP_ERR_INVAL;
    if (gated && q->w->n_out % 32) return WR_HIP_ERR_INVAL;
    const bool rows32 = q->out == WR_HIP_MIX_OUT_ROWS_F32 || (q->out == WR_HIP_MIX_OUT_SPLIT && q->n_split < q->w->n_out) || split_gated;
    const uint32_t n_rows = q->out == WR_HIP_MIX_OUT_SPLIT ? q->w->n_out - q->n_split : split_gated ? q->n_split : q->w->n_out;
    if (rows32 && (!q->y_f32 || q->ldy % 4 || q->ldy < n_rows)) return WR_HIP_ERR_INVAL;
    if (q->out == WR_HIP_MIX_OUT_ROWS_F32 && batch > 1 && (q->col_z % 4 || (uint64_t)q->col_z * (batch - 1) + n_rows > q->ldy))
        return WR_HIP_ERR_INVAL;
    if (q->out == WR_HIP_MIX_OUT_ROWS && (!q->y_act || q->ldy % 8 || q->ldy < n_rows)) return WR_HIP_ERR_INVAL;
    if (((q->out == WR_HIP_MIX_OUT_ROWS_F32 && !q->col_z) || q->out == WR_HIP_MIX_OUT_ROWS) && batch != 1) return WR_HIP_ERR_INVAL;
    if (q->group_expert && (q->rows % 16 || (q->tile_groups != 1 && q->tile_groups != 8))) return WR_HIP_ERR_INVAL;
    if (q->group_expert && q->rows / 16 % q->tile_groups) return WR_HIP_ERR_INVAL;
    if (q->bias && (batch != 1 || q->out == WR_HIP_MIX_OUT_GATED || q->group_expert)) return WR_HIP_ERR_INVAL;
    if (q->x_scale && !q->group_expert) return WR_HIP_ERR_INVAL;
    if (q->x_perm && (!q->group_expert || q->tile_groups != 1)) return WR_HIP_ERR_INVAL;
    ENTER();
    MixGemmArgs a = {};
    a.w = reinterpret_cast<const bf16x8*>(q->w->tiles);
    a.x = static_cast<const uint8_t*>(q->x) + (size_t)q->x_kt0 * 512 * (f32 ? 4 : 2);
    a.ntiles = q->w->n_out / 16;
    a.ktiles = ktiles;
    a.x_kt = q->x_kt;
    a.x_kt_z = q->x_kt_z;
    a.rows = q->rows;
    a.groups = (q->rows + 15) / 16;
    a.group_expert = q->group_expert;
    a.out = q->out;
    a.ldy = q->ldy;
    a.h_kt = q->h_kt;
    a.col_z = q->col_z;
    a.n_split = q->n_split;
    a.silu_end = q->silu_end;
    a.sigmoid_end = std::max(q->sigmoid_end, q->silu_end);
    a.tanh_end = q->tanh_end;
    a.relu2 = q->relu2;
    a.gelu = q->gelu;
    a.scale = q->scale;
    a.limit = q->limit;
    a.slope = q->slope;
    a.up_bias = q->up_bias;
    a.bias = q->bias;
    a.x_perm = q->x_perm;
    a.x_scale = q->x_scale;
    a.y = q->y_f32;
    a.ya = q->y_act;
    a.h = frag ? static_cast<uint8_t*>(q->h) + (size_t)q->h_kt0 * 512 * (f32 ? 4 : 2) : q->h;
    if (q->group_expert) {
        if (!f32 && q->tile_groups == 8) return launch_lds<4>(a, 1);
        if (f32) return gated ? launch_stream<true, 2, 1>(a, 1) : launch_stream<true, 1, 1>(a, 1);
        return gated ? launch_stream<false, 2, 1>(a, 1) : launch_stream<false, 1, 1>(a, 1);
    }
    if (f32) {
        if (a.groups <= 1) return gated ? launch_stream<true, 2, 1>(a, batch) : launch_stream<true, 1, 1>(a, batch);
        return launch_stream<true, 2, 2>(a, batch);
    }
    if (a.groups >= 4) {
        // the largest tile that still gives every compute unit a workgroup; over a short input range a smaller
        // one, of which a unit holds three: most of such a launch is its ends
        const uint64_t panels = (uint64_t)(a.ntiles + 7) / 8 * batch;
        if (a.ktiles > 16 && panels * ((a.groups + 15) / 16) >= 256) return launch_lds<8>(a, batch);
        if (panels * ((a.groups + 7) / 8) >= 256) return launch_lds<4>(a, batch);
        if (panels * ((a.groups + 3) / 4) >= 256) return launch_lds<2>(a, batch);
        const uint64_t tiles44 = (uint64_t)((a.ntiles + 3) / 4) * ((a.groups + 3) / 4) * batch;
        if (tiles44 >= 256) return launch_stream<false, 4, 4>(a, batch);
        if (tiles44 >= 64) return launch_stream<false, 2, 4>(a, batch);
        return gated ? launch_stream<false, 2, 1>(a, batch) : launch_stream<false, 1, 1>(a, batch);
    }
    if (a.groups >= 2) return launch_stream<false, 2, 2>(a, batch);
    // a short input range: more outputs per workgroup, or the launch is all workgroups and no work
    if (!gated && a.ktiles <= 8 && a.ntiles % 4 == 0 && a.ntiles * batch >= 1024) return launch_stream<false, 4, 1>(a, batch);
    return gated || a.ntiles * batch >= 4096 ? launch_stream<false, 2, 1>(a, batch) : launch_stream<false, 1, 1>(a, batch);
}

// -------------------------------------------------------------- lightning --

template <bool F32>
static int lightning_steps(const LightningArgs& a, uint32_t n)
{
    if (n == 0) return WR_HIP_OK;
    const dim3 grid(n, a.heads, (a.vdim + 63) / 64), block(256);
    if (a.dim <= 32) MIX_LAUNCH((lightning_step_kernel<F32, 8>), grid, block, 0, a);
    else if (a.dim <= 64) MIX_LAUNCH((lightning_step_kernel<F32, 16>), grid, block, 0, a);
    else if (a.dim <= 128) MIX_LAUNCH((lightning_step_kernel<F32, 32>), grid, block, 0, a);
    else if (a.dim <= 256) MIX_LAUNCH((lightning_step_kernel<F32, 64>), grid, block, 0, a);
    else MIX_LAUNCH((lightning_step_kernel<F32, 128>), grid, block, 0, a);
    return WR_HIP_OK;
}

template <bool F32>
static int lightning_chunks(const LightningArgs& a, uint32_t n_chunks, uint32_t n_long)
{
    const dim3 grid(n_chunks, a.heads, (a.vdim + kLightSlice - 1) / kLightSlice), block(256);
    const size_t l1 = lightning_state_lds(a.dim, a.vdim), l3 = lightning_out_lds(a.dim, a.vdim);
    int rc = allow_lds<lightning_chunk_state_kernel<F32>>(l1);
    if (rc == WR_HIP_OK) rc = allow_lds<lightning_chunk_out_kernel<F32>>(l3);
    if (rc) return rc;
    MIX_LAUNCH(lightning_chunk_state_kernel<F32>, grid, block, l1, a);
    const size_t elems = (size_t)a.heads * a.dim * a.vdim;
    MIX_LAUNCH(lightning_scan_kernel, dim3(n_long, (uint32_t)((elems + 255) / 256)), block, 0, a);
    MIX_LAUNCH(lightning_chunk_out_kernel<F32>, grid, block, l3, a);
    return WR_HIP_OK;
}

template <int KT>
static int lightning_chunks_bf16(wr_hip_mix_step* s, const LightningArgs& a)
{
    LightFragArgs q = {a, nullptr, (a.vdim + 31) / 32 * 2};
    int rc = ensure_device(s->state_frag, (size_t)s->n_chunks * a.heads * KT * q.vt * 2 * 1024);
    if (rc) return rc;
    q.frag = reinterpret_cast<bf16x8*>(s->state_frag.p);
    const dim3 grid(s->n_chunks, a.heads, (a.vdim + kLightSlice - 1) / kLightSlice), block(256);
    MIX_LAUNCH(lightning_state_bf16_kernel<KT>, grid, block, 0, q);
    const uint32_t threads = a.heads * KT * 4 * q.vt * 16;
    MIX_LAUNCH(lightning_scan_bf16_kernel<KT>, dim3(s->n_long, (threads + 255) / 256), block, 0, q);
    MIX_LAUNCH(lightning_out_bf16_kernel<KT>, grid, block, 0, q);
    return WR_HIP_OK;
}

int wr_hip_mix_lightning(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, uint32_t heads, uint32_t dim,
                         uint32_t vdim, const float* decay_dev, const void* qkv_dev, uint32_t ld, uint32_t col_k,
                         uint32_t col_v, float* o_dev, uint32_t ldo)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !pool || run >= pool->state.size() || !heads || !dim || !vdim || !decay_dev || !qkv_dev || !o_dev)
        return WR_HIP_ERR_INVAL;
    if (dim > WR_HIP_MIX_MAX_STATE_DIM) return WR_HIP_ERR_LIMIT;
    if ((uint64_t)heads * dim * vdim != pool->state_elems[run]) return WR_HIP_ERR_INVAL;
    const uint64_t hd = (uint64_t)heads * dim, hv = (uint64_t)heads * vdim;
    if (hd > ld || col_k + hd > ld || col_v + hv > ld || hv > ldo) return WR_HIP_ERR_INVAL;
    ENTER();
    LightningArgs a = {};
    a.seqs = s->d<MixSeq>(s->o_seqs);
    a.chunks = s->d<MixChunk>(s->o_chunks);
    a.heads = heads;
    a.dim = dim;
    a.vdim = vdim;
    a.ld = ld;
    a.col_k = col_k;
    a.col_v = col_v;
    a.ldo = ldo;
    a.decay = decay_dev;
    a.qkv = qkv_dev;
    a.o = o_dev;
    a.state = pool->state[run];
    const bool chunked = s->n_long && dim <= (uint32_t)kLightMaxDim;
    int rc;
    if (chunked) {
        rc = ensure_device(s->chunk_state, (size_t)s->n_chunks * heads * dim * vdim * 4);
        if (rc) return rc;
        a.chunk_state = reinterpret_cast<float*>(s->chunk_state.p);
        a.list = s->d<uint32_t>(s->o_long);
        // bfloat16 operands are loaded eight at a time, also past a head's last column
        const bool bf16 = !f32 && !g.force_generic && dim % 8 == 0 && vdim % 8 == 0 && col_k % 8 == 0 && col_v % 8 == 0 &&
                          ld % 8 == 0 && ldo % 4 == 0 && hd + 32 <= ld && col_k + hd + 32 <= ld && col_v + hv + 32 <= ld;
        if (f32) rc = lightning_chunks<true>(a, s->n_chunks, s->n_long);
        else if (!bf16) rc = lightning_chunks<false>(a, s->n_chunks, s->n_long);
        else if (dim <= 32) rc = lightning_chunks_bf16<1>(s, a);
        else if (dim <= 64) rc = lightning_chunks_bf16<2>(s, a);
        else rc = lightning_chunks_bf16<4>(s, a);
        if (rc) return rc;
    }
    a.list = s->d<uint32_t>(chunked ? s->o_short : s->o_all);
    const uint32_t n = chunked ? s->n_short : s->n_seq;
    return f32 ? lightning_steps<true>(a, n) : lightning_steps<false>(a, n);
}

int wr_hip_mix_gate_norm(wr_hip_mix_step* s, int f32, const float* o_dev, uint32_t ldo, uint32_t n, const void* g_dev,
                         uint32_t ldg, const float* norm_dev, float eps, void* h_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    const uint32_t npad = round32(n);
    if (!s || !s->rows || !o_dev || !n || !g_dev || !norm_dev || !h_dev || ldo < npad || ldg < npad || ldo % 4 || ldg % 8)
        return WR_HIP_ERR_INVAL;
    ENTER();
    MixGateNormArgs a = {s->rows, n, npad, ldo, ldg, eps, o_dev, norm_dev, g_dev, h_dev};
    if (s->rows >= 64) {
        const dim3 grid((s->rows + 3) / 4), block(MixRowShape<4>::kThreads);
        if (f32) MIX_LAUNCH((mix_gate_norm_kernel<true, 4>), grid, block, 0, a);
        else MIX_LAUNCH((mix_gate_norm_kernel<false, 4>), grid, block, 0, a);
    } else {
        const dim3 grid(s->rows), block(MixRowShape<1>::kThreads);
        if (f32) MIX_LAUNCH((mix_gate_norm_kernel<true, 1>), grid, block, 0, a);
        else MIX_LAUNCH((mix_gate_norm_kernel<false, 1>), grid, block, 0, a);
    }
    return WR_HIP_OK;
}

// ------------------------------------------------------------- recurrence --

template <bool F32, bool DELTA>
static int recur_steps(const RecurArgs& a, uint32_t n)
{
    if (n == 0) return WR_HIP_OK;
    const dim3 grid(n, a.heads);
    if (a.dim <= 16) MIX_LAUNCH((recur_step_kernel<F32, 16, DELTA>), grid, dim3(64), 0, a);
    else if (a.dim <= 32) MIX_LAUNCH((recur_step_kernel<F32, 32, DELTA>), grid, dim3(128), 0, a);
    else if (a.dim <= 64) MIX_LAUNCH((recur_step_kernel<F32, 64, DELTA>), grid, dim3(256), 0, a);
    else if (a.dim <= 128) MIX_LAUNCH((recur_step_kernel<F32, 128, DELTA>), grid, dim3(512), 0, a);
    else MIX_LAUNCH((recur_step_kernel<F32, 256, DELTA>), grid, dim3(1024), 0, a);
    return WR_HIP_OK;
}

constexpr uint32_t kSegMax = 8, kSegSubs = 6;

template <bool F32, int KT, int RULE, int VT>
static int recur_chunks(wr_hip_mix_step* s, RecurArgs& a)
{
    constexpr bool DELTA = RULE == kRecurDelta;
    // FORGET: the value columns in slices of VT tiles, a workgroup each
    const uint32_t slices = RULE == kRecurForget ? (a.vdim + 16 * VT - 1) / (16 * VT) : 1;
    a.vtiles = VT * slices;
    constexpr size_t unit = (size_t)recur_unit_kib(KT, DELTA, VT) * 1024;
    int rc = ensure_device(s->recur_ops, (size_t)s->n_chunks * kRecurSubs * a.heads * recur_unit_kib(KT, DELTA, a.vtiles) * 1024);
    if (rc == WR_HIP_OK) rc = ensure_device(s->recur_out, (size_t)s->n_chunks * kMixChunk * a.heads * a.vtiles * 16 * 4);
    constexpr size_t l1 = (size_t)4 * recur_chunk_lds(KT, DELTA) * 4, l2 = recur_ring(KT, DELTA) * unit;
    constexpr size_t l3 = l2 - (size_t)recur_ring(KT, DELTA) * RecurUnit<KT, DELTA>::kG * 1024;      // without the outputs' part
    if (rc == WR_HIP_OK) rc = allow_lds<recur_chunk_kernel<F32, KT, RULE>>(l1);
    if (rc == WR_HIP_OK) rc = allow_lds<recur_chain_kernel<F32, KT, DELTA, VT, false>>(l2);
    if (rc == WR_HIP_OK) rc = allow_lds<recur_chain_kernel<F32, KT, DELTA, VT, true>>(l2);
    if (rc) return rc;
    uint32_t longest = 0;
    for (uint32_t i = 0; i < s->n_long; i++) longest = std::max(longest, (s->long_rows[i] + kRecurSub - 1) / kRecurSub);
    // Segments: as many as give every compute unit a walk (below three the two walks cost more than one), none shorter
    // than kSegSubs.
    a.n_seg = std::min({(uint32_t)g.n_cus / (s->n_long * a.heads * slices), longest / kSegSubs, kSegMax});
    if (a.n_seg < 3) a.n_seg = 1;
    a.seg_len = (longest + a.n_seg - 1) / a.n_seg;
    if (a.n_seg > 1) {
        const size_t c = (size_t)32 * KT * 16 * a.vtiles, x = DELTA ? (size_t)32 * KT * 32 * KT : 32 * KT;
        const size_t items = (size_t)s->n_long * a.n_seg * a.heads;
        rc = ensure_device(s->recur_segs, items * (c + x) * 4);
        if (rc) return rc;
        a.seg_c = reinterpret_cast<float*>(s->recur_segs.p);
        a.seg_x = a.seg_c + items * c;
    }
    a.ops = reinterpret_cast<unsigned char*>(s->recur_ops.p);
    a.o = reinterpret_cast<float*>(s->recur_out.p);
    const uint32_t whole = !((a.dim | a.ld | a.ldz | a.col_r | a.col_k | a.col_a) % 4);
    MIX_LAUNCH((recur_chunk_kernel<F32, KT, RULE>), dim3(s->n_chunks, a.heads), dim3(256), l1, a, whole);
    if (a.n_seg > 1)
        MIX_LAUNCH((recur_chain_kernel<F32, KT, DELTA, VT, true>), dim3(s->n_long * (a.n_seg - 1), a.heads, DELTA ? 2 : slices),
                   dim3(64 * VT), l3, a);
    MIX_LAUNCH((recur_chain_kernel<F32, KT, DELTA, VT, false>), dim3(s->n_long * a.n_seg, a.heads, slices), dim3(64 * VT), l2, a);
    MIX_LAUNCH(recur_gate_kernel<F32>, dim3(s->n_chunks, a.heads), dim3(256), 0, a);
    return WR_HIP_OK;
}

// Ranks (in tiles of 32) up to which a decoded token's decays are made in passing.
constexpr uint32_t kDecayTiles = 4;

template <bool F32, bool DELTA>
static int recur_run(wr_hip_mix_step* s, RecurArgs& a, const wr_hip_mix_recurrence* q)
{
    const bool chunked = s->n_long && a.dim <= (uint32_t)kRecurMaxDim;
    if (!s->n_long && a.low_kt <= kDecayTiles) {
        a.wd = reinterpret_cast<const bf16x8*>(q->w_decay->tiles);
        a.low = q->low;
    } else {
        wr_hip_mix_gemm d = {};
        d.w = q->w_decay;
        d.x = q->low;
        d.x_kt = a.low_kt;
        d.rows = s->rows;
        d.out = WR_HIP_MIX_OUT_ROWS_F32;
        d.y_f32 = q->z;
        d.ldy = a.ldz;
        const int rc = wr_hip_mix_gemm_run(F32, &d);
        if (rc) return rc;
    }
    if (chunked) {
        a.list = s->d<uint32_t>(s->o_long);
        int rc;
        constexpr int RULE = DELTA ? kRecurDelta : kRecurBonus;
        if (a.dim <= 16) rc = recur_chunks<F32, 1, RULE, 1>(s, a);
        else if (a.dim <= 32) rc = recur_chunks<F32, 1, RULE, 2>(s, a);
        else if (a.dim <= 64) rc = recur_chunks<F32, 2, RULE, 4>(s, a);
        else rc = recur_chunks<F32, 4, RULE, 8>(s, a);
        if (rc) return rc;
    }
    a.list = s->d<uint32_t>(chunked ? s->o_short : s->o_all);
    return recur_steps<F32, DELTA>(a, chunked ? s->n_short : s->n_seq);
}

template <bool F32, int DPT>
static int forget_steps_v(const RecurArgs& a, uint32_t n)
{
    const dim3 grid(n, a.heads);
    if (a.vdim <= 32) MIX_LAUNCH((recur_forget_step_kernel<F32, DPT, 32>), grid, dim3(128), 0, a);
    else if (a.vdim <= 64) MIX_LAUNCH((recur_forget_step_kernel<F32, DPT, 64>), grid, dim3(256), 0, a);
    else if (a.vdim <= 128) MIX_LAUNCH((recur_forget_step_kernel<F32, DPT, 128>), grid, dim3(512), 0, a);
    else MIX_LAUNCH((recur_forget_step_kernel<F32, DPT, 256>), grid, dim3(1024), 0, a);
    return WR_HIP_OK;
}

template <bool F32, int KT>
static int forget_chunks(wr_hip_mix_step* s, RecurArgs& a)
{
    return a.vdim <= 32 ? recur_chunks<F32, KT, kRecurForget, 2>(s, a) : recur_chunks<F32, KT, kRecurForget, 4>(s, a);
}

template <bool F32>
static int forget_run(wr_hip_mix_step* s, RecurArgs& a)
{
    const bool chunked = s->n_long && a.dim <= (uint32_t)kRecurMaxDim;
    if (chunked) {
        a.list = s->d<uint32_t>(s->o_long);
        const int rc = a.dim <= 32 ? forget_chunks<F32, 1>(s, a) : a.dim <= 64 ? forget_chunks<F32, 2>(s, a) : forget_chunks<F32, 4>(s, a);
        if (rc) return rc;
    }
    a.list = s->d<uint32_t>(chunked ? s->o_short : s->o_all);
    const uint32_t n = chunked ? s->n_short : s->n_seq;
    if (n == 0) return WR_HIP_OK;
    if (a.dim <= 32) return forget_steps_v<F32, 8>(a, n);
    if (a.dim <= 64) return forget_steps_v<F32, 16>(a, n);
    if (a.dim <= 128) return forget_steps_v<F32, 32>(a, n);
    return forget_steps_v<F32, 64>(a, n);
}

int wr_hip_mix_recur(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, const wr_hip_mix_recurrence* q)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !pool || run >= pool->state.size() || !q || !q->heads || !q->dim || !q->w0 || !q->norm || !q->in ||
        !q->h || q->rule > WR_HIP_MIX_RULE_FORGET)
        return WR_HIP_ERR_INVAL;
    const bool delta = q->rule == WR_HIP_MIX_RULE_DELTA, forget = q->rule == WR_HIP_MIX_RULE_FORGET;
    if (delta ? !q->a_bias : forget ? !q->lower || !q->vdim : !q->u) return WR_HIP_ERR_INVAL;
    if (!forget && (!q->w_decay || !q->low || !q->z)) return WR_HIP_ERR_INVAL;
    const uint32_t vdim = forget ? q->vdim : q->dim;
    if (q->dim > WR_HIP_MIX_MAX_RECUR_DIM || vdim > WR_HIP_MIX_MAX_RECUR_DIM) return WR_HIP_ERR_LIMIT;
    const uint64_t hd = (uint64_t)q->heads * q->dim, hv = (uint64_t)q->heads * vdim;
    if (hd * vdim != pool->state_elems[run]) return WR_HIP_ERR_INVAL;
    if (q->col_r + hd > q->ld || q->col_k + hd > q->ld || q->col_v + hv > q->ld || (!forget && q->col_g + hd > q->ld) ||
        (delta && q->col_a + hd > q->ld) || q->col_h + (hv + 31) / 32 * 32 > (uint64_t)q->h_kt * 32)
        return WR_HIP_ERR_INVAL;
    if (!forget && (q->w_decay->batch != 1 || q->w_decay->n_out < hd)) return WR_HIP_ERR_INVAL;
    ENTER();
    RecurArgs a = {};
    a.seqs = s->d<MixSeq>(s->o_seqs);
    a.chunks = s->d<MixChunk>(s->o_chunks);
    a.heads = q->heads;
    a.dim = q->dim;
    a.vdim = vdim;
    a.gate = forget ? kRecurGateNone : q->gate_silu ? kRecurGateSilu : kRecurGateLogistic;
    a.norm_step = forget ? 0 : vdim;
    a.gain = q->gain;
    a.unit_eps = q->unit_eps;
    a.eps = q->eps;
    a.out_scale = q->out_scale;
    a.w0 = q->w0;
    a.u = forget ? q->lower : q->u;
    a.ab = q->a_bias;
    a.norm = q->norm;
    a.in = q->in;
    a.ld = q->ld;
    a.col_r = q->col_r;
    a.col_k = q->col_k;
    a.col_v = q->col_v;
    a.col_a = delta ? q->col_a : 0;
    a.col_g = forget ? 0 : q->col_g;
    a.z = forget ? q->in + q->col_k : q->z;
    a.ldz = forget ? q->ld : q->w_decay->n_out;
    a.low_kt = forget ? 0 : q->w_decay->n_in / 32;
    a.state = pool->state[run];
    a.h = q->h;
    a.h_kt = q->h_kt;
    a.col_h = q->col_h;
    if (forget) return f32 ? forget_run<true>(s, a) : forget_run<false>(s, a);
    if (f32) return delta ? recur_run<true, true>(s, a, q) : recur_run<true, false>(s, a, q);
    return delta ? recur_run<false, true>(s, a, q) : recur_run<false, false>(s, a, q);
}

int wr_hip_mix_min_gru(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, const wr_hip_mix_gru* q)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !pool || run >= pool->state.size() || !q || !q->width || !q->in || !q->h) return WR_HIP_ERR_INVAL;
    const uint32_t wp = round32(q->width);
    if (pool->state_elems[run] != wp || (q->ld | q->col_z | q->col_x | q->col_g) % 4 || q->col_h % 8 ||
        (uint64_t)std::max({q->col_z, q->col_x, q->col_g}) + wp > q->ld || (uint64_t)q->col_h + wp > (uint64_t)q->h_kt * 32)
        return WR_HIP_ERR_INVAL;
    ENTER();
    GruArgs a = {s->d<MixSeq>(s->o_seqs), s->d<uint32_t>(s->o_long), wp, q->in, q->ld, q->col_z, q->col_x, q->col_g,
                 pool->state[run], q->h, q->h_kt, q->col_h};
    if (s->n_long) {
        const dim3 grid(wp / 16, s->n_long);
        const bool many = *std::max_element(s->long_rows, s->long_rows + s->n_long) > 64;
        if (many && f32) MIX_LAUNCH((gru_scan_kernel<true, 16>), grid, dim3(1024), 0, a);
        else if (many) MIX_LAUNCH((gru_scan_kernel<false, 16>), grid, dim3(1024), 0, a);
        else if (f32) MIX_LAUNCH((gru_scan_kernel<true, 4>), grid, dim3(256), 0, a);
        else MIX_LAUNCH((gru_scan_kernel<false, 4>), grid, dim3(256), 0, a);
    }
    if (s->n_short) {
        a.list = s->d<uint32_t>(s->o_short);
        const dim3 grid(wp / 16, s->n_short);
        if (f32) MIX_LAUNCH((gru_scan_kernel<true, 1>), grid, dim3(64), 0, a);
        else MIX_LAUNCH((gru_scan_kernel<false, 1>), grid, dim3(64), 0, a);
    }
    return WR_HIP_OK;
}

// ----------------------------------------------------------------- latent --

uint32_t wr_hip_mix_latent_rank_pad(uint32_t rank)
{
    for (uint32_t p = 64; p <= 512; p *= 2)
        if (rank <= p) return p;
    return round32(rank);
}

static int check_latent(const wr_hip_mix_latent* q)
{
    if (!q || !q->heads || !q->rank || q->rank_pad % 32 || q->rot_pad % 32 || q->rank > q->rank_pad || q->rot > q->rot_pad ||
        q->rot_half * 2 > q->rot || !q->window)
        return WR_HIP_ERR_INVAL;
    return WR_HIP_OK;
}

static LatentArgs latent_args(const wr_hip_mix_step* s, const wr_hip_mix_latent* q)
{
    LatentArgs a = {};
    a.seqs = s->d<MixSeq>(s->o_seqs);
    a.row_seq = s->d<uint32_t>(s->o_seq);
    a.row_pos = s->d<uint32_t>(s->o_pos);
    a.pages = s->d<uint32_t>(s->o_pages);
    a.rows = s->rows;
    a.heads = q->heads;
    a.rank = q->rank;
    a.rank_pad = q->rank_pad;
    a.rot = q->rot;
    a.rot_pad = q->rot_pad;
    a.half = q->rot_half;
    a.window = q->window;
    a.scale = q->scale;
    return a;
}

int wr_hip_mix_rope_table(wr_hip_mix_step* s, const double* freq_dev, uint32_t half, float gain, float* table_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !freq_dev || !half || !table_dev) return WR_HIP_ERR_INVAL;
    ENTER();
    MIX_LAUNCH(mix_rope_table_kernel, dim3((s->rows * half + 255) / 256), dim3(256), 0, s->d<uint32_t>(s->o_pos), s->rows,
               freq_dev, half, gain, table_dev);
    return WR_HIP_OK;
}

int wr_hip_mix_latent_append(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, const wr_hip_mix_latent* q,
                             const float* d_dev, uint32_t ldd, uint32_t q_rank, const float* q_norm_dev,
                             const float* kv_norm_dev, float eps, const float* table_dev, void* cq_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    int rc = check_latent(q);
    if (rc) return rc;
    if (!s || !s->rows || !pool || run >= pool->latent.size() || pool->latent_dim[run] != q->rank_pad + q->rot_pad ||
        pool->f32 != (f32 != 0) || !d_dev || !q_rank || !q_norm_dev || !kv_norm_dev || (q->rot_half && !table_dev) || !cq_dev ||
        ldd < round32(q_rank) + round32(q->rank) + q->rot)
        return WR_HIP_ERR_INVAL;
    ENTER();
    LatentArgs a = latent_args(s, q);
    a.cache = pool->latent[run];
    a.d = d_dev;
    a.ldd = ldd;
    a.q_rank = q_rank;
    a.q_norm = q_norm_dev;
    a.kv_norm = kv_norm_dev;
    a.eps = eps;
    a.table = table_dev;
    a.cq = cq_dev;
    if (f32) MIX_LAUNCH(latent_append_kernel<true>, dim3(s->rows), dim3(256), 0, a);
    else MIX_LAUNCH(latent_append_kernel<false>, dim3(s->rows), dim3(256), 0, a);
    return WR_HIP_OK;
}

int wr_hip_mix_latent_qrope(wr_hip_mix_step* s, int f32, const wr_hip_mix_latent* q, const float* qr_dev, uint32_t ldq,
                            const float* table_dev, void* q_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    int rc = check_latent(q);
    if (rc) return rc;
    if (!s || !s->rows || !qr_dev || ldq < q->heads * q->rot || (q->rot_half && !table_dev) || !q_dev) return WR_HIP_ERR_INVAL;
    if (q->rot_pad == 0) return WR_HIP_OK;
    ENTER();
    LatentArgs a = latent_args(s, q);
    a.qr = qr_dev;
    a.ldq = ldq;
    a.table = table_dev;
    a.q_out = q_dev;
    const uint32_t n = s->rows * q->heads * (q->rot_pad / 8);
    if (f32) MIX_LAUNCH(latent_qrope_kernel<true>, dim3((n + 255) / 256), dim3(256), 0, a);
    else MIX_LAUNCH(latent_qrope_kernel<false>, dim3((n + 255) / 256), dim3(256), 0, a);
    return WR_HIP_OK;
}

static bool latent_mfma_shape(int f32, const wr_hip_mix_latent* q)
{
    if (f32 || g.force_generic || q->rot_pad < 32 || q->rot_pad > 64) return false;
    return q->rank_pad == 64 || q->rank_pad == 128 || q->rank_pad == 256 || q->rank_pad == 512;
}

template <int RT, int KR, int KP>
static int latent_decode(wr_hip_mix_step* s, LatentMfmaArgs& q)
{
    using Sh = LatentDecodeShape<RT, KR, KP>;
    const LatentArgs& a = q.a;
    const uint32_t n = s->n_short_rows, tiles = (a.heads + 15) / 16, groups = (tiles + 4 / KP - 1) / (4 / KP);
    const LatentRow* rows = s->h<LatentRow>(s->o_short_rows);
    uint32_t keys = 1;                                     // of the row that sees the most, from its first tile on
    for (uint32_t i = 0; i < n; i++) {
        const uint32_t lo = rows[i].pos + 1 > a.window ? rows[i].pos + 1 - a.window : 0;
        keys = std::max(keys, rows[i].pos + 1 - lo / 32 * 32);
    }
    // Shares: a workgroup per compute unit at a time; a round costs about three iterations before its first
    // and one for each it makes.
    uint64_t best = ~(uint64_t)0;
    for (uint32_t iters = 1; iters <= 256; iters++) {
        const uint32_t share = iters * 32 * KP, splits = (keys + share - 1) / share;
        if (splits > 1024) continue;
        const uint64_t rounds = ((uint64_t)n * groups * splits + g.n_cus - 1) / g.n_cus, cost = rounds * (iters + 3);
        if (cost < best) {
            best = cost;
            q.split_keys = share;
            q.splits = splits;
        }
        if (splits == 1) break;
    }
    q.drows = s->d<LatentRow>(s->o_short_rows);
    if (q.splits > 1) {
        const size_t part = (size_t)n * tiles * q.splits * 16;
        int rc = ensure_device(s->partial, part * (RT * 32 + 2) * 4);
        if (rc) return rc;
        q.part_o = reinterpret_cast<float*>(s->partial.p);
        q.part_ml = q.part_o + part * RT * 32;
    }
    int rc = allow_lds<latent_decode_kernel<RT, KR, KP>>(Sh::kLds);
    if (rc) return rc;
    launch_main(latent_decode_kernel<RT, KR, KP>, dim3(n * groups, q.splits), dim3(256), q, Sh::kLds);
    HIP_TRY(hipGetLastError(), "latent decode launch", 0);
    if (q.splits > 1) MIX_LAUNCH(latent_combine_kernel<RT>, dim3(n, a.heads), dim3(RT * 32), 0, q);
    return WR_HIP_OK;
}

template <int RT, int KR>
static int latent_mfma(wr_hip_mix_step* s, LatentMfmaArgs& q)
{
    const LatentArgs& a = q.a;
    if (s->n_long) {
        uint32_t tiles = 0;
        for (uint32_t i = 0; i < s->n_long; i++) tiles += (s->long_rows[i] * a.heads + 127) / 128;
        q.list = s->d<uint32_t>(s->o_long);
        q.n_list = s->n_long;
        int rc = allow_lds<latent_prefill_kernel<RT, KR>>(latent_prefill_lds(RT, KR));
        if (rc) return rc;
        launch_main(latent_prefill_kernel<RT, KR>, dim3(tiles), dim3(LatentPrefillShape<RT>::kWaves * 64), q, latent_prefill_lds(RT, KR));
        HIP_TRY(hipGetLastError(), "latent prefill launch", 0);
    }
    if (s->n_short_rows) {
        const uint32_t head_tiles = (a.heads + 15) / 16;
        if (head_tiles == 1) return latent_decode<RT, KR, 4>(s, q);
        if (head_tiles == 2) return latent_decode<RT, KR, 2>(s, q);
        return latent_decode<RT, KR, 1>(s, q);
    }
    return WR_HIP_OK;
}

int wr_hip_mix_latent_attend(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, const wr_hip_mix_latent* q,
                             const void* q_dev, void* o_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    int rc = check_latent(q);
    if (rc) return rc;
    if (!s || !s->rows || !pool || run >= pool->latent.size() || pool->latent_dim[run] != q->rank_pad + q->rot_pad ||
        pool->f32 != (f32 != 0) || !q_dev || !o_dev)
        return WR_HIP_ERR_INVAL;
    ENTER();
    g.calls.fetch_add(s->n_seq, std::memory_order_relaxed);
    LatentArgs a = latent_args(s, q);
    a.cache = pool->latent[run];
    a.q = q_dev;
    a.o = o_dev;
    if (latent_mfma_shape(f32, q)) {
        LatentMfmaArgs m = {};
        m.a = a;
        switch (q->rank_pad / 32 * 2 + (q->rot_pad / 32 - 1)) {
        case 4: return latent_mfma<2, 1>(s, m);
        case 5: return latent_mfma<2, 2>(s, m);
        case 8: return latent_mfma<4, 1>(s, m);
        case 9: return latent_mfma<4, 2>(s, m);
        case 16: return latent_mfma<8, 1>(s, m);
        case 17: return latent_mfma<8, 2>(s, m);
        case 32: return latent_mfma<16, 1>(s, m);
        default: return latent_mfma<16, 2>(s, m);
        }
    }
    const size_t lds = ((size_t)2 * q->rank_pad + q->rot_pad + 64) * 4;
    rc = f32 ? allow_lds<latent_attend_any_kernel<true>>(lds) : allow_lds<latent_attend_any_kernel<false>>(lds);
    if (rc) return rc;
    if (f32) MIX_LAUNCH(latent_attend_any_kernel<true>, dim3(s->rows, q->heads), dim3(64), lds, a);
    else MIX_LAUNCH(latent_attend_any_kernel<false>, dim3(s->rows, q->heads), dim3(64), lds, a);
    return WR_HIP_OK;
}

// --------------------------------------------------- windowed attention --

uint32_t wr_hip_mix_window_pad(uint32_t dim)
{
    for (uint32_t p = 32; p <= 128; p *= 2)
        if (dim <= p) return p;
    return round32(dim);
}

static int check_window(const wr_hip_mix_step* s, const wr_hip_mix_pool* pool, uint32_t run, int f32, const wr_hip_mix_window* q)
{
    if (!s || !s->rows || !pool || run >= pool->latent.size() || pool->f32 != (f32 != 0) || !q || !q->heads || !q->kv_heads ||
        q->heads % q->kv_heads || !q->dim || !q->vdim || q->dim_pad % 32 || q->vdim_pad % 32 || q->dim > q->dim_pad ||
        q->vdim > q->vdim_pad || q->rot_half * 2 > q->dim || (!q->window && !q->chunk) || q->maps < 1 || q->maps > 2)
        return WR_HIP_ERR_INVAL;
    if (q->turn_values && (q->vdim % 2 || q->maps != 1)) return WR_HIP_ERR_INVAL;
    if ((uint64_t)q->kv_heads * ((uint64_t)q->maps * q->dim_pad + q->vdim_pad) != pool->latent_dim[run]) return WR_HIP_ERR_INVAL;
    return WR_HIP_OK;
}

static WindowArgs window_args(const wr_hip_mix_step* s, const wr_hip_mix_pool* pool, uint32_t run, const wr_hip_mix_window* q)
{
    WindowArgs a = {};
    a.seqs = s->d<MixSeq>(s->o_seqs);
    a.row_seq = s->d<uint32_t>(s->o_seq);
    a.row_pos = s->d<uint32_t>(s->o_pos);
    a.pages = s->d<uint32_t>(s->o_pages);
    a.rows = s->rows;
    a.heads = q->heads;
    a.kvh = q->kv_heads;
    a.group = q->heads / q->kv_heads;
    a.dim = q->dim;
    a.dimp = q->dim_pad;
    a.vdim = q->vdim;
    a.vdimp = q->vdim_pad;
    a.half = q->rot_half;
    a.window = q->window;
    a.chunk = q->chunk;
    a.gate_wide = q->gate_wide;
    a.vtable = q->turn_values;
    a.norm_values = q->norm_values;
    a.maps = q->maps;
    a.dimk = q->maps * q->dim_pad;
    a.neighbours = q->neighbours;
    a.softcap = q->softcap;
    a.diff = q->diff;
    a.q_norm = q->q_norm;
    a.k_norm = q->k_norm;
    a.scale = q->scale;
    a.out_scale = q->out_scale;
    a.eps = q->eps;
    a.cache = pool->latent[run];
    return a;
}

int wr_hip_mix_window_append(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, const wr_hip_mix_window* q,
                             const float* in_dev, uint32_t ld, uint32_t col_q, uint32_t col_k, uint32_t col_v,
                             const float* table_dev, void* q_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    int rc = check_window(s, pool, run, f32, q);
    if (rc) return rc;
    const bool keys = col_k != WR_HIP_MIX_NO_KEYS;
    if (!in_dev || !q_dev || (q->rot_half && !table_dev) || (uint64_t)col_q + (uint64_t)q->heads * q->maps * q->dim > ld ||
        (keys && ((uint64_t)col_k + (uint64_t)q->kv_heads * q->maps * q->dim > ld ||
                  (uint64_t)col_v + (uint64_t)q->kv_heads * q->vdim > ld)))
        return WR_HIP_ERR_INVAL;
    ENTER();
    WindowArgs a = window_args(s, pool, run, q);
    a.in = in_dev;
    a.ld = ld;
    a.col_q = col_q;
    a.col_k = col_k;
    a.col_v = col_v;
    a.table = table_dev;
    a.q = q_dev;
    a.key_heads = keys ? a.kvh : 0;
    const dim3 grid((s->rows + 3) / 4, a.key_heads + (4 * a.heads * (a.dimk / 8) + kWindowQUnits - 1) / kWindowQUnits);
    if (f32) MIX_LAUNCH(window_append_kernel<true>, grid, dim3(256), 0, a);
    else MIX_LAUNCH(window_append_kernel<false>, grid, dim3(256), 0, a);
    return WR_HIP_OK;
}

// Workgroups of a prefill launch of `rows` (token, head of the group) rows each.
static uint64_t window_tiles(const wr_hip_mix_step* s, const WindowArgs& a, uint32_t rows)
{
    uint64_t tiles = 0;
    for (uint32_t i = 0; i < s->n_long; i++) tiles += ((uint64_t)s->long_rows[i] * a.group + rows - 1) / rows;
    return tiles * a.kvh;
}

template <int KQ, int VT, int MAPS, int NR>
static int window_prefill(wr_hip_mix_step* s, WindowArgs& a)
{
    const uint64_t tiles = window_tiles(s, a, 64 * NR / MAPS);
    a.list = s->d<uint32_t>(s->o_long);
    a.n_list = s->n_long;
    constexpr size_t lds = window_prefill_lds(MAPS * KQ, VT);
    int rc = allow_lds<window_prefill_kernel<KQ, VT, MAPS, NR>>(lds);
    if (rc) return rc;
    launch_main(window_prefill_kernel<KQ, VT, MAPS, NR>, dim3((uint32_t)tiles), dim3(256), a, lds);
    HIP_TRY(hipGetLastError(), "windowed prefill launch", 0);
    return WR_HIP_OK;
}

template <int KQ, int VT, int MAPS>
static int window_mfma(wr_hip_mix_step* s, WindowArgs& a)
{
    if (s->n_long) {
        // 32 rows a wave, or 16 where the launch would be little more than what the device holds at once (two workgroups
        // a compute unit): its time is then that of the workgroup with the most keys
        int rc;
        if constexpr (MAPS == 2) rc = window_prefill<KQ, VT, 2, 2>(s, a);
        else if (window_tiles(s, a, 128) > 3 * (uint64_t)g.n_cus) rc = window_prefill<KQ, VT, 1, 2>(s, a);
        else rc = window_prefill<KQ, VT, 1, 1>(s, a);
        if (rc) return rc;
    }
    const uint32_t n = s->n_short_rows;
    if (n == 0) return WR_HIP_OK;
    const LatentRow* rows = s->h<LatentRow>(s->o_short_rows);
    uint32_t keys = 1;                                     // of the row that sees the most, from its first block on
    for (uint32_t i = 0; i < n; i++) {
        const uint32_t lo = window_lo(rows[i].pos, a.window, a.chunk);
        keys = std::max(keys, rows[i].pos + 1 - lo / 32 * 32);
    }
    const uint32_t groups = a.kvh * ((a.group * MAPS + 15) / 16);
    // Shares: two workgroups per compute unit at a time; a round costs about three iterations before its first and one
    // for each it makes, and the shares' sums about two more to put together.
    uint64_t best = ~(uint64_t)0;
    for (uint32_t iters = 1; iters <= 256; iters++) {
        const uint64_t share = (uint64_t)iters * 128, splits = (keys + share - 1) / share;
        if (splits > kWindowSplits) continue;
        const uint64_t rounds = ((uint64_t)n * groups * splits + 2 * g.n_cus - 1) / (2 * g.n_cus);
        const uint64_t cost = rounds * (iters + 3) + (splits > 1 ? 2 : 0);
        if (cost < best) {
            best = cost;
            a.split_keys = (uint32_t)share;
            a.splits = (uint32_t)splits;
        }
        if (splits == 1) break;
    }
    a.drows = s->d<LatentRow>(s->o_short_rows);
    if (a.splits > 1) {
        const size_t part = (size_t)n * a.heads * MAPS * a.splits;
        int rc = ensure_device(s->partial, part * (VT * 32 + 2) * 4);
        if (rc) return rc;
        a.part_o = reinterpret_cast<float*>(s->partial.p);
        a.part_ml = a.part_o + part * VT * 32;
    }
    launch_main(window_decode_kernel<MAPS * KQ, VT, MAPS>, dim3(n * groups, a.splits), dim3(256), a);
    HIP_TRY(hipGetLastError(), "windowed decode launch", 0);
    if (a.splits > 1) MIX_LAUNCH((window_combine_kernel<VT, MAPS>), dim3(n, a.heads), dim3(64 * MAPS), 0, a);
    return WR_HIP_OK;
}

template <int KQ, int MAPS>
static int window_mfma_v(wr_hip_mix_step* s, WindowArgs& a)
{
    if (a.vdimp == 32) return window_mfma<KQ, 1, MAPS>(s, a);
    if (a.vdimp == 64) return window_mfma<KQ, 2, MAPS>(s, a);
    return window_mfma<KQ, 4, MAPS>(s, a);
}

template <int MAPS>
static int window_mfma_k(wr_hip_mix_step* s, WindowArgs& a)
{
    if (a.dimp == 32) return window_mfma_v<1, MAPS>(s, a);
    if (a.dimp == 64) return window_mfma_v<2, MAPS>(s, a);
    return window_mfma_v<4, MAPS>(s, a);
}

int wr_hip_mix_window_attend(wr_hip_mix_step* s, wr_hip_mix_pool* pool, uint32_t run, int f32, const wr_hip_mix_window* q,
                             const void* q_dev, const float* sink_dev, const float* gate_dev, uint32_t ldg, void* o_dev,
                             uint32_t o_kt)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    int rc = check_window(s, pool, run, f32, q);
    if (rc) return rc;
    if (!q_dev || !o_dev || (uint64_t)q->heads * q->vdim_pad > (uint64_t)o_kt * 32 || (gate_dev && ldg < (q->gate_wide ? q->heads * q->vdim : q->heads)))
        return WR_HIP_ERR_INVAL;
    if (q->gate_wide && (!gate_dev || ldg % 4)) return WR_HIP_ERR_INVAL;
    ENTER();
    g.calls.fetch_add(s->n_seq, std::memory_order_relaxed);
    WindowArgs a = window_args(s, pool, run, q);
    a.q = const_cast<void*>(q_dev);
    a.sink = sink_dev;
    a.gate = gate_dev;
    a.ldg = ldg;
    a.o = o_dev;
    a.o_kt = o_kt;
    auto fits = [](uint32_t p) { return p == 32 || p == 64 || p == 128; };
    if (!f32 && !g.force_generic && fits(a.dimp) && fits(a.vdimp)) {
        return a.maps == 2 ? window_mfma_k<2>(s, a) : window_mfma_k<1>(s, a);
    }
    const size_t lds = ((size_t)a.dimp + (size_t)a.maps * a.vdimp + 64) * 4;
    rc = f32 ? allow_lds<window_attend_any_kernel<true>>(lds) : allow_lds<window_attend_any_kernel<false>>(lds);
    if (rc) return rc;
    if (f32) MIX_LAUNCH(window_attend_any_kernel<true>, dim3(s->rows, a.heads), dim3(64), lds, a);
    else MIX_LAUNCH(window_attend_any_kernel<false>, dim3(s->rows, a.heads), dim3(64), lds, a);
    return WR_HIP_OK;
}

// ---------------------------------------------------------------- experts --

uint32_t wr_hip_mix_route_groups(uint32_t rows, uint32_t experts, uint32_t top, uint32_t tile_groups)
{
    const uint64_t pairs = (uint64_t)rows * top, run = (uint64_t)tile_groups * 16;
    // every expert in use can waste at most all but one slot of its last run
    const uint64_t runs = pairs / run + std::min<uint64_t>(pairs, experts);
    return (uint32_t)(runs * tile_groups);
}

int wr_hip_mix_route(wr_hip_mix_step* s, const float* z_dev, uint32_t ldz, const wr_hip_mix_router* q, uint32_t tile_groups,
                     float* gate_dev, float* side_dev, float* slot_weight_dev, uint32_t* slot_dev, uint32_t* perm_dev,
                     int32_t* group_expert_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !z_dev || !q || !q->experts || !q->top || !tile_groups || !gate_dev || !slot_dev || !perm_dev ||
        !group_expert_dev)
        return WR_HIP_ERR_INVAL;
    const uint64_t outputs = (uint64_t)q->experts + q->identity;
    if (outputs > WR_HIP_MIX_MAX_EXPERTS || q->top > WR_HIP_MIX_MAX_TOP || q->groups > WR_HIP_MIX_MAX_GROUPS) return WR_HIP_ERR_LIMIT;
    if (ldz < outputs + (q->shared_gate != 0) || ((q->identity || q->shared_gate) && !side_dev) || (q->correction && !q->softmax_all))
        return WR_HIP_ERR_INVAL;
    if (q->logistic && q->softmax_all) return WR_HIP_ERR_INVAL;
    if (q->groups && (outputs % q->groups || !q->keep || q->keep > q->groups)) return WR_HIP_ERR_INVAL;
    if (q->top > (q->groups ? outputs / q->groups * q->keep : outputs)) return WR_HIP_ERR_INVAL;
    ENTER();
    MixRouteArgs a = {};
    a.z = z_dev;
    a.ldz = ldz;
    a.rows = s->rows;
    a.outputs = (uint32_t)outputs;
    a.experts = q->experts;
    a.top = q->top;
    a.tile_groups = tile_groups;
    a.n_groups = wr_hip_mix_route_groups(s->rows, q->experts, q->top, tile_groups);
    a.kinds = q->groups;
    a.keep = q->keep;
    a.softmax_all = q->softmax_all;
    a.shared_gate = q->shared_gate;
    a.logistic = q->logistic;
    a.slot_weight = slot_weight_dev;
    a.scale = q->scale;
    a.correction = q->correction;
    a.gate = gate_dev;
    a.side = side_dev;
    a.slot = slot_dev;
    a.perm = perm_dev;
    a.group_expert = group_expert_dev;
    static_assert(WR_HIP_MIX_MAX_TOP * kOrderRows <= kOrderPairs, "choices of a short step");
    if (s->rows <= kOrderRows) {
        if (outputs <= 64) MIX_LAUNCH(mix_order_kernel<1>, dim3(1), dim3(1024), 0, a);
        else if (outputs <= 256) MIX_LAUNCH(mix_order_kernel<4>, dim3(1), dim3(1024), 0, a);
        else MIX_LAUNCH(mix_order_kernel<16>, dim3(1), dim3(1024), 0, a);
        return WR_HIP_OK;
    }
    const dim3 grid((s->rows + 3) / 4), block(256);
    if (outputs <= 64) MIX_LAUNCH(mix_top_kernel<1>, grid, block, 0, a);
    else if (outputs <= 256) MIX_LAUNCH(mix_top_kernel<4>, grid, block, 0, a);
    else MIX_LAUNCH(mix_top_kernel<16>, grid, block, 0, a);
    MIX_LAUNCH(mix_order_kernel<0>, dim3(1), dim3(1024), 0, a);
    return WR_HIP_OK;
}

int wr_hip_mix_route_gather(wr_hip_mix_step* s, int f32, const void* h_dev, uint32_t kt, uint32_t n_groups,
                            const uint32_t* perm_dev, const int32_t* group_expert_dev, void* xs_dev)
{
    if (!g.inited) return WR_HIP_ERR_STATE;
    if (!s || !s->rows || !h_dev || !kt || !n_groups || !perm_dev || !group_expert_dev || !xs_dev) return WR_HIP_ERR_INVAL;
    ENTER();
    const dim3 grid((kt * 64 + 255) / 256, n_groups), block(256);
    if (f32) MIX_LAUNCH(mix_gather_kernel<true>, grid, block, 0, h_dev, kt, n_groups, perm_dev, group_expert_dev, xs_dev);
    else MIX_LAUNCH(mix_gather_kernel<false>, grid, block, 0, h_dev, kt, n_groups, perm_dev, group_expert_dev, xs_dev);
    return WR_HIP_OK;
}

