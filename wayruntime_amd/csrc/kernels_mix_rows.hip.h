// Row steps of mixer-stack models: embedding with its norm, the norm-residual-
// norm step between sublayers, the gated norm after the recurrence, the expert
// router and its ordering.
#pragma once

#include "mix_common.hip.h"

namespace wr {

// A workgroup serves RPW rows (1: few rows, latency; 4: many rows, so that the
// fragment is written in pieces of 64 bytes).  Thread t
// works on row t % RPW and the chunks of eight features t / RPW, + THREADS / RPW ...
template <int RPW>
struct MixRowShape {
    static constexpr int kThreads = RPW == 1 ? 256 : 512;
    static constexpr int kPerRow = kThreads / RPW;
    static constexpr int kHeld = RPW == 1 ? 2 : 4;       // chunks a thread can hold: 4096 features
};

// Sum over the threads of a row; every thread gets its row's sum.
template <int RPW>
__device__ __forceinline__ float mix_row_sum(float v, float* red)
{
    const int t = threadIdx.x, lane = t & 63, wave = t >> 6;
    constexpr int WAVES = MixRowShape<RPW>::kThreads / 64;
    if constexpr (RPW == 1) {
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) v += wave_xor_f32(v, off);
        if (lane == 0) red[wave] = v;
        __syncthreads();
        float s = 0.f;
#pragma unroll
        for (int w = 0; w < WAVES; w++) s += red[w];
        __syncthreads();
        return s;
    } else {
#pragma unroll
        for (int off = RPW; off <= 32; off <<= 1) v += wave_xor_f32(v, off);
        if (lane < RPW) red[wave * RPW + lane] = v;
        __syncthreads();
        float s = 0.f;
#pragma unroll
        for (int w = 0; w < WAVES; w++) s += red[w * RPW + t % RPW];
        __syncthreads();
        return s;
    }
}

__device__ __forceinline__ void mix_load8(const float* p, float (&v)[8])
{
    const f32x4 lo = *reinterpret_cast<const f32x4*>(p), hi = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; j++) {
        v[j] = lo[j];
        v[4 + j] = hi[j];
    }
}
__device__ __forceinline__ void mix_load8(const __bf16* p, float (&v)[8])
{
    const bf16x8 x = *reinterpret_cast<const bf16x8*>(p);
#pragma unroll
    for (int j = 0; j < 8; j++) v[j] = (float)x[j];
}
__device__ __forceinline__ void mix_store8(float* p, const float (&v)[8])
{
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}
template <bool F32>
__device__ __forceinline__ void mix_store_unit(void* h, size_t unit, const float (&v)[8])
{
    typename MixAct<F32>::V8 o;
#pragma unroll
    for (int j = 0; j < 8; j++) o[j] = (typename MixAct<F32>::E)v[j];
    reinterpret_cast<typename MixAct<F32>::V8*>(h)[unit] = o;
}

struct MixRowArgs {
    uint32_t rows, width, wpad;      // wpad: width padded to 32, the row stride of x, y, add and the norms
    float eps;
    float* x;
    const float *y, *post, *add, *next;
    const float *pair_y[2], *pair_post[2];      // two more outputs, each normed
    const float* gate;                // nullptr: ones
    const uint32_t* slot;
    uint32_t top;
    const float *side, *shared;      // weights of the input's own row and of the shared expert's, [rows][2]
    const void* ident;               // frag rows of the sublayer's input; may be h
    const uint32_t* gather;          // rows to read (the step's wanted rows), or nullptr
    void* h;
    // embedding
    const uint16_t* table;
    const uint32_t* tokens;
    const float* norm;               // nullptr: times scale instead
    float scale;
    float* x0;
};

// the sublayer output's chunk q of row r: plain, or the experts' rows weighted
template <bool F32>
__device__ __forceinline__ void mix_sub_chunk(const MixRowArgs& a, uint32_t r, uint32_t q, float (&v)[8])
{
    if (!a.top) {
        mix_load8(a.y + (size_t)r * a.wpad + q * 8, v);
        return;
    }
#pragma unroll
    for (int j = 0; j < 8; j++) v[j] = 0.f;
    for (uint32_t t0 = 0; t0 < a.top; t0 += 4) {           // four experts' rows in flight
        float gt[4], e[4][8];
        uint32_t slot[4];
#pragma unroll
        for (uint32_t i = 0; i < 4; i++) {
            const size_t at = (size_t)r * a.top + min(t0 + i, a.top - 1);
            gt[i] = a.gate ? a.gate[at] : 1.0f;
            slot[i] = t0 + i < a.top ? a.slot[at] : 0xFFFFFFFFu;
        }
#pragma unroll
        for (uint32_t i = 0; i < 4; i++)
            if (slot[i] != 0xFFFFFFFFu) mix_load8(a.y + (size_t)slot[i] * a.wpad + q * 8, e[i]);
#pragma unroll
        for (uint32_t i = 0; i < 4; i++)
            if (slot[i] != 0xFFFFFFFFu) {
#pragma unroll
                for (int j = 0; j < 8; j++) v[j] = fmaf(gt[i], e[i][j], v[j]);
            }
    }
    if (!a.side) return;
    float e[8];
    if (a.ident) {                                         // (read by the thread that writes this unit of h later)
        const float own = a.side[(size_t)r * 2];
        mix_load8(reinterpret_cast<const typename MixAct<F32>::E*>(a.ident) + frag_unit(r, q, a.wpad / 32) * 8, e);
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = fmaf(own, e[j], v[j]);
    }
    if (a.shared) {
        const float gt = a.side[(size_t)r * 2 + 1];
        mix_load8(a.shared + (size_t)r * a.wpad + q * 8, e);
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = fmaf(gt, e[j], v[j]);
    }
}

// x <- x + rmsnorm(y) * post (or + y) + add; h <- rmsnorm(x) * next
// (EMBED: x <- rmsnorm(table[token]) * norm, or table[token] * scale, first;
// PAIR: + rmsnorm(pair_y[i]) * pair_post[i] for both).
template <bool F32, int RPW, bool EMBED, bool HELD, bool PAIR>
__global__ __launch_bounds__(MixRowShape<RPW>::kThreads) void mix_residual_kernel(const MixRowArgs a)
{
    using Sh = MixRowShape<RPW>;
    constexpr int CH = HELD ? Sh::kHeld : 1;
    __shared__ float red[64];
    const uint32_t t = threadIdx.x;
    const uint32_t row = blockIdx.x * RPW + t % RPW, lr = t / RPW;
    const bool live = row < a.rows;
    const uint32_t rr = live ? row : a.rows - 1;
    const uint32_t r = a.gather ? a.gather[rr] : rr;
    const uint32_t nq = a.wpad / 8, kt = a.wpad / 32;
    const float invw = 1.0f / (float)a.width;
    float* xr = a.x + (size_t)r * a.wpad;
    float held[CH][8];
    float ss = 0.f;

    // the value to be normed into x: the sublayer's output, or the embedding row
    auto first = [&](uint32_t q, float (&v)[8]) {
        if constexpr (EMBED) {
            const uint16_t* e = a.table + (size_t)a.tokens[r] * a.width;
            if ((a.width & 7) == 0) {                      // rows of whole 16-byte units
                if (q * 8 < a.width) {
                    mix_load8(reinterpret_cast<const __bf16*>(e + q * 8), v);
                } else {
#pragma unroll
                    for (int j = 0; j < 8; j++) v[j] = 0.f;
                }
                return;
            }
#pragma unroll
            for (int j = 0; j < 8; j++) {
                const uint32_t k = q * 8 + j;
                v[j] = k < a.width ? __uint_as_float((uint32_t)e[k] << 16) : 0.f;
            }
        } else {
            mix_sub_chunk<F32>(a, r, q, v);
        }
    };
    const bool some = EMBED || a.y != nullptr;            // uniform: there is a value
    const bool normed = EMBED ? a.norm != nullptr : a.post != nullptr;
    float inv = EMBED ? a.scale : 1.0f;
    if (some) {
        if constexpr (HELD) {
#pragma unroll
            for (int i = 0; i < CH; i++) {
                const uint32_t q = lr + i * Sh::kPerRow;
                if (q < nq) {
                    first(q, held[i]);
#pragma unroll
                    for (int j = 0; j < 8; j++) ss = fmaf(held[i][j], held[i][j], ss);
                }
            }
        } else {
            for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
                float v[8];
                first(q, v);
#pragma unroll
                for (int j = 0; j < 8; j++) ss = fmaf(v[j], v[j], ss);
            }
        }
        if (normed) inv = 1.0f / sqrtf(mix_row_sum<RPW>(ss, red) * invw + a.eps);
    }
    float pair[PAIR ? 2 : 1][HELD && PAIR ? CH : 1][8], pinv[2];
    if constexpr (PAIR) {
#pragma unroll
        for (int k = 0; k < 2; k++) {
            const float* p = a.pair_y[k] + (size_t)r * a.wpad;
            float ps = 0.f;
            if constexpr (HELD) {
#pragma unroll
                for (int i = 0; i < CH; i++) {
                    const uint32_t q = lr + i * Sh::kPerRow;
                    if (q >= nq) continue;
                    mix_load8(p + q * 8, pair[k][i]);
#pragma unroll
                    for (int j = 0; j < 8; j++) ps = fmaf(pair[k][i][j], pair[k][i][j], ps);
                }
            } else {
                for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
                    mix_load8(p + q * 8, pair[k][0]);
#pragma unroll
                    for (int j = 0; j < 8; j++) ps = fmaf(pair[k][0][j], pair[k][0][j], ps);
                }
            }
            pinv[k] = 1.0f / sqrtf(mix_row_sum<RPW>(ps, red) * invw + a.eps);
        }
    }

    // x of one chunk, from the value above
    auto second = [&](uint32_t q, float (&v)[8], [[maybe_unused]] int at) {
        if constexpr (EMBED) {
            if (normed) {
                float w[8];
                mix_load8(a.norm + q * 8, w);
#pragma unroll
                for (int j = 0; j < 8; j++) v[j] = v[j] * inv * w[j];
            } else {
#pragma unroll
                for (int j = 0; j < 8; j++) v[j] *= inv;
            }
        } else {
            float x[8];
            mix_load8(xr + q * 8, x);
            if (a.y && !normed) {
#pragma unroll
                for (int j = 0; j < 8; j++) x[j] += v[j];
            } else if (a.y) {
                float w[8];
                mix_load8(a.post + q * 8, w);
#pragma unroll
                for (int j = 0; j < 8; j++) x[j] += v[j] * inv * w[j];
            }
            if constexpr (PAIR) {
#pragma unroll
                for (int k = 0; k < 2; k++) {
                    float w[8];
                    if constexpr (!HELD) mix_load8(a.pair_y[k] + (size_t)r * a.wpad + q * 8, pair[k][0]);
                    mix_load8(a.pair_post[k] + q * 8, w);
#pragma unroll
                    for (int j = 0; j < 8; j++) x[j] = fmaf(pair[k][HELD ? at : 0][j] * pinv[k], w[j], x[j]);
                }
            }
            if (a.add) {
                float w[8];
                mix_load8(a.add + (size_t)r * a.wpad + q * 8, w);
#pragma unroll
                for (int j = 0; j < 8; j++) x[j] += w[j];
            }
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] = x[j];
        }
        if (live && (EMBED || PAIR || a.y || a.add)) {
            mix_store8(xr + q * 8, v);
            if (EMBED && a.x0) mix_store8(a.x0 + (size_t)r * a.wpad + q * 8, v);
        }
    };
    ss = 0.f;
    if constexpr (HELD) {
#pragma unroll
        for (int i = 0; i < CH; i++) {
            const uint32_t q = lr + i * Sh::kPerRow;
            if (q < nq) {
                second(q, held[i], i);
#pragma unroll
                for (int j = 0; j < 8; j++) ss = fmaf(held[i][j], held[i][j], ss);
            }
        }
    } else {
        for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
            float v[8];
            if (some) first(q, v);
            second(q, v, 0);
#pragma unroll
            for (int j = 0; j < 8; j++) ss = fmaf(v[j], v[j], ss);
        }
    }
    if (!a.next) return;                                   // uniform
    inv = 1.0f / sqrtf(mix_row_sum<RPW>(ss, red) * invw + a.eps);
    auto third = [&](uint32_t q, float (&v)[8]) {
        float w[8];
        mix_load8(a.next + q * 8, w);
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = v[j] * inv * w[j];
        if (live) mix_store_unit<F32>(a.h, frag_unit(row, q, kt), v);
    };
    if constexpr (HELD) {
#pragma unroll
        for (int i = 0; i < CH; i++) {
            const uint32_t q = lr + i * Sh::kPerRow;
            if (q < nq) third(q, held[i]);
        }
    } else {
        for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
            float v[8];
            if (a.add || a.y || EMBED || PAIR) {
                if (live) {
                    mix_load8(xr + q * 8, v);              // this thread's own writes
                } else {
#pragma unroll
                    for (int j = 0; j < 8; j++) v[j] = 0.f;
                }
            } else {
                mix_load8(xr + q * 8, v);
            }
            third(q, v);
        }
    }
}

// Token shift (wr_hip_mix_shift): one row of eight features a thread and turn; the row before is normed again
// rather than waited for.
struct MixShiftArgs {
    const MixSeq* seqs;
    const uint32_t* row_seq;
    uint32_t rows, width, wpad, n_mix;
    float eps;
    const float *x, *y, *norm, *mu;
    float* x_out;
    float* state;                    // [buffer][wpad]
    void* out;
};
constexpr uint32_t kShiftMixes = 5;  // factors fetched ahead of the norms where a row has a workgroup to itself

template <bool F32, int RPW, bool HELD>
__global__ __launch_bounds__(MixRowShape<RPW>::kThreads) void mix_shift_kernel(const MixShiftArgs a)
{
    using Sh = MixRowShape<RPW>;
    constexpr int CH = HELD ? Sh::kHeld : 1;
    constexpr bool EARLY = HELD && RPW == 1;
    __shared__ float red[64];
    const uint32_t t = threadIdx.x, row = blockIdx.x * RPW + t % RPW, lr = t / RPW;
    const bool live = row < a.rows;
    const uint32_t r = live ? row : a.rows - 1, nq = a.wpad / 8;
    auto load = [&](uint32_t rr, uint32_t q, float (&v)[8]) {
        mix_load8(a.x + (size_t)rr * a.wpad + q * 8, v);
        if (a.y) {
            float w[8];
            mix_load8(a.y + (size_t)rr * a.wpad + q * 8, w);
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] += w[j];
        }
    };
    float hr[CH][8], hp[CH][8], hn[EARLY ? CH : 1][8], hm[EARLY ? kShiftMixes : 1][EARLY ? CH : 1][8];
    float sr = 0.f, sp = 0.f;
    if constexpr (HELD) {                                  // (first what does not wait for the request's description)
#pragma unroll
        for (int i = 0; i < CH; i++) {
            const uint32_t q = lr + i * Sh::kPerRow;
            if (q >= nq) continue;
            load(r, q, hr[i]);
            if constexpr (EARLY) {
                mix_load8(a.norm + q * 8, hn[i]);
#pragma unroll
                for (uint32_t m = 0; m < kShiftMixes; m++)
                    if (m < a.n_mix) mix_load8(a.mu + (size_t)m * a.wpad + q * 8, hm[m][i]);
            }
        }
    }
    const MixSeq s = a.seqs[a.row_seq[r]];
    const bool first = r == s.row0, last = r + 1 == s.row0 + s.rows;
    const uint32_t p = first ? r : r - 1;
    // h of the row before, not yet normed: its residual, or what the state holds (normed already)
    auto before = [&](uint32_t q, float (&v)[8]) {
        if (!first) {
            load(p, q, v);
        } else if (s.pos0 > 0) {
            mix_load8(a.state + (size_t)s.state_in * a.wpad + q * 8, v);
        } else {
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] = 0.f;
        }
    };
    auto square = [&](const float (&v)[8], const float (&w)[8]) {
#pragma unroll
        for (int j = 0; j < 8; j++) {
            sr = fmaf(v[j], v[j], sr);
            sp = fmaf(w[j], w[j], sp);
        }
    };
    if constexpr (HELD) {
#pragma unroll
        for (int i = 0; i < CH; i++) {
            const uint32_t q = lr + i * Sh::kPerRow;
            if (q >= nq) continue;
            before(q, hp[i]);
            square(hr[i], hp[i]);
        }
    } else {
        for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
            load(r, q, hr[0]);
            before(q, hp[0]);
            square(hr[0], hp[0]);
        }
    }
    const float invw = 1.0f / (float)a.width;
    const float ir = 1.0f / sqrtf(mix_row_sum<RPW>(sr, red) * invw + a.eps);
    float ip = 1.0f;
    if (RPW > 1 || !first) ip = 1.0f / sqrtf(mix_row_sum<RPW>(sp, red) * invw + a.eps);      // (one row: uniform)
    if (!live) return;
    auto mix = [&](uint32_t q, float (&v)[8], float (&w)[8], int i) {
        float n[8];
        if (a.y) mix_store8(a.x_out + (size_t)r * a.wpad + q * 8, v);
        if constexpr (EARLY) {
#pragma unroll
            for (int j = 0; j < 8; j++) n[j] = hn[i][j];
        } else {
            mix_load8(a.norm + q * 8, n);
        }
#pragma unroll
        for (int j = 0; j < 8; j++) {
            v[j] *= ir * n[j];
            if (!first) w[j] *= ip * n[j];
        }
        if (last) mix_store8(a.state + (size_t)s.state_out * a.wpad + q * 8, v);
        auto put = [&](uint32_t m, const float (&u)[8]) {
            float o[8];
#pragma unroll
            for (int j = 0; j < 8; j++) o[j] = v[j] + (w[j] - v[j]) * u[j];
            mix_store_unit<F32>(a.out, frag_unit(r, m * nq + q, a.n_mix * (a.wpad / 32)), o);
        };
        if constexpr (EARLY) {
#pragma unroll
            for (uint32_t m = 0; m < kShiftMixes; m++)
                if (m < a.n_mix) put(m, hm[m][i]);
        }
        for (uint32_t m = EARLY ? kShiftMixes : 0; m < a.n_mix; m++) {
            float u[8];
            mix_load8(a.mu + (size_t)m * a.wpad + q * 8, u);
            put(m, u);
        }
    };
    if constexpr (HELD) {
#pragma unroll
        for (int i = 0; i < CH; i++) {
            const uint32_t q = lr + i * Sh::kPerRow;
            if (q < nq) mix(q, hr[i], hp[i], i);
        }
    } else {
        for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
            load(r, q, hr[0]);
            before(q, hp[0]);
            mix(q, hr[0], hp[0], 0);
        }
    }
}

// h <- rmsnorm(o) * norm * g over n features (o 32-bit rows; g activation rows)
struct MixGateNormArgs {
    uint32_t rows, n, npad, ldo, ldg;
    float eps;
    const float *o, *norm;
    const void* g;
    void* h;
};
template <bool F32, int RPW>
__global__ __launch_bounds__(MixRowShape<RPW>::kThreads) void mix_gate_norm_kernel(const MixGateNormArgs a)
{
    using Sh = MixRowShape<RPW>;
    using E = typename MixAct<F32>::E;
    __shared__ float red[64];
    const uint32_t t = threadIdx.x, row = blockIdx.x * RPW + t % RPW, lr = t / RPW;
    const bool live = row < a.rows;
    const uint32_t r = live ? row : a.rows - 1, nq = a.npad / 8;
    const float* orow = a.o + (size_t)r * a.ldo;
    const E* grow = reinterpret_cast<const E*>(a.g) + (size_t)r * a.ldg;
    float ss = 0.f;
    for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
        float v[8];
        mix_load8(orow + q * 8, v);
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const float x = q * 8 + j < a.n ? v[j] : 0.f;              // (the pads of o are nobody's)
            ss = fmaf(x, x, ss);
        }
    }
    const float inv = 1.0f / sqrtf(mix_row_sum<RPW>(ss, red) / (float)a.n + a.eps);
    for (uint32_t q = lr; q < nq; q += Sh::kPerRow) {
        float v[8], w[8], g[8];
        mix_load8(orow + q * 8, v);
        mix_load8(a.norm + q * 8, w);
        mix_load8(grow + q * 8, g);
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = q * 8 + j < a.n ? v[j] * inv * w[j] * g[j] : 0.f;
        if (live) mix_store_unit<F32>(a.h, frag_unit(row, q, a.npad / 32), v);
    }
}

// ---- experts ---------------------------------------------------------------

struct MixRouteArgs {
    const float* z;
    uint32_t ldz, rows, outputs, experts, top, tile_groups, n_groups;     // outputs: experts, then those that pass the input on
    uint32_t kinds, keep, softmax_all, shared_gate, logistic;             // kinds: groups of neighbouring outputs, or 0
    float scale;
    const float* correction;
    float *gate, *side, *slot_weight;
    uint32_t* slot;                  // first the chosen output, then the slot
    uint32_t* perm;
    int32_t* group_expert;
};

__device__ __forceinline__ float mix_wave_max(float v)
{
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) v = fmaxf(v, wave_xor_f32(v, off));
    return v;
}

// One wave: the `top` outputs of a row with the largest choice value (lowest index among equals) and their weights.
// Lane l holds outputs l, l + 64, ...; put(t, output) is called by lane t.
template <int PER, typename Put>
__device__ __forceinline__ void mix_top(const MixRouteArgs& a, uint32_t row, int lane, Put put)
{
    float v[PER], s[PER];                                  // choice values (NaN: none, or taken) and softmax terms
    const float* z = a.z + (size_t)row * a.ldz;
    const float shared = a.shared_gate ? z[a.outputs] : 0.f;
#pragma unroll
    for (int i = 0; i < PER; i++) {
        const uint32_t e = lane + 64 * i;
        v[i] = e < a.outputs ? z[e] : __builtin_nanf("");
    }
    float zinv = 1.f;
    if (a.softmax_all) {                                   // choice: the softmax over all outputs, corrected
        float zmax = v[0], zs = 0.f;
#pragma unroll
        for (int i = 1; i < PER; i++) zmax = fmaxf(zmax, v[i]);
        zmax = mix_wave_max(zmax);
#pragma unroll
        for (int i = 0; i < PER; i++) {
            s[i] = lane + 64u * i < a.outputs ? expf(v[i] - zmax) : 0.f;
            zs += s[i];
        }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) zs += wave_xor_f32(zs, off);
        zinv = 1.0f / zs;
#pragma unroll
        for (int i = 0; i < PER; i++) {
            const uint32_t e = lane + 64 * i;
            if (e < a.outputs) v[i] = s[i] * zinv + (a.correction ? a.correction[e] : 0.f);
        }
    }
    if (a.kinds) {                                         // lane g holds the largest choice value of group g
        const uint32_t size = a.outputs / a.kinds;
        float mine = -INFINITY;
        for (uint32_t k = 0; k < a.kinds; k++) {
            float best = -INFINITY;
#pragma unroll
            for (int i = 0; i < PER; i++) {
                const uint32_t e = lane + 64 * i;
                if (e >= k * size && e < (k + 1) * size) best = fmaxf(best, v[i]);
            }
            best = mix_wave_max(best);
            if ((uint32_t)lane == k) mine = best;
        }
        uint32_t ahead = 0;                                // groups that are better than this lane's
        for (uint32_t k = 0; k < a.kinds; k++) {
            const float other = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(mine), k));
            ahead += other > mine || (other == mine && k < (uint32_t)lane);
        }
        const uint64_t kept = __ballot((uint32_t)lane < a.kinds && ahead < a.keep);
#pragma unroll
        for (int i = 0; i < PER; i++) {
            const uint32_t e = lane + 64 * i;
            if (e < a.outputs && !((kept >> (e / size)) & 1u)) v[i] = -INFINITY;
        }
    }
    float best0 = 0.f, sum = 0.f, mine = 0.f, own = 0.f;
    for (uint32_t t = 0; t < a.top; t++) {
        float bv = v[0];
#pragma unroll
        for (int i = 1; i < PER; i++) bv = fmaxf(bv, v[i]);
        bv = mix_wave_max(bv);
        uint32_t be = a.outputs - 1;                       // (NaN logits: still an output)
#pragma unroll
        for (int i = PER - 1; i >= 0; i--) {
            const uint64_t at = __ballot(v[i] == bv);
            if (at) be = 64 * i + __ffsll((unsigned long long)at) - 1;
        }
        float term = 0.f;
#pragma unroll
        for (int i = 0; i < PER; i++)
            if (lane + 64u * i == be) {
                v[i] = __builtin_nanf("");
                if (a.softmax_all) term = s[i];
            }
        if (t == 0) best0 = bv;
        const float g = a.softmax_all ? __int_as_float(__builtin_amdgcn_readlane(__float_as_int(term), be & 63u)) * zinv
                        : a.logistic  ? 1.0f / (1.0f + expf(-bv)) : expf(bv - best0);
        sum += g;
        if (be >= a.experts) own += g;
        if ((uint32_t)lane == t) {
            mine = g;
            put(t, be);
        }
    }
    const bool as_is = a.softmax_all || a.logistic;
    const float over = a.softmax_all ? a.scale / (sum + 1e-20f) : 1.0f;
    if ((uint32_t)lane < a.top) a.gate[(size_t)row * a.top + lane] = as_is ? mine * over : mine / sum;
    if (a.side && lane == 0) {
        a.side[(size_t)row * 2] = as_is ? own * over : own / sum;
        a.side[(size_t)row * 2 + 1] = a.shared_gate ? 1.0f / (1.0f + expf(-shared)) : 0.f;
    }
}

template <int PER>
__global__ __launch_bounds__(256) void mix_top_kernel(const MixRouteArgs a)
{
    const uint32_t row = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row < a.rows) mix_top<PER>(a, row, threadIdx.x & 63, [&](uint32_t t, uint32_t e) { a.slot[(size_t)row * a.top + t] = e; });
}

constexpr uint32_t kOrderRows = 64, kOrderPairs = kOrderRows * 64;      // of a step whose choice is made with the order

// One workgroup: orders the chosen (row, expert) pairs by expert.  Each expert's
// pairs take whole runs of tile_groups groups of 16 slots.  Which slot of its
// expert a pair gets may differ from run to run; nothing computed for it does
// (a slot's column of a matrix product depends on that column alone).
// PER: outputs a lane holds where the choice is made here too (few rows), else 0.
template <int PER>
__global__ __launch_bounds__(1024) void mix_order_kernel(const MixRouteArgs a)
{
    constexpr bool TOP = PER > 0;
    __shared__ uint32_t count[1024], wave_sum[16];
    __shared__ uint16_t pick[TOP ? kOrderPairs : 1];
    const uint32_t t = threadIdx.x, lane = t & 63, wave = t >> 6;
    const uint32_t n_slots = a.n_groups * 16, pairs = a.rows * a.top, run = a.tile_groups * 16;
    count[t] = 0;
    for (uint32_t i = t; i < n_slots; i += 1024) {
        a.perm[i] = 0xFFFFFFFFu;
        if (a.slot_weight) a.slot_weight[i] = 0.f;
    }
    for (uint32_t i = t; i < a.n_groups; i += 1024) a.group_expert[i] = -1;
    __syncthreads();
    if constexpr (TOP) {
        for (uint32_t r = wave; r < a.rows; r += 16)
            mix_top<PER>(a, r, lane, [&](uint32_t k, uint32_t e) {
                pick[r * a.top + k] = (uint16_t)e;
                if (e < a.experts) atomicAdd(&count[e], 1u);
            });
    } else {
        for (uint32_t i = t; i < pairs; i += 1024)
            if (a.slot[i] < a.experts) atomicAdd(&count[a.slot[i]], 1u);
    }
    __syncthreads();
    const uint32_t mine = (count[t] + run - 1) / run * run;
    uint32_t upto = mine;                                  // slots of the experts up to this one
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const uint32_t v = __shfl_up(upto, off, 64);
        if (lane >= (uint32_t)off) upto += v;
    }
    if (lane == 63) wave_sum[wave] = upto;
    __syncthreads();
    for (uint32_t w = 0; w < wave; w++) upto += wave_sum[w];
    for (uint32_t g = 0; g < mine / 16; g++) a.group_expert[(upto - mine) / 16 + g] = (int32_t)t;
    count[t] = upto - mine;                                // from here on: the expert's next slot
    __syncthreads();
    for (uint32_t i = t; i < pairs; i += 1024) {
        uint32_t e;
        if constexpr (TOP) e = pick[i];
        else e = a.slot[i];
        if (e >= a.experts) {                              // the input itself: nothing to compute
            a.slot[i] = 0xFFFFFFFFu;
            continue;
        }
        const uint32_t s = atomicAdd(&count[e], 1u);
        a.slot[i] = s;
        a.perm[s] = i / a.top;
        if (a.slot_weight) a.slot_weight[s] = a.gate[i];   // (made here: ahead of two barriers)
    }
}

// xs: the rows of h in slot order; one thread per unit of eight
template <bool F32>
__global__ __launch_bounds__(256) void mix_gather_kernel(const void* h, uint32_t kt, uint32_t n_groups,
                                                         const uint32_t* perm, const int32_t* group_expert, void* xs)
{
    using V8 = typename MixAct<F32>::V8;
    const uint32_t grp = blockIdx.y;
    if (group_expert[grp] < 0) return;
    const uint32_t u = blockIdx.x * 256 + threadIdx.x;     // unit of the group
    if (u >= kt * 64) return;
    const uint32_t row = perm[grp * 16 + (u & 15)];
    V8 v;
    if (row == 0xFFFFFFFFu) {
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = (typename MixAct<F32>::E)0.f;
    } else {
        v = reinterpret_cast<const V8*>(h)[((size_t)(row >> 4) * kt + (u >> 6)) * 64 + (u & 48) + (row & 15)];
    }
    reinterpret_cast<V8*>(xs)[(size_t)grp * kt * 64 + u] = v;
}

}  // namespace wr
