// Matrix-state recurrence with a decay per head and key channel made from the input:
// per head a state S [dim][vdim] (key channel by value column) in 32-bit floats,
//
//   BONUS   o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t    S_t = diag(w_t) S_(t-1) + k_t v_t^T
//   DELTA   S_t = diag(w_t) S_(t-1) - b_t (n_t^T S_(t-1)) + k_t v_t^T     o_t = S_t^T r_t
//   FORGET  S_t = diag(w_t) S_(t-1) + (1 - w_t) v_t^T     o_t = S_t^T r_t
//
// n_t the unit key, b_t = a_t n_t (BONUS, DELTA: vdim = dim).  Everything between the projections' 32-bit rows
// and the next product's operand happens here: decays, rates, unit keys, the
// recurrence, each head's norm and the gate.
//
// Token by token (decoded tokens and short portions): one workgroup per (request,
// head) holds the head's state in registers, a value column and a quarter of the key
// channels to a thread; both sums over the channels that a token needs are taken from
// the old state, so it is one reduction per token.  One decoded token is one read and
// one write of the state.
//
// By chunks of 16 rows (longer portions).  With p_t = n_t^T S_(t-1) and, inside a
// chunk that starts from S_0, rho(s, t) the product of the decays after token s up to
// and including token t, per channel:
//
//   P = T (N~ S_0 + A_nk V)       T = (I + A_nb)^-1, N~_t = n_t rho(before the chunk, t-1)
//   O = R~ S_0 + A_rk V - A_rb P
//   S_16 = rho(chunk) S_0 + K^T V - B^T P
//   A_xy[t][s] = sum over channels of x_t y_s rho(s, t or t-1),  K, B: k_s, b_s times rho(s, end)
//
// (BONUS, FORGET: P, N, B fall away; DELTA, FORGET: r_t comes times w_t.)  Two launches:
//   recur_chunk_kernel   parallel over (chunk, head), a wave each: the operands
//                        T N~, R~, [K | -B], [A_rk | -A_rb], T A_nk and V
//   recur_chain_kernel   a workgroup per (request, head), a wave per 16 value columns:
//                        walks the chunks with S in registers, operands through LDS
//                        (FORGET: per slice of the value columns, whose number is free)
// and recur_gate_kernel norms and gates their rows.  Where requests times heads leave
// most of the device idle, a request's chunks are walked in segments side by side: a
// first walk takes every segment but the last from S = 0 (and, DELTA, from S = I
// without values) without outputs, which gives the segment as S -> X S + C; the second
// starts each segment from the earlier ones applied to the request's state.
//
// No decay is ever divided by: tokens s < t that differ first in bit L of their place
// in the chunk meet in a product of two factors, rho from s to the end of its aligned
// block of 2^L and rho from the start of t's block to t, both at most one.  The four
// levels' scores are four products of differently scaled operands, of which each
// keeps its own pairs; the level after the last gives the factors to the chunk's ends.
//
// Products: with 32-bit activations on the 32-bit matrix instructions, else every
// operand as two bfloat16 terms, high and low, without the product of the low ones.
// In an operand's eight elements e of lane 16g + c, channel 32k + 16 (e / 4) + 4g + e % 4:
// the order in which an accumulator tile pair of S already lies, so S is the next
// product's operand where it stands.
#pragma once

#include "mix_common.hip.h"
#include "kernels_mix_rows.hip.h"

namespace wr {

struct RecurArgs {
    const MixSeq* seqs;
    const MixChunk* chunks;
    const uint32_t* list;           // requests of this launch
    uint32_t heads, dim, vdim, vtiles;      // vtiles: value tiles of sixteen, chunked form
    uint32_t gate;                  // kRecurGate*
    uint32_t norm_step;             // from one head's norm weights to the next's: vdim, or 0 where the heads share them
    float gain, unit_eps, eps, out_scale;
    const float *w0, *u, *ab, *norm;        // FORGET: w0 the gate's bias, u its lower bound
    const float* in;
    uint32_t ld, col_r, col_k, col_v, col_a, col_g;
    const float* z;
    uint32_t ldz;
    const bf16x8* wd;               // token by token: the decay's matrix, or nullptr where z is there already
    const void* low;
    uint32_t low_kt;
    float* state;                   // [buffer][heads][dim][dim]
    void* h;
    uint32_t h_kt, col_h;
    // chunked
    unsigned char* ops;             // [sub-chunk][heads][recur_unit_kib KiB]
    float* o;                       // [sub-chunk][16][heads][16 vtiles]
    uint32_t n_seg, seg_len;        // segments of a request, sub-chunks of one
    float *seg_c, *seg_x;           // [request of the list][segment][heads]: C [32 KT][16 VT], X [32 KT][32 KT] or its diagonal
};

enum { kRecurBonus = 0, kRecurDelta = 1, kRecurForget = 2 };
enum { kRecurGateLogistic = 0, kRecurGateSilu = 1, kRecurGateNone = 2 };

__device__ __forceinline__ float recur_decay(const RecurArgs& a, float z)
{
    return expf(a.gain > 0.f ? -a.gain / (1.0f + expf(-z)) : -expf(z));
}
__device__ __forceinline__ float recur_gate(const RecurArgs& a, float g)
{
    const float s = 1.0f / (1.0f + expf(-g));
    return a.gate == kRecurGateSilu ? g * s : s;
}
// FORGET: the decay low + (1 - low) logistic(z) and what it leaves of one.
__device__ __forceinline__ void recur_forget(float z, float low, float& w, float& k)
{
    const float e = expf(-fabsf(z)), over = 1.0f / (1.0f + e), s = z < 0.f ? e * over : over, t = z < 0.f ? over : e * over;
    w = fmaf(1.0f - low, s, low);
    k = (1.0f - low) * t;
}

// ---- token by token ---------------------------------------------------------

// Sum over a wave, in every lane.
__device__ __forceinline__ float recur_wave_sum(float v)
{
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) v += wave_xor_f32(v, off);
    return v;
}

// Row r's product with output n of the decay's matrix.
template <bool F32>
__device__ __forceinline__ float recur_z(const RecurArgs& a, uint32_t r, uint32_t n)
{
    using V8 = typename MixAct<F32>::V8;
    float z = 0.f;
    for (uint32_t kt = 0; kt < a.low_kt; kt++) {
        bf16x8 w[4];
        V8 x[4];
#pragma unroll
        for (int g = 0; g < 4; g++) {
            w[g] = a.wd[((size_t)(n / 16) * a.low_kt + kt) * 64 + 16 * g + n % 16];
            x[g] = reinterpret_cast<const V8*>(a.low)[frag_unit(r, kt * 4 + g, a.low_kt)];
        }
#pragma unroll
        for (int g = 0; g < 4; g++)
#pragma unroll
            for (int j = 0; j < 8; j++) z = fmaf((float)w[g][j], (float)x[g][j], z);
    }
    return z;
}

// grid (requests, heads), 4 DP threads: thread t has value column t % DP, channels DPT (t / DP) .. +DPT
template <bool F32, int DP, bool DELTA>
__global__ __launch_bounds__(4 * DP) void recur_step_kernel(const RecurArgs a)
{
    constexpr int DPT = DP / 4, WV = DP >= 64 ? DP / 64 : 1;       // waves that hold the channels' own values
    __shared__ float sr[DP], sk[DP], sw[DP], sn[DP], sb[DP], red[8 * DP], sums[3 * WV], sq[WV];
    const uint32_t t = threadIdx.x, head = blockIdx.y, part = t / DP, c = t % DP, d0 = part * DPT, D = a.dim;
    const uint32_t lane = t & 63, wave = t >> 6;
    const bool has = c < D, own = t < DP && has;                  // (own: also the thread of channel c's values)
    const MixSeq s = a.seqs[a.list[blockIdx.x]];
    const size_t head_elems = (size_t)D * D;
    const float* in = a.state + ((size_t)s.state_in * a.heads + head) * head_elems;
    float* out = a.state + ((size_t)s.state_out * a.heads + head) * head_elems;
    const uint32_t hd = head * D, npad = (a.heads * D + 31) / 32 * 32;
    float S[DPT];
#pragma unroll
    for (int j = 0; j < DPT; j++) S[j] = (s.pos0 > 0 && has && d0 + j < D) ? in[(size_t)(d0 + j) * D + c] : 0.f;
    const float w0 = own ? a.w0[hd + c] : 0.f, nrm = own ? a.norm[hd + c] : 0.f;
    const float ub = own ? (DELTA ? a.ab[hd + c] : a.u[hd + c]) : 0.f;
    for (uint32_t i = 0; i < s.rows; i++) {
        const uint32_t r = s.row0 + i;
        const float* row = a.in + (size_t)r * a.ld + hd;
        const float vv = has ? row[a.col_v + c] : 0.f;
        float g = 0.f;
        if (wave < WV) {
            const float rr = own ? row[a.col_r + c] : 0.f, kk = own ? row[a.col_k + c] : 0.f;
            const float w = own ? recur_decay(a, (a.wd ? recur_z<F32>(a, r, hd + c) : a.z[(size_t)r * a.ldz + hd + c]) + w0) : 0.f;
            g = own ? row[a.col_g + c] : 0.f;
            if constexpr (DELTA) {
                const float rate = own ? 1.0f / (1.0f + expf(-(row[a.col_a + c] + ub))) : 0.f;
                const float k2 = recur_wave_sum(kk * kk), rk = recur_wave_sum(rr * kk), rak = recur_wave_sum(rr * rate * kk);
                if (lane == 0) {
                    sums[wave] = k2;
                    sums[WV + wave] = rk;
                    sums[2 * WV + wave] = rak;
                }
                if (t < DP) {
                    sr[t] = rr * w;
                    sk[t] = kk;
                    sw[t] = w;
                    sn[t] = kk;
                    sb[t] = rate * kk;
                }
            } else {
                const float ruk = recur_wave_sum(rr * ub * kk);
                if (lane == 0) sums[wave] = ruk;
                if (t < DP) {
                    sr[t] = rr;
                    sk[t] = kk;
                    sw[t] = w;
                }
            }
        }
        __syncthreads();
        float tot[3] = {0.f, 0.f, 0.f};
#pragma unroll
        for (int q = 0; q < (DELTA ? 3 : 1); q++)
#pragma unroll
            for (int x = 0; x < WV; x++) tot[q] += sums[q * WV + x];
        float p = 0.f, o = 0.f;
#pragma unroll
        for (int j = 0; j < DPT; j++) {
            o = fmaf(sr[d0 + j], S[j], o);
            if constexpr (DELTA) p = fmaf(sn[d0 + j], S[j], p);
        }
        red[t] = o;
        if constexpr (DELTA) red[4 * DP + t] = p;
        __syncthreads();
        o = (red[c] + red[DP + c]) + (red[2 * DP + c] + red[3 * DP + c]);
        if constexpr (DELTA) {
            // n = k / sqrt(k . k + eps): once for what is read along it, once for what is removed
            const float inv = 1.0f / sqrtf(tot[0] + a.unit_eps);
            p = ((red[4 * DP + c] + red[5 * DP + c]) + (red[6 * DP + c] + red[7 * DP + c])) * inv * inv;
            o = o - tot[2] * p + tot[1] * vv;
        } else {
            o = fmaf(tot[0], vv, o);
        }
#pragma unroll
        for (int j = 0; j < DPT; j++) {
            float n = sw[d0 + j] * S[j];
            if constexpr (DELTA) n = fmaf(-sb[d0 + j], p, n);
            S[j] = fmaf(sk[d0 + j], vv, n);
        }
        if (wave < WV) {                                          // the head's norm and the gate
            const float ss = recur_wave_sum(own ? o * o : 0.f);
            if constexpr (WV > 1) {
                if (lane == 0) sq[wave] = ss;
            } else {
                if (own) {
                    const float inv = 1.0f / sqrtf(ss / (float)D + a.eps);
                    reinterpret_cast<typename MixAct<F32>::E*>(a.h)[frag_elem(r, a.col_h + hd + c, a.h_kt)] =
                        (typename MixAct<F32>::E)(o * inv * nrm * recur_gate(a, g) * a.out_scale);
                }
            }
        }
        __syncthreads();                                          // the row's values in LDS are done with
        if constexpr (WV > 1) {
            if (own) {
                float ss = 0.f;
#pragma unroll
                for (int x = 0; x < WV; x++) ss += sq[x];
                const float inv = 1.0f / sqrtf(ss / (float)D + a.eps);
                reinterpret_cast<typename MixAct<F32>::E*>(a.h)[frag_elem(r, a.col_h + hd + c, a.h_kt)] =
                    (typename MixAct<F32>::E)(o * inv * nrm * recur_gate(a, g) * a.out_scale);
            }
            // (sq is written again only after the next row's two barriers)
        }
        if (head + 1 == a.heads && t < npad - a.heads * D)        // pads of the operand
            reinterpret_cast<typename MixAct<F32>::E*>(a.h)[frag_elem(r, a.col_h + a.heads * D + t, a.h_kt)] =
                (typename MixAct<F32>::E)0.f;
    }
#pragma unroll
    for (int j = 0; j < DPT; j++)
        if (has && d0 + j < D) out[(size_t)(d0 + j) * D + c] = S[j];
}

// FORGET.  grid (requests, heads), 4 CP threads: thread t has value column t % CP, channels DPT (t / CP) .. +DPT
template <bool F32, int DPT, int CP>
__global__ __launch_bounds__(4 * CP) void recur_forget_step_kernel(const RecurArgs a)
{
    using E = typename MixAct<F32>::E;
    constexpr int DP = 4 * DPT, WV = CP >= 64 ? CP / 64 : 1;       // waves that put the columns together
    __shared__ float sr[DP], sk[DP], sw[DP], red[4 * CP], sq[WV];
    const uint32_t t = threadIdx.x, head = blockIdx.y, part = t / CP, c = t % CP, d0 = part * DPT, D = a.dim, V = a.vdim;
    const uint32_t lane = t & 63, wave = t >> 6;
    const bool has = c < V, own = t < CP && has;
    const MixSeq s = a.seqs[a.list[blockIdx.x]];
    const size_t head_elems = (size_t)D * V;
    const float* in = a.state + ((size_t)s.state_in * a.heads + head) * head_elems;
    float* out = a.state + ((size_t)s.state_out * a.heads + head) * head_elems;
    float S[DPT];
#pragma unroll
    for (int j = 0; j < DPT; j++) S[j] = (s.pos0 > 0 && has && d0 + j < D) ? in[(size_t)(d0 + j) * V + c] : 0.f;
    const float nrm = own ? a.norm[head * a.norm_step + c] * a.out_scale : 0.f;
    const uint32_t npad = (a.heads * V + 31) / 32 * 32;
    for (uint32_t i = 0; i < s.rows; i++) {
        const uint32_t r = s.row0 + i;
        const float* row = a.in + (size_t)r * a.ld;
        const float vv = has ? row[a.col_v + head * V + c] : 0.f;
        for (uint32_t d = t; d < DP; d += 4 * CP) {
            float w = 1.0f, k = 0.f;
            if (d < D) recur_forget(row[a.col_k + head * D + d] + a.w0[head * D + d], a.u[head * D + d], w, k);
            sw[d] = w;
            sk[d] = k;
            sr[d] = d < D ? row[a.col_r + head * D + d] : 0.f;
        }
        __syncthreads();
        float o = 0.f;
#pragma unroll
        for (int j = 0; j < DPT; j++) {
            S[j] = fmaf(sk[d0 + j], vv, sw[d0 + j] * S[j]);
            o = fmaf(sr[d0 + j], S[j], o);
        }
        red[t] = o;
        __syncthreads();
        o = own ? (red[c] + red[CP + c]) + (red[2 * CP + c] + red[3 * CP + c]) : 0.f;
        if (wave < WV) {
            const float ss = recur_wave_sum(o * o);
            if (lane == 0) sq[wave] = ss;
        }
        __syncthreads();
        if (own) {
            float ss = 0.f;
#pragma unroll
            for (int x = 0; x < WV; x++) ss += sq[x];
            reinterpret_cast<E*>(a.h)[frag_elem(r, a.col_h + head * V + c, a.h_kt)] = (E)(o / sqrtf(ss / (float)V + a.eps) * nrm);
        }
        // (sr, sk, sw: read ahead of the last two barriers; red and sq: written again only after the next row's)
        if (head + 1 == a.heads && t < npad - a.heads * V)        // pads of the operand
            reinterpret_cast<E*>(a.h)[frag_elem(r, a.col_h + a.heads * V + t, a.h_kt)] = (E)0.f;
    }
#pragma unroll
    for (int j = 0; j < DPT; j++)
        if (has && d0 + j < D) out[(size_t)(d0 + j) * V + c] = S[j];
}

// ---- by chunks --------------------------------------------------------------

constexpr uint32_t kRecurSub = 16;           // rows of a chunk: one matrix tile
constexpr uint32_t kRecurSubs = kMixChunk / kRecurSub;
constexpr int kRecurMaxDim = 128;            // the chunked form's limit on dim

// Eight (four) operand elements of a lane: in memory two (one) planes of 16 bytes a lane.
template <bool F32> struct RecurOp8;
template <> struct RecurOp8<true> {
    f32x4 p[2];
};
template <> struct RecurOp8<false> {
    bf16x8 p[2];                             // high terms, low terms
};
template <bool F32> struct RecurOp4;
template <> struct RecurOp4<true> {
    f32x4 p;
};
template <> struct RecurOp4<false> {
    bf16x8 p;                                // four high terms, four low terms
};

// Two values as high and low terms (in pairs: one conversion instruction does two).
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
typedef float f32x2v __attribute__((ext_vector_type(2)));
__device__ __forceinline__ void recur_split2(float x, float y, bf16x2& hi, bf16x2& lo)
{
    hi = __builtin_convertvector((f32x2v{x, y}), bf16x2);
    lo = __builtin_convertvector((f32x2v{x - (float)hi[0], y - (float)hi[1]}), bf16x2);
}
__device__ __forceinline__ bf16x8 recur_cat(bf16x2 a, bf16x2 b, bf16x2 c, bf16x2 d)
{
    return __builtin_shufflevector(__builtin_shufflevector(a, b, 0, 1, 2, 3), __builtin_shufflevector(c, d, 0, 1, 2, 3), 0, 1, 2, 3,
                                   4, 5, 6, 7);
}
template <bool F32>
__device__ __forceinline__ RecurOp8<F32> recur_op8(const float (&v)[8])
{
    RecurOp8<F32> r;
    if constexpr (F32) {
        r.p[0] = f32x4{v[0], v[1], v[2], v[3]};
        r.p[1] = f32x4{v[4], v[5], v[6], v[7]};
    } else {
        bf16x2 h[4], l[4];
#pragma unroll
        for (int j = 0; j < 4; j++) recur_split2(v[2 * j], v[2 * j + 1], h[j], l[j]);
        r.p[0] = recur_cat(h[0], h[1], h[2], h[3]);
        r.p[1] = recur_cat(l[0], l[1], l[2], l[3]);
    }
    return r;
}
template <bool F32>
__device__ __forceinline__ RecurOp8<F32> recur_op8(f32x4 lo, f32x4 hi)
{
    float v[8];
#pragma unroll
    for (int j = 0; j < 4; j++) {
        v[j] = lo[j];
        v[4 + j] = hi[j];
    }
    return recur_op8<F32>(v);
}
template <bool F32>
__device__ __forceinline__ RecurOp4<F32> recur_op4(f32x4 v)
{
    RecurOp4<F32> r;
    if constexpr (F32) {
        r.p = v;
    } else {
        bf16x2 h[2], l[2];
#pragma unroll
        for (int j = 0; j < 2; j++) recur_split2(v[2 * j], v[2 * j + 1], h[j], l[j]);
        r.p = recur_cat(h[0], h[1], l[0], l[1]);
    }
    return r;
}
// the first four elements from a, the others from b
__device__ __forceinline__ RecurOp8<true> recur_join(const RecurOp4<true>& a, const RecurOp4<true>& b)
{
    return RecurOp8<true>{{a.p, b.p}};
}
__device__ __forceinline__ RecurOp8<false> recur_join(const RecurOp4<false>& a, const RecurOp4<false>& b)
{
    return RecurOp8<false>{{__builtin_shufflevector(a.p, b.p, 0, 1, 2, 3, 8, 9, 10, 11),
                            __builtin_shufflevector(a.p, b.p, 4, 5, 6, 7, 12, 13, 14, 15)}};
}

// acc + A B over 32 inputs
__device__ __forceinline__ f32x4 recur_mm(const RecurOp8<true>& a, const RecurOp8<true>& b, f32x4 acc)
{
#pragma unroll
    for (int h = 0; h < 2; h++)
#pragma unroll
        for (int j = 0; j < 4; j++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.p[h][j], b.p[h][j], acc, 0, 0, 0);
    return acc;
}
__device__ __forceinline__ f32x4 recur_mm(const RecurOp8<false>& a, const RecurOp8<false>& b, f32x4 acc)
{
    return mix_mfma(a.p[0], b.p[0], mix_mfma(a.p[0], b.p[1], mix_mfma(a.p[1], b.p[0], acc)));
}
// over 16 inputs
__device__ __forceinline__ f32x4 recur_mm(const RecurOp4<true>& a, const RecurOp4<true>& b, f32x4 acc)
{
#pragma unroll
    for (int j = 0; j < 4; j++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.p[j], b.p[j], acc, 0, 0, 0);
    return acc;
}
// The eight elements of a lane are its four high and four low terms: one product over 32 "inputs" of
// (high, low) with (high, high), one of (high, low) with (low, 0).
__device__ __forceinline__ f32x4 recur_mm(const RecurOp4<false>& a, const RecurOp4<false>& b, f32x4 acc)
{
    bf16x8 zero;
#pragma unroll
    for (int j = 0; j < 8; j++) zero[j] = (__bf16)0.f;
    const bf16x8 bh = __builtin_shufflevector(b.p, b.p, 0, 1, 2, 3, 0, 1, 2, 3), bl = __builtin_shufflevector(b.p, zero, 4, 5, 6, 7, 8, 8, 8, 8);
    return mix_mfma(a.p, bh, mix_mfma(a.p, bl, acc));
}

// KiB of a sub-chunk's operands for one head, and where each lies.
template <int KT, bool DELTA>
struct RecurUnit {
    static constexpr int kR = 0;                                  // R~          [KT] op8
    static constexpr int kA = kR + 2 * KT;                        // A_rk, or [A_rk | -A_rb]: op4 / op8
    static constexpr int kG = kA + (DELTA ? 2 : 1);               // rho(chunk)  [32 KT] floats; from here on: what moves S
    static constexpr int kK = kG + 1;                             // K^T, or [K | -B]^T: [2 KT tiles] op4 / op8
    static constexpr int kW = kK + 2 * KT * (DELTA ? 2 : 1);      // T N~        [KT] op8
    static constexpr int kM = kW + (DELTA ? 2 * KT : 0);          // T A_nk      op4
    static constexpr int kV = kM + (DELTA ? 1 : 0);               // V           [value tiles] op4
};
__host__ __device__ constexpr int recur_unit_kib(int kt, bool delta, int vtiles)
{
    return (delta ? RecurUnit<0, true>::kV + 8 * kt : RecurUnit<0, false>::kV + 4 * kt) + vtiles;
}
static_assert(RecurUnit<2, true>::kV == RecurUnit<0, true>::kV + 16 && RecurUnit<2, false>::kV == RecurUnit<0, false>::kV + 8, "KiB");

template <bool F32>
__device__ __forceinline__ void recur_put(unsigned char* unit, int kib, int lane, const RecurOp8<F32>& v)
{
    using P = decltype(v.p[0]);
#pragma unroll
    for (int h = 0; h < 2; h++)
        *reinterpret_cast<std::remove_cv_t<std::remove_reference_t<P>>*>(unit + (kib + h) * 1024 + lane * 16) = v.p[h];
}
template <bool F32>
__device__ __forceinline__ void recur_put(unsigned char* unit, int kib, int lane, const RecurOp4<F32>& v)
{
    using P = decltype(v.p);
    *reinterpret_cast<std::remove_cv_t<std::remove_reference_t<P>>*>(unit + kib * 1024 + lane * 16) = v.p;
}
template <bool F32>
__device__ __forceinline__ RecurOp8<F32> recur_get8(const unsigned char* unit, int kib, int lane)
{
    RecurOp8<F32> r;
    using P = std::remove_reference_t<decltype(r.p[0])>;
#pragma unroll
    for (int h = 0; h < 2; h++) r.p[h] = *reinterpret_cast<const P*>(unit + (kib + h) * 1024 + lane * 16);
    return r;
}
template <bool F32>
__device__ __forceinline__ RecurOp4<F32> recur_get4(const unsigned char* unit, int kib, int lane)
{
    RecurOp4<F32> r;
    using P = decltype(r.p);
    r.p = *reinterpret_cast<const P*>(unit + kib * 1024 + lane * 16);
    return r;
}

// Four consecutive values from channel d on, zeros past n.
__device__ __forceinline__ f32x4 recur_load4(const float* p, uint32_t d, uint32_t n, bool whole)
{
    if (whole) return d < n ? *reinterpret_cast<const f32x4*>(p + d) : f32x4{0.f, 0.f, 0.f, 0.f};
    f32x4 v;
#pragma unroll
    for (int j = 0; j < 4; j++) v[j] = d + j < n ? p[d + j] : 0.f;
    return v;
}

// LDS floats of one wave: rows of N~, K and B [16][32 KT + 4], A_nb and T [16][20].  (BONUS: K alone.)
__host__ __device__ constexpr int recur_chunk_lds(int kt, bool delta)
{
    return (delta ? 3 : 1) * 16 * (32 * kt + 4) + (delta ? 2 * 16 * 20 : 0);
}

// grid (chunks of 64 rows, heads): wave w of four has rows 16w .. 16w + 15.  `whole`: dim and every column are
// multiples of four.
template <bool F32, int KT, int RULE>
__global__ __launch_bounds__(256, KT <= 2 ? 2 : 1) void recur_chunk_kernel(const RecurArgs a, const uint32_t whole)
{
    constexpr bool DELTA = RULE == kRecurDelta, FORGET = RULE == kRecurForget;
    using U = RecurUnit<KT, DELTA>;
    constexpr int LD = 32 * KT + 4;
    extern __shared__ __attribute__((aligned(16))) float recur_smem[];
    const MixChunk ch = a.chunks[blockIdx.x];
    const uint32_t head = blockIdx.y, D = a.dim, hd = head * D;
    const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const uint32_t wave = threadIdx.x >> 6, vtiles = a.vtiles;
    float* ln = recur_smem + wave * recur_chunk_lds(KT, DELTA);   // DELTA: N~; the rows of K stand first otherwise
    float* lk = DELTA ? ln + 16 * LD : ln;
    float* lb = lk + 16 * LD;
    float* la = lb + 16 * LD;
    float* lt = la + 16 * 20;
    const uint32_t i = wave * kRecurSub + c;
    const bool live = i < ch.rows;                                // (other rows: zeros, decay one)
    const uint32_t r = ch.row0 + min(i, ch.rows - 1);
    const float* row = a.in + (size_t)r * a.ld + hd;
    const float* zrow = a.z + (size_t)r * a.ldz + hd;
    unsigned char* unit = a.ops + ((size_t)(blockIdx.x * kRecurSubs + wave) * a.heads + head) *
                                      (size_t)recur_unit_kib(KT, DELTA, vtiles) * 1024;

    float q[KT][8], k[KT][8], n[DELTA ? KT : 1][8], b[DELTA ? KT : 1][8];      // q: r, times this token's decay but in BONUS
    float E[KT][8], F[KT][8], B[KT][8];                           // rho: after the token in its block, ahead of it, the block
    float k2 = 0.f, drk = 0.f, drb = 0.f;
#pragma unroll
    for (int t = 0; t < KT; t++)
#pragma unroll
        for (int h = 0; h < 2; h++) {
            const uint32_t d = 32 * t + 16 * h + 4 * g;
            const f32x4 r4 = recur_load4(row + a.col_r, d, D, whole);
            f32x4 k4 = r4;
            if constexpr (!FORGET) k4 = recur_load4(row + a.col_k, d, D, whole);
            const f32x4 z4 = recur_load4(zrow, d, D, whole), w4 = recur_load4(a.w0 + hd, d, D, whole);
            const f32x4 x4 = recur_load4((DELTA ? a.ab : a.u) + hd, d, D, whole);
            f32x4 a4 = x4;
            if constexpr (DELTA) a4 = recur_load4(row + a.col_a, d, D, whole);
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const bool on = live && d + j < D;
                const float rr = on ? r4[j] : 0.f;
                float kk, w;
                if constexpr (FORGET) {
                    recur_forget(z4[j] + w4[j], x4[j], w, kk);
                    w = on ? w : 1.0f;
                    kk = on ? kk : 0.f;
                } else {
                    kk = on ? k4[j] : 0.f;
                    w = on ? recur_decay(a, z4[j] + w4[j]) : 1.0f;
                }
                const int e = 4 * h + j;
                q[t][e] = DELTA || FORGET ? rr * w : rr;
                k[t][e] = kk;
                B[t][e] = w;
                E[t][e] = F[t][e] = 1.0f;
                if constexpr (DELTA) {
                    const float rate = 1.0f / (1.0f + expf(-(a4[j] + x4[j])));
                    n[t][e] = kk;
                    b[t][e] = rate * kk;
                    k2 = fmaf(kk, kk, k2);
                    drk = fmaf(rr, kk, drk);
                    drb = fmaf(rr, rate * kk, drb);
                } else {
                    drk = fmaf(FORGET ? rr : rr * x4[j], kk, drk);
                }
            }
        }
    auto over_g = [](float v) {
        v += wave_xor_f32(v, 16);
        return v + wave_xor_f32(v, 32);
    };
    drk = over_g(drk);
    if constexpr (DELTA) {
        const float inv = 1.0f / sqrtf(over_g(k2) + a.unit_eps);
        drb = over_g(drb) * inv;
#pragma unroll
        for (int t = 0; t < KT; t++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                n[t][e] *= inv;
                b[t][e] *= inv;
            }
    }

    const f32x4 zero = f32x4{0.f, 0.f, 0.f, 0.f};
    f32x4 ark = zero, arb = zero, ank = zero, anb = zero;         // ark, arb: key row 4g + i, query column c; ank, anb the other way
#pragma unroll
    for (int L = 0; L < 4; L++) {
        f32x4 xrk = zero, xrb = zero, xnk = zero, xnb = zero;
#pragma unroll
        for (int t = 0; t < KT; t++) {
            float v[8];
            auto times = [&](const float (&x)[8], const float (&y)[8]) {
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = x[e] * y[e];
                return recur_op8<F32>(v);
            };
            const RecurOp8<F32> qo = times(q[t], F[t]), ko = times(k[t], E[t]);
            xrk = recur_mm(ko, qo, xrk);
            if constexpr (DELTA) {
                const RecurOp8<F32> no = times(n[t], F[t]), bo = times(b[t], E[t]);
                xrb = recur_mm(bo, qo, xrb);
                xnk = recur_mm(no, ko, xnk);
                xnb = recur_mm(no, bo, xnb);
            }
        }
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int m = 4 * g + j;                              // rows of the tile; columns are c
            const bool col_later = (c >> L) == (m >> L) + 1 && ((c >> L) & 1), row_later = (m >> L) == (c >> L) + 1 && ((m >> L) & 1);
            if (col_later) {
                ark[j] = xrk[j];
                arb[j] = xrb[j];
            }
            if (row_later) {
                ank[j] = xnk[j];
                anb[j] = xnb[j];
            }
        }
        const bool upper = (c >> L) & 1;
#pragma unroll
        for (int t = 0; t < KT; t++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const float o = wave_xor_f32(B[t][e], 1 << L);
                E[t][e] *= upper ? 1.0f : o;
                F[t][e] *= upper ? o : 1.0f;
                B[t][e] *= o;
            }
    }
    if (c >> 2 == g) {                                            // a token with itself
#pragma unroll
        for (int j = 0; j < 4; j++)
            if ((c & 3) == j) {
                ark[j] = drk;
                arb[j] = drb;
            }
    }

    // rows for the operands that want tokens innermost
#pragma unroll
    for (int t = 0; t < KT; t++)
#pragma unroll
        for (int h = 0; h < 2; h++) {
            f32x4 x, y, z;
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const int e = 4 * h + j;
                x[j] = k[t][e] * E[t][e];
                if constexpr (DELTA) {
                    y[j] = -b[t][e] * E[t][e];
                    z[j] = n[t][e] * F[t][e];
                }
            }
            const int at = c * LD + 32 * t + 16 * h + 4 * g;
            *reinterpret_cast<f32x4*>(lk + at) = x;
            if constexpr (DELTA) {
                *reinterpret_cast<f32x4*>(lb + at) = y;
                *reinterpret_cast<f32x4*>(ln + at) = z;
            }
        }
    if constexpr (DELTA) {
#pragma unroll
        for (int j = 0; j < 4; j++) la[(4 * g + j) * 20 + c] = anb[j];         // zero on and above the diagonal
    }
    __syncthreads();

    f32x4 tt = zero;                                              // T[c][4g + j]
    if constexpr (DELTA) {
        // T = (I + A_nb)^-1 by rows, a column to each of the sixteen lanes (the four groups do the same)
        float T[16];
#pragma unroll
        for (int t = 0; t < 16; t++) {
            float v = t == c ? 1.0f : 0.f;
#pragma unroll
            for (int s4 = 0; s4 < (t + 3) / 4; s4++) {
                const f32x4 A = *reinterpret_cast<const f32x4*>(la + t * 20 + 4 * s4);
#pragma unroll
                for (int j = 0; j < 4; j++)
                    if (4 * s4 + j < t) v = fmaf(-A[j], T[4 * s4 + j], v);
            }
            T[t] = v;
        }
        if (g == 0) {
#pragma unroll
            for (int t = 0; t < 16; t++) lt[t * 20 + c] = T[t];
        }
        __syncthreads();
        tt = *reinterpret_cast<const f32x4*>(lt + c * 20 + 4 * g);
    }
    if (wave * kRecurSub >= ch.rows) return;

#pragma unroll
    for (int t = 0; t < KT; t++) {
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] = q[t][e] * F[t][e];
        recur_put<F32>(unit, U::kR + 2 * t, lane, recur_op8<F32>(v));
        if (c == 0) {
            float* G = reinterpret_cast<float*>(unit + U::kG * 1024) + 32 * t + 4 * g;
            *reinterpret_cast<f32x4*>(G) = f32x4{B[t][0], B[t][1], B[t][2], B[t][3]};
            *reinterpret_cast<f32x4*>(G + 16) = f32x4{B[t][4], B[t][5], B[t][6], B[t][7]};
        }
    }
    auto column = [&](const float* rows, int d) {                 // tokens 4g .. 4g + 3 of channel d
        return f32x4{rows[(4 * g) * LD + d], rows[(4 * g + 1) * LD + d], rows[(4 * g + 2) * LD + d], rows[(4 * g + 3) * LD + d]};
    };
#pragma unroll
    for (int t = 0; t < 2 * KT; t++) {
        const f32x4 kc = column(lk, 16 * t + c);
        if constexpr (DELTA) recur_put<F32>(unit, U::kK + 2 * t, lane, recur_op8<F32>(kc, column(lb, 16 * t + c)));
        else recur_put<F32>(unit, U::kK + t, lane, recur_op4<F32>(kc));
    }
    if constexpr (DELTA) {
        f32x4 nb;
#pragma unroll
        for (int j = 0; j < 4; j++) nb[j] = -arb[j];
        recur_put<F32>(unit, U::kA, lane, recur_op8<F32>(ark, nb));
        const RecurOp4<F32> to = recur_op4<F32>(tt);
#pragma unroll
        for (int t = 0; t < KT; t++) {
            const f32x4 lo = recur_mm(recur_op4<F32>(column(ln, 32 * t + c)), to, zero);
            const f32x4 hi = recur_mm(recur_op4<F32>(column(ln, 32 * t + 16 + c)), to, zero);
            recur_put<F32>(unit, U::kW + 2 * t, lane, recur_op8<F32>(lo, hi));
        }
        recur_put<F32>(unit, U::kM, lane, recur_op4<F32>(recur_mm(recur_op4<F32>(ank), to, zero)));
    } else {
        recur_put<F32>(unit, U::kA, lane, recur_op4<F32>(ark));
    }
    for (uint32_t t = 0; t < vtiles; t++) {
        f32x4 v;
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const uint32_t tok = wave * kRecurSub + 4 * g + j, col = 16 * t + c;
            v[j] = tok < ch.rows && col < a.vdim ? a.in[(size_t)(ch.row0 + tok) * a.ld + a.col_v + head * a.vdim + col] : 0.f;
        }
        recur_put<F32>(unit, U::kV + t, lane, recur_op4<F32>(v));
    }
}

// Sub-chunks whose operands lie in LDS at once.
__host__ __device__ constexpr int recur_ring(int kt, bool delta) { return kt >= 4 || delta ? 3 : 4; }

// One sub-chunk's operands in a wave's registers.
template <bool F32, int KT, bool DELTA, bool CARRY>
struct RecurHeld {
    RecurOp8<F32> R[KT], W[DELTA ? KT : 1], K8[DELTA ? 2 * KT : 1], A8;
    RecurOp4<F32> K4[DELTA ? 1 : 2 * KT], A4, M, V;
    f32x4 G[2 * KT];

    __device__ __forceinline__ void fetch(const unsigned char* unit, uint32_t wave, int lane, int g, bool values)
    {
        using U = RecurUnit<KT, DELTA>;
        constexpr int K0 = CARRY ? U::kG : 0;                     // first KiB that is there
        V = recur_get4<F32>(unit, U::kV - K0 + wave, lane);
        if (CARRY && DELTA && !values) {
#pragma unroll
            for (int j = 0; j < (int)(sizeof(V.p) / sizeof(V.p[0])); j++) V.p[j] = (std::remove_reference_t<decltype(V.p[0])>)0.f;
        }
        if constexpr (DELTA) M = recur_get4<F32>(unit, U::kM - K0, lane);
        if constexpr (!CARRY) {
            if constexpr (DELTA) A8 = recur_get8<F32>(unit, U::kA, lane);
            else A4 = recur_get4<F32>(unit, U::kA, lane);
        }
#pragma unroll
        for (int t = 0; t < KT; t++) {
            if constexpr (DELTA) W[t] = recur_get8<F32>(unit, U::kW - K0 + 2 * t, lane);
            if constexpr (!CARRY) R[t] = recur_get8<F32>(unit, U::kR + 2 * t, lane);
        }
#pragma unroll
        for (int t = 0; t < 2 * KT; t++) {
            if constexpr (DELTA) K8[t] = recur_get8<F32>(unit, U::kK - K0 + 2 * t, lane);
            else K4[t] = recur_get4<F32>(unit, U::kK - K0 + t, lane);
            G[t] = *reinterpret_cast<const f32x4*>(unit + (U::kG - K0) * 1024 + (16 * t + 4 * g) * 4);
        }
    }
};

// acc + sum over t of A[t] B[t], in chains of their own where there are several terms
template <int N>
__device__ __forceinline__ f32x4 recur_mm_many(const RecurOp8<true> (&a)[N], const RecurOp8<true> (&b)[N], f32x4 acc)
{
#pragma unroll
    for (int t = 0; t < N; t++) acc = recur_mm(a[t], b[t], acc);
    return acc;
}
template <int N>
__device__ __forceinline__ f32x4 recur_mm_many(const RecurOp8<false> (&a)[N], const RecurOp8<false> (&b)[N], f32x4 acc)
{
    f32x4 x = f32x4{0.f, 0.f, 0.f, 0.f}, y = x;
#pragma unroll
    for (int t = 0; t < N; t++) {
        acc = mix_mfma(a[t].p[0], b[t].p[0], acc);
        x = mix_mfma(a[t].p[0], b[t].p[1], x);
        y = mix_mfma(a[t].p[1], b[t].p[0], y);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) acc[i] += x[i] + y[i];
    return acc;
}

// Grid (requests * segments, heads), a wave per 16 value columns (1, 2, 4 or 8 of them, VT).  A stage of the ring is
// read into registers a step before it is used, and copied over from then on.  CARRY: the walk without outputs, of
// every segment but the last; DELTA has z = 1 for the walk from S = I.  Without DELTA z is the slice of VT value tiles.
template <bool F32, int KT, bool DELTA, int VT, bool CARRY>
__global__ __launch_bounds__(64 * VT, 2) void recur_chain_kernel(const RecurArgs a)
{
    using U = RecurUnit<KT, DELTA>;
    constexpr int K0 = CARRY ? U::kG : 0, UNIT = recur_unit_kib(KT, DELTA, VT) - K0;
    constexpr int RING = recur_ring(KT, DELTA), CPW = (UNIT + VT - 1) / VT, STORES = CARRY ? 0 : 4;
    // what is on its way behind the stage waited for: RING - 2 stages, and the stores of each step made since
    constexpr int EARLY = (RING - 2) * CPW, FULL = (RING - 2) * (CPW + STORES) + STORES, FIRST = (RING - 1) * CPW;
    static_assert(FULL < 64 && FIRST < 64, "vmcnt");
    constexpr uint32_t KP = 32 * KT;
    // a sub-chunk's operands and value columns in all, and those ahead of this slice
    const uint32_t all = (uint32_t)U::kV + a.vtiles, CP = 16 * a.vtiles, first_tile = DELTA ? 0 : blockIdx.z * VT;
    extern __shared__ __attribute__((aligned(16))) unsigned char recur_lds[];
    const uint32_t segs = CARRY ? a.n_seg - 1 : a.n_seg, item = blockIdx.x / segs, seg = blockIdx.x % segs;
    const MixSeq s = a.seqs[a.list[item]];
    const uint32_t n_sub = (s.rows + kRecurSub - 1) / kRecurSub, begin = seg * a.seg_len, end = min(n_sub, begin + a.seg_len);
    if (begin >= n_sub || (CARRY && end == n_sub)) return;        // uniform over the workgroup
    const bool values = !(CARRY && DELTA) || blockIdx.z == 0;     // (else: from S = I, without values)
    const uint32_t head = blockIdx.y, D = a.dim, sub0 = s.chunk0 * kRecurSubs;
    const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t col = (first_tile + wave) * 16 + c, V = a.vdim;
    const uint32_t lds0 = (uint32_t)__builtin_amdgcn_readfirstlane((uint32_t)(uintptr_t)recur_lds);
    auto issue = [&](uint32_t sub) {                              // (past the end: the last one again)
        const unsigned char* base =
            uniform_ptr(a.ops + (((size_t)(sub0 + min(begin + sub, end - 1)) * a.heads + head) * all + K0) * 1024);
        const uint32_t to = lds0 + sub % RING * UNIT * 1024;
#pragma unroll
        for (int i = 0; i < CPW; i++) {
            const uint32_t k = min(wave * CPW + i, (uint32_t)(UNIT - 1));        // (a repeat copies the same bytes)
            const uint32_t from = k + (k >= (uint32_t)(U::kV - K0) ? first_tile : 0u);
            lds_direct_load(to + k * 1024, base + (size_t)from * 1024, lane * 16);
        }
    };
    const size_t head_elems = (size_t)D * V;
    const float* in = a.state + ((size_t)s.state_in * a.heads + head) * head_elems;
    float* out = a.state + ((size_t)s.state_out * a.heads + head) * head_elems;
    auto seg_at = [&](uint32_t q) { return ((size_t)item * a.n_seg + q) * a.heads + head; };
    f32x4 S[2 * KT], gp[2 * KT];                                  // channels 16t + 4g + i, column col
#pragma unroll
    for (int t = 0; t < 2 * KT; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t d = 16 * t + 4 * g + i;
            if constexpr (CARRY) S[t][i] = values || d != col ? 0.f : 1.0f;
            else S[t][i] = (s.pos0 > 0 && d < D && col < V) ? in[(size_t)d * V + col] : 0.f;
            gp[t][i] = 1.0f;
        }
    if constexpr (!CARRY) {
        for (uint32_t q = 0; q < seg; q++) {                      // S <- X S + C of the segments before
            const float* C = a.seg_c + seg_at(q) * KP * CP + col;
            f32x4 next[2 * KT];
#pragma unroll
            for (int t = 0; t < 2 * KT; t++)
#pragma unroll
                for (int i = 0; i < 4; i++) next[t][i] = C[(size_t)(16 * t + 4 * g + i) * CP];
            if constexpr (DELTA) {
                RecurOp8<F32> So[KT];
#pragma unroll
                for (int k = 0; k < KT; k++) So[k] = recur_op8<F32>(S[2 * k], S[2 * k + 1]);
                const float* X = a.seg_x + seg_at(q) * KP * KP + (size_t)c * KP + 4 * g;
#pragma unroll
                for (int t = 0; t < 2 * KT; t++) {
#pragma unroll
                    for (int k = 0; k < KT; k++) {
                        const f32x4 lo = *reinterpret_cast<const f32x4*>(X + (size_t)16 * t * KP + 32 * k);
                        f32x4 hi = f32x4{0.f, 0.f, 0.f, 0.f};
                        if (32 * k + 16 < 16 * VT) hi = *reinterpret_cast<const f32x4*>(X + (size_t)16 * t * KP + 32 * k + 16);
                        next[t] = recur_mm(recur_op8<F32>(lo, hi), So[k], next[t]);
                    }
                    if constexpr (KT >= 4) __builtin_amdgcn_sched_barrier(0);    // (not every row's operands at once)
                }
            } else {
                const float* X = a.seg_x + seg_at(q) * KP + 4 * g;
#pragma unroll
                for (int t = 0; t < 2 * KT; t++) {
                    const f32x4 x = *reinterpret_cast<const f32x4*>(X + 16 * t);
#pragma unroll
                    for (int i = 0; i < 4; i++) next[t][i] = fmaf(x[i], S[t][i], next[t][i]);
                }
            }
#pragma unroll
            for (int t = 0; t < 2 * KT; t++) S[t] = next[t];
        }
    }
    // nothing of the state is on its way any more: what follows counts loads and stores
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    const uint32_t ldo = a.heads * CP, n = end - begin;
    float* o = a.o + ((size_t)(sub0 + begin) * kRecurSub + 4 * g) * ldo + head * CP + col;
    using Held = RecurHeld<F32, KT, DELTA, CARRY>;
    Held x, y;
#pragma unroll
    for (int i = 0; i < RING; i++) issue(i);
    asm volatile("s_waitcnt vmcnt(%0)\n\ts_barrier" ::"n"(FIRST) : "memory");
    x.fetch(recur_lds, wave, lane, g, values);
    // a step: the next stage has landed and is fetched into `after`, the stage of `now` (in registers everywhere) is
    // copied over, and `now` moves the state
    auto step = [&](uint32_t sub, const Held& now, Held& after) {
        if (sub < (uint32_t)RING - 1)
            asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(EARLY) : "memory");
        else
            asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(FULL) : "memory");
        issue(sub + RING);
        after.fetch(recur_lds + (sub + 1) % RING * UNIT * 1024, wave, lane, g, values);
        if constexpr (KT <= 2 && !DELTA) __builtin_amdgcn_sched_barrier(0);      // (left alone, the reads sink to their uses)
        RecurOp8<F32> So[KT];
        if constexpr (DELTA || !CARRY) {
#pragma unroll
            for (int t = 0; t < KT; t++) So[t] = recur_op8<F32>(S[2 * t], S[2 * t + 1]);
        }
        const f32x4 zero = f32x4{0.f, 0.f, 0.f, 0.f};
        f32x4 O = zero;
        if constexpr (DELTA) {
            const f32x4 P = recur_mm_many<KT>(now.W, So, recur_mm(now.M, now.V, zero));
            if constexpr (!CARRY) O = recur_mm_many<KT>(now.R, So, O);
#pragma unroll
            for (int t = 0; t < 2 * KT; t++)
#pragma unroll
                for (int i = 0; i < 4; i++) S[t][i] *= now.G[t][i];
            const RecurOp8<F32> VP = recur_join(now.V, recur_op4<F32>(P));
#pragma unroll
            for (int t = 0; t < 2 * KT; t++) S[t] = recur_mm(now.K8[t], VP, S[t]);
            if constexpr (!CARRY) O = recur_mm(now.A8, VP, O);
        } else {
#pragma unroll
            for (int t = 0; t < 2 * KT; t++)
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    S[t][i] *= now.G[t][i];
                    if constexpr (CARRY) gp[t][i] *= now.G[t][i];
                }
#pragma unroll
            for (int t = 0; t < 2 * KT; t++) S[t] = recur_mm(now.K4[t], now.V, S[t]);
            if constexpr (!CARRY) O = recur_mm_many<KT>(now.R, So, recur_mm(now.A4, now.V, O));
        }
        if constexpr (!CARRY) {
            // (rows past the request's end have room of their own)
#pragma unroll
            for (int i = 0; i < 4; i++) o[(size_t)i * ldo] = O[i];
            o += (size_t)kRecurSub * ldo;
        }
    };
    for (uint32_t sub = 0; sub < n; sub += 2) {                   // uniform
        step(sub, x, y);
        if (sub + 1 < n) step(sub + 1, y, x);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");              // the last copies still target the ring
    if constexpr (CARRY) {
        float* to = values ? a.seg_c + seg_at(seg) * KP * CP + col : a.seg_x + seg_at(seg) * KP * KP + col;
        const uint32_t ld = values ? CP : KP;
#pragma unroll
        for (int t = 0; t < 2 * KT; t++)
#pragma unroll
            for (int i = 0; i < 4; i++) to[(size_t)(16 * t + 4 * g + i) * ld] = S[t][i];
        if (!DELTA && first_tile + wave == 0 && c == 0) {
#pragma unroll
            for (int t = 0; t < 2 * KT; t++) *reinterpret_cast<f32x4*>(a.seg_x + seg_at(seg) * KP + 16 * t + 4 * g) = gp[t];
        }
        return;
    }
    if (end < n_sub) return;
#pragma unroll
    for (int t = 0; t < 2 * KT; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t d = 16 * t + 4 * g + i;
            if (d < D && col < V) out[(size_t)d * V + col] = S[t][i];
        }
}

// grid (chunks of 64 rows, heads): four threads a row
template <bool F32>
__global__ __launch_bounds__(256) void recur_gate_kernel(const RecurArgs a)
{
    using E = typename MixAct<F32>::E;
    const MixChunk ch = a.chunks[blockIdx.x];
    const uint32_t head = blockIdx.y, D = a.vdim, hd = head * D, vp = a.vtiles * 16;
    const float* norm = a.norm + head * a.norm_step;
    const uint32_t i = threadIdx.x / 4, q = threadIdx.x % 4;
    if (i >= ch.rows) return;                                     // (no barrier below)
    const uint32_t r = ch.row0 + i, npad = (a.heads * D + 31) / 32 * 32;
    const float* o = a.o + ((size_t)blockIdx.x * kMixChunk + i) * a.heads * vp + (size_t)head * vp;
    const float* g = a.in + (size_t)r * a.ld + a.col_g + hd;
    E* h = reinterpret_cast<E*>(a.h);
    float ss = 0.f;
    const bool whole = D % 8 == 0 && a.ld % 4 == 0 && a.col_g % 4 == 0 && a.col_h % 8 == 0;
    if (whole) {
        for (uint32_t d = q * 8; d < D; d += 32) {
            float v[8];
            mix_load8(o + d, v);
#pragma unroll
            for (int j = 0; j < 8; j++) ss = fmaf(v[j], v[j], ss);
        }
    } else {
        for (uint32_t d = q; d < D; d += 4) ss = fmaf(o[d], o[d], ss);
    }
    ss += wave_xor_f32(ss, 1);
    ss += wave_xor_f32(ss, 2);
    const float inv = a.out_scale / sqrtf(ss / (float)D + a.eps);
    if (whole) {
        for (uint32_t d = q * 8; d < D; d += 32) {
            float v[8], w[8], x[8];
            mix_load8(o + d, v);
            mix_load8(norm + d, w);
            if (a.gate != kRecurGateNone) {                       // (uniform)
                mix_load8(g + d, x);
#pragma unroll
                for (int j = 0; j < 8; j++) w[j] *= recur_gate(a, x[j]);
            }
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] *= inv * w[j];
            mix_store_unit<F32>(h, frag_unit(r, (a.col_h + hd + d) / 8, a.h_kt), v);
        }
    } else {
        for (uint32_t d = q; d < D; d += 4)
            h[frag_elem(r, a.col_h + hd + d, a.h_kt)] = (E)(o[d] * inv * norm[d] * (a.gate != kRecurGateNone ? recur_gate(a, g[d]) : 1.0f));
    }
    if (head + 1 == a.heads)
        for (uint32_t d = a.heads * D + q; d < npad; d += 4) h[frag_elem(r, a.col_h + d, a.h_kt)] = (E)0.f;
}

}  // namespace wr
