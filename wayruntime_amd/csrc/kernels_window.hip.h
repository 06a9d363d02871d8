// Attention over grouped keys and values inside a sliding window, or inside chunks of
// positions (a row sees its own chunk from the chunk's first position on).  Optionally each
// head has a sink s: its weights are exp(score) / (exp(s) + sum of exp(score)), so a row may
// attend to nothing at all.  Scores may be capped (cap * tanh(score / cap)), and a head's
// output gated, whole or element by element.  Values may be turned by their position like
// the keys; a row's output is then turned back by the row's.
//
// With two maps every head weighs the same values twice, by two queries over two keys, and
// its output is the first sum less `diff` times the second, over its root mean square.
// Prefill gives a wave the two maps of sixteen rows where it has 32 rows otherwise, so each
// value operand feeds both and the difference is taken in registers.  Decode takes both maps
// as columns of one product over keys twice as long, a column's query being zero where the
// other map's keys lie: one running softmax and one product with the values serve both.
//
// A page (64 positions) holds each key/value head's block one after the other:
//
//   K  [64/16][maps * dim_pad/32][64][8]  lane 16g + c of a tile: position 16s + c, elements 32k + 8g .. +8
//   V  [64/32][vdim_pad/16][64][8]    lane 16g + c of a tile: column 16t + c, element e of its eight:
//                                     position 32b + 16 (e / 4) + 4g + e % 4
//
// both the A operands of the products as they lie: scores S^T = K Q^T leave lane 16g + c with
// positions 4g .. 4g+3 of two 16-position halves for row c, which is the B operand of
// O^T = V^T P^T in the order V is stored.
//
//   window_append_kernel    queries normed and rotated into an operand, keys the same way and values into the cache
//   window_prefill_kernel   128 or 64 (token, head, map) rows of one key/value head a workgroup, a page at a
//                           time through LDS
//   window_decode_kernel    a workgroup per (token, key/value head, share of the keys)
//   window_attend_any_kernel  any geometry, both activation types
#pragma once

#include "kernels_latent_mfma.hip.h"

namespace wr {

struct WindowArgs {
    const MixSeq* seqs;
    const uint32_t *row_seq, *row_pos, *pages;
    uint32_t rows, heads, kvh, group;            // group = heads / kvh
    uint32_t dim, dimp, vdim, vdimp, half, window, chunk, norm_values;
    uint32_t maps, dimk, neighbours, key_heads;  // dimk = maps * dimp; key_heads: key/value heads to append (0 or kvh)
    float scale, out_scale, eps, softcap, diff;
    const float *q_norm, *k_norm, *gate;
    uint32_t ldg, gate_wide;                     // gate_wide: an element's own, head by head
    const float* vtable;                         // angles of the step's rows over the values, [rows][vdim / 2][2]
    void* cache;
    const float* in;
    uint32_t ld, col_q, col_k, col_v;
    const float *table, *sink;
    void *q, *o;
    uint32_t o_kt;
    // matrix forms
    const uint32_t* list;
    uint32_t n_list;
    const LatentRow* drows;
    uint32_t splits, split_keys;
    float *part_o, *part_ml;
};

// First position the row at `pos` sees.
__host__ __device__ __forceinline__ uint32_t window_lo(uint32_t pos, uint32_t window, uint32_t chunk)
{
    if (chunk) return pos - pos % chunk;
    return pos + 1 > window ? pos + 1 - window : 0;
}

// element of (position in page, column) inside a head's V block
__device__ __forceinline__ uint32_t window_v_elem(uint32_t at, uint32_t d, uint32_t vdimp)
{
    return (((at / 32) * (vdimp / 16) + d / 16) * 64 + 16 * (at % 16 / 4) + d % 16) * 8 + (at % 32 / 16) * 4 + at % 4;
}

constexpr uint32_t kWindowQUnits = 512;          // query units of eight a workgroup rotates

// Eight elements i0 .. i0 + 7 of the vector x, times inv and the norm's weights where there are any, rotated.
__device__ __forceinline__ void window_turn8(const WindowArgs& a, const float* x, const float* norm, float inv, const float* tab,
                                             uint32_t i0, float (&v)[8])
{
    if (!norm && !a.neighbours) {
        latent_rotate8(x, tab, i0, a.dim, a.half, v);
        return;
    }
    auto at = [&](uint32_t i) { return i < a.dim ? (norm ? x[i] * inv * norm[i] : x[i]) : 0.f; };
#pragma unroll
    for (uint32_t j = 0; j < 8; j += 2) {
        const uint32_t i = i0 + j;
        const float e = at(i), o = at(i + 1);
        if (a.neighbours) {
            const bool turn = i < 2 * a.half;
            const float c = turn ? tab[i] : 1.0f, sn = turn ? tab[i + 1] : 0.f;
            v[j] = e * c - o * sn;
            v[j + 1] = o * c + e * sn;
        } else {
#pragma unroll
            for (uint32_t k = 0; k < 2; k++) {
                const uint32_t d = i + k;
                const float own = k ? o : e;
                if (d < a.half) v[j + k] = own * tab[2 * d] - at(d + a.half) * tab[2 * d + 1];
                else if (d < 2 * a.half) v[j + k] = own * tab[2 * (d - a.half)] + at(d - a.half) * tab[2 * (d - a.half) + 1];
                else v[j + k] = own;
            }
        }
    }
}

// One over the root mean square of the vector x, whose units of eight (this thread's: i0 ..) are held by every fourth
// lane of a run of lanes.
__device__ __forceinline__ float window_inv_rms(const WindowArgs& a, const float* x, uint32_t i0)
{
    float ss = 0.f;
    if (a.dimp == 32 || a.dimp == 64 || a.dimp == 128) {
#pragma unroll
        for (uint32_t j = 0; j < 8; j++) {
            const float e = i0 + j < a.dim ? x[i0 + j] : 0.f;
            ss = fmaf(e, e, ss);
        }
        ss += wave_xor_f32(ss, 4);
        ss += wave_xor_f32(ss, 8);
        if (a.dimp >= 64) ss += wave_xor_f32(ss, 16);
        if (a.dimp >= 128) ss += wave_xor_f32(ss, 32);
    } else {
        for (uint32_t i = 0; i < a.dim; i++) ss = fmaf(x[i], x[i], ss);
    }
    return 1.0f / sqrtf(ss / (float)a.dim + a.eps);
}

// Whether units of eight lie whole inside a vector and inside or outside its rotated part, so that they go in as vectors.
__device__ __forceinline__ bool window_whole(const WindowArgs& a, uint32_t col)
{
    return a.neighbours && a.dim % 8 == 0 && a.half % 4 == 0 && a.ld % 4 == 0 && col % 4 == 0 && (a.dimp == 32 || a.dimp == 64 || a.dimp == 128);
}

// Unit i0 .. i0 + 7 of the vector x, normed and rotated (neighbours): the other units of x are held by every fourth lane.
__device__ __forceinline__ void window_unit(const WindowArgs& a, const float* x, const float* norm, const float* tab, uint32_t i0,
                                            float (&v)[8])
{
    const bool some = i0 < a.dim;
    if (some) {
        mix_load8(x + i0, v);
    } else {
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = 0.f;
    }
    if (norm) {                                            // uniform
        float ss = 0.f, w[8];
#pragma unroll
        for (int j = 0; j < 8; j++) ss = fmaf(v[j], v[j], ss);
        ss += wave_xor_f32(ss, 4);
        ss += wave_xor_f32(ss, 8);
        if (a.dimp >= 64) ss += wave_xor_f32(ss, 16);
        if (a.dimp >= 128) ss += wave_xor_f32(ss, 32);
        const float inv = 1.0f / sqrtf(ss / (float)a.dim + a.eps);
        if (some) {
            mix_load8(norm + i0, w);
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] *= inv * w[j];
        }
    }
    if (i0 < 2 * a.half) {
        float cs[8];
        mix_load8(tab + i0, cs);
#pragma unroll
        for (int j = 0; j < 8; j += 2) {
            const float e = v[j], o = v[j + 1];
            v[j] = e * cs[j] - o * cs[j + 1];
            v[j + 1] = o * cs[j] + e * cs[j + 1];
        }
    }
}

// Element d of row r's value, turned where values are.
__device__ __forceinline__ float window_value(const WindowArgs& a, uint32_t r, uint32_t kvh, uint32_t d)
{
    const float* v = a.in + (size_t)r * a.ld + a.col_v + kvh * a.vdim;
    if (!a.vtable) return v[d];                            // uniform
    const float* cs = a.vtable + (size_t)r * a.vdim + (d & ~1u);
    return v[d] * cs[0] + (d & 1 ? v[d - 1] : -v[d + 1]) * cs[1];
}

// grid (rows / 4, key_heads + slices of 4 rows' query units)
template <bool F32>
__global__ __launch_bounds__(256) void window_append_kernel(const WindowArgs a)
{
    using E = typename MixAct<F32>::E;
    using V4 = typename MixAct<F32>::V4;
    __shared__ float s_inv[4];
    const uint32_t t = threadIdx.x, r0 = blockIdx.x * 4, n = min(4u, a.rows - r0), per_map = a.dimp / 8;
    const bool whole = window_whole(a, blockIdx.y >= a.key_heads ? a.col_q : a.col_k);       // uniform
    if (blockIdx.y >= a.key_heads) {
        const uint32_t per = a.heads * a.maps * per_map, u0 = (blockIdx.y - a.key_heads) * kWindowQUnits;
        for (uint32_t u = u0 + t; u < min(u0 + kWindowQUnits, 4 * per); u += 256) {
            const uint32_t i = u % 4, q = u / 4, r = r0 + min(i, n - 1);
            const float* x = a.in + (size_t)r * a.ld + a.col_q + q / per_map * a.dim;
            float v[8];
            if (whole) {
                window_unit(a, x, a.q_norm, a.table + (size_t)r * 2 * a.half, q % per_map * 8, v);
                if (i < n) mix_store_unit<F32>(a.q, frag_unit(r, q, a.heads * (a.dimk / 32)), v);
                continue;
            }
            const float inv = a.q_norm ? window_inv_rms(a, x, q % per_map * 8) : 1.0f;
            if (i >= n) continue;
            window_turn8(a, x, a.q_norm, inv, a.table + (size_t)r * 2 * a.half, q % per_map * 8, v);
            mix_store_unit<F32>(a.q, frag_unit(r, q, a.heads * (a.dimk / 32)), v);
        }
        return;
    }
    const uint32_t kvh = blockIdx.y, block = kMixPage * (a.dimk + a.vdimp);
    auto head_block = [&](uint32_t r) {
        const MixSeq s = a.seqs[a.row_seq[r]];
        return reinterpret_cast<E*>(a.cache) + ((size_t)a.pages[s.page0 + a.row_pos[r] / kMixPage] * a.kvh + kvh) * block;
    };
    for (uint32_t u = t; u < 4 * a.maps * per_map; u += 256) {
        const uint32_t i = u % 4, q = u / 4, r = r0 + min(i, n - 1);
        const float* x = a.in + (size_t)r * a.ld + a.col_k + (kvh * a.maps + q / per_map) * a.dim;
        float v[8];
        if (whole) {
            window_unit(a, x, a.k_norm, a.table + (size_t)r * 2 * a.half, q % per_map * 8, v);
            if (i < n) mix_store_unit<F32>(head_block(r), frag_unit(a.row_pos[r] % kMixPage, q, a.dimk / 32), v);
            continue;
        }
        const float inv = a.k_norm ? window_inv_rms(a, x, q % per_map * 8) : 1.0f;
        if (i >= n) continue;
        window_turn8(a, x, a.k_norm, inv, a.table + (size_t)r * 2 * a.half, q % per_map * 8, v);
        mix_store_unit<F32>(head_block(r), frag_unit(a.row_pos[r] % kMixPage, q, a.dimk / 32), v);
    }
    const uint32_t wave = t >> 6, lane = t & 63;
    if (wave < n) {
        float ss = 0.f;
        if (a.norm_values) {
            const float* v = a.in + (size_t)(r0 + wave) * a.ld + a.col_v + kvh * a.vdim;
            for (uint32_t d = lane; d < a.vdim; d += 64) ss = fmaf(v[d], v[d], ss);
#pragma unroll
            for (int off = 32; off >= 1; off >>= 1) ss += wave_xor_f32(ss, off);
        }
        if (lane == 0) s_inv[wave] = a.norm_values ? 1.0f / sqrtf(ss / (float)a.vdim + a.eps) : 1.0f;
    }
    __syncthreads();
    const uint32_t p0 = a.row_pos[r0];
    const bool run = n == 4 && p0 % 4 == 0 && a.row_seq[r0] == a.row_seq[r0 + 3];
    for (uint32_t d = t; d < a.vdimp; d += 256) {
        V4 x;
#pragma unroll
        for (uint32_t i = 0; i < 4; i++)
            x[i] = (E)(i < n && d < a.vdim ? window_value(a, r0 + min(i, n - 1), kvh, d) * s_inv[i] : 0.f);
        if (run) {                                         // four positions of one column side by side
            *reinterpret_cast<V4*>(head_block(r0) + kMixPage * a.dimk + window_v_elem(p0 % kMixPage, d, a.vdimp)) = x;
        } else {
            for (uint32_t i = 0; i < n; i++)
                head_block(r0 + i)[kMixPage * a.dimk + window_v_elem(a.row_pos[r0 + i] % kMixPage, d, a.vdimp)] = x[i];
        }
    }
}

// What head h's output of row r is multiplied by, besides what its own sum calls for.
template <bool F32>
__device__ __forceinline__ float window_factor(const WindowArgs& a, uint32_t r, uint32_t h)
{
    return a.gate && !a.gate_wide ? a.out_scale * mix_sigmoid<F32>(a.gate[(size_t)r * a.ldg + h]) : a.out_scale;
}

// Column col of head h's output of row r, turned back and times the element's gate; pair: the column it is paired with.
template <bool F32>
__device__ __forceinline__ float window_finish(const WindowArgs& a, uint32_t r, uint32_t h, uint32_t col, float v, float pair)
{
    if (col >= a.vdim) return v;                           // (zeros)
    if (a.vtable) {                                        // uniform, like the gate
        const float* cs = a.vtable + (size_t)r * a.vdim + (col & ~1u);
        v = v * cs[0] + (col & 1 ? -pair : pair) * cs[1];
    }
    return a.gate_wide ? v * mix_sigmoid<F32>(a.gate[(size_t)r * a.ldg + h * a.vdim + col]) : v;
}

// Columns col .. col + 3 of it (col a multiple of four).
__device__ __forceinline__ f32x4 window_finish4(const WindowArgs& a, uint32_t r, uint32_t h, uint32_t col, f32x4 v)
{
    if (a.vdim % 4 == 0) {
        if (col >= a.vdim) return v;
        if (a.vtable) {
            const f32x4 cs = *reinterpret_cast<const f32x4*>(a.vtable + (size_t)r * a.vdim + col);
            v = f32x4{v[0] * cs[0] + v[1] * cs[1], v[1] * cs[0] - v[0] * cs[1], v[2] * cs[2] + v[3] * cs[3], v[3] * cs[2] - v[2] * cs[3]};
        }
        if (a.gate_wide) {
            const f32x4 gt = *reinterpret_cast<const f32x4*>(a.gate + (size_t)r * a.ldg + h * a.vdim + col);
#pragma unroll
            for (int i = 0; i < 4; i++) v[i] *= mix_sigmoid<false>(gt[i]);
        }
        return v;
    }
    f32x4 o;
#pragma unroll
    for (int i = 0; i < 4; i++) o[i] = window_finish<false>(a, r, h, col + i, v[i], v[i ^ 1]);
    return o;
}

// One wave per (row, head), a lane per key of a page.  LDS: a query row and every map's output row as floats, 64 weights.
template <bool F32>
__global__ __launch_bounds__(64) void window_attend_any_kernel(const WindowArgs a)
{
    using E = typename MixAct<F32>::E;
    using V8 = typename MixAct<F32>::V8;
    extern __shared__ __attribute__((aligned(16))) float window_smem[];
    const uint32_t lane = threadIdx.x, r = blockIdx.x, h = blockIdx.y, kd = a.dimk / 32, per_map = a.dimp / 8;
    float *q = window_smem, *w = q + a.dimp, *outs = w + 64;
    const V8* qf = reinterpret_cast<const V8*>(a.q);
    const MixSeq s = a.seqs[a.row_seq[r]];
    const uint32_t pos = a.row_pos[r], lo = window_lo(pos, a.window, a.chunk);
    for (uint32_t m = 0; m < a.maps; m++) {
        float* o = outs + m * a.vdimp;
        for (uint32_t u = lane; u < per_map; u += 64) {
            const V8 x = qf[frag_unit(r, h * kd * 4 + m * per_map + u, a.heads * kd)];
#pragma unroll
            for (int j = 0; j < 8; j++) q[u * 8 + j] = (float)x[j];
        }
        for (uint32_t k = lane; k < a.vdimp; k += 64) o[k] = 0.f;
        __syncthreads();
        float mx = a.sink ? a.sink[h] : -INFINITY, sum = a.sink ? 1.0f : 0.f;
        for (uint32_t j0 = lo / kMixPage * kMixPage; j0 <= pos; j0 += kMixPage) {
            const uint32_t j = j0 + lane;
            const V8* page = reinterpret_cast<const V8*>(
                reinterpret_cast<const E*>(a.cache) +
                ((size_t)a.pages[s.page0 + j0 / kMixPage] * a.kvh + h / a.group) * kMixPage * (a.dimk + a.vdimp));
            float sc = 0.f;
            for (uint32_t u = 0; u < per_map; u++) {
                const V8 x = page[frag_unit(lane, m * per_map + u, kd)];
#pragma unroll
                for (int e = 0; e < 8; e++) sc = fmaf((float)x[e], q[u * 8 + e], sc);
            }
            sc *= a.scale;
            if (a.softcap > 0.f) sc = a.softcap * tanhf(sc / a.softcap);
            sc = (j >= lo && j <= pos) ? sc : -INFINITY;
            float bm = sc;
#pragma unroll
            for (int off = 32; off >= 1; off >>= 1) bm = fmaxf(bm, wave_xor_f32(bm, off));
            const float nm = fmaxf(mx, bm), p = expf(sc - nm), corr = expf(mx - nm);
            float bs = p;
#pragma unroll
            for (int off = 32; off >= 1; off >>= 1) bs += wave_xor_f32(bs, off);
            sum = sum * corr + bs;
            mx = nm;
            w[lane] = p;
            __syncthreads();
            const V8* vb = page + kMixPage * a.dimk / 8;
            for (uint32_t k = lane; k < a.vdimp; k += 64) {
                float acc = o[k] * corr;
                for (uint32_t u = 0; u < 8; u++) {         // 32-position block u / 4, lane group u % 4
                    const V8 x = vb[(u / 4 * (a.vdimp / 16) + k / 16) * 64 + 16 * (u % 4) + k % 16];
#pragma unroll
                    for (int e = 0; e < 8; e++) {
                        // (positions past the row's own may hold anything: their weight is zero, their value is not used)
                        const float p8 = w[32 * (u / 4) + 16 * (e / 4) + 4 * (u % 4) + e % 4];
                        acc = fmaf(p8, p8 != 0.f ? (float)x[e] : 0.f, acc);
                    }
                }
                o[k] = acc;
            }
            __syncthreads();
        }
        for (uint32_t k = lane; k < a.vdimp; k += 64) o[k] /= sum;     // (this lane's own columns, here and below)
    }
    float factor = window_factor<F32>(a, r, h);
    if (a.maps == 2) {
        float ss = 0.f;
        for (uint32_t k = lane; k < a.vdimp; k += 64) {
            outs[k] -= a.diff * outs[a.vdimp + k];
            ss = fmaf(outs[k], outs[k], ss);
        }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) ss += wave_xor_f32(ss, off);
        factor /= sqrtf(ss / (float)a.vdim + a.eps);
    }
    E* out = reinterpret_cast<E*>(a.o);
    __syncthreads();                                       // (a pair's other column is another lane's)
    for (uint32_t k = lane; k < a.vdimp; k += 64)
        out[frag_elem(r, h * a.vdimp + k, a.o_kt)] = (E)(window_finish<F32>(a, r, h, k, outs[k], outs[k ^ 1u]) * factor);
}

// ---- matrix forms (bfloat16; head sizes padded to 32, 64 or 128) -------------

// Products to scores in units of log2 e: times mul, and with cap > 0 (its own log2 e in it) capped; a capped score's mul
// is 2 log2 e times scale over cap.
struct WindowScore {
    float mul, cap;
    __device__ __forceinline__ explicit WindowScore(const WindowArgs& a)
        : mul(a.softcap > 0.f ? a.scale / a.softcap * 2.0f * kLog2e : a.scale * kLog2e), cap(a.softcap * kLog2e) {}
};

// The running softmax of one row tile over N x 16 keys from j0 on; s[n][i]: product with key j0 + 16n + 4g + i.
// Leaves the probabilities in s and returns by how much the old sums shrink.
template <int N, bool MASK>
__device__ __forceinline__ float window_softmax(f32x4 (&s)[N], uint32_t j0, int g, uint32_t lo, uint32_t pos, WindowScore score,
                                                float& mx, float& sum)
{
    float bm = kLatentNone;
    if (score.cap > 0.f) {                                 // uniform; tanh(x) = 1 - 2 / (exp(2x) + 1)
#pragma unroll
        for (int n = 0; n < N; n++)
#pragma unroll
            for (int i = 0; i < 4; i++)
                s[n][i] = score.cap - 2.0f * score.cap * __builtin_amdgcn_rcpf(fast_exp2(s[n][i] * score.mul) + 1.0f);
    } else {
#pragma unroll
        for (int n = 0; n < N; n++)
#pragma unroll
            for (int i = 0; i < 4; i++) s[n][i] *= score.mul;
    }
#pragma unroll
    for (int n = 0; n < N; n++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            if constexpr (MASK) {
                const uint32_t j = j0 + 16 * n + 4 * g + i;
                if (j < lo || j > pos) s[n][i] = kLatentNone;
            }
            bm = fmaxf(bm, s[n][i]);
        }
    bm = fmaxf(bm, wave_xor_f32(bm, 16));
    bm = fmaxf(bm, wave_xor_f32(bm, 32));
    const float nm = fmaxf(mx, bm), corr = fast_exp2(mx - nm);
    mx = nm;
    float bs = 0.f;
#pragma unroll
    for (int n = 0; n < N; n++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            float e = fast_exp2(s[n][i] - nm);
            if constexpr (MASK) e = s[n][i] > 0.5f * kLatentNone ? e : 0.f;
            bs += e;
            s[n][i] = e;
        }
    bs += wave_xor_f32(bs, 16);
    bs += wave_xor_f32(bs, 32);
    sum = sum * corr + bs;
    return corr;
}

__device__ __forceinline__ bf16x8 window_pack(f32x4 a, f32x4 b)
{
    bf16x8 p;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        p[i] = (__bf16)a[i];
        p[4 + i] = (__bf16)b[i];
    }
    return p;
}


constexpr size_t window_prefill_lds(int kq, int vt) { return (size_t)2 * 4 * (kq + vt) * 1024; }

// The difference of two maps' outputs of one row, each over its own sum: over its root mean square times factor.
// a, b: this lane's columns; the row's others are held by the lanes 16 and 32 away.
template <int N>
__device__ __forceinline__ float window_difference(const WindowArgs& a, f32x4 (&x)[N], const f32x4 (&y)[N], float ix, float iy)
{
    float ss = 0.f;
    iy *= a.diff;
#pragma unroll
    for (int k = 0; k < N; k++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            x[k][i] = x[k][i] * ix - y[k][i] * iy;
            ss = fmaf(x[k][i], x[k][i], ss);
        }
    ss += wave_xor_f32(ss, 16);
    ss += wave_xor_f32(ss, 32);
    return 1.0f / sqrtf(ss / (float)a.vdim + a.eps);
}

// KQ, VT: head sizes in tiles of 32.  Grid: tiles of 64 NR (token, head of the group, map) rows times key/value heads, the
// key/value head innermost: with eight of them each XCD keeps to one.  A wave's two row tiles are 32 rows, or the two
// maps of 16.
template <int KQ, int VT, int MAPS, int NR>
__global__ __launch_bounds__(256, 2) void window_prefill_kernel(const WindowArgs a)
{
    static_assert(NR % MAPS == 0, "a wave has all maps of its rows");
    constexpr int CPW = MAPS * KQ + VT, STAGE = 4 * CPW * 1024, WROWS = 16 * NR / MAPS, ROWS = 4 * WROWS;
    extern __shared__ __attribute__((aligned(16))) unsigned char window_lds[];
    const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t kvh = blockIdx.x % a.kvh, H = a.group;
    uint32_t tile = blockIdx.x / a.kvh, pick_seq = 0, n_tiles = 0;
    for (uint32_t i = 0; i < a.n_list; i++) {
        n_tiles = (a.seqs[a.list[i]].rows * H + ROWS - 1) / ROWS;
        pick_seq = a.list[i];
        if (tile < n_tiles) break;
        tile -= n_tiles;
    }
    tile = n_tiles - 1 - tile;                             // the last tiles see the most keys and go first
    const MixSeq s = a.seqs[pick_seq];
    const uint32_t m_end = s.rows * H, m0 = tile * ROWS;
    const uint32_t pos_first = s.pos0 + m0 / H, pos_last = s.pos0 + (min(m0 + ROWS, m_end) - 1) / H;
    const uint32_t j_begin = window_lo(pos_first, a.window, a.chunk) / kMixPage * kMixPage, j_end = pos_last + 1;
    const WindowScore score(a);

    uint32_t m[NR], pos[NR], lo[NR];
    bf16x8 qv[NR][KQ];
    float mx[NR], sum[NR];
#pragma unroll
    for (int t = 0; t < NR; t++) {
        m[t] = m0 + wave * WROWS + (MAPS == 1 ? t * 16 : 0) + c;
        const uint32_t mm = min(m[t], m_end - 1), head = kvh * H + mm % H;
        pos[t] = s.pos0 + mm / H;
        lo[t] = window_lo(pos[t], a.window, a.chunk);
#pragma unroll
        for (int k = 0; k < KQ; k++)
            qv[t][k] = reinterpret_cast<const bf16x8*>(a.q)[frag_unit(
                s.row0 + mm / H, ((MAPS == 1 ? head : head * MAPS + t) * KQ + k) * 4 + g, a.heads * MAPS * KQ)];
        mx[t] = a.sink ? a.sink[head] * kLog2e : kLatentNone;
        sum[t] = a.sink ? 1.0f : 0.f;
    }
    // positions this wave's rows span: a page between them needs no mask
    const uint32_t w0 = min(m0 + wave * WROWS, m_end - 1), w1 = min(m0 + wave * WROWS + WROWS - 1, m_end - 1);
    const uint32_t w_pos0 = s.pos0 + w0 / H, w_pos1 = s.pos0 + w1 / H;
    const uint32_t w_lo0 = window_lo(w_pos0, a.window, a.chunk), w_lo1 = window_lo(w_pos1, a.window, a.chunk);
    f32x4 acc[NR][2 * VT];
#pragma unroll
    for (int t = 0; t < NR; t++)
#pragma unroll
        for (int k = 0; k < 2 * VT; k++) acc[t][k] = f32x4{0.f, 0.f, 0.f, 0.f};

    const uint32_t lds0 = (uint32_t)__builtin_amdgcn_readfirstlane((uint32_t)(uintptr_t)window_lds);
    auto issue = [&](uint32_t j0, uint32_t stage) {        // a head's block of a page is contiguous
        const uint32_t page = (uint32_t)__builtin_amdgcn_readfirstlane(a.pages[s.page0 + j0 / kMixPage]);
        const unsigned char* base = uniform_ptr(reinterpret_cast<const unsigned char*>(a.cache) + ((size_t)page * a.kvh + kvh) * STAGE);
#pragma unroll
        for (int i = 0; i < CPW; i++) {
            const uint32_t ch = wave * CPW + i;
            lds_direct_load(lds0 + stage * STAGE + ch * 1024, base + (size_t)ch * 1024, lane * 16);
        }
    };
    issue(j_begin, 0);
    uint32_t stage = 0;
    for (uint32_t j0 = j_begin; j0 < j_end; j0 += kMixPage, stage ^= 1) {
        // this page has landed, everybody is done with the one before
        asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
        if (j0 + kMixPage < j_end) issue(j0 + kMixPage, stage ^ 1);
        if (j0 > w_pos1 || j0 + kMixPage <= w_lo0) continue;              // uniform over the wave: none of its keys
        const bf16x8* kt = reinterpret_cast<const bf16x8*>(window_lds + stage * STAGE) + lane;
        const bf16x8* vt = kt + 4 * MAPS * KQ * 64;
        f32x4 sc[NR][4];
#pragma unroll
        for (int t = 0; t < NR; t++)
#pragma unroll
            for (int n = 0; n < 4; n++) sc[t][n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KQ; k++)
#pragma unroll
            for (int n = 0; n < 4; n++) {
                if constexpr (MAPS == 1) {
                    const bf16x8 kv = kt[(n * KQ + k) * 64];
#pragma unroll
                    for (int t = 0; t < NR; t++) sc[t][n] = mix_mfma(kv, qv[t][k], sc[t][n]);
                } else {
#pragma unroll
                    for (int t = 0; t < NR; t++) sc[t][n] = mix_mfma(kt[((n * MAPS + t) * KQ + k) * 64], qv[t][k], sc[t][n]);
                }
            }
        const bool inside = j0 + kMixPage - 1 <= w_pos0 && j0 >= w_lo1;
        bf16x8 p[NR][2];
#pragma unroll
        for (int t = 0; t < NR; t++) {
            const float corr = inside ? window_softmax<4, false>(sc[t], j0, g, lo[t], pos[t], score, mx[t], sum[t])
                                      : window_softmax<4, true>(sc[t], j0, g, lo[t], pos[t], score, mx[t], sum[t]);
            if (__any(corr != 1.0f)) {
#pragma unroll
                for (int k = 0; k < 2 * VT; k++)
#pragma unroll
                    for (int i = 0; i < 4; i++) acc[t][k][i] *= corr;
            }
            p[t][0] = window_pack(sc[t][0], sc[t][1]);
            p[t][1] = window_pack(sc[t][2], sc[t][3]);
        }
#pragma unroll
        for (int b = 0; b < 2; b++)
#pragma unroll
            for (int k = 0; k < 2 * VT; k++) {
                const bf16x8 v = vt[(b * 2 * VT + k) * 64];
#pragma unroll
                for (int t = 0; t < NR; t++) acc[t][k] = mix_mfma(v, p[t][b], acc[t][k]);
            }
    }
    __bf16* out = reinterpret_cast<__bf16*>(a.o);
    float norm = 1.0f;
    if constexpr (MAPS == 2) norm = window_difference(a, acc[0], acc[1], 1.0f / sum[0], 1.0f / sum[1]);
#pragma unroll
    for (int t = 0; t < NR / MAPS; t++) {
        if (m[t] >= m_end) continue;
        const uint32_t r = s.row0 + m[t] / H, h = kvh * H + m[t] % H;
        const float inv = window_factor<false>(a, r, h) * (MAPS == 2 ? norm : 1.0f / sum[t]);
#pragma unroll
        for (int k = 0; k < 2 * VT; k++) {
            bf16x4 o;
            const f32x4 v = window_finish4(a, r, h, k * 16 + 4 * g, acc[t][k]);
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] = (__bf16)(v[i] * inv);
            *reinterpret_cast<bf16x4*>(out + frag_elem(r, h * VT * 32 + k * 16 + 4 * g, a.o_kt)) = o;
        }
    }
}

// grid (rows of the launch * kvh * tiles of 16 (head, map) columns of a group, splits).  The four waves take every fourth
// block of 32 keys of the share, straight into registers, one block ahead.  KQ: tiles of all maps' keys.
template <int KQ, int VT, int MAPS>
__global__ __launch_bounds__(256, KQ + VT > 8 ? 1 : 2) void window_decode_kernel(const WindowArgs a)
{
    __shared__ f32x4 box[3 * (2 * VT + 1) * 64];
    const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t columns = a.group * MAPS, tiles = (columns + 15) / 16, split = blockIdx.y;
    const uint32_t kvh = blockIdx.x % a.kvh, tile = blockIdx.x / a.kvh % tiles, ri = blockIdx.x / a.kvh / tiles;
    const LatentRow lr = a.drows[ri];
    const uint32_t r = lr.row, pos = lr.pos, lo = window_lo(pos, a.window, a.chunk);
    const uint32_t first = lo / 32 * 32 + split * a.split_keys, end = min(pos + 1, first + a.split_keys);
    const WindowScore score(a);
    const uint32_t member = tile * 16 + c, column = min(member, columns - 1), head = kvh * a.group + column / MAPS, map = column % MAPS;

    bf16x8 kA[2 * KQ], vA[2 * VT], kB[2 * KQ], vB[2 * VT];
    const uint32_t j_last = pos / 32 * 32;                 // (a block past the end reads the last one again)
    auto load = [&](bf16x8 (&k)[2 * KQ], bf16x8 (&v)[2 * VT], uint32_t j) {
        const uint32_t j0 = min(j, j_last);
        const uint32_t page = (uint32_t)__builtin_amdgcn_readfirstlane(a.pages[lr.page0 + j0 / kMixPage]), b = j0 % kMixPage / 32;
        const bf16x8* base = reinterpret_cast<const bf16x8*>(a.cache) + ((size_t)page * a.kvh + kvh) * 4 * (KQ + VT) * 64 + lane;
#pragma unroll
        for (int i = 0; i < 2 * KQ; i++) k[i] = __builtin_nontemporal_load(&base[(b * 2 * KQ + i) * 64]);
#pragma unroll
        for (int i = 0; i < 2 * VT; i++) v[i] = __builtin_nontemporal_load(&base[(4 * KQ + b * 2 * VT + i) * 64]);
    };
    bf16x8 qv[KQ];
#pragma unroll
    for (int k = 0; k < KQ; k++) {
        qv[k] = reinterpret_cast<const bf16x8*>(a.q)[frag_unit(r, (head * KQ + k) * 4 + g, a.heads * KQ)];
        if (MAPS > 1 && (uint32_t)k / (KQ / MAPS) != map) {
#pragma unroll
            for (int i = 0; i < 8; i++) qv[k][i] = (__bf16)0.f;
        }
    }
    f32x4 acc[2 * VT];
#pragma unroll
    for (int k = 0; k < 2 * VT; k++) acc[k] = f32x4{0.f, 0.f, 0.f, 0.f};
    const bool sinks = a.sink && split == 0 && wave == 0;
    float mx = sinks ? a.sink[head] * kLog2e : kLatentNone, sum = sinks ? 1.0f : 0.f;
    auto step = [&](const bf16x8 (&k)[2 * KQ], const bf16x8 (&v)[2 * VT], uint32_t j0) {
        if (j0 >= end) return;                             // uniform over the wave
        f32x4 sc[2];
        sc[0] = sc[1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < KQ; i++) {
            sc[0] = mix_mfma(k[i], qv[i], sc[0]);
            sc[1] = mix_mfma(k[KQ + i], qv[i], sc[1]);
        }
        const float corr = window_softmax<2, true>(sc, j0, g, lo, end - 1, score, mx, sum);
        if (__any(corr != 1.0f)) {
#pragma unroll
            for (int i = 0; i < 2 * VT; i++)
#pragma unroll
                for (int x = 0; x < 4; x++) acc[i][x] *= corr;
        }
        const bf16x8 p = window_pack(sc[0], sc[1]);
#pragma unroll
        for (int i = 0; i < 2 * VT; i++) acc[i] = mix_mfma(v[i], p, acc[i]);
    };
    uint32_t j = first + wave * 32;
    if (j < end) {
        load(kA, vA, j);
        for (; j < end; j += 256) {
            load(kB, vB, j + 128);
            step(kA, vA, j);
            load(kA, vA, j + 256);
            step(kB, vB, j + 128);
        }
    }
    constexpr int BOX = (2 * VT + 1) * 64;
    if (wave) {
        f32x4* to = box + (wave - 1) * BOX + lane;
#pragma unroll
        for (int k = 0; k < 2 * VT; k++) to[k * 64] = acc[k];
        to[2 * VT * 64] = f32x4{mx, sum, 0.f, 0.f};
    }
    __syncthreads();
    if (wave) return;
    for (int o = 0; o < 3; o++) {
        const f32x4* from = box + o * BOX + lane;
        const f32x4 ml = from[2 * VT * 64];
        const float nm = fmaxf(mx, ml[0]), s0 = fast_exp2(mx - nm), s1 = fast_exp2(ml[0] - nm);
        mx = nm;
        sum = sum * s0 + ml[1] * s1;
#pragma unroll
        for (int k = 0; k < 2 * VT; k++) {
            const f32x4 v = from[k * 64];
#pragma unroll
            for (int i = 0; i < 4; i++) acc[k][i] = acc[k][i] * s0 + v[i] * s1;
        }
    }
    if (member >= columns) return;                         // (the two maps of a head go together)
    if (a.splits == 1) {
        float inv = window_factor<false>(a, r, head);
        if constexpr (MAPS == 2) {                         // the other map is the next lane's
            f32x4 other[2 * VT];
#pragma unroll
            for (int k = 0; k < 2 * VT; k++)
#pragma unroll
                for (int i = 0; i < 4; i++) other[k][i] = wave_xor_f32(acc[k][i], 1);
            inv *= window_difference(a, acc, other, 1.0f / sum, 1.0f / wave_xor_f32(sum, 1));
            if (map) return;
        } else {
            inv /= sum;
        }
        __bf16* out = reinterpret_cast<__bf16*>(a.o);
#pragma unroll
        for (int k = 0; k < 2 * VT; k++) {
            bf16x4 o;
            const f32x4 v = window_finish4(a, r, head, k * 16 + 4 * g, acc[k]);
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] = (__bf16)(v[i] * inv);
            *reinterpret_cast<bf16x4*>(out + frag_elem(r, head * VT * 32 + k * 16 + 4 * g, a.o_kt)) = o;
        }
        return;
    }
    const size_t at = (((size_t)ri * a.heads + head) * MAPS + map) * a.splits + split;
    if (g == 0) {
        a.part_ml[at * 2] = mx;
        a.part_ml[at * 2 + 1] = sum;
    }
#pragma unroll
    for (int k = 0; k < 2 * VT; k++) *reinterpret_cast<f32x4*>(a.part_o + at * VT * 32 + k * 16 + 4 * g) = acc[k];
}

constexpr uint32_t kWindowSplits = 64;          // shares of the keys at most: a lane each

// grid (rows of the launch, heads), a wave per map: the shares of one row and head together
template <int VT, int MAPS>
__global__ __launch_bounds__(64 * MAPS) void window_combine_kernel(const WindowArgs a)
{
    constexpr int COLS = (VT * 32 + 63) / 64;
    __shared__ float wt[MAPS][kWindowSplits], second[MAPS == 2 ? COLS * 64 : 1];
    const uint32_t h = blockIdx.y, r = a.drows[blockIdx.x].row, t = threadIdx.x & 63, map = threadIdx.x >> 6;
    const size_t at = (((size_t)blockIdx.x * a.heads + h) * MAPS + map) * a.splits;
    const bool has = t < a.splits;
    const float m = has ? a.part_ml[(at + t) * 2] : kLatentNone, l = has ? a.part_ml[(at + t) * 2 + 1] : 0.f;
    float factor = window_factor<false>(a, r, h);
    const float mx = mix_wave_max(m);
    const float w = l != 0.f ? fast_exp2(m - mx) : 0.f;    // zero: a share past the row's keys
    float sum = w * l;
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) sum += wave_xor_f32(sum, off);
    const float inv = 1.0f / sum;
    wt[map][t] = w * inv;
    __syncthreads();
    float o[COLS];
#pragma unroll
    for (int i = 0; i < COLS; i++) {
        const uint32_t col = t + 64 * i;
        o[i] = 0.f;
        if (col >= VT * 32) continue;
#pragma unroll 4
        for (uint32_t s = 0; s < a.splits; s++) o[i] = fmaf(wt[map][s], a.part_o[(at + s) * VT * 32 + col], o[i]);
    }
    if constexpr (MAPS == 2) {
        if (map) {
#pragma unroll
            for (int i = 0; i < COLS; i++) second[t + 64 * i] = o[i];
        }
        __syncthreads();
        if (map) return;
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < COLS; i++) {
            o[i] -= a.diff * second[t + 64 * i];
            ss = fmaf(o[i], o[i], ss);
        }
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) ss += wave_xor_f32(ss, off);
        factor /= sqrtf(ss / (float)a.vdim + a.eps);
    }
    __bf16* out = reinterpret_cast<__bf16*>(a.o);
#pragma unroll
    for (int i = 0; i < COLS; i++) {
        const uint32_t col = t + 64 * i;
        const float pair = wave_xor_f32(o[i], 1);
        if (col < VT * 32) out[frag_elem(r, h * VT * 32 + col, a.o_kt)] = (__bf16)(window_finish<false>(a, r, h, col, o[i], pair) * factor);
    }
}

}  // namespace wr
