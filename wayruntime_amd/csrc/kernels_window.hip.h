// Sliding-window attention over grouped keys and values.  Optionally each head has a sink
// s: its weights are exp(score) / (exp(s) + sum of exp(score)), so a row may attend to
// nothing at all.
//
// A page (64 positions) holds each key/value head's block one after the other:
//
//   K  [64/16][dim_pad/32][64][8]     lane 16g + c of a tile: position 16s + c, elements 32k + 8g .. +8
//   V  [64/32][vdim_pad/16][64][8]    lane 16g + c of a tile: column 16t + c, element e of its eight:
//                                     position 32b + 16 (e / 4) + 4g + e % 4
//
// both the A operands of the products as they lie: scores S^T = K Q^T leave lane 16g + c with
// positions 4g .. 4g+3 of two 16-position halves for row c, which is the B operand of
// O^T = V^T P^T in the order V is stored.
//
//   window_append_kernel    queries rotated into an operand, keys rotated and values normed into the cache
//   window_prefill_kernel   128 (token, head) rows of one key/value head a workgroup, a page at a time
//                           through LDS
//   window_decode_kernel    a workgroup per (token, key/value head, share of the keys)
//   window_attend_any_kernel  any geometry, both activation types
#pragma once

#include "kernels_latent_mfma.hip.h"

namespace wr {

struct WindowArgs {
    const MixSeq* seqs;
    const uint32_t *row_seq, *row_pos, *pages;
    uint32_t rows, heads, kvh, group;            // group = heads / kvh
    uint32_t dim, dimp, vdim, vdimp, half, window, norm_values;
    float scale, out_scale, eps;
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

// element of (position in page, column) inside a head's V block
__device__ __forceinline__ uint32_t window_v_elem(uint32_t at, uint32_t d, uint32_t vdimp)
{
    return (((at / 32) * (vdimp / 16) + d / 16) * 64 + 16 * (at % 16 / 4) + d % 16) * 8 + (at % 32 / 16) * 4 + at % 4;
}

constexpr uint32_t kWindowQUnits = 512;          // query units of eight a workgroup rotates

// grid (rows / 4, kvh + slices of 4 rows' query units)
template <bool F32>
__global__ __launch_bounds__(256) void window_append_kernel(const WindowArgs a)
{
    using E = typename MixAct<F32>::E;
    using V4 = typename MixAct<F32>::V4;
    __shared__ float s_inv[4];
    const uint32_t t = threadIdx.x, r0 = blockIdx.x * 4, n = min(4u, a.rows - r0);
    if (blockIdx.y >= a.kvh) {
        const uint32_t per = a.heads * (a.dimp / 8), u0 = (blockIdx.y - a.kvh) * kWindowQUnits;
        for (uint32_t u = u0 + t; u < min(u0 + kWindowQUnits, 4 * per); u += 256) {
            const uint32_t i = u % 4, q = u / 4, h = q / (a.dimp / 8), r = r0 + i;
            if (i >= n) continue;
            float v[8];
            latent_rotate8(a.in + (size_t)r * a.ld + a.col_q + h * a.dim, a.table + (size_t)r * 2 * a.half, q % (a.dimp / 8) * 8,
                           a.dim, a.half, v);
            mix_store_unit<F32>(a.q, frag_unit(r, q, a.heads * (a.dimp / 32)), v);
        }
        return;
    }
    const uint32_t kvh = blockIdx.y, block = kMixPage * (a.dimp + a.vdimp);
    auto head_block = [&](uint32_t r) {
        const MixSeq s = a.seqs[a.row_seq[r]];
        return reinterpret_cast<E*>(a.cache) + ((size_t)a.pages[s.page0 + a.row_pos[r] / kMixPage] * a.kvh + kvh) * block;
    };
    for (uint32_t u = t; u < n * (a.dimp / 8); u += 256) {
        const uint32_t i = u % n, q = u / n, r = r0 + i;
        float v[8];
        latent_rotate8(a.in + (size_t)r * a.ld + a.col_k + kvh * a.dim, a.table + (size_t)r * 2 * a.half, q * 8, a.dim, a.half, v);
        mix_store_unit<F32>(head_block(r), frag_unit(a.row_pos[r] % kMixPage, q, a.dimp / 32), v);
    }
    const uint32_t wave = t >> 6, lane = t & 63;
    if (wave < n) {
        const float* v = a.in + (size_t)(r0 + wave) * a.ld + a.col_v + kvh * a.vdim;
        float ss = 0.f;
        for (uint32_t d = lane; d < a.vdim; d += 64) ss = fmaf(v[d], v[d], ss);
#pragma unroll
        for (int off = 32; off >= 1; off >>= 1) ss += wave_xor_f32(ss, off);
        if (lane == 0) s_inv[wave] = a.norm_values ? 1.0f / sqrtf(ss / (float)a.vdim + a.eps) : 1.0f;
    }
    __syncthreads();
    const uint32_t p0 = a.row_pos[r0];
    const bool run = n == 4 && p0 % 4 == 0 && a.row_seq[r0] == a.row_seq[r0 + 3];
    for (uint32_t d = t; d < a.vdimp; d += 256) {
        V4 x;
#pragma unroll
        for (uint32_t i = 0; i < 4; i++)
            x[i] = (E)(i < n && d < a.vdim ? a.in[(size_t)(r0 + min(i, n - 1)) * a.ld + a.col_v + kvh * a.vdim + d] * s_inv[i] : 0.f);
        if (run) {                                         // four positions of one column side by side
            *reinterpret_cast<V4*>(head_block(r0) + kMixPage * a.dimp + window_v_elem(p0 % kMixPage, d, a.vdimp)) = x;
        } else {
            for (uint32_t i = 0; i < n; i++)
                head_block(r0 + i)[kMixPage * a.dimp + window_v_elem(a.row_pos[r0 + i] % kMixPage, d, a.vdimp)] = x[i];
        }
    }
}

// One wave per (row, head), a lane per key of a page.  LDS: the query row and the output row as floats, 64 weights.
template <bool F32>
__global__ __launch_bounds__(64) void window_attend_any_kernel(const WindowArgs a)
{
    using E = typename MixAct<F32>::E;
    using V8 = typename MixAct<F32>::V8;
    extern __shared__ __attribute__((aligned(16))) float window_smem[];
    const uint32_t lane = threadIdx.x, r = blockIdx.x, h = blockIdx.y, kd = a.dimp / 32;
    float *q = window_smem, *o = q + a.dimp, *w = o + a.vdimp;
    const V8* qf = reinterpret_cast<const V8*>(a.q);
    for (uint32_t u = lane; u < a.dimp / 8; u += 64) {
        const V8 x = qf[frag_unit(r, h * kd * 4 + u, a.heads * kd)];
#pragma unroll
        for (int j = 0; j < 8; j++) q[u * 8 + j] = (float)x[j];
    }
    for (uint32_t k = lane; k < a.vdimp; k += 64) o[k] = 0.f;
    __syncthreads();
    const MixSeq s = a.seqs[a.row_seq[r]];
    const uint32_t pos = a.row_pos[r], lo = pos + 1 > a.window ? pos + 1 - a.window : 0;
    float mx = a.sink ? a.sink[h] : -INFINITY, sum = a.sink ? 1.0f : 0.f;
    for (uint32_t j0 = lo / kMixPage * kMixPage; j0 <= pos; j0 += kMixPage) {
        const uint32_t j = j0 + lane;
        const V8* page = reinterpret_cast<const V8*>(
            reinterpret_cast<const E*>(a.cache) +
            ((size_t)a.pages[s.page0 + j0 / kMixPage] * a.kvh + h / a.group) * kMixPage * (a.dimp + a.vdimp));
        float sc = 0.f;
        for (uint32_t u = 0; u < a.dimp / 8; u++) {
            const V8 x = page[frag_unit(lane, u, kd)];
#pragma unroll
            for (int e = 0; e < 8; e++) sc = fmaf((float)x[e], q[u * 8 + e], sc);
        }
        sc = (j >= lo && j <= pos) ? sc * a.scale : -INFINITY;
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
        const V8* vb = page + kMixPage * a.dimp / 8;
        for (uint32_t k = lane; k < a.vdimp; k += 64) {
            float acc = o[k] * corr;
            for (uint32_t u = 0; u < 8; u++) {             // 32-position block u / 4, lane group u % 4
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
    const float inv = a.out_scale / sum;
    E* out = reinterpret_cast<E*>(a.o);
    for (uint32_t k = lane; k < a.vdimp; k += 64) out[frag_elem(r, h * a.vdimp + k, a.o_kt)] = (E)(o[k] * inv);
}

// ---- matrix forms (bfloat16; head sizes padded to 32, 64 or 128) -------------

// The running softmax of one row tile over N x 16 keys from j0 on; s[n][i]: score of key j0 + 16n + 4g + i.
// Leaves the probabilities in s and returns by how much the old sums shrink.
template <int N, bool MASK>
__device__ __forceinline__ float window_softmax(f32x4 (&s)[N], uint32_t j0, int g, uint32_t lo, uint32_t pos, float scale,
                                                float& mx, float& sum)
{
    float bm = kLatentNone;
#pragma unroll
    for (int n = 0; n < N; n++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            s[n][i] *= scale;
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

// KQ, VT: head sizes in tiles of 32.  Grid: tiles of 128 (token, head of the group) rows times key/value heads, the
// key/value head innermost: with eight of them each XCD keeps to one.
template <int KQ, int VT>
__global__ __launch_bounds__(256, 2) void window_prefill_kernel(const WindowArgs a)
{
    constexpr int NR = 2, STAGE = 4 * (KQ + VT) * 1024, CPW = KQ + VT;
    extern __shared__ __attribute__((aligned(16))) unsigned char window_lds[];
    const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t kvh = blockIdx.x % a.kvh, H = a.group;
    uint32_t tile = blockIdx.x / a.kvh, pick_seq = 0, n_tiles = 0;
    for (uint32_t i = 0; i < a.n_list; i++) {
        n_tiles = (a.seqs[a.list[i]].rows * H + 127) / 128;
        pick_seq = a.list[i];
        if (tile < n_tiles) break;
        tile -= n_tiles;
    }
    tile = n_tiles - 1 - tile;                             // the last tiles see the most keys and go first
    const MixSeq s = a.seqs[pick_seq];
    const uint32_t m_end = s.rows * H, m0 = tile * 128;
    const uint32_t pos_first = s.pos0 + m0 / H, pos_last = s.pos0 + (min(m0 + 128, m_end) - 1) / H;
    const uint32_t j_begin = (pos_first + 1 > a.window ? pos_first + 1 - a.window : 0) / kMixPage * kMixPage, j_end = pos_last + 1;
    const float scale = a.scale * kLog2e;

    uint32_t m[NR], pos[NR], lo[NR];
    bf16x8 qv[NR][KQ];
    float mx[NR], sum[NR];
#pragma unroll
    for (int t = 0; t < NR; t++) {
        m[t] = m0 + (wave * NR + t) * 16 + c;
        const uint32_t mm = min(m[t], m_end - 1), head = kvh * H + mm % H;
        pos[t] = s.pos0 + mm / H;
        lo[t] = pos[t] + 1 > a.window ? pos[t] + 1 - a.window : 0;
#pragma unroll
        for (int k = 0; k < KQ; k++)
            qv[t][k] = reinterpret_cast<const bf16x8*>(a.q)[frag_unit(s.row0 + mm / H, (head * KQ + k) * 4 + g, a.heads * KQ)];
        mx[t] = a.sink ? a.sink[head] * kLog2e : kLatentNone;
        sum[t] = a.sink ? 1.0f : 0.f;
    }
    // positions this wave's rows span: a page between them needs no mask
    const uint32_t w0 = min(m0 + wave * NR * 16, m_end - 1), w1 = min(m0 + wave * NR * 16 + NR * 16 - 1, m_end - 1);
    const uint32_t w_pos0 = s.pos0 + w0 / H, w_pos1 = s.pos0 + w1 / H, w_lo1 = w_pos1 + 1 > a.window ? w_pos1 + 1 - a.window : 0;
    const uint32_t w_lo0 = w_pos0 + 1 > a.window ? w_pos0 + 1 - a.window : 0;
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
        const bf16x8* vt = kt + 4 * KQ * 64;
        f32x4 sc[NR][4];
#pragma unroll
        for (int t = 0; t < NR; t++)
#pragma unroll
            for (int n = 0; n < 4; n++) sc[t][n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KQ; k++)
#pragma unroll
            for (int n = 0; n < 4; n++) {
                const bf16x8 kv = kt[(n * KQ + k) * 64];
#pragma unroll
                for (int t = 0; t < NR; t++) sc[t][n] = mix_mfma(kv, qv[t][k], sc[t][n]);
            }
        const bool inside = j0 + kMixPage - 1 <= w_pos0 && j0 >= w_lo1;
        bf16x8 p[NR][2];
#pragma unroll
        for (int t = 0; t < NR; t++) {
            const float corr = inside ? window_softmax<4, false>(sc[t], j0, g, lo[t], pos[t], scale, mx[t], sum[t])
                                      : window_softmax<4, true>(sc[t], j0, g, lo[t], pos[t], scale, mx[t], sum[t]);
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
#pragma unroll
    for (int t = 0; t < NR; t++) {
        if (m[t] >= m_end) continue;
        const uint32_t r = s.row0 + m[t] / H, h = kvh * H + m[t] % H;
        const float inv = a.out_scale / sum[t];
#pragma unroll
        for (int k = 0; k < 2 * VT; k++) {
            bf16x4 o;
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] = (__bf16)(acc[t][k][i] * inv);
            *reinterpret_cast<bf16x4*>(out + frag_elem(r, h * VT * 32 + k * 16 + 4 * g, a.o_kt)) = o;
        }
    }
}

// grid (rows of the launch * kvh * tiles of 16 heads of a group, splits).  The four waves take every fourth block of 32
// keys of the share, straight into registers, one block ahead.
template <int KQ, int VT>
__global__ __launch_bounds__(256, 2) void window_decode_kernel(const WindowArgs a)
{
    __shared__ f32x4 box[3 * (2 * VT + 1) * 64];
    const int lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t tiles = (a.group + 15) / 16, split = blockIdx.y;
    const uint32_t kvh = blockIdx.x % a.kvh, tile = blockIdx.x / a.kvh % tiles, ri = blockIdx.x / a.kvh / tiles;
    const LatentRow lr = a.drows[ri];
    const uint32_t r = lr.row, pos = lr.pos, lo = pos + 1 > a.window ? pos + 1 - a.window : 0;
    const uint32_t first = lo / 32 * 32 + split * a.split_keys, end = min(pos + 1, first + a.split_keys);
    const float scale = a.scale * kLog2e;
    const uint32_t member = tile * 16 + c, head = kvh * a.group + min(member, a.group - 1);

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
    for (int k = 0; k < KQ; k++) qv[k] = reinterpret_cast<const bf16x8*>(a.q)[frag_unit(r, (head * KQ + k) * 4 + g, a.heads * KQ)];
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
        const float corr = window_softmax<2, true>(sc, j0, g, lo, end - 1, scale, mx, sum);
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
    if (member >= a.group) return;
    if (a.splits == 1) {
        const float inv = a.out_scale / sum;
        __bf16* out = reinterpret_cast<__bf16*>(a.o);
#pragma unroll
        for (int k = 0; k < 2 * VT; k++) {
            bf16x4 o;
#pragma unroll
            for (int i = 0; i < 4; i++) o[i] = (__bf16)(acc[k][i] * inv);
            *reinterpret_cast<bf16x4*>(out + frag_elem(r, head * VT * 32 + k * 16 + 4 * g, a.o_kt)) = o;
        }
        return;
    }
    const size_t at = ((size_t)ri * a.heads + head) * a.splits + split;
    if (g == 0) {
        a.part_ml[at * 2] = mx;
        a.part_ml[at * 2 + 1] = sum;
    }
#pragma unroll
    for (int k = 0; k < 2 * VT; k++) *reinterpret_cast<f32x4*>(a.part_o + at * VT * 32 + k * 16 + 4 * g) = acc[k];
}

constexpr uint32_t kWindowSplits = 64;          // shares of the keys at most: a lane each

// grid (rows of the launch, heads), one wave: the shares of one row and head together
template <int VT>
__global__ __launch_bounds__(64) void window_combine_kernel(const WindowArgs a)
{
    __shared__ float wt[kWindowSplits];
    const uint32_t h = blockIdx.y, r = a.drows[blockIdx.x].row, t = threadIdx.x;
    const size_t at = ((size_t)blockIdx.x * a.heads + h) * a.splits;
    const bool has = t < a.splits;
    const float m = has ? a.part_ml[(at + t) * 2] : kLatentNone, l = has ? a.part_ml[(at + t) * 2 + 1] : 0.f;
    float mx = m;
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) mx = fmaxf(mx, wave_xor_f32(mx, off));
    const float w = l != 0.f ? fast_exp2(m - mx) : 0.f;    // zero: a share past the row's keys
    float sum = w * l;
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) sum += wave_xor_f32(sum, off);
    const float inv = a.out_scale / sum;
    wt[t] = w;
    __syncthreads();
    __bf16* out = reinterpret_cast<__bf16*>(a.o);
    for (uint32_t col = t; col < VT * 32; col += 64) {
        float o = 0.f;
        for (uint32_t s = 0; s < a.splits; s++) o = fmaf(wt[s], a.part_o[(at + s) * VT * 32 + col], o);
        out[frag_elem(r, h * VT * 32 + col, a.o_kt)] = (__bf16)(o * inv);
    }
}

}  // namespace wr
