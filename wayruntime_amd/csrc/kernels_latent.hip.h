// Attention through a low-rank latent with a shared rotated key part, inside a
// sliding window.  The per-head key and value matrices are absorbed: a query is
// brought into the latent's space before, the weighted latents are taken out of
// it after (both matrix products elsewhere), so here all heads of a token share
// one cached row [latent | rotated part] per position, and the values are that
// row's first part.
//
// Cache pages (64 positions) hold the rows in operand order, [64/16][KD][64][8]
// with KD = row elements / 32: lane 16g + c of a tile holds position 16 s + c,
// elements 32 kt + 8g .. +8.
#pragma once

#include "mix_common.hip.h"
#include "kernels_mix_rows.hip.h"

namespace wr {

struct LatentArgs {
    const MixSeq* seqs;
    const uint32_t* row_seq;        // request of each row
    const uint32_t* row_pos;
    const uint32_t* pages;
    uint32_t rows, heads, rank, rank_pad, rot, rot_pad, half;
    uint32_t window;
    float scale;
    void* cache;                    // this layer run's pages
    const void* q;
    void* o;
    // append
    const float* d;
    uint32_t ldd, q_rank;
    const float *q_norm, *kv_norm, *table;
    float eps;
    void* cq;
    // rotated query part
    const float* qr;
    uint32_t ldq;
    void* q_out;
};

// (cos, sin) of position * freq, times gain; angles reduced in double
__global__ __launch_bounds__(256) void mix_rope_table_kernel(const uint32_t* row_pos, uint32_t rows, const double* freq,
                                                             uint32_t half, float gain, float* table)
{
    const uint32_t i = blockIdx.x * 256 + threadIdx.x;
    if (i >= rows * half) return;
    const double ang = (double)row_pos[i / half] * freq[i % half];
    const double turns = ang * 0.15915494309189533577;
    const float x = (float)((turns - rint(turns)) * 6.283185307179586477);
    float s, c;
    sincosf(x, &s, &c);
    table[2 * (size_t)i] = c * gain;
    table[2 * (size_t)i + 1] = s * gain;
}

// Eight rotated elements i0 .. i0 + 7 of x (zero past rot).
__device__ __forceinline__ void latent_rotate8(const float* x, const float* tab, uint32_t i0, uint32_t rot, uint32_t half,
                                               float (&v)[8])
{
    if (half % 8 == 0 && i0 + 8 <= 2 * half) {             // whole units: all eight in the same half
        const bool upper = i0 >= half;
        const uint32_t p0 = upper ? i0 - half : i0;
        float own[8], other[8], cs[16];
#pragma unroll
        for (int j = 0; j < 8; j++) {
            own[j] = x[i0 + j];
            other[j] = x[upper ? p0 + j : i0 + half + j];
            cs[2 * j] = tab[2 * (p0 + j)];
            cs[2 * j + 1] = tab[2 * (p0 + j) + 1];
        }
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = upper ? own[j] * cs[2 * j] + other[j] * cs[2 * j + 1]
                                                 : own[j] * cs[2 * j] - other[j] * cs[2 * j + 1];
        return;
    }
#pragma unroll
    for (int j = 0; j < 8; j++) {
        const uint32_t i = i0 + j;
        float y = 0.f;
        if (i < rot) {
            if (i < half)
                y = x[i] * tab[2 * i] - x[i + half] * tab[2 * i + 1];
            else if (i < 2 * half)
                y = x[i] * tab[2 * (i - half)] + x[i - half] * tab[2 * (i - half) + 1];
            else
                y = x[i];
        }
        v[j] = y;
    }
}

// One workgroup a row: the q latent normed to cq (frag), the kv latent normed and
// the key part rotated into the cache.  The pads of d and of the norms are zeros.
template <bool F32>
__global__ __launch_bounds__(256) void latent_append_kernel(const LatentArgs a)
{
    using E = typename MixAct<F32>::E;
    __shared__ float red[64];
    const uint32_t t = threadIdx.x, r = blockIdx.x;
    const float* d = a.d + (size_t)r * a.ldd;
    const uint32_t qp = (a.q_rank + 31) / 32 * 32, kp = (a.rank + 31) / 32 * 32;
    const float *dc = d + qp, *dr = dc + kp;
    float sq = 0.f, sk = 0.f;
    for (uint32_t q = t; q < (qp + kp) / 8; q += 256) {
        float v[8];
        mix_load8(d + q * 8, v);
        float s = 0.f;
#pragma unroll
        for (int j = 0; j < 8; j++) s = fmaf(v[j], v[j], s);
        if (q < qp / 8) sq += s;
        else sk += s;
    }
    const MixSeq s = a.seqs[a.row_seq[r]];
    const uint32_t pos = a.row_pos[r], kd = (a.rank_pad + a.rot_pad) / 32;
    const uint32_t page = a.pages[s.page0 + pos / kMixPage], at = pos % kMixPage;
    const float qi = 1.0f / sqrtf(mix_row_sum<1>(sq, red) / (float)a.q_rank + a.eps);
    const float ki = 1.0f / sqrtf(mix_row_sum<1>(sk, red) / (float)a.rank + a.eps);
    for (uint32_t q = t; q < qp / 8; q += 256) {
        float v[8], w[8];
        mix_load8(d + q * 8, v);
        mix_load8(a.q_norm + q * 8, w);
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = v[j] * qi * w[j];
        mix_store_unit<F32>(a.cq, frag_unit(r, q, qp / 32), v);
    }
    E* base = reinterpret_cast<E*>(a.cache) + (size_t)page * kMixPage * (a.rank_pad + a.rot_pad);
    const float* tab = a.table + (size_t)r * 2 * a.half;
    for (uint32_t q = t; q < (a.rank_pad + a.rot_pad) / 8; q += 256) {
        float v[8], w[8];
        if (q < kp / 8) {
            mix_load8(dc + q * 8, v);
            mix_load8(a.kv_norm + q * 8, w);
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] = v[j] * ki * w[j];
        } else if (q >= a.rank_pad / 8) {
            latent_rotate8(dr, tab, q * 8 - a.rank_pad, a.rot, a.half, v);
        } else {
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] = 0.f;
        }
        mix_store_unit<F32>(base, frag_unit(at, q, kd), v);
    }
}

// Rotated query part of every (row, head) into columns rank_pad .. of the head.
template <bool F32>
__global__ __launch_bounds__(256) void latent_qrope_kernel(const LatentArgs a)
{
    const uint32_t per = a.rot_pad / 8;
    const uint32_t i0 = blockIdx.x * 256 + threadIdx.x;
    if (i0 >= a.rows * a.heads * per) return;
    const uint32_t q = i0 % per, m = i0 / per, r = m / a.heads, h = m % a.heads;
    const float* x = a.qr + (size_t)r * a.ldq + h * a.rot;
    const float* tab = a.table + (size_t)r * 2 * a.half;
    float v[8];
    latent_rotate8(x, tab, q * 8, a.rot, a.half, v);
    const uint32_t kd = (a.rank_pad + a.rot_pad) / 32;
    mix_store_unit<F32>(a.q_out, frag_unit(r, h * kd * 4 + (a.rank_pad >> 3) + q, a.heads * kd), v);
}

// Any geometry, both activation types: one wave per (row, head), a lane per key of
// a run of 64.  LDS: the query row and the output row as floats, 64 weights.
template <bool F32>
__global__ __launch_bounds__(64) void latent_attend_any_kernel(const LatentArgs a)
{
    using E = typename MixAct<F32>::E;
    using V8 = typename MixAct<F32>::V8;
    extern __shared__ __attribute__((aligned(16))) float latent_smem[];
    const uint32_t lane = threadIdx.x, r = blockIdx.x, h = blockIdx.y;
    const uint32_t dk = a.rank_pad + a.rot_pad, kd = dk / 32;
    float *q = latent_smem, *o = q + dk, *w = o + a.rank_pad;
    const V8* qf = reinterpret_cast<const V8*>(a.q);
    for (uint32_t u = lane; u < dk / 8; u += 64) {
        const V8 x = qf[frag_unit(r, h * kd * 4 + u, a.heads * kd)];
#pragma unroll
        for (int j = 0; j < 8; j++) q[u * 8 + j] = (float)x[j];
    }
    for (uint32_t k = lane; k < a.rank_pad; k += 64) o[k] = 0.f;
    __syncthreads();
    const MixSeq s = a.seqs[a.row_seq[r]];
    const uint32_t pos = a.row_pos[r], lo = pos + 1 > a.window ? pos + 1 - a.window : 0;
    float mx = -INFINITY, sum = 0.f;
    for (uint32_t j0 = lo / 64 * 64; j0 <= pos; j0 += 64) {
        const uint32_t j = j0 + lane;
        const V8* page = reinterpret_cast<const V8*>(reinterpret_cast<const E*>(a.cache) +
                                                     (size_t)a.pages[s.page0 + j0 / kMixPage] * kMixPage * dk);
        float sc = 0.f;
        for (uint32_t u = 0; u < dk / 8; u++) {
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
        for (uint32_t k = lane; k < a.rank_pad; k += 64) {
            float acc = o[k] * corr;
            const E* col = reinterpret_cast<const E*>(page + frag_unit(0, k >> 3, kd)) + (k & 7);
            for (uint32_t jj = 0; jj < 64; jj++) {
                // positions past the row's own may hold anything: their weight is zero, their value is not read
                const float x = w[jj] != 0.f ? (float)col[((size_t)(jj >> 4) * kd * 64 + (jj & 15)) * 8] : 0.f;
                acc = fmaf(w[jj], x, acc);
            }
            o[k] = acc;
        }
        __syncthreads();
    }
    const float inv = 1.0f / sum;
    E* out = reinterpret_cast<E*>(a.o);
    for (uint32_t k = lane; k < a.rank_pad; k += 64)
        out[frag_elem(r, h * a.rank_pad + k, a.heads * a.rank_pad / 32)] = (E)(o[k] * inv);
}

}  // namespace wr
