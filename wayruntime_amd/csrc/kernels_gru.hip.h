// Element-wise gated recurrence, gates and candidates made from the input and not from the state (minGRU):
//
//   S_t = (1 - z_t) S_(t-1) + z_t c_t      z = logistic(zl), c = u + 1/2 for u >= 0, else logistic(u)
//   out = S_t * SiLU(g_t)
//
// zl, u and g are 32-bit rows of the layer's input product.  A token is the map S -> A S + B, so
// tokens can be put together in any grouping: a workgroup has sixteen channels of a request, a
// wave sixteen rows of them (lane 16g + c: row c, channels 4g .. +3), scans its rows across lanes,
// and the waves' totals are put together in LDS while the next rows are on their way.  Decoded
// tokens and short portions take one wave.
#pragma once

#include "mix_common.hip.h"
#include "kernels_mix_rows.hip.h"

namespace wr {

struct GruArgs {
    const MixSeq* seqs;
    const uint32_t* list;           // requests of this launch
    uint32_t wpad;                  // channels, padded to 32
    const float* in;
    uint32_t ld, col_z, col_x, col_g;
    float* state;                   // [buffer][wpad]
    void* h;
    uint32_t h_kt, col_h;
};

// The value `by` rows up in the sixteen lanes of a row group, `none` above the first.
template <int BY>
__device__ __forceinline__ float gru_up(float v, float none)
{
    return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(none), __float_as_int(v), 0x110 + BY, 0xF, 0xF, false));
}

template <int BY>
__device__ __forceinline__ void gru_join(f32x4& A, f32x4& B)
{
#pragma unroll
    for (int j = 0; j < 4; j++) {
        const float a = gru_up<BY>(A[j], 1.0f), b = gru_up<BY>(B[j], 0.f);
        B[j] = fmaf(A[j], b, B[j]);
        A[j] *= a;
    }
}

// logistic(z) and what it leaves of one
template <bool F32>
__device__ __forceinline__ void gru_logistic(float z, float& s, float& t)
{
    float e, over;
    if constexpr (F32) {
        e = expf(-fabsf(z));
        over = 1.0f / (1.0f + e);
    } else {
        e = __builtin_amdgcn_exp2f(-fabsf(z) * 1.44269504088896340736f);
        over = __builtin_amdgcn_rcpf(1.0f + e);
    }
    s = z < 0.f ? e * over : over;
    t = z < 0.f ? over : e * over;
}

// What this wave did in LDS is done, and everybody's: loads from memory stay on their way.
__device__ __forceinline__ void gru_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// grid (channels / 16, requests), NW waves
template <bool F32, int NW>
__global__ __launch_bounds__(64 * NW) void gru_scan_kernel(const GruArgs a)
{
    __shared__ __attribute__((aligned(16))) float tot[NW][2][16], start[NW][16];
    const MixSeq s = a.seqs[a.list[blockIdx.y]];
    const uint32_t lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4, wave = threadIdx.x >> 6;
    // the two halves of a row's 128 bytes go to workgroups of one XCD
    const uint32_t b = blockIdx.x, slab = gridDim.x % 16 == 0 ? (b / 16 * 8 + b % 8) * 2 + b / 8 % 2 : b;
    const uint32_t ch = slab * 16 + 4 * g;
    float carry = 0.f;                                     // wave 0, lanes below 16: the state of a channel each
    if (threadIdx.x < 16 && s.pos0 > 0) carry = a.state[(size_t)s.state_in * a.wpad + slab * 16 + lane];
    struct Rows {
        f32x4 z, u, q;
    };
    auto load = [&](Rows& x, uint32_t row) {               // (rows past the request's repeat its last one)
        const float* p = a.in + (size_t)(s.row0 + min(row, s.rows - 1)) * a.ld + ch;
        x.z = *reinterpret_cast<const f32x4*>(p + a.col_z);
        x.u = *reinterpret_cast<const f32x4*>(p + a.col_x);
        x.q = *reinterpret_cast<const f32x4*>(p + a.col_g);
    };
    // sixteen rows a wave from row0 on; x is theirs, and then those of the turn after the next
    auto turn = [&](Rows& x, uint32_t row0) {
        const uint32_t row = row0 + wave * 16 + c;
        f32x4 A, B, o;
#pragma unroll
        for (int j = 0; j < 4; j++) {
            float zs, zt, us, ut, qs, qt;
            gru_logistic<F32>(x.z[j], zs, zt);
            gru_logistic<F32>(x.u[j], us, ut);
            gru_logistic<F32>(x.q[j], qs, qt);
            A[j] = row < s.rows ? zt : 1.0f;
            B[j] = row < s.rows ? zs * (x.u[j] >= 0.f ? x.u[j] + 0.5f : us) : 0.f;
            o[j] = x.q[j] * qs;
        }
        load(x, row + 32 * NW);
        gru_join<1>(A, B);
        gru_join<2>(A, B);
        gru_join<4>(A, B);
        gru_join<8>(A, B);
        if (c == 15) {
            *reinterpret_cast<f32x4*>(&tot[wave][0][4 * g]) = A;
            *reinterpret_cast<f32x4*>(&tot[wave][1][4 * g]) = B;
        }
        gru_barrier();
        if (threadIdx.x < 16) {
#pragma unroll
            for (int w = 0; w < NW; w++) {
                start[w][lane] = carry;
                carry = fmaf(tot[w][0][lane], carry, tot[w][1][lane]);
            }
        }
        gru_barrier();                                     // (tot is written again behind it, start behind the next one)
        const f32x4 S = *reinterpret_cast<const f32x4*>(&start[wave][4 * g]);
        if (row < s.rows) {
            typename MixAct<F32>::V4 out;
#pragma unroll
            for (int j = 0; j < 4; j++) out[j] = (typename MixAct<F32>::E)(o[j] * fmaf(A[j], S[j], B[j]));
            *reinterpret_cast<typename MixAct<F32>::V4*>(reinterpret_cast<typename MixAct<F32>::E*>(a.h) +
                                                         frag_elem(s.row0 + row, a.col_h + ch, a.h_kt)) = out;
        }
    };
    Rows even, odd;
    load(even, wave * 16 + c);
    load(odd, 16 * NW + wave * 16 + c);
    for (uint32_t row0 = 0; row0 < s.rows; row0 += 32 * NW) {      // uniform
        turn(even, row0);
        if (row0 + 16 * NW < s.rows) turn(odd, row0 + 16 * NW);
    }
    if (threadIdx.x < 16) a.state[(size_t)s.state_out * a.wpad + slab * 16 + lane] = carry;
}

}  // namespace wr
