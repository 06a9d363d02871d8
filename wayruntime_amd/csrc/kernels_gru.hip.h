// Gated recurrence element by element whose gates read the current token alone (minGRU):
//
//   S_t = (1 - z_t) S_(t-1) + z_t c_t      z = logistic(zl), c = u + 1/2 for u >= 0, else logistic(u)
//   out = S_t * SiLU(g_t)
//
// zl, u and g are 32-bit rows of the layer's input product.  A token is the map S -> A S + B, so
// tokens can be put together in any grouping: a workgroup has 32 channels of a request, a wave
// sixteen rows of them (lane 16g + c: row c, channels 8g .. +7, which is the next product's
// operand), scans its rows across lanes, and the waves' totals are put together in LDS.  Decoded
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
__device__ __forceinline__ void gru_join(float (&A)[8], float (&B)[8])
{
#pragma unroll
    for (int j = 0; j < 8; j++) {
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

// grid (channels / 32, requests), NW waves
template <bool F32, int NW>
__global__ __launch_bounds__(64 * NW) void gru_scan_kernel(const GruArgs a)
{
    __shared__ float tot[NW][2][32], start[NW][32];
    const MixSeq s = a.seqs[a.list[blockIdx.y]];
    const uint32_t lane = threadIdx.x & 63, c = lane & 15, g = lane >> 4, wave = threadIdx.x >> 6;
    const uint32_t ch = blockIdx.x * 32 + 8 * g;
    float carry = 0.f;                                     // wave 0, lanes below 32: the state of a channel each
    if (threadIdx.x < 32 && s.pos0 > 0) carry = a.state[(size_t)s.state_in * a.wpad + blockIdx.x * 32 + lane];
    float z[8], u[8], q[8];
    auto load = [&](uint32_t row) {                        // (rows past the request's repeat its last one)
        const float* p = a.in + (size_t)(s.row0 + min(row, s.rows - 1)) * a.ld + ch;
        mix_load8(p + a.col_z, z);
        mix_load8(p + a.col_x, u);
        mix_load8(p + a.col_g, q);
    };
    load(wave * 16 + c);
    for (uint32_t row0 = 0; row0 < s.rows; row0 += 16 * NW) {
        const uint32_t row = row0 + wave * 16 + c;
        float A[8], B[8], o[8];
#pragma unroll
        for (int j = 0; j < 8; j++) {
            float zs, zt, us, ut, qs, qt;
            gru_logistic<F32>(z[j], zs, zt);
            gru_logistic<F32>(u[j], us, ut);
            gru_logistic<F32>(q[j], qs, qt);
            A[j] = row < s.rows ? zt : 1.0f;
            B[j] = row < s.rows ? zs * (u[j] >= 0.f ? u[j] + 0.5f : us) : 0.f;
            o[j] = q[j] * qs;
        }
        if (row0 + 16 * NW < s.rows) load(row + 16 * NW);  // uniform
        gru_join<1>(A, B);
        gru_join<2>(A, B);
        gru_join<4>(A, B);
        gru_join<8>(A, B);
        if (c == 15) {
            mix_store8(&tot[wave][0][8 * g], A);
            mix_store8(&tot[wave][1][8 * g], B);
        }
        __syncthreads();
        if (threadIdx.x < 32) {
#pragma unroll
            for (int w = 0; w < NW; w++) {
                start[w][lane] = carry;
                carry = fmaf(tot[w][0][lane], carry, tot[w][1][lane]);
            }
        }
        __syncthreads();                                   // (tot is written again behind it, start behind the next one)
        float S[8];
        mix_load8(&start[wave][8 * g], S);
#pragma unroll
        for (int j = 0; j < 8; j++) o[j] *= fmaf(A[j], S[j], B[j]);
        if (row < s.rows) mix_store_unit<F32>(a.h, frag_unit(s.row0 + row, (a.col_h + ch) / 8, a.h_kt), o);
    }
    if (threadIdx.x < 32) a.state[(size_t)s.state_out * a.wpad + blockIdx.x * 32 + lane] = carry;
}

}  // namespace wr
