// Matrix products of mixer-stack models: bfloat16 weights in operand order,
// activation rows in fragment order (mix_common.hip.h), and the output put where
// the next step wants it: 32-bit or activation-type rows, or directly the
// fragment of the next product.
//
//   mix_gemm_stream_kernel  any row count, both activation types: a workgroup's
//                           four waves share one run of NT x 16 outputs and GR x 16
//                           rows and split the input range; weights stream from HBM
//                           once (decode: HBM-bound on the weight bytes)
//   mix_gemm_lds_kernel     prompt-sized row counts, bfloat16: 128-output tiles
//                           staged through LDS (MFMA-bound)
#pragma once

#include "mix_common.hip.h"

namespace wr {

constexpr uint32_t kMixOutRowsF32 = 0, kMixOutRows = 1, kMixOutFrag = 2, kMixOutSplit = 3, kMixOutGated = 4,
                   kMixOutSplitGated = 5;

struct MixGemmArgs {
    const bf16x8* w;
    const void* x;
    uint32_t ntiles, ktiles;         // of one matrix
    uint32_t x_kt, x_kt_z;
    uint32_t rows, groups;
    const int32_t* group_expert;
    uint32_t out, ldy, h_kt, col_z, n_split, silu_end, sigmoid_end, tanh_end, relu2, gelu;
    float scale, limit, slope, up_bias;
    const float* bias;
    const uint32_t* x_perm;
    const float* x_scale;            // a factor per row of the input (applied to its products), or nullptr
    float* y;
    void* ya;
    void* h;
};

__global__ __launch_bounds__(256) void mix_pack_kernel(const uint16_t* __restrict__ w, u32x4* __restrict__ tiles,
                                                       uint64_t units, uint32_t K)
{
    const uint64_t unit = (uint64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (unit >= units) return;
    const uint32_t lane = (uint32_t)(unit & 63);
    const uint64_t tile = unit >> 6;
    const uint32_t kt = (uint32_t)(tile % (K / 32));
    const uint64_t nt = tile / (K / 32);
    tiles[unit] = *reinterpret_cast<const u32x4*>(w + ((nt * 16 + (lane & 15)) * K + kt * 32 + (lane >> 4) * 8));
}

template <bool F32>
__device__ __forceinline__ void mix_put4(void* p, size_t elem, f32x4 v)
{
    typename MixAct<F32>::V4 o;
#pragma unroll
    for (int i = 0; i < 4; i++) o[i] = (typename MixAct<F32>::E)v[i];
    *reinterpret_cast<typename MixAct<F32>::V4*>(reinterpret_cast<typename MixAct<F32>::E*>(p) + elem) = o;
}

// The gated unit of one gate and one up output.
template <bool F32>
__device__ __forceinline__ float mix_gated(const MixGemmArgs& a, float gate, float up)
{
    if (a.limit > 0.f) {                                   // (uniform, like gelu)
        gate = fminf(gate, a.limit);
        up = fminf(fmaxf(up, -a.limit), a.limit) + a.up_bias;
        return gate * mix_sigmoid<F32>(a.slope * gate) * up;
    }
    // the tanh form of GELU is x * logistic(2 y), y the argument of its tanh
    const float y = a.gelu ? 1.5957691216057308f * (gate + 0.044715f * gate * gate * gate) : gate;
    return gate * mix_sigmoid<F32>(y) * up;
}

// Bias and activation of outputs n .. n + 3.
template <bool F32>
__device__ __forceinline__ f32x4 mix_activate(const MixGemmArgs& a, f32x4 v, uint32_t n)
{
    if (a.bias) {
        const f32x4 b = *reinterpret_cast<const f32x4*>(a.bias + n);
#pragma unroll
        for (int i = 0; i < 4; i++) v[i] += b[i];
    }
    if (n < a.sigmoid_end) {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float s = mix_sigmoid<F32>(v[i]);
            v[i] = n + i < a.silu_end ? v[i] * s : (n + i < a.sigmoid_end ? s : v[i]);
        }
    } else if (n < a.tanh_end) {
#pragma unroll
        for (int i = 0; i < 4; i++) v[i] = n + i < a.tanh_end ? tanhf(v[i]) : v[i];
    } else if (a.relu2) {
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const float p = fmaxf(v[i], 0.f);
            v[i] = p * p;
        }
    }
    return v;
}

// Accumulator tile nt of row group `group`: lane 16g + c holds outputs
// 16 nt + 4g .. +3 of row 16 group + c.  `up`: the tile's partner (GATED, SPLIT_GATED).
template <bool F32>
__device__ __forceinline__ void mix_store_tile(const MixGemmArgs& a, f32x4 v, f32x4 up, uint32_t nt, uint32_t group,
                                               uint32_t z, int lane)
{
    const uint32_t c = lane & 15, g = lane >> 4, row = group * 16 + c, n = nt * 16 + 4 * g;
    if (row >= a.rows || nt >= a.ntiles) return;
    if (a.x_scale) {
        const float s = a.x_scale[row];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            v[i] *= s;
            up[i] *= s;
        }
    }
    if (a.out >= kMixOutGated) {
        if (a.out == kMixOutSplitGated && nt * 16 < a.n_split) {
            *reinterpret_cast<f32x4*>(a.y + (size_t)row * a.ldy + n) = mix_activate<F32>(a, v, n);
            *reinterpret_cast<f32x4*>(a.y + (size_t)row * a.ldy + n + 16) = mix_activate<F32>(a, up, n + 16);
            return;
        }
#pragma unroll
        for (int i = 0; i < 4; i++) v[i] = mix_gated<F32>(a, v[i], up[i]);
        const uint32_t to = nt - (a.out == kMixOutSplitGated ? a.n_split / 16 : 0u);
        mix_put4<F32>(a.h, frag_elem(row, to / 2 * 16 + 4 * g, a.h_kt), v);
        return;
    }
    v = mix_activate<F32>(a, v, n);
    if (a.scale != 0.f) {
#pragma unroll
        for (int i = 0; i < 4; i++) v[i] *= a.scale;
    }
    if (a.out == kMixOutRowsF32) {
        *reinterpret_cast<f32x4*>(a.y + (size_t)row * a.ldy + (size_t)z * a.col_z + n) = v;
    } else if (a.out == kMixOutRows) {
        mix_put4<F32>(a.ya, (size_t)row * a.ldy + n, v);
    } else if (a.out == kMixOutSplit && n >= a.n_split) {
        *reinterpret_cast<f32x4*>(a.y + (size_t)row * a.ldy + n - a.n_split) = v;
    } else {
        mix_put4<F32>(a.h, frag_elem(row, z * a.col_z + n, a.h_kt), v);
    }
}

template <bool F32, int NT, int GR>
__global__ __launch_bounds__(256) void mix_gemm_stream_kernel(const MixGemmArgs a)
{
    using V8 = typename MixAct<F32>::V8;
    // k-steps in flight per buffer: about eight KiB of operands
    constexpr int KB = (F32 ? 4 : 8) / (NT > GR ? NT : GR) > 0 ? (F32 ? 4 : 8) / (NT > GR ? NT : GR) : 1;
    __shared__ f32x4 s_part[3 * NT * GR * 64];
    const int lane = threadIdx.x & 63;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t nt0 = blockIdx.x * NT, group0 = blockIdx.y * GR, z = blockIdx.z;
    uint32_t mat = z;
    if (a.group_expert) {                                  // GR == 1
        const int e = a.group_expert[group0];
        if (e < 0) return;                                 // uniform over the workgroup
        mat = (uint32_t)e;
    }
    const uint32_t k_begin = a.ktiles * wave / 4, k_end = a.ktiles * (wave + 1) / 4, klast = a.ktiles - 1;

    const bf16x8* wp[NT];
    const V8* xp[GR];
#pragma unroll
    for (int t = 0; t < NT; t++)
        wp[t] = a.w + ((size_t)mat * a.ntiles + min(nt0 + t, a.ntiles - 1)) * a.ktiles * 64 + lane;
#pragma unroll
    for (int i = 0; i < GR; i++)
        xp[i] = reinterpret_cast<const V8*>(a.x) + ((size_t)min(group0 + i, a.groups - 1) * a.x_kt + (size_t)z * a.x_kt_z) * 64 + lane;
    if constexpr (GR == 1) {
        if (a.x_perm) {                                    // rows picked one by one: the operand's lanes fetch their own
            const uint32_t pick = a.x_perm[group0 * 16 + (lane & 15)], row = pick == 0xFFFFFFFFu ? 0 : pick;
            xp[0] = reinterpret_cast<const V8*>(a.x) + (size_t)(row >> 4) * a.x_kt * 64 + (lane & 48) + (row & 15);
        }
    }

    f32x4 acc[NT][GR];
#pragma unroll
    for (int t = 0; t < NT; t++)
#pragma unroll
        for (int i = 0; i < GR; i++) acc[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};

    // loads are unconditional (a k-step past the end re-reads the last one and is
    // not multiplied), so the batch asked for ahead stays in flight
    bf16x8 wa[KB][NT], wb[KB][NT];
    V8 xa[KB][GR], xb[KB][GR];
    auto load = [&](bf16x8 (&w)[KB][NT], V8 (&x)[KB][GR], uint32_t k0) {
#pragma unroll
        for (int u = 0; u < KB; u++) {
            const size_t k = (size_t)min(k0 + u, klast) * 64;
#pragma unroll
            for (int t = 0; t < NT; t++) w[u][t] = __builtin_nontemporal_load(&wp[t][k]);
#pragma unroll
            for (int i = 0; i < GR; i++) x[u][i] = xp[i][k];
        }
    };
    auto multiply = [&](const bf16x8 (&w)[KB][NT], const V8 (&x)[KB][GR], uint32_t k0) {
#pragma unroll
        for (int u = 0; u < KB; u++) {
            if (k0 + u < k_end) {                          // uniform
#pragma unroll
                for (int i = 0; i < GR; i++)
#pragma unroll
                    for (int t = 0; t < NT; t++) acc[t][i] = mix_mfma(w[u][t], x[u][i], acc[t][i]);
            }
        }
    };
    if (k_begin < k_end) {
        load(wa, xa, k_begin);
        for (uint32_t kt = k_begin; kt < k_end; kt += 2 * KB) {
            load(wb, xb, kt + KB);
            multiply(wa, xa, kt);
            load(wa, xa, kt + 2 * KB);
            multiply(wb, xb, kt + KB);
        }
    }
    if (wave > 0) {
#pragma unroll
        for (int t = 0; t < NT; t++)
#pragma unroll
            for (int i = 0; i < GR; i++) s_part[(((wave - 1) * NT + t) * GR + i) * 64 + lane] = acc[t][i];
    }
    __syncthreads();
    if (wave > 0) return;
#pragma unroll 1
    for (int p = 0; p < 3; p++) {
#pragma unroll
        for (int t = 0; t < NT; t++)
#pragma unroll
            for (int i = 0; i < GR; i++) {
                const f32x4 o = s_part[((p * NT + t) * GR + i) * 64 + lane];
#pragma unroll
                for (int j = 0; j < 4; j++) acc[t][i][j] += o[j];
            }
    }
    if (a.out >= kMixOutGated) {
        if constexpr (NT % 2 == 0) {
#pragma unroll
            for (int t = 0; t < NT; t += 2)
#pragma unroll
                for (int i = 0; i < GR; i++)
                    mix_store_tile<F32>(a, acc[t][i], acc[t + 1][i], nt0 + t, group0 + i, z, lane);
        }
        return;
    }
#pragma unroll
    for (int t = 0; t < NT; t++)
#pragma unroll
        for (int i = 0; i < GR; i++) mix_store_tile<F32>(a, acc[t][i], acc[t][i], nt0 + t, group0 + i, z, lane);
}

// 2 x 2 waves of 64 outputs x 16 GROUPS rows each: 128 outputs x 32 GROUPS rows a
// workgroup.  Per k-step 8 weight tiles and 2 GROUPS fragments, one KiB each and
// already in operand order, go to LDS by direct loads two k-steps ahead in a ring
// of three stages; lane i reads its operands back at 16 i.  With group_expert a
// workgroup's row groups share one expert.
template <int GROUPS>
constexpr size_t mix_gemm_lds_bytes() { return (size_t)3 * (8 + 2 * GROUPS) * 1024; }

template <int GROUPS>
__global__ __launch_bounds__(256, 2) void mix_gemm_lds_kernel(const MixGemmArgs a)
{
    extern __shared__ __attribute__((aligned(16))) unsigned char mix_smem[];
    constexpr int NT = 4, CHUNKS = 8 + 2 * GROUPS, CPW = CHUNKS / 4, RING = 3;
    static_assert(CHUNKS % 4 == 0, "every wave copies the same number of chunks");
    constexpr uint32_t STAGE = CHUNKS * 1024;
    const int lane = threadIdx.x & 63;
    const uint32_t wave = (uint32_t)__builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t wn = wave & 1, wr = wave >> 1;
    // XCD x takes the output panels x, x + 8, ...: one after the other through all row panels; with experts
    // up to four side by side, so that the rows (few per expert, and each expert has weights of its own) are
    // fetched into the XCD's L2 once for the four
    const uint32_t nx = (a.ntiles + 7) / 8, ny = (a.groups + 2 * GROUPS - 1) / (2 * GROUPS);
    const uint32_t xcd = blockIdx.x % 8, slot = blockIdx.x / 8, share = (nx + 7) / 8;
    const uint32_t side = a.group_expert ? (share % 4 == 0 ? 4u : (share % 2 == 0 ? 2u : 1u)) : 1u;
    // (fewer panels than XCDs: panels and rows dealt out as they come, or most XCDs would stand idle)
    const bool few = nx < 8;
    const uint32_t px = few ? blockIdx.x % nx : (slot / (ny * side) * side + slot % side) * 8 + xcd;
    const uint32_t py = few ? blockIdx.x / nx : slot / side % ny, z = blockIdx.y;
    if (px >= nx) return;
    const uint32_t nt_wg = px * 8, g_wg = py * 2 * GROUPS;
    uint32_t mat = z;
    if (a.group_expert) {
        const int e = a.group_expert[g_wg];
        if (e < 0) return;
        mat = (uint32_t)e;
    }
    const uint32_t klast = a.ktiles - 1;
    const uint32_t lds0 = (uint32_t)__builtin_amdgcn_readfirstlane((uint32_t)(uintptr_t)mix_smem);
    const unsigned char* src[CPW];
#pragma unroll
    for (int i = 0; i < CPW; i++) {
        const uint32_t c = wave * CPW + i;
        const unsigned char* p =
            c < 8 ? reinterpret_cast<const unsigned char*>(a.w) +
                        ((size_t)mat * a.ntiles + min(nt_wg + c, a.ntiles - 1)) * a.ktiles * 1024
                  : reinterpret_cast<const unsigned char*>(a.x) +
                        ((size_t)min(g_wg + c - 8, a.groups - 1) * a.x_kt + (size_t)z * a.x_kt_z) * 1024;
        src[i] = uniform_ptr(p);
    }
    const uint32_t lane_off = lane * 16;
    auto issue = [&](uint32_t kt) {
        const size_t k = (size_t)min(kt, klast) * 1024;
        const uint32_t to = lds0 + (kt % RING) * STAGE + wave * CPW * 1024;
#pragma unroll
        for (int i = 0; i < CPW; i++) lds_direct_load(to + i * 1024, src[i] + k, lane_off);
    };

    f32x4 acc[NT][GROUPS];
#pragma unroll
    for (int t = 0; t < NT; t++)
#pragma unroll
        for (int i = 0; i < GROUPS; i++) acc[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};

    issue(0);
    issue(1);
    const uint32_t w_off = wn * NT * 1024 + lane * 16, x_off = (8 + wr * GROUPS) * 1024 + lane * 16;
    for (uint32_t kt = 0; kt < a.ktiles; kt++) {
        // this wave's copies of stage kt have landed (those of kt + 1 may be in flight),
        // and everybody has finished reading stage kt - 1
        asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" ::"n"(CPW) : "memory");
        issue(kt + 2);
        const unsigned char* st = mix_smem + (kt % RING) * STAGE;
        bf16x8 wv[NT], xv[GROUPS];
#pragma unroll
        for (int t = 0; t < NT; t++) wv[t] = *reinterpret_cast<const bf16x8*>(st + w_off + t * 1024);
#pragma unroll
        for (int i = 0; i < GROUPS; i++) xv[i] = *reinterpret_cast<const bf16x8*>(st + x_off + i * 1024);
#pragma unroll
        for (int i = 0; i < GROUPS; i++)
#pragma unroll
            for (int t = 0; t < NT; t++) acc[t][i] = mix_mfma(wv[t], xv[i], acc[t][i]);
        __builtin_amdgcn_sched_group_barrier(0x100, NT + GROUPS, 0);
        __builtin_amdgcn_sched_group_barrier(0x008, NT * GROUPS, 0);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");       // the last steps' copies still target the ring

    const uint32_t nt0 = nt_wg + wn * NT, group0 = g_wg + wr * GROUPS;
    if (nt0 >= a.ntiles || group0 >= a.groups) return;
    if (a.out >= kMixOutGated) {
#pragma unroll
        for (int t = 0; t < NT; t += 2)
#pragma unroll
            for (int i = 0; i < GROUPS; i++)
                mix_store_tile<false>(a, acc[t][i], acc[t + 1][i], nt0 + t, group0 + i, z, lane);
        return;
    }
#pragma unroll
    for (int t = 0; t < NT; t++)
#pragma unroll
        for (int i = 0; i < GROUPS; i++)
            mix_store_tile<false>(a, acc[t][i], acc[t][i], nt0 + t, group0 + i, z, lane);
}

}  // namespace wr
