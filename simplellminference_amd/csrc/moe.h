// moe.h — a mixture of experts on gfx950: each token uses the `top` experts with the largest router logits, weighted by
// the softmax over the chosen logits; an expert is down(silu(gate h) * (up h)).
//   * batches and prompts: moe_topk_kernel (a wave per token; a few tokens: in the next launch), moe_group_kernel sorts the (token, expert) pairs by expert
//     into row blocks of one tile height (a stable order: the same batch gives the same blocks), then two grouped GEMMs
//     (prefill.h PgGroups) read the token rows through the row map and write expert rows, which gated.h weights and adds;
//   * one token: the choice runs in the prologue of the gate / up GEMV (EpiMoeUp), which streams the chosen experts'
//     rows as one matrix, and moe_down_kernel sums the experts' down projections as column parts of one GEMV.
// Weights: gate / up [E][ffp pairs {gate i, up i}][Dp], down [E][Dn][FFp].
#pragma once
#include "attn_mfma.h"
#include "canon.h"
#include "common.h"
#include "gemv.h"
#include "prefill.h"
#include "step_state.h"

namespace sli {

constexpr int kMoeMaxExperts = 1024;
constexpr int kMoeMaxTop = 64;
constexpr int kMoeGroupRoutes = 16;  // rows at most whose choices moe_group_kernel makes
constexpr int kMoeFusedExperts = 256, kMoeFusedTop = 16;  // the one-token form

// One wave: f(k, expert) for the `top` largest of z[0 .. E), largest first, the lower index first among equals (uniform)
template <int NV, class F>
__device__ __forceinline__ void wave_topk(const float* z, int E, int top, F&& f) {
    const int lane = threadIdx.x & 63;
    unsigned long long key[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int e = lane + 64 * i;
        key[i] = e < E ? argmax_key(z[e], (unsigned)e) : 0ull;
    }
    for (int k = 0; k < top; ++k) {
        unsigned long long b = key[0];
#pragma unroll
        for (int i = 1; i < NV; ++i) b = key[i] > b ? key[i] : b;
        const int e = (int)min(argmax_key_index(wave_max_u64(b)), (unsigned)(E - 1));  // (in range whatever z holds)
        f(k, e);
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (lane + 64 * i == e) key[i] = 0ull;
    }
}
// the choice of one row by one wave: lane k (< top) returns expert k and its weight
template <int NV>
__device__ __forceinline__ void wave_route(const float* z, int E, int top, int& expert, float& weight) {
    const int lane = threadIdx.x & 63;
    expert = 0;
    wave_topk<NV>(z, E, top, [&](int k, int e) { expert = lane == k ? e : expert; });
    const float v = lane < top ? z[expert] : -INFINITY;
    const float p = expf(v - wave_max(v));  // 0 past top
    weight = p / wave_sum(p);
}

// one wave: the choice of row m
struct MoeRoute {
    const float* z;  // [M][E]
    const RowRef* rows;
    int M, E, top;
    int32_t* sel;  // [M][top], -1 for padding rows: no pairs
    float* wsel;
};
template <int NV>
__device__ __forceinline__ void moe_route_row(const MoeRoute& r, int m) {
    const int lane = threadIdx.x & 63;
    int e;
    float w;
    wave_route<NV>(r.z + (size_t)m * r.E, r.E, r.top, e, w);
    if (lane < r.top) {
        r.sel[(size_t)m * r.top + lane] = r.rows[m].slot < 0 ? -1 : e;
        r.wsel[(size_t)m * r.top + lane] = w;
    }
}
template <int NV>
__global__ void __launch_bounds__(256) moe_topk_kernel(MoeRoute r) {
    const int m = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (m < r.M) moe_route_row<NV>(r, m);
}

// Pairs p = token * top + k with sel[p] = expert, in expert order: at[p] = row of the pair, rowmap[row] = token, each
// expert's rows from a multiple of bm on (rows that fill up its last block read token 0), tiles[i] = {expert, first row}.
// One workgroup; wave w handles experts w, w + 16, ... NV > 0 (few rows): it also makes the choices, a wave per row.
template <int NV>
__global__ void __launch_bounds__(1024) moe_group_kernel(MoeRoute r, int bm, int32_t* __restrict__ at,
                                                         int32_t* __restrict__ rowmap, int2* __restrict__ tiles,
                                                         int32_t* __restrict__ ntiles) {
    __shared__ int base[kMoeMaxExperts + 1];  // first block of each expert
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, P = r.M * r.top, top = r.top, E = r.E;
    const int32_t* sel = r.sel;
    if constexpr (NV > 0) {
        for (int m = wave; m < r.M; m += 16) moe_route_row<NV>(r, m);
        __syncthreads();
    }
    constexpr int kU = 8;  // loads in flight
    int se[kU];
    auto load = [&](int p0) {  // pairs p0 + 64 j + lane (-1 past the last)
#pragma unroll
        for (int j = 0; j < kU; ++j) {
            const int p = p0 + 64 * j + lane;
            se[j] = sel[min(p, P - 1)];
            if (p >= P) se[j] = -1;
        }
    };
    for (int e = wave; e < E; e += 16) {
        int n = 0;
        for (int p0 = 0; p0 < P; p0 += 64 * kU) {
            load(p0);
#pragma unroll
            for (int j = 0; j < kU; ++j) n += (int)__popcll(__ballot(se[j] == e));
        }
        if (lane == 0) base[e + 1] = (n + bm - 1) / bm;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        base[0] = 0;
        for (int e = 0; e < E; ++e) base[e + 1] += base[e];
        *ntiles = base[E];
    }
    __syncthreads();
    for (int e = wave; e < E; e += 16) {
        const int r0 = base[e] * bm, r1 = base[e + 1] * bm;
        int n = 0;
        for (int p0 = 0; p0 < P && r1 > r0; p0 += 64 * kU) {
            load(p0);
#pragma unroll
            for (int j = 0; j < kU; ++j) {
                const bool mine = se[j] == e;
                const unsigned long long b = __ballot(mine);
                if (mine) {
                    const int p = p0 + 64 * j + lane, row = r0 + n + (int)__popcll(b & ((1ull << lane) - 1));
                    at[p] = row;
                    rowmap[row] = p / top;
                }
                n += (int)__popcll(b);
            }
        }
        for (int i = r0 + n + lane; i < r1; i += 64) rowmap[i] = 0;
        for (int t = base[e] + lane; t < base[e + 1]; t += 64) tiles[t] = make_int2(e, t * bm);
    }
}
// Router logits of a prompt's rows, z[m][e] = w[e] . x[m] + b[e] (few rows of weights: as part of a wide GEMM they would
// cost a column of its tiles). Grid (M / 16, E / 16), 4 waves that split K: A = 16 experts' rows, B = 16 tokens, both
// straight from memory.
static __global__ void __launch_bounds__(256) moe_router_kernel(const __half* __restrict__ w, const __half* __restrict__ x,
                                                                const float* __restrict__ b, int K, int E, float* __restrict__ z) {
    constexpr int kU = 8;
    __shared__ float4 red[3][64];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, i16 = lane & 15, g = lane >> 4;
    const int e0 = blockIdx.y * 16, m = blockIdx.x * 16 + i16;
    const int nkb = K / 32, kb0 = nkb * wave / 4, kb1 = nkb * (wave + 1) / 4;
    const __half* wp = w + (size_t)min(e0 + i16, E - 1) * K + 8 * g;
    const __half* xp = x + (size_t)m * K + 8 * g;
    am_float4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int k0 = kb0; k0 < kb1; k0 += kU) {
        u32x4 a[kU], v[kU];
#pragma unroll
        for (int j = 0; j < kU; ++j) {
            const int kb = min(k0 + j, kb1 - 1);
            a[j] = load16<false>(wp + 32 * kb);
            v[j] = load16<false>(xp + 32 * kb);
        }
#pragma unroll
        for (int j = 0; j < kU; ++j)
            if (k0 + j < kb1) acc = am_mfma(a[j], v[j], acc);
    }
    if (wave > 0) red[wave - 1][lane] = make_float4(acc[0], acc[1], acc[2], acc[3]);
    __syncthreads();
    if (wave > 0) return;
#pragma unroll
    for (int i = 0; i < 3; ++i) {
        const float4 r = red[i][lane];
        acc[0] += r.x, acc[1] += r.y, acc[2] += r.z, acc[3] += r.w;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
        if (e0 + 4 * g + i < E) z[(size_t)m * E + e0 + 4 * g + i] = acc[i] + b[e0 + 4 * g + i];
}

// row blocks P pairs can need
inline int moe_max_tiles(int P, int E, int bm) { return P / bm + std::min(E, P); }

__device__ __forceinline__ float silu_mul(float g, float u) { return g / (1.0f + expf(-g)) * u; }

// grouped gate / up: act[row][i] = silu(gate) * up
template <typename OT>
struct MoeAct {
    OT* act;
    int ld, ff;
    __device__ void pair(int u, int m, float g, float up) const {
        if (u < ff) act[(size_t)m * ld + u] = from_f32<OT>(silu_mul(g, up));
    }
    __device__ void pair2(int u, int m, const float* a, bool) const {  // u even, ld even
        if (u + 1 < ff) {
            const float y[2] = {silu_mul(a[0], a[1]), silu_mul(a[2], a[3])};
            store2(act + (size_t)m * ld + u, y);
            return;
        }
        pair(u, m, a[0], a[1]);
    }
};

// ---------------------------------------------------------------- one token
// gate / up rows of the chosen experts: unit u = pair u % ff of choice u / ff; act [top][ldk] fp32. Every wave routes for
// itself; the first wave of the first workgroup also writes the choice for moe_down_kernel.
struct EpiMoeUp {
    const float* z;
    int E, top, ff, ffp, ldk;
    float* act;
    int32_t* sel;
    float* wsel;
    int* ids;  // [kMoeFusedTop] in LDS
    __device__ int units() const { return top * ff; }
    __device__ void prefetch_a(int) {
        int e;
        float w;
        wave_route<kMoeFusedExperts / 64>(z, E, top, e, w);
        const int lane = threadIdx.x & 63;
        if (lane < top) {
            ids[lane] = e;  // (every wave stores the same values; a wave reads its own)
            if (blockIdx.x == 0 && threadIdx.x < 64) {
                sel[lane] = e;
                wsel[lane] = w;
            }
        }
        __builtin_amdgcn_wave_barrier();
    }
    __device__ void prefetch_b(int) {}
    __device__ void rows(int u, int* r) const {
        const int k = u / ff;
        r[0] = 2 * (ids[k] * ffp + u - k * ff);
        r[1] = r[0] + 1;
    }
    __device__ void store(int u, const int*, const float* v) const {
        const int k = u / ff;
        act[(size_t)k * ldk + u - k * ff] = silu_mul(v[0], v[1]);
    }
    __device__ void finish(float*) const {}
};

template <typename WT, bool SPLIT, int U>
__global__ void __launch_bounds__(kGemvThreads) moe_up_kernel(const WT* __restrict__ W, GemvIn in, EpiMoeUp epi_in) {
    __shared__ int ids[kMoeFusedTop];
    extern __shared__ __attribute__((aligned(16))) float smem[];
    EpiMoeUp epi = epi_in;
    epi.ids = ids;
    XStage<Vec16<WT>::N / 4> stage;
    gemv_block<WT, 2, U, true, EpiMoeUp, XStage<Vec16<WT>::N / 4>, 2, SPLIT>(W, in, epi, stage, smem);
}

// y[u] = sum_k wsel[k] (down row u of expert sel[k]) . act[k]: the choices are the GEMV's column parts
struct EpiMoeDown {
    static constexpr bool kParts = true;
    const int32_t* sel;
    int top, Dn, D;
    float* y;
    int* ids;  // [kMoeFusedTop] in LDS
    __device__ int units() const { return D; }
    __device__ void prefetch_a(int) {
        const int lane = threadIdx.x & 63;
        if (lane < top) ids[lane] = sel[lane];
        __builtin_amdgcn_wave_barrier();
    }
    __device__ void prefetch_b(int) {}
    __device__ void rows(int u, int* r) const { r[0] = u; }
    __device__ void rows_part(int u, int p, int* r) const { r[0] = ids[p] * Dn + u; }
    __device__ void store(int u, const int*, const float* v) const { y[u] = v[0]; }
    __device__ void finish(float*) const {}
};
// the choices' products, each times its weight (parts [csplit][cols])
template <int G>
struct XStageMoe {
    const float *act, *wsel;
    float4 xr[kGemvStageV4];
    float wr[kGemvStageV4];
    __device__ __forceinline__ void issue(const GemvIn& in) {
        const int n4 = in.cols >> 2, tot = n4 * in.csplit;
#pragma unroll
        for (int k = 0; k < kGemvStageV4; ++k) {
            const int f = min((int)threadIdx.x + k * kGemvThreads, tot - 1);
            xr[k] = reinterpret_cast<const float4*>(act)[f];
            wr[k] = wsel[f / n4];
        }
    }
    __device__ __forceinline__ void put(float* smem, int f, int n4, const float4& x, float w) const {
        const int p = f / n4, l = f - p * n4;
        reinterpret_cast<float4*>(smem + kGemvLdsHead)[p * n4 + xswz<G>(l)] = mul4(x, w);
    }
    __device__ __forceinline__ void commit(float* smem, const GemvIn& in) {
        const int n4 = in.cols >> 2, tot = n4 * in.csplit;
#pragma unroll
        for (int k = 0; k < kGemvStageV4; ++k) {
            const int f = (int)threadIdx.x + k * kGemvThreads;
            if (f < tot) put(smem, f, n4, xr[k], wr[k]);
        }
        for (int f = (int)threadIdx.x + kGemvStageV4 * kGemvThreads; f < tot; f += kGemvThreads)
            put(smem, f, n4, reinterpret_cast<const float4*>(act)[f], wsel[f / n4]);
    }
};
template <typename WT, int U>
__global__ void __launch_bounds__(kGemvThreads) moe_down_kernel(const WT* __restrict__ W, GemvIn in, EpiMoeDown epi_in,
                                                                const float* act, const float* wsel) {
    __shared__ int ids[kMoeFusedTop];
    extern __shared__ __attribute__((aligned(16))) float smem[];
    EpiMoeDown epi = epi_in;
    epi.ids = ids;
    using Stage = XStageMoe<Vec16<WT>::N / 4>;
    Stage stage{act, wsel};
    gemv_block<WT, 1, U, true, EpiMoeDown, Stage, 2, true>(W, in, epi, stage, smem);
}

constexpr size_t kMoeLdsMax = 159 * 1024;  // dynamic; a few words are static
inline size_t moe_down_lds(int cols, int top, int rows, int grid) {
    return gemv_lds_bytes(cols * top) + sizeof(float) * gemv_res_floats(rows, grid, 1, top);
}
template <typename WT>
hipError_t launch_moe_up(const WT* W, const float* x, int cols, const EpiMoeUp& e, hipStream_t s) {
    GemvIn in{x, nullptr, 0.0f, cols};
    const int units = e.top * e.ff;
    const GemvSplit sp = gemv_split<WT, 4>(units, cols);
    in.csplit = sp.cs;
    const int grid = sp.cs == 1 ? gemv_balanced_blocks(units) : gemv_blocks(units, sp.cs);
    const size_t lds = gemv_lds_bytes(cols) + sizeof(float) * gemv_res_floats(units, grid, 2, sp.cs);
    if (sp.cs == 1)
        hipLaunchKernelGGL((moe_up_kernel<WT, false, 4>), dim3(grid), dim3(kGemvThreads), lds, s, W, in, e);
    else if (sp.u == 4)
        hipLaunchKernelGGL((moe_up_kernel<WT, true, 4>), dim3(grid), dim3(kGemvThreads), lds, s, W, in, e);
    else if (sp.u == 2)
        hipLaunchKernelGGL((moe_up_kernel<WT, true, 2>), dim3(grid), dim3(kGemvThreads), lds, s, W, in, e);
    else
        hipLaunchKernelGGL((moe_up_kernel<WT, true, 1>), dim3(grid), dim3(kGemvThreads), lds, s, W, in, e);
    return hipGetLastError();
}
template <typename WT>
hipError_t launch_moe_down(const WT* W, const float* act, const float* wsel, int cols, const EpiMoeDown& e, hipStream_t s) {
    GemvIn in{nullptr, nullptr, 0.0f, cols};
    in.csplit = e.top;
    const int grid = gemv_blocks(e.D, e.top);
    const size_t lds = moe_down_lds(cols, e.top, e.D, grid);
    if (lds > kMoeLdsMax) return hipErrorInvalidValue;
    hipLaunchKernelGGL((moe_down_kernel<WT, 4>), dim3(grid), dim3(kGemvThreads), lds, s, W, in, e, act, wsel);
    return hipGetLastError();
}
template <typename WT>
hipError_t moe_allow_lds() {
    return hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_down_kernel<WT, 4>),
                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMoeLdsMax);
}

}  // namespace sli
