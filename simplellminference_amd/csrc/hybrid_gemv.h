// hybrid_gemv.h — the two weight-streaming launches of a block-stack layer at batch 1 (gemv.h schedules):
//   * hy_in_kernel: norm + input convolution (canon.h) computed in the prologue, the mixer's and the feed-forward's input
//     projections as two workgroup ranges of one launch (each range stages its own sublayer's input);
//   * hy_out_kernel: the mixer's output (retention: normalised per head and gated in the prologue) next to the
//     feed-forward product, and one pass over [W_o | W_down] adds both sublayers to the residual.
#pragma once
#include "canon.h"
#include "gemv.h"
#include "hybrid_kernels.h"

namespace sli {

// ---------------------------------------------------------------- input side
// One float4 of the row per thread (ld <= 4 * kGemvThreads), taps == kCanonFusedTaps. All ring rows are loaded, in row
// order, so no address waits for the position; which row is which tap is sorted out in commit. The ring row of this
// position is not read (the row itself takes its place), so the first workgroup may overwrite it meanwhile.
template <int G>
struct XStageCanon {
    CanonArgs a;
    const float* f;  // this sublayer's coefficients
    bool write;      // this workgroup stores the new ring row
    using Args = CanonArgs;
    __device__ __forceinline__ XStageCanon(const CanonArgs& a_, bool second, bool first_block)
        : a(a_), f(second ? a_.f2 : a_.f1), write(first_block) {}
    float4 x, r[kCanonFusedTaps], c[kCanonFusedTaps];
    int pos = 0, slot = 0;
    __device__ __forceinline__ void issue(const GemvIn& in) {
        const int n4 = in.cols >> 2, i = min((int)threadIdx.x, n4 - 1);
        slot = a.rows->slot;
        pos = a.rows->pos;
        const float4* ring = reinterpret_cast<const float4*>(a.ring + (size_t)slot * kCanonFusedTaps * a.ld);
        x = reinterpret_cast<const float4*>(a.x)[i];
#pragma unroll
        for (int j = 0; j < kCanonFusedTaps; ++j) {
            r[j] = ring[(size_t)j * n4 + i];
            c[j] = reinterpret_cast<const float4*>(f)[(size_t)j * n4 + i];
        }
    }
    // + coefficient J times the row J positions back (ring row R), zero before the sequence's start
    template <int J, int R>
    __device__ __forceinline__ float4 tap(const float4& s) const {
        return pos >= J ? fma4(c[J], r[R], s) : s;
    }
    __device__ __forceinline__ void commit(float* smem, const GemvIn& in) {
        static_assert(kCanonFusedTaps == 4, "taps");
        float* red = smem;
        const int tid = threadIdx.x, n4 = in.cols >> 2, i = min(tid, n4 - 1);
        float ss = wave_sum(tid < n4 ? sq4(x) : 0.0f);
        if ((tid & 63) == 0) red[tid >> 6] = ss;
        __syncthreads();
        float t = 0.0f;
#pragma unroll
        for (int w = 0; w < (kGemvThreads >> 6); ++w) t += red[w];
        const float4 n = mul4(x, 1.0f / sqrtf(t / (float)a.D + a.eps));
        float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
        switch (pos & 3) {  // uniform: the row of position p is p % 4
            case 0: s = tap<1, 3>(tap<2, 2>(tap<3, 1>(s))); break;
            case 1: s = tap<1, 0>(tap<2, 3>(tap<3, 2>(s))); break;
            case 2: s = tap<1, 1>(tap<2, 0>(tap<3, 3>(s))); break;
            default: s = tap<1, 2>(tap<2, 1>(tap<3, 0>(s))); break;
        }
        s = fma4(c[0], n, s);
        reinterpret_cast<float4*>(smem + kGemvLdsHead)[xswz<G>(i)] = s;
        if (write && tid < n4)
            reinterpret_cast<float4*>(a.ring + ((size_t)slot * kCanonFusedTaps + (pos & 3)) * a.ld)[i] = n;
    }
};

// workgroups [0, b1): pairs [0, n1) with the first sublayer's input; [b1, grid): pairs [u2, u2 + n2) with the second's
// (Stage(args, second, first workgroup): what a range stages)
template <typename WT, class Epi, class Stage, bool SPLIT>
__global__ void __launch_bounds__(kGemvThreads) hy_in_kernel(const WT* __restrict__ W, GemvIn in_, typename Stage::Args a,
                                                             Epi epi, int n1, int u2, int n2, int b1) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    const bool second = (int)blockIdx.x >= b1;  // uniform
    GemvIn in = in_;
    in.blk0 = second ? b1 : 0;
    in.blk1 = second ? (int)gridDim.x : b1;
    Stage stage(a, second, blockIdx.x == 0);
    GvPair<Epi> e{epi, second ? n2 : n1, second ? u2 : 0};
    gemv_block<WT, 2, 4, true, GvPair<Epi>, Stage, 2, SPLIT, true>(W + (second ? (size_t)2 * u2 * in.cols : 0), in, e, stage,
                                                                   smem);
}

template <typename WT, template <int> class StageT = XStageCanon, class Epi, class SA>
hipError_t launch_hy_in(const WT* W, const SA& a, const Epi& epi, int n1, int u2, int n2, hipStream_t s) {
    using Stage = StageT<Vec16<WT>::N / 4>;
    GemvIn in{nullptr, nullptr, 0.0f, a.ld};
    constexpr int waves = kGemvThreads / 64;
    // two column parts per pair where the rows are long enough: waves then differ by half a pair
    const int cs = a.ld / Vec16<WT>::N > 4 * 64 ? 2 : 1;
    in.csplit = cs;
    int b1 = std::max(1, std::min(n1, (n1 * cs + waves - 1) / waves)), b2 = n2 ? std::max(1, std::min(n2, (n2 * cs + waves - 1) / waves)) : 0;
    const int maxb = gemv_max_blocks();
    if (b1 + b2 > maxb) {
        const int g = std::max(2, maxb);
        b1 = n2 ? std::max(1, std::min(g - 1, (int)((long long)g * n1 / (n1 + n2)))) : g;
        // the split whose fuller range has the fewest items per wave
        auto worst = [&](int b) {
            auto per = [&](int n, int w) { return (n * cs + w * waves - 1) / (w * waves); };
            return n2 ? std::max(per(n1, b), per(n2, g - b)) : per(n1, b);
        };
        if (n2)
            for (int b : {b1 - 4, b1 - 3, b1 - 2, b1 - 1, b1 + 1, b1 + 2, b1 + 3, b1 + 4})
                if (b >= 1 && b < g && worst(b) < worst(b1)) b1 = b;
        b2 = n2 ? g - b1 : 0;
    }
    const size_t res = std::max(gemv_res_floats(n1, b1, 2, cs), n2 ? gemv_res_floats(n2, b2, 2, cs) : 0);
    const size_t lds = gemv_lds_bytes(in.cols) + sizeof(float) * res;
    if (cs > 1)
        hipLaunchKernelGGL((hy_in_kernel<WT, Epi, Stage, true>), dim3(b1 + b2), dim3(kGemvThreads), lds, s, W, in, a, epi, n1, u2, n2, b1);
    else
        hipLaunchKernelGGL((hy_in_kernel<WT, Epi, Stage, false>), dim3(b1 + b2), dim3(kGemvThreads), lds, s, W, in, a, epi, n1, u2, n2, b1);
    return hipGetLastError();
}

// ---------------------------------------------------------------- output side
constexpr int kHyOutSlices = 8;  // retention slices per head held in registers (more are read in commit)
constexpr int kHyOutAct = 4;     // float4 of the feed-forward product per thread

// The mixer part (KA = 4 * float4s, one per thread: KA <= 4 * kGemvThreads; vdim % 4 == 0), then the feed-forward part.
struct HyOutIn {
    const float* cat;   // [KA + KF]: the mixer's output (attention), the feed-forward product at KA
    int KA, KF, mixw, vdim;
    // retention: raw o, silu gate, sums of o^2 per (head, slice)
    const float *o, *gate, *ssq;
    int nsl;
    float eps;
};

template <int G, bool RET>
struct XStageCat {
    HyOutIn a;
    float4 act[kHyOutAct];
    float4 mix, gate;
    float sq[RET ? kHyOutSlices : 1];
    __device__ __forceinline__ void issue(const GemvIn&) {
        const int tid = threadIdx.x, f = min(4 * tid, a.mixw - 4);
        if constexpr (RET) {
            const int h = f / a.vdim;
            mix = *reinterpret_cast<const float4*>(a.o + f);
            gate = *reinterpret_cast<const float4*>(a.gate + f);
#pragma unroll
            for (int s = 0; s < kHyOutSlices; ++s) sq[s] = a.ssq[(size_t)h * a.nsl + min(s, a.nsl - 1)];
        } else {
            mix = *reinterpret_cast<const float4*>(a.cat + f);
        }
        const int na = max(a.KF >> 2, 1);
        const float4* src = reinterpret_cast<const float4*>(a.cat + (a.KF ? a.KA : 0));
#pragma unroll
        for (int k = 0; k < kHyOutAct; ++k) act[k] = src[min(tid + k * kGemvThreads, na - 1)];
    }
    __device__ __forceinline__ void commit(float* smem, const GemvIn&) {
        float4* xs4 = reinterpret_cast<float4*>(smem + kGemvLdsHead);
        const int tid = threadIdx.x, n4 = a.KA >> 2;
        float4 y = mix;
        if constexpr (RET) {
            const int h = min(4 * tid, a.mixw - 4) / a.vdim;
            float t = 0.0f;
#pragma unroll
            for (int s = 0; s < kHyOutSlices; ++s)
                if (s < a.nsl) t += sq[s];
            for (int s = kHyOutSlices; s < a.nsl; ++s) t += a.ssq[(size_t)h * a.nsl + s];
            const float inv = 1.0f / sqrtf(t / (float)a.vdim + a.eps);
            y = make_float4(y.x * inv * gate.x, y.y * inv * gate.y, y.z * inv * gate.z, y.w * inv * gate.w);
        }
        if (tid < n4) xs4[xswz<G>(tid)] = 4 * tid < a.mixw ? y : make_float4(0.f, 0.f, 0.f, 0.f);
        const int na = a.KF >> 2;
#pragma unroll
        for (int k = 0; k < kHyOutAct; ++k)
            if (tid + k * kGemvThreads < na) xs4[xswz<G>(n4 + tid + k * kGemvThreads)] = act[k];
    }
};

template <typename WT, bool RET, int U, bool SPLIT>
__global__ void __launch_bounds__(kGemvThreads) hy_out_kernel(const WT* __restrict__ W, GemvIn in, HyOutIn a, EpiStore<1> epi_in) {
    EpiStore<1> epi = epi_in;
    extern __shared__ __attribute__((aligned(16))) float smem[];
    constexpr int G = Vec16<WT>::N / 4;
    XStageCat<G, RET> stage{a};
    gemv_block<WT, 1, U, true, EpiStore<1>, XStageCat<G, RET>, 2, SPLIT>(W, in, epi, stage, smem);
}

inline bool hy_out_fits(int KA, int KF, int mixw, int vdim) {
    return KA <= 4 * kGemvThreads && KF <= 4 * kGemvThreads * kHyOutAct && vdim % 4 == 0 && mixw >= 4;
}

// (the widest input, 20480 columns, takes more LDS than a launch gets by default)
template <typename WT>
hipError_t hy_out_allow_lds() {
    hipError_t r = hipSuccess;
    auto allow = [&](auto* k) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize,
                                                 160 * 1024);
        if (e != hipSuccess) r = e;
    };
    allow(&hy_out_kernel<WT, true, 4, true>);
    allow(&hy_out_kernel<WT, true, 4, false>);
    allow(&hy_out_kernel<WT, false, 4, true>);
    allow(&hy_out_kernel<WT, false, 4, false>);
    return r;
}

template <typename WT, bool RET>
hipError_t launch_hy_out(const WT* W, const HyOutIn& a, const EpiStore<1>& e, int rows, hipStream_t s) {
    GemvIn in{nullptr, nullptr, 0.0f, a.KA + a.KF};
    constexpr int U = 4, waves = kGemvThreads / 64;
    const int cpr = (in.cols / Vec16<WT>::N + 64 * U - 1) / (64 * U);
    int cs = 1;
    while (cs < 8 && 2 * cs <= cpr && rows * cs < gemv_max_blocks() * waves) cs *= 2;
    in.csplit = cs;
    const int grid = cs == 1 ? gemv_balanced_blocks(rows) : gemv_blocks(rows, cs);
    const size_t lds = gemv_lds_bytes(in.cols) + sizeof(float) * gemv_res_floats(rows, grid, 1, cs);
    if (cs == 1)
        hipLaunchKernelGGL((hy_out_kernel<WT, RET, U, false>), dim3(grid), dim3(kGemvThreads), lds, s, W, in, a, e);
    else
        hipLaunchKernelGGL((hy_out_kernel<WT, RET, U, true>), dim3(grid), dim3(kGemvThreads), lds, s, W, in, a, e);
    return hipGetLastError();
}

}  // namespace sli
