// gated.h — sublayers whose result is gated and normed before it joins the residual stream: with y the result, g the
// sublayer's gate (already through the sigmoid) and w one gain per channel, x <- x + w * RMSnorm(g * y). Everything here
// is fp32.
//   * gated_rows_kernel: rows of a batch or prompt pass; the result may be the weighted rows of a mixture (moe.h);
//   * XStageGated: the same for one row, as the input stage of the next GEMV (gemv.h), so that the residual add, the
//     norm and, where the next sublayer has one, the input convolution (canon.h, raw rows) cost no launch.
#pragma once
#include "canon.h"
#include "common.h"
#include "gemv.h"
#include "step_state.h"

namespace sli {

struct GatedArgs {
    const float *x, *y, *g, *w;  // [M][ld] rows (padding zero); w [ld]
    float* xout;                 // may be x where one launch owns a row (gated_rows_kernel)
    float eps;
    int D, ld;
    const RowRef* rows;
    __half* xh = nullptr;        // the new rows as fp16 (nullable; zeros for padding rows)
    // mixture: y holds expert rows, token m's result is sum_k wsel[m][k] y[at[m][k]]
    const int32_t* at = nullptr;
    const float* wsel = nullptr;
    int top = 0;
};

inline size_t gated_lds(int ld) { return sizeof(float) * ((size_t)ld + 4); }

template <bool MIX>
__global__ void __launch_bounds__(256) gated_rows_kernel(GatedArgs a) {
    extern __shared__ __attribute__((aligned(16))) float gt_sm[];
    float4* t = reinterpret_cast<float4*>(gt_sm);
    float* red = gt_sm + a.ld;
    const int m = blockIdx.x, n4 = a.ld / 4;
    if (a.rows[m].slot < 0) {
        if (a.xh)
            for (int i = threadIdx.x; i < n4; i += 256) store4(a.xh + (size_t)m * a.ld + 4 * i, make_float4(0.f, 0.f, 0.f, 0.f));
        return;
    }
    const float4* g = reinterpret_cast<const float4*>(a.g + (size_t)m * a.ld);
    float ss = 0.0f;
    for (int i = threadIdx.x; i < n4; i += 256) {
        float4 y;
        if constexpr (MIX) {
            y = make_float4(0.f, 0.f, 0.f, 0.f);
            for (int k = 0; k < a.top; ++k) {
                const float p = a.wsel[(size_t)m * a.top + k];
                y = fma4(reinterpret_cast<const float4*>(a.y + (size_t)a.at[(size_t)m * a.top + k] * a.ld)[i],
                         make_float4(p, p, p, p), y);
            }
        } else {
            y = reinterpret_cast<const float4*>(a.y + (size_t)m * a.ld)[i];
        }
        const float4 gv = g[i];
        y = make_float4(y.x * gv.x, y.y * gv.y, y.z * gv.z, y.w * gv.w);
        t[i] = y;
        ss += sq4(y);
    }
    ss = wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.D + a.eps);
    for (int i = threadIdx.x; i < n4; i += 256) {
        const float4 w = reinterpret_cast<const float4*>(a.w)[i];
        const float4 x = fma4(mul4(t[i], inv), w, reinterpret_cast<const float4*>(a.x + (size_t)m * a.ld)[i]);
        reinterpret_cast<float4*>(a.xout + (size_t)m * a.ld)[i] = x;
        if (a.xh) store4(a.xh + (size_t)m * a.ld + 4 * i, x);
    }
}

// One float4 of the row per thread (ld <= 4 * kGemvThreads). Every workgroup computes the new row; the first stores it to
// xout (another buffer than x, which the others still read) and its ring row. CONV: the first range of the launch stages
// the convolved row, the second the row itself.
struct GatedStageArgs {
    GatedArgs gt;
    CanonArgs cv;  // raw rows, kCanonFusedTaps taps
    int ld;
};
template <int G, bool CONV>
struct XStageGatedT {
    using Args = GatedStageArgs;
    GatedArgs a;
    CanonArgs cv;
    bool conv, write;
    float4 x, y, g, w, r[CONV ? kCanonFusedTaps : 1], c[CONV ? kCanonFusedTaps : 1];
    int pos = 0, slot = 0;
    __device__ __forceinline__ XStageGatedT(const Args& s, bool second, bool first_block)
        : a(s.gt), cv(s.cv), conv(CONV && !second), write(first_block) {}
    __device__ __forceinline__ void issue(const GemvIn& in) {
        const int n4 = in.cols >> 2, i = min((int)threadIdx.x, n4 - 1);
        x = reinterpret_cast<const float4*>(a.x)[i];
        y = reinterpret_cast<const float4*>(a.y)[i];
        g = reinterpret_cast<const float4*>(a.g)[i];
        w = reinterpret_cast<const float4*>(a.w)[i];
        if constexpr (CONV) {
            slot = cv.rows->slot;
            pos = cv.rows->pos;
            const float4* ring = reinterpret_cast<const float4*>(cv.ring + (size_t)slot * kCanonFusedTaps * cv.ld);
#pragma unroll
            for (int j = 0; j < kCanonFusedTaps; ++j) {
                r[j] = ring[(size_t)j * n4 + i];
                c[j] = reinterpret_cast<const float4*>(cv.f1)[(size_t)j * n4 + i];
            }
        }
    }
    // + coefficient J times the row J positions back (ring row R), zero before the sequence's start
    template <int J, int R>
    __device__ __forceinline__ float4 tap(const float4& s) const {
        return pos >= J ? fma4(c[J], r[R], s) : s;
    }
    __device__ __forceinline__ void commit(float* smem, const GemvIn& in) {
        float* red = smem;
        const int tid = threadIdx.x, n4 = in.cols >> 2, i = min(tid, n4 - 1);
        const float4 t = make_float4(y.x * g.x, y.y * g.y, y.z * g.z, y.w * g.w);
        const float ss = wave_sum(tid < n4 ? sq4(t) : 0.0f);
        if ((tid & 63) == 0) red[tid >> 6] = ss;
        __syncthreads();
        float sum = 0.0f;
#pragma unroll
        for (int k = 0; k < (kGemvThreads >> 6); ++k) sum += red[k];
        const float4 n = fma4(mul4(t, 1.0f / sqrtf(sum / (float)a.D + a.eps)), w, x);
        float4 s = n;
        if constexpr (CONV) {
            if (conv) {
                static_assert(kCanonFusedTaps == 4, "taps");
                s = make_float4(0.f, 0.f, 0.f, 0.f);
                switch (pos & 3) {  // uniform: the row of position p is p % 4
                    case 0: s = tap<1, 3>(tap<2, 2>(tap<3, 1>(s))); break;
                    case 1: s = tap<1, 0>(tap<2, 3>(tap<3, 2>(s))); break;
                    case 2: s = tap<1, 1>(tap<2, 0>(tap<3, 3>(s))); break;
                    default: s = tap<1, 2>(tap<2, 1>(tap<3, 0>(s))); break;
                }
                s = fma4(c[0], n, s);
            }
        }
        reinterpret_cast<float4*>(smem + kGemvLdsHead)[xswz<G>(i)] = s;
        if (write && tid < n4) {
            reinterpret_cast<float4*>(a.xout)[i] = n;
            if constexpr (CONV)
                reinterpret_cast<float4*>(cv.ring + ((size_t)slot * kCanonFusedTaps + (pos & 3)) * cv.ld)[i] = n;
        }
    }
};
template <int G>
using XStageGated = XStageGatedT<G, false>;
template <int G>
using XStageGatedCanon = XStageGatedT<G, true>;

}  // namespace sli
