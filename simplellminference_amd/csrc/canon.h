// canon.h — the input convolution of a sublayer on gfx950: what a sublayer reads, h_t, becomes
// h_t + sum_j w[:, j] * h_(t - taps + 1 + j) per channel (causal, zeros before the sequence's start), with
// h = RMS norm of the residual stream times one gain per sublayer.
//
// The gain is a scalar, so both sublayers of a parallel block read the same unit-gain row n_t = x_t / rms(x_t):
// a sublayer's gain and its "+ h_t" term are folded into its taps at load (c_t = sum_j f_j * n_(t-j), f_0 = g (1 +
// w_last), f_j = g w_(last-j)), and ONE ring of past n rows per layer run and sequence slot is the state of both
// convolutions: position p lives in ring row p % taps, so a decode step overwrites the row no tap reads any more.
// Everything here is fp32. CanonArgs::raw: the same for a sublayer that reads the residual stream without a norm.
#pragma once
#include "common.h"
#include "gemv.h"
#include "step_state.h"

namespace sli {

constexpr int kCanonMaxTaps = 32;
constexpr int kCanonFusedTaps = 4;  // the GEMV prologue's tap count (fewer taps are padded with zero coefficients)

struct CanonArgs {
    const float* x;       // [M][ld] residual rows
    float* ring;          // [slots][taps][ld]
    const float* f1;      // [taps][ld] folded coefficients, f[j] of the row j positions back
    const float* f2;      // second sublayer's (nullable)
    const RowRef* rows;   // [M]
    float eps;
    int D, ld, taps, M;
    bool raw = false;     // no norm: h is the residual row itself (the ring holds x rows); c2, where given without f2, is
                          // a copy of it
};

template <typename T>
__device__ __forceinline__ void store4(T* p, const float4& v);
template <>
__device__ __forceinline__ void store4<float>(float* p, const float4& v) { *reinterpret_cast<float4*>(p) = v; }
template <>
__device__ __forceinline__ void store4<__half>(__half* p, const float4& v) {
    const __half h[4] = {__float2half_rn(v.x), __float2half_rn(v.y), __float2half_rn(v.z), __float2half_rn(v.w)};
    *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(h);
}
__device__ __forceinline__ float4 fma4(const float4& a, const float4& b, const float4& c) {
    return make_float4(fmaf(a.x, b.x, c.x), fmaf(a.y, b.y, c.y), fmaf(a.z, b.z, c.z), fmaf(a.w, b.w, c.w));
}
__device__ __forceinline__ float4 mul4(const float4& a, float s) {
    return make_float4(a.x * s, a.y * s, a.z * s, a.w * s);
}
__device__ __forceinline__ float sq4(const float4& a) { return a.x * a.x + a.y * a.y + a.z * a.z + a.w * a.w; }

// 256 threads: 1 / rms of one row
__device__ __forceinline__ float row_inv_rms(const float* xr, int ld, int D, float eps, float* red) {
    float ss = 0.0f;
    for (int i = threadIdx.x; i < ld / 4; i += 256) ss += sq4(reinterpret_cast<const float4*>(xr)[i]);
    ss = wave_sum(ss);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    return 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)D + eps);
}

// One workgroup per row. write_ring: the launch holds one row per sequence (a decode step), so this row's n may go
// to the ring at once; a prompt pass writes its last rows with canon_ring_kernel after every row has read the ring.
template <typename OT>
__global__ void __launch_bounds__(256) canon_rows_kernel(CanonArgs a, OT* c1, OT* c2, int write_ring) {
    __shared__ float red[4];
    const int m = blockIdx.x;
    const RowRef r = a.rows[m];
    if (r.slot < 0) {  // padding: zeros, so that a GEMM over whole tiles reads finite numbers
        for (int i = threadIdx.x; i < a.ld / 4; i += 256) {
            store4(c1 + (size_t)m * a.ld + 4 * i, make_float4(0.f, 0.f, 0.f, 0.f));
            if (c2) store4(c2 + (size_t)m * a.ld + 4 * i, make_float4(0.f, 0.f, 0.f, 0.f));
        }
        return;
    }
    __shared__ float inv[kCanonMaxTaps];
    const int nin = min(min(a.taps - 1, r.pos), m - r.first);  // earlier rows of this pass under the taps
    for (int j = 0; j <= nin; ++j) {
        const float v = a.raw ? 1.0f : row_inv_rms(a.x + (size_t)(m - j) * a.ld, a.ld, a.D, a.eps, red);
        if (threadIdx.x == 0) inv[j] = v;
    }
    __syncthreads();
    float* ring = a.ring + (size_t)r.slot * a.taps * a.ld;
    const int nall = min(a.taps - 1, r.pos);
    for (int i = threadIdx.x; i < a.ld / 4; i += 256) {
        float4 s1 = make_float4(0.f, 0.f, 0.f, 0.f), s2 = s1;
        for (int j = nall; j >= 0; --j) {
            float4 n;
            if (j <= nin)
                n = mul4(reinterpret_cast<const float4*>(a.x + (size_t)(m - j) * a.ld)[i], inv[j]);
            else
                n = reinterpret_cast<const float4*>(ring + (size_t)((r.pos - j) % a.taps) * a.ld)[i];
            s1 = fma4(n, reinterpret_cast<const float4*>(a.f1 + (size_t)j * a.ld)[i], s1);
            if (a.f2) s2 = fma4(n, reinterpret_cast<const float4*>(a.f2 + (size_t)j * a.ld)[i], s2);
            if (j == 0 && !a.f2) s2 = n;
            if (j == 0 && write_ring) reinterpret_cast<float4*>(ring + (size_t)(r.pos % a.taps) * a.ld)[i] = n;
        }
        store4(c1 + (size_t)m * a.ld + 4 * i, s1);
        if (c2) store4(c2 + (size_t)m * a.ld + 4 * i, s2);
    }
}

// The same for kCanonFusedTaps taps and ld <= 4 * blockDim.x: one float4 of a row per thread, every row and coefficient
// in flight at once, the rows' sums in one exchange. RAW: CanonArgs::raw.
template <typename OT, bool RAW>
__global__ void __launch_bounds__(1024) canon4_rows_kernel(CanonArgs a, OT* c1, OT* c2, int write_ring) {
    constexpr int TAPS = kCanonFusedTaps;
    __shared__ float red[16][TAPS];
    const int m = blockIdx.x, n4 = a.ld / 4, tid = threadIdx.x, i = min(tid, n4 - 1);
    const RowRef r = a.rows[m];
    if (r.slot < 0) {
        if (tid < n4) {
            store4(c1 + (size_t)m * a.ld + 4 * i, make_float4(0.f, 0.f, 0.f, 0.f));
            if (c2) store4(c2 + (size_t)m * a.ld + 4 * i, make_float4(0.f, 0.f, 0.f, 0.f));
        }
        return;
    }
    const int nall = min(TAPS - 1, r.pos), nin = min(nall, m - r.first);
    float* ring = a.ring + (size_t)r.slot * TAPS * a.ld;
    float4 n[TAPS], f1[TAPS], f2[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
        const float* src = j <= nin ? a.x + (size_t)(m - j) * a.ld
                                    : j <= nall ? ring + (size_t)((r.pos - j) % TAPS) * a.ld : a.x + (size_t)m * a.ld;
        n[j] = reinterpret_cast<const float4*>(src)[i];
        f1[j] = reinterpret_cast<const float4*>(a.f1 + (size_t)j * a.ld)[i];
        if constexpr (!RAW) f2[j] = reinterpret_cast<const float4*>((c2 ? a.f2 : a.f1) + (size_t)j * a.ld)[i];
    }
    float4 s1 = make_float4(0.f, 0.f, 0.f, 0.f), s2 = s1;
    if constexpr (RAW) {
#pragma unroll
        for (int j = TAPS - 1; j >= 0; --j)  // (selects, no branches: the loads stay together)
            s1 = fma4(n[j], mul4(f1[j], j <= nall ? 1.0f : 0.0f), s1);
        s2 = n[0];
    } else {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) {
            const float ss = wave_sum(tid < n4 ? sq4(n[j]) : 0.0f);
            if ((tid & 63) == 0) red[tid >> 6][j] = ss;
        }
        __syncthreads();
#pragma unroll
        for (int j = TAPS - 1; j >= 0; --j) {
            if (j > nall) continue;
            if (j <= nin) {
                float t = 0.0f;
                for (int w = 0; w < (int)blockDim.x / 64; ++w) t += red[w][j];
                n[j] = mul4(n[j], 1.0f / sqrtf(t / (float)a.D + a.eps));
            }
            s1 = fma4(n[j], f1[j], s1);
            s2 = fma4(n[j], f2[j], s2);
        }
    }
    if (tid >= n4) return;
    if (write_ring) reinterpret_cast<float4*>(ring + (size_t)(r.pos % TAPS) * a.ld)[i] = n[0];
    store4(c1 + (size_t)m * a.ld + 4 * i, s1);
    if (c2) store4(c2 + (size_t)m * a.ld + 4 * i, s2);
}

template <typename OT>
hipError_t launch_canon_rows(const CanonArgs& a, OT* c1, OT* c2, int write_ring, hipStream_t s) {
    const dim3 bl((a.ld / 4 + 63) / 64 * 64);
    const bool four = a.taps == kCanonFusedTaps && a.ld <= 4096;
    if (four && a.raw)
        hipLaunchKernelGGL((canon4_rows_kernel<OT, true>), dim3(a.M), bl, 0, s, a, c1, c2, write_ring);
    else if (four)
        hipLaunchKernelGGL((canon4_rows_kernel<OT, false>), dim3(a.M), bl, 0, s, a, c1, c2, write_ring);
    else
        hipLaunchKernelGGL(canon_rows_kernel<OT>, dim3(a.M), dim3(256), 0, s, a, c1, c2, write_ring);
    return hipGetLastError();
}

// the last min(n, taps - 1) rows of every portion into the ring (after canon_rows_kernel of the same pass)
static __global__ void __launch_bounds__(256) canon_ring_kernel(CanonArgs a) {
    __shared__ float red[4];
    const int m = blockIdx.x;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    const int later = m + a.taps - 1;  // a later row of the portion that far ahead: this row is out of every tap's reach
    if (later < a.M && a.rows[later].slot >= 0 && a.rows[later].first == r.first) return;
    const float inv = a.raw ? 1.0f : row_inv_rms(a.x + (size_t)m * a.ld, a.ld, a.D, a.eps, red);
    float* ring = a.ring + ((size_t)r.slot * a.taps + r.pos % a.taps) * a.ld;
    for (int i = threadIdx.x; i < a.ld / 4; i += 256)
        reinterpret_cast<float4*>(ring)[i] = mul4(reinterpret_cast<const float4*>(a.x + (size_t)m * a.ld)[i], inv);
}

// plain RMS norm of gathered rows with a gain per channel: y[i] = x[idx[i]] / rms * g   (idx null: row i)
template <typename OT>
__global__ void __launch_bounds__(256) norm_rows_kernel(const float* __restrict__ x, const int32_t* __restrict__ idx,
                                                        const float* __restrict__ g, OT* __restrict__ y, int D, int ld,
                                                        float eps) {
    __shared__ float red[4];
    const int m = blockIdx.x;
    const float* xr = x + (size_t)(idx ? idx[m] : m) * ld;
    const float inv = row_inv_rms(xr, ld, D, eps, red);
    for (int i = threadIdx.x; i < ld / 4; i += 256) {
        const float4 v = reinterpret_cast<const float4*>(xr)[i], w = reinterpret_cast<const float4*>(g)[i];
        store4(y + (size_t)m * ld + 4 * i,
               make_float4(v.x * inv * w.x, v.y * inv * w.y, v.z * inv * w.z, v.w * inv * w.w));
    }
}

}  // namespace sli
