// retention.h — linear attention with a fixed decay per head on gfx950: S_t = decay S_(t-1) + k_t v_t^T (fp32,
// [dim][vdim] per head and sequence), o_t = S_t^T q_t, no softmax and no denominator.
//
// The state is cut into slices of kRetCols value columns, each a contiguous [dim][kRetCols] block
// (slot, head, slice), so one workgroup owns a slice in every form:
//   * ret_step_kernel: one token per sequence (decode): S read, updated and written once, 16-byte accesses;
//   * ret_scan_kernel: a portion token by token with the slice in LDS (the fp32 form, and any dim);
//   * retention_chunk.h: a portion 32 tokens at a time on the matrix cores.
// The raw o rows are then normalised per head and gated (ret_gate_kernel).
#pragma once
#include "canon.h"
#include "common.h"
#include "step_state.h"

namespace sli {

constexpr int kRetCols = 32;  // value columns per state slice

struct RetArgs {
    const float* q;      // [M][H dim] rotated
    const float* k;      // [M][H dim] rotated, scaled
    const float* v;      // [M][H vdim]
    float* S;            // [slots][H][nsl][dim][kRetCols]
    float* o;            // [M][H vdim] raw
    const float* decay;  // [H]
    const RowRef* rows;
    const SegRef* segs;  // portions of the pass (scan / chunk forms)
    const int32_t* nsegs;
    int H, dim, vdim, nsl;
    float* ssq = nullptr;  // [M][H][nsl] sums of o^2 over a slice (step form, nullable)
};

__device__ __forceinline__ float* ret_slice(const RetArgs& a, int slot, int h, int sl) {
    return a.S + (((size_t)slot * a.H + h) * a.nsl + sl) * (size_t)a.dim * kRetCols;
}

// grid (nsl, H, M), 256 threads: thread = (4 columns, one of 32 row groups)
__global__ void __launch_bounds__(256) ret_step_kernel(RetArgs a) {
    const int sl = blockIdx.x, h = blockIdx.y, m = blockIdx.z;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    __shared__ float4 red[4][8];
    const int c4 = threadIdx.x & 7, g = threadIdx.x >> 3;
    const int col = sl * kRetCols + 4 * c4;
    float* S = ret_slice(a, r.slot, h, sl);
    const float* qr = a.q + ((size_t)m * a.H + h) * a.dim;
    const float* kr = a.k + ((size_t)m * a.H + h) * a.dim;
    const float* vr = a.v + ((size_t)m * a.H + h) * a.vdim;
    const float dec = a.decay[h];
    const bool fresh = r.pos == 0;  // the state starts at zero: whatever the slot held is not read
    float4 v;
    v.x = col + 0 < a.vdim ? vr[col + 0] : 0.0f;
    v.y = col + 1 < a.vdim ? vr[col + 1] : 0.0f;
    v.z = col + 2 < a.vdim ? vr[col + 2] : 0.0f;
    v.w = col + 3 < a.vdim ? vr[col + 3] : 0.0f;
    float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
    constexpr int U = 8;
    for (int i0 = g; i0 < a.dim; i0 += 32 * U) {
        float4 s[U];
        float kk[U], qq[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = min(i0 + 32 * u, a.dim - 1);
            s[u] = reinterpret_cast<const float4*>(S + (size_t)i * kRetCols)[c4];
            kk[u] = kr[i];
            qq[u] = qr[i];
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int i = i0 + 32 * u;
            if (i >= a.dim) break;
            const float4 p = fresh ? make_float4(0.f, 0.f, 0.f, 0.f) : mul4(s[u], dec);
            const float4 n = make_float4(fmaf(kk[u], v.x, p.x), fmaf(kk[u], v.y, p.y), fmaf(kk[u], v.z, p.z),
                                         fmaf(kk[u], v.w, p.w));
            reinterpret_cast<float4*>(S + (size_t)i * kRetCols)[c4] = n;
            acc = make_float4(fmaf(n.x, qq[u], acc.x), fmaf(n.y, qq[u], acc.y), fmaf(n.z, qq[u], acc.z),
                              fmaf(n.w, qq[u], acc.w));
        }
    }
    // the 8 row groups of a wave (lanes 8 apart), then the 4 waves
    acc = make_float4(stride_sum<8>(acc.x), stride_sum<8>(acc.y), stride_sum<8>(acc.z), stride_sum<8>(acc.w));
    if ((threadIdx.x & 63) < 8) red[threadIdx.x >> 6][c4] = acc;
    __syncthreads();
    if (threadIdx.x < 8) {
        float4 t = red[0][c4];
        for (int w = 1; w < 4; ++w)
            t = make_float4(t.x + red[w][c4].x, t.y + red[w][c4].y, t.z + red[w][c4].z, t.w + red[w][c4].w);
        float* o = a.o + ((size_t)m * a.H + h) * a.vdim;
        if (col + 0 < a.vdim) o[col + 0] = t.x;
        if (col + 1 < a.vdim) o[col + 1] = t.y;
        if (col + 2 < a.vdim) o[col + 2] = t.z;
        if (col + 3 < a.vdim) o[col + 3] = t.w;
        // (columns past vdim are zero: their v is)
        const float q2 = group_sum<8>(sq4(t));
        if (a.ssq && c4 == 0) a.ssq[((size_t)m * a.H + h) * a.nsl + sl] = q2;
    }
}

// grid (nsl, H, portions), 256 threads; dynamic LDS: the slice [dim][kRetCols], then q and k of one token
inline size_t ret_scan_lds(int dim) { return sizeof(float) * ((size_t)dim * kRetCols + 2 * dim + 8 * kRetCols); }
__global__ void __launch_bounds__(256) ret_scan_kernel(RetArgs a) {
    extern __shared__ __attribute__((aligned(16))) float rs_sm[];
    const int sl = blockIdx.x, h = blockIdx.y;
    if ((int)blockIdx.z >= *a.nsegs) return;
    const SegRef sg = a.segs[blockIdx.z];
    float* S = rs_sm;
    float* qs = S + (size_t)a.dim * kRetCols;
    float* ks = qs + a.dim;
    float* red = ks + a.dim;  // [8][kRetCols]
    const int c = threadIdx.x & 31, g = threadIdx.x >> 5;
    const int col = sl * kRetCols + c;
    float* Sg = ret_slice(a, sg.slot, h, sl);
    const float dec = a.decay[h];
    for (int i = threadIdx.x; i < a.dim * kRetCols; i += 256) S[i] = sg.pos0 == 0 ? 0.0f : Sg[i];
    for (int t = 0; t < sg.n; ++t) {
        const size_t row = (size_t)(sg.row0 + t) * a.H + h;
        __syncthreads();
        for (int i = threadIdx.x; i < a.dim; i += 256) {
            qs[i] = a.q[row * a.dim + i];
            ks[i] = a.k[row * a.dim + i];
        }
        const float v = col < a.vdim ? a.v[row * a.vdim + col] : 0.0f;
        __syncthreads();
        float acc = 0.0f;
        for (int i = g; i < a.dim; i += 8) {
            const float n = fmaf(ks[i], v, dec * S[i * kRetCols + c]);
            S[i * kRetCols + c] = n;
            acc = fmaf(n, qs[i], acc);
        }
        red[g * kRetCols + c] = acc;
        __syncthreads();
        if (g == 0 && col < a.vdim) {
            float s = 0.0f;
            for (int w = 0; w < 8; ++w) s += red[w * kRetCols + c];
            a.o[row * a.vdim + col] = s;
        }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < a.dim * kRetCols; i += 256) Sg[i] = S[i];
}

// out[m][h vdim + d] = o / sqrt(mean_d(o^2) + eps) * gate   (one wave per row and head; gate = silu(g) already)
template <typename OT>
__global__ void __launch_bounds__(256) ret_gate_kernel(const float* __restrict__ o, const float* __restrict__ gate,
                                                       const RowRef* __restrict__ rows, OT* __restrict__ out, int ldo,
                                                       int M, int H, int vdim, float eps) {
    const int w = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (w >= M * H) return;
    const int m = w / H, h = w - m * H;
    if (rows[m].slot < 0) return;
    const float* orow = o + (size_t)w * vdim;
    float ss = 0.0f;
    for (int d = lane; d < vdim; d += 64) ss += orow[d] * orow[d];
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)vdim + eps);
    for (int d = lane; d < vdim; d += 64)
        out[(size_t)m * ldo + (size_t)h * vdim + d] = from_f32<OT>(orow[d] * inv * gate[(size_t)w * vdim + d]);
}

}  // namespace sli
