// attn_rows.h — softmax attention of packed rows (one query row per token of any sequence slot) over the slots'
// K/V caches, with two additions that any attention layer can switch on:
//   * a distance bias: score(i, j) = (q_i . k_j) scale - r1_h ln(1 + r2_h (i - j));
//   * a sink: the softmax denominator also holds exp(sink_h), which has no key, no value, no scale and no bias.
// attn_rows_kernel is the form for every shape and element type (one wave per row and query head, fp32 sums); the
// matrix-core forms of the same arithmetic are prefill.h pf_attn_mfma_kernel and attn_mfma.h, whose split partials
// attn_sink_merge_kernel finishes.
#pragma once
#include "attention.h"
#include "common.h"
#include "step_state.h"

namespace sli {

constexpr int kAttnRowsMaxV = 512;  // value dims per head

struct AttnRowsArgs {
    const float* q;  // [M][H][hd] (dims past `dim` zero)
    const void* kc;  // [slots][G][T][hd]
    const void* vc;
    const RowRef* rows;
    const float *r1, *r2, *sink;  // [H] each, nullable (r1 and r2 together)
    int H, G, dim, vdim, hd, T, M;
    float scale;
};

template <typename KT, typename OT>
__global__ void __launch_bounds__(64) attn_rows_kernel(AttnRowsArgs a, OT* out, int ldo) {
    extern __shared__ float ar_sm[];  // q[dim], p[64]
    float* qs = ar_sm;
    float* ps = ar_sm + a.dim;
    const int h = blockIdx.x, m = blockIdx.y, lane = threadIdx.x;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    const int kvh = h / (a.H / a.G);
    const KT* kc = (const KT*)a.kc + ((size_t)r.slot * a.G + kvh) * a.T * a.hd;
    const KT* vc = (const KT*)a.vc + ((size_t)r.slot * a.G + kvh) * a.T * a.hd;
    for (int d = lane; d < a.dim; d += 64) qs[d] = a.q[((size_t)m * a.H + h) * a.hd + d];
    __syncthreads();
    const float r1 = a.r1 ? a.r1[h] : 0.0f, r2 = a.r2 ? a.r2[h] : 0.0f;
    float mx = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.0f : 0.0f;
    constexpr int NV = kAttnRowsMaxV / 64;
    float o[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) o[i] = 0.0f;
    for (int t0 = 0; t0 <= r.pos; t0 += 64) {
        const int t = t0 + lane;
        float s = -INFINITY;
        if (t <= r.pos) {
            float d = 0.0f;
            for (int e = 0; e < a.dim; ++e) d = fmaf(qs[e], to_f32(kc[(size_t)t * a.hd + e]), d);
            s = d * a.scale;
            if (a.r1) s -= r1 * logf(1.0f + r2 * (float)(r.pos - t));
        }
        const float mn = fmaxf(mx, wave_max(s));
        const float corr = expf(mx - mn), p = expf(s - mn);
        l = l * corr + wave_sum(p);
        mx = mn;
        __syncthreads();
        ps[lane] = p;
        __syncthreads();
        const int n = min(64, r.pos - t0 + 1);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int d = lane + 64 * i;
            if (d >= a.vdim) break;
            float acc = o[i] * corr;
            for (int j = 0; j < n; ++j) acc = fmaf(ps[j], to_f32(vc[(size_t)(t0 + j) * a.hd + d]), acc);
            o[i] = acc;
        }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int d = lane + 64 * i;
        if (d < a.vdim) out[(size_t)m * ldo + (size_t)h * a.vdim + d] = from_f32<OT>(o[i] / l);
    }
}

// Merge of split partials [M H][max_splits][hd + pad] (o, m, l: attn_mfma.h) with the sink: row m's live splits are
// those that start at or before its position. grid (H, M), 128 threads, one value dim each.
template <typename OT>
__global__ void __launch_bounds__(128) attn_sink_merge_kernel(const float* __restrict__ part, AttnRowsArgs a, int max_splits,
                                                              int ppwg, OT* out, int ldo) {
    const int h = blockIdx.x, m = blockIdx.y;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    const int ns = min(r.pos / ppwg + 1, max_splits), ps = a.hd + kAttnPartPad;
    const float* p = part + (size_t)(m * a.H + h) * max_splits * ps;
    float M = a.sink[h];
    for (int s = 0; s < ns; ++s) M = fmaxf(M, p[(size_t)s * ps + a.hd]);
    for (int d = threadIdx.x; d < a.vdim; d += 128) {
        float o = 0.0f, L = expf(a.sink[h] - M);
        for (int s = 0; s < ns; ++s) {
            const float w = expf(p[(size_t)s * ps + a.hd] - M);
            o = fmaf(w, p[(size_t)s * ps + d], o);
            L = fmaf(w, p[(size_t)s * ps + a.hd + 1], L);
        }
        out[(size_t)m * ldo + (size_t)h * a.vdim + d] = from_f32<OT>(o / L);
    }
}

}  // namespace sli
