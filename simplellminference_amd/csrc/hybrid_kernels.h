// hybrid_kernels.h — the row-level kernels and projection epilogues of block-stack models (hybrid.h): embedding,
// the q/k/v(/gate) + feed-forward input projection's epilogue, the residual add of the fused output projection, a
// plain fp32 projection for every shape, and the adapters that run one epilogue under the GEMV (gemv.h), the batched
// MFMA projection (bgemm.h) and the prompt GEMM (prefill.h).
//
// Weight rows are stored in PAIRS: pair u is rows 2u and 2u + 1 of the fused matrix, the two rows whose sums are
// consumed together (a rotation pair {d, d + rot_dims / 2}, a {gate i, up i} pair, or two neighbours), so an epilogue
// sees complete pairs under all three kernels' tilings.
#pragma once
#include "bgemm.h"
#include "common.h"
#include "gemv.h"
#include "prefill.h"
#include "step_state.h"

namespace sli {

// ---------------------------------------------------------------- embedding
// rows of a decode step from the engine's states: one row per slot
// (rows B .. M - 1: padding)
static __global__ void hy_rows_kernel(const DevState* st, RowRef* rows, int B, int M) {
    for (int b = threadIdx.x; b < M; b += blockDim.x)
        rows[b] = b < B ? RowRef{b, st[b].pos, st[b].token, b} : RowRef{-1, 0, 0, b};
}

// (pos: learned position rows [positions][D], nullable; the context never exceeds them)
template <typename WT>
__global__ void __launch_bounds__(256) hy_embed_kernel(const RowRef* __restrict__ rows, const WT* __restrict__ emb,
                                                       const WT* __restrict__ pos, float scale, float* __restrict__ x,
                                                       int V, int D, int ld) {
    const int m = blockIdx.x;
    const RowRef r = rows[m];
    const bool ok = r.tok >= 0 && r.tok < V;
    for (int i = threadIdx.x; i < ld; i += 256)
        x[(size_t)m * ld + i] = r.slot < 0 || i >= D ? 0.0f
                                : ok ? to_f32(emb[(size_t)r.tok * D + i]) * scale +
                                           (pos ? to_f32(pos[(size_t)r.pos * D + i]) : 0.0f)
                                     : __int_as_float(0x7FC00000);
}

// ---------------------------------------------------------------- epilogues: pair(u, m, v0, v1)
// (pair2: pairs u and u + 1 at once, u even)
__device__ __forceinline__ void store2(float* p, const float* v) { *reinterpret_cast<float2*>(p) = make_float2(v[0], v[1]); }
__device__ __forceinline__ void store2(__half* p, const float* v) {
    *reinterpret_cast<__half2*>(p) = __halves2half2(__float2half_rn(v[0]), __float2half_rn(v[1]));
}
// The fused input projection. Pairs [0, e_g): the mixer's q, k, v(, g) heads; pairs [u1p, u1p + ff): {gate, up}.
// OT: element type of the feed-forward product in the output projection's input.
template <typename KT, typename OT>
struct HyIn {
    int retention;
    int H, G, dim, vdim, hpq, hpv;   // hpq / hpv: pairs per q,k / v,g head
    int e_q, e_k, e_v, e_g, u1p, ff;  // pair ranges
    int rh;                          // rotation pairs per head (rot_dims / 2)
    int hd, T;                       // padded cache row, context
    float kscale, limit;
    const float *cs, *sn;            // [T][rh]
    float *q, *k, *v, *g;            // attention: q [M][H hd]; retention: q, k [M][H dim], v, g [M][H vdim]
    KT *kc, *vc;                     // [slots][G][T][hd]
    OT* act;
    int act_ld, act_off;
    const RowRef* rows;
    int even;                        // dim, vdim multiples of 4, rh even: two neighbouring pairs share a head and a branch
    __device__ float glu(float gate, float up) const {
        const float gt = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
        return gt / (1.0f + expf(-1.702f * gt)) * (u + 1.0f);
    }
    // pairs u and u + 1, u even: one row lookup and one head division, neighbouring results stored together
    __device__ void pair2(int u, int m, const float* a, bool second) const {
        if (!even || !second || (u < u1p ? u + 1 >= e_g : u + 1 - u1p >= ff)) {
            pair(u, m, a[0], a[1]);
            if (second) pair(u + 1, m, a[2], a[3]);
            return;
        }
        const RowRef r = rows[m];
        if (r.slot < 0) return;
        if (u >= u1p) {
            const float y[2] = {glu(a[0], a[1]), glu(a[2], a[3])};
            store2(act + (size_t)m * act_ld + act_off + (u - u1p), y);
            return;
        }
        const bool qk = u < e_k, isq = u < e_q, isv = u < e_v;
        const int uu = isq ? u : qk ? u - e_q : isv ? u - e_k : u - e_v;
        const int hp = qk ? hpq : hpv, h = uu / hp, j = uu - h * hp;
        if (qk && j < rh) {  // two rotation pairs {j, j + rh}, {j + 1, j + 1 + rh} (retention only)
            const size_t at = (size_t)r.pos * rh + j;
            const float c0 = cs[at], s0 = sn[at], c1 = cs[at + 1], s1 = sn[at + 1], f = isq ? 1.0f : kscale;
            float* p = (isq ? q : k) + ((size_t)m * H + h) * dim + j;
            const float lo[2] = {(a[0] * c0 - a[1] * s0) * f, (a[2] * c1 - a[3] * s1) * f};
            const float hi[2] = {(a[1] * c0 + a[0] * s0) * f, (a[3] * c1 + a[2] * s1) * f};
            store2(p, lo);
            store2(p + rh, hi);
            return;
        }
        if (!retention) {
            if (isq) {
                *reinterpret_cast<float4*>(q + ((size_t)m * H + h) * hd + 2 * j) = make_float4(a[0], a[1], a[2], a[3]);
            } else {
                KT* p = (qk ? kc : vc) + (((size_t)r.slot * G + h) * T + r.pos) * hd + 2 * j;
                store2(p, a);
                store2(p + 2, a + 2);
            }
            return;
        }
        float4 y = make_float4(a[0], a[1], a[2], a[3]);
        if (qk && !isq) y = make_float4(y.x * kscale, y.y * kscale, y.z * kscale, y.w * kscale);
        if (!isv)
            y = make_float4(y.x / (1.0f + expf(-y.x)), y.y / (1.0f + expf(-y.y)), y.z / (1.0f + expf(-y.z)),
                            y.w / (1.0f + expf(-y.w)));
        float* p = isq ? q : qk ? k : isv ? v : g;
        *reinterpret_cast<float4*>(p + ((size_t)m * H + h) * (qk ? dim : vdim) + 2 * j) = y;
    }
    __device__ void dims(int j, int n, int& d0, int& d1) const {  // pair j of a head of n dims (d1 < 0: none)
        if (j < rh) {
            d0 = j, d1 = j + rh;
        } else {
            d0 = 2 * j;  // rot_dims + 2 (j - rh)
            d1 = d0 + 1 < n ? d0 + 1 : -1;
        }
    }
    __device__ void pair(int u, int m, float a0, float a1) const {
        const RowRef r = rows[m];
        if (r.slot < 0) return;
        if (u >= u1p) {
            const int i = u - u1p;
            if (i >= ff) return;
            act[(size_t)m * act_ld + act_off + i] = from_f32<OT>(glu(a0, a1));
            return;
        }
        if (u >= e_g) return;
        int d0, d1;
        if (u < e_k) {
            const bool isq = u < e_q;
            const int uu = isq ? u : u - e_q, h = uu / hpq, j = uu - h * hpq;
            dims(j, dim, d0, d1);
            if (j < rh) {
                const float c = cs[(size_t)r.pos * rh + j], s = sn[(size_t)r.pos * rh + j];
                const float t0 = a0 * c - a1 * s, t1 = a1 * c + a0 * s;
                a0 = t0, a1 = t1;
            }
            if (!retention) {
                if (isq) {
                    float* p = q + ((size_t)m * H + h) * hd;
                    p[d0] = a0;
                    if (d1 >= 0) p[d1] = a1;
                } else {
                    KT* p = kc + (((size_t)r.slot * G + h) * T + r.pos) * hd;
                    p[d0] = from_f32<KT>(a0);
                    if (d1 >= 0) p[d1] = from_f32<KT>(a1);
                }
            } else {
                float* p = (isq ? q : k) + ((size_t)m * H + h) * dim;
                const float f = isq ? 1.0f : kscale;
                p[d0] = a0 * f;
                if (d1 >= 0) p[d1] = a1 * f;
            }
            return;
        }
        const bool isv = u < e_v;
        const int uu = isv ? u - e_k : u - e_v, h = uu / hpv, j = uu - h * hpv;
        d0 = 2 * j;
        d1 = d0 + 1 < vdim ? d0 + 1 : -1;
        if (!retention) {
            KT* p = vc + (((size_t)r.slot * G + h) * T + r.pos) * hd;
            p[d0] = from_f32<KT>(a0);
            if (d1 >= 0) p[d1] = from_f32<KT>(a1);
        } else {
            if (!isv) {  // silu of the gate
                a0 = a0 / (1.0f + expf(-a0));
                a1 = a1 / (1.0f + expf(-a1));
            }
            float* p = (isv ? v : g) + ((size_t)m * H + h) * vdim;
            p[d0] = a0;
            if (d1 >= 0) p[d1] = a1;
        }
    }
};

// x[m][row] += mult * sum, rows 2u and 2u + 1
struct HyOut {
    float* x;
    int ld, D;
    float mult;
    __device__ void pair(int u, int m, float v0, float v1) const {
        float* p = x + (size_t)m * ld + 2 * u;
        if (2 * u < D) p[0] = fmaf(mult, v0, p[0]);
        if (2 * u + 1 < D) p[1] = fmaf(mult, v1, p[1]);
    }
    __device__ void pair2(int u, int m, const float* a, bool) const {  // u even, ld a multiple of 4
        float* p = x + (size_t)m * ld + 2 * u;
        if (2 * u + 3 < D) {
            const float4 r = *reinterpret_cast<const float4*>(p);
            *reinterpret_cast<float4*>(p) =
                make_float4(fmaf(mult, a[0], r.x), fmaf(mult, a[1], r.y), fmaf(mult, a[2], r.z), fmaf(mult, a[3], r.w));
            return;
        }
        pair(u, m, a[0], a[1]);
        pair(u + 1, m, a[2], a[3]);
    }
};

// y[m][row] = sum
struct HyStore {
    float* y;
    int ld, D;
    __device__ void pair(int u, int m, float v0, float v1) const {
        float* p = y + (size_t)m * ld + 2 * u;
        if (2 * u < D) p[0] = v0;
        if (2 * u + 1 < D) p[1] = v1;
    }
    __device__ void pair2(int u, int m, const float* a, bool) const {  // u even, ld a multiple of 4
        if (2 * u + 3 < D) {
            *reinterpret_cast<float4*>(y + (size_t)m * ld + 2 * u) = make_float4(a[0], a[1], a[2], a[3]);
            return;
        }
        pair(u, m, a[0], a[1]);
        pair(u + 1, m, a[2], a[3]);
    }
};

struct HyLogits {
    float* y;  // [M][n]
    int n, M;
    __device__ void pair(int u, int m, float v0, float v1) const {
        if (m >= M) return;
        float* p = y + (size_t)m * n + 2 * u;
        if (2 * u < n) p[0] = v0;
        if (2 * u + 1 < n) p[1] = v1;
    }
    __device__ void pair2(int u, int m, const float* a, bool) const {
        pair(u, m, a[0], a[1]);
        pair(u + 1, m, a[2], a[3]);
    }
};

// ---------------------------------------------------------------- adapters
// (u0: first pair of the matrix part a launch covers; the launch's W starts at row 2 u0)
template <class Epi>
struct GvPair {  // gemv.h, R = 2
    Epi e;
    int n, u0;
    __device__ int units() const { return n; }
    __device__ void rows(int u, int* r) const {
        r[0] = 2 * u;
        r[1] = 2 * u + 1;
    }
    __device__ void prefetch_a(int) {}
    __device__ void prefetch_b(int) {}
    __device__ void store(int u, const int*, const float* v) const { e.pair(u0 + u, 0, v[0], v[1]); }
    __device__ void finish(float*) const {}
};

template <class Epi>
struct BgPair {  // bgemm.h: tile rows i and i + 8 are pair 8 t + i
    Epi e;
    int n, u0;
    __device__ int row(int t, int i) const { return 2 * min(8 * t + (i & 7), n - 1) + (i >> 3); }
    __device__ void pre_a(int, int, int) {}
    __device__ void pre_b() {}
    __device__ void store(int t, int i, int b, float v0, float v1, unsigned long long*) const {
        if (8 * t + i < n) e.pair(u0 + 8 * t + i, b, v0, v1);
    }
    __device__ void finish(unsigned long long*, int, int) const {}
};

template <class Epi>
struct PgPair {  // prefill.h: plain 16-row tiles, 4 consecutive rows per store
    Epi e;
    int n, u0;
    __device__ int row(int t, int i) const { return t * 16 + i; }
    __device__ void store(int t, int i0, int m, const float* v, const PfState*) const {
        const int u = t * 8 + (i0 >> 1);
        if (u < n) e.pair2(u0 + u, m, v, u + 1 < n);
    }
};

// ---------------------------------------------------------------- the plain projection
// y = x W^T in fp32 for any row count: a workgroup owns 16 rows x 32 pairs, both operands through LDS 32 columns at a
// time (K a multiple of 32). The fp32 models' prompt and batch form. GR: row blocks with weights of their own (prefill.h
// PgGroups, blocks of kRowsGemmTile rows).
constexpr int kRowsGemmTile = 16;
template <typename WT, class Epi, bool GR = false>
__global__ void __launch_bounds__(256) rows_gemm_kernel(const WT* __restrict__ W, const float* __restrict__ X, int K,
                                                        int npairs, int u0, int M, Epi epi, PgGroups grp) {
    constexpr int BM = kRowsGemmTile, BU = 32, BK = 32;
    __shared__ float xs[BM][BK + 1];
    __shared__ float ws[2 * BU][BK + 1];
    const int ub = blockIdx.x * BU, mb = blockIdx.y * BM;
    int2 tile = make_int2(0, 0);
    if constexpr (GR) {
        if ((int)blockIdx.y >= *grp.ntiles) return;
        tile = grp.tiles[blockIdx.y];
        W += (size_t)tile.x * grp.wstride;
    }
    const int tm = threadIdx.x >> 4, tu = threadIdx.x & 15;
    float acc[2][2] = {};
    for (int k0 = 0; k0 < K; k0 += BK) {
        __syncthreads();
        for (int i = threadIdx.x; i < BM * BK; i += 256) {
            const int r = i / BK, c = i % BK;
            int m = mb + r;
            if constexpr (GR) m = grp.rowmap ? grp.rowmap[m] : tile.y + r;
            xs[r][c] = GR || m < M ? X[(size_t)m * K + k0 + c] : 0.0f;
        }
        for (int i = threadIdx.x; i < 2 * BU * BK; i += 256) {
            const int r = i / BK, c = i % BK;
            ws[r][c] = ub + r / 2 < npairs ? to_f32(W[(size_t)(2 * ub + r) * K + k0 + c]) : 0.0f;
        }
        __syncthreads();
        for (int k = 0; k < BK; ++k) {
            const float x = xs[tm][k];
#pragma unroll
            for (int p = 0; p < 2; ++p)
#pragma unroll
                for (int e = 0; e < 2; ++e) acc[p][e] = fmaf(x, ws[2 * (tu + 16 * p) + e][k], acc[p][e]);
        }
    }
    if (!GR && mb + tm >= M) return;
#pragma unroll
    for (int p = 0; p < 2; ++p)
        if (ub + tu + 16 * p < npairs) epi.pair(u0 + ub + tu + 16 * p, mb + tm, acc[p][0], acc[p][1]);
}

template <typename WT, class Epi>
hipError_t launch_rows_gemm(const WT* W, const float* X, int K, int npairs, int u0, int M, const Epi& e, hipStream_t s) {
    hipLaunchKernelGGL((rows_gemm_kernel<WT, Epi>), dim3((npairs + 31) / 32, (M + 15) / 16), dim3(256), 0, s, W, X, K,
                       npairs, u0, M, e, PgGroups{});
    return hipGetLastError();
}
template <typename WT, class Epi>
hipError_t launch_rows_gemm_grouped(const WT* W, const float* X, int K, int npairs, const PgGroups& g, int maxtiles,
                                    const Epi& e, hipStream_t s) {
    hipLaunchKernelGGL((rows_gemm_kernel<WT, Epi, true>), dim3((npairs + 31) / 32, maxtiles), dim3(256), 0, s, W, X, K,
                       npairs, 0, maxtiles * kRowsGemmTile, e, g);
    return hipGetLastError();
}

// first-maximum keys of whole logits rows: keys[b] over logits [B][n]
static __global__ void __launch_bounds__(256) hy_keys_kernel(const float* __restrict__ logits, int n,
                                                      unsigned long long* keys, int key_ld) {
    __shared__ unsigned long long red[4];
    const float* y = logits + (size_t)blockIdx.x * n;
    unsigned long long b = 0;
    for (int i = blockIdx.y * 256 + threadIdx.x; i < n; i += 256 * gridDim.y) {
        const unsigned long long k = argmax_key(y[i], (unsigned)i);
        b = k > b ? k : b;
    }
    b = wave_max_u64(b);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = b;
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w = 1; w < 4; ++w) b = red[w] > b ? red[w] : b;
        keys[(size_t)blockIdx.x * key_ld + blockIdx.y] = red[0] > b ? red[0] : b;
    }
}

// ---------------------------------------------------------------- weights
// rows of a source matrix [nrows][ncols] into rows map[r] of a fused matrix (row stride ld), from column col0 on
struct HySrcBuf {
    const float* p;
    __device__ float operator()(size_t i) const { return p[i]; }
};
template <typename WT, class Src>
__global__ void __launch_bounds__(256) hy_place_kernel(WT* __restrict__ dst, int ld, int col0,
                                                       const int32_t* __restrict__ map, int ncols, Src src) {
    const int r = blockIdx.x;
    WT* d = dst + (size_t)map[r] * ld + col0;
    for (int c = threadIdx.x; c < ncols; c += 256) d[c] = from_f32<WT>(src((size_t)r * ncols + c));
}

}  // namespace sli
