// latent.h — latent attention on gfx950: every token caches ONE RMS-normed row c of R values, and each head's keys and
// values are projections of it, k = U_k c, v = U_v c (no positions). A query sees the last `window` positions up to its
// own. The caches hold [slots][T][Rp] rows (Rp = R padded to 64, the padding zero).
//
// Two forms of the same attention:
//   * decode (and every shape and precision): absorbed. q . (U_k c) = (U_k^T q) . c, so a head's query becomes one row
//     of R values (lat_rows_kernel), all heads attend over the SAME rows c, which serve as keys and as values
//     (lat_attn_kernel on the matrix cores, lat_attn_rows_kernel plain), and U_v is applied to the R-value result
//     (lat_out_kernel). A step streams R values per past token, whatever the number of heads.
//   * prompts (fp16): expanded. K and V rows of the positions a pass can see are computed by one grouped GEMM straight
//     from the cache rows into scratch [heads][rows][hd] (lat_tiles_kernel lays the portions out), then prefill.h
//     pf_attn_mfma_kernel runs over them: (dim + vdim) multiply-adds per query, key and head instead of 2 R.
#pragma once
#include "attn_mfma.h"
#include "canon.h"
#include "common.h"
#include "prefill.h"
#include "step_state.h"

namespace sli {

constexpr int kLatMaxRank = 2048;
constexpr int kLatMfmaRank = 512;  // lat_attn_kernel: padded rank at most
constexpr int kLatKeys = 64;       // keys per tile of the decode attention
constexpr int kLatHeads = 16;      // heads per workgroup of it: the columns of an MFMA
constexpr int kLatMaxSplits = 32;
constexpr int kLatCols = 128;      // columns per workgroup of the absorbed query
constexpr int kLatTile = 64;       // cache rows per tile of the expansion
constexpr int kLatOutRows = 32;    // value rows per workgroup of lat_out_kernel

struct LatArgs {
    const float* lat;    // [M][Rp] rows of the down projection (padding zero)
    const float* lnorm;  // [Rp] gains (padding zero)
    void* cache;         // [slots][T][Rp]
    const RowRef* rows;
    const float* q;      // [M][H * dim]
    const void* uk;      // [H * dim][Rp]
    const void* uv;      // [H * vdim][Rp]
    float* qa;           // [M][H][Rp] absorbed queries
    float* part;         // [M][H][splits][Rp + kAttnPartPad]: o, m, l
    const float* gate;   // [M][H * vdim], already through the sigmoid
    int H, dim, vdim, R, Rp, T, window, splits;
    float scale, eps;
};
// keys a row sees, and their split over workgroups: tiles [s * per, (s + 1) * per) of the row's nt tiles
struct LatSpan {
    int lo, nt, per, ns;
};
__device__ __forceinline__ LatSpan lat_span(int pos, int window, int splits) {
    LatSpan s;
    s.lo = max(0, pos - window + 1);
    s.nt = (pos - s.lo + kLatKeys) / kLatKeys;
    s.per = (s.nt + splits - 1) / splits;
    s.ns = (s.nt + s.per - 1) / s.per;
    return s;
}

// Workgroup 0 of a row: its normed latent into the cache. Workgroups 1 .. H * chunks (decode): kLatCols columns of one
// head's absorbed query, U_k read along its rows (16 bytes of a row per lane, the rows of the head over lane groups).
template <typename KT, typename WT>
__global__ void __launch_bounds__(256) lat_rows_kernel(LatArgs a) {
    constexpr int VE = Vec16<WT>::N, LPR = kLatCols / VE, NG = 256 / LPR;
    __shared__ float red[NG][kLatCols];
    const int m = blockIdx.y, tid = threadIdx.x;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    if (blockIdx.x == 0) {
        const float* x = a.lat + (size_t)m * a.Rp;
        const float inv = row_inv_rms(x, a.Rp, a.R, a.eps, &red[0][0]);
        KT* dst = (KT*)a.cache + ((size_t)r.slot * a.T + r.pos) * a.Rp;
        for (int i = tid; i < a.Rp / 4; i += 256) {
            const float4 v = reinterpret_cast<const float4*>(x)[i], w = reinterpret_cast<const float4*>(a.lnorm)[i];
            store4(dst + 4 * i, make_float4(v.x * inv * w.x, v.y * inv * w.y, v.z * inv * w.z, v.w * inv * w.w));
        }
        return;
    }
    const int nch = (a.Rp + kLatCols - 1) / kLatCols, b = blockIdx.x - 1, h = b / nch, c0 = (b - h * nch) * kLatCols;
    const int g = tid / LPR, l = tid - g * LPR, col = c0 + l * VE;
    float acc[VE];
#pragma unroll
    for (int e = 0; e < VE; ++e) acc[e] = 0.0f;
    if (col < a.Rp) {
        const WT* w = (const WT*)a.uk + (size_t)h * a.dim * a.Rp + col;
        const float* q = a.q + ((size_t)m * a.H + h) * a.dim;
#pragma unroll 8
        for (int d = g; d < a.dim; d += NG) {
            float f[VE];
            Vec16<WT>::unpack(load16<false>(w + (size_t)d * a.Rp), f);
            const float qd = q[d];
#pragma unroll
            for (int e = 0; e < VE; ++e) acc[e] = fmaf(f[e], qd, acc[e]);
        }
    }
#pragma unroll
    for (int e = 0; e < VE; ++e) red[g][l * VE + e] = acc[e];
    __syncthreads();
    if (tid < kLatCols && c0 + tid < a.Rp) {
        float s = 0.0f;
#pragma unroll
        for (int j = 0; j < NG; ++j) s += red[j][tid];
        a.qa[((size_t)m * a.H + h) * a.Rp + c0 + tid] = s;
    }
}

// ---------------------------------------------------------------- decode attention on the matrix cores (fp16 cache)
// Grid (splits, head groups of 16, rows), 4 waves. A tile is 64 cache rows in LDS, read once for both products:
//   * S[key][head] = C Q^T: wave w owns keys 16 w .. + 15; A = rows of C, B = the group's absorbed queries as fp16
//     hi + lo fragments in LDS (shared by the waves);
//   * the tile's maximum per head through LDS, then P as hi + lo, written as the B fragments of the second product: a
//     lane's 4 accumulator rows are 4 of the 8 keys of its fragment;
//   * O[r][head] += C^T P^T: wave w owns columns r in [16 NB w, 16 NB (w + 1)), C^T by ds_read_b64_tr_b16.
// 16-byte chunks of a row are XOR-swizzled so that the row reads (16 rows, one chunk) and the transposed reads (8 rows,
// two chunks) both touch every bank once.
template <int NB>
struct LatGeo {
    static constexpr int RP = 64 * NB, ROWB = 2 * RP, CPR = ROWB / 16, STEPS = RP / 32;
    static constexpr int TILE = kLatKeys * ROWB, PIECES = TILE / 1024 / 4;  // LDS-DMA instructions per wave
    static constexpr int NBUF = NB <= 4 ? 2 : 1;
    static constexpr int QB = STEPS * 1024;                                // one of hi, lo
    static constexpr int OFF_Q = NBUF * TILE, OFF_P = OFF_Q + 2 * QB, OFF_M = OFF_P + 4096;
    static constexpr int LDS = OFF_M + 4 * 16 * 4;
    static_assert(LDS <= 160 * 1024, "LDS");
};
template <int NB>
__device__ __forceinline__ int lat_swz(int row) {
    const int r = row & 15;
    return NB % 2 == 0 ? ((r & 7) << 1) | (r >> 3) : (((r >> 1) & 3) << 1) | (r >> 3);
}
// the transposed reads of N (at most 4) tiles landed: their registers are named in the wait, so nothing that uses them
// moves above it
template <int N>
__device__ __forceinline__ void lat_wait_tr(uint2 (&x)[N], uint2 (&y)[N]) {
    static_assert(N >= 1 && N <= 4, "tiles per wait");
    if constexpr (N == 1)
        asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(x[0]), "+v"(y[0])::"memory");
    else if constexpr (N == 2)
        asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(x[0]), "+v"(x[1]), "+v"(y[0]), "+v"(y[1])::"memory");
    else if constexpr (N == 3)
        asm volatile("s_waitcnt lgkmcnt(0)"
                     : "+v"(x[0]), "+v"(x[1]), "+v"(x[2]), "+v"(y[0]), "+v"(y[1]), "+v"(y[2])::"memory");
    else
        asm volatile("s_waitcnt lgkmcnt(0)"
                     : "+v"(x[0]), "+v"(x[1]), "+v"(x[2]), "+v"(x[3]), "+v"(y[0]), "+v"(y[1]), "+v"(y[2]),
                       "+v"(y[3])::"memory");
}

template <int NB>
__global__ void __launch_bounds__(256) lat_attn_kernel(LatArgs a) {
    using G = LatGeo<NB>;
    extern __shared__ __attribute__((aligned(1024))) char la_sm[];
    const int m = blockIdx.z, split = blockIdx.x, h0 = blockIdx.y * kLatHeads;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    const LatSpan sp = lat_span(r.pos, a.window, a.splits);
    if (split >= sp.ns) return;  // (uniform)
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int g = lane >> 4, i16 = lane & 15;
    const int t_end = min(sp.nt, (split + 1) * sp.per);
    const __half* cache = (const __half*)a.cache + (size_t)r.slot * a.T * G::RP;
    const unsigned base = (unsigned)(uintptr_t)(const __attribute__((address_space(3))) char*)la_sm;
    u32x4* qf = reinterpret_cast<u32x4*>(la_sm + G::OFF_Q);
    float* wm = reinterpret_cast<float*>(la_sm + G::OFF_M);  // [4 waves][16 heads]

    auto issue = [&](int t) {
        const int k0 = sp.lo + t * kLatKeys;
        const unsigned dst = base + (unsigned)((t % G::NBUF) * G::TILE);
#pragma unroll
        for (int j = 0; j < G::PIECES; ++j) {
            const int p = wave * G::PIECES + j, f = p * 64 + lane, row = f / G::CPR, c = (f - row * G::CPR) ^ lat_swz<NB>(row);
            am_dma<true>(cache + (size_t)min(k0 + row, r.pos) * G::RP + c * 8, dst + (unsigned)(p * 1024));
        }
    };
    // the group's queries as B fragments: step s, lane l holds head l & 15, values 32 s + 8 (l >> 4) .. + 7
    constexpr int QPT = (G::STEPS * 64 + 255) / 256;
    float4 qv[QPT][2];
#pragma unroll
    for (int j = 0; j < QPT; ++j) {
        const int f = min(tid + 256 * j, G::STEPS * 64 - 1), s = f >> 6, l = f & 63, h = min(h0 + (l & 15), a.H - 1);
        const float4* qp = reinterpret_cast<const float4*>(a.qa + ((size_t)m * a.H + h) * G::RP + 32 * s + 8 * (l >> 4));
        qv[j][0] = qp[0], qv[j][1] = qp[1];
    }
    issue(split * sp.per);
#pragma unroll
    for (int j = 0; j < QPT; ++j) {
        const int f = tid + 256 * j;
        if (f >= G::STEPS * 64) break;
        const bool live = h0 + (f & 15) < a.H;
        const float v[8] = {qv[j][0].x, qv[j][0].y, qv[j][0].z, qv[j][0].w, qv[j][1].x, qv[j][1].y, qv[j][1].z, qv[j][1].w};
        __half hi[8], lo[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) pf_split(live ? v[e] : 0.0f, hi[e], lo[e]);
        qf[f] = *reinterpret_cast<const u32x4*>(hi);
        qf[G::STEPS * 64 + f] = *reinterpret_cast<const u32x4*>(lo);
    }
    am_float4 o[NB];
#pragma unroll
    for (int t = 0; t < NB; ++t) o[t] = am_float4{0.0f, 0.0f, 0.0f, 0.0f};
    float mx = -INFINITY, l = 0.0f;
    const int kr = wave * 16 + i16, ksw = lat_swz<NB>(kr);
    for (int t = split * sp.per; t < t_end; ++t) {
        if (G::NBUF == 1 && t > split * sp.per) {
            __syncthreads();  // every wave is done with the tile before
            issue(t);
        }
        am_wait_vm<0>();
        __syncthreads();  // the tile (and, first, the query fragments) landed; the other buffer is free
        if (G::NBUF == 2 && t + 1 < t_end) issue(t + 1);
        const int boff = (t % G::NBUF) * G::TILE;
        const char* krow = la_sm + boff + kr * G::ROWB;
        am_float4 sh = am_float4{0.0f, 0.0f, 0.0f, 0.0f}, sl = sh;
#pragma unroll
        for (int s = 0; s < G::STEPS; ++s) {
            const u32x4 kf = *reinterpret_cast<const u32x4*>(krow + ((4 * s + g) ^ ksw) * 16);
            sh = am_mfma(kf, qf[s * 64 + lane], sh);
            sl = am_mfma(kf, qf[(G::STEPS + s) * 64 + lane], sl);
        }
        // this lane: keys 16 wave + 4 g + e of head i16
        float sv[4], cmax = -INFINITY;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int key = sp.lo + t * kLatKeys + wave * 16 + 4 * g + e;
            sv[e] = key <= r.pos ? (sh[e] + sl[e]) * a.scale : -INFINITY;
            cmax = fmaxf(cmax, sv[e]);
        }
        cmax = fmaxf(cmax, __shfl_xor(cmax, 16));
        cmax = fmaxf(cmax, __shfl_xor(cmax, 32));
        if (lane < 16) wm[wave * 16 + lane] = cmax;
        __syncthreads();
        const float mn = fmaxf(fmaxf(fmaxf(wm[i16], wm[16 + i16]), fmaxf(wm[32 + i16], wm[48 + i16])), mx);
        const float corr = expf(mx - mn);  // (a tile holds at least one visible key: mn is finite)
        mx = mn;
        __half ph[4], pl[4];
        l *= corr;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float p = expf(sv[e] - mn);
            l += p;
            pf_split(p, ph[e], pl[e]);
        }
        char* pf = la_sm + G::OFF_P + ((wave >> 1) * 64 + lane) * 16 + (wave & 1) * 8;
        *reinterpret_cast<uint2*>(pf) = *reinterpret_cast<const uint2*>(ph);
        *reinterpret_cast<uint2*>(pf + 2048) = *reinterpret_cast<const uint2*>(pl);
        __syncthreads();
#pragma unroll
        for (int n = 0; n < NB; ++n) o[n] *= corr;
        const int q4 = i16 >> 2, p4 = lane & 3;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {  // 32 keys: k order {4 g .. + 3, 16 + 4 g .. + 3} of the block
            const u32x4 bh = *reinterpret_cast<const u32x4*>(la_sm + G::OFF_P + (kb * 64 + lane) * 16);
            const u32x4 bl = *reinterpret_cast<const u32x4*>(la_sm + G::OFF_P + 2048 + (kb * 64 + lane) * 16);
            const int r1 = kb * 32 + 4 * g + q4, sw = lat_swz<NB>(r1);
            const unsigned a1 = base + boff + r1 * G::ROWB + 8 * (p4 & 1), a2 = a1 + 16 * G::ROWB;
            auto tiles = [&](auto cnt, int n0) {
                constexpr int N = decltype(cnt)::value;
                uint2 x[N], y[N];
#pragma unroll
                for (int n = 0; n < N; ++n) {
                    const int c = (2 * (wave * NB + n0 + n) + (p4 >> 1)) ^ sw;
                    x[n] = am_tr_read(a1 + c * 16);
                    y[n] = am_tr_read(a2 + c * 16);
                }
                lat_wait_tr<N>(x, y);
#pragma unroll
                for (int n = 0; n < N; ++n) {
                    const u32x4 vf = u32x4{x[n].x, x[n].y, y[n].x, y[n].y};
                    o[n0 + n] = am_mfma(vf, bh, o[n0 + n]);
                    o[n0 + n] = am_mfma(vf, bl, o[n0 + n]);
                }
            };
            tiles(std::integral_constant<int, (NB < 4 ? NB : 4)>{}, 0);
            if constexpr (NB > 4) tiles(std::integral_constant<int, NB - 4>{}, 4);
        }
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    __syncthreads();  // (the maxima of the last tile were read)
    if (lane < 16) wm[wave * 16 + lane] = l;
    __syncthreads();
    if (h0 + i16 >= a.H) return;
    float* dst = a.part + (((size_t)m * a.H + h0 + i16) * a.splits + split) * (G::RP + kAttnPartPad);
#pragma unroll
    for (int n = 0; n < NB; ++n)
        *reinterpret_cast<float4*>(dst + 16 * (wave * NB + n) + 4 * g) = make_float4(o[n][0], o[n][1], o[n][2], o[n][3]);
    if (wave == 0 && g == 0) {
        dst[G::RP] = mx;
        dst[G::RP + 1] = wm[i16] + wm[16 + i16] + wm[32 + i16] + wm[48 + i16];
    }
}

// ---------------------------------------------------------------- the form for every shape and precision
// One workgroup per (head, row): 64 keys at a time, one wave per key and dot product. Writes its result as one split.
inline size_t lat_rows_lds(int Rp) { return sizeof(float) * (size_t)(Rp + 128); }
template <typename KT>
__global__ void __launch_bounds__(256) lat_attn_rows_kernel(LatArgs a) {
    extern __shared__ float lr_sm[];
    float *qs = lr_sm, *ss = lr_sm + a.Rp, *ps = ss + 64;
    const int h = blockIdx.x, m = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    const KT* c = (const KT*)a.cache + (size_t)r.slot * a.T * a.Rp;
    for (int i = tid; i < a.Rp; i += 256) qs[i] = a.qa[((size_t)m * a.H + h) * a.Rp + i];
    constexpr int NV = kLatMaxRank / 256;
    float o[NV], mx = -INFINITY, l = 0.0f;
#pragma unroll
    for (int i = 0; i < NV; ++i) o[i] = 0.0f;
    for (int t0 = max(0, r.pos - a.window + 1); t0 <= r.pos; t0 += 64) {
        __syncthreads();
        for (int j = wave; j < 64; j += 4) {
            const int t = t0 + j;
            float d = 0.0f;
            if (t <= r.pos)
                for (int i = lane; i < a.Rp; i += 64) d = fmaf(qs[i], to_f32(c[(size_t)t * a.Rp + i]), d);
            d = wave_sum(d);
            if (lane == 0) ss[j] = t <= r.pos ? d * a.scale : -INFINITY;
        }
        __syncthreads();
        const float s = ss[lane], mn = fmaxf(mx, wave_max(s)), corr = expf(mx - mn), p = expf(s - mn);
        l = l * corr + wave_sum(p);
        mx = mn;
        if (wave == 0) ps[lane] = p;
        __syncthreads();
        const int n = min(64, r.pos - t0 + 1);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int d = tid + 256 * i;
            if (d >= a.Rp) break;
            float acc = o[i] * corr;
            for (int j = 0; j < n; ++j) acc = fmaf(ps[j], to_f32(c[(size_t)(t0 + j) * a.Rp + d]), acc);
            o[i] = acc;
        }
    }
    float* dst = a.part + ((size_t)m * a.H + h) * (a.Rp + kAttnPartPad);
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if (tid + 256 * i < a.Rp) dst[tid + 256 * i] = o[i];
    if (tid == 0) {
        dst[a.Rp] = mx;
        dst[a.Rp + 1] = l;
    }
}

// The splits merged, U_v applied, the gate: out[m][h * vdim + v]. Grid (value rows / 32, H, M): a wave owns 8 value rows
// (their first 16 bytes per lane in flight before the merge). The merge: thread groups of Rp / 4 threads take every ng-th
// split, kLatMerge loads of each in flight; lane s has split s's maximum and sum.
constexpr int kLatMerge = 8;
inline size_t lat_out_lds(int Rp) { return sizeof(float) * (size_t)std::max(Rp, 1024); }
template <typename WT, typename OT>
__global__ void __launch_bounds__(256) lat_out_kernel(LatArgs a, OT* out, int ldo) {
    extern __shared__ __attribute__((aligned(16))) float lo_sm[];  // [ng][Rp]
    __shared__ float se[kLatMaxSplits];
    constexpr int VE = Vec16<WT>::N, NR = kLatOutRows / 4;
    const int h = blockIdx.y, m = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const RowRef r = a.rows[m];
    if (r.slot < 0) return;
    const int v0 = blockIdx.x * kLatOutRows + wave * NR, nvec = a.Rp / VE;
    const WT* w = (const WT*)a.uv + (size_t)h * a.vdim * a.Rp;
    const int ns = lat_span(r.pos, a.window, a.splits).ns, ps = a.Rp + kAttnPartPad;
    const float* p = a.part + ((size_t)m * a.H + h) * a.splits * ps;
    const int n4 = a.Rp / 4, ng = max(1, 256 / n4), grp = n4 > 256 ? 0 : tid / n4, c0 = tid - grp * n4;
    float4 v[kLatMerge];
    auto load = [&](int s0, int c) {
#pragma unroll
        for (int j = 0; j < kLatMerge; ++j)
            v[j] = *reinterpret_cast<const float4*>(p + (size_t)min(s0 + j * ng, ns - 1) * ps + 4 * min(c, n4 - 1));
    };
    const float ms = p[(size_t)min(lane, ns - 1) * ps + a.Rp], ls = p[(size_t)min(lane, ns - 1) * ps + a.Rp + 1];
    load(grp, c0);
    u32x4 wf[NR];
#pragma unroll
    for (int j = 0; j < NR; ++j)
        wf[j] = load16<false>(w + (size_t)min(v0 + j, a.vdim - 1) * a.Rp + min(lane, nvec - 1) * VE);
    const float M = wave_max(ms), e = lane < ns ? expf(ms - M) : 0.0f, L = wave_sum(e * ls);
    if (wave == 0 && lane < kLatMaxSplits) se[lane] = e / L;  // 0 past the last split
    __syncthreads();
    if (grp < ng)
        for (int c = c0; c < n4; c += 256) {
            if (c != c0) load(grp, c);
            float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
            for (int s0 = grp; s0 < ns; s0 += ng * kLatMerge) {
                if (s0 != grp) load(s0, c);
#pragma unroll
                for (int j = 0; j < kLatMerge; ++j) {
                    const int s = s0 + j * ng;
                    const float es = s < kLatMaxSplits ? se[s] : 0.0f;
                    o = fma4(v[j], make_float4(es, es, es, es), o);
                }
            }
            reinterpret_cast<float4*>(lo_sm)[grp * n4 + c] = o;
        }
    __syncthreads();
    if (ng > 1) {
        for (int c = tid; c < n4; c += 256) {
            float4 o = reinterpret_cast<const float4*>(lo_sm)[c];
            for (int g = 1; g < ng; ++g) o = fma4(reinterpret_cast<const float4*>(lo_sm)[g * n4 + c], make_float4(1.f, 1.f, 1.f, 1.f), o);
            reinterpret_cast<float4*>(lo_sm)[c] = o;
        }
        __syncthreads();
    }
#pragma unroll
    for (int j = 0; j < NR; ++j) {
        if (v0 + j >= a.vdim) break;  // (uniform in the wave)
        float s = 0.0f;
        for (int c = lane; c < nvec; c += 64) {
            float f[VE];
            Vec16<WT>::unpack(c == lane ? wf[j] : load16<false>(w + (size_t)(v0 + j) * a.Rp + c * VE), f);
#pragma unroll
            for (int e = 0; e < VE; ++e) s = fmaf(f[e], lo_sm[c * VE + e], s);
        }
        s = wave_sum(s);
        const size_t at = (size_t)m * a.H * a.vdim + (size_t)h * a.vdim + v0 + j;
        if (lane == 0) out[(size_t)m * ldo + (size_t)h * a.vdim + v0 + j] = from_f32<OT>(s * a.gate[at]);
    }
}

// ---------------------------------------------------------------- prompts: the expansion's layout
// For one window, the portions of a pass: portion s needs cache rows lo_s .. pos0_s + n_s - 1, lo_s = max(0, pos0_s -
// window + 1), in tiles of kLatTile rows, one portion after the other. tiles[i] = {0, first cache row}; koff[g]: of the
// pass's rows 32 g .. + 31, what turns a position into a scratch row.
static __global__ void __launch_bounds__(1024) lat_tiles_kernel(const SegRef* segs, const int32_t* nsegs, int T, int window,
                                                         int2* tiles, int32_t* ntiles, int32_t* koff) {
    const int n = *nsegs;
    int at = 0;
    for (int s = 0; s < n; ++s) {  // (uniform: every thread walks the portions)
        const SegRef g = segs[s];
        const int lo = max(0, g.pos0 - window + 1), nt = (g.pos0 + g.n - lo + kLatTile - 1) / kLatTile;
        for (int i = threadIdx.x; i < nt; i += 1024) tiles[at + i] = make_int2(0, g.slot * T + lo + i * kLatTile);
        for (int i = threadIdx.x; i < (g.n + 31) / 32; i += 1024) koff[g.row0 / 32 + i] = at * kLatTile - lo;
        at += nt;
    }
    if (threadIdx.x == 0) *ntiles = at;
}
inline int lat_tiles(int pos0, int n, int window) {
    const int lo = pos0 - window + 1 > 0 ? pos0 - window + 1 : 0;
    return (pos0 + n - lo + kLatTile - 1) / kLatTile;
}

// The expansion's epilogue: fused rows [U_k (padded to 4 rows) ; U_v] at scratch row m -> K, V [heads][cap][hd]
struct LatExpand {
    __half *k, *v;
    int Hq, dim, Hv, vdim, v0, cap, hd;  // v0: first U_v row
    __device__ void put(int row, int m, float x) const {
        const bool isv = row >= v0;
        const int i = isv ? row - v0 : row, n = isv ? vdim : dim;
        if (i >= (isv ? Hv : Hq)) return;
        const int h = i / n;
        (isv ? v : k)[((size_t)h * cap + m) * hd + i - h * n] = __float2half_rn(x);
    }
    __device__ void pair(int u, int m, float a0, float a1) const {
        put(2 * u, m, a0);
        put(2 * u + 1, m, a1);
    }
    __device__ void pair2(int u, int m, const float* a, bool second) const {  // u even
        const int row = 2 * u;
        const bool isv = row >= v0;
        const int i = isv ? row - v0 : row, n = isv ? vdim : dim;
        if (n % 4 == 0 && i + 3 < (isv ? Hv : Hq)) {
            const int h = i / n;
            store4((isv ? v : k) + ((size_t)h * cap + m) * hd + i - h * n, make_float4(a[0], a[1], a[2], a[3]));
            return;
        }
        pair(u, m, a[0], a[1]);
        if (second) pair(u + 1, m, a[2], a[3]);
    }
};

}  // namespace sli
