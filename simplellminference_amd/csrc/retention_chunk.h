// retention_chunk.h — retention of a prompt portion on the matrix cores, kRcTok tokens at a time (retention.h):
//   o_i = decay^(i+1) S^T q_i + sum_(j <= i) decay^(i-j) (q_i . k_j) v_j          (i, j inside the chunk)
//   S  <- decay^n S + sum_j decay^(n-1-j) k_j v_j^T                               (n tokens in the chunk)
// A workgroup of 4 waves owns one (portion, head, kRetCols value columns) and walks the portion's chunks. The state
// slice stays in fp32 accumulators (C tiles of the update's own MFMAs) from the first chunk to the last, so it is never
// rounded; where it is an operand (S^T q) it is carried as fp16 hi + lo, like the decayed scores and the decayed values.
// q, k and v enter as fp16. Operands reach their MFMA layouts through LDS; the next chunk's rows are loaded while the
// current one is computed.
#pragma once
#include "prefill.h"
#include "retention.h"

namespace sli {

constexpr int kRcTok = 32;

template <int KD>  // dim padded to a multiple of 32
struct RcGeo {
    static constexpr int QS = KD + 8, TS = kRcTok + 8;  // LDS row strides in halves (16-byte aligned, spread over banks)
    static constexpr int Q = 0, K = Q + kRcTok * QS, KT = K + kRcTok * QS, VT = KT + KD * TS,
                         VD = VT + kRetCols * TS, VDL = VD + kRetCols * TS, ST = VDL + kRetCols * TS, STL = ST + kRetCols * QS, P = STL + kRetCols * QS, PL = P + kRcTok * TS,
                         END = PL + kRcTok * TS;
    static constexpr size_t LDS = (size_t)END * 2 + 4 * 64;  // + decay powers
    static constexpr int NT = KD / 16;                     // 16-row state tiles (x 2 column tiles)
    static constexpr int TPW = (NT * 2 + 3) / 4;           // state tiles per wave
    static constexpr int VEC = kRcTok * KD / 4 / 256;      // float4 of q (and of k) per thread per chunk
    // piece i of thread tid: token and first dim (tokens 2p, 2p + 1 of one dim group are pieces of one thread: their
    // transposed copies are one 4-byte store)
    static constexpr int TOKS = VEC >= 2 ? 2 : 1;
    __device__ static void piece(int i, int tid, int& t, int& d) {
        const int e = (i / TOKS) * 256 + tid;
        t = TOKS * (e / (KD / 4)) + i % TOKS;
        d = 4 * (e % (KD / 4));
    }
    // K^T: the 8-token blocks of row d permuted by d / 16, so that the lanes of a transposed store spread over the banks
    __device__ static int kt(int d, int t) { return KT + d * TS + ((t >> 3) ^ ((d >> 4) & 3)) * 8 + (t & 7); }
};

template <int KD>
__global__ void __launch_bounds__(256) ret_chunk_kernel(RetArgs a) {
    using G = RcGeo<KD>;
    extern __shared__ __attribute__((aligned(16))) char rc_sm[];
    __half* sm = reinterpret_cast<__half*>(rc_sm);
    float* pw = reinterpret_cast<float*>(rc_sm + (size_t)G::END * 2);  // decay^0 .. decay^kRcTok
    if ((int)blockIdx.z >= *a.nsegs) return;
    const SegRef sg = a.segs[blockIdx.z];
    const int sl = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int g = lane >> 4, i16 = lane & 15;
    const float dec = a.decay[h];
    if (tid <= kRcTok) {
        double p = 1.0;
        for (int i = 0; i < tid; ++i) p *= (double)dec;
        pw[tid] = (float)p;
    }
    // the state tiles of this wave: index t = wave * TPW + i -> rows 16 (t / 2), columns 16 (t % 2); lane holds rows
    // 4 g .. + 3 of column i16
    float* S = ret_slice(a, sg.slot, h, sl);
    pf_float4 st[G::TPW];
#pragma unroll
    for (int i = 0; i < G::TPW; ++i) {
        const int t = wave * G::TPW + i, r0 = 16 * (t / 2) + 4 * g, c = 16 * (t % 2) + i16;
#pragma unroll
        for (int r = 0; r < 4; ++r)
            st[i][r] = (sg.pos0 > 0 && t < 2 * G::NT && r0 + r < a.dim) ? S[(size_t)(r0 + r) * kRetCols + c] : 0.0f;
    }
    // this chunk's rows in registers: q, k as float4 groups, v one element per (token, column) pair
    constexpr int NV = kRcTok * kRetCols / 256;
    float4 qr[G::VEC], kr[G::VEC];
    float vr[NV];
    auto load = [&](int c0) {
        const bool al = a.dim % 4 == 0;
#pragma unroll
        for (int i = 0; i < G::VEC; ++i) {
            int t, d;
            G::piece(i, tid, t, d);
            const bool ok = c0 + t < sg.n;
            const size_t row = ((size_t)(sg.row0 + c0 + (ok ? t : 0)) * a.H + h) * a.dim;
            if (al) {
                const bool in = ok && d < a.dim;
                qr[i] = in ? *reinterpret_cast<const float4*>(a.q + row + d) : make_float4(0.f, 0.f, 0.f, 0.f);
                kr[i] = in ? *reinterpret_cast<const float4*>(a.k + row + d) : make_float4(0.f, 0.f, 0.f, 0.f);
            } else {
                float f[4], w[4];
#pragma unroll
                for (int x = 0; x < 4; ++x) {
                    const bool in = ok && d + x < a.dim;
                    f[x] = in ? a.q[row + d + x] : 0.0f;
                    w[x] = in ? a.k[row + d + x] : 0.0f;
                }
                qr[i] = make_float4(f[0], f[1], f[2], f[3]);
                kr[i] = make_float4(w[0], w[1], w[2], w[3]);
            }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int e = i * 256 + tid, t = e / kRetCols, c = e % kRetCols, col = sl * kRetCols + c;
            const bool in = c0 + t < sg.n && col < a.vdim;
            vr[i] = in ? a.v[((size_t)(sg.row0 + c0 + t) * a.H + h) * a.vdim + col] : 0.0f;
        }
    };
    load(0);
    for (int c0 = 0; c0 < sg.n; c0 += kRcTok) {
        const int n = min(kRcTok, sg.n - c0);
        __syncthreads();  // the previous chunk's LDS reads are done (first chunk: pw is there)
#pragma unroll
        for (int i = 0; i < G::VEC; ++i) {
            int t, d;
            G::piece(i, tid, t, d);
            store4(sm + G::Q + t * G::QS + d, qr[i]);
            store4(sm + G::K + t * G::QS + d, kr[i]);
        }
#pragma unroll
        for (int i = 0; i < G::VEC; i += G::TOKS) {
            int t, d;
            G::piece(i, tid, t, d);
            const float f[4] = {kr[i].x, kr[i].y, kr[i].z, kr[i].w};
            const float4& k1 = kr[i + G::TOKS - 1];
            const float f1[4] = {k1.x, k1.y, k1.z, k1.w};
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                if constexpr (G::TOKS == 2)
                    *reinterpret_cast<__half2*>(sm + G::kt(d + x, t)) = __halves2half2(__float2half_rn(f[x]), __float2half_rn(f1[x]));
                else
                    sm[G::kt(d + x, t)] = __float2half_rn(f[x]);
            }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int e = i * 256 + tid, t = e / kRetCols, c = e % kRetCols;
            sm[G::VT + c * G::TS + t] = __float2half_rn(vr[i]);
            __half hi, lo;
            pf_split(vr[i] * pw[max(n - 1 - t, 0)], hi, lo);  // (rows past the portion are zero)
            sm[G::VD + c * G::TS + t] = hi;
            sm[G::VDL + c * G::TS + t] = lo;
        }
        // the state before this chunk, as the S^T q operand [column][row]
#pragma unroll
        for (int i = 0; i < G::TPW; ++i) {
            const int t = wave * G::TPW + i, r0 = 16 * (t / 2) + 4 * g, c = 16 * (t % 2) + i16;
            if (t < 2 * G::NT) {
                __half hi[4], lo[4];
#pragma unroll
                for (int r = 0; r < 4; ++r) pf_split(st[i][r], hi[r], lo[r]);
                *reinterpret_cast<uint2*>(sm + G::ST + c * G::QS + r0) = *reinterpret_cast<const uint2*>(hi);
                *reinterpret_cast<uint2*>(sm + G::STL + c * G::QS + r0) = *reinterpret_cast<const uint2*>(lo);
            }
        }
        __syncthreads();
        if (c0 + kRcTok < sg.n) load(c0 + kRcTok);
        // wave w: rows 16 (w / 2) of the chunk, key tile (scores) and column tile (output) w % 2
        const int rt = wave >> 1, ct = wave & 1;
        auto frag = [&](int base, int row, int stride, int kb) {
            return *reinterpret_cast<const u32x4*>(sm + base + row * stride + 32 * kb + 8 * g);
        };
        pf_float4 sc = {0.f, 0.f, 0.f, 0.f}, oi = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < KD / 32; ++kb) {
            const u32x4 q = frag(G::Q, rt * 16 + i16, G::QS, kb);
            sc = pf_mfma(q, frag(G::K, ct * 16 + i16, G::QS, kb), sc);
            oi = pf_mfma(q, frag(G::ST, ct * 16 + i16, G::QS, kb), oi);
            oi = pf_mfma(q, frag(G::STL, ct * 16 + i16, G::QS, kb), oi);
        }
        // lane holds rows i = 16 rt + 4 g + r, column (key j / value column) 16 ct + i16
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = rt * 16 + 4 * g + r, j = ct * 16 + i16;
            __half hi, lo;
            pf_split(j <= i ? sc[r] * pw[max(i - j, 0)] : 0.0f, hi, lo);
            sm[G::P + i * G::TS + j] = hi;
            sm[G::PL + i * G::TS + j] = lo;
            oi[r] *= pw[i + 1];
        }
        // the state update needs no scores
        const float dn = pw[n];
#pragma unroll
        for (int i = 0; i < G::TPW; ++i) {
            const int t = wave * G::TPW + i;
            if (t < 2 * G::NT) {
                st[i] *= dn;
                const u32x4 kt = *reinterpret_cast<const u32x4*>(sm + G::kt((t / 2) * 16 + i16, 8 * g));
                st[i] = pf_mfma(kt, frag(G::VD, (t % 2) * 16 + i16, G::TS, 0), st[i]);
                st[i] = pf_mfma(kt, frag(G::VDL, (t % 2) * 16 + i16, G::TS, 0), st[i]);
            }
        }
        __syncthreads();
        const u32x4 v = frag(G::VT, ct * 16 + i16, G::TS, 0);
        oi = pf_mfma(frag(G::P, rt * 16 + i16, G::TS, 0), v, oi);
        oi = pf_mfma(frag(G::PL, rt * 16 + i16, G::TS, 0), v, oi);
        const int col = sl * kRetCols + ct * 16 + i16;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = rt * 16 + 4 * g + r;
            if (i < n && col < a.vdim) a.o[((size_t)(sg.row0 + c0 + i) * a.H + h) * a.vdim + col] = oi[r];
        }
    }
#pragma unroll
    for (int i = 0; i < G::TPW; ++i) {
        const int t = wave * G::TPW + i, r0 = 16 * (t / 2) + 4 * g, c = 16 * (t % 2) + i16;
        if (t < 2 * G::NT)
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (r0 + r < a.dim) S[(size_t)(r0 + r) * kRetCols + c] = st[i][r];
    }
}

// (KD: dim rounded up to one of 32, 64, 128, 256; 0: the scan form takes it)
inline int ret_chunk_kd(int dim) { return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : dim <= 256 ? 256 : 0; }

}  // namespace sli
