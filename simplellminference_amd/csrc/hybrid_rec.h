// hybrid_rec.h — recording a projection over M rows for block-stack models (hybrid.h): which kernel runs it, by the row
// count and the element type. Base of the recorders of the two arrangements.
#pragma once
#include <type_traits>

#include "hybrid_kernels.h"
#include "hybrid_stack.h"

namespace sli {

template <typename WT>
struct HyProj {
    BlockStack* s;
    int M;      // rows of the launches
    bool one;   // one row per sequence (decode)
    int msegs;  // portions at most
    int key_tiles = 0;  // sequential arrangement: expansion tiles at most
    hipStream_t st() const { return s->stream; }

    // How a projection over M rows runs: the batch-1 GEMV, the batched MFMA projection (fp16, 2 .. 8 rows; one row past
    // the GEMV's LDS stage), the prompt GEMM (fp16, more rows), or the plain kernel (fp32, more rows or wider).
    enum Path { GV, BG, PG, RG };
    static constexpr bool F16 = std::is_same<WT, __half>::value;
    static Path path(int M, int K) {
        if (M == 1 && K <= kGemvMaxCols) return GV;
        if (!F16) return RG;
        return M <= kBgMaxBatch ? BG : PG;
    }
    // rows of the launches for n rows
    static int rows_for(int n) { return F16 && n > kBgMaxBatch ? pad_to(n, kHyTile) : n; }

    template <class Epi>
    int project(const void* W, const void* X, int K, int npairs, int u0, const Epi& e) const {
        const WT* w = (const WT*)W + (size_t)2 * u0 * K;
        const Path p = path(M, K);
        if (p == GV) {
            GemvIn in{(const float*)X, nullptr, 0.0f, K};
            SLI_HIP((launch_gemv_u<WT, 2, 4, true>(w, in, GvPair<Epi>{e, npairs, u0}, npairs, st())));
            return SLI_OK;
        }
        if constexpr (F16) {
            if (p == BG) {
                BgIn in{};
                in.x = (const float*)X;
                in.K = K;
                in.B = M;
                in.ws = s->bg_ws;
                in.counters = s->bg_cnt;
                const BgPlan pl = bg_plan((npairs + 7) / 8, K, M, false, gemv_max_blocks(), true);
                SLI_HIP((launch_bgemm(w, in, BgPair<Epi>{e, npairs, u0}, pl, st())));
                return SLI_OK;
            }
            if (p == PG) return pgemm(w, (const __half*)X, nullptr, 0, K, npairs, u0, e);
        }
        SLI_HIP((launch_rows_gemm<WT, Epi>(w, (const float*)X, K, npairs, u0, M, e, st())));
        return SLI_OK;
    }
    // pairs [0, split) read X, pairs [split, npairs) X2 (split: a multiple of kHySection; X2 null: one input)
    template <class Epi>
    int pgemm(const WT* w, const __half* X, const __half* X2, int split, int K, int npairs, int u0, const Epi& e) const {
        if constexpr (F16) {
            PgIn<__half> in{w, X, nullptr, pad_to(2 * npairs, 16), K, M};
            if (X2) in.Bhi2 = X2, in.row_b2 = 2 * split;
            return pg_pick(M, in.N, [&](auto cfg) -> int {
                SLI_HIP((launch_pgemm<PgPair<Epi>, decltype(cfg), __half>(in, PgPair<Epi>{e, npairs, u0}, nullptr, st())));
                return SLI_OK;
            });
        } else {
            return fail(SLI_ERR_ARG, "prompt GEMM: fp16 weights");
        }
    }
    // Tilings (their row count divides M) by rows and output tiles, the fastest of a sweep at 4096 x 15104 and 34304 x 4096 with the weights streamed
    // from HBM (TFLOP/s at 1024 rows 794 and 814, at 512 591 and 658, at 256 296 and 579): one 256 x 256 tile per CU
    // where the grid fills the chip with them, smaller tiles (a full grid) where the output is narrow.
    template <class F>
    static int pg_pick(int M, int N, F&& f) {
        const long long t128 = (long long)((N + 127) / 128) * (M / 128);
        if (M % 256 == 0 && M != 512 && t128 >= 512) return f(PgCfg<256, 4, 2, 4, true, 0, 1>{});
        if (M % 128 == 0 && M >= 512 && t128 >= 512) return f(PgCfg<128, 4, 2, 2, true, 0, 1>{});
        if (M % 128 == 0 && t128 >= 256) return f(PgCfg<128, 2, 3, 4, true, 0, 1>{});
        if (M % 64 == 0 && M >= 128) return f(PgCfg<64, 4, 4, 2, true, 0, 1>{});
        if (M % 64 == 0) return f(PgCfg<64, 2, 4, 2, true, 0, 1>{});
        return f(PgCfg<32, 2, 4, 2, true, 0, 1>{});
    }
    template <class Epi>
    static int allow() {
        if constexpr (F16) {
            for (auto [M, N] : {std::make_pair(32, 128), {64, 128}, {128, 128}, {128, 1 << 15}, {256, 1 << 15}, {512, 1 << 15}})
                HY_TRY(pg_pick(M, N, [&](auto cfg) -> int {
                    SLI_HIP((pgemm_allow_lds<PgPair<Epi>, decltype(cfg), __half>()));
                    return SLI_OK;
                }));
            SLI_HIP((bg_allow_lds<BgPair<Epi>, false>()));
        }
        return SLI_OK;
    }

    // Row blocks with weights of their own (prefill.h PgGroups): X fp16 for fp16 weights, else fp32
    static constexpr int group_rows(int pairs_per_group) {
        return !F16 ? kRowsGemmTile : pairs_per_group >= 192 ? 128 : pairs_per_group >= 48 ? 64 : 32;
    }
    template <class Epi>
    int grouped(const void* W, const void* X, int K, int npairs, const PgGroups& g, int bm, int maxtiles, const Epi& e) const {
        if constexpr (F16) {
            PgIn<__half> in{(const __half*)W, (const __half*)X, nullptr, pad_to(2 * npairs, 16), K, maxtiles * bm};
            in.grp = g;
            return pg_group_pick(bm, [&](auto cfg) -> int {
                SLI_HIP((launch_pgemm<PgPair<Epi>, decltype(cfg), __half>(in, PgPair<Epi>{e, npairs, 0}, nullptr, st())));
                return SLI_OK;
            });
        } else {
            SLI_HIP((launch_rows_gemm_grouped<WT, Epi>((const WT*)W, (const float*)X, K, npairs, g, maxtiles, e, st())));
            return SLI_OK;
        }
    }
    template <class F>
    static int pg_group_pick(int bm, F&& f) {
        if (bm == 128) return f(PgCfg<128, 2, 3, 4, true, 0, 1, true>{});
        if (bm == 64) return f(PgCfg<64, 4, 4, 2, true, 0, 1, true>{});
        return f(PgCfg<32, 2, 4, 2, true, 0, 1, true>{});
    }
    template <class Epi>
    static int allow_grouped() {
        if constexpr (F16)
            for (int bm : {32, 64, 128})
                HY_TRY(pg_group_pick(bm, [&](auto cfg) -> int {
                    SLI_HIP((pgemm_allow_lds<PgPair<Epi>, decltype(cfg), __half>()));
                    return SLI_OK;
                }));
        return SLI_OK;
    }
};

}  // namespace sli
