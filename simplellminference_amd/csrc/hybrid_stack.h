// hybrid_stack.h — what the files of block-stack models (hybrid.h) share: the layers, runs and buffers of a stack, weight
// placement, and the entry points of the sequential arrangement (hybrid_seq.hip).
#pragma once
#include <hip/hip_fp16.h>

#include <algorithm>
#include <map>
#include <memory>
#include <string>
#include <utility>
#include <vector>

#include "hybrid.h"

namespace sli {

#define HY_TRY(expr)                   \
    do {                               \
        int rc_ = (expr);              \
        if (rc_ != SLI_OK) return rc_; \
    } while (0)

constexpr int kHyLogitRows = 256;  // wanted rows per pass of the output head
constexpr int kHySection = 128;  // pairs: a GEMM row block (at most 256 rows) never straddles the two inputs

inline int pad_to(int n, int m) { return (n + m - 1) / m * m; }

struct HyLayer {
    sli_block_desc d{};
    int mixw = 0, KA = 0, KF = 0, Kp = 0;  // output projection input: [mixer (KA) ; feed-forward (KF)]
    int hpq = 0, hpv = 0, e_q = 0, e_k = 0, e_v = 0, e_g = 0, u1p = 0, u2p = 0;
    int hd = 0;   // attention: padded cache row
    int nsl = 0;  // retention: state slices per head
    int rot = -1;
    void *win = nullptr, *wout = nullptr;
    float *f1 = nullptr, *f2 = nullptr, *r1 = nullptr, *r2 = nullptr, *sink = nullptr, *decay = nullptr;
    // the output projection's input and the attention query rows, one buffer per shape: their padding columns are never
    // written, so they stay zero
    float *cat32 = nullptr, *q = nullptr;
    __half* cat16 = nullptr;
    float n1 = 0.0f, n2 = 0.0f;
    std::vector<float> c1, c2;  // [width][taps] as given
};

// A block of the sequential arrangement (hybrid_seq.hip): latent attention, then a mixture of experts or nothing
struct SeqLayer {
    sli_block_desc d{};
    int window = 0;                        // d.window, or the whole context
    int Hq = 0, Hv = 0, R = 0, Rp = 0;     // query rows, value rows, latent size and its padded size
    int r_kv = 0, r_g = 0, n1 = 0, u1p = 0;  // input projection: first latent / gate row, pairs, first residual-gate pair
    int v0 = 0;                            // first U_v row of ukv
    int KA = 0;                            // padded value rows (the output projection's input)
    int hd = 0;                            // expanded K / V row (0: prompts take the absorbed form)
    int z0 = 0, n2 = 0;                    // second gate matrix [rg2 ; router]: first router row, pairs
    int ffp = 0, FFp = 0, Dn = 0;          // expert pairs padded, down input padded, down rows padded
    void *win = nullptr, *wo = nullptr, *ukv = nullptr, *wg2 = nullptr, *wup = nullptr, *wdn = nullptr;
    float *f1 = nullptr, *lnorm = nullptr, *rg1b = nullptr, *rg2b = nullptr, *zb = nullptr, *w1 = nullptr, *w2 = nullptr;
    std::vector<float> c1;  // taps as given [width][taps]
    // activations whose padding columns are never written (they stay zero): one buffer per shape
    float *lat = nullptr, *q = nullptr, *cat32 = nullptr, *act32 = nullptr;
    __half *cat16 = nullptr, *act16 = nullptr;
    int win_id = -1;  // prompts: the layout of its window (SeqState::wins)
};

// The expansion's layout of one window (latent.h lat_tiles_kernel), computed once per pass
struct SeqWindow {
    int window = 0;
    int2* tiles = nullptr;
    int32_t *ntiles = nullptr, *koff = nullptr;
};

struct SeqState {
    std::vector<SeqLayer> layers;
    std::vector<SeqWindow> wins;
    int key_tiles = 0;  // expansion tiles a pass may take (scratch)
    float *x2 = nullptr, *qf = nullptr, *qa = nullptr, *part = nullptr, *gate = nullptr, *rg1 = nullptr, *rg2 = nullptr,
          *y = nullptr, *z = nullptr, *wsel = nullptr, *ye = nullptr, *zeros = nullptr;
    __half *xh = nullptr, *ks = nullptr, *vs = nullptr;
    int32_t *sel = nullptr, *at = nullptr, *rowmap = nullptr, *ntiles = nullptr;
    int2* tiles = nullptr;
};

struct HyRun {
    int layer = 0;
    void *kc = nullptr, *vc = nullptr;  // (latent attention: kc holds the cache rows)
    float *S = nullptr, *ring = nullptr;
};

struct HyRot {
    int dims = 0;
    double base = 0.0;
    float *cs = nullptr, *sn = nullptr;
};

struct BlockStack {
    sli_stack_config c{};
    hipStream_t stream = nullptr;
    bool f16 = true;
    size_t wb = 2;
    int D = 0, Dp = 0, V = 0, Vp = 0, T = 0, B = 0, taps = 0, M = 0;  // taps: padded tap count; M: rows of a pass
    std::vector<HyLayer> layers;
    std::vector<HyRun> runs;
    std::vector<HyRot> rots;
    std::unique_ptr<SeqState> seq;  // the sequential arrangement (null: parallel)
    void *emb = nullptr, *head = nullptr, *pos = nullptr;
    float *fnorm = nullptr, *fnorm_p = nullptr;  // final gain per channel; times sqrt(D / Dp)
    std::vector<float> fgain;  // one gain, or one per channel
    std::map<std::string, bool> want;  // tensor -> placed
    bool dirty = true;
    // activations of a pass
    RowRef* rows = nullptr;
    SegRef* segs = nullptr;
    int32_t *nsegs = nullptr, *widx = nullptr;
    float *x = nullptr, *q = nullptr, *k = nullptr, *v = nullptr, *g = nullptr, *o = nullptr, *lg = nullptr;
    void *c1 = nullptr, *c2 = nullptr, *xl = nullptr;  // fp32 or fp16 by path
    float* ssq = nullptr;    // retention: sums of o^2 per (head, slice) of a batch-1 step
    float* part = nullptr;   // split partials of the decode attention
    unsigned* attn_cnt = nullptr;  // its per-head arrival counters (zero between launches)
    float* bg_ws = nullptr;  // split-K partials and arrival counters of the batched projections
    unsigned* bg_cnt = nullptr;
    size_t bg_ws_bytes = 0, bg_groups = 1;  // the most any projection needs (hy_bg_need)
    std::vector<void*> allocs;
    // captured passes: {0, rows} of a decode step, {1 + key tile bucket, rows} of a prompt pass
    std::map<std::pair<int, int>, std::pair<hipGraph_t, hipGraphExec_t>> graphs;
};

// device memory of the stack (zeroed), freed with it
int hy_alloc(BlockStack* s, void** p, size_t bytes, bool zero = true);
template <typename T>
int hy_new(BlockStack* s, T** p, size_t n) {
    return hy_alloc(s, reinterpret_cast<void**>(p), sizeof(T) * n);
}

// creation: reserve the workspace of the batched projections of np pairs over K columns
int hy_bg_need(BlockStack* s, int np, int K);

// where a tensor's elements come from: host memory, or (host null) a generator on the device
struct HySrcRand {  // uniform in (-amp, amp) by element index
    uint32_t seed;
    float amp;
    __device__ float operator()(size_t i) const {
        uint32_t h = (uint32_t)i * 2654435761u ^ (uint32_t)(i >> 32) * 0x9E3779B9u ^ seed;
        h ^= h >> 16, h *= 0x7feb352du, h ^= h >> 15, h *= 0x846ca68bu, h ^= h >> 16;
        return amp * ((float)(h >> 8) * (1.0f / 8388608.0f) - 1.0f);
    }
};
struct HyFill {
    const float* host = nullptr;
    HySrcRand rand{};
};
// rows of a tensor into rows map[r] of a fused matrix (row stride ld elements), from column col0 on
int hy_place(BlockStack* s, void* dst, int ld, int col0, const std::vector<int32_t>& map, int ncols, const HyFill& f);
std::vector<int32_t> strided_rows(int n, int first, int step);
// taps [width][given] as coefficients [s->taps][Dp] of the row j positions back, "+ h" included, times gain
int hy_fold_taps(BlockStack* s, const std::vector<float>& w, float gain, float* dst);

// ---- the sequential arrangement
int seq_create(BlockStack* s);  // layers, caches of the runs, buffers
// shape of block i's tensor `leaf` (0 rows: unknown); place one tensor
void seq_shape(const BlockStack* s, int i, const std::string& leaf, int64_t* rows, int64_t* cols);
int seq_put(BlockStack* s, int i, const std::string& leaf, const HyFill& f);
int seq_prepare(BlockStack* s);
// x (embedded rows) -> x after every layer run; one run of it (for inspection). key_tiles: expansion tiles at most.
int seq_pass(BlockStack* s, int M, bool one, int msegs, int key_tiles);
int seq_run(BlockStack* s, int M, bool one, int msegs, int key_tiles, size_t run);
// expansion tiles of a portion (its layer with the widest window; 0: none)
int seq_key_tiles(const BlockStack* s, int pos0, int n);
void seq_step_bytes(const BlockStack* s, const HyRun& r, int B, double pos_sum, double* weights, double* state);

}  // namespace sli
