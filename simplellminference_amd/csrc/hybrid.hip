// hybrid.hip — block-stack models (hybrid.h): configuration checks, weight placement, caches and states, and the
// recorded launches of a decode step and of a prompt pass.
#include "hybrid.h"

#include <cmath>
#include <cstdlib>
#include <cstring>
#include <type_traits>

#include "../../include/sli_synth.h"
#include "attn_mfma.h"
#include "attn_rows.h"
#include "canon.h"
#include "hybrid_gemv.h"
#include "hybrid_kernels.h"
#include "hybrid_rec.h"
#include "hybrid_stack.h"
#include "latent.h"
#include "retention.h"
#include "retention_chunk.h"

namespace sli {

// ---------------------------------------------------------------- creation
int hy_alloc(BlockStack* s, void** p, size_t bytes, bool zero) {
    bytes = std::max<size_t>(bytes, 16);
    hipError_t e = hipMalloc(p, bytes);
    if (e != hipSuccess) return hip_fail(e, "hipMalloc");
    s->allocs.push_back(*p);
    if (zero) SLI_HIP(hipMemset(*p, 0, bytes));
    return SLI_OK;
}

static int hy_layer_init(HyLayer& l, int i) {
    const sli_block_desc& d = l.d;
    const std::string at = "block " + std::to_string(i) + ": ";
    SLI_CHECK(d.heads > 0 && d.dim > 0 && d.vdim > 0 && d.ff >= 0, SLI_ERR_SHAPE, at + "non-positive size");
    SLI_CHECK(d.mixer == SLI_MIX_ATTENTION || d.mixer == SLI_MIX_RETENTION, SLI_ERR_ARG,
              at + "a parallel block mixes with attention or retention");
    SLI_CHECK(d.experts == 0 && d.window == 0, SLI_ERR_ARG, at + "a parallel block has no experts and no window");
    l.mixw = d.heads * d.vdim;
    l.KA = pad_to(l.mixw, 64);
    l.KF = pad_to(d.ff, 64);
    l.Kp = l.KA + l.KF;
    l.hpq = (d.dim + 1) / 2;
    l.hpv = (d.vdim + 1) / 2;
    if (d.mixer == SLI_MIX_ATTENTION) {
        SLI_CHECK(d.kv_heads > 0 && d.heads % d.kv_heads == 0, SLI_ERR_SHAPE, at + "heads must be a multiple of kv_heads");
        SLI_CHECK(d.vdim <= kAttnRowsMaxV, SLI_ERR_SHAPE, at + "attention vdim must be at most 512");
        SLI_CHECK(d.dim <= 4096, SLI_ERR_SHAPE, at + "attention dim must be at most 4096");
        const int w = std::max(d.dim, d.vdim);
        l.hd = w <= 64 ? 64 : w <= 128 ? 128 : pad_to(w, 64);
        l.e_q = d.heads * l.hpq;
        l.e_k = l.e_q + d.kv_heads * l.hpq;
        l.e_v = l.e_k + d.kv_heads * l.hpv;
        l.e_g = l.e_v;
    } else {
        SLI_CHECK(d.rot_dims >= 0 && d.rot_dims % 2 == 0 && d.rot_dims <= d.dim, SLI_ERR_SHAPE, at + "bad rot_dims");
        SLI_CHECK(ret_scan_lds(d.dim) <= 160 * 1024, SLI_ERR_SHAPE, at + "retention dim too large");
        if (ret_scan_lds(d.dim) > 64 * 1024)
            SLI_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(&ret_scan_kernel),
                                        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
        l.nsl = (d.vdim + kRetCols - 1) / kRetCols;
        l.e_q = d.heads * l.hpq;
        l.e_k = l.e_q + d.heads * l.hpq;
        l.e_v = l.e_k + d.heads * l.hpv;
        l.e_g = l.e_v + d.heads * l.hpv;
    }
    l.u1p = d.ff > 0 ? pad_to(l.e_g, kHySection) : pad_to(l.e_g, 8);
    l.u2p = pad_to(d.ff, 8);
    return SLI_OK;
}

// decode attention splits per head at most (attn_mfma_tpw: at most kAmMaxSplits up to 64 tiles per wave)
static int hy_attn_splits(int T) { return std::max(kAmMaxSplits, (T + 64 * kAmWgKeys - 1) / (64 * kAmWgKeys)); }

static int hy_allow_lds();

// the batched projections of np pairs over K columns: their workspace (every row count; the head takes any number of wanted rows)
int hy_bg_need(BlockStack* s, int np, int K) {
    if (!s->f16 || np == 0) return SLI_OK;
    for (int b = 1; b <= kBgMaxBatch; ++b) {
        const BgPlan p = bg_plan((np + 7) / 8, K, b, false, gemv_max_blocks(), true);
        SLI_CHECK(p.groups > 0, SLI_ERR_SHAPE, "stack: no tiling of a batched projection fits");
        s->bg_ws_bytes = std::max(s->bg_ws_bytes, bg_part_bytes(p));
        s->bg_groups = std::max(s->bg_groups, (size_t)p.groups);
    }
    return SLI_OK;
}

// layers, rotation tables and activations of the parallel arrangement
static int par_create(BlockStack* s) {
    const sli_stack_config& c = s->c;
    s->layers.resize(c.n_blocks);
    size_t nq = 0, nk = 0, nv = 0, no = 0;
    int dec = 0;
    std::map<std::pair<int, int>, HyLayer*> by_out;             // (mixer width, ff)
    std::map<std::pair<std::pair<int, int>, int>, float*> by_q;  // (heads, dim), padded row
    for (int i = 0; i < c.n_blocks; ++i) {
        HyLayer& l = s->layers[i];
        l.d = c.blocks[i];
        HY_TRY(hy_layer_init(l, i));
        const bool att = l.d.mixer == SLI_MIX_ATTENTION;
        HY_TRY(hy_alloc(s, &l.win, s->wb * (size_t)2 * (l.u1p + l.u2p) * s->Dp));
        HY_TRY(hy_alloc(s, &l.wout, s->wb * (size_t)pad_to(s->D, 128) * l.Kp));
        const std::string p = "l" + std::to_string(i) + ".";
        for (const char* n : {"norm1", "canon1", "mix.q", "mix.k", "mix.v", "mix.o"}) s->want[p + n] = false;
        HY_TRY(hy_alloc(s, (void**)&l.f1, sizeof(float) * s->taps * s->Dp));
        if (att) {
            for (const char* n : {"mix.r1", "mix.r2", "mix.sink"}) s->want[p + n] = false;
            HY_TRY(hy_alloc(s, (void**)&l.r1, sizeof(float) * l.d.heads));
            HY_TRY(hy_alloc(s, (void**)&l.r2, sizeof(float) * l.d.heads));
            HY_TRY(hy_alloc(s, (void**)&l.sink, sizeof(float) * l.d.heads));
            float*& qb = by_q[{{l.d.heads, l.d.dim}, l.hd}];
            if (!qb) HY_TRY(hy_alloc(s, (void**)&qb, sizeof(float) * (size_t)s->M * l.d.heads * l.hd));
            l.q = qb;
        } else {
            s->want[p + "mix.g"] = false;
            SLI_CHECK(c.decay, SLI_ERR_ARG, "stack: retention needs decay values");
            HY_TRY(hy_alloc(s, (void**)&l.decay, sizeof(float) * l.d.heads));
            SLI_HIP(hipMemcpy(l.decay, c.decay + dec, sizeof(float) * l.d.heads, hipMemcpyHostToDevice));
            dec += l.d.heads;
            nq = std::max(nq, (size_t)l.d.heads * l.d.dim);
            nk = std::max(nk, (size_t)l.d.heads * l.d.dim);
            nv = std::max(nv, (size_t)l.mixw);
            if (l.d.rot_dims > 0) {
                for (size_t r = 0; r < s->rots.size(); ++r)
                    if (s->rots[r].dims == l.d.rot_dims && s->rots[r].base == l.d.rot_base) l.rot = (int)r;
                if (l.rot < 0) {
                    l.rot = (int)s->rots.size();
                    HyRot rt;
                    rt.dims = l.d.rot_dims;
                    rt.base = l.d.rot_base;
                    s->rots.push_back(rt);
                }
            }
        }
        if (l.d.ff > 0) {
            for (const char* n : {"norm2", "canon2", "mlp.gate", "mlp.up", "mlp.down"}) s->want[p + n] = false;
            HY_TRY(hy_alloc(s, (void**)&l.f2, sizeof(float) * s->taps * s->Dp));
        }
        HyLayer*& same = by_out[{l.mixw, l.d.ff}];
        if (same) {
            l.cat32 = same->cat32, l.cat16 = same->cat16;
        } else {
            HY_TRY(hy_alloc(s, (void**)&l.cat32, sizeof(float) * (size_t)s->M * l.Kp));
            if (s->f16) HY_TRY(hy_alloc(s, (void**)&l.cat16, sizeof(__half) * (size_t)s->M * l.Kp));
            same = &l;
        }
        no = std::max(no, (size_t)l.mixw);
    }
    for (HyRot& r : s->rots) {  // angles in double, the table in fp32
        const int h = r.dims / 2;
        std::vector<float> cs((size_t)s->T * h), sn((size_t)s->T * h);
        for (int j = 0; j < h; ++j) {
            const double f = std::pow(r.base, -2.0 * j / r.dims);
            for (int p = 0; p < s->T; ++p) {
                cs[(size_t)p * h + j] = (float)std::cos(p * f);
                sn[(size_t)p * h + j] = (float)std::sin(p * f);
            }
        }
        HY_TRY(hy_alloc(s, (void**)&r.cs, sizeof(float) * cs.size(), false));
        HY_TRY(hy_alloc(s, (void**)&r.sn, sizeof(float) * sn.size(), false));
        SLI_HIP(hipMemcpy(r.cs, cs.data(), sizeof(float) * cs.size(), hipMemcpyHostToDevice));
        SLI_HIP(hipMemcpy(r.sn, sn.data(), sizeof(float) * sn.size(), hipMemcpyHostToDevice));
    }
    for (HyRun& r : s->runs) {
        const HyLayer& l = s->layers[r.layer];
        HY_TRY(hy_new(s, &r.ring, (size_t)s->B * s->taps * s->Dp));
        if (l.d.mixer == SLI_MIX_ATTENTION) {
            const size_t n = (size_t)s->B * l.d.kv_heads * s->T * l.hd * (s->f16 ? 2 : 4);
            HY_TRY(hy_alloc(s, &r.kc, n));
            HY_TRY(hy_alloc(s, &r.vc, n));
        } else {
            HY_TRY(hy_new(s, &r.S, (size_t)s->B * l.d.heads * l.nsl * l.d.dim * kRetCols));
        }
    }
    const size_t M = s->M;
    HY_TRY(hy_new(s, &s->q, M * nq));
    HY_TRY(hy_new(s, &s->k, M * nk));
    HY_TRY(hy_new(s, &s->v, M * nv));
    HY_TRY(hy_new(s, &s->g, M * nv));
    HY_TRY(hy_new(s, &s->o, M * no));
    size_t nssq = 0;
    for (const HyLayer& l : s->layers) nssq = std::max(nssq, (size_t)l.d.heads * l.nsl);
    HY_TRY(hy_new(s, &s->ssq, nssq));
    const int Bp = s->B <= kBgMaxBatch ? s->B : pad_to(s->B, kHyTile);
    size_t part = 0, ncnt = 0;
    for (const HyLayer& l : s->layers) {
        if (l.d.mixer == SLI_MIX_ATTENTION)
            part = std::max(part, (size_t)Bp * l.d.heads * hy_attn_splits(s->T) * (l.hd + kAttnPartPad)),
            ncnt = std::max(ncnt, (size_t)Bp * l.d.heads);
        HY_TRY(hy_bg_need(s, l.e_g, s->Dp));
        HY_TRY(hy_bg_need(s, l.d.ff, s->Dp));
        HY_TRY(hy_bg_need(s, (s->D + 1) / 2, l.Kp));
    }
    HY_TRY(hy_new(s, &s->part, part));
    return hy_new(s, &s->attn_cnt, ncnt);
}

int hy_create(const sli_stack_config* cfg, hipStream_t stream, BlockStack** out) {
    const sli_stack_config& c = *cfg;
    SLI_CHECK(c.vocab > 0 && c.width > 0 && c.n_blocks > 0 && c.blocks && c.max_len > 0 && c.batch > 0, SLI_ERR_SHAPE,
              "stack: non-positive dimension");
    SLI_CHECK(c.taps >= 1 && c.taps <= kCanonMaxTaps, SLI_ERR_SHAPE, "stack: taps must be 1 .. 32");
    SLI_CHECK(c.loop_start >= 0 && c.loop_start <= c.loop_stop && c.loop_stop <= c.n_blocks && c.loop_times >= 1,
              SLI_ERR_SHAPE, "stack: bad loop");
    SLI_CHECK(c.w_dtype == SLI_DT_F16 || c.w_dtype == SLI_DT_F32, SLI_ERR_ARG, "stack: fp16 or fp32 weights");
    SLI_CHECK(c.arrangement == SLI_STACK_PARALLEL || c.arrangement == SLI_STACK_SEQUENTIAL, SLI_ERR_ARG,
              "stack: unknown arrangement");
    SLI_CHECK(c.positions >= 0 && (c.positions == 0 || c.max_len <= c.positions), SLI_ERR_SHAPE,
              "stack: max_len exceeds the learned positions");
    BlockStack* s = new BlockStack();
    *out = s;  // destroyed by the caller on failure
    s->c = c;
    s->stream = stream;
    s->f16 = c.w_dtype == SLI_DT_F16;
    s->wb = s->f16 ? 2 : 4;
    s->D = c.width;
    s->Dp = pad_to(c.width, 64);
    s->V = c.vocab;
    s->Vp = pad_to(c.vocab, 128);
    s->T = c.max_len;
    s->B = c.batch;
    s->taps = std::max(c.taps, kCanonFusedTaps);
    s->M = kHyMaxRows;
    if (c.arrangement == SLI_STACK_SEQUENTIAL) s->seq = std::make_unique<SeqState>();
    auto add_run = [&](int i) {
        HyRun r;
        r.layer = i;
        s->runs.push_back(r);
    };
    if (c.runs) {
        for (int i = 0; i < c.n_runs; ++i) {
            SLI_CHECK(c.runs[i] >= 0 && c.runs[i] < c.n_blocks, SLI_ERR_SHAPE, "stack: a run of no block");
            add_run(c.runs[i]);
        }
    } else {
        for (int i = 0; i < c.loop_start; ++i) add_run(i);
        for (int t = 0; t < c.loop_times; ++t)
            for (int i = c.loop_start; i < c.loop_stop; ++i) add_run(i);
        for (int i = c.loop_stop; i < c.n_blocks; ++i) add_run(i);
    }
    SLI_CHECK(!s->runs.empty(), SLI_ERR_SHAPE, "stack: no runs");
    HY_TRY(hy_alloc(s, &s->emb, s->wb * (size_t)s->V * s->D));
    HY_TRY(hy_alloc(s, &s->head, s->wb * (size_t)s->Vp * s->Dp));
    HY_TRY(hy_alloc(s, (void**)&s->fnorm, sizeof(float) * s->Dp));
    HY_TRY(hy_alloc(s, (void**)&s->fnorm_p, sizeof(float) * s->Dp));
    for (const char* n : {"embed", "head", "final.norm"}) s->want[n] = false;
    if (c.positions > 0) {
        HY_TRY(hy_alloc(s, &s->pos, s->wb * (size_t)c.positions * s->D));
        s->want["pos"] = false;
    }
    const size_t M = s->M;
    HY_TRY(hy_alloc(s, (void**)&s->rows, sizeof(RowRef) * M));
    HY_TRY(hy_alloc(s, (void**)&s->segs, sizeof(SegRef) * M));
    HY_TRY(hy_alloc(s, (void**)&s->nsegs, sizeof(int32_t)));
    HY_TRY(hy_alloc(s, (void**)&s->widx, sizeof(int32_t) * M));
    HY_TRY(hy_alloc(s, (void**)&s->x, sizeof(float) * M * s->Dp));
    HY_TRY(hy_alloc(s, &s->c1, sizeof(float) * M * s->Dp));
    HY_TRY(hy_alloc(s, &s->c2, sizeof(float) * M * s->Dp));
    HY_TRY(hy_alloc(s, &s->xl, sizeof(float) * M * s->Dp));
    HY_TRY(hy_alloc(s, (void**)&s->lg, sizeof(float) * kHyLogitRows * s->V));
    HY_TRY(hy_bg_need(s, (s->V + 1) / 2, s->Dp));
    HY_TRY(s->seq ? seq_create(s) : par_create(s));
    HY_TRY(hy_alloc(s, (void**)&s->bg_ws, s->bg_ws_bytes + 256));
    HY_TRY(hy_new(s, &s->bg_cnt, s->bg_groups));
    return hy_allow_lds();
}

void hy_destroy(BlockStack* s) {
    if (!s) return;
    for (auto& [key, g] : s->graphs) {
        if (g.second) (void)hipGraphExecDestroy(g.second);
        if (g.first) (void)hipGraphDestroy(g.first);
    }
    for (void* p : s->allocs) (void)hipFree(p);
    delete s;
}

int hy_runs(const BlockStack* s) { return (int)s->runs.size(); }
int hy_key_tiles(const BlockStack* s, int pos0, int n) { return seq_key_tiles(s, pos0, n); }
int hy_key_tiles_max(const BlockStack* s) { return s->seq ? s->seq->key_tiles : 0; }

// ---------------------------------------------------------------- weights
int hy_place(BlockStack* s, void* dst, int ld, int col0, const std::vector<int32_t>& map, int ncols,
                    const HyFill& f) {
    const size_t n = map.size() * (size_t)ncols;
    float* tmp = nullptr;
    int32_t* dm = nullptr;
    int rc = SLI_OK;
    if ((f.host && hipMalloc(&tmp, sizeof(float) * n) != hipSuccess) ||
        hipMalloc(&dm, sizeof(int32_t) * map.size()) != hipSuccess)
        rc = fail(SLI_ERR_NOMEM, "weight staging");
    if (rc == SLI_OK && ((f.host && hipMemcpy(tmp, f.host, sizeof(float) * n, hipMemcpyHostToDevice) != hipSuccess) ||
                         hipMemcpy(dm, map.data(), sizeof(int32_t) * map.size(), hipMemcpyHostToDevice) != hipSuccess))
        rc = fail(SLI_ERR_HIP, "weight upload");
    if (rc == SLI_OK) {
        const dim3 grid((unsigned)map.size()), bl(256);
        auto go = [&](auto* d, auto src) {
            using WT = std::remove_pointer_t<decltype(d)>;
            hipLaunchKernelGGL((hy_place_kernel<WT, decltype(src)>), grid, bl, 0, s->stream, d, ld, col0, dm, ncols, src);
        };
        if (s->f16)
            f.host ? go((__half*)dst, HySrcBuf{tmp}) : go((__half*)dst, f.rand);
        else
            f.host ? go((float*)dst, HySrcBuf{tmp}) : go((float*)dst, f.rand);
        if (hipGetLastError() != hipSuccess || hipStreamSynchronize(s->stream) != hipSuccess)
            rc = fail(SLI_ERR_HIP, "weight placement");
    }
    if (tmp) (void)hipFree(tmp);
    if (dm) (void)hipFree(dm);
    return rc;
}

// fused-matrix rows of a head-wise tensor: `heads` heads of n dims, rh rotation pairs, from pair u0 on
static std::vector<int32_t> head_rows(int heads, int n, int rh, int u0) {
    std::vector<int32_t> map;
    const int hp = (n + 1) / 2;
    for (int h = 0; h < heads; ++h)
        for (int d = 0; d < n; ++d) {
            const int j = d < rh ? d : d < 2 * rh ? d - rh : d / 2;
            const int e = d < rh ? 0 : d < 2 * rh ? 1 : d & 1;
            map.push_back(2 * (u0 + h * hp + j) + e);
        }
    return map;
}
std::vector<int32_t> strided_rows(int n, int first, int step) {
    std::vector<int32_t> map(n);
    for (int i = 0; i < n; ++i) map[i] = first + step * i;
    return map;
}

// shape of a tensor: rows x cols (vectors: 1 x n), 0 rows: unknown name
static void hy_shape(const BlockStack* s, const std::string& name, int* li, std::string* leaf, int64_t* rows, int64_t* cols) {
    *li = -1;
    *rows = *cols = 0;
    *leaf = name;
    if (name == "embed" || name == "head") {
        *rows = s->V, *cols = s->D;
        return;
    }
    if (name == "final.norm") {
        *rows = 1, *cols = s->seq ? s->D : 1;
        return;
    }
    if (name == "pos") {
        *rows = s->c.positions, *cols = s->D;
        return;
    }
    const size_t dot = name.find('.');
    *li = std::atoi(name.c_str() + 1);
    *leaf = name.substr(dot + 1);
    if (s->seq) return seq_shape(s, *li, *leaf, rows, cols);
    const sli_block_desc& d = s->layers[*li].d;
    const int kvh = d.mixer == SLI_MIX_ATTENTION ? d.kv_heads : d.heads;
    const std::string& t = *leaf;
    auto set = [&](int64_t r, int64_t c) { *rows = r, *cols = c; };
    if (t == "norm1" || t == "norm2") set(1, 1);
    else if (t == "canon1" || t == "canon2") set(s->D, s->c.taps);
    else if (t == "mix.q") set((int64_t)d.heads * d.dim, s->D);
    else if (t == "mix.k") set((int64_t)kvh * d.dim, s->D);
    else if (t == "mix.v") set((int64_t)kvh * d.vdim, s->D);
    else if (t == "mix.g") set((int64_t)d.heads * d.vdim, s->D);
    else if (t == "mix.o") set(s->D, (int64_t)d.heads * d.vdim);
    else if (t == "mix.r1" || t == "mix.r2" || t == "mix.sink") set(1, d.heads);
    else if (t == "mlp.gate" || t == "mlp.up") set(d.ff, s->D);
    else if (t == "mlp.down") set(s->D, d.ff);
}

static int hy_put(BlockStack* s, const std::string& name, const HyFill& f, int64_t n) {
    const float* host = f.host;  // (vectors always come from the host)
    auto it = s->want.find(name);
    SLI_CHECK(it != s->want.end(), SLI_ERR_ARG, "the model has no tensor '" + name + "'");
    int li;
    std::string t;
    int64_t rows, cols;
    hy_shape(s, name, &li, &t, &rows, &cols);
    SLI_CHECK(n == rows * cols, SLI_ERR_SHAPE, "tensor '" + name + "' has the wrong size");
    if (s->f16 && host)
        for (int64_t i = 0; i < n; ++i)
            SLI_CHECK(std::fabs(host[i]) <= 65504.0f, SLI_ERR_RANGE, "tensor '" + name + "' has values fp16 cannot hold");
    s->dirty = true;
    int rc = SLI_OK;
    if (name == "embed") {
        rc = hy_place(s, s->emb, s->D, 0, strided_rows(s->V, 0, 1), s->D, f);
    } else if (name == "head") {
        rc = hy_place(s, s->head, s->Dp, 0, strided_rows(s->V, 0, 1), s->D, f);
    } else if (name == "pos") {
        rc = hy_place(s, s->pos, s->D, 0, strided_rows(s->c.positions, 0, 1), s->D, f);
    } else if (name == "final.norm") {
        s->fgain.assign(host, host + n);
    } else if (s->seq) {
        rc = seq_put(s, li, t, f);
    } else {
        HyLayer& l = s->layers[li];
        const sli_block_desc& d = l.d;
        const int kvh = d.mixer == SLI_MIX_ATTENTION ? d.kv_heads : d.heads;
        const int rh = d.mixer == SLI_MIX_RETENTION ? d.rot_dims / 2 : 0;
        if (t == "norm1") l.n1 = host[0];
        else if (t == "norm2") l.n2 = host[0];
        else if (t == "canon1") l.c1.assign(host, host + n);
        else if (t == "canon2") l.c2.assign(host, host + n);
        else if (t == "mix.q") rc = hy_place(s, l.win, s->Dp, 0, head_rows(d.heads, d.dim, rh, 0), s->D, f);
        else if (t == "mix.k") rc = hy_place(s, l.win, s->Dp, 0, head_rows(kvh, d.dim, rh, l.e_q), s->D, f);
        else if (t == "mix.v") rc = hy_place(s, l.win, s->Dp, 0, head_rows(kvh, d.vdim, 0, l.e_k), s->D, f);
        else if (t == "mix.g") rc = hy_place(s, l.win, s->Dp, 0, head_rows(d.heads, d.vdim, 0, l.e_v), s->D, f);
        else if (t == "mix.o") rc = hy_place(s, l.wout, l.Kp, 0, strided_rows(s->D, 0, 1), l.mixw, f);
        else if (t == "mlp.gate") rc = hy_place(s, l.win, s->Dp, 0, strided_rows(d.ff, 2 * l.u1p, 2), s->D, f);
        else if (t == "mlp.up") rc = hy_place(s, l.win, s->Dp, 0, strided_rows(d.ff, 2 * l.u1p + 1, 2), s->D, f);
        else if (t == "mlp.down") rc = hy_place(s, l.wout, l.Kp, l.KA, strided_rows(s->D, 0, 1), d.ff, f);
        else {
            float* p = t == "mix.r1" ? l.r1 : t == "mix.r2" ? l.r2 : l.sink;
            SLI_HIP(hipMemcpy(p, host, sizeof(float) * n, hipMemcpyHostToDevice));
        }
    }
    if (rc == SLI_OK) it->second = true;
    return rc;
}

int hy_set_tensor(BlockStack* s, const std::string& name, const float* host, int64_t n) {
    HyFill f;
    f.host = host;
    return hy_put(s, name, f, n);
}

// seeded random weights (matrices on the device)
int hy_init_synthetic(BlockStack* s, uint32_t seed) {
    std::vector<std::string> names;
    for (auto& kv : s->want) names.push_back(kv.first);
    uint32_t id = 0;
    for (const std::string& name : names) {
        int li;
        std::string t;
        int64_t rows, cols;
        hy_shape(s, name, &li, &t, &rows, &cols);
        const int64_t n = rows * cols;
        const bool canon = t == "canon1" || t == "canon2";
        const bool gain = t == "norm1" || t == "norm2" || t == "final.norm" || t == "mix.dkv.norm";
        HyFill f;
        f.rand.seed = (seed * 0x9E3779B9u) ^ (++id * 0x85EBCA6Bu);
        f.rand.amp = canon ? 0.3f : t == "embed" ? 1.0f : rows > 1 ? 1.5f / std::sqrt((float)cols) : 1.0f;
        std::vector<float> v;
        if (rows == 1 || canon) {
            const float amp = gain ? 0.1f : t == "mix.r2" ? 0.2f : f.rand.amp;
            const bool bias = t.size() > 2 && t.compare(t.size() - 2, 2, ".b") == 0;
            const float off = gain ? 1.0f : t == "mix.r2" ? 0.25f : canon || bias ? 0.0f : 1.0f;
            uint64_t x = 0x9E3779B97F4A7C15ull * (f.rand.seed + 1ull);
            for (int64_t i = 0; i < n; ++i) {
                x ^= x >> 12, x ^= x << 25, x ^= x >> 27;
                v.push_back(off + amp * (float)((double)((x * 0x2545F4914F6CDD1Dull) >> 40) / 8388608.0 - 1.0));
            }
            f.host = v.data();
        }
        HY_TRY(hy_put(s, name, f, n));
    }
    return SLI_OK;
}

int hy_fold_taps(BlockStack* s, const std::vector<float>& w, float gain, float* dst) {
    const int given = s->c.taps;
    std::vector<float> f((size_t)s->taps * s->Dp, 0.0f);
    for (int d = 0; d < s->D; ++d)
        for (int j = 0; j < given; ++j) {
            const double c = (double)w[(size_t)d * given + given - 1 - j] + (j == 0 ? 1.0 : 0.0);
            f[(size_t)j * s->Dp + d] = (float)(gain * c);
        }
    SLI_HIP(hipMemcpy(dst, f.data(), sizeof(float) * f.size(), hipMemcpyHostToDevice));
    return SLI_OK;
}

int hy_prepare(BlockStack* s) {
    if (!s->dirty) return SLI_OK;
    for (auto& kv : s->want) SLI_CHECK(kv.second, SLI_ERR_STATE, "tensor '" + kv.first + "' was not loaded");
    SLI_HIP(hipStreamSynchronize(s->stream));
    const int Dp = s->Dp;
    if (s->seq) HY_TRY(seq_prepare(s));
    for (HyLayer& l : s->layers) {
        HY_TRY(hy_fold_taps(s, l.c1, l.n1, l.f1));
        if (l.d.ff > 0) HY_TRY(hy_fold_taps(s, l.c2, l.n2, l.f2));
    }
    std::vector<float> g(Dp, 0.0f);
    for (int d = 0; d < s->D; ++d) g[d] = s->fgain[s->fgain.size() == 1 ? 0 : d];
    SLI_HIP(hipMemcpy(s->fnorm, g.data(), sizeof(float) * Dp, hipMemcpyHostToDevice));
    for (int d = 0; d < s->D; ++d) g[d] = (float)(g[d] * std::sqrt((double)s->D / Dp));
    SLI_HIP(hipMemcpy(s->fnorm_p, g.data(), sizeof(float) * Dp, hipMemcpyHostToDevice));
    s->dirty = false;
    return SLI_OK;
}

// ---------------------------------------------------------------- the forward pass over rows
template <typename WT>
struct HyRec : HyProj<WT> {
    using KT = WT;  // fp16 weights with an fp16 cache, fp32 with fp32
    using P = HyProj<WT>;
    using P::F16, P::GV, P::s, P::M, P::one, P::msegs, P::key_tiles, P::st, P::path, P::rows_for, P::project, P::pgemm;
    template <class Epi>
    static int allow() { return P::template allow<Epi>(); }
    template <typename OT>
    static OT* cat(const HyLayer& l) {
        if constexpr (std::is_same<OT, float>::value)
            return l.cat32;
        else
            return l.cat16;
    }
    CanonArgs canon(const HyLayer& l, const HyRun& r) const {
        return CanonArgs{s->x, r.ring, l.f1, l.f2, s->rows, s->c.eps, s->D, s->Dp, s->taps, M};
    }
    template <typename OT>
    HyIn<KT, OT> in_epi(const HyLayer& l, const HyRun& r) const {
        const sli_block_desc& d = l.d;
        HyIn<KT, OT> e{};
        e.retention = d.mixer == SLI_MIX_RETENTION;
        e.H = d.heads, e.G = d.kv_heads, e.dim = d.dim, e.vdim = d.vdim, e.hpq = l.hpq, e.hpv = l.hpv;
        e.e_q = l.e_q, e.e_k = l.e_k, e.e_v = l.e_v, e.e_g = l.e_g, e.u1p = l.u1p, e.ff = d.ff;
        e.rh = l.rot >= 0 ? d.rot_dims / 2 : 0;
        e.hd = l.hd, e.T = s->T;
        e.kscale = (float)(1.0 / std::sqrt((double)d.dim));
        e.limit = d.ff_limit;
        e.even = d.dim % 4 == 0 && d.vdim % 4 == 0 && e.rh % 2 == 0;
        if (l.rot >= 0) e.cs = s->rots[l.rot].cs, e.sn = s->rots[l.rot].sn;
        e.q = l.q ? l.q : s->q, e.k = s->k, e.v = s->v, e.g = s->g;
        e.kc = (KT*)r.kc, e.vc = (KT*)r.vc;
        e.act = cat<OT>(l), e.act_ld = l.Kp, e.act_off = l.KA;
        e.rows = s->rows;
        return e;
    }
    template <typename OT>
    int mixer(const HyLayer& l, const HyRun& r) const {
        const sli_block_desc& d = l.d;
        if (d.mixer == SLI_MIX_ATTENTION) return attention<OT>(l, r);
        RetArgs a{s->q, s->k, s->v, r.S, s->o, l.decay, s->rows, s->segs, s->nsegs, d.heads, d.dim, d.vdim, l.nsl};
        const dim3 sg(l.nsl, d.heads, msegs);
        const int kd = F16 ? ret_chunk_kd(d.dim) : 0;
        if (one)
            hipLaunchKernelGGL(ret_step_kernel, dim3(l.nsl, d.heads, M), dim3(256), 0, st(), a);
        else if (kd == 32)
            hipLaunchKernelGGL(ret_chunk_kernel<32>, sg, dim3(256), RcGeo<32>::LDS, st(), a);
        else if (kd == 64)
            hipLaunchKernelGGL(ret_chunk_kernel<64>, sg, dim3(256), RcGeo<64>::LDS, st(), a);
        else if (kd == 128)
            hipLaunchKernelGGL(ret_chunk_kernel<128>, sg, dim3(256), RcGeo<128>::LDS, st(), a);
        else if (kd == 256)
            hipLaunchKernelGGL(ret_chunk_kernel<256>, sg, dim3(256), RcGeo<256>::LDS, st(), a);
        else
            hipLaunchKernelGGL(ret_scan_kernel, sg, dim3(256), ret_scan_lds(d.dim), st(), a);
        SLI_HIP(hipGetLastError());
        hipLaunchKernelGGL(ret_gate_kernel<OT>, dim3((M * d.heads + 3) / 4), dim3(256), 0, st(), s->o, s->g, s->rows,
                           cat<OT>(l), l.Kp, M, d.heads, d.vdim, s->c.eps);
        SLI_HIP(hipGetLastError());
        return SLI_OK;
    }
    template <int HD>
    void attn_split(const AttnArgs<__half>& a, int g, int blocks, bool ring) const {
        const dim3 gr(blocks), bl(64 * kAmWaves);
        switch (g * 2 + (ring ? 1 : 0)) {
            case 2: hipLaunchKernelGGL((attn_mfma_kernel<HD, 1, 1, true>), gr, bl, 0, st(), a); break;
            case 3: hipLaunchKernelGGL((attn_mfma_kernel<HD, 1, 2, true>), gr, bl, 0, st(), a); break;
            case 4: hipLaunchKernelGGL((attn_mfma_kernel<HD, 2, 1, true>), gr, bl, 0, st(), a); break;
            case 5: hipLaunchKernelGGL((attn_mfma_kernel<HD, 2, 2, true>), gr, bl, 0, st(), a); break;
            case 8: hipLaunchKernelGGL((attn_mfma_kernel<HD, 4, 1, true>), gr, bl, 0, st(), a); break;
            case 9: hipLaunchKernelGGL((attn_mfma_kernel<HD, 4, 2, true>), gr, bl, 0, st(), a); break;
            case 16: hipLaunchKernelGGL((attn_mfma_kernel<HD, 8, 1, true>), gr, bl, 0, st(), a); break;
            default: hipLaunchKernelGGL((attn_mfma_kernel<HD, 8, 2, true>), gr, bl, 0, st(), a); break;
        }
    }
    template <typename OT>
    int attention(const HyLayer& l, const HyRun& r) const {
        const sli_block_desc& d = l.d;
        const AttnRowsArgs ra{l.q, r.kc, r.vc, s->rows, l.r1, l.r2, l.sink, d.heads, d.kv_heads, d.dim, d.vdim, l.hd,
                              s->T, M, d.scale};
        if constexpr (F16) {
            if (one && l.hd <= 128) {  // split context, then the merge with the sink
                const int gq = d.heads / d.kv_heads, g = gq % 8 == 0 ? 8 : gq % 4 == 0 ? 4 : gq % 2 == 0 ? 2 : 1;
                const int kvg = gq / g, nkv = M * d.kv_heads * kvg;
                AttnArgs<__half> a{};
                a.q = l.q;
                a.k = (const __half*)r.kc;
                a.v = (const __half*)r.vc;
                a.pos_stride = l.hd;
                a.head_stride = (long long)s->T * l.hd;
                a.part = s->part;
                a.pos_dev = &s->rows->pos;
                a.slot_dev = &s->rows->slot;
                a.pos_seq_stride = sizeof(RowRef) / sizeof(int32_t);
                a.n_kv_heads = nkv;
                a.seq_heads = d.kv_heads * kvg;
                a.kv_group = kvg;
                a.scale = d.scale;
                a.bias_r1 = l.r1;
                a.bias_r2 = l.r2;
                a.sink = l.sink;
                a.counters = s->attn_cnt;
                a.vdim = d.vdim;
                a.out_ld = l.Kp;
                if constexpr (std::is_same<OT, float>::value)
                    a.out = l.cat32;
                else
                    a.defer_merge = 2;
                const int tpw = attn_mfma_tpw(nkv, s->T, device_cus());
                a.ppwg = kAmWgKeys * tpw;
                a.max_splits = (s->T + a.ppwg - 1) / a.ppwg;
                SLI_CHECK(a.max_splits <= hy_attn_splits(s->T), SLI_ERR_SHAPE, "attention: more splits than the buffer holds");
                if (l.hd == 64)
                    attn_split<64>(a, g, nkv * a.max_splits, tpw > 1);
                else
                    attn_split<128>(a, g, nkv * a.max_splits, tpw > 1);
                SLI_HIP(hipGetLastError());
                if (a.defer_merge == 0) return SLI_OK;  // merged into out by the launch itself
                hipLaunchKernelGGL(attn_sink_merge_kernel<OT>, dim3(d.heads, M), dim3(128), 0, st(), s->part, ra,
                                   a.max_splits, a.ppwg, cat<OT>(l), l.Kp);
                SLI_HIP(hipGetLastError());
                return SLI_OK;
            }
            if constexpr (!std::is_same<OT, float>::value) {
                if (!one && l.hd <= 128) {
                    const PfAttnArgs<__half> pa{l.q, (const __half*)r.kc, (const __half*)r.vc, cat<OT>(l), nullptr,
                                                d.heads, d.kv_heads, s->T, d.scale};
                    const PfRowsArgs px{s->rows, l.r1, l.r2, l.sink, l.Kp, d.vdim};
                    const dim3 gr(M / 16, d.heads);
                    if (l.hd == 64)
                        hipLaunchKernelGGL((pf_attn_mfma_kernel<64, 1>), gr, dim3(256), 0, st(), pa, nullptr, px);
                    else
                        hipLaunchKernelGGL((pf_attn_mfma_kernel<128, 1>), gr, dim3(256), 0, st(), pa, nullptr, px);
                    SLI_HIP(hipGetLastError());
                    return SLI_OK;
                }
            }
        }
        hipLaunchKernelGGL((attn_rows_kernel<KT, OT>), dim3(d.heads, M), dim3(64), sizeof(float) * (d.dim + 64), st(), ra,
                           cat<OT>(l), l.Kp);
        SLI_HIP(hipGetLastError());
        return SLI_OK;
    }
    int layer(const HyRun& r) const {
        if constexpr (F16)
            if (M > kBgMaxBatch) return layer_as<__half>(r);
        return layer_as<float>(r);
    }
    // Batch 1: the layer as three launches (hybrid_gemv.h), where its shape fits their prologues
    bool fits_fused(const HyLayer& l) const {
        const sli_block_desc& d = l.d;
        if (M != 1 || !one || s->taps != kCanonFusedTaps || s->Dp > 4 * kGemvThreads) return false;
        if (!hy_out_fits(l.KA, l.KF, l.mixw, d.vdim)) return false;
        return d.mixer == SLI_MIX_RETENTION || (F16 && l.hd <= 128);
    }
    int layer_fused(const HyRun& r) const {
        const HyLayer& l = s->layers[r.layer];
        const sli_block_desc& d = l.d;
        SLI_HIP((launch_hy_in<WT>((const WT*)l.win, canon(l, r), in_epi<float>(l, r), l.e_g, l.u1p, (int)d.ff, st())));
        HyOutIn o{};
        o.cat = l.cat32;
        o.KA = l.KA, o.KF = l.KF, o.mixw = l.mixw, o.vdim = d.vdim;
        o.o = s->o, o.gate = s->g, o.ssq = s->ssq, o.nsl = l.nsl;
        o.eps = s->c.eps;
        const EpiStore<1> e{s->x, s->x, nullptr, s->c.residual_mult, s->D};
        if (d.mixer == SLI_MIX_ATTENTION) {
            HY_TRY(attention<float>(l, r));
            SLI_HIP((launch_hy_out<WT, false>((const WT*)l.wout, o, e, s->D, st())));
        } else {
            RetArgs a{s->q, s->k, s->v, r.S, s->o, l.decay, s->rows, s->segs, s->nsegs, d.heads, d.dim, d.vdim, l.nsl};
            a.ssq = s->ssq;
            hipLaunchKernelGGL(ret_step_kernel, dim3(l.nsl, d.heads, 1), dim3(256), 0, st(), a);
            SLI_HIP(hipGetLastError());
            SLI_HIP((launch_hy_out<WT, true>((const WT*)l.wout, o, e, s->D, st())));
        }
        return SLI_OK;
    }
    template <typename OT>
    int layer_as(const HyRun& r) const {
        const HyLayer& l = s->layers[r.layer];
        if (fits_fused(l)) return layer_fused(r);
        const CanonArgs ca = canon(l, r);
        SLI_HIP((launch_canon_rows<OT>(ca, (OT*)s->c1, l.d.ff > 0 ? (OT*)s->c2 : (OT*)nullptr, one ? 1 : 0, st())));
        if (!one) {
            hipLaunchKernelGGL(canon_ring_kernel, dim3(M), dim3(256), 0, st(), ca);
            SLI_HIP(hipGetLastError());
        }
        const auto ei = in_epi<OT>(l, r);
        if constexpr (!std::is_same<OT, float>::value) {
            if (l.d.ff > 0)
                HY_TRY(pgemm((const WT*)l.win, (const __half*)s->c1, (const __half*)s->c2, l.u1p, s->Dp, l.u1p + l.d.ff, 0, ei));
            else
                HY_TRY(pgemm((const WT*)l.win, (const __half*)s->c1, nullptr, 0, s->Dp, l.e_g, 0, ei));
        } else {
            HY_TRY(project(l.win, s->c1, s->Dp, l.e_g, 0, ei));
            if (l.d.ff > 0) HY_TRY(project(l.win, s->c2, s->Dp, l.d.ff, l.u1p, ei));
        }
        HY_TRY(mixer<OT>(l, r));
        if constexpr (std::is_same<OT, float>::value) {
            if (path(M, l.Kp) == GV) {
                GemvIn in{l.cat32, nullptr, 0.0f, l.Kp};
                const EpiStore<1> e{s->x, s->x, nullptr, s->c.residual_mult, s->D};
                SLI_HIP((launch_gemv_u<WT, 1, 6, true>((const WT*)l.wout, in, e, s->D, st())));
                return SLI_OK;
            }
        }
        const HyOut eo{s->x, s->Dp, s->D, s->c.residual_mult};
        return project(l.wout, cat<OT>(l), l.Kp, (s->D + 1) / 2, 0, eo);
    }
    int embed() const {
        hipLaunchKernelGGL(hy_embed_kernel<WT>, dim3(M), dim3(256), 0, st(), s->rows, (const WT*)s->emb, (const WT*)s->pos,
                           s->c.emb_scale, s->x, s->V, s->D, s->Dp);
        SLI_HIP(hipGetLastError());
        return SLI_OK;
    }
    // logits [n][V] of rows idx (null: rows 0 .. n - 1)
    int logits(const int32_t* idx, int n, float* y) const {
        HyRec h = *this;
        h.M = rows_for(n);
        if constexpr (F16)
            if (h.M > kBgMaxBatch) return h.template logits_as<__half>(idx, n, y);
        return h.template logits_as<float>(idx, n, y);
    }
    template <typename OT>
    int logits_as(const int32_t* idx, int n, float* y) const {
        hipLaunchKernelGGL(norm_rows_kernel<OT>, dim3(n), dim3(256), 0, st(), s->x, idx, s->fnorm, (OT*)s->xl, s->D, s->Dp,
                           s->c.eps);
        SLI_HIP(hipGetLastError());
        return project(s->head, s->xl, s->Dp, (s->V + 1) / 2, 0, HyLogits{y, s->V, n});
    }
    int pass() const {
        HY_TRY(embed());
        if (s->seq) return seq_pass(s, M, one, msegs, key_tiles);
        for (const HyRun& r : s->runs) HY_TRY(layer(r));
        return SLI_OK;
    }
    int run(size_t r) const { return s->seq ? seq_run(s, M, one, msegs, key_tiles, r) : layer(s->runs[r]); }
    int step(const DevState* dst, int B, float* y, unsigned long long* keys, int key_ld, int* nkeys) const {
        hipLaunchKernelGGL(hy_rows_kernel, dim3(1), dim3(256), 0, st(), dst, s->rows, B, M);
        SLI_HIP(hipGetLastError());
        HY_TRY(pass());
        if (B == 1 && path(1, s->Dp) == GV) {
            // the norm over the padded row: x / sqrt(sum / D + eps) = sqrt(D / Dp) x / sqrt(sum / Dp + eps D / Dp)
            GemvIn in{s->x, s->fnorm_p, (float)((double)s->c.eps * s->D / s->Dp), s->Dp};
            const EpiLogits<2> e{y, keys, nullptr, s->V, 0, 0ull};
            const int units = (s->V + 1) / 2, cs = gemv_split<WT, 4>(units, s->Dp).cs;
            *nkeys = cs == 1 ? gemv_balanced_blocks(units) : gemv_blocks(units, cs);  // launch_gemv's grid
            SLI_HIP((launch_gemv_u<WT, 2, 4, true>((const WT*)s->head, in, e, units, st())));
            return SLI_OK;
        }
        HY_TRY(logits(nullptr, B, y));
        *nkeys = std::max(1, std::min({key_ld, 64, s->V / 1024}));
        hipLaunchKernelGGL(hy_keys_kernel, dim3(B, *nkeys), dim3(256), 0, st(), y, s->V, keys, key_ld);
        SLI_HIP(hipGetLastError());
        return SLI_OK;
    }
    static int allow_all() {
        HY_TRY((allow<HyIn<KT, float>>()));
        HY_TRY((allow<HyIn<KT, __half>>()));
        HY_TRY((allow<HyOut>()));
        return allow<HyLogits>();
    }
};

static int hy_allow_lds() {
    SLI_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(&ret_chunk_kernel<256>),
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)RcGeo<256>::LDS));
    SLI_HIP(hy_out_allow_lds<__half>());
    SLI_HIP(hy_out_allow_lds<float>());
    return HyRec<__half>::allow_all();
}

#define HY_DISPATCH(s, M, one, msegs, kt, CALL)                             \
    ((s)->f16 ? HyRec<__half>{{(s), (M), (one), (msegs), (kt)}}.CALL \
              : HyRec<float>{{(s), (M), (one), (msegs), (kt)}}.CALL)

int hy_key_ld(const BlockStack*, int) { return std::max(1, gemv_max_blocks()); }

int hy_record_step(BlockStack* s, const DevState* st, int B, float* logits, unsigned long long* keys, int key_ld,
                   int* nkeys) {
    const int M = s->f16 ? HyRec<__half>::rows_for(B) : B;
    return HY_DISPATCH(s, M, true, M, 0, step(st, B, logits, keys, key_ld, nkeys));
}

static int hy_capture(BlockStack* s, std::pair<hipGraph_t, hipGraphExec_t>& g, int M, bool one, int msegs,
                      int key_tiles) {
    if (g.second) return SLI_OK;
    SLI_HIP(hipStreamBeginCapture(s->stream, hipStreamCaptureModeRelaxed));
    const int rc = HY_DISPATCH(s, M, one, msegs, key_tiles, pass());
    hipGraph_t gr = nullptr;
    const hipError_t e = hipStreamEndCapture(s->stream, &gr);
    if (rc != SLI_OK || e != hipSuccess) {
        if (gr) (void)hipGraphDestroy(gr);
        return rc != SLI_OK ? rc : hip_fail(e, "hipStreamEndCapture");
    }
    g.first = gr;
    SLI_HIP(hipGraphInstantiate(&g.second, gr, nullptr, nullptr, 0));
    return SLI_OK;
}

int hy_pass(BlockStack* s, const std::vector<RowRef>& rows_in, const std::vector<SegRef>& segs, bool one,
            const std::vector<int32_t>& want, float* logits_host, float* hidden_host) {
    const int n = (int)rows_in.size();
    SLI_CHECK(n >= 1 && n <= s->M && !segs.empty() && (int)segs.size() <= s->M, SLI_ERR_SHAPE, "pass: too many rows");
    // a decode step runs its rows as they are; a prompt pass is padded to a row count with a captured graph
    int M = s->f16 ? HyRec<__half>::rows_for(n) : n, kt = 0;
    SLI_CHECK(!one || n <= s->B, SLI_ERR_SHAPE, "pass: more sequences than slots");
    if (!one) {
        M = kHyTile;
        while (M < n) M *= 2;
        for (const SegRef& g : segs) kt += seq_key_tiles(s, g.pos0, g.n);
        SLI_CHECK(kt <= hy_key_tiles_max(s), SLI_ERR_SHAPE, "pass: too many expanded rows");
        if (kt > 0) {  // (the grid of the expansion: a power of two, so that few graphs are captured)
            int p = M / kLatTile + 1;
            while (p < kt) p *= 2;
            kt = std::min(p, hy_key_tiles_max(s));
        }
    }
    std::vector<RowRef> rows(rows_in);
    rows.resize(M, RowRef{-1, 0, 0, 0});
    const int32_t ns = (int32_t)segs.size();
    SLI_HIP(hipMemcpyAsync(s->rows, rows.data(), sizeof(RowRef) * M, hipMemcpyHostToDevice, s->stream));
    SLI_HIP(hipMemcpyAsync(s->segs, segs.data(), sizeof(SegRef) * ns, hipMemcpyHostToDevice, s->stream));
    SLI_HIP(hipMemcpyAsync(s->nsegs, &ns, sizeof(ns), hipMemcpyHostToDevice, s->stream));
    const int msegs = one ? M : std::min(s->B, M / kHyTile);
    if (hidden_host) {  // eager, with a copy after every run
        HY_TRY(HY_DISPATCH(s, M, one, msegs, kt, embed()));
        for (size_t r = 0; r < s->runs.size(); ++r) {
            HY_TRY(HY_DISPATCH(s, M, one, msegs, kt, run(r)));
            SLI_HIP(hipMemcpy2DAsync(hidden_host + r * (size_t)n * s->D, sizeof(float) * s->D, s->x, sizeof(float) * s->Dp,
                                     sizeof(float) * s->D, n, hipMemcpyDeviceToHost, s->stream));
        }
    } else {
        auto& g = s->graphs[{one ? 0 : 1 + kt, M}];
        SLI_HIP(hipStreamSynchronize(s->stream));
        HY_TRY(hy_capture(s, g, M, one, msegs, kt));
        SLI_HIP(hipGraphLaunch(g.second, s->stream));
    }
    if (!want.empty()) {
        const int nw = (int)want.size();
        SLI_HIP(hipMemcpyAsync(s->widx, want.data(), sizeof(int32_t) * nw, hipMemcpyHostToDevice, s->stream));
        for (int w = 0; w < nw; w += kHyLogitRows) {
            const int n = std::min(kHyLogitRows, nw - w);
            HY_TRY(HY_DISPATCH(s, M, one, msegs, kt, logits(s->widx + w, n, s->lg)));
            SLI_HIP(hipMemcpyAsync(logits_host + (size_t)w * s->V, s->lg, sizeof(float) * (size_t)n * s->V,
                                   hipMemcpyDeviceToHost, s->stream));
        }
    }
    SLI_HIP(hipStreamSynchronize(s->stream));
    return SLI_OK;
}

// ---------------------------------------------------------------- bench helpers
__global__ void hy_fill_kernel(void* p, size_t n, int f16, uint32_t seed) {
    for (size_t i = blockIdx.x * (size_t)blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) {
        uint32_t h = (uint32_t)(i * 2654435761u) ^ seed;
        h ^= h >> 16, h *= 0x7feb352du, h ^= h >> 15;
        const float f = (float)(h & 0xFFFF) / 32768.0f - 1.0f;
        if (f16)
            ((__half*)p)[i] = __float2half_rn(f);
        else
            ((float*)p)[i] = f;
    }
}

int hy_fill_context(BlockStack* s, uint32_t seed, int) {
    for (HyRun& r : s->runs) {
        auto fill = [&](void* p, size_t n, int f16) {
            if (p) hipLaunchKernelGGL(hy_fill_kernel, dim3(1024), dim3(256), 0, s->stream, p, n, f16, seed);
        };
        fill(r.ring, (size_t)s->B * s->taps * s->Dp, 0);
        if (s->seq) {
            fill(r.kc, (size_t)s->B * s->T * s->seq->layers[r.layer].Rp, s->f16);
            SLI_HIP(hipGetLastError());
            continue;
        }
        const HyLayer& l = s->layers[r.layer];
        fill(r.S, (size_t)s->B * l.d.heads * l.nsl * l.d.dim * kRetCols, 0);
        const size_t n = (size_t)s->B * l.d.kv_heads * s->T * l.hd;
        fill(r.kc, n, s->f16);
        fill(r.vc, n, s->f16);
        SLI_HIP(hipGetLastError());
    }
    return SLI_OK;
}

void hy_step_bytes(const BlockStack* s, int B, double pos_sum, double* weight_bytes, double* state_bytes) {
    double w = (double)s->V * s->D * s->wb, k = 0.0;
    for (const HyRun& r : s->runs) {
        if (s->seq) {
            seq_step_bytes(s, r, B, pos_sum, &w, &k);
            continue;
        }
        const HyLayer& l = s->layers[r.layer];
        const sli_block_desc& d = l.d;
        w += s->wb * (2.0 * (l.e_g + d.ff) * s->D + (double)s->D * (l.mixw + d.ff));
        k += 4.0 * B * s->taps * s->D;
        if (d.mixer == SLI_MIX_ATTENTION)
            k += pos_sum * d.kv_heads * (d.dim + d.vdim) * (s->f16 ? 2 : 4);
        else
            k += 2.0 * 4.0 * B * d.heads * d.dim * d.vdim;
    }
    *weight_bytes = w;
    *state_bytes = k;
}

}  // namespace sli
