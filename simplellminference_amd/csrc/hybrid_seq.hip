// hybrid_seq.hip — the sequential arrangement of block-stack models (hybrid.h): x <- x + norm1(rg1 * mixer(c)), then
// x <- x + norm2(rg2 * ff(x)), with latent attention (latent.h), a mixture of experts (moe.h), gated sublayers (gated.h)
// and an input convolution over the raw residual rows (canon.h). Layer set-up, weight placement and the recorded
// launches; hybrid.hip has what both arrangements share (embedding, head, passes, graphs).
//
// Fused weights of a layer: [q | latent down | gate ; rg1] over the model width (two inputs: the convolved row, the row
// itself), [U_k | U_v] over the latent, W_o, [rg2 | router] over the width, and the experts' gate / up pairs and downs.
#include <cmath>
#include <cstdlib>
#include <type_traits>

#include "gated.h"
#include "hybrid_gemv.h"
#include "hybrid_kernels.h"
#include "hybrid_rec.h"
#include "hybrid_stack.h"
#include "latent.h"
#include "moe.h"

namespace sli {

__device__ __forceinline__ float sigmoid_f(float v) { return 1.0f / (1.0f + expf(-v)); }

// ---------------------------------------------------------------- epilogues
// Row sections start at multiples of 4 rows, so four consecutive rows never straddle two of them.
struct SeqIn {  // [q | latent | gate ; residual gate]
    int Hq, dim, hq_ld;       // query rows; values and stride of a head in q
    int r_kv, R, Rp, r_g, Hv, r_rg, D, ld;
    float *q, *lat, *gate, *rg;
    const float* rgb;
    size_t q_ld;
    __device__ void put(int row, int m, float v) const {
        if (row >= r_rg) {
            const int i = row - r_rg;
            if (i < D) rg[(size_t)m * ld + i] = sigmoid_f(v + rgb[i]);
        } else if (row >= r_g) {
            const int i = row - r_g;
            if (i < Hv) gate[(size_t)m * Hv + i] = sigmoid_f(v);
        } else if (row >= r_kv) {
            const int i = row - r_kv;
            if (i < R) lat[(size_t)m * Rp + i] = v;
        } else if (row < Hq) {
            const int h = row / dim;
            q[m * q_ld + h * hq_ld + row - h * dim] = v;
        }
    }
    __device__ void pair(int u, int m, float v0, float v1) const {
        put(2 * u, m, v0);
        put(2 * u + 1, m, v1);
    }
    __device__ void pair2(int u, int m, const float* a, bool second) const {  // u even
        const int row = 2 * u;
        float* dst = nullptr;
        float4 y = make_float4(a[0], a[1], a[2], a[3]);
        if (row >= r_rg) {
            const int i = row - r_rg;
            if (i + 3 < D) {
                const float4 b = *reinterpret_cast<const float4*>(rgb + i);
                dst = rg + (size_t)m * ld + i;
                y = make_float4(sigmoid_f(y.x + b.x), sigmoid_f(y.y + b.y), sigmoid_f(y.z + b.z), sigmoid_f(y.w + b.w));
            }
        } else if (row >= r_g) {
            const int i = row - r_g;
            if (i + 3 < Hv && Hv % 4 == 0) {
                dst = gate + (size_t)m * Hv + i;
                y = make_float4(sigmoid_f(y.x), sigmoid_f(y.y), sigmoid_f(y.z), sigmoid_f(y.w));
            }
        } else if (row >= r_kv) {
            if (row - r_kv + 3 < R) dst = lat + (size_t)m * Rp + row - r_kv;
        } else if (row + 3 < Hq && dim % 4 == 0) {
            const int h = row / dim;
            dst = q + m * q_ld + h * hq_ld + row - h * dim;
        }
        if (dst) {
            *reinterpret_cast<float4*>(dst) = y;
            return;
        }
        pair(u, m, a[0], a[1]);
        if (second) pair(u + 1, m, a[2], a[3]);
    }
};

struct SeqGates {  // [rg2 ; router]
    float* rg;
    const float* rgb;
    int D, ld, z0, E;
    float* z;  // [M][E]
    const float* zb;
    __device__ void put(int row, int m, float v) const {
        if (row < D) rg[(size_t)m * ld + row] = sigmoid_f(v + rgb[row]);
        else if (row >= z0 && row - z0 < E) z[(size_t)m * E + row - z0] = v + zb[row - z0];
    }
    __device__ void pair(int u, int m, float v0, float v1) const {
        put(2 * u, m, v0);
        put(2 * u + 1, m, v1);
    }
    __device__ void pair2(int u, int m, const float* a, bool second) const {  // u even
        if (2 * u + 3 < D) {
            const float4 b = *reinterpret_cast<const float4*>(rgb + 2 * u);
            *reinterpret_cast<float4*>(rg + (size_t)m * ld + 2 * u) =
                make_float4(sigmoid_f(a[0] + b.x), sigmoid_f(a[1] + b.y), sigmoid_f(a[2] + b.z), sigmoid_f(a[3] + b.w));
            return;
        }
        pair(u, m, a[0], a[1]);
        if (second) pair(u + 1, m, a[2], a[3]);
    }
};

// ---------------------------------------------------------------- set-up
static int seq_layer_init(BlockStack* s, SeqLayer& l, int i) {
    const sli_block_desc& d = l.d;
    const std::string at = "block " + std::to_string(i) + ": ";
    SLI_CHECK(d.mixer == SLI_MIX_LATENT, SLI_ERR_ARG, at + "a sequential block mixes with latent attention");
    SLI_CHECK(d.heads > 0 && d.dim > 0 && d.vdim > 0 && d.kv_rank > 0 && d.window >= 0, SLI_ERR_SHAPE,
              at + "non-positive size");
    SLI_CHECK(d.kv_rank <= kLatMaxRank, SLI_ERR_SHAPE, at + "kv_rank must be at most 2048");
    SLI_CHECK(d.ff >= 0 && (d.ff == 0) == (d.experts == 0), SLI_ERR_SHAPE,
              at + "a sequential block's feed-forward is a mixture (ff and experts), or none");
    SLI_CHECK(d.experts == 0 || (d.experts > 0 && d.experts <= kMoeMaxExperts && d.top > 0 && d.top <= d.experts &&
                                 d.top <= kMoeMaxTop),
              SLI_ERR_SHAPE, at + "bad experts / top");
    l.window = d.window > 0 ? std::min(d.window, s->T) : s->T;
    l.Hq = d.heads * d.dim;
    l.Hv = d.heads * d.vdim;
    l.R = d.kv_rank;
    l.Rp = pad_to(l.R, 64);
    l.r_kv = pad_to(l.Hq, 4);
    l.r_g = l.r_kv + pad_to(l.R, 4);
    l.n1 = (l.r_g + pad_to(l.Hv, 4)) / 2;
    l.u1p = pad_to(l.n1, kHySection);
    l.v0 = pad_to(l.Hq, 4);
    l.KA = pad_to(l.Hv, 64);
    const int w = std::max(d.dim, d.vdim);
    l.hd = !s->f16 || w > 128 ? 0 : w <= 64 ? 64 : 128;
    l.z0 = pad_to(s->D, 4);
    l.n2 = (l.z0 + d.experts + 1) / 2;
    l.ffp = pad_to(d.ff, 8);
    l.FFp = pad_to(d.ff, 64);
    l.Dn = pad_to(s->D, 16);
    return SLI_OK;
}

static int bm_for(const BlockStack* s, int M, int top, int E) {
    const int per = M * top / E;
    return s->f16 ? HyProj<__half>::group_rows(per) : HyProj<float>::group_rows(per);
}
static int lat_splits(const SeqLayer& l, int M) {
    const int tiles = (l.window + kLatKeys - 1) / kLatKeys, hg = (l.d.heads + kLatHeads - 1) / kLatHeads;
    return std::max(1, std::min({tiles, kLatMaxSplits, device_cus() / std::max(1, M * hg)}));
}

static int seq_allow_lds();

int seq_create(BlockStack* s) {
    const sli_stack_config& c = s->c;
    SeqState& q = *s->seq;
    q.layers.resize(c.n_blocks);
    const size_t wb = s->wb, M = s->M;
    const int D = s->D, Dp = s->Dp, Bp = s->f16 ? HyProj<__half>::rows_for(s->B) : s->B;
    std::map<int, float*> by_rank;
    std::map<int, SeqLayer*> by_v, by_ff;
    std::map<std::pair<int, int>, float*> by_q;
    size_t qf = 0, qa = 0, part = 0, gate = 0, nz = 0, pairs = 0, erows = 0, etiles = 0, kv = 0, wmax = 0;
    for (int i = 0; i < c.n_blocks; ++i) {
        SeqLayer& l = q.layers[i];
        l.d = c.blocks[i];
        HY_TRY(seq_layer_init(s, l, i));
        const sli_block_desc& d = l.d;
        const std::string p = "l" + std::to_string(i) + ".";
        for (const char* n : {"norm1", "canon1", "rg1", "rg1.b", "mix.q", "mix.dkv", "mix.dkv.norm", "mix.uk", "mix.uv", "mix.g",
                              "mix.o"})
            s->want[p + n] = false;
        HY_TRY(hy_alloc(s, &l.win, wb * (size_t)(2 * l.u1p + pad_to(D, 128)) * Dp));
        HY_TRY(hy_alloc(s, &l.ukv, wb * (size_t)pad_to(l.v0 + l.Hv, 128) * l.Rp));
        HY_TRY(hy_alloc(s, &l.wo, wb * (size_t)pad_to(D, 128) * l.KA));
        HY_TRY(hy_new(s, &l.f1, (size_t)s->taps * Dp));
        HY_TRY(hy_new(s, &l.lnorm, (size_t)l.Rp));
        HY_TRY(hy_new(s, &l.rg1b, (size_t)Dp));
        HY_TRY(hy_new(s, &l.w1, (size_t)Dp));
        if (d.experts > 0) {
            for (const char* n : {"norm2", "rg2", "rg2.b", "mlp.router", "mlp.router.b"}) s->want[p + n] = false;
            for (int e = 0; e < d.experts; ++e)
                for (const char* n : {"gate", "up", "down"}) s->want[p + "mlp.e" + std::to_string(e) + "." + n] = false;
            HY_TRY(hy_alloc(s, &l.wg2, wb * (size_t)pad_to(2 * l.n2, 128) * Dp));
            HY_TRY(hy_alloc(s, &l.wup, wb * (size_t)d.experts * 2 * l.ffp * Dp));
            HY_TRY(hy_alloc(s, &l.wdn, wb * (size_t)d.experts * l.Dn * l.FFp));
            HY_TRY(hy_new(s, &l.rg2b, (size_t)Dp));
            HY_TRY(hy_new(s, &l.w2, (size_t)Dp));
            HY_TRY(hy_new(s, &l.zb, (size_t)d.experts));
            for (int m = 1; m <= (int)M; ++m) {
                const int bm = bm_for(s, m, d.top, d.experts), t = moe_max_tiles(m * d.top, d.experts, bm);
                erows = std::max(erows, (size_t)t * bm);
                etiles = std::max(etiles, (size_t)t);
            }
            pairs = std::max(pairs, M * d.top);
            nz = std::max(nz, M * d.experts);
            HY_TRY(hy_bg_need(s, l.n2, Dp));
        }
        HY_TRY(hy_bg_need(s, l.n1, Dp));
        HY_TRY(hy_bg_need(s, (D + 1) / 2, Dp));
        HY_TRY(hy_bg_need(s, (D + 1) / 2, l.KA));
        float*& lat = by_rank[l.R];
        if (!lat) HY_TRY(hy_new(s, &lat, M * l.Rp));
        l.lat = lat;
        SeqLayer*& sv = by_v[l.Hv];
        if (sv) {
            l.cat32 = sv->cat32, l.cat16 = sv->cat16;
        } else {
            HY_TRY(hy_new(s, &l.cat32, M * l.KA));
            if (s->f16) HY_TRY(hy_new(s, &l.cat16, M * l.KA));
            sv = &l;
        }
        // absorbed attention: the rows of a decode step, or (no expanded form) of any pass
        const size_t ra = l.hd ? (size_t)Bp : std::max(M, (size_t)Bp);
        qf = std::max(qf, ra * l.Hq);
        qa = std::max(qa, ra * d.heads * l.Rp);
        size_t sp = 1;
        for (int m = 1; m <= Bp; ++m) sp = std::max(sp, (size_t)m * lat_splits(l, m));
        part = std::max(part, std::max(ra, sp) * d.heads * (l.Rp + kAttnPartPad));
        gate = std::max(gate, M * l.Hv);
        if (l.hd) {
            float*& qb = by_q[{d.heads, d.dim * 256 + l.hd}];
            if (!qb) HY_TRY(hy_new(s, &qb, M * d.heads * l.hd));
            l.q = qb;
            kv = std::max(kv, (size_t)d.heads * l.hd);
            wmax = std::max(wmax, (size_t)l.window);
            for (size_t w = 0; w < q.wins.size(); ++w)
                if (q.wins[w].window == l.window) l.win_id = (int)w;
            if (l.win_id < 0) {
                l.win_id = (int)q.wins.size();
                q.wins.push_back(SeqWindow{l.window});
            }
        }
    }
    for (SeqLayer& l : q.layers) {  // (the rows of the largest batch of experts)
        if (l.d.experts == 0) continue;
        SeqLayer*& sf = by_ff[l.d.ff];
        if (sf) {
            l.act32 = sf->act32, l.act16 = sf->act16;
            continue;
        }
        HY_TRY(hy_new(s, &l.act32, (s->f16 ? (size_t)kMoeFusedTop : std::max(erows, (size_t)kMoeFusedTop)) * l.FFp));
        if (s->f16) HY_TRY(hy_new(s, &l.act16, erows * l.FFp));
        sf = &l;
    }
    for (HyRun& r : s->runs) {
        const SeqLayer& l = q.layers[r.layer];
        HY_TRY(hy_new(s, &r.ring, (size_t)s->B * s->taps * Dp));
        // (tiles of the expansion may read up to one tile past the last row)
        HY_TRY(hy_alloc(s, &r.kc, wb * ((size_t)s->B * s->T + kLatTile) * l.Rp));
    }
    if (kv > 0) {
        // one portion of a whole pass always fits; more portions up to 32768 rows or what a batch can need
        const int one = (int)std::min<size_t>(wmax + M, (size_t)s->T) / kLatTile + 2;
        const int any = std::min(s->B, kHyMaxRows / kHyTile) * (int)(std::min<size_t>(wmax, (size_t)s->T) / kLatTile + 2) +
                        kHyMaxRows / kLatTile;
        q.key_tiles = std::max(one, std::min(any, 32768 / kLatTile));
        for (SeqWindow& w : q.wins) {
            HY_TRY(hy_new(s, &w.tiles, (size_t)q.key_tiles));
            HY_TRY(hy_new(s, &w.ntiles, 1));
            HY_TRY(hy_new(s, &w.koff, M / 32));
        }
        HY_TRY(hy_new(s, &q.ks, kv * q.key_tiles * kLatTile));
        HY_TRY(hy_new(s, &q.vs, kv * q.key_tiles * kLatTile));
    }
    HY_TRY(hy_new(s, &q.x2, (size_t)Dp));
    HY_TRY(hy_new(s, &q.zeros, (size_t)Dp));
    HY_TRY(hy_new(s, &q.qf, qf));
    HY_TRY(hy_new(s, &q.qa, qa));
    HY_TRY(hy_new(s, &q.part, part));
    HY_TRY(hy_new(s, &q.gate, gate));
    HY_TRY(hy_new(s, &q.rg1, M * Dp));
    HY_TRY(hy_new(s, &q.rg2, M * Dp));
    HY_TRY(hy_new(s, &q.y, M * Dp));
    HY_TRY(hy_new(s, &q.z, nz));
    HY_TRY(hy_new(s, &q.sel, pairs));
    HY_TRY(hy_new(s, &q.at, pairs));
    HY_TRY(hy_new(s, &q.wsel, pairs));
    HY_TRY(hy_new(s, &q.rowmap, erows));
    HY_TRY(hy_new(s, &q.tiles, etiles));
    HY_TRY(hy_new(s, &q.ntiles, 1));
    HY_TRY(hy_new(s, &q.ye, erows * Dp));
    if (s->f16) HY_TRY(hy_new(s, &q.xh, M * Dp));
    return seq_allow_lds();
}

// ---------------------------------------------------------------- weights
void seq_shape(const BlockStack* s, int i, const std::string& t, int64_t* rows, int64_t* cols) {
    const SeqLayer& l = s->seq->layers[i];
    auto set = [&](int64_t r, int64_t c) { *rows = r, *cols = c; };
    if (t == "norm1" || t == "norm2" || t == "rg1.b" || t == "rg2.b") set(1, s->D);
    else if (t == "canon1") set(s->D, s->c.taps);
    else if (t == "rg1" || t == "rg2") set(s->D, s->D);
    else if (t == "mix.q") set(l.Hq, s->D);
    else if (t == "mix.dkv") set(l.R, s->D);
    else if (t == "mix.dkv.norm") set(1, l.R);
    else if (t == "mix.uk") set(l.Hq, l.R);
    else if (t == "mix.uv") set(l.Hv, l.R);
    else if (t == "mix.g") set(l.Hv, s->D);
    else if (t == "mix.o") set(s->D, l.Hv);
    else if (t == "mlp.router") set(l.d.experts, s->D);
    else if (t == "mlp.router.b") set(1, l.d.experts);
    else if (t.compare(0, 5, "mlp.e") == 0) t.back() == 'n' ? set(s->D, l.d.ff) : set(l.d.ff, s->D);  // down, or gate and up
}

int seq_put(BlockStack* s, int i, const std::string& t, const HyFill& f) {
    SeqLayer& l = s->seq->layers[i];
    const int D = s->D, Dp = s->Dp;
    auto vec = [&](float* dst, int n) -> int {
        SLI_HIP(hipMemcpy(dst, f.host, sizeof(float) * n, hipMemcpyHostToDevice));
        return SLI_OK;
    };
    auto mat = [&](void* dst, int ld, int n, int first, int step, int cols) {
        return hy_place(s, dst, ld, 0, strided_rows(n, first, step), cols, f);
    };
    if (t == "norm1") return vec(l.w1, D);
    if (t == "norm2") return vec(l.w2, D);
    if (t == "rg1.b") return vec(l.rg1b, D);
    if (t == "rg2.b") return vec(l.rg2b, D);
    if (t == "mix.dkv.norm") return vec(l.lnorm, l.R);
    if (t == "mlp.router.b") return vec(l.zb, l.d.experts);
    if (t == "canon1") {
        l.c1.assign(f.host, f.host + (size_t)D * s->c.taps);
        return SLI_OK;
    }
    if (t == "mix.q") return mat(l.win, Dp, l.Hq, 0, 1, D);
    if (t == "mix.dkv") return mat(l.win, Dp, l.R, l.r_kv, 1, D);
    if (t == "mix.g") return mat(l.win, Dp, l.Hv, l.r_g, 1, D);
    if (t == "rg1") return mat(l.win, Dp, D, 2 * l.u1p, 1, D);
    if (t == "mix.uk") return mat(l.ukv, l.Rp, l.Hq, 0, 1, l.R);
    if (t == "mix.uv") return mat(l.ukv, l.Rp, l.Hv, l.v0, 1, l.R);
    if (t == "mix.o") return mat(l.wo, l.KA, D, 0, 1, l.Hv);
    if (t == "rg2") return mat(l.wg2, Dp, D, 0, 1, D);
    if (t == "mlp.router") return mat(l.wg2, Dp, l.d.experts, l.z0, 1, D);
    const int e = std::atoi(t.c_str() + 5);  // mlp.e<e>.{gate,up,down}
    if (t.back() == 'n') return mat(l.wdn, l.FFp, D, e * l.Dn, 1, l.d.ff);
    return mat(l.wup, Dp, l.d.ff, 2 * e * l.ffp + (t.back() == 'p' ? 1 : 0), 2, D);
}

int seq_prepare(BlockStack* s) {
    for (SeqLayer& l : s->seq->layers) HY_TRY(hy_fold_taps(s, l.c1, 1.0f, l.f1));
    return SLI_OK;
}

int seq_key_tiles(const BlockStack* s, int pos0, int n) {
    int t = 0;
    if (s->seq)
        for (const SeqWindow& w : s->seq->wins) t = std::max(t, lat_tiles(pos0, n, w.window));
    return t;
}

void seq_step_bytes(const BlockStack* s, const HyRun& r, int B, double pos_sum, double* weights, double* state) {
    const SeqLayer& l = s->seq->layers[r.layer];
    const sli_block_desc& d = l.d;
    const double D = s->D;
    double w = (l.Hq + l.R + l.Hv + D) * D + (double)(l.Hq + l.Hv) * l.R + D * l.Hv;
    if (d.experts > 0) {  // experts a batch uses, were the choices independent and even
        const double used = d.experts * (1.0 - std::pow(1.0 - (double)d.top / d.experts, B));
        w += (D + d.experts) * D + used * 3.0 * d.ff * D;
    }
    *weights += w * s->wb;
    *state += B * std::min(pos_sum / B, (double)l.window) * l.R * s->wb + 4.0 * B * s->taps * D;
}

// ---------------------------------------------------------------- the recorded launches
template <typename WT>
struct SeqRec : HyProj<WT> {
    using P = HyProj<WT>;
    using P::F16, P::s, P::M, P::one, P::key_tiles, P::st, P::project, P::pgemm, P::grouped;
    SeqState& q() const { return *s->seq; }

    // what the last sublayer leaves for the next launch: the row before it, its result, gate and norm gains
    struct Pending {
        float* x;
        const float *y, *g, *w;
    };

    CanonArgs canon(const SeqLayer& l, const HyRun& r) const {
        return CanonArgs{s->x, r.ring, l.f1, nullptr, s->rows, s->c.eps, s->D, s->Dp, s->taps, M, true};
    }
    bool absorbed(const SeqLayer& l) const { return one || l.hd == 0; }
    SeqIn in_epi(const SeqLayer& l) const {
        const bool flat = absorbed(l);
        SeqIn e{};
        e.Hq = l.Hq, e.dim = l.d.dim, e.hq_ld = flat ? l.d.dim : l.hd;
        e.r_kv = l.r_kv, e.R = l.R, e.Rp = l.Rp, e.r_g = l.r_g, e.Hv = l.Hv, e.r_rg = 2 * l.u1p, e.D = s->D, e.ld = s->Dp;
        e.q = flat ? q().qf : l.q;
        e.lat = l.lat, e.gate = q().gate, e.rg = q().rg1, e.rgb = l.rg1b;
        e.q_ld = flat ? (size_t)l.Hq : (size_t)l.d.heads * l.hd;
        return e;
    }
    SeqGates gate_epi(const SeqLayer& l) const {
        return SeqGates{q().rg2, l.rg2b, s->D, s->Dp, l.z0, (int)l.d.experts, q().z, l.zb};
    }
    GatedArgs gated(const Pending& p, float* xout) const {
        GatedArgs a{};
        a.x = p.x, a.y = p.y, a.g = p.g, a.w = p.w, a.xout = xout;
        a.eps = s->c.eps, a.D = s->D, a.ld = s->Dp, a.rows = s->rows;
        return a;
    }
    LatArgs lat(const SeqLayer& l, const HyRun& r) const {
        LatArgs a{};
        a.lat = l.lat, a.lnorm = l.lnorm, a.cache = r.kc, a.rows = s->rows, a.q = q().qf;
        a.uk = l.ukv, a.uv = (const WT*)l.ukv + (size_t)l.v0 * l.Rp, a.qa = q().qa, a.part = q().part, a.gate = q().gate;
        a.H = l.d.heads, a.dim = l.d.dim, a.vdim = l.d.vdim, a.R = l.R, a.Rp = l.Rp, a.T = s->T, a.window = l.window;
        a.splits = mfma_decode(l) ? lat_splits(l, M) : 1;
        a.scale = l.d.scale, a.eps = s->c.eps;
        return a;
    }
    bool mfma_decode(const SeqLayer& l) const { return F16 && one && l.Rp <= kLatMfmaRank; }

    template <int NB>
    int attn_mfma(const LatArgs& a) const {
        if constexpr (F16) {
            const dim3 gr(a.splits, (a.H + kLatHeads - 1) / kLatHeads, M);
            hipLaunchKernelGGL(lat_attn_kernel<NB>, gr, dim3(256), LatGeo<NB>::LDS, st(), a);
            SLI_HIP(hipGetLastError());
        }
        return SLI_OK;
    }
    template <class F>
    static int rank_pick(int Rp, F&& f) {
        switch (Rp / 64) {
            case 1: return f(std::integral_constant<int, 1>{});
            case 2: return f(std::integral_constant<int, 2>{});
            case 3: return f(std::integral_constant<int, 3>{});
            case 4: return f(std::integral_constant<int, 4>{});
            case 5: return f(std::integral_constant<int, 5>{});
            case 6: return f(std::integral_constant<int, 6>{});
            case 7: return f(std::integral_constant<int, 7>{});
            case 8: return f(std::integral_constant<int, 8>{});
        }
        return fail(SLI_ERR_SHAPE, "latent attention: rank past the matrix-core form");
    }
    // projections of the convolved row are in place -> cat: gated heads, the output projection's input
    template <typename OT>
    int mixer(const SeqLayer& l, const HyRun& r, OT* cat) const {
        const sli_block_desc& d = l.d;
        const LatArgs a = lat(l, r);
        if (absorbed(l)) {
            const int nch = (l.Rp + kLatCols - 1) / kLatCols;
            hipLaunchKernelGGL((lat_rows_kernel<WT, WT>), dim3(1 + d.heads * nch, M), dim3(256), 0, st(), a);
            SLI_HIP(hipGetLastError());
            if (mfma_decode(l)) {
                HY_TRY(rank_pick(l.Rp, [&](auto nb) { return attn_mfma<decltype(nb)::value>(a); }));
            } else {
                hipLaunchKernelGGL(lat_attn_rows_kernel<WT>, dim3(d.heads, M), dim3(256), lat_rows_lds(l.Rp), st(), a);
                SLI_HIP(hipGetLastError());
            }
            hipLaunchKernelGGL((lat_out_kernel<WT, OT>), dim3((d.vdim + kLatOutRows - 1) / kLatOutRows, d.heads, M), dim3(256),
                               lat_out_lds(l.Rp), st(), a, cat, l.KA);
            SLI_HIP(hipGetLastError());
            return SLI_OK;
        }
        hipLaunchKernelGGL((lat_rows_kernel<WT, WT>), dim3(1, M), dim3(256), 0, st(), a);
        SLI_HIP(hipGetLastError());
        if constexpr (std::is_same<OT, __half>::value) {
            const SeqWindow& w = q().wins[l.win_id];
            const int cap = q().key_tiles * kLatTile;
            PgGroups g{};
            g.tiles = w.tiles, g.ntiles = w.ntiles;
            const LatExpand e{q().ks, q().vs, l.Hq, (int)d.dim, l.Hv, (int)d.vdim, l.v0, cap, l.hd};
            HY_TRY(grouped(l.ukv, r.kc, l.Rp, (l.v0 + l.Hv + 1) / 2, g, kLatTile, key_tiles, e));
            const PfAttnArgs<__half> pa{l.q, q().ks, q().vs, cat, nullptr, (int)d.heads, (int)d.heads, cap, d.scale};
            PfRowsArgs px{};
            px.rows = s->rows, px.ldo = l.KA, px.vdim = d.vdim, px.window = l.window, px.koff = w.koff, px.gate = q().gate;
            const dim3 gr(M / 16, d.heads);
            if (l.hd == 64)
                hipLaunchKernelGGL((pf_attn_mfma_kernel<64, 2>), gr, dim3(256), 0, st(), pa, nullptr, px);
            else
                hipLaunchKernelGGL((pf_attn_mfma_kernel<128, 2>), gr, dim3(256), 0, st(), pa, nullptr, px);
            SLI_HIP(hipGetLastError());
            return SLI_OK;
        } else {
            return fail(SLI_ERR_STATE, "expanded attention: fp16 prompt passes");
        }
    }

    // ---- one row: the layer as eight launches, each sublayer's residual add and norm in the next launch's input stage
    bool fits_fused(const SeqLayer& l) const {
        const sli_block_desc& d = l.d;
        if (M != 1 || !one || s->taps != kCanonFusedTaps || s->Dp > 4 * kGemvThreads || l.KA > kGemvMaxCols) return false;
        if (d.experts == 0) return true;
        return d.experts <= kMoeFusedExperts && d.top <= kMoeFusedTop &&
               moe_down_lds(l.FFp, d.top, s->D, gemv_blocks(s->D, d.top)) <= kMoeLdsMax;
    }
    bool fused() const {
        for (const SeqLayer& l : q().layers)
            if (!fits_fused(l)) return false;
        return true;
    }
    int layer_fused(const HyRun& r, Pending& p) const {
        const SeqLayer& l = q().layers[r.layer];
        const sli_block_desc& d = l.d;
        auto other = [&](const float* x) { return x == s->x ? q().x2 : s->x; };
        float* x1 = other(p.x);
        const GatedStageArgs sa{gated(p, x1), canon(l, r), s->Dp};
        SLI_HIP((launch_hy_in<WT, XStageGatedCanon>((const WT*)l.win, sa, in_epi(l), l.n1, l.u1p, (s->D + 1) / 2, st())));
        HY_TRY(mixer<float>(l, r, l.cat32));
        GemvIn in{l.cat32, nullptr, 0.0f, l.KA};
        SLI_HIP((launch_gemv_u<WT, 1, 6, true>((const WT*)l.wo, in, EpiStore<1>{q().y, nullptr, nullptr, 1.0f, s->D}, s->D, st())));
        p = Pending{x1, q().y, q().rg1, l.w1};
        if (d.experts == 0) return SLI_OK;
        float* x2 = other(p.x);
        const GatedStageArgs sb{gated(p, x2), CanonArgs{}, s->Dp};
        SLI_HIP((launch_hy_in<WT, XStageGated>((const WT*)l.wg2, sb, gate_epi(l), l.n2, 0, 0, st())));
        const EpiMoeUp up{q().z, (int)d.experts, (int)d.top, (int)d.ff, l.ffp, l.FFp, l.act32, q().sel, q().wsel, nullptr};
        SLI_HIP(launch_moe_up<WT>((const WT*)l.wup, x2, s->Dp, up, st()));
        const EpiMoeDown dn{q().sel, (int)d.top, l.Dn, s->D, q().y, nullptr};
        SLI_HIP(launch_moe_down<WT>((const WT*)l.wdn, l.act32, q().wsel, l.FFp, dn, st()));
        p = Pending{x2, q().y, q().rg2, l.w2};
        return SLI_OK;
    }
    int add_rows(const GatedArgs& a, bool mix) const {
        if (mix)
            hipLaunchKernelGGL(gated_rows_kernel<true>, dim3(M), dim3(256), gated_lds(a.ld), st(), a);
        else
            hipLaunchKernelGGL(gated_rows_kernel<false>, dim3(M), dim3(256), gated_lds(a.ld), st(), a);
        SLI_HIP(hipGetLastError());
        return SLI_OK;
    }

    // the choices of a pass and its expert rows' layout
    template <int NV>
    int route(const MoeRoute& r, int bm) const {
        if (M <= kMoeGroupRoutes) {
            hipLaunchKernelGGL(moe_group_kernel<NV>, dim3(1), dim3(1024), 0, st(), r, bm, q().at, q().rowmap, q().tiles,
                               q().ntiles);
        } else {
            hipLaunchKernelGGL(moe_topk_kernel<NV>, dim3((M + 3) / 4), dim3(256), 0, st(), r);
            SLI_HIP(hipGetLastError());
            hipLaunchKernelGGL(moe_group_kernel<0>, dim3(1), dim3(1024), 0, st(), r, bm, q().at, q().rowmap, q().tiles,
                               q().ntiles);
        }
        SLI_HIP(hipGetLastError());
        return SLI_OK;
    }

    // ---- any rows
    template <typename OT>
    int layer_rows(const HyRun& r) const {
        constexpr bool half = std::is_same<OT, __half>::value;
        const SeqLayer& l = q().layers[r.layer];
        const sli_block_desc& d = l.d;
        const CanonArgs ca = canon(l, r);
        SLI_HIP((launch_canon_rows<OT>(ca, (OT*)s->c1, half ? (OT*)s->c2 : (OT*)nullptr, one ? 1 : 0, st())));
        if (!one) {
            hipLaunchKernelGGL(canon_ring_kernel, dim3(M), dim3(256), 0, st(), ca);
            SLI_HIP(hipGetLastError());
        }
        const SeqIn ei = in_epi(l);
        const int np = (s->D + 1) / 2;
        OT* cat;
        if constexpr (half) {
            HY_TRY(pgemm((const WT*)l.win, (const __half*)s->c1, (const __half*)s->c2, l.u1p, s->Dp, l.u1p + np, 0, ei));
            cat = l.cat16;
        } else {
            HY_TRY(project(l.win, s->c1, s->Dp, l.n1, 0, ei));
            HY_TRY(project(l.win, s->x, s->Dp, np, l.u1p, ei));
            cat = l.cat32;
        }
        HY_TRY(mixer<OT>(l, r, cat));
        HY_TRY(project(l.wo, cat, l.KA, np, 0, HyStore{q().y, s->Dp, s->D}));
        GatedArgs a = gated(Pending{s->x, q().y, q().rg1, l.w1}, s->x);
        a.xh = q().xh;
        HY_TRY(add_rows(a, false));
        if (d.experts == 0) return SLI_OK;

        const void* xin = half ? (const void*)q().xh : (const void*)s->x;
        if constexpr (half) {
            HY_TRY(project(l.wg2, xin, s->Dp, np, 0, gate_epi(l)));
            hipLaunchKernelGGL(moe_router_kernel, dim3(M / 16, (d.experts + 15) / 16), dim3(256), 0, st(),
                               (const __half*)l.wg2 + (size_t)l.z0 * s->Dp, q().xh, l.zb, s->Dp, (int)d.experts, q().z);
            SLI_HIP(hipGetLastError());
        } else {
            HY_TRY(project(l.wg2, xin, s->Dp, l.n2, 0, gate_epi(l)));
        }
        const int E = d.experts, top = d.top, bm = bm_for(s, M, top, E), mt = moe_max_tiles(M * top, E, bm);
        const MoeRoute mr{q().z, s->rows, M, E, top, q().sel, q().wsel};
        HY_TRY(E <= 64 ? route<1>(mr, bm) : E <= 256 ? route<4>(mr, bm) : route<kMoeMaxExperts / 64>(mr, bm));
        PgGroups g{};
        g.tiles = q().tiles, g.ntiles = q().ntiles, g.rowmap = q().rowmap, g.wstride = (size_t)2 * l.ffp * s->Dp;
        PgGroups gd = g;
        gd.rowmap = nullptr, gd.wstride = (size_t)l.Dn * l.FFp;
        const HyStore ed{q().ye, s->Dp, s->D};
        if constexpr (F16) {
            HY_TRY(grouped(l.wup, q().xh, s->Dp, d.ff, g, bm, mt, MoeAct<__half>{l.act16, l.FFp, (int)d.ff}));
            HY_TRY(grouped(l.wdn, l.act16, l.FFp, np, gd, bm, mt, ed));
        } else {
            HY_TRY(grouped(l.wup, s->x, s->Dp, d.ff, g, bm, mt, MoeAct<float>{l.act32, l.FFp, (int)d.ff}));
            HY_TRY(grouped(l.wdn, l.act32, l.FFp, np, gd, bm, mt, ed));
        }
        a = gated(Pending{s->x, q().ye, q().rg2, l.w2}, s->x);
        a.at = q().at, a.wsel = q().wsel, a.top = top;
        return add_rows(a, true);
    }
    int layout() const {  // prompts: where each window's expanded rows go
        if (one) return SLI_OK;
        for (const SeqWindow& w : q().wins) {
            hipLaunchKernelGGL(lat_tiles_kernel, dim3(1), dim3(1024), 0, st(), s->segs, s->nsegs, s->T, w.window, w.tiles, w.ntiles,
                               w.koff);
            SLI_HIP(hipGetLastError());
        }
        return SLI_OK;
    }
    int runs(size_t r0, size_t r1) const {
        if (fused()) {
            Pending p{s->x, q().zeros, q().zeros, q().zeros};
            for (size_t r = r0; r < r1; ++r) HY_TRY(layer_fused(s->runs[r], p));
            return add_rows(gated(p, s->x), false);
        }
        HY_TRY(layout());
        for (size_t r = r0; r < r1; ++r) {
            if constexpr (F16) {
                HY_TRY(M > kBgMaxBatch ? layer_rows<__half>(s->runs[r]) : layer_rows<float>(s->runs[r]));
            } else {
                HY_TRY(layer_rows<float>(s->runs[r]));
            }
        }
        return SLI_OK;
    }
    static int allow_all() {
        HY_TRY((P::template allow<SeqIn>()));
        HY_TRY((P::template allow<SeqGates>()));
        HY_TRY((P::template allow<HyStore>()));
        HY_TRY((P::template allow_grouped<HyStore>()));
        HY_TRY((P::template allow_grouped<MoeAct<__half>>()));
        HY_TRY((P::template allow_grouped<LatExpand>()));
        for (int nb = 1; nb <= kLatMfmaRank / 64; ++nb)
            HY_TRY(rank_pick(64 * nb, [&](auto n) -> int {
                constexpr int NB = decltype(n)::value;
                SLI_HIP(hipFuncSetAttribute(reinterpret_cast<const void*>(&lat_attn_kernel<NB>),
                                            hipFuncAttributeMaxDynamicSharedMemorySize, LatGeo<NB>::LDS));
                return SLI_OK;
            }));
        return SLI_OK;
    }
};

static int seq_allow_lds() {
    SLI_HIP(moe_allow_lds<__half>());
    SLI_HIP(moe_allow_lds<float>());
    for (const void* k : {reinterpret_cast<const void*>(&gated_rows_kernel<true>),
                          reinterpret_cast<const void*>(&gated_rows_kernel<false>)})
        SLI_HIP(hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024));
    return SeqRec<__half>::allow_all();
}

#define SEQ_DISPATCH(s, M, one, msegs, kt, CALL)                           \
    ((s)->f16 ? SeqRec<__half>{{(s), (M), (one), (msegs), (kt)}}.CALL \
              : SeqRec<float>{{(s), (M), (one), (msegs), (kt)}}.CALL)

int seq_pass(BlockStack* s, int M, bool one, int msegs, int key_tiles) {
    return SEQ_DISPATCH(s, M, one, msegs, key_tiles, runs(0, s->runs.size()));
}
int seq_run(BlockStack* s, int M, bool one, int msegs, int key_tiles, size_t run) {
    return SEQ_DISPATCH(s, M, one, msegs, key_tiles, runs(run, run + 1));
}

}  // namespace sli
