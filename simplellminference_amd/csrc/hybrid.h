// hybrid.h — block-stack models behind the engine's model handle (engine.hip): a decoder whose layers are described
// by data (sli_stack_config, include/sli.h), in one of two arrangements: parallel blocks x += mult * (mixer(c1) + ff(c2))
// with an attention or a retention mixer (hybrid.hip), or sequential sublayers x += norm(gate * sublayer(x)) with latent
// attention and a mixture of experts (hybrid_seq.hip); both with an input convolution (canon.h) and with blocks that may
// run several times with shared weights and one cache or state per run.
//
// The engine keeps what every model has (device decode state, prompts, history, graphs, greedy sampling); this file's
// functions are the forward pass over packed rows (step_state.h RowRef): a decode step has one row per sequence,
// a prompt pass up to kHyMaxRows rows of any portions.
#pragma once
#include <string>
#include <vector>

#include "common.h"
#include "step_state.h"

namespace sli {

constexpr int kHyMaxRows = 1024;  // rows of one pass
constexpr int kHyTile = 32;      // a portion's rows start at a multiple of this (one sequence per row tile)

struct BlockStack;

int hy_create(const sli_stack_config* cfg, hipStream_t stream, BlockStack** out);
void hy_destroy(BlockStack* s);
int hy_set_tensor(BlockStack* s, const std::string& name, const float* host, int64_t n);
int hy_init_synthetic(BlockStack* s, uint32_t seed);
int hy_fill_context(BlockStack* s, uint32_t seed, int upto);
// before a capture or an eager pass: every tensor is there, the folded coefficients and tables are uploaded
int hy_prepare(BlockStack* s);
int hy_runs(const BlockStack* s);
// A prompt pass also expands cached rows (latent attention): what a portion of n tokens at pos0 adds, and the most a pass
// may hold (one portion of kHyMaxRows rows always fits)
int hy_key_tiles(const BlockStack* s, int pos0, int n);
int hy_key_tiles_max(const BlockStack* s);

// Decode step of every slot, from the engine's device states: embedding .. logits [B][V] and the argmax keys
// (*nkeys per sequence at keys[b * key_ld]).
int hy_record_step(BlockStack* s, const DevState* st, int B, float* logits, unsigned long long* keys, int key_ld,
                   int* nkeys);
int hy_key_ld(const BlockStack* s, int B);

// One pass over given rows (at most kHyMaxRows): rows[i] and segs describe it (host copies are uploaded on the
// stream). Runs the layers; then, for each of n_want row indices, logits into logits_host [n_want][V].
// hidden_host (nullable): the residual rows after every layer run, [runs][n_rows][width].
// one: every portion is one token (a decode step).
int hy_pass(BlockStack* s, const std::vector<RowRef>& rows, const std::vector<SegRef>& segs, bool one,
            const std::vector<int32_t>& want, float* logits_host, float* hidden_host);

void hy_step_bytes(const BlockStack* s, int B, double pos_sum, double* weight_bytes, double* state_bytes);

}  // namespace sli
