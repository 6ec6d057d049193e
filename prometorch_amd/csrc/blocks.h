// The layers of a block decoder (ptm_block_config): what ptm_decoder runs in place of its fixed layer shape.
#pragma once
#include "dense.h"

namespace ptm {

struct BlockStack;
int blocks_create(const ptm_block_config& cfg, BlockStack** out);
void blocks_destroy(BlockStack* b);
int blocks_runs(const BlockStack* b);
// Layers that carry state from token to token, which no position can be taken out of again.  blocks_state_copy keeps a copy of
// all of it, or puts the copy back.
bool blocks_recurrent(const BlockStack* b);
int blocks_state_copy(BlockStack* b, bool restore, hipStream_t s);
// One token (id in *d_token, position *d_past) through all layer runs.  trace: [runs][2][hidden], after the mixer branch and
// at the end of the layer.
int blocks_token(BlockStack* b, const int* d_token, const int64_t* d_past, float* trace, hipStream_t s);
// Scratch for chunks of up to `rows` prompt rows.
int blocks_reserve(BlockStack* b, int rows);
// M prompt rows at positions pos0 ..; trace: [runs][M][hidden], at the end of every layer.
int blocks_rows(BlockStack* b, const int* tokens_host, int M, int64_t pos0, float* trace, hipStream_t s);
// Final norm and vocabulary projection of the token (row < 0) or of prompt row `row`; adv: also the greedy argmax and the step's
// bookkeeping.
int blocks_head(BlockStack* b, int row, float* logits, float* xn, int64_t* d_next, void* argmax_ws, const ArgmaxAdvance* adv,
                hipStream_t s);

}  // namespace ptm
