// lv_block.h — block models (include/llava_hip.h, lv_block_model_upload) behind the session interface of lv_api.hip: weights
// and their layouts, the per-sequence state, and the two forms of a step (one token, a batch of tokens).
#pragma once

#include "lv_common.h"

namespace lv {

struct BlockModel;
struct BlockSession;

int block_model_create(hipStream_t st, const void *base, uint64_t base_size, const lv_block_hparams *hp, const lv_block_spec *blocks,
                       const lv_tensor_desc *table, uint32_t n_tensors, int compute, BlockModel **out);
void block_model_destroy(BlockModel *m);
uint64_t block_model_bytes(const BlockModel *m);
// layers as a sequence runs through them: each pass of a loop counts, and has a state of its own
uint32_t block_model_passes(const BlockModel *m);

int block_session_create(const BlockModel *m, hipStream_t st, BlockSession **out);
void block_session_destroy(BlockSession *s);
// room for positions 0 .. positions - 1
int block_session_reserve(BlockSession *s, uint32_t positions);
uint32_t block_session_position(const BlockSession *s);
// the state no longer stands at any position (a failed step): only a new sequence may follow
void block_session_invalidate(BlockSession *s);

// Where a traced step leaves the residual stream: rows of `stride` floats, row z of buffer `which` of a layer at
// slot(layer, which, z).  Null slot: not traced.
struct BlockTrace {
    float *base = nullptr;
    uint32_t rows = 0, stride = 0, kinds = 0;
    float *slot(uint32_t layer, int which, uint32_t row) const { return base + (((size_t)layer * kinds + which) * rows + row) * stride; }
};

// Token cfg[1 + idx] at position cfg[0] + idx, as launches on the session's stream (capturable).  logits: null or vocab floats.
int block_step_token(BlockSession *s, const uint32_t *cfg, uint32_t idx, float *logits, const BlockTrace *trace);
// Tokens cfg[1 + idx0] .. of the step at position pos on, n of them together.  logits_all: null or [n][vocab]; logits_last: null or
// vocab floats.
int block_step_batch(BlockSession *s, const uint32_t *cfg, uint32_t pos, uint32_t idx0, uint32_t n, float *logits_last, float *logits_all,
                     const BlockTrace *trace);
// to be called when a step's launches are on the stream: the state stands at pos from now on
void block_session_advance(BlockSession *s, uint32_t pos);

uint64_t block_state_bytes(const BlockSession *s, uint32_t layer, uint32_t n_tokens);
int block_state_copy(BlockSession *s, uint32_t layer, uint32_t n_tokens, void *host, bool write);

constexpr uint32_t kBlockBatch = 2048;   // tokens evaluated together at most
constexpr uint32_t kBlockBatchMin = 16;  // shorter steps go token by token

}  // namespace lv
