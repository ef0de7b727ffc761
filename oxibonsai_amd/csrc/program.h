// program.h — layer programs: models described by a DesignConfig, run through the same model handle, cache manager, decode
// graph and token loops as the fixed Qwen3 sequence (model.hip calls these where a model carries a program).
#pragma once
#include "design.h"
#include "model_internal.h"
#include "safetensors.h"

namespace oxb {

static constexpr uint32_t kNoPosition = 0xFFFFFFFFu;

// Uploads the tensors, creates the model and its embedding table.  dt: OXB_DT_*.
int program_create(const DesignConfig& c, const TensorMap& tensors, int dt, uint32_t max_seq, uint32_t batch, uint64_t* model,
                   uint64_t* embedding);
void program_release(Program& p);
int program_check_handles(Model& m);
// One decode step of the whole batch on m.hidden / m.pos -> m.logits, m.tokens (capturable: allocates nothing).
int program_decode_step(Model& m);
int program_prefill_buffers(Model& m, uint32_t rows, uint32_t pos_start);
// M tokens of one sequence, embedding rows in m.pf_hidden.  Logits of the wanted rows (host indices into the portion; null:
// the last row only) -> d_logits [n_want][vocab]; n_want 0: none.
int program_prefill(Model& m, uint32_t seq, uint32_t M, uint32_t pos_start, const uint32_t* want, uint32_t n_want, float* d_logits);
// Recurrent memory: whether sequence `seq` can take tokens from position `pos` on, and where it stands afterwards
// (kNoPosition while a call is under way; 0 once its slot is free).
int program_begin(Model& m, uint32_t seq, uint32_t pos);
void program_commit(Model& m, uint32_t seq, uint32_t next);
// Bytes of cache per position over all layer runs.
size_t program_cache_row_bytes(const Program& p);

}  // namespace oxb
