// Sessions over a mixed layer stack: every layer described by itself (include/nerva_hip_api.h, NervaHipStackLayer).
// The session object, its lifecycle, sampler, slots and graphs are decode_session.hip's; here are the weights' layout,
// the cache and state of such a stack, and its two ways through the layers:
//   a decode step (16-bit precision): per sublayer a weight-streaming GEMV whose prologue is the seam between the
//     sublayers and whose epilogue is the activation or the recurrence (gemv_stream.cuh), attention in between; in
//     parallel layers of attention over latents and experts what does not wait for each other shares a launch
//     (gemv_layer.cuh);
//   blocks of token rows (prompts, portions, every step of a 32-bit session, and steps of layers the above does not
//     take): norms, projections, attention or scan, projection, experts - row kernels, the projections on the streaming
//     multi-row kernels where a shape has one.
#pragma once

#include <memory>
#include <vector>

#include "session.hpp"

namespace nv {

// Token rows a block holds at most. Layers of latents and experts take larger ones: an expert sees a few of a block's
// tokens, and its weights are read once a block whatever it sees.
constexpr uint32_t kStackBlockTokens = kGemmDeepMaxTokens, kExpertBlockTokens = 2048;

// Tensors of one layer in device memory. Row-concatenated: w_in is [q; k; v; gate] ([q; gate] where the keys are
// another layer's), [z; candidate; gate] or [query latent; latent and rotated key part; gate].
struct StackLayer {
  NervaHipStackLayer spec{};
  const uint16_t *norm[8] = {};   // norm1 w, b, norm1b w, b, norm2 w, b, norm2b w, b (parallel layers: norm1 w, norm2 w)
  const uint16_t *w_in = nullptr, *w_out = nullptr, *talk = nullptr, *sink = nullptr, *z_bias = nullptr, *x_bias = nullptr,
                 *w_up = nullptr, *w_down = nullptr, *act = nullptr;
  const uint16_t *q_norm = nullptr, *kv_norm = nullptr, *w_uq = nullptr, *w_uk = nullptr, *w_uv = nullptr;   // latent attention
  // experts: [experts][gate rows; up rows] and [experts][down], the shared one likewise
  const uint16_t *router = nullptr, *e_in = nullptr, *e_out = nullptr, *shared_in = nullptr, *shared_out = nullptr;
  uint32_t in_rows = 0, out_cols = 0;
  uint32_t q_col = 0, k_col = 0, v_col = 0, gate_col = 0;
  uint32_t rotation = 0;          // first column of the layer's angles in a token's rotation row
  uint32_t cache_layer = 0;       // the layer whose cache it reads (attention)
  // where the layer has a cache of its own
  uint64_t k_offset = 0, v_offset = 0;   // bytes into the session's cache area
  uint32_t table_offset = 0;             // entries into the session's block tables
  uint32_t ring_blocks = 0;
  uint64_t state_offset = 0;             // floats into the session's recurrent state (minGRU)
  bool own_cache() const {
    return spec.mixer == NERVA_HIP_MIXER_LATENT || (spec.mixer == NERVA_HIP_MIXER_ATTENTION && spec.kv_layer == NERVA_HIP_OWN_KEYS);
  }
  uint32_t q_rows() const { return spec.heads * (spec.key_dim + spec.rotary_key_dim); }   // latent attention
};

struct StackModel {
  std::vector<StackLayer> layers;
  uint32_t precision = NERVA_HIP_PRECISION_16;
  uint32_t block_tokens = kStackBlockTokens;
  uint32_t arrangement = NERVA_HIP_STACK_SANDWICH;
  float embedding_scale = 1.0f, logit_scale = 1.0f;
  const uint16_t *final_w = nullptr, *final_b = nullptr;
  // widest input projection, mixer output, feed-forward (activations of a token), query latent, queries, router, choices
  uint32_t max_in = 0, max_mix = 0, max_ff = 0, max_q_rank = 0, max_q = 0, max_experts = 0, max_top = 0;
  uint64_t plan_bytes = 0;                        // routing of a block (moe_rows.cuh)
  std::vector<float> angle_step;                  // per angle: radians per position
  std::vector<uint32_t> angle_cos, angle_sin;     // ... and its two columns in a token's rotation row
  uint32_t rotation_columns = 0;
  uint64_t cache_bytes = 0, state_floats = 0;
  uint32_t table_entries = 0, logical_blocks = 0;
};

constexpr uint32_t kStackWantedRows = 32;                    // rows whose logits are computed at a time

hipError_t stack_setup_state(Session *s, int32_t *failure_stage, bool with_weights);
// One decode step at the device cursor, head and sampler included.
hipError_t stack_enqueue_step(Session *s);
uint64_t stack_step_launches(const Session *s);
// Tokens begin .. end-1 of s->prompt through the layers in blocks, the last one with the head and the sampler.
// wanted / logits / residuals: as NervaHipSessionExtendRequest (host memory; the call then waits for them).
hipError_t stack_prompt(Session *s, uint32_t begin, uint32_t end, const uint32_t *wanted, uint32_t wanted_count, float *logits,
                        float *residuals, NervaHipHfDecodeSequenceResult *out);

}  // namespace nv
