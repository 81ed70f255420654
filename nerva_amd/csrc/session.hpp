// A decode session's object and what the translation units that implement its steps share of it.
#pragma once

#include <atomic>
#include <memory>
#include <vector>

#include "argmax.cuh"
#include "attn_decode.cuh"
#include "gemm_rows.cuh"
#include "gemv_stream.cuh"
#include "runtime_state.hpp"
#include "sampler.cuh"

namespace nv {

using Slot = NervaHipSyntheticTokenSlot;

struct LayerDev {
  const uint16_t *rms_attn, *rms_mlp, *wqkv, *q_norm, *k_norm, *q_bias, *k_bias, *v_bias, *wo, *o_bias,
      *wgu, *wdown;
};

enum StepMode { kDecodeStep = 0, kPromptStep = 1, kPromptHeadStep = 2 };
enum LaunchKind { kLEmbed = 0, kLQkv, kLAttn, kLO, kLGateUp, kLDown, kLHead, kLAdvance, kLKinds };

// The weight arena of a session and of every session forked from it (one stream of the weights can
// then serve a token row of each of them); freed by the last of them to go.
struct SharedWeights {
  char *origin = nullptr;  // what the allocator returned (and takes back)
  char *base = nullptr;    // the first kMatrixAlign boundary in it: offsets of the weight layout count from here
  uint64_t bytes = 0;
  std::atomic<uint32_t> refs{1};
};

// What a batch step needs to know of each of its sequences, in device memory: the cache and position
// for the attention launches, the token slots for the embedding.
struct BatchTable {
  AttnSeq seq[kGemmMaxTokens];
  const Slot *slots[kGemmMaxTokens];
  SamplerParams sample[kGemmMaxTokens];
};

struct StackModel;   // layer_stack.hpp

}  // namespace nv

struct NervaHipHfDecodeSequenceSession {
  uint32_t dtype = 0, hidden = 0, heads = 0, kv_heads = 0, head_dim = 0, intermediate = 0, vocab = 0,
           layers = 0, max_ctx = 0;
  float eps = 0.0f, theta = 0.0f;
  hipStream_t stream = nullptr;
  nv::SharedWeights *weights = nullptr;  // shared with forks
  char *arena = nullptr;             // everything but the weights: KV cache, sequence state, activations, workspaces
  uint32_t pair_gap = 0;             // elements between a layer's gate rows and its up rows (see kPairGapElems)
  bool arena_in_weights = false;     // `arena` lies behind the weights in their allocation (the creating session)
  uint64_t state_bytes = 0;          // size of `arena`
  uint64_t arena_bytes = 0;          // weights + state, as reported to the caller
  char *pinned = nullptr;
  uint64_t pinned_bytes = 0;
  std::vector<nv::LayerDev> layer;
  const uint16_t *emb = nullptr, *final_norm = nullptr, *lm_head = nullptr;
  uint16_t *kc = nullptr, *vc = nullptr;
  uint32_t block_count = 0;
  uint32_t *table = nullptr, *prompt = nullptr;
  uint32_t *state = nullptr;  // state[0] cursor, state[1] prompt count, state[2] steps executed so far,
                              // state[3] fault word (set by a kernel whose bounded wait gave up; cleared by start)
  nv::Slot *slots = nullptr;
  float *x = nullptr, *r = nullptr, *qkv = nullptr, *logits = nullptr, *rope_freq = nullptr, *rope_cs = nullptr;
  uint16_t *attn16 = nullptr, *ff16 = nullptr;
  void *attn_ws = nullptr, *sample_ws = nullptr;
  uint32_t attn_splits = 1;
  uint32_t attn_single_blocks = 0;   // contexts of up to this many blocks go to one split (0 with a forced split factor)
  uint64_t *attn_tagged = nullptr;   // tagged split partials of the decode step kernel
  uint32_t *attn_plan = nullptr;     // this step's split plan of the decode attention (attn_plan_fill), or null
  uint64_t *attn_trace = nullptr;  // NERVA_HIP_ATTN_TRACE=1: per-layer stage timestamps of selected attention workgroups
  nv::Slot *host_slots = nullptr;
  uint32_t *host_prompt = nullptr;
  uint32_t *host_state = nullptr;    // 64 words
  // captured steps: 0 decode step with the greedy finish, 1 prompt step, 2 decode step with the
  // temperature / top-k / top-p sampler (its parameters live in device memory, so one capture
  // serves every such configuration)
  hipGraph_t graph[3] = {nullptr, nullptr, nullptr};
  hipGraphExec_t exec[3] = {nullptr, nullptr, nullptr};
  uint64_t graph_nodes[3] = {0, 0, 0};
  // prompt blocks: up to prefill_block_tokens prompt tokens per pass through the layers (weights streamed
  // once per block on the matrix cores); false = one prompt step per token
  bool block_prefill = false;
  // the multi-row kernels take this model's shapes (prompt blocks and batch steps need it)
  bool rows_ready = false;
  float *blogits = nullptr;          // [NERVA_HIP_BATCH_MAX_BLOCK_TOKENS][vocab] logits of a batch step
  nv::BatchTable *btable = nullptr, *host_btable = nullptr;
  nv::Slot *bslots = nullptr, *host_bslots = nullptr;   // a batch step's published slots, gathered for one copy
  float *px = nullptr, *pr = nullptr, *pqkv = nullptr, *prope = nullptr;
  uint16_t *pxn16 = nullptr, *pattn16 = nullptr, *pff16 = nullptr;
  char *pattn_ws = nullptr;
  uint64_t pattn_ws_stride = 0;
  char *pgemm_ws = nullptr;        // partial sums of the K-sliced projections of a prompt block
  uint64_t pgemm_ws_bytes = 0;
  uint32_t prefill_block_tokens = nv::kGemmMaxTokens;   // tokens per prompt block: 512 or 256 where every projection has the kernel for it
  nv::SamplerDev sampler{};            // normalised configuration of the active sequence
  nv::SamplerDev *sampler_dev = nullptr;
  uint64_t *sampler_keys = nullptr;
  hipEvent_t ev0 = nullptr, ev1 = nullptr;
  // test hook: the next decode step is launched kernel by kernel and every intermediate vector is
  // copied behind the previous one into this caller-owned device buffer (step_trace_bytes)
  char *trace_buf = nullptr;
  uint64_t trace_used = 0;
  // echo of the caller's weight plan
  uint32_t planned_weight_blocks = 0, planned_gpu_resident_blocks = 0, planned_gpu_staged_blocks = 0,
           planned_weight_descriptor_count = 0;
  uint64_t planned_weight_bytes = 0, planned_gpu_resident_weight_bytes = 0,
           planned_gpu_staged_weight_bytes = 0, planned_weight_descriptor_hash = 0;
  uint64_t resident_weight_bytes = 0, kv_bytes = 0;
  // A mixed layer stack (layer_stack.hpp) instead of the uniform decoder layers above: its layers and weights, shared
  // with forks, and this sequence's part of it. The members above that describe one uniform layer are then unused or
  // hold the largest sizes; hidden, vocab, max_ctx, the prompt, the slots, the cursor words, the sampler, the graphs
  // and the lifecycle are the same.
  std::shared_ptr<const nv::StackModel> stack;
  char *stack_cache = nullptr;       // keys and values of the layers that have any, each layer in its own block ring
  uint32_t *stack_tables = nullptr;  // logical block -> block of the layer's ring, per caching layer
  float *stack_state = nullptr;      // recurrent state, f32, all recurrent layers
  uint64_t stack_state_bytes = 0;
  float *y = nullptr, *py = nullptr; // output of the sublayer under way, before its norm: decode row, token rows
  uint64_t stack_launches = 0;       // kernel launches of the step enqueued last (where the layers do not tell)
  // layers whose sublayers read the same row: the feed-forward's normalised rows and output
  void *pxn2 = nullptr;
  float *pz = nullptr;
  void *pql = nullptr;               // latent attention: normalised query latents, queries
  float *pq = nullptr;
  float *prouter = nullptr, *pslots = nullptr;   // experts: router logits, one output row per (token, choice)
  void *pplan = nullptr;             // ... and the block's routing (MoePlan)
  void *pwant = nullptr;             // normalised rows whose logits are asked for, with their row numbers and logits
  uint32_t *pwant_rows = nullptr;
  float *pwant_logits = nullptr;
  void *pxn = nullptr, *pmix = nullptr, *pff = nullptr;   // 16-bit or f32 token rows (the session's precision)
  // active sequence
  bool started = false, finished = false;
  uint32_t prompt_count = 0, observed = 0, cursor = 0, seed_token = 0, has_eos = 0, eos = 0;
};

namespace nv {

using Session = NervaHipHfDecodeSequenceSession;

struct Carver {
  uint64_t offset = 0;
  uint64_t take(uint64_t bytes, uint64_t align = 256) {
    const uint64_t at = (offset + align - 1) & ~(align - 1);
    offset = at + ((bytes + 255u) & ~uint64_t{255});
    return at;
  }
};
// Weight matrices start on 8 MiB boundaries of device memory (the arena's first such boundary is its origin for
// the weight layout). What the gate/up launch costs depends on its matrix's address modulo 8 MiB - the up rows lie
// a fixed 96 MiB behind the gate rows, and the memory channels are chosen by a hash that reaches up to those bits:
// with the rotated walk 31.0 us at 0 modulo 8 MiB, 31.4 at 2 and 6 MiB, 31.8 at 4 MiB, 32.1 at an odd KiB (the
// plain walk: 33.0 / 31.7 / 31.3 / 31.8 / 31.7). At most 8 MiB a matrix is left unused: under 1.2 GB for 36 layers.
constexpr uint64_t kMatrixAlign = 8u << 20;

// Moves the sequence's device-side position words (decode_session.hip).
hipError_t set_device_position(Session *s, uint32_t cursor, uint32_t prompt_count, uint32_t clear_fault);
void destroy_session(Session *s);
void fill_create_result(const Session *s, NervaHipHfDecodeSequenceSessionCreateResult *out);
// Stream, the arena of s->weights->bytes (with_weights) + s->state_bytes, the pinned mirrors and the events.
hipError_t allocate_session(Session *s, int32_t *failure_stage, bool with_weights);

}  // namespace nv
