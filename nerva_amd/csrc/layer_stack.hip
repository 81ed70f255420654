// Sessions over a mixed layer stack (see layer_stack.hpp).
#include "layer_stack.hpp"

#include <math.h>

#include <algorithm>
#include <new>

#include "attn_latent.cuh"
#include "attn_mixed.cuh"
#include "gemm_any.cuh"
#include "gemv_layer.cuh"
#include "mingru.cuh"
#include "moe_rows.cuh"
#include "norm_join.cuh"
#include "norm_rms.cuh"
#include "synth_fill.cuh"
#include "weight_plan.hpp"

using namespace nv;

namespace {

struct Angles {
  const float *step;
  const uint32_t *cos_col, *sin_col;
  uint32_t count, columns;
};

// Embedding rows and rotation tables of the tokens at positions first .. first + gridDim.x - 1, or of the one at the
// device cursor (a prompt token, or the token the position before it published).
template <uint32_t DT>
__global__ __launch_bounds__(kBlock) void stack_embed_kernel(const uint16_t *emb, const uint32_t *prompt, const Slot *slots,
                                                             const uint32_t *state, bool at_cursor, uint32_t first,
                                                             uint32_t max_steps, uint32_t hidden, uint32_t vocab, float scale, float *x,
                                                             Angles angles, float *rope) {
  const uint32_t t = blockIdx.x, pos = at_cursor ? state[0] : first + t;
  if (pos >= max_steps) return;
  for (uint32_t i = threadIdx.x; i < angles.count; i += kBlock) {
    float sn, cs;
    sincosf(static_cast<float>(pos) * angles.step[i], &sn, &cs);
    float *row = rope + static_cast<uint64_t>(t) * angles.columns;
    row[angles.cos_col[i]] = cs;
    row[angles.sin_col[i]] = sn;
  }
  uint32_t token = !at_cursor || pos < state[1] ? prompt[pos] : slots[pos - 1].token;
  if (token >= vocab) token = 0;   // prompts are validated on the host; sampled ids are < vocab
  const uint16_t *row = emb + static_cast<uint64_t>(token) * hidden;
  for (uint32_t i = threadIdx.x; i < hidden; i += kBlock) x[static_cast<uint64_t>(t) * hidden + i] = dec16<DT>(row[i]) * scale;
}

// Identity plus noise for a synthetic mixing matrix (the noise is there already).
__global__ void add_identity_kernel(uint16_t *m, uint32_t n) {
  const uint32_t i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) m[static_cast<uint64_t>(i) * n + i] = f32_to_bf16(bf16_to_f32(m[static_cast<uint64_t>(i) * n + i]) + 1.0f);
}

bool wide(const Session *s) { return s->stack->precision == NERVA_HIP_PRECISION_32; }
bool parallel(const Session *s) { return s->stack->arrangement == NERVA_HIP_STACK_PARALLEL; }
// Whether the decode step is decode_step_16's; every other step is a block of one token row at the device cursor.
bool sandwich_step(const Session *s) {
  if (wide(s) || parallel(s)) return false;
  for (const StackLayer &w : s->stack->layers)
    if (w.spec.mixer == NERVA_HIP_MIXER_LATENT) return false;
  return true;
}

// Whether it is parallel_step_16's.
bool parallel_step(const Session *s) {
  if (wide(s) || !parallel(s) || s->stack->logit_scale == 0.0f) return false;
  for (const StackLayer &w : s->stack->layers) {
    const NervaHipStackLayer &d = w.spec;
    if (d.mixer != NERVA_HIP_MIXER_LATENT || d.ff != 0 ||
        !layer_gemv_takes(s->hidden, d.q_rank, w.out_cols, d.experts, d.experts_per_token, d.expert_ff, d.shared_ff))
      return false;
  }
  return true;
}

// The seam that is due before the next projection: the norm of the sublayer output in s->y / s->py, if there is one.
struct Seam {
  const uint16_t *post_w = nullptr, *post_b = nullptr;
};

// What a parallel layer has put out and the residual has not taken in yet.
struct Sum {
  const float *mixer = nullptr, *ff = nullptr, *slot_rows = nullptr, *slot_weights = nullptr;
  uint32_t slots = 0;
};

// ---- decode step, 16-bit precision -----------------------------------------------------------

struct DecodeRow {
  float *x, *next;   // the residual row, and where the next seam leaves it
  Seam due;
};

JoinNorm decode_seam(Session *s, DecodeRow &row, const uint16_t *pre_w, const uint16_t *pre_b) {
  JoinNorm j{};
  j.x = row.x;
  j.pre_w = pre_w;
  j.pre_b = pre_b;
  j.eps = s->eps;
  if (row.due.post_w != nullptr) {
    j.y = s->y;
    j.post_w = row.due.post_w;
    j.post_b = row.due.post_b;
    j.x_out = row.next;
    std::swap(row.x, row.next);
    row.due = Seam{};
  }
  return j;
}

GemvParams decode_gemv(Session *s, const uint16_t *w, uint32_t rows, uint32_t cols) {
  GemvParams p{};
  p.w = w;
  p.rows = rows;
  p.cols = cols;
  p.cursor = s->state;
  p.max_steps = s->max_ctx;
  return p;
}

MixedAttnParams attention_params(Session *s, const StackLayer &layer, const float *proj, const float *rope) {
  const StackModel &m = *s->stack;
  const StackLayer &owner = m.layers[layer.cache_layer];
  MixedAttnParams a{};
  a.proj = proj;
  a.proj_stride = layer.in_rows;
  a.q_col = layer.q_col;
  a.k_col = layer.k_col;
  a.v_col = layer.v_col;
  a.gate_col = layer.gate_col;
  a.talk = layer.talk;
  a.sink = layer.sink;
  a.k_cache = s->stack_cache + owner.k_offset;
  a.v_cache = s->stack_cache + owner.v_offset;
  a.table = s->stack_tables + owner.table_offset;
  a.rope_cs = rope + layer.rotation;
  a.rot_dims = layer.spec.rotary_dims;
  a.rope_stride = m.rotation_columns;
  a.heads = layer.spec.heads;
  a.kv_heads = layer.spec.kv_heads;
  a.key_dim = layer.spec.key_dim;
  a.value_dim = layer.spec.value_dim;
  a.chunk = layer.spec.chunk_tokens;
  a.scale = layer.spec.score_scale;
  a.cache32 = wide(s) ? 1u : 0u;
  a.max_steps = s->max_ctx;
  a.workspace = s->attn_ws;
  a.last_block = m.logical_blocks - 1;
  return a;
}

// Rotation, cache rows, attention of the token rows in `a`.
bool takes_wide(const Session *s, const StackLayer &w) {
  return !wide(s) && mixed_attention_wide(w.spec.heads, w.spec.kv_heads, w.spec.key_dim, w.spec.value_dim) &&
         tuning(kTuneMixedAttentionWide) != 2;
}
uint32_t attention_launches(const Session *s, const StackLayer &w, bool decode) {
  return takes_wide(s, w) ? (decode ? 2u : 3u) : (w.own_cache() ? 2u : 1u);
}
hipError_t attend(Session *s, const StackLayer &w, const MixedAttnParams &a) {
  if (takes_wide(s, w)) return launch_mixed_attention_wide(s->dtype, a, w.own_cache(), s->stream);
  hipError_t err = w.own_cache() ? launch_mixed_publish(s->dtype, a, s->stream) : hipSuccess;
  return err == hipSuccess ? launch_mixed_attention(s->dtype, a, s->stream) : err;
}

LatentAttnParams latent_params(Session *s, const StackLayer &w, const float *proj, const float *q, const float *rope) {
  const StackModel &m = *s->stack;
  LatentAttnParams a{};
  a.proj = proj;
  a.proj_stride = w.in_rows;
  a.q_col = w.q_col;
  a.kv_col = w.k_col;
  a.gate_col = w.gate_col;
  a.q_norm = w.q_norm;
  a.kv_norm = w.kv_norm;
  a.eps = s->eps;
  a.q = q;
  a.w_uk = w.w_uk;
  a.w_uv = w.w_uv;
  a.cache = s->stack_cache + w.k_offset;
  a.table = s->stack_tables + w.table_offset;
  a.rope_cs = rope + w.rotation;
  a.rot_dims = w.spec.rotary_dims;
  a.rope_stride = m.rotation_columns;
  a.heads = w.spec.heads;
  a.key_dim = w.spec.key_dim;
  a.rot_dim = w.spec.rotary_key_dim;
  a.value_dim = w.spec.value_dim;
  a.q_rank = w.spec.q_rank;
  a.kv_rank = w.spec.kv_rank;
  a.window = w.spec.window_tokens;
  a.scale = w.spec.score_scale;
  a.cache32 = wide(s) ? 1u : 0u;
  a.max_steps = s->max_ctx;
  a.workspace = s->attn_ws;
  a.last_block = m.logical_blocks - 1;
  return a;
}
bool takes_latent_wide(const Session *s, const NervaHipStackLayer &d) {
  return !wide(s) && latent_attention_wide(d.heads, d.key_dim, d.rotary_key_dim, d.value_dim, d.kv_rank) && tuning(kTuneLatentAttentionWide) != 2;
}

// Final norm, head, sampler of the row in (row.x, s->y): logits, slot[cursor], cursor + 1.
hipError_t decode_head(Session *s, DecodeRow &row) {
  const StackModel &m = *s->stack;
  GemvParams p = decode_gemv(s, s->lm_head, s->vocab, s->hidden);
  if (parallel(s)) {
    p.xf = row.x;
    p.gamma = m.final_w;
    p.eps = s->eps;
    p.gain = m.logit_scale;
  } else {
    p.join = decode_seam(s, row, m.final_w, m.final_b);
  }
  p.out_f32 = s->logits;
  sample_bind_workspace(p.sample, s->sample_ws);
  p.sample.slots = s->slots;
  p.sample.cursor_rw = s->state;
  uint32_t candidates = 0;
  hipError_t err = launch_gemv(s->dtype, parallel(s) ? kProRmsNorm : kProJoin, kEpiArgmax, p, s->stream, nullptr, &candidates);
  if (err != hipSuccess) return err;
  if (s->sampler.mode == kSamplerGreedy) return launch_sample_finish(p.sample, candidates, s->state, s->max_ctx, s->stream);
  SamplerParams sp{};
  sp.logits = s->logits;
  sp.vocab = s->vocab;
  sp.config = s->sampler_dev;
  sp.keys = s->sampler_keys;
  sp.out = p.sample;
  sp.cursor = s->state;
  sp.max_steps = s->max_ctx;
  return launch_sampler(sp, s->stream);
}

hipError_t embed_rows(Session *s, bool at_cursor, uint32_t first, uint32_t tokens, float *x) {
  const StackModel &m = *s->stack;
  const uint32_t *cols = reinterpret_cast<const uint32_t *>(s->rope_freq + m.angle_step.size());
  const uint32_t n = static_cast<uint32_t>(m.angle_step.size());
  const Angles angles{s->rope_freq, cols, cols + n, n, m.rotation_columns};
  hipLaunchKernelGGL(stack_embed_kernel<kBF16>, dim3(tokens), dim3(kBlock), 0, s->stream, s->emb, s->prompt, s->slots, s->state,
                     at_cursor, first, s->max_ctx, s->hidden, s->vocab, m.embedding_scale, x, angles, s->prope);
  return hipGetLastError();
}

hipError_t decode_step_16(Session *s) {
  const StackModel &m = *s->stack;
  hipStream_t st = s->stream;
  hipError_t err = embed_rows(s, true, 0, 1, s->x);
  DecodeRow row{s->x, s->r, Seam{}};
  for (size_t l = 0; err == hipSuccess && l < m.layers.size(); ++l) {
    const StackLayer &w = m.layers[l];
    GemvParams p = decode_gemv(s, w.w_in, w.in_rows, s->hidden);
    p.join = decode_seam(s, row, w.norm[0], w.norm[1]);
    if (w.spec.mixer == NERVA_HIP_MIXER_ATTENTION) {
      p.out_f32 = s->qkv;
      err = launch_gemv(s->dtype, kProJoin, kEpiF32, p, st);
      MixedAttnParams a = attention_params(s, w, s->qkv, s->prope);
      a.cursor = s->state;
      a.tokens = 1;
      a.out16 = s->attn16;
      if (err == hipSuccess) err = attend(s, w, a);
    } else {
      p.rows = w.spec.width;
      p.out16 = s->attn16;
      p.bias = w.z_bias;
      p.bias2 = w.x_bias;
      p.state = s->stack_state + w.state_offset;
      err = launch_gemv(s->dtype, kProJoin, kEpiMinGru, p, st);
    }
    if (err == hipSuccess) {
      p = decode_gemv(s, w.w_out, s->hidden, w.out_cols);
      p.x16 = s->attn16;
      p.out_f32 = s->y;
      err = launch_gemv(s->dtype, kProX16, kEpiF32, p, st);
      row.due = Seam{w.norm[2], w.norm[3]};
    }
    if (err != hipSuccess || w.spec.ff == 0) continue;
    p = decode_gemv(s, w.w_up, w.spec.ff, s->hidden);
    p.join = decode_seam(s, row, w.norm[4], w.norm[5]);
    p.act = w.act;
    p.out16 = s->ff16;
    err = launch_gemv(s->dtype, kProJoin, kEpiXielu, p, st);
    if (err == hipSuccess) {
      p = decode_gemv(s, w.w_down, s->hidden, w.spec.ff);
      p.x16 = s->ff16;
      p.out_f32 = s->y;
      err = launch_gemv(s->dtype, kProX16, kEpiF32, p, st);
      row.due = Seam{w.norm[6], w.norm[7]};
    }
  }
  return err == hipSuccess ? decode_head(s, row) : err;
}

// Parallel layers of attention over latents and routed experts.
hipError_t parallel_step_16(Session *s) {
  const StackModel &m = *s->stack;
  hipStream_t st = s->stream;
  hipError_t err = embed_rows(s, true, 0, 1, s->x);
  uint64_t launches = 1;
  for (size_t l = 0; err == hipSuccess && l < m.layers.size(); ++l) {
    const StackLayer &w = m.layers[l];
    const NervaHipStackLayer &d = w.spec;
    const MoePlan plan = moe_plan_at(s->pplan, 1, d.experts_per_token, d.experts, true);
    LayerFront f{};
    f.x = s->x;
    f.mixer_norm = w.norm[0];
    f.ff_norm = d.experts != 0 ? w.norm[1] : nullptr;
    f.eps = s->eps;
    f.hidden = s->hidden;
    f.w_in = w.w_in;
    f.in_rows = w.gate_col + w.out_cols;
    f.in = s->qkv;
    f.router = w.router;
    f.experts = d.experts;
    f.logits = s->prouter;
    f.shared_in = w.shared_in;
    f.shared_ff = d.shared_ff;
    f.shared_limit = d.shared_limit;
    f.shared_act = s->ff16;
    f.h16 = static_cast<uint16_t *>(s->pxn2);
    f.cursor = s->state;
    f.max_steps = s->max_ctx;
    err = launch_layer_front(s->dtype, f, st);
    LayerMiddle g{};
    g.latent = s->qkv + w.q_col;
    g.latent_norm = w.q_norm;
    g.eps = s->eps;
    g.w_uq = w.w_uq;
    g.q_rank = d.q_rank;
    g.q_rows = w.q_rows();
    g.q = s->pq;
    g.h16 = f.h16;
    g.logits = s->prouter;
    g.hidden = s->hidden;
    g.experts = d.experts;
    g.top = d.experts_per_token;
    g.e_in = w.e_in;
    g.ff = d.expert_ff;
    g.limit = d.expert_limit;
    g.act = static_cast<uint16_t *>(s->pff);
    g.ids = plan.ids;
    g.weights = plan.weights;
    g.cursor = s->state;
    g.max_steps = s->max_ctx;
    if (err == hipSuccess) err = launch_layer_middle(s->dtype, g, st);
    LatentAttnParams a = latent_params(s, w, s->qkv, s->pq, s->prope);
    a.cursor = s->state;
    a.tokens = 1;
    a.out16 = s->attn16;
    const bool fast = takes_latent_wide(s, d);
    if (!fast) a.q_latent16 = static_cast<uint16_t *>(s->pql);   // (the middle launch has its own)
    if (err == hipSuccess && !fast) err = launch_latent_prepare(s->dtype, a, st);
    if (err == hipSuccess) err = fast ? launch_latent_attention_wide(s->dtype, a, st, &launches) : launch_latent_attention(s->dtype, a, st);
    LayerBack b{};
    b.x = s->x;
    b.hidden = s->hidden;
    b.w_o = w.w_out;
    b.mixed = s->attn16;
    b.mix_cols = w.out_cols;
    b.e_out = w.e_out;
    b.act = g.act;
    b.ids = plan.ids;
    b.weights = plan.weights;
    b.ff = d.expert_ff;
    b.top = d.experts != 0 ? d.experts_per_token : 0u;
    b.shared_out = w.shared_out;
    b.shared_act = s->ff16;
    b.shared_ff = d.shared_ff;
    b.cursor = s->state;
    b.max_steps = s->max_ctx;
    if (err == hipSuccess) err = launch_layer_back(s->dtype, b, st);
    launches += 3 + (fast ? 0 : 2);
  }
  s->stack_launches = launches + (s->sampler.mode == kSamplerGreedy ? 2 : 3);
  DecodeRow row{s->x, nullptr, Seam{}};
  return err == hipSuccess ? decode_head(s, row) : err;
}

// ---- blocks of token rows --------------------------------------------------------------------

// Token tiles of the matrix-operand order a projection's input takes, 0 where its shape goes through gemm_any.
uint32_t operand_tiles(const Session *s, int epilogue, uint32_t rows, uint32_t cols, uint32_t tokens) {
  if (wide(s) || cols % 32 != 0) return 0;
  tokens = std::min(tokens, kGemmDeepMaxTokens);   // (larger blocks go in pieces)
  const bool taken = tokens <= kGemmMaxTokens       ? gemm_rows_supported(rows, cols, tokens)
                     : tokens <= kGemmWideMaxTokens ? gemm_wide_slices(epilogue, rows, cols, tokens, s->pgemm_ws_bytes) != 0
                                                    : gemm_deep_slices(epilogue, rows, cols, tokens, s->pgemm_ws_bytes) != 0;
  return taken ? gemm_packed_tiles(tokens) : 0u;
}

struct Block {
  Session *s;
  uint32_t tokens, first;
  bool at_cursor;      // the one token at the device cursor (the steps that sandwich_step does not take)
  Seam due;
  uint64_t launches;
  Sum sum{};           // parallel layers

  hipError_t join(const uint16_t *pre_w, const uint16_t *pre_b, uint32_t tiles) {
    JoinRows j{};
    j.x = s->px;
    if (due.post_w != nullptr) {
      j.y = s->py;
      j.post_w = due.post_w;
      j.post_b = due.post_b;
      due = Seam{};
    }
    j.pre_w = pre_w;
    j.pre_b = pre_b;
    if (pre_w != nullptr) {
      if (wide(s)) j.out32 = static_cast<float *>(s->pxn);
      else j.out16 = static_cast<uint16_t *>(s->pxn);
    }
    j.packed_tiles = tiles;
    j.tokens = tokens;
    j.cols = s->hidden;
    j.eps = s->eps;
    launches += 1;
    return launch_join_rows(s->dtype, j, s->stream);
  }

  // x: the 16-bit or f32 rows of `tiles` layout; out: f32 rows, or for the activation 16-bit rows of out_tiles layout
  hipError_t project(int epilogue, const uint16_t *w, uint32_t rows, uint32_t cols, const void *x, uint32_t tiles, void *out,
                     uint32_t out_tiles, const uint16_t *act) {
    launches += 1;
    const bool narrow = epilogue == kGemmXielu && !wide(s);
    if (tiles != 0 && tokens > kGemmDeepMaxTokens) {
      // pieces of kGemmDeepMaxTokens rows; the last one has the others' layout, so enough rows for that are multiplied
      hipError_t err = hipSuccess;
      const uint32_t all = tokens;
      for (uint32_t at = 0; err == hipSuccess && at < all; at += kGemmDeepMaxTokens) {
        tokens = std::min(kGemmDeepMaxTokens, std::max(all - at, kGemmWideMaxTokens + 1));
        const uint64_t done = static_cast<uint64_t>(at) * rows;
        err = project(epilogue, w, rows, cols, static_cast<const uint16_t *>(x) + static_cast<uint64_t>(at) * cols, tiles,
                      narrow ? static_cast<void *>(static_cast<uint16_t *>(out) + done) : static_cast<void *>(static_cast<float *>(out) + done),
                      out_tiles, act);
      }
      tokens = all;
      return err;
    }
    if (tiles != 0) {
      GemmRowsParams g{};
      g.w = w;
      g.x16 = static_cast<const uint16_t *>(x);
      g.x_packed = tiles;
      g.rows = rows;
      g.cols = cols;
      g.tokens = tokens;
      g.workspace = s->pgemm_ws;
      g.workspace_bytes = s->pgemm_ws_bytes;
      g.act = act;
      if (narrow) {
        g.out16 = static_cast<uint16_t *>(out);
        g.out_packed_tiles = out_tiles;
      } else {
        g.out_f32 = static_cast<float *>(out);
      }
      return launch_gemm_rows(s->dtype, epilogue, g, s->stream);
    }
    GemmAnyParams g{};
    g.w = w;
    if (wide(s)) g.x32 = static_cast<const float *>(x);
    else g.x16 = static_cast<const uint16_t *>(x);
    g.rows = rows;
    g.cols = cols;
    g.tokens = tokens;
    g.act = act;
    if (narrow) {
      g.out16 = static_cast<uint16_t *>(out);
      g.out_packed_tiles = out_tiles;
    } else {
      g.out_f32 = static_cast<float *>(out);
    }
    return launch_gemm_any(s->dtype, epilogue, g, s->stream);
  }

  // The residual rows with the sum that is due, and their norms: for the mixer into s->pxn, for the feed-forward into
  // s->pxn2 (either may be left out). A picked output goes to `picked` instead, the rows stay as they are.
  hipError_t rms(const uint16_t *for_mixer, uint32_t mixer_tiles, const uint16_t *for_ff, uint32_t ff_tiles) {
    RmsRows r = rms_rows();
    r.out[0] = rms_out(for_mixer, s->pxn, mixer_tiles);
    r.out[1] = rms_out(for_ff, s->pxn2, ff_tiles);
    r.tokens = tokens;
    sum = Sum{};
    launches += 1;
    return launch_rms_rows(s->dtype, r, s->stream);
  }
  RmsRows rms_rows() const {
    RmsRows r{};
    r.x = s->px;
    r.y[0] = sum.mixer;
    r.y[1] = sum.ff;
    r.slot_rows = sum.slot_rows;
    r.slot_weights = sum.slot_weights;
    r.slots = sum.slots;
    r.gain = 1.0f;
    r.cols = s->hidden;
    r.eps = s->eps;
    return r;
  }
  RmsOut rms_out(const uint16_t *gamma, void *to, uint32_t tiles) const {
    RmsOut o{};
    o.gamma = gamma;
    if (wide(s)) o.out32 = static_cast<float *>(to);
    else o.out16 = static_cast<uint16_t *>(to);
    o.packed_tiles = tiles;
    return o;
  }

  uint32_t mixer_tiles(const StackLayer &w) const { return operand_tiles(s, kGemmF32, w.in_rows, s->hidden, tokens); }
  // h: the normalised rows, in that layout; the output goes to s->py
  hipError_t mixer(const StackLayer &w, const void *h) {
    const uint32_t out_tiles = operand_tiles(s, kGemmF32, s->hidden, w.out_cols, tokens);
    hipError_t err = project(kGemmF32, w.w_in, w.in_rows, s->hidden, h, mixer_tiles(w), s->pqkv, 0, nullptr);
    if (err != hipSuccess) return err;
    if (w.spec.mixer == NERVA_HIP_MIXER_LATENT) {
      const uint32_t q_tiles = operand_tiles(s, kGemmF32, w.q_rows(), w.spec.q_rank, tokens);
      LatentAttnParams a = latent_params(s, w, s->pqkv, s->pq, s->prope);
      a.position = first;
      a.tokens = tokens;
      if (at_cursor) a.cursor = s->state;
      if (wide(s)) a.q_latent32 = static_cast<float *>(s->pql);
      else a.q_latent16 = static_cast<uint16_t *>(s->pql);
      a.q_latent_tiles = q_tiles;
      if (wide(s)) a.out32 = static_cast<float *>(s->pmix);
      else a.out16 = static_cast<uint16_t *>(s->pmix);
      a.packed_tiles = out_tiles;
      err = launch_latent_prepare(s->dtype, a, s->stream);
      if (err == hipSuccess) err = project(kGemmF32, w.w_uq, w.q_rows(), w.spec.q_rank, s->pql, q_tiles, s->pq, 0, nullptr);
      const bool fast = takes_latent_wide(s, w.spec);
      if (err == hipSuccess) err = fast ? launch_latent_attention_wide(s->dtype, a, s->stream, &launches) : launch_latent_attention(s->dtype, a, s->stream);
      launches += fast ? 0 : 1;
    } else if (w.spec.mixer == NERVA_HIP_MIXER_ATTENTION) {
      MixedAttnParams a = attention_params(s, w, s->pqkv, s->prope);
      a.position = first;
      a.tokens = tokens;
      if (at_cursor) a.cursor = s->state;
      if (wide(s)) a.out32 = static_cast<float *>(s->pmix);
      else a.out16 = static_cast<uint16_t *>(s->pmix);
      a.packed_tiles = out_tiles;
      err = attend(s, w, a);
      launches += attention_launches(s, w, false) - 1;
    } else {
      MinGruRows g{};
      g.zxg = s->pqkv;
      g.z_bias = w.z_bias;
      g.x_bias = w.x_bias;
      g.state = s->stack_state + w.state_offset;
      if (wide(s)) g.out32 = static_cast<float *>(s->pmix);
      else g.out16 = static_cast<uint16_t *>(s->pmix);
      g.packed_tiles = out_tiles;
      g.tokens = tokens;
      g.width = w.spec.width;
      if (at_cursor) {
        g.cursor = s->state;
        g.max_steps = s->max_ctx;
      }
      err = launch_mingru_rows(s->dtype, g, s->stream);
    }
    launches += 1;
    if (err == hipSuccess) err = project(kGemmF32, w.w_out, s->hidden, w.out_cols, s->pmix, out_tiles, s->py, 0, nullptr);
    return err;
  }

  uint32_t ff_tiles(const StackLayer &w) const {
    return w.spec.ff != 0 ? operand_tiles(s, kGemmXielu, w.spec.ff, s->hidden, tokens) : 0u;
  }
  hipError_t feed_forward(const StackLayer &w, const void *h, float *out) {
    const uint32_t down_tiles = operand_tiles(s, kGemmF32, s->hidden, w.spec.ff, tokens);
    hipError_t err = project(kGemmXielu, w.w_up, w.spec.ff, s->hidden, h, ff_tiles(w), s->pff, down_tiles, w.act);
    if (err == hipSuccess) err = project(kGemmF32, w.w_down, s->hidden, w.spec.ff, s->pff, down_tiles, out, 0, nullptr);
    return err;
  }

  // Routed experts on the rows h ([token][column]): one row per (token, choice) in s->pslots, the shared expert's in s->pz.
  hipError_t experts(const StackLayer &w, const void *h) {
    const NervaHipStackLayer &d = w.spec;
    MoeRouteRows r{};
    r.logits = s->prouter;
    r.tokens = tokens;
    r.experts = d.experts;
    r.top = d.experts_per_token;
    r.plan = moe_plan_at(s->pplan, tokens, r.top, r.experts, wide(s));
    ExpertRows e{};
    if (wide(s)) {
      e.x32 = static_cast<const float *>(h);
      e.act32 = static_cast<float *>(s->pff);
    } else {
      e.x16 = static_cast<const uint16_t *>(h);
      e.act16 = static_cast<uint16_t *>(s->pff);
    }
    e.hidden = s->hidden;
    e.tokens = tokens;
    hipError_t err = hipSuccess;
    if (d.shared_ff != 0) {
      e.w_gate_up = w.shared_in;
      e.w_down = w.shared_out;
      e.out = s->pz;
      e.ff = d.shared_ff;
      e.limit = d.shared_limit;
      e.top = e.experts = 1;
      err = launch_expert_gate_up(s->dtype, e, s->stream);
      if (err == hipSuccess) err = launch_expert_down(s->dtype, e, s->stream);
      launches += 2;
    }
    if (err == hipSuccess) err = project(kGemmF32, w.router, d.experts, s->hidden, h, 0, s->prouter, 0, nullptr);
    if (err == hipSuccess) err = launch_moe_route_rows(r, s->stream);
    e.w_gate_up = w.e_in;
    e.w_down = w.e_out;
    e.out = s->pslots;
    e.ff = d.expert_ff;
    e.limit = d.expert_limit;
    e.top = r.top;
    e.experts = r.experts;
    e.plan = &r.plan;
    if (err == hipSuccess) err = launch_expert_gate_up(s->dtype, e, s->stream);
    if (err == hipSuccess) err = launch_expert_down(s->dtype, e, s->stream);
    launches += 4;
    sum.ff = d.shared_ff != 0 ? s->pz : nullptr;
    sum.slot_rows = s->pslots;
    sum.slot_weights = r.plan.weights;
    sum.slots = r.top;
    return err;
  }

  hipError_t sandwich_layer(const StackLayer &w) {
    hipError_t err = join(w.norm[0], w.norm[1], mixer_tiles(w));
    if (err == hipSuccess) err = mixer(w, s->pxn);
    due = Seam{w.norm[2], w.norm[3]};
    if (err != hipSuccess || w.spec.ff == 0) return err;
    err = join(w.norm[4], w.norm[5], ff_tiles(w));
    if (err == hipSuccess) err = feed_forward(w, s->pxn, s->py);
    due = Seam{w.norm[6], w.norm[7]};
    return err;
  }

  hipError_t parallel_layer(const StackLayer &w) {
    const bool ff = w.spec.ff != 0 || w.spec.experts != 0;
    hipError_t err = rms(w.norm[0], mixer_tiles(w), ff ? w.norm[1] : nullptr, ff_tiles(w));
    if (err == hipSuccess) err = mixer(w, s->pxn);
    if (err == hipSuccess && w.spec.experts != 0) {
      err = experts(w, s->pxn2);
    } else if (err == hipSuccess && w.spec.ff != 0) {
      err = feed_forward(w, s->pxn2, s->pz);
      sum.ff = s->pz;
    }
    sum.mixer = s->py;
    return err;
  }

  // x' where nothing follows that would take the last layer's output in.
  hipError_t settle() { return parallel(s) ? rms(nullptr, 0, nullptr, 0) : join(nullptr, nullptr, 0); }

  // residuals: host [layers][row_stride] f32, the block's rows of every layer, or null
  hipError_t layers(float *residuals, uint64_t row_stride) {
    hipError_t err = embed_rows(s, at_cursor, first, tokens, s->px);
    launches += 1;
    const StackModel &m = *s->stack;
    for (size_t l = 0; err == hipSuccess && l < m.layers.size(); ++l) {
      err = parallel(s) ? parallel_layer(m.layers[l]) : sandwich_layer(m.layers[l]);
      if (err == hipSuccess && residuals != nullptr) {
        err = settle();
        if (err == hipSuccess)
          err = hipMemcpyAsync(residuals + l * row_stride, s->px, static_cast<uint64_t>(tokens) * s->hidden * sizeof(float),
                               hipMemcpyDeviceToHost, s->stream);
      }
    }
    return err;
  }

  // Logits of the block's rows pick[0 .. count) into s->pwant_logits (count <= kStackWantedRows) or, for the one row of
  // a block of one token, into `logits`. Leaves the residual rows as they are where rows are picked.
  hipError_t logits_of(const uint32_t *pick, uint32_t count, float *logits) {
    const StackModel &m = *s->stack;
    const uint32_t tiles = !wide(s) && s->hidden % 32 == 0 && gemm_rows_supported(s->vocab, s->hidden, count) ? gemm_packed_tiles(count) : 0u;
    hipError_t err;
    if (parallel(s)) {
      RmsRows r = rms_rows();
      r.out[0] = rms_out(m.final_w, s->pwant, tiles);
      r.pick = pick;
      r.gain = m.logit_scale;
      r.tokens = count;
      err = launch_rms_rows(s->dtype, r, s->stream);
    } else {
      JoinRows j{};
      j.x = s->px;
      if (due.post_w != nullptr) {
        j.y = s->py;
        j.post_w = due.post_w;
        j.post_b = due.post_b;
      }
      j.pre_w = m.final_w;
      j.pre_b = m.final_b;
      j.pick = pick;
      if (wide(s)) j.out32 = static_cast<float *>(s->pwant);
      else j.out16 = static_cast<uint16_t *>(s->pwant);
      j.packed_tiles = tiles;
      j.tokens = count;
      j.cols = s->hidden;
      j.eps = s->eps;
      err = launch_join_rows(s->dtype, j, s->stream);
    }
    const uint32_t rows = tokens;
    tokens = count;
    if (err == hipSuccess) err = project(kGemmF32, s->lm_head, s->vocab, s->hidden, s->pwant, tiles, logits, 0, nullptr);
    tokens = rows;
    launches += 1;
    return err;
  }
};

// The sampler from s->logits (sessions whose head is not the decode step's).
hipError_t sample_logits(Session *s) {
  SamplerParams sp{};
  sp.logits = s->logits;
  sp.vocab = s->vocab;
  sp.config = s->sampler_dev;
  sp.keys = s->sampler_keys;
  sample_bind_workspace(sp.out, s->sample_ws);
  sp.out.slots = s->slots;
  sp.out.cursor_rw = s->state;
  sp.cursor = s->state;
  sp.max_steps = s->max_ctx;
  return launch_sampler(sp, s->stream);
}

}  // namespace

hipError_t nv::stack_enqueue_step(Session *s) {
  if (sandwich_step(s)) return decode_step_16(s);
  if (parallel_step(s)) return parallel_step_16(s);
  Block b{s, 1, 0, true, Seam{}, 0};
  hipError_t err = b.layers(nullptr, 0);
  if (err == hipSuccess) err = b.logits_of(nullptr, 1, s->logits);
  if (err == hipSuccess) err = sample_logits(s);
  s->stack_launches = b.launches + 2;
  return err;
}

uint64_t nv::stack_step_launches(const Session *s) {
  if (!sandwich_step(s)) return s->stack_launches;
  uint64_t n = 1 + (s->sampler.mode == kSamplerGreedy ? 2 : 3);
  for (const StackLayer &w : s->stack->layers) {
    n += w.spec.mixer == NERVA_HIP_MIXER_ATTENTION ? 2 + attention_launches(s, w, true) : 2;
    if (w.spec.ff != 0) n += 2;
  }
  return n;
}

hipError_t nv::stack_prompt(Session *s, uint32_t begin, uint32_t end, const uint32_t *wanted, uint32_t wanted_count, float *logits,
                            float *residuals, NervaHipHfDecodeSequenceResult *out) {
  hipError_t err = hipSuccess;
  uint32_t next_wanted = 0;
  const uint64_t H = s->hidden;
  const uint32_t most = s->stack->block_tokens;
  for (uint32_t first = begin; err == hipSuccess && first < end; first += most) {
    Block b{s, std::min(most, end - first), first, false, Seam{}, 0};
    err = b.layers(residuals != nullptr ? residuals + static_cast<uint64_t>(first - begin) * H : nullptr,
                   static_cast<uint64_t>(end - begin) * H);
    while (err == hipSuccess && next_wanted < wanted_count && wanted[next_wanted] < first + b.tokens - begin) {
      uint32_t *rows = s->host_state, count = 0;   // (pinned; the copies below are waited for before it is written again)
      while (count < kStackWantedRows && next_wanted + count < wanted_count && wanted[next_wanted + count] < first + b.tokens - begin) {
        rows[count] = wanted[next_wanted + count] - (first - begin);
        count += 1;
      }
      err = hipMemcpyAsync(s->pwant_rows, rows, count * sizeof(uint32_t), hipMemcpyHostToDevice, s->stream);
      if (err == hipSuccess) err = b.logits_of(s->pwant_rows, count, s->pwant_logits);
      if (err == hipSuccess)
        err = hipMemcpyAsync(logits + static_cast<uint64_t>(next_wanted) * s->vocab, s->pwant_logits,
                             static_cast<uint64_t>(count) * s->vocab * sizeof(float), hipMemcpyDeviceToHost, s->stream);
      if (err == hipSuccess) err = hipStreamSynchronize(s->stream);
      out->d2h_bytes += static_cast<uint64_t>(count) * s->vocab * sizeof(float);
      out->sync_calls += 1;
      next_wanted += count;
    }
    if (err == hipSuccess && first + b.tokens == end) {
      // the sequence's last token so far: head and sampler at its position
      err = set_device_position(s, end - 1, end, 0);
      const uint64_t last = b.tokens - 1;
      if (err == hipSuccess && sandwich_step(s)) {
        // (with residuals read back the last seam is done already)
        err = hipMemcpyAsync(s->x, s->px + last * H, H * sizeof(float), hipMemcpyDeviceToDevice, s->stream);
        if (err == hipSuccess) err = hipMemcpyAsync(s->y, s->py + last * H, H * sizeof(float), hipMemcpyDeviceToDevice, s->stream);
        DecodeRow row{s->x, s->r, b.due};
        if (err == hipSuccess) err = decode_head(s, row);
      } else if (err == hipSuccess && parallel_step(s)) {
        err = b.settle();
        if (err == hipSuccess) err = hipMemcpyAsync(s->x, s->px + last * H, H * sizeof(float), hipMemcpyDeviceToDevice, s->stream);
        DecodeRow row{s->x, nullptr, Seam{}};
        if (err == hipSuccess) err = decode_head(s, row);
      } else if (err == hipSuccess) {
        s->host_state[kStackWantedRows] = static_cast<uint32_t>(last);
        err = hipMemcpyAsync(s->pwant_rows, s->host_state + kStackWantedRows, sizeof(uint32_t), hipMemcpyHostToDevice, s->stream);
        if (err == hipSuccess) err = b.logits_of(s->pwant_rows, 1, s->logits);
        if (err == hipSuccess) err = sample_logits(s);
      }
      b.launches += 3;
    }
    out->kernel_launches += b.launches;
  }
  return err;
}

// ---- layout ----------------------------------------------------------------------------------

namespace {

struct LayerOffsets {
  uint64_t norm[8], w_in, w_out, talk, sink, z_bias, x_bias, w_up, w_down, act, q_norm, kv_norm, w_uq, w_uk, w_uv, router, e_in, e_out,
      shared_in, shared_out;
};

// Most tokens any reader of layer l's cache looks back over, itself included (0: one of them looks at everything).
uint32_t widest_view(const std::vector<StackLayer> &layers, size_t l) {
  uint32_t widest = 0;
  if (layers[l].spec.mixer == NERVA_HIP_MIXER_LATENT) return layers[l].spec.window_tokens;
  for (const StackLayer &r : layers) {
    if (r.spec.mixer != NERVA_HIP_MIXER_ATTENTION || r.cache_layer != l) continue;
    if (r.spec.chunk_tokens == 0) return 0;
    widest = std::max(widest, r.spec.chunk_tokens);
  }
  return widest;
}

bool rotation_valid(const NervaHipStackLayer &d, uint32_t dims) {
  return d.rotary_dims % 2 == 0 && d.rotary_dims <= dims && (d.rotary_dims == 0 || (d.rotary_base > 0.0f && isfinite(d.rotary_base)));
}

bool layer_valid(const NervaHipStackLayer *layers, uint32_t count, uint32_t l, uint32_t arrangement) {
  const NervaHipStackLayer &d = layers[l];
  constexpr uint64_t kMostColumns = 60 * 1024 / 2;
  if (d.ff > kMostColumns) return false;
  if (d.experts != 0) {
    if (arrangement != NERVA_HIP_STACK_PARALLEL || d.ff != 0 || d.experts > kMaxExperts || d.experts_per_token == 0 ||
        d.experts_per_token > d.experts || d.experts_per_token > kMaxTop || d.expert_ff == 0 || d.expert_ff > kMostColumns ||
        d.shared_ff > kMostColumns || !(d.expert_limit >= 0.0f) || (d.shared_ff != 0 && !(d.shared_limit >= 0.0f)))
      return false;
  } else if (d.shared_ff != 0) {
    return false;
  }
  if (d.mixer == NERVA_HIP_MIXER_LATENT)
    return d.heads != 0 && d.heads <= 65535u && d.key_dim != 0 && d.value_dim != 0 && d.q_rank != 0 && d.kv_rank != 0 &&
           d.q_rank <= kMostColumns && d.kv_rank <= kLatentMaxRank && static_cast<uint64_t>(d.kv_rank) + d.rotary_key_dim <= kLatentMaxRow &&
           static_cast<uint64_t>(d.heads) * d.value_dim <= kMostColumns && static_cast<uint64_t>(d.heads) * d.key_dim <= (1u << 24) &&
           isfinite(d.score_scale) && rotation_valid(d, d.rotary_key_dim);
  if (d.mixer == NERVA_HIP_MIXER_MINGRU) return d.width != 0 && static_cast<uint64_t>(d.width) * 2 <= 60 * 1024;
  if (d.mixer != NERVA_HIP_MIXER_ATTENTION) return false;
  if (d.heads == 0 || d.kv_heads == 0 || d.heads % d.kv_heads != 0 || d.key_dim == 0 || d.value_dim == 0 || !rotation_valid(d, d.key_dim) || d.value_dim > kMixedMaxValueDim || static_cast<uint64_t>(d.kv_heads) * d.key_dim > kMixedMaxFolded ||
      static_cast<uint64_t>(d.heads) * d.value_dim * 2 > 60 * 1024 || !isfinite(d.score_scale))
    return false;
  if (d.kv_layer == NERVA_HIP_OWN_KEYS) return true;
  // the layer it borrows from comes before it, has keys of its own, and they have this layer's shape
  if (d.kv_layer >= count || d.kv_layer >= l) return false;
  const NervaHipStackLayer &o = layers[d.kv_layer];
  return o.mixer == NERVA_HIP_MIXER_ATTENTION && o.kv_layer == NERVA_HIP_OWN_KEYS && o.kv_heads == d.kv_heads && o.key_dim == d.key_dim &&
         o.value_dim == d.value_dim;
}

// Rows of an input projection in the arena: as many as the matrix-core kernel for whole prompt blocks takes (a multiple of
// 192 or 256) where the padding is small; the rows past the layer's own hold nothing and are not read.
uint32_t padded_rows(uint32_t rows) {
  if (rows < 1536) return rows;
  return std::min((rows + 191) / 192 * 192, (rows + 255) / 256 * 256);
}

template <typename F>
bool create_checks(const NervaHipStackSessionCreateRequest *rq, bool synthetic, F &&unsupported) {
  if (rq == nullptr || rq->hidden == 0 || rq->vocab_size == 0 || rq->layer_count == 0 || rq->max_context_tokens == 0 ||
      rq->layers == nullptr || rq->precision > NERVA_HIP_PRECISION_32 || !(rq->norm_eps >= 0.0f) || !isfinite(rq->norm_eps) ||
      rq->arrangement > NERVA_HIP_STACK_PARALLEL || !isfinite(rq->embedding_scale) || !isfinite(rq->logit_scale) ||
      (rq->arrangement == NERVA_HIP_STACK_SANDWICH && rq->logit_scale != 1.0f))
    return false;
  if (rq->dtype != NERVA_HIP_DTYPE_BF16 || static_cast<uint64_t>(rq->hidden) * 2 > 60 * 1024) {
    unsupported();
    return false;
  }
  for (uint32_t l = 0; l < rq->layer_count; ++l)
    if (!layer_valid(rq->layers, rq->layer_count, l, rq->arrangement)) return false;
  // the weights come through a complete plan
  return synthetic || (rq->planned_weight_blocks != 0 && rq->planned_weight_bytes != 0 && rq->planned_weight_descriptors != nullptr &&
                       rq->planned_weight_descriptor_count == rq->planned_weight_blocks && rq->planned_weight_descriptor_hash != 0);
}

int create_stack(const NervaHipStackSessionCreateRequest *rq, bool synthetic, uint64_t seed, float weight_std,
                 NervaHipHfDecodeSequenceSessionCreateResult *out, Session **session_out) {
  if (!begin_result(out)) return -1;
  if (session_out == nullptr) return -1;
  *session_out = nullptr;
  out->failure_stage = 1;
  if (!create_checks(rq, synthetic, [&] { out->hip_error = NERVA_HIP_ERROR_NOT_SUPPORTED; })) return -1;
  if (!device_ready(&out->hip_error)) return -1;

  std::shared_ptr<StackModel> model(new (std::nothrow) StackModel());
  Session *s = new (std::nothrow) Session();
  if (s == nullptr || model == nullptr) {
    delete s;
    return -1;
  }
  s->weights = new (std::nothrow) SharedWeights();
  if (s->weights == nullptr) {
    delete s;
    return -1;
  }
  const uint64_t H = rq->hidden, V = rq->vocab_size;
  const uint32_t L = rq->layer_count;
  s->dtype = rq->dtype;
  s->hidden = rq->hidden;
  s->vocab = rq->vocab_size;
  s->layers = L;
  s->max_ctx = rq->max_context_tokens;
  s->eps = rq->norm_eps;
  s->planned_weight_blocks = rq->planned_weight_blocks;
  s->planned_gpu_resident_blocks = rq->planned_gpu_resident_blocks;
  s->planned_gpu_staged_blocks = rq->planned_gpu_staged_blocks;
  s->planned_weight_bytes = rq->planned_weight_bytes;
  s->planned_gpu_resident_weight_bytes = rq->planned_gpu_resident_weight_bytes;
  s->planned_gpu_staged_weight_bytes = rq->planned_gpu_staged_weight_bytes;
  s->planned_weight_descriptor_count = rq->planned_weight_descriptor_count;
  s->planned_weight_descriptor_hash = rq->planned_weight_descriptor_hash;

  // ---- layers: columns of the projections, rotations, caches, states
  StackModel &m = *model;
  m.precision = rq->precision;
  m.arrangement = rq->arrangement;
  m.embedding_scale = rq->embedding_scale;
  m.logit_scale = rq->logit_scale;
  const bool sandwich = m.arrangement == NERVA_HIP_STACK_SANDWICH;
  m.layers.resize(L);
  m.logical_blocks = (s->max_ctx + kKvBlockTokens - 1) / kKvBlockTokens;
  const uint64_t cache_elem = rq->precision == NERVA_HIP_PRECISION_32 ? 4 : 2;
  std::vector<std::pair<uint32_t, float>> rotations;   // (dims, base) met so far, in the order of their columns
  std::vector<uint32_t> rotation_at;
  // first column of a layer's angles in a token's rotation row
  const auto rotation_of = [&](const NervaHipStackLayer &d) {
    size_t r = 0;
    while (r < rotations.size() && rotations[r] != std::make_pair(d.rotary_dims, d.rotary_base)) ++r;
    if (r == rotations.size()) {
      rotations.emplace_back(d.rotary_dims, d.rotary_base);
      rotation_at.push_back(m.rotation_columns);
      const uint32_t half = d.rotary_dims / 2;
      for (uint32_t i = 0; i < half; ++i) {
        m.angle_step.push_back(static_cast<float>(pow(static_cast<double>(d.rotary_base), -2.0 * i / d.rotary_dims)));
        m.angle_cos.push_back(m.rotation_columns + i);
        m.angle_sin.push_back(m.rotation_columns + half + i);
      }
      m.rotation_columns += d.rotary_dims;
    }
    return rotation_at[r];
  };
  for (uint32_t l = 0; l < L; ++l) {
    StackLayer &w = m.layers[l];
    w.spec = rq->layers[l];
    const NervaHipStackLayer &d = w.spec;
    if (d.mixer == NERVA_HIP_MIXER_ATTENTION) {
      const bool own = d.kv_layer == NERVA_HIP_OWN_KEYS;
      w.cache_layer = own ? l : d.kv_layer;
      w.out_cols = d.heads * d.value_dim;
      w.k_col = w.q_col + d.heads * d.key_dim;
      w.v_col = w.k_col + (own ? d.kv_heads * d.key_dim : 0u);
      w.gate_col = w.v_col + (own ? d.kv_heads * d.value_dim : 0u);
      w.in_rows = w.gate_col + w.out_cols;
      w.rotation = rotation_of(d);
      s->heads = std::max(s->heads, d.heads);
      s->kv_heads = std::max(s->kv_heads, d.kv_heads);
      s->head_dim = std::max(s->head_dim, d.key_dim);
    } else if (d.mixer == NERVA_HIP_MIXER_LATENT) {
      w.cache_layer = l;
      w.out_cols = d.heads * d.value_dim;
      w.k_col = w.q_col + d.q_rank;
      w.gate_col = w.k_col + d.kv_rank + d.rotary_key_dim;
      w.in_rows = padded_rows(w.gate_col + w.out_cols);
      w.rotation = rotation_of(d);
      m.max_q_rank = std::max(m.max_q_rank, d.q_rank);
      m.max_q = std::max(m.max_q, w.q_rows());
      s->heads = std::max(s->heads, d.heads);
      s->kv_heads = std::max(s->kv_heads, 1u);
      s->head_dim = std::max(s->head_dim, d.key_dim + d.rotary_key_dim);
    } else {
      w.out_cols = d.width;
      w.in_rows = 3 * d.width;
      w.state_offset = m.state_floats;
      m.state_floats += (d.width + 63u) & ~63u;
    }
    m.max_in = std::max(m.max_in, w.in_rows);
    m.max_mix = std::max(m.max_mix, w.out_cols);
    m.max_ff = std::max({m.max_ff, d.ff, d.experts_per_token * d.expert_ff, d.shared_ff});
    if (d.experts != 0) {
      m.max_experts = std::max(m.max_experts, d.experts);
      m.max_top = std::max(m.max_top, d.experts_per_token);
    }
  }
  s->intermediate = m.max_ff;
  bool experts = !sandwich;
  for (const StackLayer &w : m.layers) experts = experts && w.spec.mixer == NERVA_HIP_MIXER_LATENT && w.spec.ff == 0;
  if (experts) m.block_tokens = kExpertBlockTokens;
  for (const StackLayer &w : m.layers)
    if (w.spec.experts != 0)
      m.plan_bytes = std::max(m.plan_bytes, moe_plan_bytes(m.block_tokens, w.spec.experts_per_token, w.spec.experts));
  for (uint32_t l = 0; l < L; ++l) {
    StackLayer &w = m.layers[l];
    if (!w.own_cache()) continue;
    // A block of token rows writes all its keys before its first query looks back: the oldest key that query may see
    // and the newest key written lie less than view + block_tokens positions apart, one block more for the edges.
    const uint32_t view = widest_view(m.layers, l);
    const uint64_t reach = (static_cast<uint64_t>(view) + m.block_tokens + kKvBlockTokens - 1) / kKvBlockTokens + 1;
    w.ring_blocks = view == 0 || reach > m.logical_blocks ? m.logical_blocks : static_cast<uint32_t>(reach);
    const auto area = [&](uint32_t dim) {
      const uint64_t at = m.cache_bytes;
      m.cache_bytes += (static_cast<uint64_t>(w.ring_blocks) * kKvBlockTokens * dim * cache_elem + 255u) & ~uint64_t{255};
      return at;
    };
    if (w.spec.mixer == NERVA_HIP_MIXER_LATENT) {
      w.k_offset = area(w.spec.kv_rank + w.spec.rotary_key_dim);
    } else {
      w.k_offset = area(w.spec.kv_heads * w.spec.key_dim);
      w.v_offset = area(w.spec.kv_heads * w.spec.value_dim);
    }
    w.table_offset = m.table_entries;
    m.table_entries += m.logical_blocks;
  }

  // ---- weight arena layout
  Carver c;
  const auto matrix = [&](uint64_t rows, uint64_t cols) {
    const uint64_t bytes = rows * cols * 2;
    return c.take(bytes, bytes >= kMatrixAlign ? kMatrixAlign : 8192u);
  };
  const uint64_t off_emb = matrix(V, H);
  std::vector<LayerOffsets> lo(L);
  for (uint32_t l = 0; l < L; ++l) {
    const StackLayer &w = m.layers[l];
    const NervaHipStackLayer &d = w.spec;
    for (uint64_t &at : lo[l].norm) at = c.take(H * 2);
    lo[l].w_in = matrix(w.in_rows, H);
    lo[l].w_out = matrix(H, w.out_cols);
    if (d.mixer == NERVA_HIP_MIXER_ATTENTION) {
      lo[l].talk = c.take(static_cast<uint64_t>(d.heads) * d.heads * 2);
      lo[l].sink = c.take(d.heads * 2ull);
    } else if (d.mixer == NERVA_HIP_MIXER_LATENT) {
      lo[l].q_norm = c.take(d.q_rank * 2ull);
      lo[l].kv_norm = c.take(d.kv_rank * 2ull);
      lo[l].w_uq = matrix(w.q_rows(), d.q_rank);
      lo[l].w_uk = matrix(d.heads * d.key_dim, d.kv_rank);
      lo[l].w_uv = matrix(w.out_cols, d.kv_rank);
    } else {
      lo[l].z_bias = c.take(d.width * 2ull);
      lo[l].x_bias = c.take(d.width * 2ull);
    }
    if (d.ff != 0) {
      lo[l].w_up = matrix(d.ff, H);
      lo[l].w_down = matrix(H, d.ff);
      lo[l].act = c.take(4);
    }
    if (d.experts != 0) {
      lo[l].router = matrix(d.experts, H);
      lo[l].e_in = matrix(2ull * d.experts * d.expert_ff, H);
      lo[l].e_out = matrix(d.experts * H, d.expert_ff);
      if (d.shared_ff != 0) {
        lo[l].shared_in = matrix(2ull * d.shared_ff, H);
        lo[l].shared_out = matrix(H, d.shared_ff);
      }
    }
  }
  const uint64_t off_final_w = c.take(H * 2), off_final_b = c.take(H * 2);
  const uint64_t off_head = sandwich ? off_emb : matrix(V, H);
  s->weights->bytes = c.offset;

  // ---- the plan's order of tensors: (offset in the arena, elements, kind of synthetic value)
  enum Kind { kMatrix, kUnit, kZero, kTalk };
  struct Piece {
    uint64_t off, elems;
    Kind kind;
    uint32_t n;
  };
  std::vector<Piece> pieces;
  const auto piece = [&](uint64_t off, uint64_t elems, Kind kind, uint32_t n = 0) { pieces.push_back(Piece{off, elems, kind, n}); };
  piece(off_emb, V * H, kMatrix);
  for (uint32_t l = 0; l < L; ++l) {
    const StackLayer &w = m.layers[l];
    const NervaHipStackLayer &d = w.spec;
    const bool ff = d.ff != 0 || d.experts != 0;
    for (uint32_t i = 0; i < (sandwich ? 4u : 1u) * (ff ? 2u : 1u); ++i) piece(lo[l].norm[i], H, i % 2 == 0 || !sandwich ? kUnit : kZero);
    const auto rows_of = [&](uint32_t first, uint32_t rows) { piece(lo[l].w_in + static_cast<uint64_t>(first) * H * 2, rows * H, kMatrix); };
    if (d.mixer == NERVA_HIP_MIXER_ATTENTION) {
      rows_of(w.q_col, d.heads * d.key_dim);
      if (w.own_cache()) {
        rows_of(w.k_col, d.kv_heads * d.key_dim);
        rows_of(w.v_col, d.kv_heads * d.value_dim);
      }
      rows_of(w.gate_col, w.out_cols);
      piece(lo[l].talk, static_cast<uint64_t>(d.heads) * d.heads, kTalk, d.heads);
      piece(lo[l].sink, d.heads, kZero);
    } else if (d.mixer == NERVA_HIP_MIXER_LATENT) {
      rows_of(w.q_col, d.q_rank);
      rows_of(w.k_col, d.kv_rank + d.rotary_key_dim);
      rows_of(w.gate_col, w.out_cols);
      piece(lo[l].q_norm, d.q_rank, kUnit);
      piece(lo[l].kv_norm, d.kv_rank, kUnit);
      piece(lo[l].w_uq, static_cast<uint64_t>(w.q_rows()) * d.q_rank, kMatrix);
      piece(lo[l].w_uk, static_cast<uint64_t>(d.heads) * d.key_dim * d.kv_rank, kMatrix);
      piece(lo[l].w_uv, static_cast<uint64_t>(w.out_cols) * d.kv_rank, kMatrix);
    } else {
      for (uint32_t i = 0; i < 3; ++i) rows_of(i * d.width, d.width);
      piece(lo[l].z_bias, d.width, kZero);
      piece(lo[l].x_bias, d.width, kZero);
    }
    piece(lo[l].w_out, H * w.out_cols, kMatrix);
    if (d.ff != 0) {
      piece(lo[l].w_up, d.ff * H, kMatrix);
      piece(lo[l].w_down, H * d.ff, kMatrix);
      piece(lo[l].act, 2, kZero);
    }
    if (d.experts != 0) {
      piece(lo[l].router, d.experts * H, kMatrix);
      const auto expert = [&](uint64_t in, uint64_t out, uint64_t i, uint64_t width) {
        const uint64_t n = width * H;
        piece(in + 4 * i * n, n, kMatrix);
        piece(in + (4 * i + 2) * n, n, kMatrix);
        piece(out + 2 * i * n, n, kMatrix);
      };
      for (uint32_t i = 0; i < d.experts; ++i) expert(lo[l].e_in, lo[l].e_out, i, d.expert_ff);
      if (d.shared_ff != 0) expert(lo[l].shared_in, lo[l].shared_out, 0, d.shared_ff);
    }
  }
  piece(off_final_w, H, kUnit);
  if (sandwich) piece(off_final_b, H, kZero);
  else piece(off_head, V * H, kMatrix);
  uint64_t elems = 0;
  for (const Piece &p : pieces) elems += p.elems;
  s->resident_weight_bytes = elems * 2;
  if (!synthetic && !validate_weight_descriptors(rq, s->resident_weight_bytes)) {
    destroy_session(s);
    return -1;
  }

  s->stack = model;
  hipError_t err = latent_wide_setup();
  if (err == hipSuccess) err = expert_rows_setup();
  if (err == hipSuccess) err = stack_setup_state(s, &out->failure_stage, true);
  uint64_t h2d = 0, syncs = 1;
  if (err == hipSuccess) {
    char *base = s->weights->base;
    const auto w16 = [&](uint64_t off) { return reinterpret_cast<const uint16_t *>(base + off); };
    s->emb = w16(off_emb);
    s->lm_head = w16(off_head);
    m.final_w = w16(off_final_w);
    m.final_b = w16(off_final_b);
    for (uint32_t l = 0; l < L; ++l) {
      StackLayer &w = m.layers[l];
      for (int i = 0; i < 8; ++i) w.norm[i] = w16(lo[l].norm[i]);
      w.w_in = w16(lo[l].w_in);
      w.w_out = w16(lo[l].w_out);
      if (w.spec.mixer == NERVA_HIP_MIXER_ATTENTION) {
        w.talk = w16(lo[l].talk);
        w.sink = w16(lo[l].sink);
      } else if (w.spec.mixer == NERVA_HIP_MIXER_LATENT) {
        w.q_norm = w16(lo[l].q_norm);
        w.kv_norm = w16(lo[l].kv_norm);
        w.w_uq = w16(lo[l].w_uq);
        w.w_uk = w16(lo[l].w_uk);
        w.w_uv = w16(lo[l].w_uv);
      } else {
        w.z_bias = w16(lo[l].z_bias);
        w.x_bias = w16(lo[l].x_bias);
      }
      if (w.spec.ff != 0) {
        w.w_up = w16(lo[l].w_up);
        w.w_down = w16(lo[l].w_down);
        w.act = w16(lo[l].act);
      }
      if (w.spec.experts != 0) {
        w.router = w16(lo[l].router);
        w.e_in = w16(lo[l].e_in);
        w.e_out = w16(lo[l].e_out);
        if (w.spec.shared_ff != 0) {
          w.shared_in = w16(lo[l].shared_in);
          w.shared_out = w16(lo[l].shared_out);
        }
      }
    }
    out->failure_stage = 4;
    if (synthetic) {
      for (size_t i = 0; err == hipSuccess && i < pieces.size(); ++i) {
        const Piece &p = pieces[i];
        err = launch_synth_16(base + p.off, s->dtype, seed, i + 1, p.elems, p.kind == kUnit ? 1.0f : 0.0f, weight_std, s->stream);
        if (err == hipSuccess && p.kind == kTalk) {
          hipLaunchKernelGGL(add_identity_kernel, dim3((p.n + 255u) / 256u), dim3(256), 0, s->stream,
                             reinterpret_cast<uint16_t *>(base + p.off), p.n);
          err = hipGetLastError();
        }
      }
      if (err == hipSuccess) err = hipStreamSynchronize(s->stream);
    } else {
      std::vector<WeightSegment> segments;
      uint64_t logical = 0;
      for (const Piece &p : pieces) {
        segments.push_back(WeightSegment{logical, p.elems * 2, base + p.off});
        logical += p.elems * 2;
      }
      err = copy_weight_descriptors(rq, segments, s->stream, &h2d, &syncs);
    }
  }
  if (err != hipSuccess) {
    out->hip_error = static_cast<int32_t>(err);
    destroy_session(s);
    return -1;
  }
  out->failure_stage = 0;
  fill_create_result(s, out);
  out->prefill_chunk_tokens = m.block_tokens;
  out->h2d_bytes = h2d;
  out->sync_calls = syncs;
  out->status = 0;
  *session_out = s;
  return 0;
}

}  // namespace

hipError_t nv::stack_setup_state(Session *s, int32_t *failure_stage, bool with_weights) {
  const StackModel &m = *s->stack;
  const uint64_t H = s->hidden, V = s->vocab, T = m.block_tokens, es = wide(s) ? 4 : 2;
  s->block_count = m.logical_blocks;
  s->kv_bytes = m.cache_bytes;
  s->stack_state_bytes = m.state_floats * sizeof(float);
  s->pgemm_ws_bytes = wide(s) ? 0 : gemm_block_workspace_bytes(static_cast<uint32_t>(std::max<uint64_t>({H, m.max_in, m.max_ff, m.max_q})));
  Carver c;
  const uint64_t off_cache = c.take(m.cache_bytes), off_tables = c.take(m.table_entries * 4ull), off_rec = c.take(s->stack_state_bytes);
  const uint64_t off_prompt = c.take(s->max_ctx * 4ull), off_slots = c.take(static_cast<uint64_t>(s->max_ctx) * sizeof(Slot)),
                 off_state = c.take(64);
  const uint64_t off_x = c.take(H * 4), off_r = c.take(H * 4), off_y = c.take(H * 4), off_in = c.take(m.max_in * 4ull),
                 off_logits = c.take(V * 4), off_mix16 = c.take(m.max_mix * 2ull), off_ff16 = c.take(m.max_ff * 2ull);
  const uint64_t angles = m.angle_step.size();
  const uint64_t off_angles = c.take(angles * 12 + 4);
  const uint64_t off_sample_ws = c.take(sample_workspace_bytes()), off_sampler_dev = c.take(sizeof(SamplerDev)),
                 off_sampler_keys = c.take(sampler_workspace_bytes(s->vocab));
  const uint64_t off_px = c.take(T * H * 4), off_py = c.take(T * H * 4), off_pin = c.take(T * m.max_in * 4),
                 off_pxn = c.take(T * H * es), off_pmix = c.take(T * m.max_mix * es), off_pff = c.take(T * m.max_ff * es),
                 off_prope = c.take(T * m.rotation_columns * 4ull + 4), off_pgemm = c.take(s->pgemm_ws_bytes);
  uint64_t attn_ws_bytes = 0;
  for (const StackLayer &w : m.layers)
    if (w.spec.mixer == NERVA_HIP_MIXER_ATTENTION && !wide(s) &&
        mixed_attention_wide(w.spec.heads, w.spec.kv_heads, w.spec.key_dim, w.spec.value_dim))
      attn_ws_bytes = std::max(attn_ws_bytes, mixed_attention_workspace_bytes(w.spec.heads, m.block_tokens));
    else if (w.spec.mixer == NERVA_HIP_MIXER_LATENT && !wide(s) &&
             latent_attention_wide(w.spec.heads, w.spec.key_dim, w.spec.rotary_key_dim, w.spec.value_dim, w.spec.kv_rank))
      attn_ws_bytes = std::max(attn_ws_bytes, latent_workspace_bytes(w.spec.heads, w.spec.rotary_key_dim, w.spec.kv_rank, m.block_tokens));
  const uint64_t off_attn_ws = c.take(attn_ws_bytes);
  const uint64_t off_want = c.take(kStackWantedRows * H * es), off_want_rows = c.take(kStackWantedRows * 4ull),
                 off_want_logits = c.take(kStackWantedRows * V * 4ull);
  const uint64_t both = parallel(s) ? T * H : 0;   // layers whose sublayers read the same row
  const uint64_t off_pxn2 = c.take(both * es), off_pz = c.take(both * 4), off_pql = c.take(T * m.max_q_rank * es),
                 off_pq = c.take(T * m.max_q * 4ull), off_router = c.take(T * m.max_experts * 4ull),
                 off_slots_rows = c.take(T * m.max_top * H * 4), off_plan = c.take(m.plan_bytes);
  s->state_bytes = c.offset;
  hipError_t err = allocate_session(s, failure_stage, with_weights);
  if (err != hipSuccess) return err;
  *failure_stage = 5;
  const auto f32 = [&](uint64_t off) { return reinterpret_cast<float *>(s->arena + off); };
  s->stack_cache = s->arena + off_cache;
  s->stack_tables = reinterpret_cast<uint32_t *>(s->arena + off_tables);
  s->stack_state = f32(off_rec);
  s->prompt = reinterpret_cast<uint32_t *>(s->arena + off_prompt);
  s->slots = reinterpret_cast<Slot *>(s->arena + off_slots);
  s->state = reinterpret_cast<uint32_t *>(s->arena + off_state);
  s->x = f32(off_x);
  s->r = f32(off_r);
  s->y = f32(off_y);
  s->qkv = f32(off_in);
  s->logits = f32(off_logits);
  s->attn16 = reinterpret_cast<uint16_t *>(s->arena + off_mix16);
  s->ff16 = reinterpret_cast<uint16_t *>(s->arena + off_ff16);
  s->rope_freq = f32(off_angles);
  s->sample_ws = s->arena + off_sample_ws;
  s->sampler_dev = reinterpret_cast<SamplerDev *>(s->arena + off_sampler_dev);
  s->sampler_keys = reinterpret_cast<uint64_t *>(s->arena + off_sampler_keys);
  s->px = f32(off_px);
  s->py = f32(off_py);
  s->pqkv = f32(off_pin);
  s->pxn = s->arena + off_pxn;
  s->pmix = s->arena + off_pmix;
  s->pff = s->arena + off_pff;
  s->prope = f32(off_prope);
  s->pgemm_ws = s->arena + off_pgemm;
  s->attn_ws = s->arena + off_attn_ws;
  s->pxn2 = s->arena + off_pxn2;
  s->pz = f32(off_pz);
  s->pql = s->arena + off_pql;
  s->pq = f32(off_pq);
  s->prouter = f32(off_router);
  s->pslots = f32(off_slots_rows);
  s->pplan = s->arena + off_plan;
  s->pwant = s->arena + off_want;
  s->pwant_rows = reinterpret_cast<uint32_t *>(s->arena + off_want_rows);
  s->pwant_logits = f32(off_want_logits);

  std::vector<uint32_t> tables(m.table_entries);
  for (const StackLayer &w : m.layers)
    if (w.own_cache())
      for (uint32_t b = 0; b < m.logical_blocks; ++b) tables[w.table_offset + b] = b % w.ring_blocks;
  if (!tables.empty()) err = hipMemcpy(s->stack_tables, tables.data(), tables.size() * 4, hipMemcpyHostToDevice);
  if (err == hipSuccess && angles != 0) {
    err = hipMemcpy(s->rope_freq, m.angle_step.data(), angles * 4, hipMemcpyHostToDevice);
    if (err == hipSuccess) err = hipMemcpy(s->rope_freq + angles, m.angle_cos.data(), angles * 4, hipMemcpyHostToDevice);
    if (err == hipSuccess) err = hipMemcpy(s->rope_freq + 2 * angles, m.angle_sin.data(), angles * 4, hipMemcpyHostToDevice);
  }
  if (err == hipSuccess) err = hipMemsetAsync(s->stack_cache, 0, m.cache_bytes, s->stream);
  if (err == hipSuccess && s->stack_state_bytes != 0) err = hipMemsetAsync(s->stack_state, 0, s->stack_state_bytes, s->stream);
  if (err == hipSuccess) err = hipMemsetAsync(s->slots, 0, static_cast<uint64_t>(s->max_ctx) * sizeof(Slot), s->stream);
  if (err == hipSuccess) err = hipMemsetAsync(s->state, 0, 64, s->stream);
  if (err == hipSuccess) err = hipMemsetAsync(s->sample_ws, 0, sample_workspace_bytes(), s->stream);
  if (err == hipSuccess) err = hipMemsetAsync(s->sampler_dev, 0, sizeof(SamplerDev), s->stream);
  if (err == hipSuccess) err = hipStreamSynchronize(s->stream);
  return err;
}

extern "C" {

int nerva_hip_stack_session_create(const NervaHipStackSessionCreateRequest *request, NervaHipHfDecodeSequenceSessionCreateResult *out,
                                   NervaHipHfDecodeSequenceSession **session) {
  return create_stack(request, false, 0, 0.0f, out, session);
}

int nerva_hip_bench_stack_session_create_synthetic(const NervaHipStackSessionCreateRequest *request, uint64_t seed, float weight_std,
                                                   NervaHipHfDecodeSequenceSessionCreateResult *out,
                                                   NervaHipHfDecodeSequenceSession **session) {
  return create_stack(request, true, seed, weight_std, out, session);
}

}  // extern "C"
