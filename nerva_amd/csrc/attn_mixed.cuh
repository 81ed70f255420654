// Attention whose heads' scores are mixed before the softmax ("talking heads"), with optional parts around it:
//   s_g    = scale * (rotate(q_g) . k_{g's kv head})                      every query head g, every visible key
//   s'_h   = sum_g M[h][g] s_g                                            M: learned [heads][heads]; absent = identity
//   p_h    = exp(s'_h - m) / (exp(sink_h - m) + sum_keys exp(s'_h - m))   sink: learned per head; absent = no such term
//   out_h  = sigmoid(gate_h) * sum_keys p_h v_{h's kv head}               gate: a projection of the layer's input, optional
// and a visibility rule by chunks: with chunk != 0 a query at position i sees the keys of its own chunk,
// chunk * (i / chunk) .. i, positions counted from the start of the sequence; chunk == 0 sees everything before it.
// Rotation covers the first rot_dims of a head (element i goes with element i + rot_dims / 2), the rest passes.
//
// Keys and values are cached per layer in blocks of 16 tokens behind a block table (attn_decode.cuh), after rotation,
// with their own widths (key_dim, value_dim), 16-bit or f32. A layer may read the cache of another one. A layer whose
// readers all look at bounded chunks keeps a ring of blocks: the table repeats, and a block is written again once no
// reader can look back that far.
//
// Since the mixing is linear, s'_h = (scale * sum_g M[h][g] rotate(q_g)) . K with the kv heads side by side: the
// general kernel folds M into one query of kv_heads * key_dim elements per head (f32). The kernels for wide layers mix
// scores instead (attn_mixed_wide.hip).
#pragma once

#include "attn_decode.cuh"

namespace nv {

constexpr uint32_t kNoColumn = ~0u;

struct MixedAttnParams {
  // projections of the token rows: [tokens][proj_stride] f32, first columns of the parts (gate_col may be kNoColumn)
  const float *proj;
  uint32_t proj_stride, q_col, k_col, v_col, gate_col;
  const uint16_t *talk;        // optional [heads][heads]
  const uint16_t *sink;        // optional [heads]
  void *k_cache, *v_cache;     // this layer's cache area: [block][kv_head][16][dim]
  const uint32_t *table;       // logical block -> block of the area
  const float *rope_cs;        // [tokens][rot_dims]: cos of the rot_dims / 2 angles, then sin
  uint32_t rot_dims, rope_stride;
  uint32_t heads, kv_heads, key_dim, value_dim;
  uint32_t chunk;
  float scale;
  uint32_t cache32;            // cache elements are f32
  uint32_t position;           // of the first token row; with `cursor` set the position is read from there
  const uint32_t *cursor;
  uint32_t max_steps, tokens;
  uint16_t *out16;             // [tokens][heads * value_dim], or null
  float *out32;                // likewise f32, used when out16 is null
  uint32_t packed_tiles;       // out16: != 0 -> matrix-operand order with that many token tiles
  void *workspace;             // the wide kernels' split partials (mixed_attention_workspace_bytes)
  uint32_t last_block;         // highest logical block a launch may meet (sizes the split grid of a captured step)
};

// Element d of a head after rotation; cs = cos | sin of the row's angles.
__device__ __forceinline__ float rotated_elem(const float *head, const float *cs, uint32_t rot_dims, uint32_t d) {
  if (d >= rot_dims) return head[d];
  const uint32_t half = rot_dims / 2;
  return d < half ? head[d] * cs[d] - head[d + half] * cs[half + d] : head[d] * cs[d - half] + head[d - half] * cs[d];
}

// Rotates the token rows' keys and writes keys and values to the cache.
hipError_t launch_mixed_publish(uint32_t dtype, const MixedAttnParams &p, hipStream_t stream);
// Attention of the token rows, whose own keys and values are in the cache. Any shape.
hipError_t launch_mixed_attention(uint32_t dtype, const MixedAttnParams &p, hipStream_t stream);
// Wide layers, 16-bit cache (attn_mixed_wide.hip): rotation, cache rows (append) and attention of a decode step (cursor
// set, one token: two launches) or of a block of token rows (three launches).
bool mixed_attention_wide(uint32_t heads, uint32_t kv_heads, uint32_t key_dim, uint32_t value_dim);
uint64_t mixed_attention_workspace_bytes(uint32_t heads, uint32_t max_tokens);
hipError_t launch_mixed_attention_wide(uint32_t dtype, const MixedAttnParams &p, bool append, hipStream_t stream);

constexpr uint32_t kMixedMaxValueDim = 1024;
constexpr uint32_t kMixedMaxFolded = 12288;   // kv_heads * key_dim (the folded query lies in LDS as f32)

}  // namespace nv
