// Attention over normalised latents (multi-head latent attention). A layer projects its input down to
//   dq  [q_rank], dkv [kv_rank], one rotated key part [rot_dim] for all heads, and a gate [heads * value_dim]
// and from there
//   q_h = W_uq rms(dq)  ([key_dim unrotated, rot_dim rotated] per head),  c = rms(dkv)
//   s   = scale * ((W_uk,h c) . q_h,unrotated + rotate(k) . rotate(q_h,rotated))
//   o_h = sigmoid(gate_h) * W_uv,h sum_j softmax(s)_j c_j
// with a sliding window: a query at position i sees i - window + 1 .. i (window 0: everything before it).
//
// What is cached per token is c and the rotated key part, side by side (kv_rank + rot_dim elements, after norm and
// rotation), one row for all heads, 16-bit or f32, in blocks of 16 tokens behind a block table (attn_decode.cuh). Scores
// are taken against the latent itself: W_uk is applied to the query instead of to every key, and W_uv to the weighted sum
// of latents, so that nothing is ever expanded per key. The cache of a layer with a window is a ring of blocks.
#pragma once

#include "attn_decode.cuh"

namespace nv {

constexpr uint32_t kLatentMaxRank = 2048, kLatentMaxRow = 4096;

// Element of (token row, dim) inside a cache block. Rows of whole 32-element runs lie in matrix-operand order: run by
// run, lane l = (d % 32 / 8) * 16 + row holding eight dims - one 1 KiB piece per run and block.
__host__ __device__ __forceinline__ uint32_t latent_elem(uint32_t width, uint32_t row, uint32_t d) {
  if (width % 32 != 0) return row * width + d;
  return d / 32u * 512u + ((d % 32u) / 8u * 16u + row) * 8u + d % 8u;
}

struct LatentAttnParams {
  // down projections of the token rows: [tokens][proj_stride] f32, first columns of the parts
  const float *proj;
  uint32_t proj_stride, q_col, kv_col, gate_col;
  const uint16_t *q_norm, *kv_norm;   // [q_rank], [kv_rank]
  float eps;
  const float *q;              // [tokens][heads * (key_dim + rot_dim)]: W_uq's output
  const uint16_t *w_uk;        // [heads * key_dim][kv_rank]
  const uint16_t *w_uv;        // [heads * value_dim][kv_rank]
  void *cache;                 // this layer's cache area: [block][16 x (kv_rank + rot_dim)]
  const uint32_t *table;       // logical block -> block of the area
  const float *rope_cs;        // [tokens][rope_stride]: cos of the rot_dims / 2 angles, then sin
  uint32_t rot_dims, rope_stride;   // rotation covers the first rot_dims of the rot_dim elements
  uint32_t heads, key_dim, rot_dim, value_dim, q_rank, kv_rank;
  uint32_t window;
  float scale;
  uint32_t cache32;            // cache elements are f32
  uint32_t position;           // of the first token row; with `cursor` set the position is read from there
  const uint32_t *cursor;
  uint32_t max_steps, tokens;
  uint16_t *q_latent16;        // launch_latent_prepare: rms(dq) as 16-bit rows [tokens][q_rank] ...
  float *q_latent32;           // ... or f32 ones
  uint32_t q_latent_tiles;     // q_latent16: != 0 -> matrix-operand order with that many token tiles
  uint16_t *out16;             // [tokens][heads * value_dim], or null
  float *out32;                // likewise f32, used when out16 is null
  uint32_t packed_tiles;       // out16: != 0 -> matrix-operand order with that many token tiles
  void *workspace;             // the wide kernels' queries, weighted latents and split partials (latent_workspace_bytes)
  uint32_t last_block;         // highest logical block a launch may meet (sizes the split grid of a captured step)
};

__device__ __forceinline__ uint32_t window_start(uint32_t pos, uint32_t window) {
  return window != 0 && pos >= window ? pos - window + 1 : 0u;
}

// Both norms of the token rows: rms(dq) for W_uq, the latent and the rotated key part into the cache.
hipError_t launch_latent_prepare(uint32_t dtype, const LatentAttnParams &p, hipStream_t stream);
// Attention of the token rows, whose own latents are in the cache. Any shape.
hipError_t launch_latent_attention(uint32_t dtype, const LatentAttnParams &p, hipStream_t stream);
// Wide layers, 16-bit cache (attn_latent_wide.hip): the same for a block of token rows (launch_latent_prepare has run) or
// for a decode step (cursor set, one token), which also writes the token's cache row.
bool latent_attention_wide(uint32_t heads, uint32_t key_dim, uint32_t rot_dim, uint32_t value_dim, uint32_t kv_rank);
uint64_t latent_workspace_bytes(uint32_t heads, uint32_t rot_dim, uint32_t kv_rank, uint32_t max_tokens);
hipError_t latent_wide_setup();   // once per process, outside stream capture
// (launches: counted up)
hipError_t launch_latent_attention_wide(uint32_t dtype, const LatentAttnParams &p, hipStream_t stream, uint64_t *launches);

}  // namespace nv
