// minGRU over a block of token rows: the gates of every token are known before the recurrence starts (they read the
// token alone), so S_t = (1 - z_t) S_{t-1} + z_t c_t is a first-order linear recurrence that a block of tokens
// evaluates in pieces: half a wave takes a run of consecutive tokens for 32 channels and reduces it to (product of 1 - z,
// result from a zero state); the runs' results chain through LDS; then each walks its run again - from registers, for
// blocks of up to 512 tokens - from the state it now knows and writes the gated outputs. A decode step has the recurrence in the epilogue of its
// projection (gemv_stream.cuh) instead.
#pragma once

#include "nv_common.cuh"

namespace nv {

struct MinGruRows {
  const float *zxg;          // [tokens][3 width]: gate, candidate and output-gate pre-activations
  const uint16_t *z_bias, *x_bias;   // [width]
  float *state;              // [width], advanced by `tokens` steps
  uint16_t *out16;           // [tokens][width] S_t * silu(g), or null
  float *out32;              // likewise f32, used when out16 is null
  uint32_t packed_tiles;     // out16: != 0 -> matrix-operand order with that many token tiles
  uint32_t tokens, width;
  const uint32_t *cursor;    // optional step guard: nothing happens when *cursor >= max_steps
  uint32_t max_steps;
};
hipError_t launch_mingru_rows(uint32_t dtype, const MinGruRows &p, hipStream_t stream);

}  // namespace nv
