// RMS norm of token rows in f32, x / sqrt(mean(x^2) + eps) * gamma, for stacks whose sublayers of a layer read the same
// row, each through a norm of its own (norm_rms.hip, one workgroup per row). The row first takes in what the layer before
// it put out:
//   x' = x + (y[0] + (y[1] + sum_k slot_weight[k] slot_row[k]))
// (every part optional), then one root mean square serves all the outputs asked for.
#pragma once

#include "nv_common.cuh"

namespace nv {

struct RmsOut {
  const uint16_t *gamma;       // [cols]; null: this output is not wanted
  uint16_t *out16;             // one of out16 / out32
  float *out32;
  uint32_t packed_tiles;       // out16: != 0 -> matrix-operand order with that many token tiles (gemm_rows.cuh)
};
constexpr int kRmsOuts = 3;

struct RmsRows {
  float *x;                    // [tokens][cols]; x' replaces it (not where rows are picked)
  const float *y[2];           // optional [tokens][cols]
  const float *slot_rows;      // optional [tokens][slots][cols]
  const float *slot_weights;   // [tokens][slots]
  uint32_t slots;
  const uint32_t *pick;        // optional: output row i is source row pick[i], and x stays as it is
  RmsOut out[kRmsOuts];
  float gain;                  // factor on the outputs
  uint32_t tokens, cols;
  float eps;
};
hipError_t launch_rms_rows(uint32_t dtype, const RmsRows &p, hipStream_t stream);

}  // namespace nv
