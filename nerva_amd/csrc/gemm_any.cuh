// Multi-row projection for shapes the streaming kernels (gemm_rows.cuh) do not take - any number of rows, columns and
// tokens - and for sessions that compute everything in 32 bits. Y[t][r] = sum_c W[r][c] X[t][c], W 16-bit:
//   16-bit X: 64 x 64 output tiles on the matrix cores (v_mfma_f32_16x16x32), both operands staged through LDS with the
//             next K-step's pieces in registers;
//   f32 X:    64 x 64 output tiles on the vector ALU, every product and sum in f32.
#pragma once

#include "nv_common.cuh"

namespace nv {

struct GemmAnyParams {
  const uint16_t *w;       // [rows][cols]
  const uint16_t *x16;     // [tokens][cols], or null
  const float *x32;        // [tokens][cols], used when x16 is null
  uint32_t rows, cols, tokens;
  float *out_f32;          // kGemmF32: [tokens][rows]; kGemmXielu with f32 X: likewise, the activation applied
  uint16_t *out16;         // kGemmXielu with 16-bit X: [tokens][rows]
  uint32_t out_packed_tiles;   // out16: != 0 -> matrix-operand order with that many token tiles
  const uint16_t *act;     // kGemmXielu
};
// epilogue: kGemmF32 or kGemmXielu (gemm_rows.cuh)
hipError_t launch_gemm_any(uint32_t dtype, int epilogue, const GemmAnyParams &p, hipStream_t stream);

}  // namespace nv
