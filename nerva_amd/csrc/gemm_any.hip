// Multi-row projection of any shape (see gemm_any.cuh).
#include "gemm_any.cuh"

#include "activations.cuh"
#include "gemm_rows.cuh"

namespace nv {

namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef _Float16 f16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));

template <uint32_t DT>
__device__ __forceinline__ f32x4_t mfma_k32(const uint4 &a, const uint4 &b, f32x4_t c) {
  if constexpr (DT == kBF16)
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c,
                                                   0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8_t, a), __builtin_bit_cast(f16x8_t, b), c, 0,
                                                  0, 0);
}

constexpr uint32_t kTile = 64;          // output rows and tokens of a workgroup
constexpr uint32_t kStep = 64;          // columns staged at a time (16-bit X)
constexpr uint32_t kPitch = kStep + 8;  // LDS row pitch: 16 bytes of padding

// Eight columns of a row from `c` on; columns past the end are zero.
template <bool VEC>
__device__ __forceinline__ uint4 piece8(const uint16_t *row, uint32_t c, uint32_t cols) {
  if constexpr (VEC) {
    return c < cols ? *reinterpret_cast<const uint4 *>(row + c) : make_uint4(0u, 0u, 0u, 0u);
  } else {
    uint32_t w[4];
#pragma unroll
    for (uint32_t e = 0; e < 4; ++e) {
      const uint32_t lo = c + 2 * e < cols ? row[c + 2 * e] : 0u, hi = c + 2 * e + 1 < cols ? row[c + 2 * e + 1] : 0u;
      w[e] = lo | (hi << 16);
    }
    return make_uint4(w[0], w[1], w[2], w[3]);
  }
}

template <uint32_t DT, int EPI, bool VEC>
__global__ __launch_bounds__(kBlock) void gemm_any_kernel(GemmAnyParams p) {
  __shared__ __align__(16) uint16_t ws[kTile * kPitch];
  __shared__ __align__(16) uint16_t xs[kTile * kPitch];
  const uint32_t lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
  const uint32_t row0 = blockIdx.x * kTile, tok0 = blockIdx.y * kTile;
  const uint32_t cols = p.cols;
  // staging: thread -> (row of the tile, eight columns), two rows of each operand
  const uint32_t sr = threadIdx.x / 8u, sc = (threadIdx.x % 8u) * 8u;
  const uint16_t *wr[2], *xr[2];
#pragma unroll
  for (uint32_t i = 0; i < 2; ++i) {
    wr[i] = p.w + static_cast<uint64_t>(min(row0 + sr + 32u * i, p.rows - 1)) * cols;
    xr[i] = p.x16 + static_cast<uint64_t>(min(tok0 + sr + 32u * i, p.tokens - 1)) * cols;
  }
  uint4 wq[2], xq[2];
#pragma unroll
  for (uint32_t i = 0; i < 2; ++i) {
    wq[i] = piece8<VEC>(wr[i], sc, cols);
    xq[i] = piece8<VEC>(xr[i], sc, cols);
  }
  f32x4_t acc[2][2];
#pragma unroll
  for (int a = 0; a < 2; ++a)
#pragma unroll
    for (int b = 0; b < 2; ++b) acc[a][b] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  const uint32_t n = lane & 15u, q = lane >> 4;
  const uint16_t *a_at = ws + ((wave & 1u) * 32u + n) * kPitch + q * 8u;
  const uint16_t *b_at = xs + ((wave >> 1) * 32u + n) * kPitch + q * 8u;
  for (uint32_t k = 0; k < cols; k += kStep) {
    __syncthreads();
#pragma unroll
    for (uint32_t i = 0; i < 2; ++i) {
      *reinterpret_cast<uint4 *>(ws + (sr + 32u * i) * kPitch + sc) = wq[i];
      *reinterpret_cast<uint4 *>(xs + (sr + 32u * i) * kPitch + sc) = xq[i];
    }
    __syncthreads();
    if (k + kStep < cols) {
#pragma unroll
      for (uint32_t i = 0; i < 2; ++i) {
        wq[i] = piece8<VEC>(wr[i], k + kStep + sc, cols);
        xq[i] = piece8<VEC>(xr[i], k + kStep + sc, cols);
      }
    }
#pragma unroll
    for (uint32_t s = 0; s < kStep / 32u; ++s) {
      uint4 a[2], b[2];
#pragma unroll
      for (uint32_t i = 0; i < 2; ++i) {
        a[i] = *reinterpret_cast<const uint4 *>(a_at + i * 16u * kPitch + s * 32u);
        b[i] = *reinterpret_cast<const uint4 *>(b_at + i * 16u * kPitch + s * 32u);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = mfma_k32<DT>(a[i], b[j], acc[i][j]);
    }
  }
  XieluParams act{};
  if constexpr (EPI == kGemmXielu) act = xielu_params<DT>(p.act);
#pragma unroll
  for (uint32_t j = 0; j < 2; ++j) {
    const uint32_t t = tok0 + (wave >> 1) * 32u + j * 16u + n;
    if (t >= p.tokens) continue;
#pragma unroll
    for (uint32_t i = 0; i < 2; ++i)
#pragma unroll
      for (uint32_t r = 0; r < 4; ++r) {
        const uint32_t row = row0 + (wave & 1u) * 32u + i * 16u + q * 4u + r;
        if (row >= p.rows) continue;
        const uint64_t at = static_cast<uint64_t>(t) * p.rows + row;
        if constexpr (EPI == kGemmXielu)
          p.out16[p.out_packed_tiles != 0 ? gemm_x_packed_index(p.out_packed_tiles, t, row) : at] = enc16<DT>(xielu(acc[i][j][r], act));
        else
          p.out_f32[at] = acc[i][j][r];
      }
  }
}

constexpr uint32_t kStep32 = 16;   // columns staged at a time (f32 X)

template <uint32_t DT, int EPI>
__global__ __launch_bounds__(kBlock) void gemm_any_f32_kernel(GemmAnyParams p) {
  __shared__ float ws[kStep32][kTile + 4], xs[kStep32][kTile + 4];
  const uint32_t row0 = blockIdx.x * kTile, tok0 = blockIdx.y * kTile, cols = p.cols;
  const uint32_t tr = threadIdx.x % 16u, tt = threadIdx.x / 16u;
  float acc[4][4] = {};
  for (uint32_t k = 0; k < cols; k += kStep32) {
    __syncthreads();
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) {
      const uint32_t r = threadIdx.x / 16u + 16u * i, c = threadIdx.x % 16u;
      const bool in = k + c < cols;
      ws[c][r] = in ? dec16<DT>(p.w[static_cast<uint64_t>(min(row0 + r, p.rows - 1)) * cols + k + c]) : 0.0f;
      xs[c][r] = in ? p.x32[static_cast<uint64_t>(min(tok0 + r, p.tokens - 1)) * cols + k + c] : 0.0f;
    }
    __syncthreads();
#pragma unroll
    for (uint32_t c = 0; c < kStep32; ++c)
#pragma unroll
      for (uint32_t i = 0; i < 4; ++i)
#pragma unroll
        for (uint32_t j = 0; j < 4; ++j) acc[i][j] = fmaf(ws[c][tr + 16u * i], xs[c][tt + 16u * j], acc[i][j]);
  }
  XieluParams act{};
  if constexpr (EPI == kGemmXielu) act = xielu_params<DT>(p.act);
#pragma unroll
  for (uint32_t j = 0; j < 4; ++j) {
    const uint32_t t = tok0 + tt + 16u * j;
    if (t >= p.tokens) continue;
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) {
      const uint32_t row = row0 + tr + 16u * i;
      if (row >= p.rows) continue;
      float y = acc[i][j];
      if constexpr (EPI == kGemmXielu) y = xielu(y, act);
      p.out_f32[static_cast<uint64_t>(t) * p.rows + row] = y;
    }
  }
}

template <uint32_t DT, int EPI>
hipError_t launch_epi(const GemmAnyParams &p, hipStream_t stream) {
  const dim3 grid((p.rows + kTile - 1) / kTile, (p.tokens + kTile - 1) / kTile);
  if (p.x16 == nullptr) {
    hipLaunchKernelGGL((gemm_any_f32_kernel<DT, EPI>), grid, dim3(kBlock), 0, stream, p);
  } else if (p.cols % 8 == 0 && (reinterpret_cast<uintptr_t>(p.w) & 15u) == 0 && (reinterpret_cast<uintptr_t>(p.x16) & 15u) == 0) {
    hipLaunchKernelGGL((gemm_any_kernel<DT, EPI, true>), grid, dim3(kBlock), 0, stream, p);
  } else {
    hipLaunchKernelGGL((gemm_any_kernel<DT, EPI, false>), grid, dim3(kBlock), 0, stream, p);
  }
  return hipGetLastError();
}

template <uint32_t DT>
hipError_t launch_dt(int epilogue, const GemmAnyParams &p, hipStream_t stream) {
  if (epilogue == kGemmF32) return launch_epi<DT, kGemmF32>(p, stream);
  if (epilogue == kGemmXielu) return launch_epi<DT, kGemmXielu>(p, stream);
  return hipErrorInvalidValue;
}

}  // namespace

hipError_t launch_gemm_any(uint32_t dtype, int epilogue, const GemmAnyParams &p, hipStream_t stream) {
  if (p.w == nullptr || (p.x16 == nullptr) == (p.x32 == nullptr) || p.rows == 0 || p.cols == 0 || p.tokens == 0 ||
      (p.tokens + kTile - 1) / kTile > 65535u)
    return hipErrorInvalidValue;
  const bool narrow = epilogue == kGemmXielu && p.x16 != nullptr;
  if (narrow ? p.out16 == nullptr : p.out_f32 == nullptr) return hipErrorInvalidValue;
  if (epilogue == kGemmXielu && p.act == nullptr) return hipErrorInvalidValue;
  if (p.out_packed_tiles != 0 && (!narrow || p.out_packed_tiles * 16u < p.tokens || p.rows % 32 != 0)) return hipErrorInvalidValue;
  if (dtype == kBF16) return launch_dt<kBF16>(epilogue, p, stream);
  if (dtype == kF16) return launch_dt<kF16>(epilogue, p, stream);
  return hipErrorInvalidValue;
}

}  // namespace nv
