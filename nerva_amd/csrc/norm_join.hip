// The seam between two sublayers for blocks of token rows (see norm_join.cuh): one workgroup per row.
#include "norm_join.cuh"

#include "gemm_rows.cuh"

namespace nv {

namespace {

template <uint32_t DT, int WG>
__global__ __launch_bounds__(WG *kWave) void join_rows_kernel(JoinRows p) {
  __shared__ float red[WG * 3];
  const uint32_t row = blockIdx.x, src = p.pick != nullptr ? p.pick[row] : row, cols = p.cols;
  JoinNorm j;
  float *x = p.x + static_cast<uint64_t>(src) * cols;
  j.x = x;
  j.y = p.y != nullptr ? p.y + static_cast<uint64_t>(src) * cols : nullptr;
  j.post_w = p.post_w;
  j.post_b = p.post_b;
  j.pre_w = p.pre_w;
  j.pre_b = p.pre_b;
  j.x_out = p.pick == nullptr && p.y != nullptr ? x : nullptr;   // (a lane stores only what it alone has read)
  j.eps = p.eps;
  join_norm_row<DT, WG>(j, cols, true, red, [&](uint32_t c, float v) {
    if (p.out32 != nullptr) p.out32[static_cast<uint64_t>(row) * cols + c] = v;
    else if (p.packed_tiles != 0) p.out16[gemm_x_packed_index(p.packed_tiles, row, c)] = enc16<DT>(v);
    else p.out16[static_cast<uint64_t>(row) * cols + c] = enc16<DT>(v);
  });
}

// Widths that are whole runs of eight columns: the lane's pieces are 16 bytes wide.
template <uint32_t DT, int WG>
__global__ __launch_bounds__(WG *kWave) void join_rows_vec_kernel(JoinRows p) {
  extern __shared__ __align__(16) uint16_t h[];
  __shared__ float red[WG * 3];
  constexpr uint32_t TB = WG * kWave;
  const uint32_t row = blockIdx.x, src = p.pick != nullptr ? p.pick[row] : row, cols = p.cols;
  JoinNorm j;
  float *x = p.x + static_cast<uint64_t>(src) * cols;
  j.x = x;
  j.y = p.y != nullptr ? p.y + static_cast<uint64_t>(src) * cols : nullptr;
  j.post_w = p.post_w;
  j.post_b = p.post_b;
  j.pre_w = p.pre_w;
  j.pre_b = p.pre_b;
  j.x_out = p.pick == nullptr && p.y != nullptr ? x : nullptr;
  j.eps = p.eps;
  JoinRegs r[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) join_load8(j, (static_cast<uint32_t>(i) * TB + threadIdx.x) * 8u, cols, r[i]);
  join_norm_regs<DT, WG, 2>(j, cols, true, r, red, h);
  // (every lane reads back the pieces it wrote itself)
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const uint32_t c = (static_cast<uint32_t>(i) * TB + threadIdx.x) * 8u;
    if (c >= cols) continue;
    const uint4 v = *reinterpret_cast<const uint4 *>(h + c);
    if (p.packed_tiles != 0) *reinterpret_cast<uint4 *>(p.out16 + gemm_x_packed_index(p.packed_tiles, row, c)) = v;
    else *reinterpret_cast<uint4 *>(p.out16 + static_cast<uint64_t>(row) * cols + c) = v;
  }
}

template <uint32_t DT>
hipError_t launch_dt(const JoinRows &p, hipStream_t stream) {
  const auto aligned = [](const void *q) { return (reinterpret_cast<uintptr_t>(q) & 15u) == 0; };
  if (p.out16 != nullptr && p.pre_w != nullptr && p.cols % 8 == 0 && p.cols <= 16384 && aligned(p.x) && aligned(p.y) &&
      aligned(p.post_w) && aligned(p.post_b) && aligned(p.pre_w) && aligned(p.pre_b) && aligned(p.out16)) {
    const size_t lds = static_cast<size_t>(p.cols) * sizeof(uint16_t);
    if (p.cols <= 4096)
      hipLaunchKernelGGL((join_rows_vec_kernel<DT, 4>), dim3(p.tokens), dim3(4 * kWave), lds, stream, p);
    else
      hipLaunchKernelGGL((join_rows_vec_kernel<DT, 16>), dim3(p.tokens), dim3(16 * kWave), lds, stream, p);
    return hipGetLastError();
  }
  if (p.cols <= 4096)
    hipLaunchKernelGGL((join_rows_kernel<DT, 4>), dim3(p.tokens), dim3(4 * kWave), 0, stream, p);
  else
    hipLaunchKernelGGL((join_rows_kernel<DT, 16>), dim3(p.tokens), dim3(16 * kWave), 0, stream, p);
  return hipGetLastError();
}

}  // namespace

hipError_t launch_join_rows(uint32_t dtype, const JoinRows &p, hipStream_t stream) {
  if (p.x == nullptr || p.tokens == 0 || p.cols == 0) return hipErrorInvalidValue;
  if (p.y != nullptr && (p.post_w == nullptr || p.post_b == nullptr)) return hipErrorInvalidValue;
  if (p.pre_w != nullptr && (p.pre_b == nullptr || (p.out16 == nullptr) == (p.out32 == nullptr))) return hipErrorInvalidValue;
  if (p.pre_w == nullptr && p.y == nullptr) return hipErrorInvalidValue;
  if (p.packed_tiles != 0 && (p.packed_tiles * 16u < p.tokens || p.cols % 32 != 0)) return hipErrorInvalidValue;
  if (dtype == kBF16) return launch_dt<kBF16>(p, stream);
  if (dtype == kF16) return launch_dt<kF16>(p, stream);
  return hipErrorInvalidValue;
}

}  // namespace nv
