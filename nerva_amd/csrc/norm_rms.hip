// RMS norm of token rows with the residual sum in front (see norm_rms.cuh).
#include "norm_rms.cuh"

#include <algorithm>

#include "gemm_rows.cuh"

namespace nv {

namespace {

// V consecutive columns a lane at a time; rows of more than kPieces such pieces a lane are walked again for the outputs.
constexpr int kPieces = 4;

template <int V>
struct Piece {
  float v[V];
};
template <int V>
__device__ __forceinline__ Piece<V> load_piece(const float *p) {
  Piece<V> r;
  if constexpr (V == 4) {
    const float4 q = *reinterpret_cast<const float4 *>(p);
    r.v[0] = q.x;
    r.v[1] = q.y;
    r.v[2] = q.z;
    r.v[3] = q.w;
  } else {
    r.v[0] = *p;
  }
  return r;
}
template <int V>
__device__ __forceinline__ void store_piece(float *p, const Piece<V> &r) {
  if constexpr (V == 4) *reinterpret_cast<float4 *>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
  else *p = r.v[0];
}

template <uint32_t DT, int WG, int V>
__global__ __launch_bounds__(WG *kWave) void rms_rows_kernel(RmsRows p) {
  __shared__ float red[WG];
  constexpr uint32_t TB = WG * kWave;
  const uint32_t row = blockIdx.x, src = p.pick != nullptr ? p.pick[row] : row, cols = p.cols;
  const uint64_t base = static_cast<uint64_t>(src) * cols;
  const float *weights = p.slot_rows != nullptr ? p.slot_weights + static_cast<uint64_t>(src) * p.slots : nullptr;
  const bool add = p.y[0] != nullptr || p.y[1] != nullptr || p.slot_rows != nullptr;
  const bool held = cols <= TB * V * kPieces;
  const auto joined = [&](uint32_t c) {
    Piece<V> x = load_piece<V>(p.x + base + c);
    if (!add) return x;
    Piece<V> s{};
    if (p.y[1] != nullptr) s = load_piece<V>(p.y[1] + base + c);
    if (p.slot_rows != nullptr) {
      Piece<V> e{};
      for (uint32_t k = 0; k < p.slots; ++k) {
        const Piece<V> r = load_piece<V>(p.slot_rows + (static_cast<uint64_t>(src) * p.slots + k) * cols + c);
#pragma unroll
        for (int i = 0; i < V; ++i) e.v[i] = fmaf(weights[k], r.v[i], e.v[i]);
      }
#pragma unroll
      for (int i = 0; i < V; ++i) s.v[i] += e.v[i];
    }
    if (p.y[0] != nullptr) {
      const Piece<V> y = load_piece<V>(p.y[0] + base + c);
#pragma unroll
      for (int i = 0; i < V; ++i) s.v[i] += y.v[i];
    }
#pragma unroll
    for (int i = 0; i < V; ++i) x.v[i] += s.v[i];
    return x;
  };
  Piece<V> keep[kPieces];
  float ss = 0.0f;
#pragma unroll
  for (int i = 0; i < kPieces; ++i) {
    const uint32_t c = (static_cast<uint32_t>(i) * TB + threadIdx.x) * V;
    keep[i] = Piece<V>{};
    if (c < cols) keep[i] = joined(c);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(keep[i].v[e], keep[i].v[e], ss);
  }
  if (!held)
    for (uint32_t c = (kPieces * TB + threadIdx.x) * V; c < cols; c += TB * V) {
      const Piece<V> x = joined(c);
#pragma unroll
      for (int e = 0; e < V; ++e) ss = fmaf(x.v[e], x.v[e], ss);
    }
  const float scale = p.gain / sqrtf(block_sum_n<WG>(ss, red) / static_cast<float>(cols) + p.eps);
  const auto emit = [&](uint32_t c, const Piece<V> &x) {
#pragma unroll
    for (int o = 0; o < kRmsOuts; ++o) {
      const RmsOut &out = p.out[o];
      if (out.gamma == nullptr) continue;
      Piece<V> h;
#pragma unroll
      for (int e = 0; e < V; ++e) h.v[e] = x.v[e] * scale * dec16<DT>(out.gamma[c + e]);
      const uint64_t at = static_cast<uint64_t>(row) * cols + c;
      if (out.out32 != nullptr) {
        store_piece<V>(out.out32 + at, h);
      } else {
        // (four columns stay together in operand order)
        uint16_t *to = out.out16 + (out.packed_tiles != 0 ? gemm_x_block_index(out.packed_tiles, row, c, cols) : at);
        if constexpr (V == 4)
          *reinterpret_cast<uint2 *>(to) = make_uint2(enc16<DT>(h.v[0]) | (static_cast<uint32_t>(enc16<DT>(h.v[1])) << 16),
                                                      enc16<DT>(h.v[2]) | (static_cast<uint32_t>(enc16<DT>(h.v[3])) << 16));
        else
          *to = enc16<DT>(h.v[0]);
      }
    }
    // (a lane stores only what it alone has read)
    if (add && p.pick == nullptr) store_piece<V>(p.x + base + c, x);
  };
#pragma unroll
  for (int i = 0; i < kPieces; ++i) {
    const uint32_t c = (static_cast<uint32_t>(i) * TB + threadIdx.x) * V;
    if (c < cols) emit(c, keep[i]);
  }
  if (!held)
    for (uint32_t c = (kPieces * TB + threadIdx.x) * V; c < cols; c += TB * V) emit(c, joined(c));
}

template <uint32_t DT>
hipError_t launch_dt(const RmsRows &p, hipStream_t stream) {
  const auto aligned = [](const void *q) { return (reinterpret_cast<uintptr_t>(q) & 15u) == 0; };
  bool vec = p.cols % 4 == 0 && aligned(p.x) && aligned(p.y[0]) && aligned(p.y[1]) && aligned(p.slot_rows);
  for (const RmsOut &o : p.out) vec = vec && aligned(o.out16) && aligned(o.out32);
  if (!vec) hipLaunchKernelGGL((rms_rows_kernel<DT, 4, 1>), dim3(p.tokens), dim3(4 * kWave), 0, stream, p);
  else if (p.cols <= 4096) hipLaunchKernelGGL((rms_rows_kernel<DT, 4, 4>), dim3(p.tokens), dim3(4 * kWave), 0, stream, p);
  else hipLaunchKernelGGL((rms_rows_kernel<DT, 16, 4>), dim3(p.tokens), dim3(16 * kWave), 0, stream, p);
  return hipGetLastError();
}

}  // namespace

hipError_t launch_rms_rows(uint32_t dtype, const RmsRows &p, hipStream_t stream) {
  if (p.x == nullptr || p.tokens == 0 || p.cols == 0) return hipErrorInvalidValue;
  if (p.slot_rows != nullptr && (p.slot_weights == nullptr || p.slots == 0)) return hipErrorInvalidValue;
  for (const RmsOut &o : p.out) {
    if (o.gamma != nullptr && (o.out16 == nullptr) == (o.out32 == nullptr)) return hipErrorInvalidValue;
    if (o.packed_tiles != 0 && (o.packed_tiles * 16u < std::min(p.tokens, kGemmDeepMaxTokens) || p.cols % 32 != 0)) return hipErrorInvalidValue;
  }
  if (dtype == kBF16) return launch_dt<kBF16>(p, stream);
  return hipErrorInvalidValue;
}

}  // namespace nv
