// minGRU over a block of token rows (see mingru.cuh).
#include "mingru.cuh"

#include "activations.cuh"
#include "gemm_rows.cuh"

namespace nv {

namespace {

constexpr uint32_t kRuns = 16;       // runs of tokens of a workgroup
constexpr uint32_t kChannels = 32;   // channels of a workgroup: two runs a wave
constexpr uint32_t kHeld = 32;       // tokens of a run whose gates stay in registers between the two walks

template <uint32_t DT>
__global__ __launch_bounds__(kRuns *kChannels) void mingru_rows_kernel(MinGruRows p) {
  __shared__ float keep_s[kRuns][kChannels], add_s[kRuns][kChannels];
  if (p.cursor != nullptr && *p.cursor >= p.max_steps) return;
  const uint32_t lane = threadIdx.x % kChannels, run = threadIdx.x / kChannels;
  const uint32_t ch = blockIdx.x * kChannels + lane, W = p.width, T = p.tokens;
  const bool on = ch < W;
  const uint32_t c = on ? ch : W - 1;   // lanes past the width repeat its last channel and store nothing
  const uint32_t len = (T + kRuns - 1) / kRuns, t0 = min(run * len, T), t1 = min(t0 + len, T);
  const float zb = dec16<DT>(p.z_bias[c]), xb = dec16<DT>(p.x_bias[c]);
  const float start = p.state[c];
  const uint64_t stride = 3ull * W;
  const float *row = p.zxg + c;
  const bool held = len <= kHeld;   // (the same for the whole launch)
  float z[kHeld], cand[kHeld];
  float keep = 1.0f, add = 0.0f;
  if (held) {
#pragma unroll
    for (uint32_t i = 0; i < kHeld; ++i) {   // all requests of a run first; past its end they repeat the last token
      const float *at = row + min(t0 + i, T - 1) * stride;
      z[i] = at[0];
      cand[i] = at[W];
    }
#pragma unroll
    for (uint32_t i = 0; i < kHeld; ++i) {
      const bool in = t0 + i < t1;
      z[i] = in ? sigmoid(z[i] + zb) : 0.0f;   // a gate of zero leaves the state alone
      cand[i] = mingru_candidate(cand[i] + xb);
      keep *= 1.0f - z[i];
      add = (1.0f - z[i]) * add + z[i] * cand[i];
    }
  } else {
    for (uint32_t t = t0; t < t1; ++t) {
      const float *at = row + t * stride;
      const float g = sigmoid(at[0] + zb), u = mingru_candidate(at[W] + xb);
      keep *= 1.0f - g;
      add = (1.0f - g) * add + g * u;
    }
  }
  keep_s[run][lane] = keep;
  add_s[run][lane] = add;
  __syncthreads();
  float s = start;
  for (uint32_t r = 0; r < run; ++r) s = keep_s[r][lane] * s + add_s[r][lane];
  const auto store = [&](uint32_t t, float gate) {
    const float y = s * silu(gate);
    if (!on) return;
    if (p.out16 == nullptr) p.out32[static_cast<uint64_t>(t) * W + ch] = y;
    else if (p.packed_tiles != 0) p.out16[gemm_x_packed_index(p.packed_tiles, t, ch)] = enc16<DT>(y);
    else p.out16[static_cast<uint64_t>(t) * W + ch] = enc16<DT>(y);
  };
  if (held) {
    float g[kHeld];
#pragma unroll
    for (uint32_t i = 0; i < kHeld; ++i) g[i] = row[min(t0 + i, T - 1) * stride + 2ull * W];
#pragma unroll
    for (uint32_t i = 0; i < kHeld; ++i) {
      s = (1.0f - z[i]) * s + z[i] * cand[i];
      if (t0 + i < t1) store(t0 + i, g[i]);
    }
  } else {
    for (uint32_t t = t0; t < t1; ++t) {
      const float *at = row + t * stride;
      s = mingru_step(at[0] + zb, at[W] + xb, s);
      store(t, at[2ull * W]);
    }
  }
  // the run that holds the last token leaves the state (every lane has read it before the barrier above)
  if (on && t1 == T && t0 < T) p.state[ch] = s;
}

}  // namespace

hipError_t launch_mingru_rows(uint32_t dtype, const MinGruRows &p, hipStream_t stream) {
  if (p.zxg == nullptr || p.z_bias == nullptr || p.x_bias == nullptr || p.state == nullptr || (p.out16 == nullptr) == (p.out32 == nullptr) ||
      p.tokens == 0 || p.width == 0)
    return hipErrorInvalidValue;
  if (p.packed_tiles != 0 && (p.out16 == nullptr || p.packed_tiles * 16u < p.tokens || p.width % 32 != 0)) return hipErrorInvalidValue;
  const dim3 grid((p.width + kChannels - 1) / kChannels);
  if (dtype == kBF16) hipLaunchKernelGGL(mingru_rows_kernel<kBF16>, grid, dim3(kRuns * kChannels), 0, stream, p);
  else if (dtype == kF16) hipLaunchKernelGGL(mingru_rows_kernel<kF16>, grid, dim3(kRuns * kChannels), 0, stream, p);
  else return hipErrorInvalidValue;
  return hipGetLastError();
}

}  // namespace nv
