// minGRU over a block of token rows (see mingru.cuh).
#include "mingru.cuh"

#include "activations.cuh"
#include "gemm_rows.cuh"

namespace nv {

namespace {

constexpr uint32_t kRuns = 16;   // waves of a workgroup = runs of tokens

template <uint32_t DT>
__global__ __launch_bounds__(kRuns *kWave) void mingru_rows_kernel(MinGruRows p) {
  __shared__ float keep_s[kRuns][kWave], add_s[kRuns][kWave];
  if (p.cursor != nullptr && *p.cursor >= p.max_steps) return;
  const uint32_t lane = threadIdx.x & (kWave - 1), run = threadIdx.x / kWave;
  const uint32_t ch = blockIdx.x * kWave + lane, W = p.width, T = p.tokens;
  const bool on = ch < W;
  const uint32_t c = on ? ch : W - 1;   // lanes past the width repeat its last channel and store nothing
  const uint32_t len = (T + kRuns - 1) / kRuns, t0 = min(run * len, T), t1 = min(t0 + len, T);
  const float zb = dec16<DT>(p.z_bias[c]), xb = dec16<DT>(p.x_bias[c]);
  const float start = p.state[c];
  const uint64_t stride = 3ull * W;
  const float *row = p.zxg + c;
  float keep = 1.0f, add = 0.0f;
  for (uint32_t t = t0; t < t1; ++t) {
    const float *at = row + t * stride;
    const float z = sigmoid(at[0] + zb), cand = mingru_candidate(at[W] + xb);
    keep *= 1.0f - z;
    add = (1.0f - z) * add + z * cand;
  }
  keep_s[run][lane] = keep;
  add_s[run][lane] = add;
  __syncthreads();
  float s = start;
  for (uint32_t r = 0; r < run; ++r) s = keep_s[r][lane] * s + add_s[r][lane];
  for (uint32_t t = t0; t < t1; ++t) {
    const float *at = row + t * stride;
    s = mingru_step(at[0] + zb, at[W] + xb, s);
    const float y = s * silu(at[2ull * W]);
    if (!on) continue;
    if (p.out16 == nullptr) p.out32[static_cast<uint64_t>(t) * W + ch] = y;
    else if (p.packed_tiles != 0) p.out16[gemm_x_packed_index(p.packed_tiles, t, ch)] = enc16<DT>(y);
    else p.out16[static_cast<uint64_t>(t) * W + ch] = enc16<DT>(y);
  }
  // the run that holds the last token leaves the state (every wave has read it before the barrier above)
  if (on && t1 == T && t0 < T) p.state[ch] = s;
}

}  // namespace

hipError_t launch_mingru_rows(uint32_t dtype, const MinGruRows &p, hipStream_t stream) {
  if (p.zxg == nullptr || p.z_bias == nullptr || p.x_bias == nullptr || p.state == nullptr || (p.out16 == nullptr) == (p.out32 == nullptr) ||
      p.tokens == 0 || p.width == 0)
    return hipErrorInvalidValue;
  if (p.packed_tiles != 0 && (p.out16 == nullptr || p.packed_tiles * 16u < p.tokens || p.width % 32 != 0)) return hipErrorInvalidValue;
  const dim3 grid((p.width + kWave - 1) / kWave);
  if (dtype == kBF16) hipLaunchKernelGGL(mingru_rows_kernel<kBF16>, grid, dim3(kRuns * kWave), 0, stream, p);
  else if (dtype == kF16) hipLaunchKernelGGL(mingru_rows_kernel<kF16>, grid, dim3(kRuns * kWave), 0, stream, p);
  else return hipErrorInvalidValue;
  return hipGetLastError();
}

}  // namespace nv
