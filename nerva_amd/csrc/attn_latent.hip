// Attention over normalised latents, for any shape (see attn_latent.cuh).
#include "attn_latent.cuh"

#include <algorithm>

#include "activations.cuh"
#include "attn_mixed.cuh"
#include "gemm_rows.cuh"

namespace nv {

namespace {

template <uint32_t DT, bool F32>
__device__ __forceinline__ void latent_store(void *base, uint64_t at, float v) {
  if constexpr (F32) static_cast<float *>(base)[at] = v;
  else static_cast<uint16_t *>(base)[at] = enc16<DT>(v);
}
template <uint32_t DT, bool F32>
__device__ __forceinline__ float latent_load(const void *base, uint64_t at) {
  if constexpr (F32) return static_cast<const float *>(base)[at];
  else return dec16<DT>(static_cast<const uint16_t *>(base)[at]);
}

// One workgroup per token row.
template <uint32_t DT, bool F32>
__global__ __launch_bounds__(kBlock) void latent_prepare_kernel(LatentAttnParams p) {
  __shared__ float red[kWavesPerBlock];
  const uint32_t t = blockIdx.x;
  const uint32_t pos = p.cursor != nullptr ? *p.cursor : p.position + t;
  if (p.cursor != nullptr && pos >= p.max_steps) return;
  const float *src = p.proj + static_cast<uint64_t>(t) * p.proj_stride;
  const float *cs = p.rope_cs + static_cast<uint64_t>(t) * p.rope_stride;
  const auto root = [&](const float *row, uint32_t n) {
    float ss = 0.0f;
    for (uint32_t i = threadIdx.x; i < n; i += kBlock) ss = fmaf(row[i], row[i], ss);
    return 1.0f / sqrtf(block_sum(ss, red) / static_cast<float>(n) + p.eps);
  };
  const float qs = root(src + p.q_col, p.q_rank), ks = root(src + p.kv_col, p.kv_rank);
  for (uint32_t i = threadIdx.x; i < p.q_rank; i += kBlock) {
    const float v = src[p.q_col + i] * qs * dec16<DT>(p.q_norm[i]);
    if (p.q_latent32 != nullptr) p.q_latent32[static_cast<uint64_t>(t) * p.q_rank + i] = v;
    else p.q_latent16[p.q_latent_tiles != 0 ? gemm_x_block_index(p.q_latent_tiles, t, i, p.q_rank) : static_cast<uint64_t>(t) * p.q_rank + i] = enc16<DT>(v);
  }
  const uint32_t width = p.kv_rank + p.rot_dim, row = pos % kKvBlockTokens;
  const uint64_t block = static_cast<uint64_t>(p.table[pos / kKvBlockTokens]) * kKvBlockTokens * width;
  for (uint32_t i = threadIdx.x; i < width; i += kBlock) {
    const float v = i < p.kv_rank ? src[p.kv_col + i] * ks * dec16<DT>(p.kv_norm[i])
                                  : rotated_elem(src + p.kv_col + p.kv_rank, cs, p.rot_dims, i - p.kv_rank);
    latent_store<DT, F32>(p.cache, block + latent_elem(width, row, i), v);
  }
}

// One workgroup per (token row, head): lanes take keys for the scores and latent columns for the sums.
constexpr uint32_t kRankRegs = kLatentMaxRank / kBlock;
template <uint32_t DT, bool F32>
__global__ __launch_bounds__(kBlock) void latent_attention_kernel(LatentAttnParams p) {
  extern __shared__ __align__(16) float q_s[];   // the head's query against a cache row [kv_rank + rot_dim]
  __shared__ float w_s[kBlock];                  // weights of the tile's keys
  __shared__ uint32_t block_s[kBlock / kKvBlockTokens + 1];
  __shared__ float red[kWavesPerBlock];
  const uint32_t t = blockIdx.x, h = blockIdx.y;
  const uint32_t pos = p.cursor != nullptr ? *p.cursor : p.position + t;
  if (p.cursor != nullptr && pos >= p.max_steps) return;
  const float *src = p.proj + static_cast<uint64_t>(t) * p.proj_stride;
  const float *cs = p.rope_cs + static_cast<uint64_t>(t) * p.rope_stride;
  const uint32_t R = p.kv_rank, width = R + p.rot_dim, head = p.key_dim + p.rot_dim;
  const float *q = p.q + (static_cast<uint64_t>(t) * p.heads + h) * head;
  const uint16_t *uk = p.w_uk + static_cast<uint64_t>(h) * p.key_dim * R;
  for (uint32_t i = threadIdx.x; i < width; i += kBlock) {
    float v = 0.0f;
    if (i < R)
      for (uint32_t d = 0; d < p.key_dim; ++d) v = fmaf(q[d], dec16<DT>(uk[static_cast<uint64_t>(d) * R + i]), v);
    else
      v = rotated_elem(q + p.key_dim, cs, p.rot_dims, i - R);
    q_s[i] = v * p.scale;
  }
  const uint32_t lo = window_start(pos, p.window);
  float m = -INFINITY, l = 0.0f;
  float acc[kRankRegs];
#pragma unroll
  for (uint32_t i = 0; i < kRankRegs; ++i) acc[i] = 0.0f;
  for (uint32_t base = lo / kKvBlockTokens * kKvBlockTokens; base <= pos; base += kBlock) {
    __syncthreads();   // the query is there; the last tile's weights and blocks are done with
    if (threadIdx.x < kBlock / kKvBlockTokens) {
      const uint32_t b = base / kKvBlockTokens + threadIdx.x;
      block_s[threadIdx.x] = p.table[min(b, pos / kKvBlockTokens)];
    }
    __syncthreads();
    const uint32_t key = base + threadIdx.x, row = threadIdx.x % kKvBlockTokens;
    const bool seen = key >= lo && key <= pos;
    float s = -INFINITY;
    if (seen) {
      s = 0.0f;
      const uint64_t tile = static_cast<uint64_t>(block_s[threadIdx.x / kKvBlockTokens]) * kKvBlockTokens * width;
      if (width % 8 == 0) {   // eight dims of a row lie together in every tile order
        for (uint32_t d = 0; d < width; d += 8) {
          const uint64_t at = tile + latent_elem(width, row, d);
#pragma unroll
          for (uint32_t e = 0; e < 8; ++e) s = fmaf(q_s[d + e], latent_load<DT, F32>(p.cache, at + e), s);
        }
      } else {
        for (uint32_t d = 0; d < width; ++d) s = fmaf(q_s[d], latent_load<DT, F32>(p.cache, tile + latent_elem(width, row, d)), s);
      }
    }
    float top = wave_max(s);
    if ((threadIdx.x & (kWave - 1)) == 0) red[threadIdx.x / kWave] = top;
    __syncthreads();
    top = m;
#pragma unroll
    for (int w = 0; w < kWavesPerBlock; ++w) top = fmaxf(top, red[w]);
    const float keep = m > -INFINITY ? expf(m - top) : 0.0f;
    const float weight = seen ? expf(s - top) : 0.0f;
    w_s[threadIdx.x] = weight;
    m = top;
    l = l * keep + block_sum(weight, red);   // (its barriers also publish w_s)
    const uint32_t n = min(pos + 1 - base, static_cast<uint32_t>(kBlock)), first = base < lo ? lo - base : 0u;
#pragma unroll
    for (uint32_t i = 0; i < kRankRegs; ++i) {
      const uint32_t d = i * kBlock + threadIdx.x;
      if (d >= R) break;
      float a = acc[i] * keep;
      for (uint32_t k = first; k < n; ++k)
        a = fmaf(w_s[k],
                 latent_load<DT, F32>(p.cache, static_cast<uint64_t>(block_s[k / kKvBlockTokens]) * kKvBlockTokens * width +
                                                   latent_elem(width, k % kKvBlockTokens, d)),
                 a);
      acc[i] = a;
    }
  }
  __syncthreads();   // the query is done with: the weighted latent takes its room
#pragma unroll
  for (uint32_t i = 0; i < kRankRegs; ++i) {
    const uint32_t d = i * kBlock + threadIdx.x;
    if (d < R) q_s[d] = acc[i] / l;
  }
  __syncthreads();
  const uint64_t out_width = static_cast<uint64_t>(p.heads) * p.value_dim;
  for (uint32_t j = threadIdx.x; j < p.value_dim; j += kBlock) {
    const uint32_t e = h * p.value_dim + j;
    const uint16_t *uv = p.w_uv + static_cast<uint64_t>(e) * R;
    float o = 0.0f;
    for (uint32_t d = 0; d < R; ++d) o = fmaf(dec16<DT>(uv[d]), q_s[d], o);
    o *= sigmoid(src[p.gate_col + e]);
    if (p.out16 == nullptr) p.out32[t * out_width + e] = o;
    else if (p.packed_tiles != 0) p.out16[gemm_x_block_index(p.packed_tiles, t, e, p.heads * p.value_dim)] = enc16<DT>(o);
    else p.out16[t * out_width + e] = enc16<DT>(o);
  }
}

bool shape_ok(const LatentAttnParams &p) {
  return p.proj != nullptr && p.cache != nullptr && p.table != nullptr && p.q_norm != nullptr && p.kv_norm != nullptr && p.heads != 0 &&
         p.heads <= 65535u && p.key_dim != 0 && p.value_dim != 0 && p.q_rank != 0 && p.kv_rank != 0 && p.kv_rank <= kLatentMaxRank &&
         p.kv_rank + p.rot_dim <= kLatentMaxRow && p.rot_dims % 2 == 0 && p.rot_dims <= p.rot_dim &&
         (p.rot_dims == 0 || p.rope_cs != nullptr) && p.tokens != 0 && (p.cursor == nullptr || p.tokens == 1);
}

}  // namespace

hipError_t launch_latent_prepare(uint32_t dtype, const LatentAttnParams &p, hipStream_t stream) {
  if (!shape_ok(p) || dtype != kBF16 || (p.q_latent16 == nullptr) == (p.q_latent32 == nullptr) ||
      (p.q_latent_tiles != 0 && (p.q_latent16 == nullptr || p.q_latent_tiles * 16u < std::min(p.tokens, kGemmDeepMaxTokens) || p.q_rank % 32 != 0)))
    return hipErrorInvalidValue;
  if (p.cache32) hipLaunchKernelGGL((latent_prepare_kernel<kBF16, true>), dim3(p.tokens), dim3(kBlock), 0, stream, p);
  else hipLaunchKernelGGL((latent_prepare_kernel<kBF16, false>), dim3(p.tokens), dim3(kBlock), 0, stream, p);
  return hipGetLastError();
}

hipError_t launch_latent_attention(uint32_t dtype, const LatentAttnParams &p, hipStream_t stream) {
  if (!shape_ok(p) || dtype != kBF16 || p.q == nullptr || p.w_uk == nullptr || p.w_uv == nullptr || (p.out16 == nullptr) == (p.out32 == nullptr))
    return hipErrorInvalidValue;
  if (p.packed_tiles != 0 && (p.out16 == nullptr || p.packed_tiles * 16u < std::min(p.tokens, kGemmDeepMaxTokens) || p.heads * p.value_dim % 32 != 0))
    return hipErrorInvalidValue;
  const size_t lds = static_cast<size_t>(p.kv_rank + p.rot_dim) * sizeof(float);
  const dim3 grid(p.tokens, p.heads);
  if (p.cache32) hipLaunchKernelGGL((latent_attention_kernel<kBF16, true>), grid, dim3(kBlock), lds, stream, p);
  else hipLaunchKernelGGL((latent_attention_kernel<kBF16, false>), grid, dim3(kBlock), lds, stream, p);
  return hipGetLastError();
}

}  // namespace nv
