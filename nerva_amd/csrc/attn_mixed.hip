// Attention with mixed heads, sink, output gate and chunks, for any shape (see attn_mixed.cuh).
#include "attn_mixed.cuh"

#include "activations.cuh"
#include "gemm_rows.cuh"

namespace nv {

namespace {

template <uint32_t DT, bool F32>
__device__ __forceinline__ void cache_store(void *base, uint64_t at, float v) {
  if constexpr (F32) static_cast<float *>(base)[at] = v;
  else static_cast<uint16_t *>(base)[at] = enc16<DT>(v);
}
template <uint32_t DT, bool F32>
__device__ __forceinline__ float cache_load(const void *base, uint64_t at) {
  if constexpr (F32) return static_cast<const float *>(base)[at];
  else return dec16<DT>(static_cast<const uint16_t *>(base)[at]);
}
template <uint32_t DT, bool F32>
__global__ __launch_bounds__(kBlock) void mixed_publish_kernel(MixedAttnParams p) {
  const uint32_t t = blockIdx.x;
  const uint32_t pos = p.cursor != nullptr ? *p.cursor : p.position + t;
  if (p.cursor != nullptr && pos >= p.max_steps) return;
  const uint32_t block = p.table[pos / kKvBlockTokens], row = pos % kKvBlockTokens;
  const float *src = p.proj + static_cast<uint64_t>(t) * p.proj_stride;
  const float *cs = p.rope_cs + static_cast<uint64_t>(t) * p.rope_stride;
  const uint32_t nk = p.kv_heads * p.key_dim, nv_ = p.kv_heads * p.value_dim;
  for (uint32_t i = threadIdx.x; i < nk; i += kBlock) {
    const uint32_t h = i / p.key_dim, d = i % p.key_dim;
    cache_store<DT, F32>(p.k_cache, kv_tile_offset(0, p.kv_heads, p.key_dim, 0, block, h) + kv_k_elem(p.key_dim, row, d),
                         rotated_elem(src + p.k_col + h * p.key_dim, cs, p.rot_dims, d));
  }
  for (uint32_t i = threadIdx.x; i < nv_; i += kBlock) {
    const uint32_t h = i / p.value_dim, d = i % p.value_dim;
    cache_store<DT, F32>(p.v_cache, kv_tile_offset(0, p.kv_heads, p.value_dim, 0, block, h) + kv_v_elem(p.value_dim, row, d),
                         src[p.v_col + i]);
  }
}

// One workgroup per (token row, head): lanes take keys for the scores and value columns for the sums.
constexpr uint32_t kValueRegs = kMixedMaxValueDim / kBlock;
template <uint32_t DT, bool F32>
__global__ __launch_bounds__(kBlock) void mixed_attention_kernel(MixedAttnParams p) {
  extern __shared__ __align__(16) float q_s[];   // folded query [kv_heads * key_dim]
  __shared__ float w_s[kBlock];                  // weights of the tile's keys
  __shared__ uint32_t block_s[kBlock / kKvBlockTokens + 1];
  __shared__ float red[kWavesPerBlock];
  const uint32_t t = blockIdx.x, h = blockIdx.y, group = p.heads / p.kv_heads;
  const uint32_t pos = p.cursor != nullptr ? *p.cursor : p.position + t;
  if (p.cursor != nullptr && pos >= p.max_steps) return;
  const float *src = p.proj + static_cast<uint64_t>(t) * p.proj_stride;
  const float *cs = p.rope_cs + static_cast<uint64_t>(t) * p.rope_stride;
  const uint32_t D = p.key_dim, folded = p.kv_heads * D, VD = p.value_dim;
  for (uint32_t i = threadIdx.x; i < folded; i += kBlock) {
    const uint32_t c = i / D, d = i % D;
    float sum = 0.0f;
    for (uint32_t r = 0; r < group; ++r) {
      const uint32_t g = c * group + r;
      const float m = p.talk != nullptr ? dec16<DT>(p.talk[h * p.heads + g]) : (g == h ? 1.0f : 0.0f);
      sum = fmaf(m, rotated_elem(src + p.q_col + g * D, cs, p.rot_dims, d), sum);
    }
    q_s[i] = sum * p.scale;
  }
  const uint32_t lo = p.chunk != 0 ? pos / p.chunk * p.chunk : 0u;
  const uint32_t kvh = h / group;
  // the sink is a key with its own score and no value: it starts the running maximum and sum
  float m = p.sink != nullptr ? dec16<DT>(p.sink[h]) : -INFINITY, l = p.sink != nullptr ? 1.0f : 0.0f;
  float acc[kValueRegs];
#pragma unroll
  for (uint32_t i = 0; i < kValueRegs; ++i) acc[i] = 0.0f;
  for (uint32_t base = lo / kKvBlockTokens * kKvBlockTokens; base <= pos; base += kBlock) {
    __syncthreads();   // the folded query is there; the last tile's weights and blocks are done with
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
      const uint32_t block = block_s[threadIdx.x / kKvBlockTokens];
      for (uint32_t c = 0; c < p.kv_heads; ++c) {
        const uint64_t tile = kv_tile_offset(0, p.kv_heads, D, 0, block, c);
        const float *q = q_s + c * D;
        if (D % 8 == 0) {   // eight dims of a row lie together in every tile order
          for (uint32_t d = 0; d < D; d += 8) {
            const uint64_t at = tile + kv_k_elem(D, row, d);
#pragma unroll
            for (uint32_t e = 0; e < 8; ++e) s = fmaf(q[d + e], cache_load<DT, F32>(p.k_cache, at + e), s);
          }
        } else {
          for (uint32_t d = 0; d < D; ++d) s = fmaf(q[d], cache_load<DT, F32>(p.k_cache, tile + kv_k_elem(D, row, d)), s);
        }
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
    for (uint32_t i = 0; i < kValueRegs; ++i) {
      const uint32_t d = i * kBlock + threadIdx.x;
      if (d >= VD) break;
      float a = acc[i] * keep;
      for (uint32_t k = first; k < n; ++k)
        a = fmaf(w_s[k],
                 cache_load<DT, F32>(p.v_cache, kv_tile_offset(0, p.kv_heads, VD, 0, block_s[k / kKvBlockTokens], kvh) +
                                                    kv_v_elem(VD, k % kKvBlockTokens, d)),
                 a);
      acc[i] = a;
    }
  }
  const uint64_t width = static_cast<uint64_t>(p.heads) * VD;
#pragma unroll
  for (uint32_t i = 0; i < kValueRegs; ++i) {
    const uint32_t d = i * kBlock + threadIdx.x;
    if (d >= VD) break;
    float o = l > 0.0f ? acc[i] / l : 0.0f;
    const uint32_t e = h * VD + d;
    if (p.gate_col != kNoColumn) o *= sigmoid(src[p.gate_col + e]);
    if (p.out16 == nullptr) p.out32[t * width + e] = o;
    else if (p.packed_tiles != 0) p.out16[gemm_x_packed_index(p.packed_tiles, t, e)] = enc16<DT>(o);
    else p.out16[t * width + e] = enc16<DT>(o);
  }
}

bool shape_ok(const MixedAttnParams &p) {
  return p.proj != nullptr && p.k_cache != nullptr && p.v_cache != nullptr && p.table != nullptr && p.heads != 0 && p.kv_heads != 0 &&
         p.heads % p.kv_heads == 0 && p.key_dim != 0 && p.value_dim != 0 && p.value_dim <= kMixedMaxValueDim &&
         p.kv_heads * p.key_dim <= kMixedMaxFolded && p.rot_dims % 2 == 0 && p.rot_dims <= p.key_dim &&
         (p.rot_dims == 0 || p.rope_cs != nullptr) && p.tokens != 0 && (p.cursor == nullptr || p.tokens == 1);
}

}  // namespace

hipError_t launch_mixed_publish(uint32_t dtype, const MixedAttnParams &p, hipStream_t stream) {
  if (!shape_ok(p) || dtype != kBF16) return hipErrorInvalidValue;
  if (p.cache32) hipLaunchKernelGGL((mixed_publish_kernel<kBF16, true>), dim3(p.tokens), dim3(kBlock), 0, stream, p);
  else hipLaunchKernelGGL((mixed_publish_kernel<kBF16, false>), dim3(p.tokens), dim3(kBlock), 0, stream, p);
  return hipGetLastError();
}

hipError_t launch_mixed_attention(uint32_t dtype, const MixedAttnParams &p, hipStream_t stream) {
  if (!shape_ok(p) || dtype != kBF16 || (p.out16 == nullptr) == (p.out32 == nullptr) || p.heads > 65535u) return hipErrorInvalidValue;
  if (p.packed_tiles != 0 && (p.out16 == nullptr || p.packed_tiles * 16u < p.tokens || p.heads * p.value_dim % 32 != 0))
    return hipErrorInvalidValue;
  const size_t lds = static_cast<size_t>(p.kv_heads) * p.key_dim * sizeof(float);
  const dim3 grid(p.tokens, p.heads);
  if (p.cache32) hipLaunchKernelGGL((mixed_attention_kernel<kBF16, true>), grid, dim3(kBlock), lds, stream, p);
  else hipLaunchKernelGGL((mixed_attention_kernel<kBF16, false>), grid, dim3(kBlock), lds, stream, p);
  return hipGetLastError();
}

}  // namespace nv
