// Attention with mixed heads (attn_mixed.cuh) for wide layers: head width 128, 16-bit cache. The heads' scores are mixed
// as scores - not folded into the query, which would cost kv_heads times the products - and since every head needs every
// other head's scores for the same key, a workgroup holds all heads: one wave per kv head.
//
// Decode step (mixed_decode_kernel): split-KV. A workgroup takes a run of 16-key blocks; its waves request the K and V
// tiles of four blocks at once (matrix-operand order, attn_decode.cuh), leave their heads' scores of 64 keys in LDS, and
// each reads back all heads' scores with one key per lane to form its own heads' mixed scores in f32. Queries and weights
// enter the matrix cores as hi + lo 16-bit halves in separate columns of the tile.
//
// Prompt blocks (mixed_prompt_kernel): a workgroup takes eight consecutive tokens - the sixteen columns of a tile are
// eight tokens x two heads - and 32 keys at a time. The scores of all heads meet in LDS as [key][token][head], where the
// mixing is a matrix product again: M (exact in 16 bits) times the scores as three 16-bit pieces each (hi + mid + lo =
// the f32 value to its last bits), in place, each wave its own columns; then every wave reads its heads back and goes on
// as in ordinary attention. Splits of the key range run along the fastest grid dimension, so that the workgroups of an
// XCD read the same keys.
//
// Either way a split leaves un-normalised sums with their maximum and denominator, and a second launch merges the splits,
// adds the sink to the denominator and applies the output gate.
#include <algorithm>
#include <mutex>

#include "activations.cuh"
#include "attn_mixed.cuh"
#include "attn_tile.cuh"
#include "gemm_rows.cuh"

namespace nv {

namespace {

using namespace attn;

constexpr uint32_t kDecodeSplits = 256, kMinBlocksPerSplit = 4;
constexpr uint32_t kPromptTokens = 8;          // tokens of a workgroup
constexpr uint32_t kPromptWorkgroups = 256;    // split the keys until about so many are there
constexpr uint32_t kPromptSplits = 64;
constexpr uint32_t kWideHeads = 32;            // heads a prompt workgroup mixes (one K-step of the mixing product)

// Split partials: sums [(token * splits + split) * heads + head][128], then the maxima, then the denominators.
struct Partials {
  float *sum, *m, *l;
};
__host__ __device__ __forceinline__ Partials partials_of(void *ws, uint64_t entries) {
  Partials r;
  r.sum = static_cast<float *>(ws);
  r.m = r.sum + entries * kHD;
  r.l = r.m + entries;
  return r;
}

struct Range {
  uint32_t first, count, per_split, active;   // units of keys: first unit, units, units of a split, splits that have any
};
__device__ __forceinline__ Range split_range(uint32_t first, uint32_t count, uint32_t splits, uint32_t least) {
  const uint32_t per = max((count + splits - 1) / splits, least);
  return Range{first, count, per, (count + per - 1) / per};
}
__device__ __forceinline__ uint32_t first_seen(const MixedAttnParams &p, uint32_t pos) {
  return p.chunk != 0 ? pos / p.chunk * p.chunk : 0u;
}
__device__ __forceinline__ Range decode_range(const MixedAttnParams &p, uint32_t pos, uint32_t splits) {
  const uint32_t b0 = first_seen(p, pos) / kKvBlockTokens;
  return split_range(b0, pos / kKvBlockTokens - b0 + 1, splits, kMinBlocksPerSplit);
}
// Units of two blocks.
__device__ __forceinline__ Range prompt_range(const MixedAttnParams &p, uint32_t tile, uint32_t splits) {
  const uint32_t t0 = tile * kPromptTokens, t1 = min(t0 + kPromptTokens, p.tokens) - 1;
  const uint32_t b0 = first_seen(p, p.position + t0) / kKvBlockTokens;
  return split_range(b0, ((p.position + t1) / kKvBlockTokens - b0) / 2 + 1, splits, 1);
}

__device__ __forceinline__ uint32_t pack16(float a, float b) {
  return enc16_finite<kBF16>(a) | (static_cast<uint32_t>(enc16_finite<kBF16>(b)) << 16);
}

// ---- decode step -----------------------------------------------------------------------------

constexpr uint32_t kKeysPitch = 68;   // floats of a head's 64 scores in LDS
template <int R>
__global__ __launch_bounds__(512, 2) void mixed_decode_kernel(MixedAttnParams p, uint32_t splits, uint32_t append) {
  constexpr uint32_t DT = kBF16;
  extern __shared__ __align__(16) float lds[];
  const uint32_t H = p.heads;
  float *s_s = lds, *t_s = s_s + H * kHD;   // (the scores' room holds the queries first: 128 floats a head)
  uint16_t *w_s = reinterpret_cast<uint16_t *>(t_s + H * H);   // [hi | lo][head][64]
  const uint32_t pos = p.cursor != nullptr ? *p.cursor : p.position;
  if (p.cursor != nullptr && pos >= p.max_steps) return;
  const Range range = decode_range(p, pos, splits);
  const uint32_t split = blockIdx.x;
  if (split >= range.active) return;
  const uint32_t b0 = range.first + split * range.per_split, b1 = min(b0 + range.per_split, range.first + range.count);
  const uint32_t lane = threadIdx.x & (kWave - 1), c = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const uint32_t n = lane & 15u, q4 = lane >> 4;
  uint16_t *kc = static_cast<uint16_t *>(p.k_cache), *vc = static_cast<uint16_t *>(p.v_cache);

  if (append != 0 && b1 * kKvBlockTokens > pos) {   // the split with the newest block writes this token's rows first
    const uint32_t block = p.table[pos / kKvBlockTokens], row = pos % kKvBlockTokens;
    const uint64_t tile = kv_tile_offset(0, p.kv_heads, kHD, 0, block, c);
#pragma unroll
    for (uint32_t i = 0; i < 2; ++i) {
      const uint32_t d = lane + 64u * i;
      kc[tile + kv_k_elem(kHD, row, d)] = enc16<DT>(rotated_elem(p.proj + p.k_col + c * kHD, p.rope_cs, p.rot_dims, d));
      vc[tile + kv_v_elem(kHD, row, d)] = enc16<DT>(p.proj[p.v_col + c * kHD + d]);
    }
    __threadfence_block();   // (a wave reads back only the tiles of its own kv head)
  }
  uint4 kreg[4][4], vreg[4][4];
  const auto request = [&](uint32_t b) {
#pragma unroll
    for (uint32_t t = 0; t < 4; ++t) {
      const uint64_t tile = kv_tile_offset(0, p.kv_heads, kHD, 0, p.table[min(b + t, b1 - 1)], c) + lane * 8u;
#pragma unroll
      for (uint32_t j = 0; j < 4; ++j) kreg[t][j] = *reinterpret_cast<const uint4 *>(kc + tile + j * 512u);
#pragma unroll
      for (uint32_t j = 0; j < 4; ++j) vreg[t][j] = *reinterpret_cast<const uint4 *>(vc + tile + j * 512u);
    }
  };
  request(b0);   // the first four blocks are on their way while the queries are prepared

  for (uint32_t i = threadIdx.x; i < H * H; i += blockDim.x)   // M transposed: a wave's heads of one source lie together
    t_s[i % H * H + i / H] = p.talk != nullptr ? dec16<DT>(p.talk[i]) : (i / H == i % H ? 1.0f : 0.0f);
  // queries of this kv head, rotated and scaled, through LDS (the scores' room): columns 0..R-1 hi halves, 8..8+R-1 lo
  float *q_s = s_s + c * R * kHD;
#pragma unroll
  for (int r = 0; r < R; ++r)
#pragma unroll
    for (uint32_t i = 0; i < 2; ++i) {
      const uint32_t d = lane + 64u * i;
      q_s[r * kHD + d] = rotated_elem(p.proj + p.q_col + (c * R + r) * kHD, p.rope_cs, p.rot_dims, d) * (p.scale * kLog2e);
    }
  __syncthreads();
  uint4 qx[4];
  {
    const uint32_t r = n & 7u;
    const float *head = q_s + min(r, static_cast<uint32_t>(R - 1)) * kHD;
#pragma unroll
    for (uint32_t j = 0; j < 4; ++j) {
      uint32_t w[4];
#pragma unroll
      for (uint32_t e = 0; e < 4; ++e) {
        const uint32_t d = j * 32u + q4 * 8u + 2u * e;
        uint16_t h0, l0, h1, l1;
        split16<DT>(head[d], h0, l0);
        split16<DT>(head[d + 1], h1, l1);
        w[e] = n < 8u ? (h0 | (static_cast<uint32_t>(h1) << 16)) : (l0 | (static_cast<uint32_t>(l1) << 16));
      }
      qx[j] = r < static_cast<uint32_t>(R) ? make_uint4(w[0], w[1], w[2], w[3]) : make_uint4(0u, 0u, 0u, 0u);
    }
  }
  __syncthreads();   // the scores take the queries' room

  const uint32_t lo = first_seen(p, pos);
  float m[R], l[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    m[r] = -INFINITY;
    l[r] = 0.0f;
  }
  f32x4_t acc[8];
#pragma unroll
  for (int s = 0; s < 8; ++s) acc[s] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};

  for (uint32_t b = b0; b < b1; b += 4) {
    if (b != b0) request(b);
#pragma unroll
    for (uint32_t t = 0; t < 4; ++t) {
      f32x4_t s = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int j = 0; j < 4; ++j) s = mfma_k32<DT>(kreg[t][j], qx[j], s);
#pragma unroll
      for (int i = 0; i < 4; ++i) s[i] += __shfl_xor(s[i], 8, kWave);
      if (n < static_cast<uint32_t>(R))
        *reinterpret_cast<float4 *>(s_s + (c * R + n) * kKeysPitch + t * 16u + q4 * 4u) = make_float4(s[0], s[1], s[2], s[3]);
    }
    __syncthreads();
    // one key per lane: this wave's heads as combinations of all heads
    const uint32_t key = b * kKvBlockTokens + lane;
    const bool seen = key >= lo && key <= pos && b + lane / kKvBlockTokens < b1;
    float mixed[R];
#pragma unroll
    for (int r = 0; r < R; ++r) mixed[r] = 0.0f;
#pragma unroll 8
    for (uint32_t g = 0; g < H; ++g) {   // (16 or 32 heads)
      const float s = s_s[g * kKeysPitch + lane];
#pragma unroll
      for (int r = 0; r < R; ++r) mixed[r] = fmaf(t_s[g * H + c * R + r], s, mixed[r]);
    }
    float keep[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const float v = seen ? mixed[r] : -INFINITY;
      const float top = fmaxf(m[r], wave_max(v));   // finite: every block of the range has a visible key
      keep[r] = attn_exp2(m[r] - top);
      const float w = attn_exp2(v - top);
      m[r] = top;
      l[r] = l[r] * keep[r] + w;
      uint16_t hi, lo16;
      split16<DT>(w, hi, lo16);
      w_s[(c * R + r) * 64u + lane] = hi;
      w_s[(H + c * R + r) * 64u + lane] = lo16;
    }
    __syncthreads();   // the scores are done with; the weights are in LDS
    float scale = 1.0f;
#pragma unroll
    for (int r = 0; r < R; ++r) scale = (n & 7u) == static_cast<uint32_t>(r) ? keep[r] : scale;
#pragma unroll
    for (int s = 0; s < 8; ++s) acc[s] *= scale;
    const bool column = (n & 7u) < static_cast<uint32_t>(R);
    const uint16_t *w_at = w_s + ((n < 8u ? 0u : H) + c * R + (column ? n & 7u : 0u)) * 64u + q4 * 4u;
#pragma unroll
    for (uint32_t t = 0; t < 4; ++t) {
      uint2 w = *reinterpret_cast<const uint2 *>(w_at + t * 16u);
      if (!column) w = make_uint2(0u, 0u);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        acc[2 * j] = mfma_k16<DT>(make_uint2(vreg[t][j].x, vreg[t][j].y), w, acc[2 * j]);
        acc[2 * j + 1] = mfma_k16<DT>(make_uint2(vreg[t][j].z, vreg[t][j].w), w, acc[2 * j + 1]);
      }
    }
  }
  const Partials out = partials_of(p.workspace, static_cast<uint64_t>(splits) * H);
#pragma unroll
  for (int s = 0; s < 8; ++s) {
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[s][i] += __shfl_xor(acc[s][i], 8, kWave);
    if (n < static_cast<uint32_t>(R))
      *reinterpret_cast<float4 *>(out.sum + (static_cast<uint64_t>(split) * H + c * R + n) * kHD + s * 16 + q4 * 4u) =
          make_float4(acc[s][0], acc[s][1], acc[s][2], acc[s][3]);
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const float total = wave_sum(l[r]);
    if (lane == 0) {
      out.m[split * H + c * R + r] = m[r];
      out.l[split * H + c * R + r] = total;
    }
  }
}

// ---- prompt blocks ---------------------------------------------------------------------------

// Rotated, scaled queries in 16 bits, [token][head][128], and - for a layer with a cache of its own - the token's keys and
// values into the cache.
__global__ __launch_bounds__(kBlock) void mixed_prepare_kernel(MixedAttnParams p, uint16_t *q16, uint32_t append) {
  constexpr uint32_t DT = kBF16;
  const uint32_t t = blockIdx.x, pos = p.position + t;
  const float *src = p.proj + static_cast<uint64_t>(t) * p.proj_stride;
  const float *cs = p.rope_cs + static_cast<uint64_t>(t) * p.rope_stride;
  const float scale = p.scale * kLog2e;
  const uint32_t A = p.heads * kHD, KV = p.kv_heads * kHD;
  for (uint32_t i = threadIdx.x; i < A; i += kBlock)
    q16[static_cast<uint64_t>(t) * A + i] = enc16<DT>(rotated_elem(src + p.q_col + i / kHD * kHD, cs, p.rot_dims, i % kHD) * scale);
  if (append == 0) return;
  const uint32_t block = p.table[pos / kKvBlockTokens], row = pos % kKvBlockTokens;
  for (uint32_t i = threadIdx.x; i < KV; i += kBlock) {
    const uint32_t h = i / kHD, d = i % kHD;
    const uint64_t tile = kv_tile_offset(0, p.kv_heads, kHD, 0, block, h);
    static_cast<uint16_t *>(p.k_cache)[tile + kv_k_elem(kHD, row, d)] = enc16<DT>(rotated_elem(src + p.k_col + h * kHD, cs, p.rot_dims, d));
    static_cast<uint16_t *>(p.v_cache)[tile + kv_v_elem(kHD, row, d)] = enc16<DT>(src[p.v_col + i]);
  }
}

// Scores in LDS: [key of 32][token of 8][head of 32], the pitches chosen so that a wave's accesses spread over the banks.
constexpr uint32_t kTokenPitch = kWideHeads + 4, kKeyPitch = kPromptTokens * kTokenPitch + 4;
constexpr size_t kPromptLds = 2u * 32u * kKeyPitch * sizeof(float);

template <int R>
__global__ __launch_bounds__(512, 2) void mixed_prompt_kernel(MixedAttnParams p, const uint16_t *q16, uint32_t splits) {
  constexpr uint32_t DT = kBF16;
  constexpr int CT = R / 2;   // column tiles of a wave: eight tokens x two heads each
  extern __shared__ __align__(16) float lds[];
  const uint32_t split = blockIdx.x % splits, tile = blockIdx.x / splits;
  const Range range = prompt_range(p, tile, splits);
  if (split >= range.active) return;
  const uint32_t u0 = split * range.per_split, u1 = min(u0 + range.per_split, range.count);
  const uint32_t H = p.heads, G = p.kv_heads;
  const uint32_t lane = threadIdx.x & (kWave - 1), c = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const uint32_t n = lane & 15u, q4 = lane >> 4, tok = n & 7u, half = n >> 3;
  const uint16_t *kc = static_cast<const uint16_t *>(p.k_cache), *vc = static_cast<const uint16_t *>(p.v_cache);
  const uint32_t my_tok = min(tile * kPromptTokens + tok, p.tokens - 1);
  const uint32_t pos = p.position + my_tok, lo = first_seen(p, pos);
  const uint32_t last_block = (p.position + min((tile + 1) * kPromptTokens, p.tokens) - 1) / kKvBlockTokens;

  uint4 q[CT][4], talk[kWideHeads / 16];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct)
#pragma unroll
    for (int j = 0; j < 4; ++j)
      q[ct][j] = *reinterpret_cast<const uint4 *>(q16 + (static_cast<uint64_t>(my_tok) * H + c * R + 2 * ct + half) * kHD + j * 32 + q4 * 8);
#pragma unroll
  for (uint32_t ht = 0; ht < kWideHeads / 16; ++ht) {   // rows of M this lane feeds: head 16 ht + n, its eight heads 8 q4 ..
    const uint32_t h = ht * 16u + n;
    uint32_t w[4] = {0u, 0u, 0u, 0u};
    if (h < H && q4 * 8u < H) {
#pragma unroll
      for (uint32_t e = 0; e < 4; ++e) {
        const uint32_t g = q4 * 8u + 2u * e;
        if (p.talk != nullptr)
          w[e] = p.talk[h * H + g] | (static_cast<uint32_t>(p.talk[h * H + g + 1]) << 16);
        else
          w[e] = (g == h ? 0x3f80u : 0u) | (g + 1 == h ? 0x3f800000u : 0u);
      }
    }
    talk[ht] = make_uint4(w[0], w[1], w[2], w[3]);
  }

  float m[CT], l[CT];
  f32x4_t acc[CT][8];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct) {
    m[ct] = -INFINITY;
    l[ct] = 0.0f;
#pragma unroll
    for (int s = 0; s < 8; ++s) acc[ct][s] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  }
  const auto tile_at = [&](uint32_t block) {
    return kv_tile_offset(0, G, kHD, 0, p.table[min(block, last_block)], c) + lane * 8u;
  };
  uint4 kreg[2][4];
#pragma unroll
  for (uint32_t t = 0; t < 2; ++t) {
    const uint64_t at = tile_at(range.first + 2 * u0 + t);
#pragma unroll
    for (int j = 0; j < 4; ++j) kreg[t][j] = *reinterpret_cast<const uint4 *>(kc + at + j * 512);
  }
  for (uint32_t u = u0; u < u1; ++u) {
    const uint32_t b = range.first + 2 * u;
    float *s_s = lds + (u & 1u) * 32u * kKeyPitch;
    uint4 vreg[2][4];
#pragma unroll
    for (uint32_t t = 0; t < 2; ++t) {
      const uint64_t at = tile_at(b + t);
#pragma unroll
      for (int j = 0; j < 4; ++j) vreg[t][j] = *reinterpret_cast<const uint4 *>(vc + at + j * 512);
    }
#pragma unroll
    for (uint32_t t = 0; t < 2; ++t)
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        f32x4_t s = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int j = 0; j < 4; ++j) s = mfma_k32<DT>(kreg[t][j], q[ct][j], s);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          s_s[(t * 16u + q4 * 4u + i) * kKeyPitch + tok * kTokenPitch + c * R + 2 * ct + half] = s[i];
      }
#pragma unroll
    for (uint32_t t = 0; t < 2; ++t) {   // the next unit's keys (the last unit asks for its own again)
      const uint64_t at = tile_at(range.first + 2 * min(u + 1, u1 - 1) + t);
#pragma unroll
      for (int j = 0; j < 4; ++j) kreg[t][j] = *reinterpret_cast<const uint4 *>(kc + at + j * 512);
    }
    __syncthreads();
    // mixing: sixteen columns = two keys x eight tokens at a time, all heads of a column in one wave
    for (uint32_t set = c; set < 16u; set += G) {
      float *col = s_s + (set * 2u + half) * kKeyPitch + tok * kTokenPitch;
      float f[8];
      {
        const float4 a = *reinterpret_cast<const float4 *>(col + q4 * 8u), d = *reinterpret_cast<const float4 *>(col + q4 * 8u + 4u);
        const float t[8] = {a.x, a.y, a.z, a.w, d.x, d.y, d.z, d.w};
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = q4 * 8u < H ? t[e] : 0.0f;   // (columns past the heads hold nothing)
      }
      uint4 piece[3];
#pragma unroll
      for (int k = 0; k < 3; ++k) {
        uint32_t w[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          w[e] = pack16(f[2 * e], f[2 * e + 1]);
          f[2 * e] -= __uint_as_float(w[e] << 16);
          f[2 * e + 1] -= __uint_as_float(w[e] & 0xffff0000u);
        }
        piece[k] = make_uint4(w[0], w[1], w[2], w[3]);
      }
#pragma unroll
      for (uint32_t ht = 0; ht < kWideHeads / 16; ++ht) {
        f32x4_t d = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int k = 2; k >= 0; --k) d = mfma_k32<DT>(talk[ht], piece[k], d);
        *reinterpret_cast<float4 *>(col + ht * 16u + q4 * 4u) = make_float4(d[0], d[1], d[2], d[3]);
      }
    }
    __syncthreads();
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
      float s[2][4];
      float top = -INFINITY;
#pragma unroll
      for (uint32_t t = 0; t < 2; ++t)
#pragma unroll
        for (uint32_t i = 0; i < 4; ++i) {
          const uint32_t key = (b + t) * kKvBlockTokens + q4 * 4u + i;
          const float v = s_s[(t * 16u + q4 * 4u + i) * kKeyPitch + tok * kTokenPitch + c * R + 2 * ct + half];
          s[t][i] = key >= lo && key <= pos ? v : -INFINITY;
          top = fmaxf(top, s[t][i]);
        }
      top = fmaxf(top, __shfl_xor(top, 16, kWave));
      top = fmaxf(top, __shfl_xor(top, 32, kWave));
      top = fmaxf(top, m[ct]);
      const bool any = top > -INFINITY;   // a token may see none of this split's keys so far
      const float keep = any ? attn_exp2(m[ct] - top) : 1.0f;
      m[ct] = top;
      float sum = 0.0f;
      uint32_t hi[4], low[4];
#pragma unroll
      for (uint32_t t = 0; t < 2; ++t)
#pragma unroll
        for (uint32_t e = 0; e < 2; ++e) {
          const float w0 = any ? attn_exp2(s[t][2 * e] - top) : 0.0f, w1 = any ? attn_exp2(s[t][2 * e + 1] - top) : 0.0f;
          sum += w0 + w1;
          hi[2 * t + e] = pack16(w0, w1);
          low[2 * t + e] = pack16(w0 - __uint_as_float(hi[2 * t + e] << 16), w1 - __uint_as_float(hi[2 * t + e] & 0xffff0000u));
        }
      l[ct] = l[ct] * keep + sum;
      const uint4 whi = make_uint4(hi[0], hi[1], hi[2], hi[3]), wlo = make_uint4(low[0], low[1], low[2], low[3]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const uint4 a0 = make_uint4(vreg[0][j].x, vreg[0][j].y, vreg[1][j].x, vreg[1][j].y);
        const uint4 a1 = make_uint4(vreg[0][j].z, vreg[0][j].w, vreg[1][j].z, vreg[1][j].w);
        acc[ct][2 * j] *= keep;
        acc[ct][2 * j + 1] *= keep;
        acc[ct][2 * j] = mfma_k32<DT>(a0, whi, acc[ct][2 * j]);
        acc[ct][2 * j + 1] = mfma_k32<DT>(a1, whi, acc[ct][2 * j + 1]);
        acc[ct][2 * j] = mfma_k32<DT>(a0, wlo, acc[ct][2 * j]);
        acc[ct][2 * j + 1] = mfma_k32<DT>(a1, wlo, acc[ct][2 * j + 1]);
      }
    }
  }
  const Partials out = partials_of(p.workspace, static_cast<uint64_t>(p.tokens) * splits * H);
  if (tile * kPromptTokens + tok >= p.tokens) return;
#pragma unroll
  for (int ct = 0; ct < CT; ++ct) {
    const uint64_t at = (static_cast<uint64_t>(my_tok) * splits + split) * H + c * R + 2 * ct + half;
#pragma unroll
    for (int s = 0; s < 8; ++s)
      *reinterpret_cast<float4 *>(out.sum + at * kHD + s * 16 + q4 * 4u) = make_float4(acc[ct][s][0], acc[ct][s][1], acc[ct][s][2], acc[ct][s][3]);
    float total = l[ct];
    total += __shfl_xor(total, 16, kWave);
    total += __shfl_xor(total, 32, kWave);
    if (q4 == 0) {
      out.m[at] = m[ct];
      out.l[at] = total;
    }
  }
}

// ---- merge -----------------------------------------------------------------------------------

__device__ __forceinline__ void merged_store(const MixedAttnParams &p, uint32_t t, uint32_t e, float4 o) {
  if (p.gate_col != kNoColumn) {
    const float4 g = *reinterpret_cast<const float4 *>(p.proj + static_cast<uint64_t>(t) * p.proj_stride + p.gate_col + e);
    o.x *= sigmoid(g.x);
    o.y *= sigmoid(g.y);
    o.z *= sigmoid(g.z);
    o.w *= sigmoid(g.w);
  }
  uint16_t *out = p.out16 + (p.packed_tiles != 0 ? gemm_x_packed_index(p.packed_tiles, t, e) : static_cast<uint64_t>(t) * p.heads * kHD + e);
  *reinterpret_cast<uint2 *>(out) = make_uint2(pack16(o.x, o.y), pack16(o.z, o.w));   // (four columns stay together in operand order)
}

// Decode step: one workgroup per head; sixteen groups of 32 lanes share the splits, four columns a lane.
constexpr uint32_t kMergeGroups = 16;
__global__ __launch_bounds__(kMergeGroups * 32) void mixed_decode_merge_kernel(MixedAttnParams p, uint32_t splits) {
  __shared__ float f_s[kDecodeSplits], red[kMergeGroups * 32 / kWave];
  __shared__ float4 sum_s[kMergeGroups][32];
  const uint32_t h = blockIdx.x, H = p.heads, tid = threadIdx.x, group = tid / 32u, c4 = tid % 32u;
  const uint32_t pos = p.cursor != nullptr ? *p.cursor : p.position;
  if (p.cursor != nullptr && pos >= p.max_steps) return;
  const uint32_t active = decode_range(p, pos, splits).active;
  const Partials in = partials_of(p.workspace, static_cast<uint64_t>(splits) * H);
  const float sink = p.sink != nullptr ? dec16<kBF16>(p.sink[h]) * kLog2e : -INFINITY;
  // every request first: the lane's share of the sums, and one split's maximum and denominator (kDecodeSplits lanes
  // are enough)
  float4 v[kDecodeSplits / kMergeGroups];
#pragma unroll
  for (uint32_t i = 0; i < kDecodeSplits / kMergeGroups; ++i)
    v[i] = *reinterpret_cast<const float4 *>(in.sum + (static_cast<uint64_t>(min(group + i * kMergeGroups, active - 1)) * H + h) * kHD + c4 * 4u);
  const float ms = tid < active ? in.m[tid * H + h] : -INFINITY, ls = tid < active ? in.l[tid * H + h] : 0.0f;
  float top = wave_max(ms);
  if (tid % kWave == 0) red[tid / kWave] = top;
  __syncthreads();
  top = sink;
#pragma unroll
  for (uint32_t w = 0; w < kMergeGroups * 32 / kWave; ++w) top = fmaxf(top, red[w]);
  const float f = tid < active ? attn_exp2(ms - top) : 0.0f;
  if (tid < kDecodeSplits) f_s[tid] = f;
  const float part = wave_sum(ls * f);
  __syncthreads();
  if (tid % kWave == 0) red[tid / kWave] = part;
  __syncthreads();
  float total = p.sink != nullptr ? attn_exp2(sink - top) : 0.0f;
#pragma unroll
  for (uint32_t w = 0; w < kMergeGroups * 32 / kWave; ++w) total += red[w];
  float4 o = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
#pragma unroll
  for (uint32_t i = 0; i < kDecodeSplits / kMergeGroups; ++i) {
    const float w = f_s[group + i * kMergeGroups];   // zero past the active splits
    o.x = fmaf(v[i].x, w, o.x);
    o.y = fmaf(v[i].y, w, o.y);
    o.z = fmaf(v[i].z, w, o.z);
    o.w = fmaf(v[i].w, w, o.w);
  }
  sum_s[group][c4] = o;
  __syncthreads();
  if (group != 0) return;
#pragma unroll
  for (uint32_t i = 1; i < kMergeGroups; ++i) {
    const float4 a = sum_s[i][c4];
    o.x += a.x;
    o.y += a.y;
    o.z += a.z;
    o.w += a.w;
  }
  const float inv = 1.0f / total;
  merged_store(p, 0, h * kHD + c4 * 4u, make_float4(o.x * inv, o.y * inv, o.z * inv, o.w * inv));
}

// Prompt blocks: 32 lanes per (token, head), four columns a lane, the splits in order.
__global__ __launch_bounds__(kBlock) void mixed_prompt_merge_kernel(MixedAttnParams p, uint32_t splits) {
  const uint32_t H = p.heads, id = blockIdx.x * (kBlock / 32u) + threadIdx.x / 32u, c4 = threadIdx.x % 32u;
  const uint32_t t = id / H, h = id % H;
  if (t >= p.tokens) return;
  const uint32_t active = prompt_range(p, t / kPromptTokens, splits).active;
  const Partials in = partials_of(p.workspace, static_cast<uint64_t>(p.tokens) * splits * H);
  const uint64_t base = static_cast<uint64_t>(t) * splits * H + h;
  float top = p.sink != nullptr ? dec16<kBF16>(p.sink[h]) * kLog2e : -INFINITY;
  float total = p.sink != nullptr ? 1.0f : 0.0f;
  float4 o = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
#pragma unroll 4
  for (uint32_t s = 0; s < active; ++s) {
    const uint64_t at = base + static_cast<uint64_t>(s) * H;
    const float ms = in.m[at], ls = in.l[at];
    const float4 v = *reinterpret_cast<const float4 *>(in.sum + at * kHD + c4 * 4u);
    const float next = fmaxf(top, ms);
    const float keep = top > -INFINITY ? attn_exp2(top - next) : 0.0f;
    const float f = ms > -INFINITY ? attn_exp2(ms - next) : 0.0f;   // (a token may have seen no key of a split)
    top = next;
    total = total * keep + ls * f;
    o.x = o.x * keep + v.x * f;
    o.y = o.y * keep + v.y * f;
    o.z = o.z * keep + v.z * f;
    o.w = o.w * keep + v.w * f;
  }
  const float inv = 1.0f / total;
  merged_store(p, t, h * kHD + c4 * 4u, make_float4(o.x * inv, o.y * inv, o.z * inv, o.w * inv));
}

uint32_t decode_splits(const MixedAttnParams &p) {
  const uint32_t visible = p.chunk != 0 ? std::min(p.chunk / kKvBlockTokens + 2, p.last_block + 1) : p.last_block + 1;
  return std::max(1u, std::min(kDecodeSplits, (visible + kMinBlocksPerSplit - 1) / kMinBlocksPerSplit));
}
uint32_t prompt_tiles(uint32_t tokens) { return (tokens + kPromptTokens - 1) / kPromptTokens; }
uint32_t prompt_splits(uint32_t tokens) {
  return std::max(1u, std::min(kPromptSplits, kPromptWorkgroups / prompt_tiles(tokens)));
}
uint64_t partial_bytes(uint64_t entries) { return entries * (kHD + 2) * sizeof(float); }

template <int R>
hipError_t launch_decode(const MixedAttnParams &p, uint32_t append, hipStream_t stream) {
  const uint32_t splits = decode_splits(p);
  const size_t lds = (p.heads * static_cast<uint32_t>(kHD) + p.heads * p.heads) * sizeof(float) + 2u * p.heads * 64u * sizeof(uint16_t);
  hipLaunchKernelGGL(mixed_decode_kernel<R>, dim3(splits), dim3(p.kv_heads * kWave), lds, stream, p, splits, append);
  hipError_t err = hipGetLastError();
  if (err != hipSuccess) return err;
  hipLaunchKernelGGL(mixed_decode_merge_kernel, dim3(p.heads), dim3(kMergeGroups * 32), 0, stream, p, splits);
  return hipGetLastError();
}

template <int R>
hipError_t launch_prompt(const MixedAttnParams &p, uint32_t append, hipStream_t stream) {
  static std::once_flag once;   // (prompt blocks never run under stream capture)
  static hipError_t raised = hipSuccess;
  std::call_once(once, [] {
    raised = hipFuncSetAttribute(reinterpret_cast<const void *>(&mixed_prompt_kernel<R>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                 static_cast<int>(kPromptLds));
  });
  if (raised != hipSuccess) return raised;
  const uint32_t tiles = prompt_tiles(p.tokens), splits = prompt_splits(p.tokens);
  uint16_t *q16 = reinterpret_cast<uint16_t *>(static_cast<char *>(p.workspace) +
                                               partial_bytes(static_cast<uint64_t>(p.tokens) * splits * p.heads));
  hipLaunchKernelGGL(mixed_prepare_kernel, dim3(p.tokens), dim3(kBlock), 0, stream, p, q16, append);
  hipError_t err = hipGetLastError();
  if (err != hipSuccess) return err;
  hipLaunchKernelGGL(mixed_prompt_kernel<R>, dim3(tiles * splits), dim3(p.kv_heads * kWave), kPromptLds, stream, p,
                     static_cast<const uint16_t *>(q16), splits);
  err = hipGetLastError();
  if (err != hipSuccess) return err;
  constexpr uint32_t kRowsPerBlock = kBlock / 32u;
  hipLaunchKernelGGL(mixed_prompt_merge_kernel, dim3((p.tokens * p.heads + kRowsPerBlock - 1) / kRowsPerBlock), dim3(kBlock), 0, stream, p,
                     splits);
  return hipGetLastError();
}

}  // namespace

bool mixed_attention_wide(uint32_t heads, uint32_t kv_heads, uint32_t key_dim, uint32_t value_dim) {
  const uint32_t group = kv_heads != 0 ? heads / kv_heads : 0;
  return key_dim == static_cast<uint32_t>(kHD) && value_dim == static_cast<uint32_t>(kHD) && heads == group * kv_heads && kv_heads <= 8 &&
         (group == 2 || group == 4 || group == 8) && (heads == 16 || heads == 32);
}

uint64_t mixed_attention_workspace_bytes(uint32_t heads, uint32_t max_tokens) {
  uint64_t most = partial_bytes(static_cast<uint64_t>(kDecodeSplits) * heads);
  // (tokens a workgroup x splits is largest where the tiles do not divide the workgroups evenly; both factors bounded)
  const uint64_t entries = static_cast<uint64_t>(std::max(kPromptWorkgroups, prompt_tiles(max_tokens))) * kPromptTokens * heads;
  most = std::max(most, partial_bytes(entries) + static_cast<uint64_t>(max_tokens) * heads * kHD * sizeof(uint16_t));
  return most;
}

hipError_t launch_mixed_attention_wide(uint32_t dtype, const MixedAttnParams &p, bool append, hipStream_t stream) {
  if (dtype != kBF16 || !mixed_attention_wide(p.heads, p.kv_heads, p.key_dim, p.value_dim) || p.cache32 != 0 || p.out16 == nullptr ||
      p.workspace == nullptr || p.proj == nullptr || p.k_cache == nullptr || p.v_cache == nullptr || p.table == nullptr || p.tokens == 0 ||
      p.rot_dims % 2 != 0 || p.rot_dims > p.key_dim || (p.rot_dims != 0 && p.rope_cs == nullptr) ||
      (p.packed_tiles != 0 && p.packed_tiles * 16u < p.tokens))
    return hipErrorInvalidValue;
  const bool one = p.cursor != nullptr;
  if (one && p.tokens != 1) return hipErrorInvalidValue;
  if (!one && (p.position + p.tokens - 1) / kKvBlockTokens > p.last_block) return hipErrorInvalidValue;
  switch (p.heads / p.kv_heads) {
    case 2: return one ? launch_decode<2>(p, append, stream) : launch_prompt<2>(p, append, stream);
    case 4: return one ? launch_decode<4>(p, append, stream) : launch_prompt<4>(p, append, stream);
    default: return one ? launch_decode<8>(p, append, stream) : launch_prompt<8>(p, append, stream);
  }
}

}  // namespace nv
