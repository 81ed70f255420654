// Attention over latents (attn_latent.cuh) for wide layers, 16-bit cache, on the matrix cores. All heads of a token meet
// the same cache rows, so the rows of the products are (token, head) pairs, `heads` a token.
//
//   absorb  q' = [W_uk^T q_unrotated, rotate(q_rotated)] * scale * log2(e), 16-bit, kv_rank + rot_dim elements a row. W_uk is
//           read as it lies (rows = contraction) and turned by the transposing LDS reads. A decode step's launch also
//           writes the token's cache row.
//   rows    scores, softmax and weighted latents: two waves share 32 rows and walk the keys 32 at a time. Each takes
//           half the elements of the rows' score products, their q' in registers for the whole launch - so that a key
//           operand read once serves both row tiles - the softmax of 16 rows, and half the latent columns of the 32
//           rows' sums; partial scores and weights cross through LDS. The waves of a workgroup share the keys: two
//           cache blocks go from the cache to LDS as they lie (matrix-operand order, global_load_lds, 1 KiB a request),
//           the next two while these are worked on. The scores read them as operands; for the sums the same bytes are
//           read transposed (ds_read_b64_tr_b16), keys along the contraction - so a cache row is fetched once for both.
//           Scores come out with a lane's keys in the order the second product wants its weights in; weights enter as
//           hi + lo 16-bit halves. A running maximum is moved only when a score passes it by more than 8 (log2), so the
//           sums are rarely rescaled.
//   merge   splits of the key range into one row, where there are any (decode steps: where there are many)
//   value   o = sigmoid(gate) * W_uv (weighted latents); a decode step's launch merges few splits itself.
#include <algorithm>
#include <mutex>

#include "activations.cuh"
#include "attn_latent.cuh"
#include "attn_mixed.cuh"
#include "attn_tile.cuh"
#include "gemm_rows.cuh"

namespace nv {

namespace {

using namespace attn;

constexpr uint32_t kUnitKeys = 2 * kKvBlockTokens;   // keys a step of the rows kernel takes
constexpr uint32_t kPairRows = 32;
// [row tile][2 KiB]: the partial scores of the wave that has the row tile ([key tile][lane]), and - once it has read them -
// the tile's weights as the second product wants them ([hi, lo][lane])
constexpr size_t kPairExchange = 4096;
constexpr uint32_t kMostSplits = 256, kBlockSplits = 8, kWorkgroups = 512;   // (two a CU)
constexpr float kLazy = 8.0f;

struct Work {
  uint16_t *q16, *o16;   // [rows][kv_rank + rot_dim], [rows][kv_rank]
  float *sum, *m, *l;    // [rows][splits][kv_rank], [rows][splits]
};
__host__ __device__ __forceinline__ Work work_at(void *base, uint64_t rows, uint32_t rank, uint32_t width, uint32_t splits) {
  Work w;
  w.q16 = static_cast<uint16_t *>(base);
  w.o16 = w.q16 + (rows * width + 127u) / 128u * 128u;
  w.sum = reinterpret_cast<float *>(w.o16 + (rows * rank + 127u) / 128u * 128u);
  w.m = w.sum + rows * splits * rank;
  w.l = w.m + rows * splits;
  return w;
}

__device__ __forceinline__ uint32_t pack16(float a, float b) {
  typedef float f32x2_t __attribute__((ext_vector_type(2)));
  typedef __bf16 bf16x2_t __attribute__((ext_vector_type(2)));
  return __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2_t{a, b}), bf16x2_t));   // v_cvt_pk_bf16_f32
}
__device__ __forceinline__ uint32_t lds_address(const void *p) {
  return static_cast<uint32_t>(reinterpret_cast<uintptr_t>((__attribute__((address_space(3))) const void *)(p)));
}
typedef uint32_t u32x2_t __attribute__((ext_vector_type(2)));

// ---- absorb ----------------------------------------------------------------------------------

// A workgroup: one head, RT x 16 latent columns, 64 tokens (16 a wave); the column group past the last one prepares the
// rotated elements (and a decode step's cache row, head 0).
template <int RT>
__global__ __launch_bounds__(kBlock) void latent_absorb_kernel(LatentAttnParams p, uint16_t *q16) {
  constexpr uint32_t DT = kBF16, kCols = RT * 16;
  __shared__ __align__(16) uint16_t w_s[32 * kCols];
  __shared__ float red[kWavesPerBlock];
  const uint32_t pos0 = p.cursor != nullptr ? *p.cursor : p.position;
  if (p.cursor != nullptr && pos0 >= p.max_steps) return;
  const uint32_t R = p.kv_rank, width = R + p.rot_dim, head = p.key_dim + p.rot_dim, h = blockIdx.y;
  const uint32_t t0 = blockIdx.z * 64u, c0 = blockIdx.x * kCols;
  const float gain = p.scale * kLog2e;
  if (c0 >= R) {
    const uint32_t count = min(64u, p.tokens - t0);
    for (uint32_t i = threadIdx.x; i < count * p.rot_dim; i += kBlock) {
      const uint32_t t = t0 + i / p.rot_dim, d = i % p.rot_dim;
      const float *q = p.q + (static_cast<uint64_t>(t) * p.heads + h) * head + p.key_dim;
      q16[(static_cast<uint64_t>(t) * p.heads + h) * width + R + d] =
          enc16<DT>(rotated_elem(q, p.rope_cs + static_cast<uint64_t>(t) * p.rope_stride, p.rot_dims, d) * gain);
    }
    if (p.cursor == nullptr || h != 0) return;
    const float *src = p.proj + p.kv_col;
    float ss = 0.0f;
    for (uint32_t i = threadIdx.x; i < R; i += kBlock) ss = fmaf(src[i], src[i], ss);
    const float root = 1.0f / sqrtf(block_sum(ss, red) / static_cast<float>(R) + p.eps);
    uint16_t *block = static_cast<uint16_t *>(p.cache) + static_cast<uint64_t>(p.table[pos0 / kKvBlockTokens]) * kKvBlockTokens * width;
    for (uint32_t i = threadIdx.x; i < width; i += kBlock)
      block[latent_elem(width, pos0 % kKvBlockTokens, i)] =
          enc16<DT>(i < R ? src[i] * root * dec16<DT>(p.kv_norm[i]) : rotated_elem(src + R, p.rope_cs, p.rot_dims, i - R));
    return;
  }
  const uint32_t lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave, n = lane & 15u, q4 = lane >> 4;
  const uint32_t t = t0 + wave * 16u + n, tc = min(t, p.tokens - 1);
  const float *q = p.q + (static_cast<uint64_t>(tc) * p.heads + h) * head;
  const uint16_t *w = p.w_uk + static_cast<uint64_t>(h) * p.key_dim * R + c0;
  // transposed reads: lane i of a 16-lane group fetches columns 4 (i % 4) .. of contraction row 4 q4 + i / 4 and gets
  // column i of the group's four rows
  const uint32_t at = lds_address(w_s) + ((4u * q4 + n / 4u) * kCols + (n % 4u) * 4u) * 2u;
  f32x4_t acc[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) acc[i] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  for (uint32_t d0 = 0; d0 < p.key_dim; d0 += 32) {
    __syncthreads();
#pragma unroll
    for (uint32_t i = threadIdx.x * 8u; i < 32u * kCols; i += kBlock * 8u)
      *reinterpret_cast<uint4 *>(w_s + i) = *reinterpret_cast<const uint4 *>(w + static_cast<uint64_t>(d0 + i / kCols) * R + i % kCols);
    const float4 a = *reinterpret_cast<const float4 *>(q + d0 + 4u * q4), b = *reinterpret_cast<const float4 *>(q + d0 + 16u + 4u * q4);
    const uint4 x = make_uint4(pack16(a.x, a.y), pack16(a.z, a.w), pack16(b.x, b.y), pack16(b.z, b.w));
    __syncthreads();
#pragma unroll
    for (int i = 0; i < RT; i += 2) {
      u32x2_t lo[2], hi[2];
      asm volatile("ds_read_b64_tr_b16 %0, %4 offset:%5\n\tds_read_b64_tr_b16 %1, %4 offset:%6\n\t"
                   "ds_read_b64_tr_b16 %2, %4 offset:%7\n\tds_read_b64_tr_b16 %3, %4 offset:%8\n\ts_waitcnt lgkmcnt(0)"
                   : "=&v"(lo[0]), "=&v"(hi[0]), "=&v"(lo[1]), "=&v"(hi[1])
                   : "v"(at), "n"(i * 32), "n"(i * 32 + 16 * kCols * 2), "n"((i + 1) * 32), "n"((i + 1) * 32 + 16 * kCols * 2)
                   : "memory");
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i + j] = mfma_k32<DT>(make_uint4(lo[j].x, lo[j].y, hi[j].x, hi[j].y), x, acc[i + j]);
    }
  }
  if (t >= p.tokens) return;
  uint16_t *out = q16 + (static_cast<uint64_t>(t) * p.heads + h) * width + c0 + 4u * q4;
#pragma unroll
  for (int i = 0; i < RT; ++i)
    *reinterpret_cast<uint2 *>(out + i * 16) =
        make_uint2(pack16(acc[i][0] * gain, acc[i][1] * gain), pack16(acc[i][2] * gain, acc[i][3] * gain));
}

// ---- rows ------------------------------------------------------------------------------------

struct Units {
  uint32_t block0, count, per;   // first block, units of two blocks in all, units of a split
};
__device__ __forceinline__ Units units_of(const LatentAttnParams &p, uint32_t pos0, uint32_t first_token, uint32_t last_token, uint32_t splits) {
  const uint32_t b0 = window_start(pos0 + first_token, p.window) / kKvBlockTokens, b1 = (pos0 + last_token) / kKvBlockTokens;
  const uint32_t count = (b1 - b0) / 2u + 1u;
  return Units{b0, count, (count + splits - 1) / splits};
}

// PAIRS: pairs of waves of a workgroup, 32 rows each.
template <int R, int RD, int PAIRS>
constexpr size_t latent_rows_lds() {
  return 2u * kUnitKeys * (R + RD) * sizeof(uint16_t) + PAIRS * kPairExchange;
}

template <int R, int RD, int PAIRS>
__global__ __launch_bounds__(2 * PAIRS * kWave, 2) void latent_rows_kernel(LatentAttnParams p, uint32_t splits) {
  constexpr uint32_t DT = kBF16;
  constexpr int D = R + RD, KS = D / 32, DTL = R / 32;        // K-steps of the scores, tiles of 16 latent columns a wave
  constexpr int kTileBytes = 16 * D * 2, kBuf = 2 * kTileBytes, kPieces = kBuf / 1024, kWaves = 2 * PAIRS;
  constexpr int KH = KS / 2;                                  // ... of a wave
  static_assert(KS % 2 == 0 && KH > 2 && DTL % 2 == 0 && D % 32 == 0, "whole groups");
  extern __shared__ __align__(16) unsigned char smem[];
  const uint32_t rows = p.tokens * p.heads;
  const uint32_t split = blockIdx.x % splits, row0 = blockIdx.x / splits * (PAIRS * kPairRows);
  const uint32_t lane = threadIdx.x & (kWave - 1), wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const uint32_t pair = wave / 2u, part = wave % 2u;          // part: the wave's elements in the score products, row tile in the softmax, columns in the sums
  const uint32_t n = lane & 15u, q4 = lane >> 4;
  const Work ws = work_at(p.workspace, rows, R, D, splits);
  uint4 q[2][KH];   // of both row tiles; requested ahead of everything that depends on the position
#pragma unroll
  for (int r = 0; r < 2; ++r) {
    const uint16_t *src = ws.q16 + static_cast<uint64_t>(min(row0 + pair * kPairRows + r * 16u + n, rows - 1)) * D + part * (KH * 32u) + q4 * 8u;
#pragma unroll
    for (int j = 0; j < KH; ++j) q[r][j] = *reinterpret_cast<const uint4 *>(src + j * 32);
  }
  const uint32_t pos0 = p.cursor != nullptr ? *p.cursor : p.position;
  if (p.cursor != nullptr && pos0 >= p.max_steps) return;
  const uint32_t first_token = row0 / p.heads, last_token = (min(row0 + PAIRS * kPairRows, rows) - 1) / p.heads;
  const Units units = units_of(p, pos0, first_token, last_token, splits);
  const uint32_t u0 = split * units.per, u1 = min(u0 + units.per, units.count);
  const uint32_t row = row0 + pair * kPairRows + part * 16u + n, pos = pos0 + min(row, rows - 1) / p.heads, lo = window_start(pos, p.window);
  if (u0 >= u1) {   // a split without keys
    if (q4 == 0 && row < rows) {
      ws.m[static_cast<uint64_t>(row) * splits + split] = -INFINITY;
      ws.l[static_cast<uint64_t>(row) * splits + split] = 0.0f;
    }
    return;
  }
  const uint32_t last_block = (pos0 + last_token) / kKvBlockTokens;
  const char *cache = static_cast<const char *>(p.cache) + lane * 16u;
  // unit U -> buffer B: 1 KiB pieces, the workgroup's waves in turn
  const auto request = [&](uint32_t u, uint32_t b) {
    const uint32_t block = units.block0 + 2u * u;
    const char *src[2];
#pragma unroll
    for (uint32_t t = 0; t < 2; ++t) src[t] = cache + static_cast<uint64_t>(p.table[min(block + t, last_block)]) * kTileBytes;
#pragma unroll
    for (int i = 0; i < (kPieces + kWaves - 1) / kWaves; ++i) {
      const int piece = i * kWaves + wave;
      if (kPieces % kWaves != 0 && piece >= kPieces) break;
      const char *from = (piece >= KS ? src[1] - KS * 1024 : src[0]) + piece * 1024;
      __builtin_amdgcn_global_load_lds(reinterpret_cast<const uint32_t *>(from),
                                       (__attribute__((address_space(3))) void *)(smem + b * kBuf + piece * 1024), 16, 0, 0);
    }
  };
  request(u0, 0);
  float m = -INFINITY, l = 0.0f;
  f32x4_t acc[2][DTL];
#pragma unroll
  for (int r = 0; r < 2; ++r)
#pragma unroll
    for (int i = 0; i < DTL; ++i) acc[r][i] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  const uint32_t lds0 = lds_address(smem);
  const uint32_t first_pos = pos0 + first_token, last_lo = window_start(pos0 + last_token, p.window);

  // LDS is read and written by hand, operands a group ahead of the products that use them (the compiler would wait for the
  // requests in flight to LDS as well); the awaited registers are in/out operands of the wait.
#define NV_LR_K(DST, KT, J) asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(DST) : "v"(ka), "n"((KT) * kTileBytes + (J) * 1024) : "memory")
#define NV_LR_V(DST, KT, T) asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(DST) : "v"(va), "n"((KT) * kTileBytes + (T) * 512) : "memory")
  // (waits until at most min(LEFT_, MOST_) younger reads are outstanding)
#define NV_LR_AWAIT(LEFT_, MOST_, ...) asm volatile("s_waitcnt lgkmcnt(%c[n])" : __VA_ARGS__ : [n] "n"((LEFT_) < (MOST_) ? (LEFT_) : (MOST_)) : "memory")
  for (uint32_t u = u0; u < u1; ++u) {
    const uint32_t b = (u - u0) & 1u;
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");   // this unit is there, the last one is done with
    if (u + 1 < u1) request(u + 1, b ^ 1u);
    // addresses, made anew for every unit: kept in registers across the loop they would not fit
    uint32_t id = lane;
    asm volatile("" : "+v"(id));
    const uint32_t ka = lds0 + b * kBuf + part * (KH * 1024u) + id * 16u;
    f32x4_t part_s[2][2];   // [row tile][key tile]
#pragma unroll
    for (int r = 0; r < 2; ++r)
#pragma unroll
      for (int t = 0; t < 2; ++t) part_s[r][t] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
    {
      u32x4_t kq[5];   // K-step i / 2 of key tile i % 2, four reads ahead
      constexpr int kReads = 2 * KH;
#pragma unroll
      for (int i = 0; i < 4; ++i) NV_LR_K(kq[i], i & 1, i >> 1);
#pragma unroll
      for (int i = 0; i < kReads; ++i) {
        if (i + 4 < kReads) NV_LR_K(kq[(i + 4) % 5], i & 1, (i + 4) >> 1);
        NV_LR_AWAIT(kReads - 1 - i, 4, "+v"(kq[i % 5]));
#pragma unroll
        for (int r = 0; r < 2; ++r) part_s[r][i & 1] = mfma_k32<DT>(__builtin_bit_cast(uint4, kq[i % 5]), q[r][i >> 1], part_s[r][i & 1]);
      }
    }
    // the other wave's row tile goes to it, this one's missing half comes back
    f32x4_t s[2];
    {
      const f32x4_t give0 = part != 0 ? part_s[0][0] : part_s[1][0], give1 = part != 0 ? part_s[0][1] : part_s[1][1];
      // (the products' results are read behind the compiler's back: their latency is waited out here)
      const uint32_t s_at = lds0 + 2 * kBuf + pair * static_cast<uint32_t>(kPairExchange) + id * 16u;
      asm volatile("s_nop 15\n\ts_nop 15\n\tds_write_b128 %0, %1\n\tds_write_b128 %0, %2 offset:1024\n\ts_waitcnt lgkmcnt(0)\n\ts_barrier" ::
                   "v"(s_at + (part ^ 1u) * 2048u), "v"(give0), "v"(give1) : "memory");
      f32x4_t got0, got1;
      asm volatile("ds_read_b128 %0, %2\n\tds_read_b128 %1, %2 offset:1024\n\ts_waitcnt lgkmcnt(0)" : "=&v"(got0), "=&v"(got1) :
                   "v"(s_at + part * 2048u) : "memory");
      s[0] = (part != 0 ? part_s[1][0] : part_s[0][0]) + got0;
      s[1] = (part != 0 ? part_s[1][1] : part_s[0][1]) + got1;
    }
    const uint32_t key0 = (units.block0 + 2u * u) * kKvBlockTokens;
    if (key0 < last_lo || key0 + kUnitKeys - 1u > first_pos) {
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const uint32_t key = key0 + t * 16u + q4 * 4u + i;
          s[t][i] = key >= lo && key <= pos ? s[t][i] : -INFINITY;
        }
    }
    float top = fmaxf(fmaxf(fmaxf(s[0][0], s[0][1]), fmaxf(s[0][2], s[0][3])), fmaxf(fmaxf(s[1][0], s[1][1]), fmaxf(s[1][2], s[1][3])));
    float keep = 1.0f;
    if (__any(top > m + kLazy)) {
      top = fmaxf(top, __shfl_xor(top, 16, kWave));
      top = fmaxf(top, __shfl_xor(top, 32, kWave));
      top = fmaxf(top, m);
      keep = top > -INFINITY ? attn_exp2(m - top) : 1.0f;
      m = top;
      l *= keep;
    }
    // (the factors [row tile][lane] lie where this unit's rotated key elements were: everyone has multiplied them)
    asm volatile("" : "+v"(id));
    const uint32_t w_at = lds0 + 2 * kBuf + pair * static_cast<uint32_t>(kPairExchange) + id * 16u;
    const uint32_t f_at = lds0 + b * kBuf + R / 32 * 1024u + pair * 512u + id * 4u;
    const float ref = m > -INFINITY ? m : 0.0f;   // (a row may not have seen a key yet)
    {
      u32x4_t hi, low;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float w0 = attn_exp2(s[t][2 * e] - ref), w1 = attn_exp2(s[t][2 * e + 1] - ref);
          l += w0 + w1;
          const uint32_t h = pack16(w0, w1);
          hi[2 * t + e] = h;
          low[2 * t + e] = pack16(w0 - __uint_as_float(h << 16), w1 - __uint_as_float(h & 0xffff0000u));
        }
      asm volatile("ds_write_b128 %0, %1\n\tds_write_b128 %0, %2 offset:1024\n\tds_write_b32 %3, %4" ::
                   "v"(w_at + part * 2048u), "v"(hi), "v"(low), "v"(f_at + part * 256u), "v"(keep) : "memory");
    }
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    u32x4_t w[4];   // [row tile][hi, lo]
    asm volatile("" : "+v"(id));
    const uint32_t va = lds0 + b * kBuf + part * (DTL * 512u) + ((id % 4u / 2u) * 16u + id / 16u * 4u + id % 16u / 4u) * 16u + (id % 2u) * 8u;
    float factor[2];
    u32x2_t vq[4][2];   // a tile of columns, two key tiles; three tiles ahead
    asm volatile("ds_read_b32 %0, %2\n\tds_read_b32 %1, %2 offset:256" : "=&v"(factor[0]), "=&v"(factor[1]) : "v"(f_at) : "memory");
#pragma unroll
    for (int i = 0; i < 4; ++i) asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(w[i]) : "v"(w_at), "n"(i * 1024) : "memory");
#pragma unroll
    for (int i = 0; i < 6; ++i) NV_LR_V(vq[i >> 1][i & 1], i & 1, i >> 1);
    asm volatile("s_waitcnt lgkmcnt(6)" : "+v"(factor[0]), "+v"(factor[1]), "+v"(w[0]), "+v"(w[1]), "+v"(w[2]), "+v"(w[3]) :: "memory");
    if (__any(factor[0] != 1.0f || factor[1] != 1.0f)) {
#pragma unroll
      for (int r = 0; r < 2; ++r)
#pragma unroll
        for (int i = 0; i < DTL; ++i) acc[r][i] *= factor[r];
    }
#pragma unroll
    for (int c = 0; c < DTL; ++c) {
      if (c + 3 < DTL) {
#pragma unroll
        for (int t = 0; t < 2; ++t) NV_LR_V(vq[(c + 3) % 4][t], t, c + 3);
      }
      NV_LR_AWAIT(2 * (DTL - 1 - c), 6, "+v"(vq[c % 4][0]), "+v"(vq[c % 4][1]));
      const uint4 a = make_uint4(vq[c % 4][0].x, vq[c % 4][0].y, vq[c % 4][1].x, vq[c % 4][1].y);
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int r = 0; r < 2; ++r) acc[r][c] = mfma_k32<DT>(a, __builtin_bit_cast(uint4, w[2 * r + k]), acc[r][c]);
    }
  }
#undef NV_LR_K
#undef NV_LR_V
#undef NV_LR_AWAIT
  // the rows' denominators cross to the wave with their other columns
  float total = l;
  total += __shfl_xor(total, 16, kWave);
  total += __shfl_xor(total, 32, kWave);
  float *totals = reinterpret_cast<float *>(smem + 2 * kBuf + pair * kPairExchange);
  __syncthreads();
  if (q4 == 0) totals[part * 16u + n] = total;
  __syncthreads();
  if (q4 == 0 && row < rows && (splits != 1 || p.cursor != nullptr)) {
    ws.m[static_cast<uint64_t>(row) * splits + split] = m;
    ws.l[static_cast<uint64_t>(row) * splits + split] = total;
  }
#pragma unroll
  for (int r = 0; r < 2; ++r) {
    const uint32_t to = row0 + pair * kPairRows + r * 16u + n;
    if (to >= rows) continue;
    if (splits == 1 && p.cursor == nullptr) {
      const float inv = 1.0f / totals[r * 16u + n];
      uint16_t *out = ws.o16 + static_cast<uint64_t>(to) * R + part * (DTL * 16u) + 4u * q4;
#pragma unroll
      for (int i = 0; i < DTL; ++i)
        *reinterpret_cast<uint2 *>(out + i * 16) = make_uint2(pack16(acc[r][i][0] * inv, acc[r][i][1] * inv), pack16(acc[r][i][2] * inv, acc[r][i][3] * inv));
    } else {
      float *out = ws.sum + (static_cast<uint64_t>(to) * splits + split) * R + part * (DTL * 16u) + 4u * q4;
#pragma unroll
      for (int i = 0; i < DTL; ++i) *reinterpret_cast<float4 *>(out + i * 16) = make_float4(acc[r][i][0], acc[r][i][1], acc[r][i][2], acc[r][i][3]);
    }
  }
}

// ---- merge, value ----------------------------------------------------------------------------

// Blocks of token rows: one workgroup per row, four columns a lane.
__global__ __launch_bounds__(kBlock) void latent_merge_kernel(LatentAttnParams p, uint32_t splits) {
  const uint32_t rows = p.tokens * p.heads, R = p.kv_rank, row = blockIdx.x;
  const Work ws = work_at(p.workspace, rows, R, R + p.rot_dim, splits);
  const uint64_t base = static_cast<uint64_t>(row) * splits;
  float top = -INFINITY;
  for (uint32_t i = 0; i < splits; ++i) top = fmaxf(top, ws.m[base + i]);
  float total = 0.0f;
  for (uint32_t i = 0; i < splits; ++i) total += ws.l[base + i] * attn_exp2(ws.m[base + i] - top);
  const float inv = 1.0f / total;
  for (uint32_t c = threadIdx.x * 4u; c < R; c += kBlock * 4u) {
    float4 o = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    for (uint32_t i = 0; i < splits; ++i) {
      const float ms = ws.m[base + i];
      if (!(ms > -INFINITY)) continue;   // (such a split has left no sums)
      const float f = attn_exp2(ms - top) * inv;
      const float4 v = *reinterpret_cast<const float4 *>(ws.sum + (base + i) * R + c);
      o.x = fmaf(v.x, f, o.x);
      o.y = fmaf(v.y, f, o.y);
      o.z = fmaf(v.z, f, o.z);
      o.w = fmaf(v.w, f, o.w);
    }
    *reinterpret_cast<uint2 *>(ws.o16 + static_cast<uint64_t>(row) * R + c) = make_uint2(pack16(o.x, o.y), pack16(o.z, o.w));
  }
}

__device__ __forceinline__ void gated_store(const LatentAttnParams &p, uint32_t t, uint32_t e, const f32x4_t &o) {
  const float *g = p.proj + static_cast<uint64_t>(t) * p.proj_stride + p.gate_col + e;
  uint16_t *out = p.out16 + (p.packed_tiles != 0 ? gemm_x_block_index(p.packed_tiles, t, e, p.heads * p.value_dim) : static_cast<uint64_t>(t) * p.heads * p.value_dim + e);
  // (four columns stay together in operand order)
  *reinterpret_cast<uint2 *>(out) = make_uint2(pack16(o[0] * sigmoid(g[0]), o[1] * sigmoid(g[1])), pack16(o[2] * sigmoid(g[2]), o[3] * sigmoid(g[3])));
}

// Blocks of token rows. A workgroup: one head, up to 128 value columns, 128 tokens (32 a wave).
constexpr uint32_t kValueColumns = 128, kValueTokens = 128;
__global__ __launch_bounds__(kBlock) void latent_value_kernel(LatentAttnParams p, const uint16_t *o16) {
  constexpr uint32_t DT = kBF16, CT = kValueColumns / 16;
  const uint32_t R = p.kv_rank, h = blockIdx.y, c0 = blockIdx.x * kValueColumns;
  const uint32_t lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave, n = lane & 15u, q4 = lane >> 4;
  const uint32_t t0 = blockIdx.z * kValueTokens + wave * 32u + n;
  const uint16_t *x[2], *w[CT];
#pragma unroll
  for (uint32_t j = 0; j < 2; ++j) x[j] = o16 + (static_cast<uint64_t>(min(t0 + j * 16u, p.tokens - 1)) * p.heads + h) * R + q4 * 8u;
#pragma unroll
  for (uint32_t i = 0; i < CT; ++i)
    w[i] = p.w_uv + (static_cast<uint64_t>(h) * p.value_dim + min(c0 + i * 16u + n, p.value_dim - 1)) * R + q4 * 8u;
  f32x4_t acc[CT][2];
#pragma unroll
  for (uint32_t i = 0; i < CT; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  uint4 a[CT], b[2];
#pragma unroll
  for (uint32_t i = 0; i < CT; ++i) a[i] = *reinterpret_cast<const uint4 *>(w[i]);
#pragma unroll
  for (int j = 0; j < 2; ++j) b[j] = *reinterpret_cast<const uint4 *>(x[j]);
  for (uint32_t r = 0; r < R; r += 32) {
    const uint32_t next = r + 32 < R ? r + 32 : r;   // (the last step asks for its own again)
    uint4 an[CT], bn[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) bn[j] = *reinterpret_cast<const uint4 *>(x[j] + next);
#pragma unroll
    for (uint32_t i = 0; i < CT; ++i) an[i] = *reinterpret_cast<const uint4 *>(w[i] + next);
#pragma unroll
    for (uint32_t i = 0; i < CT; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[i][j] = mfma_k32<DT>(a[i], b[j], acc[i][j]);
#pragma unroll
    for (uint32_t i = 0; i < CT; ++i) a[i] = an[i];
#pragma unroll
    for (int j = 0; j < 2; ++j) b[j] = bn[j];
  }
#pragma unroll
  for (uint32_t j = 0; j < 2; ++j) {
    const uint32_t t = t0 + j * 16u;
    if (t >= p.tokens) continue;
#pragma unroll
    for (uint32_t i = 0; i < CT; ++i) {
      const uint32_t c = c0 + i * 16u + 4u * q4;
      if (c < p.value_dim) gated_store(p, t, h * p.value_dim + c, acc[i][j]);
    }
  }
}

// Factors of a head's splits (those that have left sums) into f_s; the lane's share of the splits' maxima and denominators
// as they were asked for. Returns 1 / denominator.
__device__ __forceinline__ float step_factors(float ms, float ls, uint32_t splits, float *f_s, float *red) {
  const uint32_t tid = threadIdx.x;
  float top = wave_max(ms);
  if (tid % kWave == 0) red[tid / kWave] = top;
  __syncthreads();
  top = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  const float f = ms > -INFINITY ? attn_exp2(ms - top) : 0.0f;
  if (tid < splits) f_s[tid] = f;
  return 1.0f / block_sum(ls * f, red);   // (its barriers publish f_s)
}
__device__ __forceinline__ uint32_t used_splits(const LatentAttnParams &p, uint32_t pos, uint32_t splits) {
  const Units u = units_of(p, pos, 0, 0, splits);
  return (u.count + u.per - 1) / u.per;
}

// Decode step with many splits: one workgroup per head and 64 latent columns - sixteen lanes a row, sixteen rows at a time;
// the merged row takes the place of the first split's.
constexpr uint32_t kMergeColumns = 64, kStepMergeSplits = 48;
__global__ __launch_bounds__(kBlock) void latent_merge_step_kernel(LatentAttnParams p, uint32_t splits) {
  __shared__ float f_s[kMostSplits], red[kWavesPerBlock];
  __shared__ float4 sum_s[kBlock];
  const uint32_t pos = *p.cursor;
  if (pos >= p.max_steps) return;
  const uint32_t R = p.kv_rank, h = blockIdx.y, tid = threadIdx.x, group = tid / 16u, c = blockIdx.x * kMergeColumns + tid % 16u * 4u;
  const Work ws = work_at(p.workspace, p.heads, R, R + p.rot_dim, splits);
  const uint64_t base = static_cast<uint64_t>(h) * splits;
  const uint32_t used = used_splits(p, pos, splits);
  constexpr uint32_t kEach = kMostSplits / 16u;
  float4 v[kEach];
#pragma unroll
  for (uint32_t i = 0; i < kEach; ++i) v[i] = *reinterpret_cast<const float4 *>(ws.sum + (base + min(group + i * 16u, used - 1)) * R + c);
  const float inv = step_factors(tid < splits ? ws.m[base + tid] : -INFINITY, tid < splits ? ws.l[base + tid] : 0.0f, splits, f_s, red);
  float4 o = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
#pragma unroll
  for (uint32_t i = 0; i < kEach; ++i) {
    const float f = group + i * 16u < used ? f_s[group + i * 16u] : 0.0f;
    o.x = fmaf(v[i].x, f, o.x);
    o.y = fmaf(v[i].y, f, o.y);
    o.z = fmaf(v[i].z, f, o.z);
    o.w = fmaf(v[i].w, f, o.w);
  }
  sum_s[tid] = o;
  __syncthreads();   // (everyone has read its splits, the first one among them)
  if (group != 0) return;
#pragma unroll
  for (uint32_t i = 1; i < 16u; ++i) {
    const float4 a = sum_s[i * 16u + tid];
    o.x += a.x;
    o.y += a.y;
    o.z += a.z;
    o.w += a.w;
  }
  *reinterpret_cast<float4 *>(ws.sum + base * R + c) = make_float4(o.x * inv, o.y * inv, o.z * inv, o.w * inv);
}

// Decode step: merges the splits of one head where that has not been done, then a wave a value column at a time.
constexpr uint32_t kStepColumns = 16;   // value columns of a workgroup
__global__ __launch_bounds__(kBlock) void latent_value_step_kernel(LatentAttnParams p, uint32_t splits, bool merged) {
  constexpr uint32_t DT = kBF16;
  __shared__ __align__(16) float o_s[kLatentMaxRank];
  __shared__ float f_s[kMostSplits], red[kWavesPerBlock];
  const uint32_t pos = *p.cursor;
  if (pos >= p.max_steps) return;
  const uint32_t R = p.kv_rank, h = blockIdx.y, tid = threadIdx.x, lane = tid & (kWave - 1), wave = tid / kWave;
  const Work ws = work_at(p.workspace, p.heads, R, R + p.rot_dim, splits);
  const uint64_t base = static_cast<uint64_t>(h) * splits;
  // the waves' weight rows are on their way while the splits are merged
  uint4 w[kStepColumns / kWavesPerBlock];
#pragma unroll
  for (uint32_t i = 0; i < kStepColumns / kWavesPerBlock; ++i) {
    const uint32_t c = min(blockIdx.x * kStepColumns + wave + i * kWavesPerBlock, p.value_dim - 1);
    w[i] = *reinterpret_cast<const uint4 *>(p.w_uv + (static_cast<uint64_t>(h) * p.value_dim + c) * R + (lane * 8u < R ? lane * 8u : 0u));
  }
  if (merged) {
    for (uint32_t c = tid * 2u; c < R; c += kBlock * 2u) *reinterpret_cast<float2 *>(o_s + c) = *reinterpret_cast<const float2 *>(ws.sum + base * R + c);
  } else {
    const float inv = step_factors(tid < splits ? ws.m[base + tid] : -INFINITY, tid < splits ? ws.l[base + tid] : 0.0f, splits, f_s, red);
    const uint32_t used = used_splits(p, pos, splits);
    for (uint32_t c = tid * 2u; c < R; c += kBlock * 2u) {
      float2 o = make_float2(0.0f, 0.0f);
#pragma unroll 16
      for (uint32_t i = 0; i < used; ++i) {
        const float2 v = *reinterpret_cast<const float2 *>(ws.sum + (base + i) * R + c);
        o.x = fmaf(v.x, f_s[i], o.x);
        o.y = fmaf(v.y, f_s[i], o.y);
      }
      o_s[c] = o.x * inv;
      o_s[c + 1] = o.y * inv;
    }
  }
  __syncthreads();
#pragma unroll
  for (uint32_t i = 0; i < kStepColumns / kWavesPerBlock; ++i) {
    const uint32_t c = blockIdx.x * kStepColumns + wave + i * kWavesPerBlock;
    if (c >= p.value_dim) break;
    float sum = 0.0f;
    for (uint32_t r = lane * 8u; r < R; r += kWave * 8u) {
      const uint4 v = r == lane * 8u ? w[i] : *reinterpret_cast<const uint4 *>(p.w_uv + (static_cast<uint64_t>(h) * p.value_dim + c) * R + r);
      const uint32_t words[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float a, b;
        unpack2<DT>(words[e], a, b);
        sum = fmaf(a, o_s[r + 2 * e], sum);
        sum = fmaf(b, o_s[r + 2 * e + 1], sum);
      }
    }
    sum = wave_sum(sum);
    const uint32_t e = h * p.value_dim + c;
    if (lane == 0) p.out16[p.packed_tiles != 0 ? gemm_x_packed_index(p.packed_tiles, 0, e) : e] = enc16<DT>(sum * sigmoid(p.proj[p.gate_col + e]));
  }
}

// ---- launches --------------------------------------------------------------------------------

uint32_t step_splits(const LatentAttnParams &p) {
  const uint32_t blocks = p.window != 0 ? std::min(p.window / kKvBlockTokens + 2, p.last_block + 1) : p.last_block + 1;
  return std::max(1u, std::min(kMostSplits, (blocks + 1) / 2));
}
uint32_t block_splits(uint32_t rows) {
  const uint32_t groups = (rows + 2 * kPairRows - 1) / (2 * kPairRows);
  return std::max(1u, std::min(kBlockSplits, kWorkgroups / groups));
}

template <int R, int RD, int PAIRS>
hipError_t launch_rows(const LatentAttnParams &p, uint32_t splits, hipStream_t stream) {
  constexpr size_t lds = latent_rows_lds<R, RD, PAIRS>();
  const uint32_t rows = p.tokens * p.heads, groups = (rows + PAIRS * kPairRows - 1) / (PAIRS * kPairRows);
  hipLaunchKernelGGL((latent_rows_kernel<R, RD, PAIRS>), dim3(groups * splits), dim3(2 * PAIRS * kWave), lds, stream, p, splits);
  return hipGetLastError();
}

template <int R, int RD>
hipError_t launch_shape(const LatentAttnParams &p, hipStream_t stream, uint64_t *launches) {
  const bool step = p.cursor != nullptr;
  const uint32_t rows = p.tokens * p.heads, splits = step ? step_splits(p) : block_splits(rows);
  const Work ws = work_at(p.workspace, rows, R, R + RD, splits);
  const uint32_t token_tiles = (p.tokens + 63) / 64;
  if (step) hipLaunchKernelGGL((latent_absorb_kernel<4>), dim3(R / 64 + 1, p.heads, 1), dim3(kBlock), 0, stream, p, ws.q16);
  else hipLaunchKernelGGL((latent_absorb_kernel<8>), dim3(R / 128 + 1, p.heads, token_tiles), dim3(kBlock), 0, stream, p, ws.q16);
  hipError_t err = hipGetLastError();
  if (err != hipSuccess) return err;
  err = rows > kPairRows ? launch_rows<R, RD, 2>(p, splits, stream) : launch_rows<R, RD, 1>(p, splits, stream);
  if (err != hipSuccess) return err;
  if (step) {
    const bool merged = splits > kStepMergeSplits;
    *launches += merged ? 4 : 3;
    if (merged) {
      hipLaunchKernelGGL(latent_merge_step_kernel, dim3(R / kMergeColumns, p.heads), dim3(kBlock), 0, stream, p, splits);
      err = hipGetLastError();
      if (err != hipSuccess) return err;
    }
    hipLaunchKernelGGL(latent_value_step_kernel, dim3((p.value_dim + kStepColumns - 1) / kStepColumns, p.heads), dim3(kBlock), 0, stream, p, splits,
                       merged);
    return hipGetLastError();
  }
  *launches += splits > 1 ? 4 : 3;
  if (splits > 1) {
    hipLaunchKernelGGL(latent_merge_kernel, dim3(rows), dim3(kBlock), 0, stream, p, splits);
    err = hipGetLastError();
    if (err != hipSuccess) return err;
  }
  hipLaunchKernelGGL(latent_value_kernel, dim3((p.value_dim + kValueColumns - 1) / kValueColumns, p.heads, (p.tokens + kValueTokens - 1) / kValueTokens),
                     dim3(kBlock), 0, stream, p,
                     static_cast<const uint16_t *>(ws.o16));
  return hipGetLastError();
}

template <int R, int RD>
hipError_t raise_lds() {
  hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_rows_kernel<R, RD, 2>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                       static_cast<int>(latent_rows_lds<R, RD, 2>()));
  if (err == hipSuccess)
    err = hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_rows_kernel<R, RD, 1>), hipFuncAttributeMaxDynamicSharedMemorySize,
                              static_cast<int>(latent_rows_lds<R, RD, 1>()));
  return err;
}

}  // namespace

bool latent_attention_wide(uint32_t heads, uint32_t key_dim, uint32_t rot_dim, uint32_t value_dim, uint32_t kv_rank) {
  const bool shape = (kv_rank == 512 && rot_dim == 64) || (kv_rank == 256 && rot_dim == 64) || (kv_rank == 128 && rot_dim == 64);
  return shape && heads != 0 && key_dim % 32 == 0 && value_dim % 16 == 0 && (key_dim + rot_dim) % 4 == 0;
}

uint64_t latent_workspace_bytes(uint32_t heads, uint32_t rot_dim, uint32_t kv_rank, uint32_t max_tokens) {
  const uint64_t width = kv_rank + rot_dim, partial = (kv_rank + 2ull) * sizeof(float);
  const auto total = [&](uint64_t rows, uint64_t splits) {
    return (rows * (width + kv_rank) + 256u) * sizeof(uint16_t) + (splits > 1 ? rows * splits * partial : 0u) + 1024u;
  };
  uint64_t most = total(heads, kMostSplits);
  for (uint32_t t = 1; t <= max_tokens; ++t) most = std::max(most, total(static_cast<uint64_t>(t) * heads, block_splits(t * heads)));
  return most;
}

hipError_t latent_wide_setup() {
  static std::once_flag once;
  static hipError_t raised = hipSuccess;
  std::call_once(once, [] {
    raised = raise_lds<512, 64>();
    if (raised == hipSuccess) raised = raise_lds<256, 64>();
    if (raised == hipSuccess) raised = raise_lds<128, 64>();
  });
  return raised;
}

hipError_t launch_latent_attention_wide(uint32_t dtype, const LatentAttnParams &p, hipStream_t stream, uint64_t *launches) {
  const auto aligned = [](const void *q, uintptr_t n) { return (reinterpret_cast<uintptr_t>(q) & (n - 1)) == 0; };
  if (dtype != kBF16 || !latent_attention_wide(p.heads, p.key_dim, p.rot_dim, p.value_dim, p.kv_rank) || p.cache32 != 0 || p.out16 == nullptr ||
      p.workspace == nullptr || p.proj == nullptr || p.q == nullptr || p.w_uk == nullptr || p.w_uv == nullptr || p.cache == nullptr ||
      p.table == nullptr || p.kv_norm == nullptr || p.tokens == 0 || p.rot_dims % 2 != 0 || p.rot_dims > p.rot_dim ||
      (p.rot_dims != 0 && p.rope_cs == nullptr) || (p.packed_tiles != 0 && (p.packed_tiles * 16u < std::min(p.tokens, kGemmDeepMaxTokens) || p.heads * p.value_dim % 32 != 0)))
    return hipErrorInvalidValue;
  if (!aligned(p.workspace, 256) || !aligned(p.cache, 16) || !aligned(p.w_uk, 16) || !aligned(p.w_uv, 16) || !aligned(p.q, 16) || !aligned(p.out16, 16))
    return hipErrorInvalidValue;
  if (p.cursor != nullptr ? p.tokens != 1 : (p.position + p.tokens - 1) / kKvBlockTokens > p.last_block) return hipErrorInvalidValue;
  if (p.kv_rank == 512) return launch_shape<512, 64>(p, stream, launches);
  if (p.kv_rank == 256) return launch_shape<256, 64>(p, stream, launches);
  return launch_shape<128, 64>(p, stream, launches);
}

}  // namespace nv
