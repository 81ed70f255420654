// Routed experts over blocks of token rows (see moe_rows.cuh).
#include "moe_rows.cuh"

#include <algorithm>
#include <mutex>

#include "activations.cuh"

namespace nv {

namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4_t mfma_k32(const uint4 &a, const uint4 &b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}

// ---- routing ---------------------------------------------------------------------------------

// One wave per token: scores in registers, `top` rounds of a wave-wide maximum.
constexpr uint32_t kScoreRegs = kMaxExperts / kWave;
__global__ __launch_bounds__(kBlock) void moe_route_rows_kernel(MoeRouteRows p) {
  const uint32_t t = blockIdx.x * kWavesPerBlock + threadIdx.x / kWave, lane = threadIdx.x % kWave;
  if (t >= p.tokens) return;
  const float *z = p.logits + static_cast<uint64_t>(t) * p.experts;
  float s[kScoreRegs];
#pragma unroll
  for (uint32_t i = 0; i < kScoreRegs; ++i) {
    const uint32_t e = i * kWave + lane;
    s[i] = -1.0f;
    if (i * kWave < p.experts && e < p.experts) s[i] = 1.0f / (1.0f + expf(-z[e]));
  }
  float sum = 0.0f, mine = 0.0f;   // lane k keeps choice k
  uint32_t mine_id = 0;
  for (uint32_t k = 0; k < p.top; ++k) {
    Best b{0.0f, 0u, 0u};
#pragma unroll
    for (uint32_t i = 0; i < kScoreRegs; ++i) {
      if (i * kWave >= p.experts) break;
      const Best c{s[i], i * kWave + lane, s[i] >= 0.0f ? 1u : 0u};
      if (better(c, b)) b = c;
    }
    b = wave_best(b);
    // (scores that are no numbers: some expert that exists, so that every slot has one)
    const uint32_t e = b.has != 0 ? b.index : k;
#pragma unroll
    for (uint32_t i = 0; i < kScoreRegs; ++i)
      if (i * kWave + lane == e) s[i] = -1.0f;
    sum += b.value;
    if (lane == k) {
      mine = b.value;
      mine_id = e;
    }
  }
  if (lane < p.top) {
    p.plan.ids[static_cast<uint64_t>(t) * p.top + lane] = mine_id;
    p.plan.weights[static_cast<uint64_t>(t) * p.top + lane] = mine / (sum + 1e-20f);
  }
}

// One workgroup: counts per expert, places, tiles.
constexpr uint32_t kSortThreads = 1024;
__global__ __launch_bounds__(kSortThreads) void moe_sort_kernel(MoeRouteRows p) {
  __shared__ uint32_t count[kMaxExperts], first[kMaxExperts], tile_at[kMaxExperts], wave_total[2][kSortThreads / kWave];
  const uint32_t slots = p.tokens * p.top, tid = threadIdx.x;
  for (uint32_t e = tid; e < kMaxExperts; e += kSortThreads) count[e] = 0;
  __syncthreads();
  for (uint32_t i = tid; i < slots; i += kSortThreads) atomicAdd(&count[min(p.plan.ids[i], p.experts - 1)], 1u);
  __syncthreads();
  // exclusive sums over the experts (one each), of slots and of tiles
  static_assert(kMaxExperts == kSortThreads, "one expert a thread");
  const uint32_t size = p.plan.tile, n = count[tid], tiles = (n + size - 1) / size;
  uint32_t a = n, b = tiles;
#pragma unroll
  for (uint32_t o = 1; o < kWave; o <<= 1) {
    const uint32_t ua = __shfl_up(a, o, kWave), ub = __shfl_up(b, o, kWave);
    if (tid % kWave >= o) {
      a += ua;
      b += ub;
    }
  }
  if (tid % kWave == kWave - 1) {
    wave_total[0][tid / kWave] = a;
    wave_total[1][tid / kWave] = b;
  }
  __syncthreads();
  for (uint32_t w = 0; w < tid / kWave; ++w) {
    a += wave_total[0][w];
    b += wave_total[1][w];
  }
  first[tid] = a - n;
  tile_at[tid] = b - tiles;
  if (tid == kSortThreads - 1) *p.plan.tile_count = b;
  for (uint32_t i = 0; i < tiles; ++i)
    p.plan.tiles[b - tiles + i] = make_uint4(tid, a - n + i * size, min(size, n - i * size), 0u);
  __syncthreads();
  for (uint32_t i = tid; i < slots; i += kSortThreads) {
    const uint32_t at = atomicAdd(&first[min(p.plan.ids[i], p.experts - 1)], 1u);
    p.plan.sorted[at] = i;
  }
}

// ---- products --------------------------------------------------------------------------------

enum : int { kExpertGateUp = 0, kExpertDown = 1 };

struct Products {
  const uint16_t *w;          // the experts' matrices
  const uint16_t *x16;
  const float *x32;
  uint16_t *act16;
  float *act32, *out;
  uint32_t rows, cols;        // output rows (gate/up: of either half), columns
  uint32_t tokens, top;
  float limit;
  const uint4 *tiles;         // null: one expert, consecutive tokens
  const uint32_t *tile_count, *sorted;
};

struct Tile {
  uint32_t expert, first, count;
};
template <uint32_t TN>
__device__ __forceinline__ bool tile_of(const Products &p, uint32_t i, Tile &t) {
  if (p.tiles == nullptr) {
    t = Tile{0u, i * TN, min(TN, p.tokens - i * TN)};
    return true;
  }
  if (i >= *p.tile_count) return false;
  const uint4 v = p.tiles[i];
  t = Tile{v.x, v.y, v.z};
  return true;
}
__device__ __forceinline__ uint32_t slot_of(const Products &p, uint32_t place) { return p.tiles == nullptr ? place : p.sorted[place]; }
// Row of the input that belongs to a slot: the token for the gate/up products, the slot itself for the down product.
template <int EPI>
__device__ __forceinline__ uint32_t input_row(const Products &p, uint32_t slot) {
  return EPI == kExpertGateUp ? slot / p.top : slot;
}

constexpr uint32_t kRows = 128;         // matrix rows of a workgroup (gate/up: 64 of each)
constexpr uint32_t kStep = 64;          // columns staged at a time
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

// TN: slots of a tile.
template <uint32_t DT, int EPI, bool VEC, uint32_t TN>
__global__ __launch_bounds__(kBlock) void expert_rows_kernel(Products p) {
  __shared__ __align__(16) uint16_t ws[kRows * kPitch];
  __shared__ __align__(16) uint16_t xs[TN * kPitch];
  __shared__ uint32_t slots[TN];
  Tile tile;
  if (!tile_of<TN>(p, blockIdx.y, tile)) return;
  const uint32_t lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
  constexpr uint32_t kOutRows = EPI == kExpertGateUp ? kRows / 2 : kRows;
  const uint32_t row0 = blockIdx.x * kOutRows, cols = p.cols;
  if (threadIdx.x < TN) slots[threadIdx.x] = slot_of(p, tile.first + min(threadIdx.x, tile.count - 1));
  __syncthreads();
  const uint16_t *w = p.w + static_cast<uint64_t>(tile.expert) * (EPI == kExpertGateUp ? 2u : 1u) * p.rows * cols;
  // staging: thread -> (row of the tile, eight columns), four rows of the matrix, TN / 32 of the input
  const uint32_t sr = threadIdx.x / 8u, sc = (threadIdx.x % 8u) * 8u;
  constexpr uint32_t XR = TN / 32, JT = TN / 32;   // input rows a thread stages, slot tiles a wave holds
  const uint16_t *wr[4], *xr[XR];
#pragma unroll
  for (uint32_t i = 0; i < 4; ++i) {
    const uint32_t r = sr + 32u * i;
    const uint32_t row = EPI == kExpertGateUp ? (r / 64u) * p.rows + min(row0 + r % 64u, p.rows - 1) : min(row0 + r, p.rows - 1);
    wr[i] = w + static_cast<uint64_t>(row) * cols;
  }
#pragma unroll
  for (uint32_t i = 0; i < XR; ++i) xr[i] = p.x16 + static_cast<uint64_t>(input_row<EPI>(p, slots[sr + 32u * i])) * cols;
  uint4 wq[4], xq[XR];
#pragma unroll
  for (uint32_t i = 0; i < 4; ++i) wq[i] = piece8<VEC>(wr[i], sc, cols);
#pragma unroll
  for (uint32_t i = 0; i < XR; ++i) xq[i] = piece8<VEC>(xr[i], sc, cols);
  // a wave: 32 gate and the 32 up rows of the same outputs (down: 64 rows), half of the slots
  f32x4_t acc[4][JT];
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (uint32_t b = 0; b < JT; ++b) acc[a][b] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  const uint32_t n = lane & 15u, q = lane >> 4, half = wave & 1u;
  const auto w_row = [&](uint32_t i) { return EPI == kExpertGateUp ? (i / 2u) * 64u + half * 32u + (i % 2u) * 16u : half * 64u + i * 16u; };
  const uint16_t *b_at = xs + ((wave >> 1) * (TN / 2) + n) * kPitch + q * 8u;
  for (uint32_t k = 0; k < cols; k += kStep) {
    __syncthreads();
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) *reinterpret_cast<uint4 *>(ws + (sr + 32u * i) * kPitch + sc) = wq[i];
#pragma unroll
    for (uint32_t i = 0; i < XR; ++i) *reinterpret_cast<uint4 *>(xs + (sr + 32u * i) * kPitch + sc) = xq[i];
    __syncthreads();
    if (k + kStep < cols) {
#pragma unroll
      for (uint32_t i = 0; i < 4; ++i) wq[i] = piece8<VEC>(wr[i], k + kStep + sc, cols);
#pragma unroll
      for (uint32_t i = 0; i < XR; ++i) xq[i] = piece8<VEC>(xr[i], k + kStep + sc, cols);
    }
#pragma unroll
    for (uint32_t s = 0; s < kStep / 32u; ++s) {
      uint4 a[4], b[JT];
#pragma unroll
      for (uint32_t i = 0; i < 4; ++i) a[i] = *reinterpret_cast<const uint4 *>(ws + (w_row(i) + n) * kPitch + q * 8u + s * 32u);
#pragma unroll
      for (uint32_t j = 0; j < JT; ++j) b[j] = *reinterpret_cast<const uint4 *>(b_at + j * 16u * kPitch + s * 32u);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (uint32_t j = 0; j < JT; ++j) acc[i][j] = mfma_k32(a[i], b[j], acc[i][j]);
    }
  }
#pragma unroll
  for (uint32_t j = 0; j < JT; ++j) {
    const uint32_t t = (wave >> 1) * (TN / 2) + j * 16u + n;
    if (t >= tile.count) continue;
    const uint64_t at = static_cast<uint64_t>(slots[t]) * p.rows;
#pragma unroll
    for (uint32_t i = 0; i < (EPI == kExpertGateUp ? 2u : 4u); ++i)
#pragma unroll
      for (uint32_t r = 0; r < 4; ++r) {
        const uint32_t row = row0 + (EPI == kExpertGateUp ? half * 32u : half * 64u) + i * 16u + q * 4u + r;
        if (row >= p.rows) continue;
        if constexpr (EPI == kExpertGateUp) p.act16[at + row] = enc16<DT>(clamped_glu(acc[i][j][r], acc[i + 2][j][r], p.limit));
        else p.out[at + row] = acc[i][j][r];
      }
  }
}

// Large tiles, whole 64-column steps: 256 matrix rows (gate/up: 128 of each) x 128 slots on eight waves, a wave 64 x 64.
// Matrix rows and gathered input rows go from global memory to LDS directly (global_load_lds, 1 KiB a request: eight rows
// of 128 bytes, whose 16-byte pieces are XORed with the row number on the way in - operand reads are then free of bank
// conflicts), three buffers, two steps ahead; one barrier a step. Operand reads are issued by hand with counted waits (the
// compiler would wait for the requests in flight as well).
constexpr uint32_t kDeepRows = 256, kDeepSlots = 2 * kExpertTile, kDeepStep = 64;
constexpr int kDeepW = kDeepRows * kDeepStep * 2, kDeepX = kDeepSlots * kDeepStep * 2, kDeepBuf = kDeepW + kDeepX;
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));

template <uint32_t DT, int EPI>
__global__ __launch_bounds__(8 * kWave, 2) void expert_deep_kernel(Products p, uint32_t row_tiles) {
  extern __shared__ __align__(16) unsigned char smem[];
  constexpr uint32_t kOutRows = EPI == kExpertGateUp ? kDeepRows / 2 : kDeepRows;
  // an XCD takes a run of consecutive (slot tile, row tile) pairs, row tiles fastest: it meets an expert's rows, and a
  // tile's slots, again while its L2 holds them
  const uint32_t all = row_tiles * (p.tiles != nullptr ? *p.tile_count : (p.tokens + kDeepSlots - 1) / kDeepSlots), run = (all + 7u) / 8u;
  const uint32_t at = (blockIdx.x % 8u) * run + blockIdx.x / 8u;
  if (blockIdx.x / 8u >= run || at >= all) return;
  Tile tile;
  if (!tile_of<kDeepSlots>(p, at / row_tiles, tile)) return;
  const uint32_t row0 = at % row_tiles * kOutRows, cols = p.cols;
  const uint32_t lane = threadIdx.x & (kWave - 1), wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const uint32_t n = lane & 15u, q = lane >> 4, th = wave & 1u, rq = wave >> 1;
  const uint16_t *w = p.w + static_cast<uint64_t>(tile.expert) * (EPI == kExpertGateUp ? 2u : 1u) * p.rows * cols;
  // requests of this wave: 32 rows of the matrix, 16 of the input, eight a request; lane (row, piece)
  const uint32_t lr = lane >> 3, lc = ((lane & 7u) ^ lr) * 8u;
  const uint16_t *wsrc[4], *xsrc[2];
#pragma unroll
  for (uint32_t i = 0; i < 4; ++i) {
    const uint32_t r = wave * 32u + i * 8u + lr;
    const uint32_t row = EPI == kExpertGateUp ? (r / 128u) * p.rows + min(row0 + r % 128u, p.rows - 1) : min(row0 + r, p.rows - 1);
    wsrc[i] = w + static_cast<uint64_t>(row) * cols + lc;
  }
#pragma unroll
  for (uint32_t i = 0; i < 2; ++i)
    xsrc[i] = p.x16 + static_cast<uint64_t>(input_row<EPI>(p, slot_of(p, tile.first + min(wave * 16u + i * 8u + lr, tile.count - 1)))) * cols + lc;
#define NV_ED_LDS(P) ((__attribute__((address_space(3))) void *)(P))
  const auto request = [&](uint32_t step, uint32_t buffer) {
    unsigned char *to = smem + buffer * kDeepBuf;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      __builtin_amdgcn_global_load_lds(reinterpret_cast<const uint32_t *>(wsrc[i] + step * kDeepStep), NV_ED_LDS(to + (wave * 4 + i) * 1024), 16, 0, 0);
#pragma unroll
    for (int i = 0; i < 2; ++i)
      __builtin_amdgcn_global_load_lds(reinterpret_cast<const uint32_t *>(xsrc[i] + step * kDeepStep), NV_ED_LDS(to + kDeepW + (wave * 2 + i) * 1024), 16, 0, 0);
  };
  const uint32_t lds0 = static_cast<uint32_t>(reinterpret_cast<uintptr_t>(NV_ED_LDS(smem)));
#undef NV_ED_LDS
  // operand addresses of the step's two K-steps: row tile i of the wave at + (gate/up: tiles 0, 1 gate, 2, 3 up) ...
  uint32_t a_at[2], b_at[2];
#pragma unroll
  for (uint32_t e = 0; e < 2; ++e) {
    const uint32_t piece = ((e * 4u + q) ^ (n & 7u)) << 4;
    a_at[e] = lds0 + (rq * (EPI == kExpertGateUp ? 32u : 64u) + n) * 128u + piece;
    b_at[e] = lds0 + kDeepW + (th * 64u + n) * 128u + piece;
  }
  constexpr auto a_tile = [](int i) { return EPI == kExpertGateUp ? (i / 2) * 128 * 128 + (i % 2) * 2048 : i * 2048; };
  f32x4_t acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.0f, 0.0f, 0.0f, 0.0f};
  const uint32_t steps = cols / kDeepStep;   // at least two
  request(0, 0);
  request(1, 1);
  uint32_t buffer = 0;
  for (uint32_t k = 0; k < steps; ++k) {
    // this step's requests are through (the next step's six may be in flight), nobody reads the last step's any more
    if (k + 1 < steps) asm volatile("s_waitcnt vmcnt(6) lgkmcnt(0)\n\ts_barrier" ::: "memory");
    else asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
    if (k + 2 < steps) request(k + 2, buffer == 0 ? 2u : buffer - 1u);
    const uint32_t off = buffer * kDeepBuf;
    u32x4_t a[2][4], b[2][4];
#pragma unroll
    for (int e = 0; e < 2; ++e) {
#pragma unroll
      for (int i = 0; i < 4; ++i) asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(a[e][i]) : "v"(a_at[e] + off), "n"(a_tile(i)) : "memory");
#pragma unroll
      for (int j = 0; j < 4; ++j) asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(b[e][j]) : "v"(b_at[e] + off), "n"(j * 2048) : "memory");
    }
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      asm volatile("s_waitcnt lgkmcnt(%c[left])" : "+v"(a[e][0]), "+v"(a[e][1]), "+v"(a[e][2]), "+v"(a[e][3]), "+v"(b[e][0]), "+v"(b[e][1]),
                   "+v"(b[e][2]), "+v"(b[e][3]) : [left] "n"(8 - 8 * e) : "memory");
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mfma_k32(__builtin_bit_cast(uint4, a[e][i]), __builtin_bit_cast(uint4, b[e][j]), acc[i][j]);
    }
    buffer = buffer == 2 ? 0u : buffer + 1u;
  }
#pragma unroll
  for (uint32_t j = 0; j < 4; ++j) {
    const uint32_t t = th * 64u + j * 16u + n;
    if (t >= tile.count) continue;
    const uint64_t to = static_cast<uint64_t>(slot_of(p, tile.first + t)) * p.rows;
#pragma unroll
    for (uint32_t i = 0; i < (EPI == kExpertGateUp ? 2u : 4u); ++i) {
      const uint32_t row = row0 + rq * (EPI == kExpertGateUp ? 32u : 64u) + i * 16u + q * 4u;
      if (row >= p.rows) continue;   // (rows are whole groups of four)
      if constexpr (EPI == kExpertGateUp) {
        uint32_t o[2];
#pragma unroll
        for (int r = 0; r < 2; ++r)
          o[r] = enc16<DT>(clamped_glu(acc[i][j][2 * r], acc[i + 2][j][2 * r], p.limit)) |
                 (static_cast<uint32_t>(enc16<DT>(clamped_glu(acc[i][j][2 * r + 1], acc[i + 2][j][2 * r + 1], p.limit))) << 16);
        *reinterpret_cast<uint2 *>(p.act16 + to + row) = make_uint2(o[0], o[1]);
      } else {
        *reinterpret_cast<float4 *>(p.out + to + row) = make_float4(acc[i][j][0], acc[i][j][1], acc[i][j][2], acc[i][j][3]);
      }
    }
  }
}

constexpr uint32_t kTile32 = 64, kStep32 = 16;   // output rows of a workgroup, columns staged at a time (f32 rows)

template <uint32_t DT, int EPI>
__global__ __launch_bounds__(kBlock) void expert_rows_f32_kernel(Products p) {
  constexpr uint32_t M = EPI == kExpertGateUp ? 2 : 1;   // matrices that meet in one output
  __shared__ float ws[M][kStep32][kTile32 + 4], xs[kStep32][kExpertTile + 4];
  __shared__ uint32_t slots[kExpertTile];
  Tile tile;
  if (!tile_of<kExpertTile>(p, blockIdx.y, tile)) return;
  const uint32_t row0 = blockIdx.x * kTile32, cols = p.cols;
  if (threadIdx.x < kExpertTile) slots[threadIdx.x] = slot_of(p, tile.first + min(threadIdx.x, tile.count - 1));
  __syncthreads();
  const uint16_t *w = p.w + static_cast<uint64_t>(tile.expert) * M * p.rows * cols;
  const uint32_t tr = threadIdx.x % 16u, tt = threadIdx.x / 16u;
  float acc[M][4][4] = {};
  for (uint32_t k = 0; k < cols; k += kStep32) {
    __syncthreads();
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) {
      const uint32_t r = threadIdx.x / 16u + 16u * i, c = threadIdx.x % 16u;
      const bool in = k + c < cols;
#pragma unroll
      for (uint32_t m = 0; m < M; ++m)
        ws[m][c][r] = in ? dec16<DT>(w[(static_cast<uint64_t>(m) * p.rows + min(row0 + r, p.rows - 1)) * cols + k + c]) : 0.0f;
      xs[c][r] = in ? p.x32[static_cast<uint64_t>(input_row<EPI>(p, slots[r])) * cols + k + c] : 0.0f;
    }
    __syncthreads();
#pragma unroll
    for (uint32_t c = 0; c < kStep32; ++c)
#pragma unroll
      for (uint32_t m = 0; m < M; ++m)
#pragma unroll
        for (uint32_t i = 0; i < 4; ++i)
#pragma unroll
          for (uint32_t j = 0; j < 4; ++j) acc[m][i][j] = fmaf(ws[m][c][tr + 16u * i], xs[c][tt + 16u * j], acc[m][i][j]);
  }
#pragma unroll
  for (uint32_t j = 0; j < 4; ++j) {
    const uint32_t t = tt + 16u * j;
    if (t >= tile.count) continue;
    const uint64_t at = static_cast<uint64_t>(slots[t]) * p.rows;
#pragma unroll
    for (uint32_t i = 0; i < 4; ++i) {
      const uint32_t row = row0 + tr + 16u * i;
      if (row >= p.rows) continue;
      if constexpr (EPI == kExpertGateUp) p.act32[at + row] = clamped_glu(acc[0][i][j], acc[M - 1][i][j], p.limit);
      else p.out[at + row] = acc[0][i][j];
    }
  }
}

template <int EPI>
hipError_t launch(const ExpertRows &e, hipStream_t stream) {
  Products p{};
  const bool narrow = e.x16 != nullptr;
  p.w = EPI == kExpertGateUp ? e.w_gate_up : e.w_down;
  p.x16 = EPI == kExpertGateUp ? e.x16 : e.act16;
  p.x32 = EPI == kExpertGateUp ? e.x32 : e.act32;
  p.act16 = e.act16;
  p.act32 = e.act32;
  p.out = e.out;
  p.rows = EPI == kExpertGateUp ? e.ff : e.hidden;
  p.cols = EPI == kExpertGateUp ? e.hidden : e.ff;
  p.tokens = e.tokens;
  p.top = e.top;
  p.limit = e.limit;
  // (f32 rows: the sort has made small tiles)
  const uint32_t size = e.plan != nullptr ? e.plan->tile : narrow ? expert_tile(e.tokens, 1) : kExpertTile;
  if (!narrow && size != kExpertTile) return hipErrorInvalidValue;
  uint32_t tiles = (e.tokens + size - 1) / size;
  if (e.plan != nullptr) {
    p.tiles = e.plan->tiles;
    p.tile_count = e.plan->tile_count;
    p.sorted = e.plan->sorted;
    tiles = moe_max_tiles(e.tokens, e.top, e.experts, size);
  }
  const bool aligned = ((reinterpret_cast<uintptr_t>(p.w) | reinterpret_cast<uintptr_t>(p.x16)) & 15u) == 0;
  if (tiles > 65535u) return hipErrorInvalidValue;
  if (!narrow) {
    hipLaunchKernelGGL((expert_rows_f32_kernel<kBF16, EPI>), dim3((p.rows + kTile32 - 1) / kTile32, tiles), dim3(kBlock), 0, stream, p);
  } else {
    constexpr uint32_t kOutRows = EPI == kExpertGateUp ? kRows / 2 : kRows;
    const dim3 grid((p.rows + kOutRows - 1) / kOutRows, tiles);
    const bool large = size != kExpertTile;
    if (large && aligned && p.cols % kDeepStep == 0 && p.cols >= 2 * kDeepStep && p.rows % 4 == 0 && (reinterpret_cast<uintptr_t>(p.out) & 15u) == 0 &&
        (reinterpret_cast<uintptr_t>(p.act16) & 7u) == 0) {
      constexpr uint32_t kDeepOut = EPI == kExpertGateUp ? kDeepRows / 2 : kDeepRows;
      const uint32_t row_tiles = (p.rows + kDeepOut - 1) / kDeepOut;
      const uint64_t most = (static_cast<uint64_t>(row_tiles) * tiles + 7u) / 8u * 8u;
      if (most > 0x7fffffffu) return hipErrorInvalidValue;
      hipLaunchKernelGGL((expert_deep_kernel<kBF16, EPI>), dim3(static_cast<uint32_t>(most)), dim3(8 * kWave), 3 * kDeepBuf, stream, p, row_tiles);
    } else if (p.cols % 8 == 0 && aligned && large) hipLaunchKernelGGL((expert_rows_kernel<kBF16, EPI, true, 2 * kExpertTile>), grid, dim3(kBlock), 0, stream, p);
    else if (p.cols % 8 == 0 && aligned) hipLaunchKernelGGL((expert_rows_kernel<kBF16, EPI, true, kExpertTile>), grid, dim3(kBlock), 0, stream, p);
    else if (large) hipLaunchKernelGGL((expert_rows_kernel<kBF16, EPI, false, 2 * kExpertTile>), grid, dim3(kBlock), 0, stream, p);
    else hipLaunchKernelGGL((expert_rows_kernel<kBF16, EPI, false, kExpertTile>), grid, dim3(kBlock), 0, stream, p);
  }
  return hipGetLastError();
}

bool rows_ok(uint32_t dtype, const ExpertRows &p) {
  return dtype == kBF16 && p.w_gate_up != nullptr && p.w_down != nullptr && (p.x16 == nullptr) != (p.x32 == nullptr) &&
         (p.x16 != nullptr ? p.act16 != nullptr : p.act32 != nullptr) && p.hidden != 0 && p.ff != 0 && p.tokens != 0 && p.top != 0 &&
         p.experts != 0 && (p.plan != nullptr ? p.experts <= kMaxExperts && p.top <= kMaxTop && p.top <= p.experts : p.experts == 1 && p.top == 1);
}

}  // namespace

uint64_t moe_plan_bytes(uint32_t tokens, uint32_t top, uint32_t experts) {
  return static_cast<uint64_t>(tokens) * top * 12 + static_cast<uint64_t>(moe_max_tiles(tokens, top, experts, kExpertTile)) * sizeof(uint4) + 64;
}

MoePlan moe_plan_at(void *base, uint32_t tokens, uint32_t top, uint32_t experts, bool small_tiles) {
  const uint64_t slots = static_cast<uint64_t>(tokens) * top;
  MoePlan m;
  m.tiles = static_cast<uint4 *>(base);
  m.ids = reinterpret_cast<uint32_t *>(m.tiles + moe_max_tiles(tokens, top, experts, kExpertTile));
  m.weights = reinterpret_cast<float *>(m.ids + slots);
  m.sorted = reinterpret_cast<uint32_t *>(m.weights + slots);
  m.tile_count = m.sorted + slots;
  m.tile = small_tiles ? kExpertTile : expert_tile(tokens * top, experts);
  return m;
}

hipError_t expert_rows_setup() {
  static std::once_flag once;
  static hipError_t raised = hipSuccess;
  std::call_once(once, [] {
    raised = hipFuncSetAttribute(reinterpret_cast<const void *>(&expert_deep_kernel<kBF16, kExpertGateUp>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                 3 * kDeepBuf);
    if (raised == hipSuccess)
      raised = hipFuncSetAttribute(reinterpret_cast<const void *>(&expert_deep_kernel<kBF16, kExpertDown>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                   3 * kDeepBuf);
  });
  return raised;
}

hipError_t launch_moe_route_rows(const MoeRouteRows &p, hipStream_t stream) {
  if (p.logits == nullptr || p.tokens == 0 || p.experts == 0 || p.experts > kMaxExperts || p.top == 0 || p.top > p.experts || p.top > kMaxTop)
    return hipErrorInvalidValue;
  hipLaunchKernelGGL(moe_route_rows_kernel, dim3((p.tokens + kWavesPerBlock - 1) / kWavesPerBlock), dim3(kBlock), 0, stream, p);
  hipError_t err = hipGetLastError();
  if (err != hipSuccess) return err;
  hipLaunchKernelGGL(moe_sort_kernel, dim3(1), dim3(kSortThreads), 0, stream, p);
  return hipGetLastError();
}

hipError_t launch_expert_gate_up(uint32_t dtype, const ExpertRows &p, hipStream_t stream) {
  return rows_ok(dtype, p) ? launch<kExpertGateUp>(p, stream) : hipErrorInvalidValue;
}
hipError_t launch_expert_down(uint32_t dtype, const ExpertRows &p, hipStream_t stream) {
  return rows_ok(dtype, p) && p.out != nullptr ? launch<kExpertDown>(p, stream) : hipErrorInvalidValue;
}

}  // namespace nv
