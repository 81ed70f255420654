// Decode-step projections of a parallel layer (see gemv_layer.cuh).
#include "gemv_layer.cuh"

#include <algorithm>

#include "activations.cuh"
#include "gemv_stream.cuh"
#include "moe_rows.cuh"

namespace nv {

namespace {

constexpr int kWaves = 8, kThreads = kWaves * kWave;
constexpr uint32_t kChunk = kWave * 8;       // columns of a load instruction
constexpr uint32_t kMaxWorkgroups = 512;     // two a CU
constexpr size_t kMaxLds = 56 * 1024;
__host__ __device__ __forceinline__ uint32_t padded(uint32_t cols) { return (cols + kChunk - 1) / kChunk * kChunk; }

// Zeros behind a staged vector, up to a whole chunk (the weights there are taken as zero as well).
__device__ __forceinline__ void clear_tail(uint16_t *xs, uint32_t cols) {
  for (uint32_t c = cols + threadIdx.x; c < padded(cols); c += kThreads) xs[c] = 0;
}

// round16(x * rsqrt(mean(x^2) + eps) * gamma) of a row, for one or two gammas. cols % 8 == 0.
template <uint32_t DT>
__device__ __forceinline__ void rms_stage(const float *x, uint32_t cols, float eps, const uint16_t *g0, uint16_t *xs0, const uint16_t *g1,
                                          uint16_t *xs1, float *red) {
  float ss = 0.0f;
  for (uint32_t c = threadIdx.x * 8u; c < cols; c += kThreads * 8u) {
    const float4 a = *reinterpret_cast<const float4 *>(x + c), b = *reinterpret_cast<const float4 *>(x + c + 4);
    ss += a.x * a.x + a.y * a.y + a.z * a.z + a.w * a.w + b.x * b.x + b.y * b.y + b.z * b.z + b.w * b.w;
  }
  const float scale = 1.0f / sqrtf(block_sum_n<kWaves>(ss, red) / static_cast<float>(cols) + eps);
  for (uint32_t c = threadIdx.x * 8u; c < cols; c += kThreads * 8u) {
    const float4 a = *reinterpret_cast<const float4 *>(x + c), b = *reinterpret_cast<const float4 *>(x + c + 4);
    const float v[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
    const auto put = [&](const uint16_t *gamma, uint16_t *xs) {
      const uint4 g = *reinterpret_cast<const uint4 *>(gamma + c);
      float w[8];
      unpack8<DT>(g, w);
      uint32_t o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e)
        o[e] = enc16<DT>(v[2 * e] * scale * w[2 * e]) | (static_cast<uint32_t>(enc16<DT>(v[2 * e + 1] * scale * w[2 * e + 1])) << 16);
      *reinterpret_cast<uint4 *>(xs + c) = make_uint4(o[0], o[1], o[2], o[3]);
    };
    put(g0, xs0);
    if (g1 != nullptr) put(g1, xs1);
  }
  clear_tail(xs0, cols);
  if (g1 != nullptr) clear_tail(xs1, cols);
}

// ---- front, middle ---------------------------------------------------------------------------

// Two rows of weights that a wave walks together, and what becomes of their sums.
struct Unit {
  const uint16_t *w0, *w1;
  uint32_t at;             // the staged input's place in LDS
  uint32_t cols;
  float *out0, *out1;      // plain rows (out1 null: there is no second one)
  uint16_t *act;           // gate and up row: one activation
  float limit;
};

constexpr int kBatch = 4;   // chunks of a request batch: 4 KiB of each row

// A wave's walk over its units first, first + stride, .. < units; unit_at(i) -> Unit (i is wave-uniform). The first two
// batches of weights are requested by start(), which does not need the staged inputs.
template <uint32_t DT, typename At>
struct PairWalk {
  At unit_at;
  uint32_t units, stride, lane;
  uint4 b0[2][kBatch], b1[2][kBatch];
  uint32_t iu, ic;      // next batch to request: unit, first column
  Unit in;
  uint32_t cu, cc;      // next batch to multiply
  Unit cur;
  float acc0, acc1;

  __device__ __forceinline__ PairWalk(At at, uint32_t n, uint32_t first, uint32_t step)
      : unit_at(at), units(n), stride(step), lane(threadIdx.x & (kWave - 1)), iu(first), ic(0), in{}, cu(first), cc(0), cur{}, acc0(0.0f), acc1(0.0f) {}
  __device__ __forceinline__ void issue(uint4 (&to)[2][kBatch]) {
    if (iu >= units) return;
#pragma unroll
    for (int u = 0; u < kBatch; ++u) {
      const uint32_t c = ic + u * kChunk + lane * 8u;
      const bool on = c < in.cols;
      to[0][u] = on ? load_stream(in.w0 + c) : make_uint4(0u, 0u, 0u, 0u);
      to[1][u] = on ? load_stream(in.w1 + c) : make_uint4(0u, 0u, 0u, 0u);
    }
    ic += kBatch * kChunk;
    if (ic >= in.cols) {
      ic = 0;
      iu += stride;
      if (iu < units) in = unit_at(iu);
    }
  }
  __device__ __forceinline__ void consume(const uint4 (&from)[2][kBatch], const uint16_t *xs) {
#pragma unroll
    for (int u = 0; u < kBatch; ++u) {
      if (cc + u * kChunk < cur.cols) {
        const uint4 x = *reinterpret_cast<const uint4 *>(xs + cur.at + cc + u * kChunk + lane * 8u);
        acc0 = dot8<DT, true>(from[0][u], x, acc0);
        acc1 = dot8<DT, true>(from[1][u], x, acc1);
      }
    }
    cc += kBatch * kChunk;
    if (cc < cur.cols) return;
    acc0 = wave_sum(acc0);
    acc1 = wave_sum(acc1);
    if (lane == 0) {
      if (cur.act != nullptr) {
        *cur.act = enc16<DT>(clamped_glu(acc0, acc1, cur.limit));
      } else {
        *cur.out0 = acc0;
        if (cur.out1 != nullptr) *cur.out1 = acc1;
      }
    }
    acc0 = acc1 = 0.0f;
    cc = 0;
    cu += stride;
    if (cu < units) cur = unit_at(cu);
  }
  __device__ __forceinline__ void start() {
    if (iu < units) in = cur = unit_at(iu);
    issue(b0);
    issue(b1);
  }
  __device__ __forceinline__ void run(const uint16_t *xs) {
    while (cu < units) {
      consume(b0, xs);
      issue(b0);
      if (cu >= units) break;
      consume(b1, xs);
      issue(b1);
    }
  }
};

__device__ __forceinline__ Unit two_rows(const uint16_t *w, uint32_t cols, uint32_t rows, uint32_t i, uint32_t at, float *out) {
  const uint32_t r0 = 2u * i, r1 = min(r0 + 1u, rows - 1u);
  return Unit{w + static_cast<uint64_t>(r0) * cols, w + static_cast<uint64_t>(r1) * cols, at, cols, out + r0, r0 + 1u < rows ? out + r1 : nullptr,
              nullptr, 0.0f};
}
__device__ __forceinline__ Unit gate_and_up(const uint16_t *w, uint32_t cols, uint32_t ff, uint32_t i, uint32_t at, uint16_t *act, float limit) {
  return Unit{w + static_cast<uint64_t>(i) * cols, w + static_cast<uint64_t>(ff + i) * cols, at, cols, nullptr, nullptr, act + i, limit};
}

template <uint32_t DT>
__global__ __launch_bounds__(kThreads, 4) void layer_front_kernel(LayerFront p) {
  extern __shared__ __align__(16) uint16_t xs[];   // the mixer's row, the feed-forward's
  __shared__ float red[kWaves];
  const uint32_t wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const uint32_t n_in = (p.in_rows + 1) / 2, n_router = (p.experts + 1) / 2, units = n_in + n_router + p.shared_ff;
  const auto unit_at = [&](uint32_t i) {
    if (i < n_router) return two_rows(p.router, p.hidden, p.experts, i, padded(p.hidden), p.logits);
    i -= n_router;
    if (i < n_in) return two_rows(p.w_in, p.hidden, p.in_rows, i, 0u, p.in);
    return gate_and_up(p.shared_in, p.hidden, p.shared_ff, i - n_in, padded(p.hidden), p.shared_act, p.shared_limit);
  };
  // (consecutive units go to different workgroups)
  PairWalk<DT, decltype(unit_at)> walk(unit_at, units, wave * gridDim.x + blockIdx.x, gridDim.x * kWaves);
  walk.start();
  if (*p.cursor >= p.max_steps) return;   // (after the requests, which do not depend on it)
  uint16_t *xs2 = xs + padded(p.hidden);
  rms_stage<DT>(p.x, p.hidden, p.eps, p.mixer_norm, xs, p.ff_norm, xs2, red);
  __syncthreads();
  if (p.ff_norm != nullptr && blockIdx.x == 0)
    for (uint32_t c = threadIdx.x * 8u; c < p.hidden; c += kThreads * 8u) *reinterpret_cast<uint4 *>(p.h16 + c) = *reinterpret_cast<const uint4 *>(xs2 + c);
  walk.run(xs);
}

template <uint32_t DT>
__global__ __launch_bounds__(kThreads, 4) void layer_middle_kernel(LayerMiddle p) {
  extern __shared__ __align__(16) uint16_t xs[];   // the query latent, the feed-forward's row
  __shared__ float red[kWaves];
  __shared__ float score[kMaxExperts];
  __shared__ uint32_t id_s[kMaxTop];
  __shared__ float s_s[kMaxTop];
  if (*p.cursor >= p.max_steps) return;
  uint16_t *xs2 = xs + padded(p.q_rank);
  const uint32_t tid = threadIdx.x;
  for (uint32_t e = tid; e < p.experts; e += kThreads) score[e] = 1.0f / (1.0f + expf(-p.logits[e]));
  if (tid < kMaxTop) {   // (scores that are no numbers choose nothing: some expert that exists)
    id_s[tid] = 0u;
    s_s[tid] = 0.0f;
  }
  __syncthreads();
  // an expert's place is the number of experts ahead of it
  for (uint32_t e = tid; e < p.experts; e += kThreads) {
    const float s = score[e];
    uint32_t ahead = 0;
#pragma unroll 8
    for (uint32_t j = 0; j < p.experts; ++j) ahead += score[j] > s || (score[j] == s && j < e) ? 1u : 0u;
    if (ahead < p.top) {
      id_s[ahead] = e;
      s_s[ahead] = s;
    }
  }
  __syncthreads();
  const uint32_t wave = __builtin_amdgcn_readfirstlane(tid / kWave);
  const uint32_t n_experts = p.experts != 0 ? p.top * p.ff : 0u, units = n_experts + (p.q_rows + 1) / 2;
  const auto unit_at = [&](uint32_t i) {
    if (i >= n_experts) return two_rows(p.w_uq, p.q_rank, p.q_rows, i - n_experts, 0u, p.q);
    const uint32_t k = i / p.ff, e = __builtin_amdgcn_readfirstlane(id_s[k]);
    return gate_and_up(p.e_in + static_cast<uint64_t>(e) * 2u * p.ff * p.hidden, p.hidden, p.ff, i - k * p.ff, padded(p.q_rank), p.act + k * p.ff,
                       p.limit);
  };
  PairWalk<DT, decltype(unit_at)> walk(unit_at, units, wave * gridDim.x + blockIdx.x, gridDim.x * kWaves);
  walk.start();
  if (p.experts != 0) {
    for (uint32_t c = tid * 8u; c < p.hidden; c += kThreads * 8u) *reinterpret_cast<uint4 *>(xs2 + c) = *reinterpret_cast<const uint4 *>(p.h16 + c);
    clear_tail(xs2, p.hidden);
    if (blockIdx.x == 0 && tid < p.top) {
      float sum = 0.0f;
      for (uint32_t k = 0; k < p.top; ++k) sum += s_s[k];
      p.ids[tid] = id_s[tid];
      p.weights[tid] = s_s[tid] / (sum + 1e-20f);
    }
  }
  rms_stage<DT>(p.latent, p.q_rank, p.eps, p.latent_norm, xs, nullptr, nullptr, red);
  __syncthreads();
  walk.run(xs);
}

// ---- back ------------------------------------------------------------------------------------

// A row's columns are the pieces' columns one after the other, each piece padded to whole chunks, as their inputs lie in
// LDS. A chunk: where it starts in row 0, bytes from row to row, lanes that have columns, what its products are worth.
struct Chunk {
  uint64_t base;
  uint16_t stride, lanes;
  float factor;
};
static_assert(sizeof(Chunk) == 16, "one LDS read");
constexpr uint32_t kMaxChunks = kMaxLds / (2 * kChunk);
constexpr int kBackBatch = 8;   // chunks of a request batch

template <uint32_t DT>
__global__ __launch_bounds__(kThreads, 4) void layer_back_kernel(LayerBack p) {
  extern __shared__ __align__(16) uint16_t xs[];   // the pieces' inputs
  __shared__ __align__(16) Chunk table[kMaxChunks + kBackBatch];
  if (*p.cursor >= p.max_steps) return;
  const uint32_t tid = threadIdx.x, lane = tid & (kWave - 1), wave = __builtin_amdgcn_readfirstlane(tid / kWave);
  const uint32_t expert_at = padded(p.mix_cols), shared_at = expert_at + p.top * padded(p.ff);
  const uint32_t chunks = (shared_at + padded(p.shared_ff)) / kChunk, batches = (chunks + kBackBatch - 1) / kBackBatch;
  if (tid < batches * kBackBatch) {
    const uint32_t at = tid * kChunk;
    const uint16_t *base = p.w_o;
    uint32_t cols = p.mix_cols, c = at;
    float factor = 1.0f;
    if (at >= shared_at) {
      base = p.shared_out;
      cols = p.shared_ff;
      c = at - shared_at;
    } else if (at >= expert_at) {
      const uint32_t k = (at - expert_at) / padded(p.ff);
      base = p.e_out + static_cast<uint64_t>(p.ids[k]) * p.hidden * p.ff;
      cols = p.ff;
      c = at - expert_at - k * padded(p.ff);
      factor = p.weights[k];
    }
    const uint32_t lanes = tid < chunks ? min((cols - c) / 8u, static_cast<uint32_t>(kWave)) : 0u;   // (the last batch's chunks past the end)
    table[tid] = Chunk{reinterpret_cast<uint64_t>(base) + 2u * (lanes != 0 ? c : 0u), static_cast<uint16_t>(2u * cols), static_cast<uint16_t>(lanes), factor};
  }
  __syncthreads();
  const uint32_t stride = gridDim.x * kWaves;
  uint4 b0[kBackBatch], b1[kBackBatch];
  uint32_t irow = wave * gridDim.x + blockIdx.x, ib = 0, crow = irow, cb = 0;
  float total = 0.0f;
  const auto issue = [&](uint4 (&to)[kBackBatch]) {
    if (irow >= p.hidden) return;
#pragma unroll
    for (int u = 0; u < kBackBatch; ++u) {
      const Chunk k = table[ib * kBackBatch + u];
      to[u] = make_uint4(0u, 0u, 0u, 0u);
      if (lane < k.lanes) to[u] = load_stream(reinterpret_cast<const char *>(k.base) + static_cast<uint64_t>(irow) * k.stride + lane * 16u);
    }
    if (++ib == batches) {
      ib = 0;
      irow += stride;
    }
  };
  const auto consume = [&](const uint4 (&from)[kBackBatch]) {
#pragma unroll
    for (int u = 0; u < kBackBatch; ++u) {
      const uint32_t i = cb * kBackBatch + u;
      if (i < chunks) total = fmaf(table[i].factor, dot8<DT, true>(from[u], *reinterpret_cast<const uint4 *>(xs + i * kChunk + lane * 8u), 0.0f), total);
    }
    if (++cb < batches) return;
    total = wave_sum(total);
    if (lane == 0) p.x[crow] += total;
    total = 0.0f;
    cb = 0;
    crow += stride;
  };
  issue(b0);
  issue(b1);
  // the inputs, under the first requests
  const auto stage = [&](const uint16_t *src, uint32_t cols, uint32_t at) {
    for (uint32_t c = tid * 8u; c < cols; c += kThreads * 8u) *reinterpret_cast<uint4 *>(xs + at + c) = *reinterpret_cast<const uint4 *>(src + c);
    clear_tail(xs + at, cols);
  };
  stage(p.mixed, p.mix_cols, 0);
  for (uint32_t k = 0; k < p.top; ++k) stage(p.act + k * p.ff, p.ff, expert_at + k * padded(p.ff));
  if (p.shared_ff != 0) stage(p.shared_act, p.shared_ff, shared_at);
  __syncthreads();
  while (crow < p.hidden) {
    consume(b0);
    issue(b0);
    if (crow >= p.hidden) break;
    consume(b1);
    issue(b1);
  }
}

uint32_t workgroups(uint32_t units) { return std::max(1u, std::min(kMaxWorkgroups, (units + kWaves - 1) / kWaves)); }
size_t back_columns(uint32_t mix_cols, uint32_t top, uint32_t ff, uint32_t shared_ff) {
  return static_cast<size_t>(padded(mix_cols)) + static_cast<size_t>(top) * padded(ff) + padded(shared_ff);
}
bool whole(const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15u) == 0; }

}  // namespace

bool layer_gemv_takes(uint32_t hidden, uint32_t q_rank, uint32_t mix_cols, uint32_t experts, uint32_t top, uint32_t ff, uint32_t shared_ff) {
  return hidden % 8 == 0 && q_rank % 8 == 0 && mix_cols % 8 == 0 && ff % 8 == 0 && shared_ff % 8 == 0 && experts <= kMaxExperts && top <= kMaxTop &&
         2u * 2u * padded(hidden) <= kMaxLds && 2u * (padded(q_rank) + padded(hidden)) <= kMaxLds && 2u * back_columns(mix_cols, top, ff, shared_ff) <= kMaxLds;
}

hipError_t launch_layer_front(uint32_t dtype, const LayerFront &p, hipStream_t stream) {
  const bool ff = p.ff_norm != nullptr;
  if (dtype != kBF16 || p.x == nullptr || p.mixer_norm == nullptr || p.w_in == nullptr || p.in == nullptr || p.in_rows == 0 || p.cursor == nullptr ||
      p.hidden == 0 || !layer_gemv_takes(p.hidden, 8, 8, p.experts, 0, 0, p.shared_ff) || (!ff && (p.experts != 0 || p.shared_ff != 0)) ||
      (ff && p.h16 == nullptr) || (p.experts != 0 && (p.router == nullptr || p.logits == nullptr)) ||
      (p.shared_ff != 0 && (p.shared_in == nullptr || p.shared_act == nullptr)) || !whole(p.x) || !whole(p.w_in) || !whole(p.router) ||
      !whole(p.shared_in) || !whole(p.mixer_norm) || !whole(p.ff_norm) || !whole(p.h16))
    return hipErrorInvalidValue;
  const uint32_t units = (p.in_rows + 1) / 2 + (p.experts + 1) / 2 + p.shared_ff;
  hipLaunchKernelGGL(layer_front_kernel<kBF16>, dim3(workgroups(units)), dim3(kThreads), 2u * 2u * padded(p.hidden), stream, p);
  return hipGetLastError();
}

hipError_t launch_layer_middle(uint32_t dtype, const LayerMiddle &p, hipStream_t stream) {
  if (dtype != kBF16 || p.latent == nullptr || p.latent_norm == nullptr || p.w_uq == nullptr || p.q == nullptr || p.q_rows == 0 || p.q_rank == 0 ||
      p.cursor == nullptr || !layer_gemv_takes(p.experts != 0 ? p.hidden : 8, p.q_rank, 8, p.experts, 0, p.experts != 0 ? p.ff : 0, 0) ||
      (p.experts != 0 && (p.h16 == nullptr || p.logits == nullptr || p.top == 0 || p.top > p.experts || p.top > kMaxTop || p.e_in == nullptr ||
                          p.ff == 0 || p.act == nullptr || p.ids == nullptr || p.weights == nullptr)) ||
      !whole(p.latent) || !whole(p.latent_norm) || !whole(p.w_uq) || !whole(p.h16) || !whole(p.e_in))
    return hipErrorInvalidValue;
  const uint32_t units = (p.q_rows + 1) / 2 + (p.experts != 0 ? p.top * p.ff : 0u);
  const size_t lds = 2u * (padded(p.q_rank) + (p.experts != 0 ? padded(p.hidden) : 0u));
  hipLaunchKernelGGL(layer_middle_kernel<kBF16>, dim3(workgroups(units)), dim3(kThreads), lds, stream, p);
  return hipGetLastError();
}

hipError_t launch_layer_back(uint32_t dtype, const LayerBack &p, hipStream_t stream) {
  if (dtype != kBF16 || p.x == nullptr || p.w_o == nullptr || p.mixed == nullptr || p.hidden == 0 || p.mix_cols == 0 || p.cursor == nullptr ||
      !layer_gemv_takes(8, 8, p.mix_cols, 0, p.top, p.top != 0 ? p.ff : 0, p.shared_ff) ||
      (p.top != 0 && (p.e_out == nullptr || p.act == nullptr || p.ids == nullptr || p.weights == nullptr || p.ff == 0)) ||
      (p.shared_ff != 0 && (p.shared_out == nullptr || p.shared_act == nullptr)) || !whole(p.w_o) || !whole(p.mixed) || !whole(p.e_out) ||
      !whole(p.act) || !whole(p.shared_out) || !whole(p.shared_act))
    return hipErrorInvalidValue;
  hipLaunchKernelGGL(layer_back_kernel<kBF16>, dim3(workgroups(p.hidden)), dim3(kThreads), 2u * back_columns(p.mix_cols, p.top, p.ff, p.shared_ff), stream, p);
  return hipGetLastError();
}

}  // namespace nv
