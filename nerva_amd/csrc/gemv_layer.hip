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

// A run of a row's columns: weights at base + row * stride, `cols` of them meet the staged inputs from `at` on.
struct Run {
  const uint16_t *base;
  uint32_t stride, cols, at;
  float factor;
};
constexpr uint32_t kMaxRuns = kMaxTop + 2;
constexpr int kBackBatch = 8;   // chunks of a request batch

template <uint32_t DT>
__global__ __launch_bounds__(kThreads, 4) void layer_back_kernel(LayerBack p) {
  extern __shared__ __align__(16) uint16_t xs[];   // the runs' inputs, each padded to whole chunks
  __shared__ Run runs[kMaxRuns];
  if (*p.cursor >= p.max_steps) return;
  const uint32_t tid = threadIdx.x, lane = tid & (kWave - 1), wave = __builtin_amdgcn_readfirstlane(tid / kWave);
  const uint32_t n_runs = 1u + p.top + (p.shared_ff != 0 ? 1u : 0u);
  const uint32_t expert_at = padded(p.mix_cols), shared_at = expert_at + p.top * padded(p.ff);
  if (tid < n_runs) {
    if (tid == 0) runs[tid] = Run{p.w_o, p.mix_cols, p.mix_cols, 0u, 1.0f};
    else if (tid <= p.top)
      runs[tid] = Run{p.e_out + static_cast<uint64_t>(p.ids[tid - 1]) * p.hidden * p.ff, p.ff, p.ff, expert_at + (tid - 1) * padded(p.ff), p.weights[tid - 1]};
    else runs[tid] = Run{p.shared_out, p.shared_ff, p.shared_ff, shared_at, 1.0f};
  }
  __syncthreads();
  const uint32_t chunks = (shared_at + padded(p.shared_ff)) / kChunk;
  // The row's chunks lie one after the other as their inputs do. Cursors over them (wave-uniform): run, column in it.
  struct Cursor {
    const uint16_t *base;
    uint32_t run, c, cols;
    float factor;
  };
  const auto open = [&](Cursor &k, uint32_t run, uint32_t row) {
    const Run &r = runs[run];
    const uint64_t base = reinterpret_cast<uint64_t>(r.base) + static_cast<uint64_t>(row) * r.stride * 2u;
    // (the builtin returns a signed word: narrowed again before it is widened to an address)
    const uint32_t low = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(base)), high = __builtin_amdgcn_readfirstlane(static_cast<uint32_t>(base >> 32));
    k.base = reinterpret_cast<const uint16_t *>(static_cast<uint64_t>(low) | static_cast<uint64_t>(high) << 32);
    k.run = run;
    k.c = 0;
    k.cols = __builtin_amdgcn_readfirstlane(r.cols);
    k.factor = r.factor;
  };
  const uint32_t stride = gridDim.x * kWaves, batches = (chunks + kBackBatch - 1) / kBackBatch;
  uint4 b0[kBackBatch], b1[kBackBatch];
  uint32_t irow = wave * gridDim.x + blockIdx.x, ib = 0, crow = irow, cb = 0;
  Cursor in{}, cur{};
  if (irow < p.hidden) {
    open(in, 0, irow);
    open(cur, 0, irow);
  }
  float acc = 0.0f, total = 0.0f;
  const auto next = [&](Cursor &k, uint32_t row) {   // one chunk further
    k.c += kChunk;
    if (k.c >= k.cols && k.run + 1 < n_runs) open(k, k.run + 1, row);
  };
#define NV_BACK_ISSUE(DST)                                                                           \
  if (irow < p.hidden) {                                                                            \
    _Pragma("unroll") for (int u = 0; u < kBackBatch; ++u) {                                        \
      const uint32_t c = in.c + lane * 8u;                                                          \
      DST[u] = ib * kBackBatch + u < chunks && c < in.cols ? load_stream(in.base + c) : make_uint4(0u, 0u, 0u, 0u); \
      if (ib * kBackBatch + u + 1 < chunks) next(in, irow);                                         \
    }                                                                                               \
    if (++ib == batches) {                                                                          \
      ib = 0;                                                                                       \
      irow += stride;                                                                               \
      if (irow < p.hidden) open(in, 0, irow);                                                       \
    }                                                                                               \
  }
#define NV_BACK_CONSUME(SRC)                                                                         \
  _Pragma("unroll") for (int u = 0; u < kBackBatch; ++u) {                                          \
    if (cb * kBackBatch + u < chunks) {                                                             \
      const uint4 x = *reinterpret_cast<const uint4 *>(xs + (cb * kBackBatch + u) * kChunk + lane * 8u); \
      acc = dot8<DT, true>(SRC[u], x, acc);                                                         \
      if (cur.c + kChunk >= cur.cols) {                                                             \
        total = fmaf(cur.factor, acc, total);                                                       \
        acc = 0.0f;                                                                                 \
      }                                                                                             \
      if (cb * kBackBatch + u + 1 < chunks) next(cur, crow);                                        \
    }                                                                                               \
  }                                                                                                 \
  if (++cb == batches) {                                                                            \
    total = wave_sum(total);                                                                        \
    if (lane == 0) p.x[crow] += total;                                                              \
    total = 0.0f;                                                                                   \
    cb = 0;                                                                                         \
    crow += stride;                                                                                 \
    if (crow < p.hidden) open(cur, 0, crow);                                                        \
  }
  NV_BACK_ISSUE(b0)
  NV_BACK_ISSUE(b1)
  const auto stage = [&](const uint16_t *src, uint32_t cols, uint32_t at) {
    for (uint32_t c = tid * 8u; c < cols; c += kThreads * 8u) *reinterpret_cast<uint4 *>(xs + at + c) = *reinterpret_cast<const uint4 *>(src + c);
    clear_tail(xs + at, cols);
  };
  stage(p.mixed, p.mix_cols, 0);
  for (uint32_t k = 0; k < p.top; ++k) stage(p.act + k * p.ff, p.ff, expert_at + k * padded(p.ff));
  if (p.shared_ff != 0) stage(p.shared_act, p.shared_ff, shared_at);
  __syncthreads();
  while (crow < p.hidden) {
    NV_BACK_CONSUME(b0)
    NV_BACK_ISSUE(b0)
    if (crow >= p.hidden) break;
    NV_BACK_CONSUME(b1)
    NV_BACK_ISSUE(b1)
  }
#undef NV_BACK_ISSUE
#undef NV_BACK_CONSUME
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
