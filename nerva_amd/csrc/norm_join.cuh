// The seam between two sublayers of a stack that normalises before AND after each of them:
//   x' = x + N_post(y)      y: what the sublayer that just ended put out
//   h  = N_pre(x')          what the next projection multiplies
// with N the layer norm (centre, divide by sqrt(mean squared deviation + eps), scale, shift), everything f32 until h.
// A decode step runs it as the prologue of the projection that reads h: every workgroup computes the whole row for
// itself (two f32 rows from L2) and one of them stores x', into another buffer than x since the others still read x.
// Blocks of token rows run it as a launch of its own, one workgroup per row (norm_join.hip).
//
// A row's mean and squared deviation come from one exchange through LDS: every wave reduces its own values around
// its own mean, and the waves' (count, mean, squared deviation) are then combined exactly as for the whole row.
#pragma once

#include "nv_common.cuh"

namespace nv {

struct JoinNorm {
  const float *x;                      // residual row
  const float *y;                      // optional: without it x' = x
  const uint16_t *post_w, *post_b;     // N_post
  const uint16_t *pre_w, *pre_b;       // N_pre (null where only x' is wanted)
  float *x_out;                        // optional: x'
  float eps;
};

// Mean and 1 / sqrt(mean squared deviation + eps) of `cols` values spread over WG waves, N per lane; in(i) says
// whether the lane's i-th value exists. `scratch`: 3 * WG floats of LDS.
template <int WG, int N, typename In>
__device__ __forceinline__ void row_moments(const float (&v)[N], In in, uint32_t cols, float eps, float *scratch, float &mean,
                                            float &rstd) {
  const int wave = threadIdx.x / kWave;
  float count = 0.0f, sum = 0.0f;
#pragma unroll
  for (int i = 0; i < N; ++i) {
    count += in(i) ? 1.0f : 0.0f;
    sum += in(i) ? v[i] : 0.0f;
  }
  count = wave_sum(count);
  const float wmean = count > 0.0f ? wave_sum(sum) / count : 0.0f;
  float dev = 0.0f;
#pragma unroll
  for (int i = 0; i < N; ++i) {
    const float d = in(i) ? v[i] - wmean : 0.0f;
    dev = fmaf(d, d, dev);
  }
  dev = wave_sum(dev);
  __syncthreads();
  if ((threadIdx.x & (kWave - 1)) == 0) {
    scratch[wave * 3] = count;
    scratch[wave * 3 + 1] = wmean;
    scratch[wave * 3 + 2] = dev;
  }
  __syncthreads();
  float total = 0.0f;
#pragma unroll
  for (int w = 0; w < WG; ++w) total = fmaf(scratch[w * 3], scratch[w * 3 + 1], total);
  mean = total / static_cast<float>(cols);
  float square = 0.0f;
#pragma unroll
  for (int w = 0; w < WG; ++w) {
    const float d = scratch[w * 3 + 1] - mean;
    square += scratch[w * 3 + 2] + scratch[w * 3] * d * d;
  }
  rstd = 1.0f / sqrtf(square / static_cast<float>(cols) + eps);
}

constexpr uint32_t kJoinPerLane = 16;   // values a lane keeps in registers between the two norms
// Any width: emit(c, h) for every column. Rows of more than kJoinPerLane values a lane are walked again for each of
// the passes instead (x' is recomputed; it may not be stored before the last read of x, so x_out must not alias x).
template <uint32_t DT, int WG, typename Emit>
__device__ __forceinline__ void join_norm_row(const JoinNorm &j, uint32_t cols, bool store, float *scratch, Emit emit) {
  constexpr uint32_t TB = WG * kWave;
  const uint32_t groups = (cols + TB * kJoinPerLane - 1) / (TB * kJoinPerLane);
  if (groups <= 1) {
    const auto in = [&](int i) { return static_cast<uint32_t>(i) * TB + threadIdx.x < cols; };
    float v[kJoinPerLane];
    float mean, rstd;
#pragma unroll
    for (int i = 0; i < static_cast<int>(kJoinPerLane); ++i) {
      const uint32_t c = static_cast<uint32_t>(i) * TB + threadIdx.x;
      v[i] = c < cols ? (j.y != nullptr ? j.y[c] : j.x[c]) : 0.0f;
    }
    if (j.y != nullptr) {
      row_moments<WG>(v, in, cols, j.eps, scratch, mean, rstd);
#pragma unroll
      for (int i = 0; i < static_cast<int>(kJoinPerLane); ++i) {
        const uint32_t c = static_cast<uint32_t>(i) * TB + threadIdx.x;
        if (c < cols) v[i] = j.x[c] + ((v[i] - mean) * rstd * dec16<DT>(j.post_w[c]) + dec16<DT>(j.post_b[c]));
      }
    }
    if (store && j.x_out != nullptr) {
#pragma unroll
      for (int i = 0; i < static_cast<int>(kJoinPerLane); ++i) {
        const uint32_t c = static_cast<uint32_t>(i) * TB + threadIdx.x;
        if (c < cols) j.x_out[c] = v[i];
      }
    }
    if (j.pre_w == nullptr) return;
    row_moments<WG>(v, in, cols, j.eps, scratch, mean, rstd);
#pragma unroll
    for (int i = 0; i < static_cast<int>(kJoinPerLane); ++i) {
      const uint32_t c = static_cast<uint32_t>(i) * TB + threadIdx.x;
      if (c < cols) emit(c, (v[i] - mean) * rstd * dec16<DT>(j.pre_w[c]) + dec16<DT>(j.pre_b[c]));
    }
    return;
  }
  // wide rows: one value a lane at a time, four walks
  const auto walk = [&](auto value, float &mean, float &rstd) {
    float sum = 0.0f;
    for (uint32_t c = threadIdx.x; c < cols; c += TB) sum += value(c);
    float one[1] = {sum};
    float dummy;
    // mean of the lanes' sums times lanes / cols is the row's mean
    row_moments<WG>(one, [](int) { return true; }, TB, 1.0f, scratch, mean, dummy);
    mean *= static_cast<float>(TB) / static_cast<float>(cols);
    float dev = 0.0f;
    for (uint32_t c = threadIdx.x; c < cols; c += TB) {
      const float d = value(c) - mean;
      dev = fmaf(d, d, dev);
    }
    one[0] = dev;
    float mean_dev;
    row_moments<WG>(one, [](int) { return true; }, TB, 1.0f, scratch, mean_dev, dummy);
    rstd = 1.0f / sqrtf(mean_dev * (static_cast<float>(TB) / static_cast<float>(cols)) + j.eps);
  };
  float ym = 0.0f, yr = 0.0f;
  if (j.y != nullptr) walk([&](uint32_t c) { return j.y[c]; }, ym, yr);
  const auto joined = [&](uint32_t c) {
    return j.y == nullptr ? j.x[c] : j.x[c] + ((j.y[c] - ym) * yr * dec16<DT>(j.post_w[c]) + dec16<DT>(j.post_b[c]));
  };
  if (j.pre_w != nullptr) {
    float mean, rstd;
    walk(joined, mean, rstd);
    for (uint32_t c = threadIdx.x; c < cols; c += TB)
      emit(c, (joined(c) - mean) * rstd * dec16<DT>(j.pre_w[c]) + dec16<DT>(j.pre_b[c]));
  }
  if (store && j.x_out != nullptr)
    for (uint32_t c = threadIdx.x; c < cols; c += TB) j.x_out[c] = joined(c);
}

// Eight consecutive columns of everything the seam reads, requested at once (the lean GEMV holds them across its first
// weight requests).
struct JoinRegs {
  float4 xa, xb, ya, yb;
  uint4 post_w, post_b, pre_w, pre_b;
};
__device__ __forceinline__ void join_load8(const JoinNorm &j, uint32_t c, uint32_t cols, JoinRegs &r) {
  if (c >= cols) return;
  r.xa = *reinterpret_cast<const float4 *>(j.x + c);
  r.xb = *reinterpret_cast<const float4 *>(j.x + c + 4);
  if (j.y != nullptr) {
    r.ya = *reinterpret_cast<const float4 *>(j.y + c);
    r.yb = *reinterpret_cast<const float4 *>(j.y + c + 4);
    r.post_w = *reinterpret_cast<const uint4 *>(j.post_w + c);
    r.post_b = *reinterpret_cast<const uint4 *>(j.post_b + c);
  }
  r.pre_w = *reinterpret_cast<const uint4 *>(j.pre_w + c);
  r.pre_b = *reinterpret_cast<const uint4 *>(j.pre_b + c);
}
template <uint32_t DT>
__device__ __forceinline__ void unpack8(const uint4 &w, float (&o)[8]) {
  unpack2<DT>(w.x, o[0], o[1]);
  unpack2<DT>(w.y, o[2], o[3]);
  unpack2<DT>(w.z, o[4], o[5]);
  unpack2<DT>(w.w, o[6], o[7]);
}
// cols % 8 == 0, cols <= WG * 64 * 8 * N: h into LDS as 16-bit values, x' to memory where `store`.
template <uint32_t DT, int WG, int N>
__device__ __forceinline__ void join_norm_regs(const JoinNorm &j, uint32_t cols, bool store, const JoinRegs (&r)[N], float *scratch,
                                               uint16_t *xs) {
  constexpr uint32_t TB = WG * kWave;
  const auto at = [&](int i) { return (static_cast<uint32_t>(i) * TB + threadIdx.x) * 8u; };
  const auto in = [&](int i) { return at(i / 8) < cols; };
  float v[8 * N];
  float mean, rstd;
  if (j.y != nullptr) {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const bool on = at(i) < cols;
      const float t[8] = {r[i].ya.x, r[i].ya.y, r[i].ya.z, r[i].ya.w, r[i].yb.x, r[i].yb.y, r[i].yb.z, r[i].yb.w};
#pragma unroll
      for (int e = 0; e < 8; ++e) v[8 * i + e] = on ? t[e] : 0.0f;
    }
    row_moments<WG>(v, in, cols, j.eps, scratch, mean, rstd);
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const bool on = at(i) < cols;
      float w[8], b[8];
      unpack8<DT>(r[i].post_w, w);
      unpack8<DT>(r[i].post_b, b);
      const float t[8] = {r[i].xa.x, r[i].xa.y, r[i].xa.z, r[i].xa.w, r[i].xb.x, r[i].xb.y, r[i].xb.z, r[i].xb.w};
#pragma unroll
      for (int e = 0; e < 8; ++e) v[8 * i + e] = on ? t[e] + ((v[8 * i + e] - mean) * rstd * w[e] + b[e]) : 0.0f;
    }
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const bool on = at(i) < cols;
      const float t[8] = {r[i].xa.x, r[i].xa.y, r[i].xa.z, r[i].xa.w, r[i].xb.x, r[i].xb.y, r[i].xb.z, r[i].xb.w};
#pragma unroll
      for (int e = 0; e < 8; ++e) v[8 * i + e] = on ? t[e] : 0.0f;
    }
  }
  if (store && j.x_out != nullptr) {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      if (at(i) < cols) {
        *reinterpret_cast<float4 *>(j.x_out + at(i)) = make_float4(v[8 * i], v[8 * i + 1], v[8 * i + 2], v[8 * i + 3]);
        *reinterpret_cast<float4 *>(j.x_out + at(i) + 4) = make_float4(v[8 * i + 4], v[8 * i + 5], v[8 * i + 6], v[8 * i + 7]);
      }
    }
  }
  row_moments<WG>(v, in, cols, j.eps, scratch, mean, rstd);
#pragma unroll
  for (int i = 0; i < N; ++i) {
    if (at(i) < cols) {
      float w[8], b[8];
      unpack8<DT>(r[i].pre_w, w);
      unpack8<DT>(r[i].pre_b, b);
      uint32_t o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float lo = (v[8 * i + 2 * e] - mean) * rstd * w[2 * e] + b[2 * e];
        const float hi = (v[8 * i + 2 * e + 1] - mean) * rstd * w[2 * e + 1] + b[2 * e + 1];
        o[e] = enc16<DT>(lo) | (static_cast<uint32_t>(enc16<DT>(hi)) << 16);
      }
      *reinterpret_cast<uint4 *>(xs + at(i)) = make_uint4(o[0], o[1], o[2], o[3]);
    }
  }
}

// ---- token rows (norm_join.hip) --------------------------------------------------------------
// The seam for `tokens` rows: x' replaces x in place (each row belongs to one workgroup), h as 16-bit rows, as 16-bit
// values in matrix-operand order, or as f32 rows.
struct JoinRows {
  float *x;                            // [tokens][cols]
  const float *y;                      // optional [tokens][cols]
  const uint16_t *post_w, *post_b, *pre_w, *pre_b;   // pre null: only x'
  const uint32_t *pick;                // optional: output row i is source row pick[i], and x stays as it is
  uint16_t *out16;                     // one of out16 / out32, where pre is given
  float *out32;
  uint32_t packed_tiles;               // out16: != 0 -> operand order with that many token tiles
  uint32_t tokens, cols;
  float eps;
};
hipError_t launch_join_rows(uint32_t dtype, const JoinRows &p, hipStream_t stream);

}  // namespace nv
