// Weights from the caller's descriptors, for every kind of session.
#pragma once

#include <stdio.h>

#include <algorithm>
#include <string>
#include <vector>

#include "runtime_state.hpp"

namespace nv {

// ---- weights from the caller's plan -----------------------------------------------------------
// A declared weight plan (weights.cu:157-160) comes with descriptors that tile the weight bytes
// [0, resident_weight_bytes) in the reference's arena order - embeddings, then per layer rms_attn,
// w_q, [q_norm], w_k, [k_norm], w_v, w_o, rms_mlp, w_gate, w_up, w_down, [q/k/v/o bias], then the
// final norm and the LM head (weights.cu:484-591, session_api_lifecycle.inc.cu:124-148) - each with a
// host-memory or a file source. The descriptors are then THE source of the weights; the tensor
// pointers of the request only say which optional tensors exist (weights.cu:18-23) and may be null
// otherwise (weights.cu:237-243). This library keeps [q;k;v] and [gate;up] as row-concatenated
// matrices elsewhere in its own arena, so a descriptor's byte range is cut along the tensor
// boundaries of that order and every piece goes to its tensor's place.
constexpr uint32_t kWeightStrategyGpuResident = 1, kWeightStrategyGpuStaged = 2;  // weight_plan.rs:3-4

struct WeightSegment {
  uint64_t logical, bytes;  // position in the reference's arena order
  char *device;
};

template <typename Request>
bool weight_plan_declared(const Request *rq) {
  return rq->planned_weight_blocks != 0 || rq->planned_weight_bytes != 0;
}

inline void hash_le(uint64_t &hash, uint64_t value, int bytes) {
  for (int i = 0; i < bytes; ++i) {
    hash ^= (value >> (8 * i)) & 0xffu;
    hash *= 0x00000100000001b3ull;
  }
}

inline bool descriptor_has_file(const NervaHipHfDecodeSequenceWeightBlock &d) {
  return d.source_file != nullptr && d.source_file_len != 0;
}

// weights.cu:411-467: contiguous from 0, even offsets and sizes, a source each, a known strategy, and
// totals, counts and the FNV-1a hash over (block_id, block_version, offset_bytes, bytes, strategy)
// equal to what the plan declares.
template <typename Request>
bool validate_weight_descriptors(const Request *rq, uint64_t resident_weight_bytes) {
  uint64_t cursor = 0, hash = 0xcbf29ce484222325ull, resident_bytes = 0, staged_bytes = 0;
  uint32_t resident_blocks = 0, staged_blocks = 0;
  for (uint32_t i = 0; i < rq->planned_weight_descriptor_count; ++i) {
    const NervaHipHfDecodeSequenceWeightBlock &d = rq->planned_weight_descriptors[i];
    if (d.bytes == 0 || d.reserved != 0 || (d.host_source == nullptr && !descriptor_has_file(d)) ||
        d.offset_bytes != cursor || d.offset_bytes % 2 != 0 || d.bytes % 2 != 0)
      return false;
    if (cursor + d.bytes < cursor) return false;
    cursor += d.bytes;
    hash_le(hash, d.block_id, 8);
    hash_le(hash, d.block_version, 8);
    hash_le(hash, d.offset_bytes, 8);
    hash_le(hash, d.bytes, 8);
    hash_le(hash, d.strategy, 4);
    if (d.strategy == kWeightStrategyGpuResident) {
      resident_blocks += 1;
      resident_bytes += d.bytes;
    } else if (d.strategy == kWeightStrategyGpuStaged) {
      staged_blocks += 1;
      staged_bytes += d.bytes;
    } else {
      return false;
    }
  }
  return cursor == resident_weight_bytes && cursor == rq->planned_weight_bytes &&
         hash == rq->planned_weight_descriptor_hash && resident_blocks == rq->planned_gpu_resident_blocks &&
         staged_blocks == rq->planned_gpu_staged_blocks && resident_bytes == rq->planned_gpu_resident_weight_bytes &&
         staged_bytes == rq->planned_gpu_staged_weight_bytes;
}

// weights.cu:797-908: every descriptor to the device, from memory directly or from its file through a
// pinned staging buffer. `segments` is sorted and gapless in the reference's order.
template <typename Request>
hipError_t copy_weight_descriptors(const Request *rq, const std::vector<WeightSegment> &segments, hipStream_t stream, uint64_t *h2d_bytes,
                                   uint64_t *sync_calls) {
  constexpr uint64_t kStagingBytes = 64ull << 20;
  char *staging = nullptr;
  hipError_t err = hipSuccess;
  size_t at = 0;  // descriptors ascend, so the segment cursor only moves forward
  for (uint32_t i = 0; err == hipSuccess && i < rq->planned_weight_descriptor_count; ++i) {
    const NervaHipHfDecodeSequenceWeightBlock &d = rq->planned_weight_descriptors[i];
    FILE *file = nullptr;
    if (d.host_source == nullptr) {
      if (staging == nullptr) err = counted_host_malloc(reinterpret_cast<void **>(&staging), kStagingBytes);
      if (err != hipSuccess) break;
      const std::string path(d.source_file, d.source_file_len);
      file = fopen(path.c_str(), "rb");
      if (file == nullptr) {
        err = hipErrorInvalidValue;
        break;
      }
    }
    uint64_t done = 0;
    while (err == hipSuccess && done < d.bytes) {
      const uint64_t logical = d.offset_bytes + done;
      while (at < segments.size() && segments[at].logical + segments[at].bytes <= logical) ++at;
      if (at == segments.size()) {
        err = hipErrorInvalidValue;
        break;
      }
      const WeightSegment &seg = segments[at];
      const uint64_t inside = logical - seg.logical;
      uint64_t piece = std::min(d.bytes - done, seg.bytes - inside);
      if (file == nullptr) {
        err = hipMemcpyAsync(seg.device + inside, reinterpret_cast<const char *>(d.host_source) + done, piece,
                             hipMemcpyHostToDevice, stream);
      } else {
        piece = std::min(piece, kStagingBytes);
        if (fseeko(file, static_cast<off_t>(d.file_offset_begin + done), SEEK_SET) != 0 ||
            fread(staging, 1, piece, file) != piece) {
          err = hipErrorInvalidValue;
          break;
        }
        err = hipMemcpyAsync(seg.device + inside, staging, piece, hipMemcpyHostToDevice, stream);
        if (err == hipSuccess) err = hipStreamSynchronize(stream);  // the one staging buffer is reused
        *sync_calls += 1;
      }
      done += piece;
    }
    if (file != nullptr) fclose(file);
    *h2d_bytes += done;
  }
  if (err == hipSuccess) err = hipStreamSynchronize(stream);
  if (staging != nullptr) (void)hipHostFree(staging);
  return err;
}

}  // namespace nv
