// Routed experts over blocks of token rows, 16-bit weights (moe_rows.hip):
//   scores s = sigmoid(router logits); the `top` largest (ties: the lower index) with weights s / (sum of them + 1e-20)
//   expert: g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit), W_down (g sigmoid(1.702 g) (u + 1))
// A (token, choice) pair is a slot, slot = token * top + choice. The slots are sorted by expert; an expert's slots are
// taken in tiles, each a product of the expert's matrix with the gathered rows. The down products leave one row per
// slot; whoever adds them (norm_rms.cuh) weighs them. One expert that takes every token (a shared one) goes through the
// same kernels without lists: slot = token.
//   16-bit rows: matrix cores (v_mfma_f32_16x16x32), both operands through LDS: small tiles and odd sizes with the next
//                K-step's pieces in registers, large tiles of whole steps with requests straight to LDS, two steps ahead;
//   f32 rows:    vector ALU, every product and sum in f32.
#pragma once

#include "nv_common.cuh"

namespace nv {

constexpr uint32_t kExpertTile = 64;        // slots of a tile; twice as many where an expert has enough of them
constexpr uint32_t kMaxExperts = 1024, kMaxTop = 64;

// Device memory of a block's routing: tokens * top slots, every array sized by moe_plan_bytes.
struct MoePlan {
  uint32_t *ids;        // [tokens][top]
  float *weights;       // [tokens][top]
  uint32_t *sorted;     // [tokens * top] slots in the order of their experts
  uint4 *tiles;         // (expert, first place in `sorted`, slots, 0)
  uint32_t *tile_count;
  uint32_t tile;        // slots of a tile
};
__host__ inline uint32_t expert_tile(uint32_t slots, uint32_t experts) {
  return slots >= 80u * experts ? 2u * kExpertTile : kExpertTile;
}
__host__ inline uint32_t moe_max_tiles(uint32_t tokens, uint32_t top, uint32_t experts, uint32_t tile) {
  const uint32_t slots = tokens * top;
  return slots / tile + (experts < slots ? experts : slots);
}
uint64_t moe_plan_bytes(uint32_t tokens, uint32_t top, uint32_t experts);
// small_tiles: kExpertTile whatever the block holds (f32 rows)
MoePlan moe_plan_at(void *base, uint32_t tokens, uint32_t top, uint32_t experts, bool small_tiles);

struct MoeRouteRows {
  const float *logits;   // [tokens][experts]
  uint32_t tokens, experts, top;
  MoePlan plan;
};
hipError_t launch_moe_route_rows(const MoeRouteRows &p, hipStream_t stream);

struct ExpertRows {
  const uint16_t *w_gate_up;   // [experts][2 * ff][hidden], gate rows first
  const uint16_t *w_down;      // [experts][hidden][ff]
  const uint16_t *x16;         // [tokens][hidden]
  const float *x32;            // likewise, used when x16 is null
  uint16_t *act16;             // [slots][ff]
  float *act32;
  float *out;                  // [slots][hidden]
  uint32_t hidden, ff, tokens, top, experts;
  float limit;
  const MoePlan *plan;         // host struct; null: one expert, slot = token (top = experts = 1)
};
hipError_t expert_rows_setup();   // once per process, outside stream capture
hipError_t launch_expert_gate_up(uint32_t dtype, const ExpertRows &p, hipStream_t stream);
hipError_t launch_expert_down(uint32_t dtype, const ExpertRows &p, hipStream_t stream);

}  // namespace nv
