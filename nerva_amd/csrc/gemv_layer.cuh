// Decode-step projections of a parallel layer (mixer and feed-forward on the same row) with attention over latents and
// routed experts: the matrices that can be multiplied at the same time share a launch.
//   front   both norms of the row; the mixer's input projection; the router; the shared expert's gate/up pairs
//   middle  the query latent's norm and the query projection; the choice of experts and their gate/up pairs
//   back    x += W_o a + sum_k weight_k W_down,k act_k + W_down,shared act: one walk over all of a row's pieces
// (gemv_layer.hip). A wave takes two rows at a time - a gate and its up row, or two neighbours - or, in the back launch,
// one output row; 1 KiB a load and row, two batches in flight. 16-bit weights and inputs, f32 sums.
#pragma once

#include "nv_common.cuh"

namespace nv {

struct LayerFront {
  const float *x;                          // residual row [hidden]
  const uint16_t *mixer_norm, *ff_norm;    // [hidden]; ff_norm null: no feed-forward
  float eps;
  uint32_t hidden;
  const uint16_t *w_in;                    // [in_rows][hidden] -> in
  uint32_t in_rows;
  float *in;
  const uint16_t *router;                  // [experts][hidden] -> logits
  uint32_t experts;
  float *logits;
  const uint16_t *shared_in;               // [2 * shared_ff][hidden] -> shared_act
  uint32_t shared_ff;
  float shared_limit;
  uint16_t *shared_act;
  uint16_t *h16;                           // the feed-forward's normalised row, for the launches after this one
  const uint32_t *cursor;
  uint32_t max_steps;
};

struct LayerMiddle {
  const float *latent;                     // [q_rank]
  const uint16_t *latent_norm;
  float eps;
  const uint16_t *w_uq;                    // [q_rows][q_rank] -> q
  uint32_t q_rank, q_rows;
  float *q;
  const uint16_t *h16;                     // [hidden]
  const float *logits;                     // [experts]
  uint32_t hidden, experts, top;           // experts 0: no feed-forward
  const uint16_t *e_in;                    // [experts][2 * ff][hidden] -> act [top][ff]
  uint32_t ff;
  float limit;
  uint16_t *act;
  uint32_t *ids;                           // [top]: the choice and its weights, for the back launch
  float *weights;
  const uint32_t *cursor;
  uint32_t max_steps;
};

struct LayerBack {
  float *x;                                // residual row [hidden], in place
  uint32_t hidden;
  const uint16_t *w_o, *mixed;             // [hidden][mix_cols], [mix_cols]
  uint32_t mix_cols;
  const uint16_t *e_out, *act;             // [experts][hidden][ff], [top][ff]
  const uint32_t *ids;
  const float *weights;
  uint32_t ff, top;                        // top 0: no feed-forward
  const uint16_t *shared_out, *shared_act;
  uint32_t shared_ff;                      // 0: no shared expert
  const uint32_t *cursor;
  uint32_t max_steps;
};

// Whether the launches take a layer's sizes (whole 16-byte pieces, vectors that fit into LDS).
bool layer_gemv_takes(uint32_t hidden, uint32_t q_rank, uint32_t mix_cols, uint32_t experts, uint32_t top, uint32_t ff, uint32_t shared_ff);
hipError_t launch_layer_front(uint32_t dtype, const LayerFront &p, hipStream_t stream);
hipError_t launch_layer_middle(uint32_t dtype, const LayerMiddle &p, hipStream_t stream);
hipError_t launch_layer_back(uint32_t dtype, const LayerBack &p, hipStream_t stream);

}  // namespace nv
