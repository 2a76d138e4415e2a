// Mixture of experts: every row uses ``top`` of ``experts`` gated feed-forwards.
//
//   route    router logits -> chosen experts and their weights, per (row, choice) pair
//   group    pairs sorted by expert and cut into tiles of at most tile_rows pairs of one expert
//   up       act[i] = silu(gate . h) * (up . h) of sorted pair i
//   down     y[i] = down . act[i]
//   (join    x += sigmoid(gate) * sum over a row's pairs of weight * y: stream_ops.hip)
#pragma once
#include "elem.h"

struct MoeTile {  // pairs [start, start + count) of the sorted list, all of one expert; expert < 0: none
  int expert, start, count, pad;
};
