// Grouped-query attention without rotation whose scores gain a learned value by distance (biased_attn.hip).
#pragma once
#include <vector>

#include "mixer.hpp"

namespace shainet {

struct BiasedConfig {
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
  double scale = 0.0;
  int bias_max = 0;  // from this distance on the last row of the table holds
};

// The row of a table of `rows` rows that distance n uses: n itself below rows / 2, then logarithmically wider
// buckets up to bias_max.
int distance_bucket(int n, int rows, int bias_max);

struct BiasedWeights {
  float *w_in = nullptr, *w_in_t = nullptr;  // [d, n_in]: W_q | W_k | W_v side by side (a borrowing layer: W_q)
  float *w_o = nullptr, *w_o_t = nullptr;    // [H vdim, d]
  int n_in = 0;
  bool w_in_t_stale = true, w_o_t_stale = true;
};

// kv_from != null: keys and values are that mixer's, which has projections of its own, the same kv_heads, dim
// and vdim, and has run the same tokens before.
int biased_attn_create(Mixer **out, int d_model, const BiasedConfig &cfg, Mixer *kv_from);
BiasedWeights &biased_attn_weights(BiasedAttn *l);
// rel: [rows, heads] on the host; max_positions: distances stay below it
int biased_attn_set_table(BiasedAttn *l, const std::vector<float> &rel, int rows, int max_positions);

}  // namespace shainet
