// Gated linear attention with a state instead of a cache as a block's mixer (hgrn2.hip).
#pragma once
#include "mixer.hpp"

namespace shainet {

struct Hgrn2Config {
  int heads = 0, dim = 0, vdim = 0;
};
struct Hgrn2Weights {
  // W_q | W_f | W_v side by side, [d, n_in], zero columns up to a multiple of 4
  float *w_in = nullptr, *w_in_t = nullptr;
  float *f_bias = nullptr, *lower = nullptr;  // [heads dim]
  float *norm = nullptr;                      // [vdim]
  float *w_o = nullptr, *w_o_t = nullptr;     // [heads vdim, d]
  int n_in = 0;
  bool w_in_t_stale = true, w_o_t_stale = true;
};
int hgrn2_create(Mixer **out, int d_model, const Hgrn2Config &cfg, double eps);
Hgrn2Weights &hgrn2_weights(Hgrn2 *l);
const Hgrn2Config &hgrn2_config(Hgrn2 *l);
const float *hgrn2_state(Hgrn2 *l);  // device [heads, dim, vdim]; zeros before the first token are not written

}  // namespace shainet
