// Feed-forwards of a block besides the SwiGLU one of llama_block.hip (feed_forward.hip).
#pragma once
#include "llama_internal.hpp"
#include "moe_kernels.hpp"

namespace shainet {

struct FeedForward {
  virtual ~FeedForward() {}
  // y = f(h), T rows of d_model, not the same buffer; proj: the block's
  virtual int forward(Projector &proj, const float *h, int T, float *y, hipStream_t stream) = 0;
};

// y = act(h W_up + b_up) W_down + b_down
struct DenseWeights {
  float *up = nullptr, *up_t = nullptr, *up_bias = nullptr;        // [d, ff], twin, [ff]
  float *down = nullptr, *down_t = nullptr, *down_bias = nullptr;  // [ff, d], twin, [d]
  Activation act;
  bool up_t_stale = true, down_t_stale = true;
};
int dense_create(FeedForward **out, int d_model, int ff, DenseWeights **weights);

// moe_kernels.hpp; expert matrices as [out, in].  The router's and the shared expert's are kept both ways round: many
// tokens take them through the ordinary products.
struct MoeWeights {
  float *router = nullptr, *correction = nullptr, *gate_up = nullptr, *down = nullptr;
  float *router_in = nullptr;                                     // [d, n_router], zero columns up to a multiple of 4
  int n_router = 0;
  float *shared_gate_up = nullptr, *shared_down = nullptr;        // [2 ff, d], [d, ff]
  float *shared_gate_up_in = nullptr, *shared_down_in = nullptr;  // [d, 2 ff], [ff, d]
};
int moe_create(FeedForward **out, const MoeShape &shape, MoeWeights **weights);

}  // namespace shainet
