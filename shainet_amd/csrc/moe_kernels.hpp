// Launchers of a mixture of SwiGLU experts behind a softmax router.  Per token, with h its row:
//   s = softmax(W_router h) over experts and identity experts together
//   chosen: the `top` largest s + correction among the `keep` groups (of `groups` equal ones, neighbours)
//           whose largest s + correction are largest; ties go to the lower index
//   weight of a chosen one: s / (sum of the chosen s + 1e-20) * scale
//   result: sum of weight * expert(h); an identity expert (the last `identity` outputs) gives h itself
// and a shared expert, if there is one, that every token takes with weight 1.
// A few tokens: a wavefront per output of every chosen expert (moe_up_kernel, moe_down_kernel).  Many: the
// tokens are sorted by expert and every expert is two MFMA products over its own rows.
// Expert matrices lie as [out, in].
#pragma once
#include <hip/hip_runtime.h>

#include <stddef.h>

namespace shainet {

constexpr int kMaxRouterOutputs = 1024;

struct MoeShape {
  int d, ff, experts, identity, top, groups, keep, shared_ff;  // shared_ff 0: no shared expert
  float scale;
};
struct MoeTensors {
  const float *router, *correction;            // [experts + identity, d], [experts + identity]
  const float *gate_up, *down;                 // [experts][2 ff, d] (gate rows, then up rows), [experts][d, ff]
  const float *shared_gate_up, *shared_down;   // [2 shared_ff, d], [d, shared_ff]
};
bool moe_shape_ok(const MoeShape &m);

constexpr int kMoeFewTokens = 8;
// y [T, d] for T <= kMoeFewTokens rows h [T, d]; scratch: moe_few_floats(m, T) floats
size_t moe_few_floats(const MoeShape &m, int T);
hipError_t launch_moe_few(const MoeShape &m, const MoeTensors &w, const float *h, float *y, int T, float *scratch,
                          hipStream_t stream);

// Any number of rows.  logits: the router's product with h, rows of `stride` floats; y [T, d] holds the shared
// expert's rows already (add_to_y) or nothing.
// scratch: moe_many_floats floats; counts: m.experts ints, zero before the first call, left zero.
size_t moe_many_floats(const MoeShape &m, int T);
hipError_t launch_moe_many(const MoeShape &m, const MoeTensors &w, const float *h, const float *logits, int stride,
                           float *y, bool add_to_y, int T, float *scratch, int *counts, hipStream_t stream);

}  // namespace shainet
