// Launchers of gated linear attention whose forget gate also decides what is written (HGRN2).  Per head,
// with a state S of dim x vdim floats that is carried from token to token:
//   q = silu(zq),  f = l + (1 - l) sigmoid(zf + b)        per channel of dim
//   S <- diag(f) S + (1 - f) v^T,   o = S^T q             v: vdim values
//   out = o / sqrt(mean(o^2) + eps) * norm                per head over vdim
// zq, zf and v are what one product made of the mixer's input, side by side in a row.
//
// A few rows go through the state one after the other (hgrn2_step_kernel).  Many rows are cut into
// chunks: what a chunk adds to the state and how much of the old one it leaves depends on the chunk
// alone (hgrn2_chunk_kernel), the states at the chunks' beginnings follow in one pass over them
// (hgrn2_scan_kernel), and then all rows of all chunks are worked out side by side
// (hgrn2_output_kernel).  Every decay that is ever formed is a product of gates over a stretch of
// tokens, at most 1: nothing is divided by one, so small gates cannot overflow.
#pragma once
#include <hip/hip_runtime.h>

namespace shainet {

struct Hgrn2Args {
  const float *raw;       // [T] rows `stride` floats apart: zq [H dim] | zf [H dim] | v [H vdim]
  long long stride;
  const float *f_bias;    // [H dim]
  const float *lower;     // [H dim] the lower bound l
  const float *norm;      // [vdim]
  float *state;           // [H, dim, vdim], read and left for the next call
  bool fresh;             // the sequence begins here: whatever lies in state, it counts as zeros
  float *out;             // [T, H vdim]
  int T, H, dim, vdim;
  float eps;
};
struct Hgrn2Plan {
  int chunk;              // rows per chunk: 64, 32 or 16; 0: one row after the other
  int chunks;             // at a time
  size_t scratch_floats;
};
// false: sizes no kernel takes (dim above 4096, vdim above 1024)
bool plan_hgrn2(int T, int H, int dim, int vdim, Hgrn2Plan &p);
hipError_t launch_hgrn2(const Hgrn2Args &a, const Hgrn2Plan &p, float *scratch, hipStream_t stream);

}  // namespace shainet
