// Launchers of what lies between two sublayers of a block that norms before and after each of them
// and convolves what a sublayer reads over time:
//   x' = x + y / rms(y) * post           the sublayer's result y joins the residual
//   h  = x' / rms(x') * pre              what the next sublayer reads, before
//   h' = h + conv(h)                     and after a causal convolution over time on each channel
// A single row is one launch.  More rows are two: the first joins y and takes the norms' factors, the second
// walks the rows of a column for the convolution.  Every part but x can be left out.
#pragma once
#include <hip/hip_runtime.h>

namespace shainet {

constexpr int kMaxConvTaps = 32;

struct ResidualArgs {
  const float *x;        // [T, d]
  const float *y;        // [T, d] or null (then x' = x)
  const float *post;     // [d], with y
  float *x_out;          // [T, d], with y; may be x
  const float *pre;      // [d] or null: no h is wanted
  const float *conv;     // [taps, d], the last tap meets the row itself; null: h' = h
  int taps;              // at most kMaxConvTaps
  const float *hist_in;  // [taps - 1, d] the h of the rows before row 0, oldest first; null: zeros
  float *hist_out;       // [taps - 1, d] the same for the next call, not hist_in; null: not kept
  float *h;              // [T, d]
  float *factors;        // [T] scratch, with pre and conv
  int T, d;
  float eps;
};
hipError_t launch_residual(const ResidualArgs &a, hipStream_t stream);

// x[i] += 1, n floats: weights stored as the distance from 1
hipError_t launch_add_one(float *x, long long n, hipStream_t stream);

}  // namespace shainet
