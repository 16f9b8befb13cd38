// Between two sublayers of a block that norms before and after each of them (residual_kernels.hpp).
// fp32 throughout: sums of squares per lane, then over the wavefront and the workgroup.
#include "residual_kernels.hpp"

#include <math.h>
#include <stdint.h>

namespace shainet {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
  return v;
}
__device__ __forceinline__ float sum4(f32x4 v) { return (v.x + v.y) + (v.z + v.w); }
__device__ __forceinline__ float inv_rms(float sq, int d, float eps) { return 1.0f / sqrtf(sq / (float)d + eps); }

// sum over the workgroup; red: one float per wavefront, used once per call site
__device__ __forceinline__ float block_sum(float v, float *red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = red[0];
  for (int w = 1; w < (int)(blockDim.x >> 6); ++w) s += red[w];
  return s;
}

// One row: everything it needs is requested at once and stays in registers.  P: 16-byte pieces per thread.
template <int P>
__global__ __launch_bounds__(1024) void residual_row_kernel(const ResidualArgs a) {
  __shared__ float red_y[16], red_x[16];
  const int d4 = a.d >> 2, nt = blockDim.x;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4 x[P], y[P], post[P], pre[P];
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int i = threadIdx.x + p * nt;
    const bool in = i < d4;
    x[p] = in ? ((const f32x4 *)a.x)[i] : zero;
    y[p] = in && a.y ? ((const f32x4 *)a.y)[i] : zero;
    post[p] = in && a.y ? ((const f32x4 *)a.post)[i] : zero;
    pre[p] = in && a.pre ? ((const f32x4 *)a.pre)[i] : zero;
  }
  if (a.y) {
    float sq = 0.f;
#pragma unroll
    for (int p = 0; p < P; ++p) sq += sum4(y[p] * y[p]);
    const float f = inv_rms(block_sum(sq, red_y), a.d, a.eps);
#pragma unroll
    for (int p = 0; p < P; ++p) {
      x[p] += y[p] * f * post[p];
      const int i = threadIdx.x + p * nt;
      if (i < d4) ((f32x4 *)a.x_out)[i] = x[p];
    }
  }
  if (!a.pre) return;
  // (the earlier rows' part of the convolution does not depend on this row's norm)
  f32x4 c[P], w_own[P];
#pragma unroll
  for (int p = 0; p < P; ++p) {
    c[p] = w_own[p] = zero;
    const int i = threadIdx.x + p * nt;
    if (!a.conv || i >= d4) continue;
    w_own[p] = ((const f32x4 *)a.conv)[(long long)(a.taps - 1) * d4 + i];
    for (int k = 0; k < a.taps - 1; ++k) {
      const f32x4 v = a.hist_in ? ((const f32x4 *)a.hist_in)[(long long)k * d4 + i] : zero;
      c[p] += v * ((const f32x4 *)a.conv)[(long long)k * d4 + i];
      if (a.hist_out && k > 0) ((f32x4 *)a.hist_out)[(long long)(k - 1) * d4 + i] = v;
    }
  }
  float sq = 0.f;
#pragma unroll
  for (int p = 0; p < P; ++p) sq += sum4(x[p] * x[p]);
  const float f = inv_rms(block_sum(sq, red_x), a.d, a.eps);
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int i = threadIdx.x + p * nt;
    if (i >= d4) continue;
    const f32x4 h = x[p] * f * pre[p];
    if (a.hist_out && a.taps > 1) ((f32x4 *)a.hist_out)[(long long)(a.taps - 2) * d4 + i] = h;
    ((f32x4 *)a.h)[i] = h + (c[p] + h * w_own[p]);
  }
}

// The two factors of the rows first - back .. first + kRows - 1 that exist, a wavefront per row.
constexpr int kRows = 8;
template <bool VEC>
__device__ __forceinline__ void row_factors(const ResidualArgs &a, int first, int back, float *fy, float *fx) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int k = wave; k < back + kRows; k += 4) {
    const int t = first - back + k;
    if (t < 0 || t >= a.T) continue;
    const float *x = a.x + (long long)t * a.d, *y = a.y ? a.y + (long long)t * a.d : nullptr;
    float f1 = 0.f;
    if (y) {
      float sq = 0.f;
      if (VEC)
        for (int i = lane; i < a.d >> 2; i += 64) sq += sum4(((const f32x4 *)y)[i] * ((const f32x4 *)y)[i]);
      else
        for (int i = lane; i < a.d; i += 64) sq += y[i] * y[i];
      f1 = inv_rms(wave_sum(sq), a.d, a.eps);
    }
    float f2 = 0.f;
    if (a.pre) {
      float sq = 0.f;
      if (VEC) {
        for (int i = lane; i < a.d >> 2; i += 64) {
          f32x4 v = ((const f32x4 *)x)[i];
          if (y) v += ((const f32x4 *)y)[i] * f1 * ((const f32x4 *)a.post)[i];
          sq += sum4(v * v);
        }
      } else {
        for (int i = lane; i < a.d; i += 64) {
          float v = x[i];
          if (y) v += y[i] * f1 * a.post[i];
          sq += v * v;
        }
      }
      f2 = inv_rms(wave_sum(sq), a.d, a.eps);
    }
    if (lane == 0) {
      fy[k] = f1;
      fx[k] = f2;
    }
  }
}

// Many rows: a workgroup takes kRows rows and works out again what it needs of the TAPS - 1 rows before
// them.  A thread walks down its columns with the last TAPS rows' h in registers.
// x_out == x would let a workgroup read a neighbour's rows after they have changed: the caller passes
// another buffer when TAPS > 1.
template <int TAPS>
__global__ __launch_bounds__(256) void residual_rows_kernel(const ResidualArgs a) {
  __shared__ float fy[TAPS - 1 + kRows], fx[TAPS - 1 + kRows];
  const int first = blockIdx.x * kRows, last = min(first + kRows, a.T);
  row_factors<true>(a, first, TAPS - 1, fy, fx);
  __syncthreads();
  const int d4 = a.d >> 2;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  for (int i = threadIdx.x; i < d4; i += 256) {
    f32x4 post = zero, pre = zero, w[TAPS], win[TAPS];
    if (a.y) post = ((const f32x4 *)a.post)[i];
    if (a.pre) pre = ((const f32x4 *)a.pre)[i];
#pragma unroll
    for (int k = 0; k < TAPS; ++k) {
      w[k] = a.conv ? ((const f32x4 *)a.conv)[(long long)k * d4 + i] : zero;
      win[k] = zero;
    }
    for (int k = 0; k < TAPS - 1 + kRows; ++k) {
      const int t = first - (TAPS - 1) + k;
      if (t >= last) break;
      f32x4 h = zero;
      if (t < 0) {
        if (a.hist_in && t >= -(TAPS - 1)) h = ((const f32x4 *)a.hist_in)[(long long)(TAPS - 1 + t) * d4 + i];
      } else {
        f32x4 x = ((const f32x4 *)a.x)[(long long)t * d4 + i];
        if (a.y) {
          x += ((const f32x4 *)a.y)[(long long)t * d4 + i] * fy[k] * post;
          if (t >= first) ((f32x4 *)a.x_out)[(long long)t * d4 + i] = x;
        }
        h = x * fx[k] * pre;
      }
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j) win[j] = win[j + 1];
      win[TAPS - 1] = h;
      if (a.hist_out) {  // the last TAPS - 1 rows of [what came in | this call's]
        const int slot = t - (a.T - (TAPS - 1));
        if (slot >= 0 && slot < TAPS - 1 && (t >= first || (t < 0 && blockIdx.x == 0)))
          ((f32x4 *)a.hist_out)[(long long)slot * d4 + i] = h;
      }
      if (t < first || !a.pre) continue;
      f32x4 c = zero;
#pragma unroll
      for (int j = 0; j < TAPS; ++j) c += win[j] * w[j];
      ((f32x4 *)a.h)[(long long)t * d4 + i] = h + c;
    }
  }
}

// Any width and number of taps: a column per thread, the window in LDS.
__global__ __launch_bounds__(256) void residual_any_kernel(const ResidualArgs a) {
  extern __shared__ float win[];  // [taps][256], row t in slot t mod taps
  __shared__ float fy[kMaxConvTaps - 1 + kRows], fx[kMaxConvTaps - 1 + kRows];
  const int taps = a.taps, back = taps - 1;
  const int first = blockIdx.x * kRows, last = min(first + kRows, a.T);
  row_factors<false>(a, first, back, fy, fx);
  __syncthreads();
  for (int i = threadIdx.x; i < a.d; i += 256) {
    for (int k = 0; k < back + kRows; ++k) {
      const int t = first - back + k;
      if (t >= last) break;
      float h = 0.f;
      if (t < 0) {
        if (a.hist_in) h = a.hist_in[(long long)(back + t) * a.d + i];
      } else {
        float x = a.x[(long long)t * a.d + i];
        if (a.y) {
          x += a.y[(long long)t * a.d + i] * fy[k] * a.post[i];
          if (t >= first) a.x_out[(long long)t * a.d + i] = x;
        }
        if (a.pre) h = x * fx[k] * a.pre[i];
      }
      win[(k % taps) * 256 + threadIdx.x] = h;
      if (a.hist_out) {
        const int slot = t - (a.T - back);
        if (slot >= 0 && slot < back && (t >= first || (t < 0 && blockIdx.x == 0)))
          a.hist_out[(long long)slot * a.d + i] = h;
      }
      if (t < first || !a.pre) continue;
      float c = 0.f;
      if (a.conv)
        for (int j = 0; j < taps; ++j) c += win[((k + 1 + j) % taps) * 256 + threadIdx.x] * a.conv[(long long)j * a.d + i];
      a.h[(long long)t * a.d + i] = h + c;
    }
  }
}

__global__ __launch_bounds__(256) void add_one_kernel(float *x, long long n) {
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] += 1.0f;
}

}  // namespace

hipError_t launch_residual(const ResidualArgs &args, hipStream_t stream) {
  ResidualArgs a = args;
  if (!a.conv) {
    a.taps = 1;
    a.hist_in = nullptr;
    a.hist_out = nullptr;
  }
  if (!a.x || a.T < 1 || a.d < 1 || (a.y && (!a.post || !a.x_out)) || (a.pre && !a.h) || (!a.y && !a.pre) ||
      (a.conv && !a.pre) || a.taps < 1 || a.taps > kMaxConvTaps || (a.hist_out && a.hist_out == a.hist_in))
    return hipErrorInvalidValue;
  const bool vec = (a.d & 3) == 0 &&
                   !(((uintptr_t)a.x | (uintptr_t)a.y | (uintptr_t)a.post | (uintptr_t)a.x_out | (uintptr_t)a.pre |
                      (uintptr_t)a.conv | (uintptr_t)a.hist_in | (uintptr_t)a.hist_out | (uintptr_t)a.h) & 15);
  const int d4 = a.d >> 2;
  if (a.T == 1 && vec && d4 <= 4096) {
    int threads = (d4 + 63) / 64 * 64;
    if (threads > 1024) threads = 1024;
    const int p = (d4 + threads - 1) / threads;
    if (p <= 1)
      hipLaunchKernelGGL(residual_row_kernel<1>, dim3(1), dim3(threads), 0, stream, a);
    else if (p <= 2)
      hipLaunchKernelGGL(residual_row_kernel<2>, dim3(1), dim3(threads), 0, stream, a);
    else
      hipLaunchKernelGGL(residual_row_kernel<4>, dim3(1), dim3(threads), 0, stream, a);
    return hipGetLastError();
  }
  const bool spread = a.taps > 1 && a.T > kRows;  // rows are read by the workgroup behind them, too
  if (spread && a.y && a.x_out == a.x) return hipErrorInvalidValue;
  const dim3 grid((unsigned)((a.T + kRows - 1) / kRows));
  if (vec && a.taps == 1)
    hipLaunchKernelGGL(residual_rows_kernel<1>, grid, dim3(256), 0, stream, a);
  else if (vec && a.taps == 2)
    hipLaunchKernelGGL(residual_rows_kernel<2>, grid, dim3(256), 0, stream, a);
  else if (vec && a.taps == 3)
    hipLaunchKernelGGL(residual_rows_kernel<3>, grid, dim3(256), 0, stream, a);
  else if (vec && a.taps == 4)
    hipLaunchKernelGGL(residual_rows_kernel<4>, grid, dim3(256), 0, stream, a);
  else
    hipLaunchKernelGGL(residual_any_kernel, grid, dim3(256), (size_t)a.taps * 256 * sizeof(float), stream, a);
  return hipGetLastError();
}

hipError_t launch_add_one(float *x, long long n, hipStream_t stream) {
  if (!x || n < 1 || (n + 255) / 256 > 0x7fffffffLL) return hipErrorInvalidValue;
  hipLaunchKernelGGL(add_one_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, x, n);
  return hipGetLastError();
}

}  // namespace shainet
