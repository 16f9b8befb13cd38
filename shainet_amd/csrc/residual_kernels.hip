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

// One row: everything it needs is requested at once and stays in registers.  P: 16-byte pieces per thread;
// TAPS: taps of the convolution that are asked for ahead (more are read when they are used).
template <int P, int TAPS>
__global__ __launch_bounds__(1024) void residual_row_kernel(const ResidualArgs a) {
  __shared__ float red_y[16], red_x[16];
  const int d4 = a.d >> 2, nt = blockDim.x;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4 x[P], y[P], post[P], pre[P], w[P][TAPS], old[P][TAPS];
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int i = threadIdx.x + p * nt;
    const bool in = i < d4;
    x[p] = in ? ((const f32x4 *)a.x)[i] : zero;
    y[p] = in && a.y ? ((const f32x4 *)a.y)[i] : zero;
    post[p] = in && a.y ? ((const f32x4 *)a.post)[i] : zero;
    pre[p] = in && a.pre ? ((const f32x4 *)a.pre)[i] : zero;
#pragma unroll
    for (int k = 0; k < TAPS; ++k) {
      w[p][k] = in && a.conv && k < a.taps ? ((const f32x4 *)a.conv)[(long long)k * d4 + i] : zero;
      old[p][k] = in && a.hist_in && k < a.taps - 1 ? ((const f32x4 *)a.hist_in)[(long long)k * d4 + i] : zero;
    }
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
  float sq = 0.f;
#pragma unroll
  for (int p = 0; p < P; ++p) sq += sum4(x[p] * x[p]);
  const float f = inv_rms(block_sum(sq, red_x), a.d, a.eps);
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int i = threadIdx.x + p * nt;
    if (i >= d4) continue;
    const f32x4 h = x[p] * f * pre[p];
    f32x4 c = zero;
    if (a.conv) {
#pragma unroll
      for (int k = 0; k < TAPS; ++k) {
        if (k < a.taps - 1) {
          c += old[p][k] * w[p][k];
          if (a.hist_out && k > 0) ((f32x4 *)a.hist_out)[(long long)(k - 1) * d4 + i] = old[p][k];
        } else if (k == a.taps - 1) {
          c += h * w[p][k];
        }
      }
      for (int k = TAPS; k < a.taps; ++k) {
        const f32x4 v = k == a.taps - 1 ? h : a.hist_in ? ((const f32x4 *)a.hist_in)[(long long)k * d4 + i] : zero;
        c += v * ((const f32x4 *)a.conv)[(long long)k * d4 + i];
        if (a.hist_out && k < a.taps - 1) ((f32x4 *)a.hist_out)[(long long)(k - 1) * d4 + i] = v;
      }
      if (a.hist_out && a.taps > 1) ((f32x4 *)a.hist_out)[(long long)(a.taps - 2) * d4 + i] = h;
    }
    ((f32x4 *)a.h)[i] = h + c;
  }
}

// Many rows, first launch: a workgroup per row.  Without a convolution h is finished here, with one its factor
// is left for the second launch.  P: 16-byte pieces per thread (0: any width, element by element).
template <int P>
__global__ __launch_bounds__(256) void residual_join_kernel(const ResidualArgs a) {
  __shared__ float red_y[4], red_x[4];
  const long long t = blockIdx.x;
  if constexpr (P > 0) {
    const int d4 = a.d >> 2;
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    const f32x4 *xr = (const f32x4 *)a.x + t * d4, *yr = a.y ? (const f32x4 *)a.y + t * d4 : nullptr;
    f32x4 x[P], y[P];
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int i = threadIdx.x + 256 * p;
      x[p] = i < d4 ? xr[i] : zero;
      y[p] = i < d4 && yr ? yr[i] : zero;
    }
    if (yr) {
      float sq = 0.f;
#pragma unroll
      for (int p = 0; p < P; ++p) sq += sum4(y[p] * y[p]);
      const float f = inv_rms(block_sum(sq, red_y), a.d, a.eps);
#pragma unroll
      for (int p = 0; p < P; ++p) {
        const int i = threadIdx.x + 256 * p;
        if (i >= d4) continue;
        x[p] += y[p] * f * ((const f32x4 *)a.post)[i];
        ((f32x4 *)a.x_out)[t * d4 + i] = x[p];
      }
    }
    if (!a.pre) return;
    float sq = 0.f;
#pragma unroll
    for (int p = 0; p < P; ++p) sq += sum4(x[p] * x[p]);
    const float f = inv_rms(block_sum(sq, red_x), a.d, a.eps);
    if (a.conv) {
      if (threadIdx.x == 0) a.factors[t] = f;
      return;
    }
#pragma unroll
    for (int p = 0; p < P; ++p) {
      const int i = threadIdx.x + 256 * p;
      if (i < d4) ((f32x4 *)a.h)[t * d4 + i] = x[p] * f * ((const f32x4 *)a.pre)[i];
    }
  } else {
    const float *xr = a.x + t * a.d;
    if (a.y) {
      float sq = 0.f;
      for (int i = threadIdx.x; i < a.d; i += 256) sq += a.y[t * a.d + i] * a.y[t * a.d + i];
      const float f = inv_rms(block_sum(sq, red_y), a.d, a.eps);
      for (int i = threadIdx.x; i < a.d; i += 256) a.x_out[t * a.d + i] = xr[i] + a.y[t * a.d + i] * f * a.post[i];
      xr = a.x_out + t * a.d;  // (a thread reads what it wrote itself)
    }
    if (!a.pre) return;
    float sq = 0.f;
    for (int i = threadIdx.x; i < a.d; i += 256) sq += xr[i] * xr[i];
    const float f = inv_rms(block_sum(sq, red_x), a.d, a.eps);
    if (a.conv) {
      if (threadIdx.x == 0) a.factors[t] = f;
      return;
    }
    for (int i = threadIdx.x; i < a.d; i += 256) a.h[t * a.d + i] = xr[i] * f * a.pre[i];
  }
}

// Second launch: kRows rows of 256 columns (of 16 bytes) per workgroup; x: the joined rows.  All rows a thread
// needs are requested before the first is used.
constexpr int kRows = 8;
template <int TAPS>
__global__ __launch_bounds__(256) void residual_conv_kernel(const ResidualArgs a, const float *__restrict__ x) {
  constexpr int BACK = TAPS - 1, N = kRows + BACK;
  const int d4 = a.d >> 2, i = blockIdx.y * 256 + threadIdx.x, first = blockIdx.x * kRows;
  if (i >= d4) return;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4 h[N], w[TAPS];
  float f[N];
#pragma unroll
  for (int k = 0; k < N; ++k) {
    const int t = first - BACK + k;
    if (t < 0) {
      h[k] = a.hist_in && t >= -BACK ? ((const f32x4 *)a.hist_in)[(long long)(BACK + t) * d4 + i] : zero;
      f[k] = 1.f;
    } else {
      h[k] = ((const f32x4 *)x)[(long long)min(t, a.T - 1) * d4 + i];
      f[k] = a.factors[min(t, a.T - 1)];
    }
  }
#pragma unroll
  for (int k = 0; k < TAPS; ++k) w[k] = ((const f32x4 *)a.conv)[(long long)k * d4 + i];
  const f32x4 pre = ((const f32x4 *)a.pre)[i];
#pragma unroll
  for (int k = 0; k < N; ++k) {
    const int t = first - BACK + k;
    if (t >= 0) h[k] = h[k] * f[k] * pre;
    if (a.hist_out && t < a.T && (k >= BACK || (t < 0 && blockIdx.x == 0))) {  // the last rows of [what came in | this call's]
      const int slot = t - (a.T - BACK);
      if (slot >= 0 && slot < BACK) ((f32x4 *)a.hist_out)[(long long)slot * d4 + i] = h[k];
    }
    if (k < BACK || t >= a.T) continue;
    f32x4 c = zero;
#pragma unroll
    for (int j = 0; j < TAPS; ++j) c += h[k - BACK + j] * w[j];
    ((f32x4 *)a.h)[(long long)t * d4 + i] = h[k] + c;
  }
}

// Any width and number of taps: an element per thread.
__global__ __launch_bounds__(256) void residual_conv_any_kernel(const ResidualArgs a, const float *__restrict__ x) {
  const int back = a.taps - 1, i = blockIdx.y * 256 + threadIdx.x;
  if (i >= a.d) return;
  auto row = [&](int t) {
    if (t < 0) return a.hist_in ? a.hist_in[(long long)(back + t) * a.d + i] : 0.f;
    return x[(long long)t * a.d + i] * a.factors[t] * a.pre[i];
  };
  const int t = blockIdx.x;
  float c = 0.f;
  for (int j = 0; j < a.taps; ++j) c += row(t - back + j) * a.conv[(long long)j * a.d + i];
  const float h = row(t);
  a.h[(long long)t * a.d + i] = h + c;
  if (!a.hist_out) return;
  if (t >= a.T - back) a.hist_out[(long long)(t - (a.T - back)) * a.d + i] = h;
  if (t == 0)
    for (int s = 0; s < back - a.T; ++s) a.hist_out[(long long)s * a.d + i] = row(s + a.T - back);
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
      hipLaunchKernelGGL((residual_row_kernel<1, 4>), dim3(1), dim3(threads), 0, stream, a);
    else if (p <= 2)
      hipLaunchKernelGGL((residual_row_kernel<2, 2>), dim3(1), dim3(threads), 0, stream, a);
    else
      hipLaunchKernelGGL((residual_row_kernel<4, 1>), dim3(1), dim3(threads), 0, stream, a);
    return hipGetLastError();
  }
  if (a.conv && !a.factors) return hipErrorInvalidValue;
  const dim3 rows((unsigned)a.T);
  const int pieces = vec ? (d4 + 255) / 256 : 99;
  {
    if (pieces <= 1)
      hipLaunchKernelGGL(residual_join_kernel<1>, rows, dim3(256), 0, stream, a);
    else if (pieces <= 2)
      hipLaunchKernelGGL(residual_join_kernel<2>, rows, dim3(256), 0, stream, a);
    else if (pieces <= 4)
      hipLaunchKernelGGL(residual_join_kernel<4>, rows, dim3(256), 0, stream, a);
    else if (pieces <= 8)
      hipLaunchKernelGGL(residual_join_kernel<8>, rows, dim3(256), 0, stream, a);
    else
      hipLaunchKernelGGL(residual_join_kernel<0>, rows, dim3(256), 0, stream, a);
  }
  if (!a.conv) return hipGetLastError();
  const float *x = a.y ? a.x_out : a.x;
  const dim3 grid((unsigned)((a.T + kRows - 1) / kRows), (unsigned)((d4 + 255) / 256));
  if (vec && a.taps == 1)
    hipLaunchKernelGGL(residual_conv_kernel<1>, grid, dim3(256), 0, stream, a, x);
  else if (vec && a.taps == 2)
    hipLaunchKernelGGL(residual_conv_kernel<2>, grid, dim3(256), 0, stream, a, x);
  else if (vec && a.taps == 3)
    hipLaunchKernelGGL(residual_conv_kernel<3>, grid, dim3(256), 0, stream, a, x);
  else if (vec && a.taps == 4)
    hipLaunchKernelGGL(residual_conv_kernel<4>, grid, dim3(256), 0, stream, a, x);
  else
    hipLaunchKernelGGL(residual_conv_any_kernel, dim3((unsigned)a.T, (unsigned)((a.d + 255) / 256)), dim3(256), 0, stream, a, x);
  return hipGetLastError();
}

hipError_t launch_add_one(float *x, long long n, hipStream_t stream) {
  if (!x || n < 1 || (n + 255) / 256 > 0x7fffffffLL) return hipErrorInvalidValue;
  hipLaunchKernelGGL(add_one_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, x, n);
  return hipGetLastError();
}

}  // namespace shainet
