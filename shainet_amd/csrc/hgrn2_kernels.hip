// HGRN2 on gfx950 (hgrn2_kernels.hpp says what is computed), fp32.
//
// MFMA layouts (lane l).  32x32x2: A[m = l % 32][k = l / 32], B[k = l / 32][n = l % 32],
// D[m = 8 (r / 4) + 4 (l / 32) + r % 4][n = l % 32].  16x16x4: A[m = l % 16][k = l / 16],
// B[k = l / 16][n = l % 16], D[m = 4 (l / 16) + r][n = l % 16].  The contraction index may be visited in
// any order as long as A and B agree.
#include "hgrn2_kernels.hpp"

#include <math.h>
#include <stdlib.h>

namespace shainet {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int kSub = 16;          // rows between which decays are formed pair by pair
constexpr int kMaxLds = 160 * 1024;
constexpr int kChunksAtOnce = 64;

__device__ __forceinline__ float fast_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
// e^-|z|: the part of |z| log2(e) that its rounding leaves out comes back to first order
__device__ __forceinline__ float exp_neg_abs(float z) {
  const float y = -fabsf(z), hi = y * 1.44269504f, lo = fmaf(y, 1.44269504f, -hi) + y * 1.925963e-8f;
  const float e = fast_exp2(hi);
  return fmaf(e, lo * 0.693147181f, e);
}
// (the hardware's reciprocal is good to the last bit or so; the argument is at least 1)
__device__ __forceinline__ float silu1(float z) {
  const float e = exp_neg_abs(z), r = __builtin_amdgcn_rcpf(1.f + e);
  return z * (z >= 0.f ? r : e * r);
}
// f and 1 - f, each to full precision
__device__ __forceinline__ void gate(float z, float l, float &f, float &k) {
  const float e = exp_neg_abs(z), r = __builtin_amdgcn_rcpf(1.f + e), lo = e * r;  // sigmoid(|z|) and sigmoid(-|z|)
  f = l + (1.f - l) * (z >= 0.f ? r : lo);
  k = (1.f - l) * (z >= 0.f ? lo : r);
}

// ---- one row after the other -------------------------------------------------------------------
// A workgroup per head.  A thread owns W neighbouring columns of rows g, g + groups, ... of the state;
// HELD: at most kHeldRows such rows, which then stay in registers over all rows of the call.
template <int W>
constexpr int kHeldRows = W == 4 ? 4 : 8;
template <int W, bool HELD>
__global__ __launch_bounds__(1024) void hgrn2_step_kernel(const Hgrn2Args a) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  __shared__ float sq_s[16];
  typedef float vec_t __attribute__((ext_vector_type(W)));
  constexpr int kHeld = kHeldRows<W>;
  const int dim = a.dim, vdim = a.vdim, h = blockIdx.x, NT = blockDim.x;
  float *qs = smem, *fs = qs + dim, *ks = fs + dim, *red = smem + (3 * dim + 3) / 4 * 4;  // red: [groups][vdim]
  const int cols = vdim / W, groups = NT / cols;
  const int c = threadIdx.x % cols, g = threadIdx.x / cols;
  const bool mine = g < groups;
  float *S = a.state + (long long)h * dim * vdim + W * c;
  vec_t s[HELD ? kHeld : 1];
  if constexpr (HELD) {
#pragma unroll
    for (int u = 0; u < kHeld; ++u) {
      const int d = g + u * groups;
      s[u] = mine && d < dim && !a.fresh ? *(const vec_t *)(S + (long long)d * vdim) : (vec_t)(0.f);
    }
  }
  for (int t = 0; t < a.T; ++t) {
    const float *row = a.raw + (long long)t * a.stride;
    const vec_t v = mine ? *(const vec_t *)(row + 2LL * a.H * dim + (long long)h * vdim + W * c) : (vec_t)(0.f);
    for (int d = threadIdx.x; d < dim; d += NT) {
      const int i = h * dim + d;
      qs[d] = silu1(row[i]);
      float f, k;
      gate(row[a.H * dim + i] + a.f_bias[i], a.lower[i], f, k);
      fs[d] = f;
      ks[d] = k;
    }
    __syncthreads();
    vec_t acc = (vec_t)(0.f);
    if (mine) {
      if constexpr (HELD) {
#pragma unroll
        for (int u = 0; u < kHeld; ++u) {
          const int d = g + u * groups;
          if (d < dim) {
            s[u] = s[u] * fs[d] + v * ks[d];
            acc += s[u] * qs[d];
          }
        }
      } else {
        for (int d = g; d < dim; d += groups) {
          vec_t *p = (vec_t *)(S + (long long)d * vdim);
          const vec_t x = (a.fresh && t == 0 ? (vec_t)(0.f) : *p * fs[d]) + v * ks[d];
          *p = x;
          acc += x * qs[d];
        }
      }
      *(vec_t *)(red + (long long)g * vdim + W * c) = acc;
    }
    __syncthreads();
    float o = 0.f;  // vdim <= NT: a thread per output
    if ((int)threadIdx.x < vdim)
      for (int k = 0; k < groups; ++k) o += red[(long long)k * vdim + threadIdx.x];
    float sq = o * o;
#pragma unroll
    for (int x = 32; x > 0; x >>= 1) sq += __shfl_xor(sq, x);
    if ((threadIdx.x & 63) == 0) sq_s[threadIdx.x >> 6] = sq;
    __syncthreads();
    float sum = 0.f;
    for (int w = 0; w < NT / 64; ++w) sum += sq_s[w];
    if ((int)threadIdx.x < vdim)
      a.out[((long long)t * a.H + h) * vdim + threadIdx.x] = o / sqrtf(sum / (float)vdim + a.eps) * a.norm[threadIdx.x];
    // (the next row's writes to LDS: qs, fs, ks and red were last read before the barrier above, sq_s is
    // written again only behind the next two)
  }
  if constexpr (HELD) {
#pragma unroll
    for (int u = 0; u < kHeld; ++u) {
      const int d = g + u * groups;
      if (mine && d < dim) *(vec_t *)(S + (long long)d * vdim) = s[u];
    }
  }
}

// ---- chunks ------------------------------------------------------------------------------------
// Column `col` of the kSub rows from `first` on (rows past the end repeat the last one).
__device__ __forceinline__ void load_column(const Hgrn2Args &a, long long col, int first, float (&x)[kSub]) {
#pragma unroll
  for (int r = 0; r < kSub; ++r) x[r] = a.raw[(long long)min(first + r, a.T - 1) * a.stride + col];
}

// The gates of one channel over the kSub rows from `first` on, made of x: body(r, f, k), f = 1 and k = 0 past the end.
template <class F>
__device__ __forceinline__ void walk_gates(const Hgrn2Args &a, int i, int first, const float (&x)[kSub], F body) {
  const float b = a.f_bias[i], l = a.lower[i];
#pragma unroll
  for (int r = 0; r < kSub; ++r) {
    float f, k;
    gate(x[r] + b, l, f, k);
    const bool in = first + r < a.T;
    body(r, in ? f : 1.f, in ? k : 0.f);
  }
}

// What chunk c leaves of the state and adds to it: decay[c][h][d] = prod f, add[c][h] = sum over its rows s of
// (prod over later rows of f) (1 - f_s) v_s^T.  blockIdx.x: head fastest.  The decayed (1 - f) go through LDS as
// the MFMAs' A operand; each of eight wavefronts takes DG tiles of 32 channels against one tile of 32 value columns.
template <int C, int DG>
__global__ __launch_bounds__(512, 4) void hgrn2_chunk_kernel(const Hgrn2Args a, int chunk0, float *__restrict__ add,
                                                             float *__restrict__ decay) {
  constexpr int NS = C / kSub;
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int dim = a.dim, vdim = a.vdim, d32 = (dim + 31) / 32 * 32;
  float *kd = smem, *tot = kd + C * d32;  // [C][d32], [NS][d32]
  const int h = blockIdx.x % a.H, c = blockIdx.x / a.H, first = (chunk0 + c) * C;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n = lane & 31, half = lane >> 5;
  const int n_vt = (vdim + 31) / 32, n_dt = d32 / 32, n_dg = (n_dt + DG - 1) / DG;
  // values of a wavefront's item: PB steps of 16 rows are asked for ahead, the first item's together with the gates
  constexpr int PB = NS < 2 ? 1 : 2;
  float b[PB][8];
  auto load_v = [&](int item, int s0) {
    const float *v = a.raw + 2LL * a.H * dim + (long long)h * vdim + min(item % n_vt * 32 + n, vdim - 1);
#pragma unroll
    for (int i = 0; i < 8; ++i) b[s0 / 16 % PB][i] = v[(long long)min(first + s0 + 2 * i + half, a.T - 1) * a.stride];
  };
  float x[kSub];
  auto load_gates = [&](int it) {
    const int j = it / d32, d = it - j * d32;
    load_column(a, (long long)a.H * dim + h * dim + min(d, dim - 1), first + j * kSub, x);
  };
  if ((int)threadIdx.x < NS * d32) load_gates(threadIdx.x);
  if (wave < n_vt * n_dg)
#pragma unroll
    for (int s0 = 0; s0 < 16 * PB; s0 += 16) load_v(wave, s0);
  for (int it = threadIdx.x; it < NS * d32; it += 512) {
    const int j = it / d32, d = it - j * d32;
    float k_[kSub], f_[kSub];
    if (it >= 512) load_gates(it);
    if (d < dim) {
      walk_gates(a, h * dim + d, first + j * kSub, x, [&](int r, float f, float k) {
        f_[r] = f;
        k_[r] = k;
      });
    } else {
#pragma unroll
      for (int r = 0; r < kSub; ++r) {
        f_[r] = 1.f;
        k_[r] = 0.f;
      }
    }
    float later = 1.f;
#pragma unroll
    for (int r = kSub - 1; r >= 0; --r) {
      kd[(j * kSub + r) * d32 + d] = k_[r] * later;
      later *= f_[r];
    }
    tot[it] = later;
  }
  __syncthreads();
  const long long at = (long long)c * a.H + h;
  for (int it = threadIdx.x; it < NS * d32; it += 512) {
    const int j = it / d32, d = it - j * d32;
    float later = 1.f;
    for (int b = NS - 1; b > j; --b) later *= tot[b * d32 + d];
#pragma unroll
    for (int r = 0; r < kSub; ++r) kd[(j * kSub + r) * d32 + d] *= later;
    if (j == 0 && d < dim) decay[at * dim + d] = later * tot[d];
  }
  __syncthreads();
  float *dst = add + at * dim * vdim;
  for (int item = wave; item < n_vt * n_dg; item += 8) {
    const int vt = item % n_vt, dt0 = item / n_vt * DG;
    const int col = vt * 32 + n;
    f32x16 acc[DG];
#pragma unroll
    for (int u = 0; u < DG; ++u)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[u][r] = 0.f;
    const float *kp[DG];
#pragma unroll
    for (int u = 0; u < DG; ++u) kp[u] = kd + half * d32 + min(dt0 + u, n_dt - 1) * 32 + n;
    if (item != wave) {
#pragma unroll
      for (int s0 = 0; s0 < 16 * PB; s0 += 16) load_v(item, s0);
    }
#pragma unroll
    for (int s0 = 0; s0 < C; s0 += 16) {
#pragma unroll
      for (int i = 0; i < 8; ++i)
#pragma unroll
        for (int u = 0; u < DG; ++u)
          acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(kp[u][(s0 + 2 * i) * d32], b[s0 / 16 % PB][i], acc[u], 0, 0, 0);
      if (s0 + 16 * PB < C) load_v(item, s0 + 16 * PB);
    }
    if (col < vdim) {
#pragma unroll
      for (int u = 0; u < DG; ++u)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int d = (dt0 + u) * 32 + 8 * (r >> 2) + 4 * half + (r & 3);
          if (d < dim) dst[(long long)d * vdim + col] = acc[u][r];
        }
    }
  }
}

// add[c] becomes the state in front of chunk c; state becomes the one behind the last.
template <int W>
__global__ __launch_bounds__(256) void hgrn2_scan_kernel(float *__restrict__ state, float *__restrict__ add,
                                                         const float *__restrict__ decay, int rows, int vdim, int chunks,
                                                         bool fresh) {
  typedef float vec_t __attribute__((ext_vector_type(W)));
  const int cols = vdim / W;
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i >= (long long)rows * cols) return;
  const int row = (int)(i / cols);
  const long long o = (long long)row * vdim + W * (i - (long long)row * cols), step = (long long)rows * vdim;
  vec_t s = fresh ? (vec_t)(0.f) : *(const vec_t *)(state + o);
  constexpr int U = 8;
  vec_t x[U];
  float f[U];
  for (int c0 = 0; c0 < chunks; c0 += U) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = min(c0 + u, chunks - 1);
      x[u] = *(const vec_t *)(add + c * step + o);
      f[u] = decay[(long long)c * rows + row];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (c0 + u < chunks) {
        *(vec_t *)(add + (c0 + u) * step + o) = s;
        s = s * f[u] + x[u];
      }
  }
  *(vec_t *)(state + o) = s;
}

// The rows of one chunk of one head: eight wavefronts.  In LDS, per row and channel: q, k = 1 - f and L, the
// log2 of the gates' product from the beginning of the row's sub-chunk of 16 up to the row itself.
//   within eight rows    P[t][s] = sum_d q_t k_s 2^(L_t - L_s), a thread per pair
//   further apart        the same sum as a product of two matrices, q_t and k_s each decayed to a row between them:
//                        the end of a sub-chunk's first eight rows, or the end of the key's sub-chunk
//   o_t = sum_s P[t][s] v_s + (q_t 2^(L_t + what came before)) S, S the state in front of the chunk
// NT: tiles of 32 value columns per wavefront.
template <int C, int NT>
__global__ __launch_bounds__(512) void hgrn2_output_kernel(const Hgrn2Args a, int chunk0, const float *__restrict__ starts) {
  constexpr int NS = C / kSub, RT = C == 64 ? 2 : 1, CW = 8 / RT, PS = C + 4;
  constexpr int PR = C < 32 ? 32 : C;  // rows of P and of q that the 32-row tiles read
  extern __shared__ __attribute__((aligned(16))) float smem[];
  __shared__ float sq_s[8 * NT][32];
  __shared__ __attribute__((aligned(16))) float inv_s[32 * RT];
  const int dim = a.dim, vdim = a.vdim, d16 = (dim + 15) / 16 * 16, ds = d16 + 4;
  float *qs = smem, *ks = qs + PR * ds, *ls = ks + C * ds, *P = ls + C * ds, *tot = P + PR * PS;  // tot: [NS][d16]
  const int h = blockIdx.x % a.H, c = blockIdx.x / a.H, first = (chunk0 + c) * C;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n = lane & 31, half = lane >> 5;
  const int rt = wave % RT, cg = wave / RT, n_vt = (vdim + 31) / 32;
  const float *start = starts + ((long long)c * a.H + h) * dim * vdim;
  const float *v0 = a.raw + 2LL * a.H * dim + (long long)h * vdim;
  // what the last part needs of memory is asked for at the beginning: rows of the state (SB k steps of 8) and of the values
  constexpr int SB = NT == 1 ? 16 : 4, VB = C / 8;
  float xs[SB][4], xv[VB][4];
  auto load_s = [&](float (&y)[4], int col, int k0) {
#pragma unroll
    for (int i = 0; i < 4; ++i) y[i] = start[(long long)min(k0 + 4 * half + i, dim - 1) * vdim + col];
  };
  auto load_tile = [&](int vt) {
    const int col = min(vt * 32 + n, vdim - 1);
#pragma unroll
    for (int b = 0; b < SB; ++b)
      if (8 * b < d16) load_s(xs[b], col, 8 * b);
#pragma unroll
    for (int b = 0; b < VB; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) xv[b][i] = v0[(long long)min(first + 8 * b + 4 * half + i, a.T - 1) * a.stride + col];
  };
  float z[kSub], q[kSub];
  auto load_gates = [&](int it) {
    const int j = it / d16, i = h * dim + min(it - j * d16, dim - 1);
    load_column(a, (long long)a.H * dim + i, first + j * kSub, z);
    load_column(a, i, first + j * kSub, q);
  };
  // (loads come back in order: what is needed first goes first)
  if ((int)threadIdx.x < NS * d16) load_gates(threadIdx.x);
  if (cg < n_vt) load_tile(cg);
  float norm[NT];
#pragma unroll
  for (int u = 0; u < NT; ++u) norm[u] = a.norm[min((cg + CW * u) * 32 + n, vdim - 1)];

  for (int it = threadIdx.x; it < NS * d16; it += 512) {
    const int j = it / d16, d = it - j * d16;
    float L = 0.f;
    if (it >= 512) load_gates(it);
#pragma unroll
    for (int r = 0; r < kSub; ++r)
      qs[(j * kSub + r) * ds + d] = d < dim && first + j * kSub + r < a.T ? silu1(q[r]) : 0.f;
    if (d < dim) {
      walk_gates(a, h * dim + d, first + j * kSub, z, [&](int r, float f, float k) {
        L += __builtin_amdgcn_logf(fmaxf(f, 0x1p-40f));  // (smaller gates leave nothing of what was there before)
        ks[(j * kSub + r) * ds + d] = k;
        ls[(j * kSub + r) * ds + d] = L;
      });
    } else {
      for (int r = 0; r < kSub; ++r) ks[(j * kSub + r) * ds + d] = ls[(j * kSub + r) * ds + d] = 0.f;
    }
    tot[it] = L;
  }
  for (int it = C * ds + threadIdx.x; it < PR * ds; it += 512) qs[it] = 0.f;
  for (int it = threadIdx.x; it < PR * PS; it += 512) P[it] = 0.f;
  __syncthreads();

  // a wavefront takes eight rows; four lanes, a quarter of the channels each, take two rows against two
  for (int p = threadIdx.x; p < C * 8; p += 512) {
    const int quarter = p & 3, ti = p >> 4 & 3, si = p >> 2 & 3, b = p / 64 * 8, t = b + 2 * ti, s = b + 2 * si, n4 = d16 >> 4;
    if (si > ti) continue;
    const int o = quarter * 4 * n4;
    const f32x4 *qp[2], *lt[2], *kp[2], *lp[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      qp[u] = (const f32x4 *)(qs + (t + u) * ds + o);
      lt[u] = (const f32x4 *)(ls + (t + u) * ds + o);
      kp[u] = (const f32x4 *)(ks + (s + u) * ds + o);
      lp[u] = (const f32x4 *)(ls + (s + u) * ds + o);
    }
    f32x4 sum[2][2];
#pragma unroll
    for (int u = 0; u < 4; ++u) sum[u >> 1][u & 1] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int i = 0; i < n4; ++i) {
      f32x4 q[2], k[2], x[2], y[2];
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        q[u] = qp[u][i];
        k[u] = kp[u][i];
        x[u] = lt[u][i];
        y[u] = lp[u][i];
      }
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int v = 0; v < 2; ++v) {
          const f32x4 e = x[u] - y[v];
          sum[u][v] += q[u] * k[v] * f32x4{fast_exp2(e.x), fast_exp2(e.y), fast_exp2(e.z), fast_exp2(e.w)};
        }
    }
    float mine = 0.f;  // of the four pairs, the one this lane writes
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const f32x4 x = sum[u >> 1][u & 1];
      float total = (x.x + x.y) + (x.z + x.w);
      total += __shfl_xor(total, 1);
      total += __shfl_xor(total, 2);
      if (quarter == u) mine = total;
    }
    const int row = t + (quarter >> 1), col = s + (quarter & 1);
    if (col <= row) P[row * PS + col] = mine;
  }
  {
    // 16 rows against 16: two sub-chunks, or rows 8 .. 15 against the first eight of two sub-chunks at once
    // (of which the squares across the sub-chunks are not used)
    const int m = lane & 15, j4 = 4 * (lane >> 4);
    constexpr int apart = NS * (NS - 1) / 2;
    for (int item = wave; item < apart + (NS + 1) / 2; item += 8) {
      int bi = 1, bj = item;
      const bool within = item >= apart;
      if (within) {
        bi = bj = min(2 * (item - apart) + (m >> 3), NS - 1);
      } else {
        while (bj >= bi) bj -= bi++;
      }
      const int q0 = (bi * kSub + (within ? 8 + (m & 7) : m)) * ds + j4, k0 = (bj * kSub + (within ? m & 7 : m)) * ds + j4;
      const float *mid = within ? ls + (bj * kSub + 7) * ds + j4 : tot + bj * d16 + j4;  // where both decay to
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      for (int i = 0; i < d16; i += 16) {
        f32x4 q = *(const f32x4 *)(qs + q0 + i), k = *(const f32x4 *)(ks + k0 + i), eq = *(const f32x4 *)(ls + q0 + i);
        const f32x4 at = *(const f32x4 *)(mid + i);
        const f32x4 ek = at - *(const f32x4 *)(ls + k0 + i);
        if (within) {
          eq -= at;
        } else {
          for (int b = bj + 1; b < bi; ++b) eq += *(const f32x4 *)(tot + b * d16 + j4 + i);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          q[e] *= fast_exp2(eq[e]);
          k[e] *= fast_exp2(ek[e]);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q[e], k[e], acc, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = j4 + r;
        if (!within)
          P[(bi * kSub + row) * PS + bj * kSub + m] = acc[r];
        else if (row >> 3 == m >> 3 && 2 * (item - apart) + (m >> 3) < NS)
          P[(bi * kSub + 8 + (row & 7)) * PS + bi * kSub + (m & 7)] = acc[r];
      }
    }
  }
  __syncthreads();
  for (int it = threadIdx.x; it < NS * d16; it += 512) {
    const int j = it / d16, d = it - j * d16;
    float before = 0.f;
    for (int b = 0; b < j; ++b) before += tot[b * d16 + d];
#pragma unroll
    for (int r = 0; r < kSub; ++r) qs[(j * kSub + r) * ds + d] *= fast_exp2(ls[(j * kSub + r) * ds + d] + before);
  }
  __syncthreads();

  f32x16 acc[NT];
#pragma unroll
  for (int u = 0; u < NT; ++u) {
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[u][r] = 0.f;
    const int vt = cg + CW * u;
    if (vt < n_vt) {
      if (u > 0) {
        __builtin_amdgcn_sched_barrier(0);  // (the loads of one tile at a time: there are no registers for more)
        load_tile(vt);
      }
      const int col = min(vt * 32 + n, vdim - 1);
      const float *qp = qs + (rt * 32 + n) * ds + 4 * half;
      for (int k0 = 0; k0 < d16; k0 += 8 * SB) {
#pragma unroll
        for (int b = 0; b < SB; ++b) {
          if (k0 + 8 * b < d16) {
            const f32x4 q = *(const f32x4 *)(qp + k0 + 8 * b);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(q[i], xs[b][i], acc[u], 0, 0, 0);
            if (k0 + 8 * (b + SB) < d16) load_s(xs[b], col, k0 + 8 * (b + SB));
          }
        }
      }
      const float *pp = P + (rt * 32 + n) * PS + 4 * half;
#pragma unroll
      for (int b = 0; b < VB; ++b) {
        if (8 * b < rt * 32 + 32) {  // (columns of P behind the row's own 32-row tile are zeros)
          const f32x4 p = *(const f32x4 *)(pp + 8 * b);
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(p[i], xv[b][i], acc[u], 0, 0, 0);
        }
      }
    }
    // squares of this tile, summed over its 32 columns: with every exchange a lane keeps half of the rows it has
    float sq[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) sq[r] = vt < n_vt && vt * 32 + n < vdim ? acc[u][r] * acc[u][r] : 0.f;
#pragma unroll
    for (int x = 16, keep = 8; x > 1; x >>= 1, keep >>= 1) {
      const bool upper = n & x;
#pragma unroll
      for (int r = 0; r < keep; ++r) {
        const float other = __shfl_xor(upper ? sq[r] : sq[r + keep], x);
        sq[r] = (upper ? sq[r + keep] : sq[r]) + other;
      }
    }
    sq[0] += __shfl_xor(sq[0], 1);
    if (!(n & 1)) sq_s[wave * NT + u][8 * (n >> 3) + 4 * half + (n >> 1 & 3)] = sq[0];
  }
  __syncthreads();
  if (threadIdx.x < 32 * RT) {
    const int row_tile = threadIdx.x >> 5;
    float sum = 0.f;
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int u = 0; u < NT; ++u) sum += sq_s[(w * RT + row_tile) * NT + u][n];
    inv_s[threadIdx.x] = 1.f / sqrtf(sum / (float)vdim + a.eps);
  }
  __syncthreads();
#pragma unroll
  for (int r4 = 0; r4 < 4; ++r4) {
    const int t0 = rt * 32 + 8 * r4 + 4 * half;
    const f32x4 inv = *(const f32x4 *)(inv_s + t0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (t0 + r >= C || first + t0 + r >= a.T) continue;
#pragma unroll
      for (int u = 0; u < NT; ++u) {
        const int col = (cg + CW * u) * 32 + n;
        if (col < vdim) a.out[((long long)(first + t0 + r) * a.H + h) * vdim + col] = acc[u][4 * r4 + r] * inv[r] * norm[u];
      }
    }
  }
}

size_t output_lds(int c, int dim) {
  const int d16 = (dim + 15) / 16 * 16, ds = d16 + 4, pr = c < 32 ? 32 : c;
  return ((size_t)(pr + 2 * c) * ds + (size_t)pr * (c + 4) + (size_t)(c / kSub) * d16) * sizeof(float);
}

template <class K>
hipError_t allow_lds(K kernel) {
  return hipFuncSetAttribute((const void *)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, kMaxLds - 8192);
}

template <int C>
hipError_t launch_chunks(const Hgrn2Args &a, const Hgrn2Plan &p, float *scratch, hipStream_t stream) {
  const int all = (a.T + C - 1) / C, d32 = (a.dim + 31) / 32 * 32;
  const size_t state = (size_t)a.H * a.dim * a.vdim;
  float *add = scratch, *decay = scratch + (size_t)p.chunks * state;
  const size_t lds_a = ((size_t)C * d32 + (size_t)(C / kSub) * d32) * sizeof(float), lds_c = output_lds(C, a.dim);
  const int n_vt = (a.vdim + 31) / 32, cw = C == 64 ? 4 : 8;
  for (int c0 = 0; c0 < all; c0 += p.chunks) {
    const int n = all - c0 < p.chunks ? all - c0 : p.chunks;
    const dim3 grid((unsigned)(n * a.H));
#define SHAINET_LAUNCH_CHUNK(DG_)                                                                                \
  do {                                                                                                           \
    static const hipError_t e_ = allow_lds(hgrn2_chunk_kernel<C, DG_>);                                          \
    if (e_ != hipSuccess) return e_;                                                                             \
    hipLaunchKernelGGL((hgrn2_chunk_kernel<C, DG_>), grid, dim3(512), lds_a, stream, a, c0, add, decay);         \
  } while (0)
    if ((long long)n_vt * ((d32 / 32 + 1) / 2) >= 8)  // (an item for every wavefront)
      SHAINET_LAUNCH_CHUNK(2);
    else
      SHAINET_LAUNCH_CHUNK(1);
#undef SHAINET_LAUNCH_CHUNK
    const int w = a.vdim % 4 == 0 ? 4 : 1;
    const long long threads = (long long)(state / w);
    const dim3 scan((unsigned)((threads + 255) / 256));
    if (w == 4)
      hipLaunchKernelGGL(hgrn2_scan_kernel<4>, scan, dim3(256), 0, stream, a.state, add, decay, a.H * a.dim, a.vdim, n,
                         a.fresh && c0 == 0);
    else
      hipLaunchKernelGGL(hgrn2_scan_kernel<1>, scan, dim3(256), 0, stream, a.state, add, decay, a.H * a.dim, a.vdim, n,
                         a.fresh && c0 == 0);
#define SHAINET_LAUNCH_OUTPUT(NT_)                                                                               \
  do {                                                                                                           \
    static const hipError_t e_ = allow_lds(hgrn2_output_kernel<C, NT_>);                                         \
    if (e_ != hipSuccess) return e_;                                                                             \
    hipLaunchKernelGGL((hgrn2_output_kernel<C, NT_>), grid, dim3(512), lds_c, stream, a, c0, add);               \
  } while (0)
    if (n_vt <= cw)
      SHAINET_LAUNCH_OUTPUT(1);
    else if (n_vt <= 2 * cw)
      SHAINET_LAUNCH_OUTPUT(2);
    else
      SHAINET_LAUNCH_OUTPUT(4);
#undef SHAINET_LAUNCH_OUTPUT
    const hipError_t e = hipGetLastError();
    if (e != hipSuccess) return e;
  }
  return hipSuccess;
}

}  // namespace

bool plan_hgrn2(int T, int H, int dim, int vdim, Hgrn2Plan &p) {
  if (T < 1 || H < 1 || dim < 1 || vdim < 1 || dim > 4096 || vdim > 1024) return false;
  p.chunk = 0;
  p.chunks = 0;
  p.scratch_floats = 0;
  if (T <= 16) return true;
  for (int c : {64, 32, 16}) {
    if (output_lds(c, dim) > (size_t)(kMaxLds - 8192) || (vdim + 31) / 32 > (c == 64 ? 16 : 32)) continue;
    const long long all = ((long long)T + c - 1) / c;
    p.chunk = c;
    p.chunks = all < kChunksAtOnce ? (int)all : kChunksAtOnce;
    if ((long long)p.chunks * H > 0x7fffffff || (long long)H * dim * vdim > 0x7fffffff) return false;
    p.scratch_floats = (size_t)p.chunks * ((size_t)H * dim * vdim + (size_t)H * dim);
    break;
  }
  return true;
}

hipError_t launch_hgrn2(const Hgrn2Args &a, const Hgrn2Plan &p, float *scratch, hipStream_t stream) {
  Hgrn2Plan want;
  if (!a.raw || !a.f_bias || !a.lower || !a.norm || !a.state || !a.out || !plan_hgrn2(a.T, a.H, a.dim, a.vdim, want) ||
      want.chunk != p.chunk || want.chunks != p.chunks || (p.scratch_floats && !scratch) ||
      a.stride < 2LL * a.H * a.dim + (long long)a.H * a.vdim)
    return hipErrorInvalidValue;
  if (p.chunk == 64) return launch_chunks<64>(a, p, scratch, stream);
  if (p.chunk == 32) return launch_chunks<32>(a, p, scratch, stream);
  if (p.chunk == 16) return launch_chunks<16>(a, p, scratch, stream);
  // (16-byte pieces of v and of the state where every row of both begins on 16 bytes)
  const int w = a.vdim % 4 == 0 && a.stride % 4 == 0 && (2LL * a.H * a.dim) % 4 == 0 ? 4 : 1;
  const int cols = a.vdim / w, groups = 1024 / cols;
  const bool held = (a.dim + groups - 1) / groups <= (w == 4 ? kHeldRows<4> : kHeldRows<1>);
  const size_t lds = ((size_t)(3 * a.dim + 3) / 4 * 4 + (size_t)groups * a.vdim) * sizeof(float);
#define SHAINET_LAUNCH_STEP(W_, HELD_)                                                                           \
  do {                                                                                                           \
    static const hipError_t e_ = allow_lds(hgrn2_step_kernel<W_, HELD_>);                                        \
    if (e_ != hipSuccess) return e_;                                                                             \
    hipLaunchKernelGGL((hgrn2_step_kernel<W_, HELD_>), dim3((unsigned)a.H), dim3(1024), lds, stream, a);         \
  } while (0)
  if (w == 4 && held)
    SHAINET_LAUNCH_STEP(4, true);
  else if (w == 4)
    SHAINET_LAUNCH_STEP(4, false);
  else if (held)
    SHAINET_LAUNCH_STEP(1, true);
  else
    SHAINET_LAUNCH_STEP(1, false);
#undef SHAINET_LAUNCH_STEP
  return hipGetLastError();
}

}  // namespace shainet
