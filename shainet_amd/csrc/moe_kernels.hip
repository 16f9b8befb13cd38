// A mixture of experts on gfx950 (moe_kernels.hpp says what is computed), fp32.
#include "moe_kernels.hpp"

#include <math.h>
#include <stdint.h>

namespace shainet {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

#define ORDER_LDS_AND_MFMA() __builtin_amdgcn_sched_barrier(0x7)

__device__ __forceinline__ float swiglu1(float g, float u) { return g / (1.f + expf(-g)) * u; }
__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
  return v;
}

// The largest of v over the wavefront and, among equal ones, the smallest index.
__device__ __forceinline__ void wave_best(float &v, int &i) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(v, o);
    const int oi = __shfl_xor(i, o);
    if (ov > v || (ov == v && oi < i)) {
      v = ov;
      i = oi;
    }
  }
}

// One wavefront chooses for one token.  logits: [n] (global); s, c: n floats of LDS each, best: m.groups floats
// of LDS.  ids, weights: m.top entries each, written by lane 0 (LDS or global).
__device__ __forceinline__ void choose(const MoeShape &m, const float *logits, const float *correction, float *s, float *c,
                                       float *best, int *ids, float *weights) {
  const int n = m.experts + m.identity, lane = threadIdx.x & 63, per = n / m.groups;
  float mx = -INFINITY;
  for (int i = lane; i < n; i += 64) mx = fmaxf(mx, logits[i]);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o));
  float sum = 0.f;
  for (int i = lane; i < n; i += 64) {
    const float e = expf(logits[i] - mx);
    s[i] = e;
    sum += e;
  }
  sum = wave_sum(sum);
  for (int i = lane; i < n; i += 64) {
    const float p = s[i] / sum;
    s[i] = p;
    c[i] = p + correction[i];
  }
  __builtin_amdgcn_wave_barrier();
  __threadfence_block();
  if (m.groups > 1) {
    for (int g = lane; g < m.groups; g += 64) {
      float b = -INFINITY;
      for (int i = 0; i < per; ++i) b = fmaxf(b, c[g * per + i]);
      best[g] = b;
    }
    __threadfence_block();
    for (int k = 0; k < m.keep; ++k) {  // a kept group's entry becomes NaN: no comparison takes it again
      float v = -INFINITY;
      int at = 0x7fffffff;
      for (int g = lane; g < m.groups; g += 64) {
        const float b = best[g];
        if (b > v || (b == v && g < at)) {
          v = b;
          at = g;
        }
      }
      wave_best(v, at);
      if (at < m.groups && lane == 0) best[at] = NAN;
      __threadfence_block();
    }
    for (int i = lane; i < n; i += 64) {
      const float b = best[i / per];
      if (b == b) c[i] = NAN;
    }
    __threadfence_block();
  }
  float total = 0.f;
  for (int k = 0; k < m.top; ++k) {
    float v = -INFINITY;
    int at = 0x7fffffff;
    for (int i = lane; i < n; i += 64) {
      const float x = c[i];
      if (x > v || (x == v && i < at)) {
        v = x;
        at = i;
      }
    }
    wave_best(v, at);
    at = min(at, n - 1);  // (only with logits that are no numbers)
    const float p = s[at];
    total += p;
    if (lane == 0) {
      ids[k] = at;
      weights[k] = p;
      c[at] = NAN;
    }
    __threadfence_block();
  }
  for (int k = lane; k < m.top; k += 64) weights[k] = weights[k] / (total + 1e-20f) * m.scale;
  __threadfence_block();
}

// ---- a few tokens ------------------------------------------------------------------------------
// this lane's share of a . b, n floats
template <bool VEC>
__device__ __forceinline__ float dot_lane(const float *a, const float *b, int n) {
  const int lane = threadIdx.x & 63;
  float s = 0.f;
  if constexpr (VEC) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const int n4 = n >> 2;
    int i = lane;
    for (; i + 192 < n4; i += 256) {
      f32x4 x[4], y[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        x[u] = __builtin_nontemporal_load((const f32x4 *)a + i + 64 * u);
        y[u] = ((const f32x4 *)b)[i + 64 * u];
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) acc += x[u] * y[u];
    }
    for (; i < n4; i += 64) acc += ((const f32x4 *)a)[i] * ((const f32x4 *)b)[i];
    s = (acc.x + acc.y) + (acc.z + acc.w);
  } else {
    for (int i = lane; i < n; i += 64) s += a[i] * b[i];
  }
  return s;
}

// logits[t][n] = router row n . h row t: a wavefront each
template <bool VEC>
__global__ __launch_bounds__(256) void moe_logits_kernel(const float *__restrict__ h, const float *__restrict__ router,
                                                         float *__restrict__ logits, int n, int d) {
  const int i = blockIdx.x * 4 + (threadIdx.x >> 6), t = blockIdx.y;
  if (i >= n) return;
  const float s = wave_sum(dot_lane<VEC>(router + (long long)i * d, h + (long long)t * d, d));
  if ((threadIdx.x & 63) == 0) logits[(long long)t * n + i] = s;
}

// hidden[t][slot][j] = silu(gate row j . h) * (up row j . h) of the slot's expert; slot `top` is the shared one.
// Every workgroup works the choice out again from the logits (a launch of its own would take longer);
// the first one of each token leaves it for moe_down_kernel.
template <bool VEC>
__global__ __launch_bounds__(256) void moe_up_kernel(MoeShape m, MoeTensors w, const float *__restrict__ h,
                                                     const float *__restrict__ logits, float *__restrict__ hidden,
                                                     int width, int *__restrict__ ids_out, float *__restrict__ weights_out) {
  extern __shared__ float smem[];  // s, c, best, weights, then ids
  const int n = m.experts + m.identity, slot = blockIdx.y, t = blockIdx.z;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const bool shared = slot == m.top;
  const int ff = shared ? m.shared_ff : m.ff;
  const int j = blockIdx.x * 4 + wave;
  const float *gate = w.shared_gate_up;
  if (!shared) {
    float *weights = smem + 2 * n + m.groups;
    int *ids = (int *)(weights + m.top);
    if (wave == 0) choose(m, logits + (long long)t * n, w.correction, smem, smem + n, smem + 2 * n, ids, weights);
    __syncthreads();
    if (blockIdx.x == 0 && slot == 0)
      for (int k = threadIdx.x; k < m.top; k += 256) {
        ids_out[t * m.top + k] = ids[k];
        weights_out[t * m.top + k] = weights[k];
      }
    const int e = ids[slot];
    if (e >= m.experts) return;
    gate = w.gate_up + (long long)e * 2 * m.ff * m.d;
  }
  if (j >= ff) return;
  const float *x = h + (long long)t * m.d;
  float g, u;
  if constexpr (VEC) {  // both rows in flight together
    const float *gp = gate + (long long)j * m.d, *up = gate + (long long)(ff + j) * m.d;
    f32x4 ga = {0.f, 0.f, 0.f, 0.f}, ua = ga;
    const int n4 = m.d >> 2;
    for (int i0 = lane; i0 < n4; i0 += 256) {
      f32x4 gv[4], uv[4], xv[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const int i = min(i0 + 64 * k, n4 - 1);
        gv[k] = __builtin_nontemporal_load((const f32x4 *)gp + i);
        uv[k] = __builtin_nontemporal_load((const f32x4 *)up + i);
        xv[k] = ((const f32x4 *)x)[i];
      }
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if (i0 + 64 * k < n4) {
          ga += gv[k] * xv[k];
          ua += uv[k] * xv[k];
        }
    }
    g = (ga.x + ga.y) + (ga.z + ga.w);
    u = (ua.x + ua.y) + (ua.z + ua.w);
  } else {
    g = dot_lane<false>(gate + (long long)j * m.d, x, m.d);
    u = dot_lane<false>(gate + (long long)(ff + j) * m.d, x, m.d);
  }
  g = wave_sum(g);
  u = wave_sum(u);
  if (lane == 0) hidden[((long long)t * (m.top + 1) + slot) * width + j] = swiglu1(g, u);
}

// y[t][j]: a wavefront per output, over all slots
template <bool VEC>
__global__ __launch_bounds__(256) void moe_down_kernel(MoeShape m, MoeTensors w, const float *__restrict__ h,
                                                       const float *__restrict__ hidden, int width,
                                                       const int *__restrict__ ids, const float *__restrict__ weights,
                                                       float *__restrict__ y) {
  const int j = blockIdx.x * 4 + (threadIdx.x >> 6), t = blockIdx.y;
  if (j >= m.d) return;
  const float *hid = hidden + (long long)t * (m.top + 1) * width;
  float s = 0.f, same = 0.f;
  for (int k = 0; k < m.top; ++k) {
    const int e = ids[t * m.top + k];
    const float wk = weights[t * m.top + k];
    if (e >= m.experts)
      same += wk;
    else
      s += wk * dot_lane<VEC>(w.down + ((long long)e * m.d + j) * m.ff, hid + (long long)k * width, m.ff);
  }
  if (m.shared_ff)
    s += dot_lane<VEC>(w.shared_down + (long long)j * m.shared_ff, hid + (long long)m.top * width, m.shared_ff);
  s = wave_sum(s);
  if ((threadIdx.x & 63) == 0) y[(long long)t * m.d + j] = s + same * h[(long long)t * m.d + j];
}

// ---- many tokens -------------------------------------------------------------------------------
// A wavefront per token chooses; a chosen expert's counter gives the token's place among its rows.
__global__ __launch_bounds__(256) void moe_select_kernel(MoeShape m, const float *__restrict__ correction,
                                                         const float *__restrict__ logits, int T, int *__restrict__ ids,
                                                         float *__restrict__ weights, int *__restrict__ rank, int *counts) {
  extern __shared__ float smem[];
  const int n = m.experts + m.identity, wave = threadIdx.x >> 6, t = blockIdx.x * 4 + wave;
  if (t >= T) return;
  float *s = smem + wave * (2 * n + m.groups + 2 * m.top), *wl = s + 2 * n + m.groups;
  int *il = (int *)(wl + m.top);
  choose(m, logits + (long long)t * n, correction, s, s + n, s + 2 * n, il, wl);
  for (int k = threadIdx.x & 63; k < m.top; k += 64) {
    const int e = il[k];
    ids[t * m.top + k] = e;
    weights[t * m.top + k] = wl[k];
    rank[t * m.top + k] = e < m.experts ? atomicAdd(counts + e, 1) : 0;
  }
}

// Where the experts' rows and tiles begin; clears the counters for the next call.
__global__ __launch_bounds__(1024) void moe_offsets_kernel(int experts, int tile, int *counts, int *__restrict__ off,
                                                           int *__restrict__ tile_off) {
  __shared__ int a[1024], b[1024];
  const int e = threadIdx.x;
  const int c = e < experts ? counts[e] : 0;
  a[e] = c;
  b[e] = (c + tile - 1) / tile;
  __syncthreads();
  for (int o = 1; o < 1024; o <<= 1) {
    const int x = e >= o ? a[e - o] : 0, y = e >= o ? b[e - o] : 0;
    __syncthreads();
    a[e] += x;
    b[e] += y;
    __syncthreads();
  }
  if (e < experts) {
    off[e + 1] = a[e];
    tile_off[e + 1] = b[e];
    counts[e] = 0;
  }
  if (e == 0) off[0] = tile_off[0] = 0;
}

__global__ __launch_bounds__(256) void moe_scatter_kernel(int n, int top, int experts, const int *__restrict__ ids,
                                                          const int *__restrict__ rank, const int *__restrict__ off,
                                                          int *__restrict__ rows) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const int e = ids[i];
  if (e < experts) rows[off[e] + rank[i]] = i / top;
}

// Rows of x (gathered, or as they lie) times the matrices of their groups, [N, K] (SWIGLU: [2N, K], gate
// rows and up rows): the layout of a product whose operands both run along K.  A workgroup of four
// wavefronts takes TM rows and TN matrix rows; both tiles go global memory -> registers -> LDS, two stages,
// row stride 36 floats, and are read 16 bytes at a time down a column of rows.  v_mfma_f32_32x32x2: MFMA i of
// a k step of 8 takes k = 8 s + 4 half + i on both sides.  With SWIGLU even blocks of 32 matrix rows are gates and
// the odd ones behind them their partners, so that a lane holds both halves of its outputs.
struct GroupedArgs {
  const float *x;
  const int *gather;       // row r of the product is row gather[r] of x; null: row r
  const int *off, *tile_off;  // [groups + 1]; null: one group of `rows` rows
  const float *w;
  float *y;                // [rows, N]
  int rows, groups, K, N;
};
template <int TM, bool SWIGLU, bool VEC>
__global__ __launch_bounds__(256, 2) void moe_product_kernel(const GroupedArgs g) {
  constexpr int TK = 32, AS = TK + 4, RW = TM / 32, CW = 4 / RW, NB = TM == 128 ? 4 : 2, TN = 32 * NB * CW;
  constexpr int NA = TM / 32, NW = TN / 32;  // 16-byte pieces per thread and stage
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float *As = smem, *Bs = smem + 2 * TM * AS;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  int grp = 0, tm = blockIdx.x, r0 = 0, r1 = g.rows;
  if (g.tile_off) {
    if (tm >= g.tile_off[g.groups]) return;
    for (int e0 = 0; e0 < g.groups; e0 += 64)
      grp += (int)__popcll(__ballot(e0 + lane < g.groups && tm >= g.tile_off[min(e0 + lane, g.groups - 1) + 1]));
    grp = __builtin_amdgcn_readfirstlane(grp);
    tm -= g.tile_off[grp];
    r0 = g.off[grp];
    r1 = g.off[grp + 1];
  }
  const int m0 = r0 + tm * TM;
  if (m0 >= r1) return;
  const int K = g.K, N = g.N, o0 = blockIdx.y * (SWIGLU ? TN / 2 : TN);
  const float *w = g.w + (long long)grp * (SWIGLU ? 2 : 1) * N * K;

  const int srow = threadIdx.x >> 3, k4 = 4 * (threadIdx.x & 7);
  const float *ap[NA], *bp[NW];
#pragma unroll
  for (int u = 0; u < NA; ++u) {
    const int r = min(m0 + srow + 32 * u, r1 - 1);
    ap[u] = g.x + (long long)(g.gather ? g.gather[r] : r) * K;
  }
#pragma unroll
  for (int u = 0; u < NW; ++u) {  // u is the block of 32 matrix rows
    const int r = SWIGLU ? (u & 1) * N + min(o0 + (u >> 1) * 32 + srow, N - 1) : min(o0 + 32 * u + srow, N - 1);
    bp[u] = w + (long long)r * K;
  }
  f32x4 sa[NA], sb[NW];
  auto piece = [&](const float *p, int k) {
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if constexpr (VEC) {
      if (k < K) v = *(const f32x4 *)(p + k);
    } else {
      if (k < K) v.x = p[k];
      if (k + 1 < K) v.y = p[k + 1];
      if (k + 2 < K) v.z = p[k + 2];
      if (k + 3 < K) v.w = p[k + 3];
    }
    return v;
  };
  auto load = [&](int k0) {
#pragma unroll
    for (int u = 0; u < NA; ++u) sa[u] = piece(ap[u], k0 + k4);
#pragma unroll
    for (int u = 0; u < NW; ++u) sb[u] = piece(bp[u], k0 + k4);
  };
  auto park = [&](int buf) {
#pragma unroll
    for (int u = 0; u < NA; ++u) *(f32x4 *)(As + (buf * TM + srow + 32 * u) * AS + k4) = sa[u];
#pragma unroll
    for (int u = 0; u < NW; ++u) *(f32x4 *)(Bs + (buf * TN + srow + 32 * u) * AS + k4) = sb[u];
  };
  const int n = lane & 31, half = lane >> 5, rw = wave % RW, cw = wave / RW;
  const float *af_p = As + (rw * 32 + n) * AS + 4 * half, *bf_p = Bs + (cw * NB * 32 + n) * AS + 4 * half;
  f32x4 af[2], bf[2][NB];
  auto fetch = [&](int par, int buf, int s) {
    af[par] = *(const f32x4 *)(af_p + buf * TM * AS + 8 * s);
#pragma unroll
    for (int b = 0; b < NB; ++b) bf[par][b] = *(const f32x4 *)(bf_p + (buf * TN + b * 32) * AS + 8 * s);
  };
  f32x16 acc[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[b][r] = 0.f;

  const int steps = (K + TK - 1) / TK;
  load(0);
  park(0);
  if (steps > 1) load(TK);
  __syncthreads();
  fetch(0, 0, 0);
  for (int kt = 0; kt < steps; ++kt) {
    const int buf = kt & 1;
    const bool more = kt + 1 < steps;
#pragma unroll
    for (int s = 0; s < TK / 8; ++s) {
      const int cur = s & 1, nxt = cur ^ 1;
      if (s + 1 < TK / 8) {
        fetch(nxt, buf, s + 1);
      } else {
        if (more) park(buf ^ 1);
        __syncthreads();
        if (kt + 2 < steps) load((kt + 2) * TK);
        if (more) fetch(nxt, buf ^ 1, 0);
      }
      ORDER_LDS_AND_MFMA();
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int b = 0; b < NB; ++b) acc[b] = __builtin_amdgcn_mfma_f32_32x32x2f32(af[cur][i], bf[cur][b][i], acc[b], 0, 0, 0);
      ORDER_LDS_AND_MFMA();
    }
  }
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int row = m0 + rw * 32 + 8 * (r >> 2) + 4 * half + (r & 3);
    if (row >= r1) continue;
    float *yr = g.y + (long long)row * N;
    if constexpr (SWIGLU) {
#pragma unroll
      for (int b = 0; b < NB; b += 2) {
        const int col = o0 + ((cw * NB + b) >> 1) * 32 + n;
        if (col < N) yr[col] = swiglu1(acc[b][r], acc[b + 1][r]);
      }
    } else {
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        const int col = o0 + (cw * NB + b) * 32 + n;
        if (col < N) yr[col] = acc[b][r];
      }
    }
  }
}

// y[t] (+)= sum over the slots of weight * the expert's row, in the slots' order
template <int W>
__global__ __launch_bounds__(256) void moe_combine_kernel(MoeShape m, const float *__restrict__ h,
                                                          const float *__restrict__ rows_y, const int *__restrict__ ids,
                                                          const float *__restrict__ weights, const int *__restrict__ rank,
                                                          const int *__restrict__ off, int add, float *__restrict__ y) {
  typedef float vec_t __attribute__((ext_vector_type(W)));
  const int t = blockIdx.x, n = m.d / W;
  for (int i = blockIdx.y * 256 + threadIdx.x; i < n; i += gridDim.y * 256) {
    vec_t s = add ? ((const vec_t *)(y + (long long)t * m.d))[i] : (vec_t)(0.f);
    for (int k = 0; k < m.top; ++k) {
      const int e = ids[t * m.top + k];
      const float *src = e < m.experts ? rows_y + (long long)(off[e] + rank[t * m.top + k]) * m.d : h + (long long)t * m.d;
      s += weights[t * m.top + k] * ((const vec_t *)src)[i];
    }
    ((vec_t *)(y + (long long)t * m.d))[i] = s;
  }
}

// floats to the next multiple of 16 bytes' worth
size_t up4(size_t n) { return (n + 3) / 4 * 4; }

struct ManyLayout {
  size_t logits, weights, ids, rank, off, tile_off, rows, hidden, rows_y, total;
};
ManyLayout many_layout(const MoeShape &m, int T) {
  ManyLayout l;
  const size_t n = (size_t)m.experts + m.identity, slots = (size_t)T * m.top;
  size_t at = 0;
  auto take = [&](size_t k) {
    const size_t here = at;
    at += up4(k);
    return here;
  };
  l.logits = take((size_t)T * n);
  l.weights = take(slots);
  l.ids = take(slots);
  l.rank = take(slots);
  l.off = take((size_t)m.experts + 1);
  l.tile_off = take((size_t)m.experts + 1);
  l.rows = take(slots);
  l.hidden = take(slots * m.ff);
  l.rows_y = take(slots * m.d);
  l.total = at;
  return l;
}

template <int TM>
hipError_t launch_product_tm(const GroupedArgs &g, bool swiglu, hipStream_t stream) {
  constexpr int TN = TM == 32 ? 256 : 128;
  const long long tiles = g.tile_off ? (long long)g.rows / TM + (g.groups < g.rows ? g.groups : g.rows) : ((long long)g.rows + TM - 1) / TM;
  const int cols = swiglu ? TN / 2 : TN, ny = (g.N + cols - 1) / cols;
  if (tiles < 1 || tiles > 0x7fffffff || ny > 65535) return hipErrorInvalidValue;
  const dim3 grid((unsigned)tiles, (unsigned)ny);
  const size_t lds = (size_t)2 * (TM + TN) * 36 * sizeof(float);
  const bool vec = (g.K & 3) == 0 && !(((uintptr_t)g.x | (uintptr_t)g.w) & 15);
#define SHAINET_LAUNCH_PRODUCT(S_, V_)                                                                           \
  do {                                                                                                           \
    static const hipError_t e_ = hipFuncSetAttribute((const void *)moe_product_kernel<TM, S_, V_>,               \
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);    \
    if (e_ != hipSuccess) return e_;                                                                             \
    hipLaunchKernelGGL((moe_product_kernel<TM, S_, V_>), grid, dim3(256), lds, stream, g);                       \
  } while (0)
  if (swiglu && vec)
    SHAINET_LAUNCH_PRODUCT(true, true);
  else if (swiglu)
    SHAINET_LAUNCH_PRODUCT(true, false);
  else if (vec)
    SHAINET_LAUNCH_PRODUCT(false, true);
  else
    SHAINET_LAUNCH_PRODUCT(false, false);
#undef SHAINET_LAUNCH_PRODUCT
  return hipGetLastError();
}

hipError_t launch_product(const GroupedArgs &g, int tm, bool swiglu, hipStream_t stream) {
  return tm == 128 ? launch_product_tm<128>(g, swiglu, stream)
         : tm == 64 ? launch_product_tm<64>(g, swiglu, stream)
                    : launch_product_tm<32>(g, swiglu, stream);
}

}  // namespace

bool moe_shape_ok(const MoeShape &m) {
  const int n = m.experts + m.identity;
  return m.d > 0 && m.ff > 0 && m.experts > 0 && m.identity >= 0 && n <= kMaxRouterOutputs && m.groups > 0 && n % m.groups == 0 &&
         m.keep > 0 && m.keep <= m.groups && m.top > 0 && m.top <= m.keep * (n / m.groups) && m.shared_ff >= 0;
}

size_t moe_few_floats(const MoeShape &m, int T) {
  const size_t width = up4(m.ff > m.shared_ff ? m.ff : m.shared_ff);
  return up4((size_t)T * (m.experts + m.identity)) + 2 * up4((size_t)T * m.top) + (size_t)T * (m.top + 1) * width;
}

hipError_t launch_moe_few(const MoeShape &m, const MoeTensors &w, const float *h, float *y, int T, float *scratch,
                          hipStream_t stream) {
  if (!moe_shape_ok(m) || T < 1 || T > kMoeFewTokens || !h || !y || !scratch || !w.router || !w.correction || !w.gate_up ||
      !w.down || (m.shared_ff && (!w.shared_gate_up || !w.shared_down)))
    return hipErrorInvalidValue;
  const int n = m.experts + m.identity, most = m.ff > m.shared_ff ? m.ff : m.shared_ff, width = (int)up4(most);
  const int slots = m.top + (m.shared_ff ? 1 : 0);
  float *logits = scratch, *weights = logits + up4((size_t)T * n);
  int *ids = (int *)(weights + up4((size_t)T * m.top));
  float *hidden = (float *)ids + up4((size_t)T * m.top);
  const dim3 g1((unsigned)((n + 3) / 4), (unsigned)T), g2((unsigned)((most + 3) / 4), (unsigned)slots, (unsigned)T),
      g3((unsigned)((m.d + 3) / 4), (unsigned)T);
  const size_t lds = (size_t)(2 * n + m.groups + 2 * m.top) * sizeof(float);
  if (slots > 65535) return hipErrorInvalidValue;
  const bool vec_d = (m.d & 3) == 0, vec_ff = ((m.ff | m.shared_ff) & 3) == 0;
  if (vec_d) {
    hipLaunchKernelGGL(moe_logits_kernel<true>, g1, dim3(256), 0, stream, h, w.router, logits, n, m.d);
    hipLaunchKernelGGL(moe_up_kernel<true>, g2, dim3(256), lds, stream, m, w, h, logits, hidden, width, ids, weights);
  } else {
    hipLaunchKernelGGL(moe_logits_kernel<false>, g1, dim3(256), 0, stream, h, w.router, logits, n, m.d);
    hipLaunchKernelGGL(moe_up_kernel<false>, g2, dim3(256), lds, stream, m, w, h, logits, hidden, width, ids, weights);
  }
  if (vec_ff)
    hipLaunchKernelGGL(moe_down_kernel<true>, g3, dim3(256), 0, stream, m, w, h, hidden, width, ids, weights, y);
  else
    hipLaunchKernelGGL(moe_down_kernel<false>, g3, dim3(256), 0, stream, m, w, h, hidden, width, ids, weights, y);
  return hipGetLastError();
}

size_t moe_many_floats(const MoeShape &m, int T) { return many_layout(m, T).total; }

hipError_t launch_moe_many(const MoeShape &m, const MoeTensors &w, const float *h, float *y, bool add_to_y, int T,
                           float *scratch, int *counts, hipStream_t stream) {
  if (!moe_shape_ok(m) || T < 1 || (long long)T * m.top > 0x3fffffff || !h || !y || !scratch || !counts || !w.router ||
      !w.correction || !w.gate_up || !w.down)
    return hipErrorInvalidValue;
  const ManyLayout l = many_layout(m, T);
  const int n = m.experts + m.identity, slots = T * m.top;
  float *logits = scratch + l.logits, *weights = scratch + l.weights, *hidden = scratch + l.hidden, *rows_y = scratch + l.rows_y;
  int *ids = (int *)(scratch + l.ids), *rank = (int *)(scratch + l.rank), *off = (int *)(scratch + l.off),
      *tile_off = (int *)(scratch + l.tile_off), *rows = (int *)(scratch + l.rows);
  GroupedArgs r = {};
  r.x = h;
  r.w = w.router;
  r.y = logits;
  r.rows = T;
  r.groups = 1;
  r.K = m.d;
  r.N = n;
  hipError_t e = launch_product(r, 32, false, stream);
  if (e != hipSuccess) return e;
  const size_t lds = (size_t)4 * (2 * n + m.groups + 2 * m.top) * sizeof(float);
  if (lds > 64 * 1024) return hipErrorInvalidValue;
  hipLaunchKernelGGL(moe_select_kernel, dim3((unsigned)((T + 3) / 4)), dim3(256), lds, stream, m, w.correction, logits, T, ids,
                     weights, rank, counts);
  const int per_expert = slots / m.experts, tm = per_expert > 96 ? 128 : per_expert > 32 ? 64 : 32;
  hipLaunchKernelGGL(moe_offsets_kernel, dim3(1), dim3(1024), 0, stream, m.experts, tm, counts, off, tile_off);
  hipLaunchKernelGGL(moe_scatter_kernel, dim3((unsigned)((slots + 255) / 256)), dim3(256), 0, stream, slots, m.top, m.experts,
                     ids, rank, off, rows);
  GroupedArgs g = {};
  g.x = h;
  g.gather = rows;
  g.off = off;
  g.tile_off = tile_off;
  g.w = w.gate_up;
  g.y = hidden;
  g.rows = slots;
  g.groups = m.experts;
  g.K = m.d;
  g.N = m.ff;
  if ((e = launch_product(g, tm, true, stream)) != hipSuccess) return e;
  g.x = hidden;
  g.gather = nullptr;
  g.w = w.down;
  g.y = rows_y;
  g.K = m.ff;
  g.N = m.d;
  if ((e = launch_product(g, tm, false, stream)) != hipSuccess) return e;
  const bool vec = (m.d & 3) == 0;
  const int per = vec ? 1024 : 256;
  const dim3 grid((unsigned)T, (unsigned)((m.d + per - 1) / per));
  if (vec)
    hipLaunchKernelGGL(moe_combine_kernel<4>, grid, dim3(256), 0, stream, m, h, rows_y, ids, weights, rank, off, add_to_y ? 1 : 0, y);
  else
    hipLaunchKernelGGL(moe_combine_kernel<1>, grid, dim3(256), 0, stream, m, h, rows_y, ids, weights, rank, off, add_to_y ? 1 : 0, y);
  return hipGetLastError();
}

}  // namespace shainet
