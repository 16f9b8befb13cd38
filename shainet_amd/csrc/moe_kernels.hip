// A mixture of experts on gfx950 (moe_kernels.hpp says what is computed), fp32.
#include "moe_kernels.hpp"

#include <math.h>
#include <stdint.h>
#include <stdlib.h>

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
  if (n <= 64) {
    // a lane per output: who comes before whom is counted instead of searched for round by round
    const bool in = lane < n;
    const float z = in ? logits[lane] : -INFINITY, corr = in ? correction[lane] : 0.f;
    float top_z = z;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) top_z = fmaxf(top_z, __shfl_xor(top_z, o));
    const float e = in ? expf(z - top_z) : 0.f;
    const float p = e / wave_sum(e), x = p + corr;
    bool open = in;
    if (m.groups > 1) {
      if (in) c[lane] = x;
      __threadfence_block();
      const int mine = (in ? lane : 0) / per;
      float gb = -INFINITY;
#pragma unroll 4
      for (int i = 0; i < per; ++i) gb = fmaxf(gb, c[mine * per + i]);
      if (in && lane == mine * per) best[mine] = gb;
      __threadfence_block();
      int before = 0;
#pragma unroll 4
      for (int g = 0; g < m.groups; ++g) {
        const float v = best[g];
        before += v > gb || (v == gb && g < mine) ? 1 : 0;
      }
      open = in && before < m.keep;
    }
    if (in) s[lane] = open ? x : -INFINITY;
    __threadfence_block();
    int before = 0;
#pragma unroll 8
    for (int k = 0; k < n; ++k) {
      const float v = s[k];
      before += v > x || (v == x && k < lane) ? 1 : 0;
    }
    const bool chosen = open && before < m.top;
    const float total = wave_sum(chosen ? p : 0.f);
    for (int k = lane; k < m.top; k += 64) {  // (only with logits that are no numbers would an entry stay like this)
      ids[k] = 0;
      weights[k] = 0.f;
    }
    __threadfence_block();
    if (chosen) {
      ids[before] = lane;
      weights[before] = p / (total + 1e-20f) * m.scale;
    }
    __threadfence_block();
    return;
  }
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
// A wavefront per output; blockIdx.x: the shared expert's outputs, then slot 0's, slot 1's ...  Every workgroup
// of a slot works the choice out again from the logits (a launch of its own would take longer) with one
// wavefront while the others bring h into LDS; the first one leaves it for moe_down_kernel.
template <bool VEC>
__global__ __launch_bounds__(256) void moe_up_kernel(MoeShape m, MoeTensors w, const float *__restrict__ h,
                                                     const float *__restrict__ logits, float *__restrict__ hidden,
                                                     int width, int shared_blocks, int slot_blocks,
                                                     int *__restrict__ ids_out, float *__restrict__ weights_out) {
  extern __shared__ __attribute__((aligned(16))) float smem[];  // h, s, c, best, weights, ids
  const int n = m.experts + m.identity, t = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const bool shared = (int)blockIdx.x < shared_blocks;
  const int slot = shared ? m.top : ((int)blockIdx.x - shared_blocks) / slot_blocks;
  const int j = (shared ? (int)blockIdx.x : ((int)blockIdx.x - shared_blocks) - slot * slot_blocks) * 4 + wave;
  const int ff = shared ? m.shared_ff : m.ff;
  const float *row = h + (long long)t * m.d;
  float *xs = smem;
  if (wave > 0) {
    if constexpr (VEC) {
      for (int i = threadIdx.x - 64; i < m.d >> 2; i += 192) ((f32x4 *)xs)[i] = ((const f32x4 *)row)[i];
    } else {
      for (int i = threadIdx.x - 64; i < m.d; i += 192) xs[i] = row[i];
    }
  } else if (shared) {
    // (nothing to choose)
  } else {
    float *s = smem + (m.d + 3) / 4 * 4, *weights = s + 2 * n + m.groups;
    int *ids = (int *)(weights + m.top);
    choose(m, logits + (long long)t * n, w.correction, s, s + n, s + 2 * n, ids, weights);
    if (slot == 0 && j == 0)
      for (int k = lane; k < m.top; k += 64) {
        ids_out[t * m.top + k] = ids[k];
        weights_out[t * m.top + k] = weights[k];
      }
  }
  __syncthreads();
  const float *gate = w.shared_gate_up;
  if (!shared) {
    const int e = ((const int *)(smem + (m.d + 3) / 4 * 4 + 2 * n + m.groups + m.top))[slot];
    if (e >= m.experts) return;
    gate = w.gate_up + (long long)e * 2 * m.ff * m.d;
  }
  if (j >= ff) return;
  float g, u;
  if constexpr (VEC) {  // both rows in flight together
    const f32x4 *gp = (const f32x4 *)(gate + (long long)j * m.d), *up = (const f32x4 *)(gate + (long long)(ff + j) * m.d);
    f32x4 ga = {0.f, 0.f, 0.f, 0.f}, ua = ga;
    const int n4 = m.d >> 2;
    constexpr int U = 8;
    for (int i0 = lane; i0 < n4; i0 += 64 * U) {
      f32x4 gv[U], uv[U];
#pragma unroll
      for (int k = 0; k < U; ++k)
        if (i0 - lane + 64 * k < n4) {
          const int i = min(i0 + 64 * k, n4 - 1);
          gv[k] = __builtin_nontemporal_load(gp + i);
          uv[k] = __builtin_nontemporal_load(up + i);
        }
#pragma unroll
      for (int k = 0; k < U; ++k)
        if (i0 + 64 * k < n4) {
          const f32x4 x = ((const f32x4 *)xs)[i0 + 64 * k];
          ga += gv[k] * x;
          ua += uv[k] * x;
        }
    }
    g = (ga.x + ga.y) + (ga.z + ga.w);
    u = (ua.x + ua.y) + (ua.z + ua.w);
  } else {
    g = dot_lane<false>(gate + (long long)j * m.d, xs, m.d);
    u = dot_lane<false>(gate + (long long)(ff + j) * m.d, xs, m.d);
  }
  g = wave_sum(g);
  u = wave_sum(u);
  if (lane == 0) hidden[((long long)t * (m.top + 1) + slot) * width + j] = swiglu1(g, u);
}

// y[t][j]: a wavefront per output, over all slots, four experts' rows in flight together
template <bool VEC>
__global__ __launch_bounds__(256) void moe_down_kernel(MoeShape m, MoeTensors w, const float *__restrict__ h,
                                                       const float *__restrict__ hidden, int width,
                                                       const int *__restrict__ ids, const float *__restrict__ weights,
                                                       float *__restrict__ y) {
  const int j = blockIdx.x * 4 + (threadIdx.x >> 6), t = blockIdx.y, lane = threadIdx.x & 63;
  if (j >= m.d) return;
  const float *hid = hidden + (long long)t * (m.top + 1) * width;
  float s = 0.f, same = 0.f;
  if constexpr (VEC) {
    constexpr int G = 4, U = 4;
    const int n4 = m.ff >> 2, s4 = m.shared_ff >> 2;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (m.shared_ff) {
      const f32x4 *a = (const f32x4 *)(w.shared_down + (long long)j * m.shared_ff), *b = (const f32x4 *)(hid + (long long)m.top * width);
      for (int i0 = 0; i0 < s4; i0 += 64 * 8) {
        f32x4 x[8], v[8];
#pragma unroll
        for (int k = 0; k < 8; ++k)
          if (i0 + 64 * k < s4) {
            const int i = min(i0 + 64 * k + lane, s4 - 1);
            x[k] = __builtin_nontemporal_load(a + i);
            v[k] = b[i];
          }
#pragma unroll
        for (int k = 0; k < 8; ++k)
          if (i0 + 64 * k + lane < s4) acc += x[k] * v[k];
      }
    }
    for (int k0 = 0; k0 < m.top; k0 += G) {
      const f32x4 *a[G], *b[G];
      float wk[G];
#pragma unroll
      for (int g = 0; g < G; ++g) {
        const int k = min(k0 + g, m.top - 1), e = ids[t * m.top + k];
        const bool real = k0 + g < m.top && e < m.experts;
        wk[g] = real ? weights[t * m.top + k] : 0.f;
        if (k0 + g < m.top && e >= m.experts) same += weights[t * m.top + k];
        a[g] = real ? (const f32x4 *)(w.down + ((long long)e * m.d + j) * m.ff) : nullptr;
        b[g] = (const f32x4 *)(hid + (long long)k * width);
      }
      for (int i0 = 0; i0 < n4; i0 += 64 * U) {
        f32x4 x[G][U], v[G][U];
#pragma unroll
        for (int g = 0; g < G; ++g)
#pragma unroll
          for (int u = 0; u < U; ++u)
            if (a[g] && i0 + 64 * u < n4) {
              const int i = min(i0 + 64 * u + lane, n4 - 1);
              x[g][u] = __builtin_nontemporal_load(a[g] + i);
              v[g][u] = b[g][i];
            }
#pragma unroll
        for (int g = 0; g < G; ++g)
#pragma unroll
          for (int u = 0; u < U; ++u)
            if (a[g] && i0 + 64 * u + lane < n4) acc += wk[g] * (x[g][u] * v[g][u]);
      }
    }
    s = (acc.x + acc.y) + (acc.z + acc.w);
  } else {
    for (int k = 0; k < m.top; ++k) {
      const int e = ids[t * m.top + k];
      const float wk = weights[t * m.top + k];
      if (e >= m.experts)
        same += wk;
      else
        s += wk * dot_lane<false>(w.down + ((long long)e * m.d + j) * m.ff, hid + (long long)k * width, m.ff);
    }
    if (m.shared_ff) s += dot_lane<false>(w.shared_down + (long long)j * m.shared_ff, hid + (long long)m.top * width, m.shared_ff);
  }
  s = wave_sum(s);
  if (lane == 0) y[(long long)t * m.d + j] = s + same * h[(long long)t * m.d + j];
}

// ---- many tokens -------------------------------------------------------------------------------
// A wavefront chooses for one token after the other; the places of a workgroup's tokens among an expert's rows
// are counted in LDS, and one addition per expert to the expert's counter gives where they begin.  tokens: per
// workgroup.
__global__ __launch_bounds__(256) void moe_select_kernel(MoeShape m, const float *__restrict__ correction,
                                                         const float *__restrict__ logits, int stride, int T, int tokens,
                                                         int *__restrict__ ids, float *__restrict__ weights,
                                                         int *__restrict__ rank, int *counts) {
  extern __shared__ float smem[];  // per wavefront: s, c, best, weights, ids; then [experts] counts
  const int n = m.experts + m.identity, wave = threadIdx.x >> 6, per_wave = 2 * n + m.groups + 2 * m.top;
  float *s = smem + wave * per_wave, *wl = s + 2 * n + m.groups;
  int *il = (int *)(wl + m.top), *cnt = (int *)(smem + 4 * per_wave);
  for (int e = threadIdx.x; e < m.experts; e += 256) cnt[e] = 0;
  __syncthreads();
  const int t0 = blockIdx.x * tokens;
  for (int i = wave; i < tokens && t0 + i < T; i += 4) {
    const int t = t0 + i;
    choose(m, logits + (long long)t * stride, correction, s, s + n, s + 2 * n, il, wl);
    for (int k = threadIdx.x & 63; k < m.top; k += 64) {
      const int e = il[k];
      ids[t * m.top + k] = e;
      weights[t * m.top + k] = wl[k];
      rank[t * m.top + k] = e < m.experts ? atomicAdd(cnt + e, 1) : 0;
    }
    __threadfence_block();
  }
  __syncthreads();
  for (int e = threadIdx.x; e < m.experts; e += 256) cnt[e] = cnt[e] ? atomicAdd(counts + e, cnt[e]) : 0;
  __syncthreads();
  const int mine = min(tokens, T - t0) * m.top;
  for (int i = threadIdx.x; i < mine; i += 256) {  // (ids and ranks of this workgroup's own tokens)
    const int at = t0 * m.top + i, e = ids[at];
    if (e < m.experts) rank[at] += cnt[e];
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
  size_t weights, ids, rank, off, tile_off, rows, hidden, rows_y, total;
};
ManyLayout many_layout(const MoeShape &m, int T) {
  ManyLayout l;
  const size_t slots = (size_t)T * m.top;
  size_t at = 0;
  auto take = [&](size_t k) {
    const size_t here = at;
    at += up4(k);
    return here;
  };
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
  float *logits = scratch, *weights = logits + up4((size_t)T * n);
  int *ids = (int *)(weights + up4((size_t)T * m.top));
  float *hidden = (float *)ids + up4((size_t)T * m.top);
  const int shared_blocks = (m.shared_ff + 3) / 4, slot_blocks = (m.ff + 3) / 4;
  const long long blocks = (long long)shared_blocks + (long long)m.top * slot_blocks;
  const dim3 g1((unsigned)((n + 3) / 4), (unsigned)T), g2((unsigned)blocks, (unsigned)T), g3((unsigned)((m.d + 3) / 4), (unsigned)T);
  const size_t lds = ((size_t)up4(m.d) + 2 * n + m.groups + 2 * m.top) * sizeof(float);
  if (blocks > 0x7fffffffLL || lds > 64 * 1024) return hipErrorInvalidValue;
  const bool vec_d = (m.d & 3) == 0, vec_ff = ((m.ff | m.shared_ff) & 3) == 0;
  if (vec_d) {
    hipLaunchKernelGGL(moe_logits_kernel<true>, g1, dim3(256), 0, stream, h, w.router, logits, n, m.d);
    hipLaunchKernelGGL(moe_up_kernel<true>, g2, dim3(256), lds, stream, m, w, h, logits, hidden, width, shared_blocks, slot_blocks,
                       ids, weights);
  } else {
    hipLaunchKernelGGL(moe_logits_kernel<false>, g1, dim3(256), 0, stream, h, w.router, logits, n, m.d);
    hipLaunchKernelGGL(moe_up_kernel<false>, g2, dim3(256), lds, stream, m, w, h, logits, hidden, width, shared_blocks, slot_blocks,
                       ids, weights);
  }
  if (vec_ff)
    hipLaunchKernelGGL(moe_down_kernel<true>, g3, dim3(256), 0, stream, m, w, h, hidden, width, ids, weights, y);
  else
    hipLaunchKernelGGL(moe_down_kernel<false>, g3, dim3(256), 0, stream, m, w, h, hidden, width, ids, weights, y);
  return hipGetLastError();
}

size_t moe_many_floats(const MoeShape &m, int T) { return many_layout(m, T).total; }

hipError_t launch_moe_many(const MoeShape &m, const MoeTensors &w, const float *h, const float *logits, int stride, float *y,
                           bool add_to_y, int T, float *scratch, int *counts, hipStream_t stream) {
  if (!moe_shape_ok(m) || T < 1 || (long long)T * m.top > 0x3fffffff || !h || !y || !logits ||
      stride < m.experts + m.identity || !scratch || !counts || !w.correction || !w.gate_up || !w.down)
    return hipErrorInvalidValue;
  const ManyLayout l = many_layout(m, T);
  const int n = m.experts + m.identity, slots = T * m.top;
  float *weights = scratch + l.weights, *hidden = scratch + l.hidden, *rows_y = scratch + l.rows_y;
  int *ids = (int *)(scratch + l.ids), *rank = (int *)(scratch + l.rank), *off = (int *)(scratch + l.off),
      *tile_off = (int *)(scratch + l.tile_off), *rows = (int *)(scratch + l.rows);
  hipError_t e = hipSuccess;
  const size_t lds = ((size_t)4 * (2 * n + m.groups + 2 * m.top) + m.experts) * sizeof(float);
  if (lds > 64 * 1024) return hipErrorInvalidValue;
  const int tokens = T <= 4096 ? 4 : 16;
  hipLaunchKernelGGL(moe_select_kernel, dim3((unsigned)((T + tokens - 1) / tokens)), dim3(256), lds, stream, m, w.correction, logits,
                     stride, T, tokens, ids, weights, rank, counts);
  // rows an expert gets if the router spreads them evenly
  const int per_expert = slots / n, best_tm = per_expert > 1024 ? 128 : per_expert > 32 ? 64 : 32;
  static const int tile_knob = getenv("SHAINET_HIP_MOE_TILE") ? atoi(getenv("SHAINET_HIP_MOE_TILE")) : 0;  // a tuning knob: 32, 64 or 128
  const int tm = tile_knob == 32 || tile_knob == 64 || tile_knob == 128 ? tile_knob : best_tm;
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
