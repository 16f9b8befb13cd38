// Latent attention on gfx950 (latent_kernels.hpp says what is computed), fp32.
//
// Decode is the absorbed form: per layer one launch that takes the queries to the latent space and
// appends the new rows, one that attends over key ranges in parallel, one that merges the ranges and
// takes the result back through W_uv.  All heads share a cached row, so 16 (row, head) pairs are the
// columns of one MFMA tile and a row is read once per 16 of them.
//
// MFMA 16x16x4 layout (lane l): A[m = l % 16][k = l / 16], B[k = l / 16][n = l % 16],
// D[m = 4 (l / 16) + r][n = l % 16] for accumulator register r.  The contraction index may be
// visited in any order as long as A and B agree.
//
// Prefill is the expanded form: latent_prefill_kernel, fp32 MFMA 32x32x2 over keys and values that a
// product made from the cached rows, the rotated key part read from the rows themselves.
#include "latent_kernels.hpp"

#include <math.h>
#include <stdint.h>
#include <stdlib.h>

namespace shainet {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float fast_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float sigmoid1(float z) { return 1.f / (1.f + expf(-z)); }

// element i of a rotated vector v of rot_dims turning elements
__device__ __forceinline__ float rotated(const float *v, int i, int rot_dims, const float2 *tab) {
  if (i >= rot_dims) return v[i];
  const float2 cs = tab[i >> 1];
  return (i & 1) ? v[i] * cs.x + v[i - 1] * cs.y : v[i] * cs.x - v[i + 1] * cs.y;
}

// One new row: 256 threads.
__device__ __forceinline__ void append_row(const LatentRows &r, const LatentShape &sh, int t) {
  __shared__ double red[4];
  const float *raw = r.raw + (long long)t * r.stride + r.kv_off;
  float *dst = r.rows + (long long)(r.start_row + t) * sh.row_w;
  double sq = 0.0;
  for (int i = threadIdx.x; i < sh.kv_rank; i += 256) sq += (double)raw[i] * (double)raw[i];
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) sq += __shfl_xor(sq, o);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = sq;
  __syncthreads();
  const double rms = sqrt(((red[0] + red[1]) + (red[2] + red[3])) / (double)sh.kv_rank + r.eps);
  const float2 *tab = r.rope_tab + (long long)(r.start_pos + t) * (sh.rot_dims >> 1);
  for (int i = threadIdx.x; i < sh.row_w; i += 256) {
    float v = 0.f;
    if (i < sh.kv_rank)
      v = (float)(((double)raw[i] / rms) * (double)r.kv_norm[i]);
    else if (i < sh.kv_rank + sh.rot_dim)
      v = rotated(raw + sh.kv_rank, i - sh.kv_rank, sh.rot_dims, tab);
    dst[i] = v;
  }
}

// q (nullable): the rotated parts of the row's queries turn in place
__global__ __launch_bounds__(256) void latent_append_kernel(LatentRows r, LatentShape sh, float *q) {
  append_row(r, sh, blockIdx.x);
  const int half = sh.rot_dims >> 1;
  if (!q || half == 0) return;
  const int qd = sh.dim + sh.rot_dim;
  float *qt = q + (long long)blockIdx.x * sh.H * qd + sh.dim;
  const float2 *tab = r.rope_tab + (long long)(r.start_pos + blockIdx.x) * half;
  for (int i = threadIdx.x; i < sh.H * half; i += 256) {
    const int h = i / half, p = i - h * half;
    float *v = qt + (long long)h * qd + 2 * p;
    const float x = v[0], y = v[1];
    const float2 cs = tab[p];
    v[0] = x * cs.x - y * cs.y;
    v[1] = y * cs.x + x * cs.y;
  }
}

// Workgroups 0 .. T - 1 append a row each; the others take 64 columns of one head of RT rows: lane =
// column, the wavefronts share the head's `dim` rows of W_uk and add up through LDS.
template <int RT>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const float *__restrict__ q, const float *__restrict__ uk,
                                                            LatentRows r, LatentShape sh, int T,
                                                            float *__restrict__ q_abs, float qscale) {
  extern __shared__ float smem[];  // [RT][dim] query rows, then [4][RT][64] sums
  if ((int)blockIdx.x < T) {
    append_row(r, sh, blockIdx.x);
    return;
  }
  const int col_tiles = (sh.kv_rank + 63) / 64;
  int w = (int)blockIdx.x - T;
  const int ct = w % col_tiles;
  w /= col_tiles;
  const int h = w % sh.H, t0 = w / sh.H * RT;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int qd = sh.dim + sh.rot_dim;
  const int nt = min(RT, T - t0);
  const float *qh = q + ((long long)t0 * sh.H + h) * qd;
  const int col = ct * 64 + lane;
  const int per = (sh.dim + 3) / 4, d0 = wave * per, d1 = min(sh.dim, d0 + per);
  const float *wp = uk + (long long)h * sh.dim * sh.kv_rank + min(col, sh.kv_rank - 1);
  // the first rows of W_uk are on their way while the queries are staged
  constexpr int U = 16;
  float wv[U];
#pragma unroll
  for (int u = 0; u < U; ++u) wv[u] = wp[(long long)min(d0 + u, sh.dim - 1) * sh.kv_rank];
  for (int i = threadIdx.x; i < RT * sh.dim; i += 256) {
    const int rr = i / sh.dim, d = i - rr * sh.dim;
    smem[i] = rr < nt ? qh[(long long)rr * sh.H * qd + d] : 0.f;
  }
  __syncthreads();
  float acc[RT];
#pragma unroll
  for (int a = 0; a < RT; ++a) acc[a] = 0.f;
  for (int db = d0; db < d1; db += U) {
    if (db > d0) {
#pragma unroll
      for (int u = 0; u < U; ++u) wv[u] = wp[(long long)min(db + u, sh.dim - 1) * sh.kv_rank];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (db + u < d1) {
#pragma unroll
        for (int a = 0; a < RT; ++a) acc[a] += smem[a * sh.dim + db + u] * wv[u];
      }
  }
  float *red = smem + RT * sh.dim;
#pragma unroll
  for (int a = 0; a < RT; ++a) red[(wave * RT + a) * 64 + lane] = acc[a];
  __syncthreads();
  for (int i = threadIdx.x; i < nt * 64; i += 256) {
    const int a = i >> 6, c = i & 63, cc = ct * 64 + c;
    if (cc >= sh.kv_rank) continue;
    const float s = (red[(0 * RT + a) * 64 + c] + red[(1 * RT + a) * 64 + c]) +
                    (red[(2 * RT + a) * 64 + c] + red[(3 * RT + a) * 64 + c]);
    q_abs[((long long)(t0 + a) * sh.H + h) * sh.row_w + cc] = s * qscale;
  }
  if (ct == 0) {  // the rotated part and the padding of these rows
    const int tail = sh.row_w - sh.kv_rank;
    for (int i = threadIdx.x; i < nt * tail; i += 256) {
      const int a = i / tail, e = i - a * tail;
      float v = 0.f;
      if (e < sh.rot_dim)
        v = rotated(qh + (long long)a * sh.H * qd + sh.dim, e, sh.rot_dims,
                    r.rope_tab + (long long)(r.start_pos + t0 + a) * (sh.rot_dims >> 1)) * qscale;
      q_abs[((long long)(t0 + a) * sh.H + h) * sh.row_w + sh.kv_rank + e] = v;
    }
  }
}

// Column c of tile ct is (row, head) pair 16 ct + c = row * H + head.  The workgroup (eight wavefronts)
// walks its share of the tile's keys in steps of KT: the cached rows go to LDS once and serve as keys
// (the scores' contraction is shared between the wavefronts) and as values (the wavefronts share the
// columns of the output, NTW tiles of 16 each).  Everything the first step needs is requested at
// once and the next step's rows while this one's are used: a launch of one new row is one step or two
// per workgroup, bound by its memory round trips.  Row stride row_w + 4 in LDS: 16-byte reads down a
// column of rows, and reads of 16 neighbours in rows 4 j apart, touch every bank once.
template <int KT, int NTW>
__global__ __launch_bounds__(512) void latent_absorbed_kernel(const float *__restrict__ q_abs,
                                                              const float *__restrict__ rows,
                                                              float *__restrict__ part_o, float *__restrict__ part_ml,
                                                              LatentShape sh, int T, int start_row, int splits,
                                                              int tiles_per_split, int v_w) {
  constexpr int NTH = 512, SUB = KT / 16, PARTS = 8 / SUB;
  constexpr int TPR = NTH / KT;                          // threads per key row; 32 per query row
  constexpr int UK = KT == 32 ? 13 : 10, UQ = KT == 32 ? 7 : 10;  // 16-byte pieces per thread: the widest rows plan_latent_absorbed admits
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int row_w = sh.row_w, ldr = row_w + 4;
  float *qs = smem, *ks = qs + 16 * ldr, *ss = ks + KT * ldr;  // ss: [PARTS][KT][17]
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n = lane & 15, j = lane >> 4;
  const int ct = blockIdx.x, sp = blockIdx.y, d_first = blockIdx.z * 1024;
  const int pairs = T * sh.H, v0 = ct * 16, v1 = min(v0 + 15, pairs - 1);
  const int lo = sh.window ? max(0, start_row + v0 / sh.H - sh.window + 1) : 0, hi = start_row + v1 / sh.H;
  const int my = min(v0 + n, pairs - 1), my_pos = start_row + my / sh.H;
  const int my_lo = sh.window ? max(0, my_pos - sh.window + 1) : 0;
  const int n_tiles = (hi - lo) / KT + 1;
  const int tile0 = sp * tiles_per_split, tile1 = min(n_tiles, tile0 + tiles_per_split);
  const int w4 = row_w >> 2;

  // a thread's pieces of its row: sub, sub + TPR, ... (past the end: the last one again, to the same place);
  // rows past the last key repeat it
  const int krow = threadIdx.x / TPR, ksub = threadIdx.x % TPR, qrow = threadIdx.x >> 5, qsub = threadIdx.x & 31;
  f32x4 kv[UK];
  auto load_keys = [&](int tile) {
    const float *src = rows + (long long)min(lo + tile * KT + krow, hi) * row_w;
#pragma unroll
    for (int u = 0; u < UK; ++u)
      if (TPR * u < w4) kv[u] = *(const f32x4 *)(src + 4 * min(ksub + TPR * u, w4 - 1));
  };
  auto park_keys = [&]() {
#pragma unroll
    for (int u = 0; u < UK; ++u)
      if (TPR * u < w4) *(f32x4 *)(ks + krow * ldr + 4 * min(ksub + TPR * u, w4 - 1)) = kv[u];
  };

  float m = -INFINITY, l = 0.f;
  f32x4 acc[NTW];
#pragma unroll
  for (int i = 0; i < NTW; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (tile0 < tile1) {
    f32x4 qv[UQ];
    const float *src = q_abs + (long long)min(v0 + qrow, v1) * row_w;
#pragma unroll
    for (int u = 0; u < UQ; ++u)
      if (32 * u < w4) qv[u] = *(const f32x4 *)(src + 4 * min(qsub + 32 * u, w4 - 1));
    load_keys(tile0);
#pragma unroll
    for (int u = 0; u < UQ; ++u)
      if (32 * u < w4) *(f32x4 *)(qs + qrow * ldr + 4 * min(qsub + 32 * u, w4 - 1)) = qv[u];
  }
  const int sub = wave % SUB, part = wave / SUB;
  const int steps = row_w >> 4, s_begin = part * steps / PARTS, s_end = (part + 1) * steps / PARTS;
  const int v_tiles = min((v_w - d_first) >> 4, 64);
  for (int tile = tile0; tile < tile1; ++tile) {
    const int k0 = lo + tile * KT;
    park_keys();
    if (tile + 1 < tile1) load_keys(tile + 1);
    __syncthreads();
    {
      f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
      const float *kp = ks + (16 * sub + n) * ldr + 4 * j, *qp = qs + n * ldr + 4 * j;
      // (fragments two steps ahead of the MFMAs that use them; the reads past the end stay inside LDS)
      f32x4 a1 = *(const f32x4 *)(kp + 16 * s_begin), b1 = *(const f32x4 *)(qp + 16 * s_begin);
      f32x4 a2 = *(const f32x4 *)(kp + 16 * min(s_begin + 1, steps - 1)), b2 = *(const f32x4 *)(qp + 16 * min(s_begin + 1, steps - 1));
      for (int i = s_begin; i < s_end; ++i) {
        const f32x4 a = a1, b = b1;
        const int ahead = min(i + 2, steps - 1);
        a1 = a2;
        b1 = b2;
        a2 = *(const f32x4 *)(kp + 16 * ahead);
        b2 = *(const f32x4 *)(qp + 16 * ahead);
        s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, s0, 0, 0, 0);
        s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, s1, 0, 0, 0);
        s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, s0, 0, 0, 0);
        s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, s1, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) ss[(part * KT + 16 * sub + 4 * j + r) * 17 + n] = s0[r] + s1[r];
    }
    __syncthreads();
    // every wavefront: the whole tile's scores of its columns, key 16 u + 4 j + r in p[u][r]
    float p[SUB][4], mx = -INFINITY;
#pragma unroll
    for (int u = 0; u < SUB; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int kk = 16 * u + 4 * j + r;
        float s = ss[kk * 17 + n];
#pragma unroll
        for (int g = 1; g < PARTS; ++g) s += ss[(g * KT + kk) * 17 + n];
        const int key = k0 + kk;
        p[u][r] = key >= my_lo && key <= my_pos ? s : -INFINITY;
        mx = fmaxf(mx, p[u][r]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float mnew = fmaxf(m, mx);
    const float mref = mnew == -INFINITY ? 0.f : mnew;  // no key of this column seen so far
    const float alpha = fast_exp2(m - mref);
    float ps = 0.f;
#pragma unroll
    for (int u = 0; u < SUB; ++u)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        p[u][r] = fast_exp2(p[u][r] - mref);
        ps += p[u][r];
      }
    l = l * alpha + ps;
    m = mnew;
#pragma unroll
    for (int i = 0; i < NTW; ++i) acc[i] *= alpha;
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      // (a wavefront without an i-th tile computes the last one again and does not store it)
      const float *vp = ks + 4 * j * ldr + d_first + 16 * min(wave + 8 * i, v_tiles - 1) + n;
#pragma unroll
      for (int u = 0; u < SUB; ++u)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(vp[(16 * u + r) * ldr], p[u][r], acc[i], 0, 0, 0);
    }
    __syncthreads();  // the rows are free for the next step's
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  const long long slot = (long long)(v0 + n) * splits + sp;
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    const int vt = wave + 8 * i;
    if (vt < v_tiles) *(f32x4 *)(part_o + slot * v_w + d_first + 16 * vt + 4 * j) = acc[i];
  }
  if (wave == 0 && j == 0 && blockIdx.z == 0) *(float2 *)(part_ml + 2 * slot) = float2{m, l};
}

// Sixteen outputs of one head, a wavefront each, for RT rows.  blockIdx.x: head fastest, so that with
// a multiple of 8 heads the workgroups that merge the same partials sit on one XCD; blockIdx.y: rows.
// The wavefronts' rows of W_uv and the partials are requested before anything is waited for.
template <int RT>
__global__ __launch_bounds__(1024) void latent_out_kernel(const float *__restrict__ part_o,
                                                          const float *__restrict__ part_ml,
                                                          const float *__restrict__ uv, const float *__restrict__ sink,
                                                          LatentRows r, LatentShape sh, int T, int splits, int v_w,
                                                          float *__restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  constexpr int WU = 4;   // 16-byte pieces of a row of W_uv per lane held in registers
  constexpr int LD = 12;  // partials in flight per thread
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int h = blockIdx.x % sh.H, t0 = blockIdx.y * RT, nt = min(RT, T - t0);
  const int v4 = v_w >> 2, groups = 1024 / v4;  // thread: column of 16 bytes c, ranges g, g + groups, ...
  const int c = threadIdx.x % v4, g = threadIdx.x / v4;
  float *lat = smem, *fac = lat + RT * v_w, *red = fac + RT * splits;  // [RT][v_w], [RT][splits], [groups][v_w]
  const int jj = (int)(blockIdx.x / sh.H) * 16 + wave;
  const float *wr = uv + ((long long)h * sh.vdim + min(jj, sh.vdim - 1)) * sh.kv_rank;
  const bool held = (sh.kv_rank & 3) == 0 && sh.kv_rank <= 256 * WU;
  f32x4 w[WU];
  if (held) {
#pragma unroll
    for (int u = 0; u < WU; ++u)
      if (256 * u < sh.kv_rank) w[u] = *(const f32x4 *)(wr + min(256 * u + 4 * lane, sh.kv_rank - 4));
  }
  for (int a = 0; a < nt; ++a) {
    const long long col = (long long)(t0 + a) * sh.H + h;
    const float *po = part_o + col * splits * v_w + 4 * c;
    f32x4 x[LD];
#pragma unroll
    for (int u = 0; u < LD; ++u)
      if (groups * u < splits) x[u] = *(const f32x4 *)(po + (long long)min(g + groups * u, splits - 1) * v_w);
    // the factor of a range: 2^(max - overall max) / denominator, the sink included in both (an empty
    // range has max -inf and sum 0: factor 0)
    if (wave == 0) {
      const float2 *ml = (const float2 *)part_ml + col * splits;
      const float sk = sink[h] * kLog2e;
      float mm = sk;
      for (int s = lane; s < splits; s += 64) mm = fmaxf(mm, ml[s].x);
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) mm = fmaxf(mm, __shfl_xor(mm, o));
      float den = 0.f;
      for (int s = lane; s < splits; s += 64) den += ml[s].y * fast_exp2(ml[s].x - mm);
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) den += __shfl_xor(den, o);
      const float inv = 1.f / (den + fast_exp2(sk - mm));
      for (int s = lane; s < splits; s += 64) fac[a * splits + s] = fast_exp2(ml[s].x - mm) * inv;
    }
    __syncthreads();
    f32x4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < LD; ++u)
      if (g + groups * u < splits) sum += fac[a * splits + g + groups * u] * x[u];
    for (int s = g + groups * LD; s < splits; s += groups) sum += fac[a * splits + s] * *(const f32x4 *)(po + (long long)s * v_w);
    if (g < groups) *(f32x4 *)(red + g * v_w + 4 * c) = sum;
    __syncthreads();
    for (int i = threadIdx.x; i < v_w; i += 1024) {
      float s = red[i];
      for (int k = 1; k < groups; ++k) s += red[k * v_w + i];
      lat[a * v_w + i] = s;
    }
    __syncthreads();
  }
  if (jj >= sh.vdim) return;
  float s[RT];
#pragma unroll
  for (int a = 0; a < RT; ++a) s[a] = 0.f;
  if (held) {
#pragma unroll
    for (int u = 0; u < WU; ++u)
      if (256 * u + 4 * lane < sh.kv_rank) {
#pragma unroll
        for (int a = 0; a < RT; ++a) {
          const f32x4 x = *(const f32x4 *)(lat + a * v_w + 256 * u + 4 * lane);
          s[a] += (w[u].x * x.x + w[u].y * x.y) + (w[u].z * x.z + w[u].w * x.w);
        }
      }
  } else {
    for (int k = lane; k < sh.kv_rank; k += 64) {
      const float wv = wr[k];
#pragma unroll
      for (int a = 0; a < RT; ++a) s[a] += wv * lat[a * v_w + k];
    }
  }
#pragma unroll
  for (int a = 0; a < RT; ++a) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) s[a] += __shfl_xor(s[a], o);
    if (lane == 0 && a < nt)
      out[((long long)(t0 + a) * sh.H + h) * sh.vdim + jj] =
          s[a] * sigmoid1(r.raw[(long long)(t0 + a) * r.stride + r.gate_off + h]);
  }
}

// ---- expanded form -----------------------------------------------------------------------------
//
// A workgroup owns 128 rows of one head, a wavefront 32 of them; all walk the keys in tiles of 32 that
// go global memory -> registers -> LDS, the next tile's loads in flight behind the MFMAs of this one
// (two workgroups share a compute unit, so that one's barriers hide behind the other's MFMAs).
// S^T = K Q^T, so that the probabilities come out of the accumulator laid out as the B operand of
// O^T += V^T P^T.  MFMA 32x32x2 layout (lane l): A[m = l % 32][k = l / 32], B[k = l / 32][n = l % 32],
// D[m = 8 (r / 4) + 4 (l / 32) + r % 4][n = l % 32] for accumulator register r.
//   scores:  m = key within the tile, n = row; lane half j = l / 32 covers d = 8 i + 4 j + 0..3 of piece i;
//            d runs over the unrotated dimensions, padded to a multiple of 8, then the rotated ones.
//   output:  tile t, m: d = NT m + t; step r of lane half j is key 8 (r / 4) + 4 j + r % 4.
// NK: pieces of 8 query / key dimensions at most; NT: tiles of 32 value dimensions.
struct LatentPrefillArgs {
  const float *q;        // [T, H (dim + rot_dim)], rotated (launch_latent_append)
  const float *kv;       // [key rows, H dim + H vdim]
  const float *key_rot;  // rotated part of key row 0; rows row_w apart
  const float *sink;
  LatentRows r;          // raw (gates), rope_tab, start_pos
  LatentShape sh;
  float *out;            // [T, H vdim]
  float *part_o, *part_ml;  // splits > 1: [blocks][splits][128][32 NT], [..][128][2]
  int T, first_key;      // row t sees key rows .. first_key + t
  int items, splits;
  float c;               // scale * log2(e)
};

template <int NK, int NT>
__global__ __launch_bounds__(256, NK <= 24 ? 2 : 1) void latent_prefill_kernel(const LatentPrefillArgs a) {
  constexpr int KSTR = NK * 8 + 4, VSTR = NT * 32;
  constexpr int KU = (NK * 2 + 7) / 8, VU = NT;  // float4 of a K (V) tile per thread: 8 threads per row
  __shared__ __attribute__((aligned(16))) float Ks[32 * KSTR];
  __shared__ __attribute__((aligned(16))) float Vs[32 * VSTR];
  const LatentShape &sh = a.sh;
  // heads fastest: with a multiple of 8 heads an XCD (index % 8) keeps to its own heads' keys and
  // values; the blocks with the most keys start first
  const int h = blockIdx.x % sh.H;
  const int chunk = (blockIdx.x / sh.H) % a.splits;
  const int item = a.items - 1 - (int)(blockIdx.x / sh.H / a.splits);
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n = lane & 31, j = lane >> 5;
  const int dn = sh.dim, dr = sh.rot_dim, dn8 = (dn + 7) / 8 * 8;
  const int row0 = item * 128, w_row0 = row0 + wave * 32;
  const bool wave_active = w_row0 < a.T;
  const int my_row = min(w_row0 + n, a.T - 1);
  const int my_hi = a.first_key + my_row, my_lo = sh.window ? max(0, my_hi - sh.window + 1) : 0;
  const int w_first = min(w_row0, a.T - 1), w_last = min(w_row0 + 31, a.T - 1);
  const int w_hi_min = a.first_key + w_first, w_hi_max = a.first_key + w_last;
  const int w_lo_min = sh.window ? max(0, w_hi_min - sh.window + 1) : 0;
  const int w_lo_max = sh.window ? max(0, w_hi_max - sh.window + 1) : 0;
  const int b_hi = a.first_key + min(row0 + 127, a.T - 1);
  const int b_lo = sh.window ? max(0, a.first_key + row0 - sh.window + 1) : 0;
  const int kt_all0 = b_lo >> 5, n_tiles = (b_hi >> 5) + 1 - kt_all0;
  const int per_chunk = (n_tiles + a.splits - 1) / a.splits;
  const int kt0 = kt_all0 + chunk * per_chunk, kt1 = min(kt_all0 + n_tiles, kt0 + per_chunk);

  // staging: 8 threads per key row, 16-byte pieces sub, sub + 8, ...; a thread without a piece of its
  // own repeats the last one (same source, same place), so no load or store is conditional
  const int srow = threadIdx.x >> 3, sub = threadIdx.x & 7;
  const unsigned kv_stride = (unsigned)(sh.H * (sh.dim + sh.vdim));
  const int n_pieces = dn >> 2, r_pieces = dr >> 2;
  const float *k_src[KU];
  unsigned k_step[KU];
  int k_dst[KU];
#pragma unroll
  for (int u = 0; u < KU; ++u) {
    const int p = min(sub + 8 * u, n_pieces + r_pieces - 1);
    const bool is_rot = p >= n_pieces;
    k_src[u] = is_rot ? a.key_rot + 4 * (p - n_pieces) : a.kv + h * dn + 4 * p;
    k_step[u] = is_rot ? (unsigned)sh.row_w : kv_stride;
    k_dst[u] = srow * KSTR + (is_rot ? dn8 + 4 * (p - n_pieces) : 4 * p);
  }
  // (pieces beyond vdim read what follows: the columns they land in are never stored)
  const float *v_src = a.kv + sh.H * dn + h * sh.vdim + 4 * sub;
  f32x4 stage[KU > VU ? KU : VU];
  auto load_k = [&](int kt) {
    const unsigned key = (unsigned)min(kt * 32 + srow, b_hi);
#pragma unroll
    for (int u = 0; u < KU; ++u) stage[u] = *(const f32x4 *)(k_src[u] + (unsigned long long)key * k_step[u]);
  };
  auto park_k = [&]() {
#pragma unroll
    for (int u = 0; u < KU; ++u) *(f32x4 *)&Ks[k_dst[u]] = stage[u];
  };
  auto load_v = [&](int kt) {
    const float *p = v_src + (unsigned long long)(unsigned)min(kt * 32 + srow, b_hi) * kv_stride;
#pragma unroll
    for (int u = 0; u < VU; ++u) stage[u] = *(const f32x4 *)(p + 32 * u);
  };
  auto park_v = [&]() {
#pragma unroll
    for (int u = 0; u < VU; ++u) *(f32x4 *)&Vs[srow * VSTR + 4 * (sub + 8 * u)] = stage[u];
  };
  if (kt0 < kt1) load_k(kt0);
  // the padding between and behind the two parts of a key: the query is zero there, so anything finite will do
  for (int i = threadIdx.x; i < 32 * KSTR; i += 256) Ks[i] = 0.f;

  float qr[NK * 4];
  {
    const float *qp = a.q + ((long long)my_row * sh.H + h) * (dn + dr);
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int d = 8 * i + 4 * j, e = d - dn8;
      f32x4 x = {0.f, 0.f, 0.f, 0.f};
      if (d < dn || (e >= 0 && e < dr)) x = *(const f32x4 *)(qp + (d < dn ? d : dn + e));
      qr[4 * i + 0] = x.x * a.c;
      qr[4 * i + 1] = x.y * a.c;
      qr[4 * i + 2] = x.z * a.c;
      qr[4 * i + 3] = x.w * a.c;
    }
  }
  f32x16 o[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[t][r] = 0.f;
  float m = -INFINITY, l = 0.f;  // reference value of the row's exponentials (log2 units), this lane half's sum
  constexpr float kTau = 8.f;    // scores may exceed it by this much before it moves

  // Per tile: the values travel while the scores are computed, the next tile's keys while the
  // values are used; each set is parked in LDS behind a barrier that says the stage is free.
  __syncthreads();
  if (kt0 < kt1) park_k();
  __syncthreads();
  for (int kt = kt0; kt < kt1; ++kt) {
    load_v(kt);
    const int k_first = kt * 32, k_last = k_first + 31;
    const bool visible = wave_active && k_first <= w_hi_max && k_last >= w_lo_min;
    f32x16 s;
#pragma unroll
    for (int r = 0; r < 16; ++r) s[r] = 0.f;
    if (visible) {
      const float *kl = &Ks[n * KSTR + 4 * j];
      constexpr int PF = 2;
      f32x4 kf[NK];
#pragma unroll
      for (int i = 0; i < PF && i < NK; ++i) kf[i] = *(const f32x4 *)(kl + 8 * i);
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        if (i + PF < NK) kf[i + PF] = *(const f32x4 *)(kl + 8 * (i + PF));
        __builtin_amdgcn_sched_barrier(0x7);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf[i].x, qr[4 * i + 0], s, 0, 0, 0);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf[i].y, qr[4 * i + 1], s, 0, 0, 0);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf[i].z, qr[4 * i + 2], s, 0, 0, 0);
        s = __builtin_amdgcn_mfma_f32_32x32x2f32(kf[i].w, qr[4 * i + 3], s, 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0x7);
      }
      if (k_first < w_lo_max || k_last > w_hi_min) {  // an edge of some row's keys lies in the tile
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = k_first + 8 * (r >> 2) + 4 * j + (r & 3);
          if (key < my_lo || key > my_hi) s[r] = -INFINITY;
        }
      }
      float mx = s[0];
#pragma unroll
      for (int r = 1; r < 16; ++r) mx = fmaxf(mx, s[r]);
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      const bool move = mx > (m == -INFINITY ? -INFINITY : m + kTau);
      if (__builtin_amdgcn_ballot_w64(move) != 0) {
        const float mnew = move ? mx : m;
        const float alpha = move && m != -INFINITY ? fast_exp2(m - mnew) : 1.f;  // (nothing to rescale before a row's first key)
        m = mnew;
        l *= alpha;
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[t][r] *= alpha;
      }
      const float mref = m == -INFINITY ? 0.f : m;
      float psum = 0.f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        s[r] = fast_exp2(s[r] - mref);
        psum += s[r];
      }
      l += psum;
    }
    park_v();
    __syncthreads();
    if (kt + 1 < kt1) load_k(kt + 1);
    if (visible) {
      constexpr int PF = 2;
      typedef float vrow_t __attribute__((ext_vector_type(NT)));
      const float *vl = &Vs[4 * j * VSTR + NT * n];
      vrow_t vv[16];
#pragma unroll
      for (int r = 0; r < PF; ++r) vv[r] = *(const vrow_t *)(vl + (8 * (r >> 2) + (r & 3)) * VSTR);
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        if (r + PF < 16) vv[r + PF] = *(const vrow_t *)(vl + (8 * ((r + PF) >> 2) + ((r + PF) & 3)) * VSTR);
        __builtin_amdgcn_sched_barrier(0x7);
#pragma unroll
        for (int t = 0; t < NT; ++t) o[t] = __builtin_amdgcn_mfma_f32_32x32x2f32(vv[r][t], s[r], o[t], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0x7);
      }
    }
    if (kt + 1 < kt1) park_k();
    __syncthreads();
  }

  l += __shfl_xor(l, 32);
  if (a.splits > 1) {
    const long long pbase = (((long long)item * sh.H + h) * a.splits + chunk) * 128 + wave * 32 + n;
    float *op = a.part_o + pbase * VSTR;
#pragma unroll
    for (int r = 0; r < 16; ++r)
#pragma unroll
      for (int t = 0; t < NT; t += 2)
        *(float2 *)(op + NT * (8 * (r >> 2) + 4 * j + (r & 3)) + t) = float2{o[t][r], o[t + 1][r]};
    if (j == 0) *(float2 *)(a.part_ml + 2 * pbase) = float2{m, l};
    return;
  }
  if (w_row0 + n >= a.T) return;
  const float sk = a.sink[h] * kLog2e, mf = fmaxf(m, sk);
  const float f = fast_exp2(m - mf), den = l * f + fast_exp2(sk - mf);
  const float factor = f / den * sigmoid1(a.r.raw[(long long)my_row * a.r.stride + a.r.gate_off + h]);
  float *op = a.out + ((long long)my_row * sh.H + h) * sh.vdim;
#pragma unroll
  for (int r = 0; r < 16; ++r)
#pragma unroll
    for (int t = 0; t < NT; t += 2) {
      const int d = NT * (8 * (r >> 2) + 4 * j + (r & 3)) + t;
      if (d < sh.vdim) *(float2 *)(op + d) = float2{o[t][r] * factor, o[t + 1][r] * factor};
    }
}

// Merges the key chunks of one (row block, head), sink and gate included; blockIdx.y: 32 of its rows.
__global__ __launch_bounds__(256) void latent_prefill_combine_kernel(const LatentPrefillArgs a, int vstr) {
  const LatentShape &sh = a.sh;
  const int h = blockIdx.x % sh.H, item = blockIdx.x / sh.H, v4 = sh.vdim >> 2;
  const long long base = ((long long)item * sh.H + h) * a.splits * 128;
  const float sk = a.sink[h] * kLog2e;
  for (int i = threadIdx.x; i < 32 * v4; i += 256) {
    const int rl = blockIdx.y * 32 + i / v4, c = i % v4, row = item * 128 + rl;
    if (row >= a.T) continue;
    float mm = sk;
    for (int s = 0; s < a.splits; ++s) mm = fmaxf(mm, a.part_ml[2 * (base + (long long)s * 128 + rl)]);
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    float den = fast_exp2(sk - mm);
    for (int s0 = 0; s0 < a.splits; s0 += 4) {
      f32x4 x[4];
      float2 ml[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const long long p = base + (long long)min(s0 + u, a.splits - 1) * 128 + rl;
        x[u] = *(const f32x4 *)(a.part_o + p * vstr + 4 * c);
        ml[u] = *(const float2 *)(a.part_ml + 2 * p);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const float f = s0 + u < a.splits ? fast_exp2(ml[u].x - mm) : 0.f;  // 0 for a chunk in which the row saw no key
        acc += f * x[u];
        den += f * ml[u].y;
      }
    }
    const float g = sigmoid1(a.r.raw[(long long)row * a.r.stride + a.r.gate_off + h]);
    *(f32x4 *)(a.out + ((long long)row * sh.H + h) * sh.vdim + 4 * c) = acc * (g / den);
  }
}

constexpr size_t kMaxLds = 160 * 1024;

bool shape_ok(const LatentShape &sh) {
  return sh.H > 0 && sh.dim > 0 && sh.rot_dim >= 0 && sh.vdim > 0 && sh.kv_rank > 0 && sh.rot_dims >= 0 &&
         sh.rot_dims <= sh.rot_dim && (sh.rot_dims & 1) == 0 && sh.row_w == latent_row_width(sh.kv_rank, sh.rot_dim) &&
         sh.window >= 0;
}
bool rows_ok(const LatentRows &r, const LatentShape &sh, int T) {
  return shape_ok(sh) && T > 0 && r.raw && r.kv_norm && (r.rope_tab || !sh.rot_dims) && r.rows && r.start_pos >= 0 &&
         r.start_row >= 0 && r.kv_off >= 0 && r.gate_off >= 0 && r.stride >= r.kv_off + sh.kv_rank + sh.rot_dim &&
         r.stride >= r.gate_off + sh.H;
}

}  // namespace

hipError_t launch_latent_append(const LatentRows &r, const LatentShape &sh, int T, float *q, hipStream_t stream) {
  if (!rows_ok(r, sh, T)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(latent_append_kernel, dim3((unsigned)T), dim3(256), 0, stream, r, sh, q);
  return hipGetLastError();
}

hipError_t launch_latent_absorb(const float *q, const float *uk, const LatentRows &r, const LatentShape &sh, int T,
                                float *q_abs, hipStream_t stream) {
  if (!rows_ok(r, sh, T) || !q || !uk || !q_abs) return hipErrorInvalidValue;
  const int rt = T == 1 ? 1 : 4;
  const size_t lds = (size_t)rt * (sh.dim + 4 * 64) * sizeof(float);
  const long long wgs = (long long)T + (long long)((sh.kv_rank + 63) / 64) * sh.H * ((T + rt - 1) / rt);
  if (lds > 64 * 1024 || wgs > 0x7fffffffLL) return hipErrorInvalidValue;
  const float qscale = sh.scale * kLog2e;
  if (rt == 1)
    hipLaunchKernelGGL(latent_absorb_kernel<1>, dim3((unsigned)wgs), dim3(256), lds, stream, q, uk, r, sh, T, q_abs, qscale);
  else
    hipLaunchKernelGGL(latent_absorb_kernel<4>, dim3((unsigned)wgs), dim3(256), lds, stream, q, uk, r, sh, T, q_abs, qscale);
  return hipGetLastError();
}

bool plan_latent_absorbed(const LatentShape &sh, int T, int start_row, LatentPlan &p) {
  if (!shape_ok(sh) || T < 1 || start_row < 0 || (long long)T * sh.H > 0x3fffffff) return false;
  p.v_w = (sh.kv_rank + 15) / 16 * 16;
  p.v_slices = (p.v_w + 1023) / 1024;
  // (what fits 160 KiB: rows of up to 800 floats in steps of 32, up to 1200 in steps of 16)
  p.key_tile = sh.row_w <= 800 ? 32 : 16;
  const size_t ldr = (size_t)sh.row_w + 4;
  p.lds_bytes = ((16 + p.key_tile) * ldr + (size_t)8 * 16 * 17) * sizeof(float);
  if (p.lds_bytes > kMaxLds) return false;
  p.col_tiles = (T * sh.H + 15) / 16;
  // the most keys a tile of columns walks: what the last of its rows sees and the rows before it saw besides
  int span = (14 + sh.H) / sh.H + 1;  // rows that 16 consecutive (row, head) pairs can touch
  if (span > T) span = T;
  long long keys = (long long)start_row + T;
  if (sh.window && keys > (long long)sh.window + span - 1) keys = (long long)sh.window + span - 1;
  const int tiles = (int)((keys + p.key_tile - 1) / p.key_tile);
  static const int target_knob = getenv("SHAINET_HIP_LATENT_WGS") ? atoi(getenv("SHAINET_HIP_LATENT_WGS")) : 0;
  const int target = target_knob > 0 ? target_knob : 256;
  int splits = target / p.col_tiles;
  if (splits > 128) splits = 128;
  if (splits > tiles) splits = tiles;
  if (splits < 1) splits = 1;
  p.tiles_per_split = (tiles + splits - 1) / splits;
  p.splits = (tiles + p.tiles_per_split - 1) / p.tiles_per_split;
  p.partial_floats = (size_t)p.col_tiles * 16 * p.splits * (p.v_w + 2);
  return true;
}

hipError_t launch_latent_absorbed(const float *q_abs, const float *rows, float *partials, const LatentShape &sh, int T,
                                  int start_row, const LatentPlan &p, hipStream_t stream) {
  LatentPlan want;
  if (!q_abs || !rows || !partials || !plan_latent_absorbed(sh, T, start_row, want) || want.splits != p.splits ||
      want.partial_floats != p.partial_floats || p.splits > 65535)
    return hipErrorInvalidValue;
  float *part_o = partials, *part_ml = partials + (size_t)p.col_tiles * 16 * p.splits * p.v_w;
  const dim3 grid((unsigned)p.col_tiles, (unsigned)p.splits, (unsigned)p.v_slices);
  const int slice = p.v_w < 1024 ? p.v_w : 1024;
  const int ntw = (slice / 16 + 7) / 8;
#define SHAINET_LAUNCH_ABSORBED(KT_, NTW_)                                                                               \
  do {                                                                                                                   \
    static const hipError_t a_ = hipFuncSetAttribute((const void *)latent_absorbed_kernel<KT_, NTW_>,                           \
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);                 \
    if (a_ != hipSuccess) return a_;                                                                                    \
    hipLaunchKernelGGL((latent_absorbed_kernel<KT_, NTW_>), grid, dim3(512), p.lds_bytes, stream, q_abs, rows, part_o,  \
                       part_ml, sh, T, start_row, p.splits, p.tiles_per_split, p.v_w);                                  \
  } while (0)
#define SHAINET_LAUNCH_ABSORBED_K(NTW_)  \
  do {                                   \
    if (p.key_tile == 32)                \
      SHAINET_LAUNCH_ABSORBED(32, NTW_); \
    else                                 \
      SHAINET_LAUNCH_ABSORBED(16, NTW_); \
  } while (0)
  if (ntw <= 1)
    SHAINET_LAUNCH_ABSORBED_K(1);
  else if (ntw <= 2)
    SHAINET_LAUNCH_ABSORBED_K(2);
  else if (ntw <= 4)
    SHAINET_LAUNCH_ABSORBED_K(4);
  else
    SHAINET_LAUNCH_ABSORBED_K(8);
#undef SHAINET_LAUNCH_ABSORBED_K
#undef SHAINET_LAUNCH_ABSORBED
  return hipGetLastError();
}

hipError_t launch_latent_out(const float *partials, const float *uv, const float *sink, const LatentRows &r,
                             const LatentShape &sh, int T, const LatentPlan &p, float *out, hipStream_t stream) {
  if (!rows_ok(r, sh, T) || !partials || !uv || !sink || !out || sh.H > 65535) return hipErrorInvalidValue;
  const float *part_ml = partials + (size_t)p.col_tiles * 16 * p.splits * p.v_w;
  const int rt = T == 1 ? 1 : 4;
  const int v4 = p.v_w / 4;
  if (v4 > 1024) return hipErrorInvalidValue;
  const size_t lds = ((size_t)rt * (p.v_w + p.splits) + (size_t)(1024 / v4) * p.v_w) * sizeof(float);
  const long long wgs = (long long)((sh.vdim + 15) / 16) * sh.H;
  if (lds > 64 * 1024 || (T + rt - 1) / rt > 65535 || wgs > 0x7fffffffLL) return hipErrorInvalidValue;
  const dim3 grid((unsigned)wgs, (unsigned)((T + rt - 1) / rt));
  if (rt == 1)
    hipLaunchKernelGGL(latent_out_kernel<1>, grid, dim3(1024), lds, stream, partials, part_ml, uv, sink, r, sh, T, p.splits,
                       p.v_w, out);
  else
    hipLaunchKernelGGL(latent_out_kernel<4>, grid, dim3(1024), lds, stream, partials, part_ml, uv, sink, r, sh, T, p.splits,
                       p.v_w, out);
  return hipGetLastError();
}

bool plan_latent_expanded(const LatentShape &sh, int T, int start_row, LatentExpandedPlan &p) {
  if (!shape_ok(sh) || T < 1 || start_row < 0) return false;
  // 16-byte pieces of the query, key and value rows
  if ((sh.dim | sh.rot_dim | sh.vdim | sh.kv_rank) & 3) return false;
  const int dk = (sh.dim + 7) / 8 * 8 + (sh.rot_dim + 7) / 8 * 8;
  if (dk > 256 || sh.vdim > 128) return false;
  p.nk = dk <= 96 ? 12 : dk <= 128 ? 16 : dk <= 192 ? 24 : 32;
  p.nt = sh.vdim <= 64 ? 2 : 4;
  const int back = sh.window && sh.window - 1 < start_row ? sh.window - 1 : start_row;
  p.first_row = start_row - back;
  p.key_rows = back + T;
  p.items = (T + 127) / 128;
  const long long blocks = (long long)p.items * sh.H;
  if (blocks > 0x3fffff) return false;
  int tiles = (p.key_rows + 31) / 32;  // of the row block with the most keys
  if (sh.window && tiles > (sh.window + 127) / 32 + 2) tiles = (sh.window + 127) / 32 + 2;
  static const int splits_knob = getenv("SHAINET_HIP_LATENT_SPLITS") ? atoi(getenv("SHAINET_HIP_LATENT_SPLITS")) : 0;
  int splits = blocks >= 384 ? 1 : (int)((512 + blocks - 1) / blocks);  // two workgroups per compute unit
  if (splits > tiles / 4) splits = tiles / 4;
  if (splits > 16) splits = 16;
  if (splits_knob > 0) splits = splits_knob;
  p.splits = splits < 1 ? 1 : splits;
  p.partial_floats = p.splits > 1 ? (size_t)blocks * p.splits * 128 * (p.nt * 32 + 2) : 0;
  // multiply-adds per (row, key, head): this form's, and its product's share; against the absorbed form's,
  // whose kernel reaches about half this one's rate
  const double pairs = (double)T * (sh.window && sh.window < p.key_rows ? sh.window : p.key_rows);
  const double here = pairs * sh.H * (8 * p.nk + 32 * p.nt) + (double)p.key_rows * sh.kv_rank * sh.H * (sh.dim + sh.vdim);
  p.pays = T > 16 && here < 2.0 * pairs * sh.H * (sh.row_w + sh.kv_rank);
  return true;
}

hipError_t launch_latent_expanded(const float *q, const float *kv, const float *sink, const LatentRows &r,
                                  const LatentShape &sh, int T, const LatentExpandedPlan &p, float *partials, float *out,
                                  hipStream_t stream) {
  LatentExpandedPlan want;
  if (!rows_ok(r, sh, T) || !q || !kv || !sink || !out || !plan_latent_expanded(sh, T, r.start_row, want) ||
      want.splits != p.splits || want.key_rows != p.key_rows || (p.splits > 1 && !partials))
    return hipErrorInvalidValue;
  if (((uintptr_t)q | (uintptr_t)kv | (uintptr_t)r.rows | (uintptr_t)out | (uintptr_t)partials) & 15) return hipErrorInvalidValue;
  LatentPrefillArgs a = {};
  a.q = q;
  a.kv = kv;
  a.key_rot = r.rows + (long long)p.first_row * sh.row_w + sh.kv_rank;
  a.sink = sink;
  a.r = r;
  a.sh = sh;
  a.out = out;
  a.part_o = partials;
  a.part_ml = partials ? partials + (size_t)p.items * sh.H * p.splits * 128 * p.nt * 32 : nullptr;
  a.T = T;
  a.first_key = r.start_row - p.first_row;
  a.items = p.items;
  a.splits = p.splits;
  a.c = sh.scale * kLog2e;
  const dim3 grid((unsigned)(p.items * sh.H * p.splits));
#define SHAINET_LAUNCH_EXPANDED(NK_)                                                               \
  do {                                                                                             \
    if (p.nt == 2)                                                                                 \
      hipLaunchKernelGGL((latent_prefill_kernel<NK_, 2>), grid, dim3(256), 0, stream, a);          \
    else                                                                                           \
      hipLaunchKernelGGL((latent_prefill_kernel<NK_, 4>), grid, dim3(256), 0, stream, a);          \
  } while (0)
  switch (p.nk) {
    case 12: SHAINET_LAUNCH_EXPANDED(12); break;
    case 16: SHAINET_LAUNCH_EXPANDED(16); break;
    case 24: SHAINET_LAUNCH_EXPANDED(24); break;
    default: SHAINET_LAUNCH_EXPANDED(32); break;
  }
#undef SHAINET_LAUNCH_EXPANDED
  const hipError_t e = hipGetLastError();
  if (e != hipSuccess || p.splits == 1) return e;
  hipLaunchKernelGGL(latent_prefill_combine_kernel, dim3((unsigned)(p.items * sh.H), 4), dim3(256), 0, stream, a, p.nt * 32);
  return hipGetLastError();
}

}  // namespace shainet
