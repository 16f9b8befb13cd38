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
#include "latent_kernels.hpp"

#include <math.h>
#include <stdint.h>
#include <stdlib.h>

namespace shainet {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

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

__global__ __launch_bounds__(256) void latent_append_kernel(LatentRows r, LatentShape sh) {
  append_row(r, sh, blockIdx.x);
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

// Column c of tile ct is (row, head) pair 16 ct + c = row * H + head.  The workgroup walks its share
// of the tile's keys in steps of KT: the cached rows go to LDS once and serve as keys (the scores'
// contraction is shared between the wavefronts) and as values (the wavefronts share the columns of
// the output, NTW tiles of 16 each).  Row stride row_w + 4 in LDS: 16-byte reads down a column of
// rows, and reads of 16 neighbours in rows 4 j apart, touch every bank once.
template <int KT, int NTW>
__global__ __launch_bounds__(256) void latent_absorbed_kernel(const float *__restrict__ q_abs,
                                                              const float *__restrict__ rows,
                                                              float *__restrict__ part_o, float *__restrict__ part_ml,
                                                              LatentShape sh, int T, int start_row, int splits,
                                                              int tiles_per_split, int v_w) {
  constexpr int SUB = KT / 16, PARTS = 4 / SUB;
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

  auto stage = [&](float *dst, const float *src, int count, int last) {  // `count` rows, the ones past `last` repeat it
    constexpr int U = 8;
    for (int i0 = threadIdx.x; i0 < count * w4; i0 += 256 * U) {
      f32x4 v[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int i = min(i0 + 256 * u, count * w4 - 1), rr = i / w4;
        v[u] = *(const f32x4 *)(src + (long long)min(rr, last) * row_w + 4 * (i - rr * w4));
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int i = i0 + 256 * u, rr = i / w4;
        if (i < count * w4) *(f32x4 *)(dst + rr * ldr + 4 * (i - rr * w4)) = v[u];
      }
    }
  };

  float m = -INFINITY, l = 0.f;
  f32x4 acc[NTW];
#pragma unroll
  for (int i = 0; i < NTW; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  if (tile0 < tile1) stage(qs, q_abs + (long long)v0 * row_w, 16, v1 - v0);
  const int sub = wave % SUB, part = wave / SUB;
  const int steps = row_w >> 4, s_begin = part * steps / PARTS, s_end = (part + 1) * steps / PARTS;
  const int v_tiles = min((v_w - d_first) >> 4, 64);
  for (int tile = tile0; tile < tile1; ++tile) {
    const int k0 = lo + tile * KT;
    stage(ks, rows + (long long)k0 * row_w, KT, hi - k0);
    __syncthreads();
    {
      f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
      const float *kp = ks + (16 * sub + n) * ldr + 4 * j, *qp = qs + n * ldr + 4 * j;
      for (int i = s_begin; i < s_end; ++i) {
        const f32x4 a = *(const f32x4 *)(kp + 16 * i), b = *(const f32x4 *)(qp + 16 * i);
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
      const int vt = wave + 4 * i;
      if (vt < v_tiles) {
        const float *vp = ks + 4 * j * ldr + d_first + 16 * vt + n;
#pragma unroll
        for (int u = 0; u < SUB; ++u)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(vp[(16 * u + r) * ldr], p[u][r], acc[i], 0, 0, 0);
      }
    }
    __syncthreads();  // the rows are free for the next step's
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  const long long slot = (long long)(v0 + n) * splits + sp;
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    const int vt = wave + 4 * i;
    if (vt < v_tiles) *(f32x4 *)(part_o + slot * v_w + d_first + 16 * vt + 4 * j) = acc[i];
  }
  if (wave == 0 && j == 0 && blockIdx.z == 0) *(float2 *)(part_ml + 2 * slot) = float2{m, l};
}

// blockIdx: x = outputs VB x .. of the head, y = head, z = rows RT z ..: the key ranges' sums of
// latents are merged into LDS, then a wavefront per output takes its row of W_uv.
template <int RT>
__global__ __launch_bounds__(256) void latent_out_kernel(const float *__restrict__ part_o,
                                                         const float *__restrict__ part_ml,
                                                         const float *__restrict__ uv, const float *__restrict__ sink,
                                                         LatentRows r, LatentShape sh, int T, int splits, int v_w,
                                                         int per_wg, float *__restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float smem[];  // [RT][v_w] latents, then [RT][splits] factors
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int h = blockIdx.y, t0 = blockIdx.z * RT, nt = min(RT, T - t0);
  float *lat = smem, *fac = smem + RT * v_w;
  // the factor of a range: 2^(max - overall max) / denominator, the sink included in both
  for (int a = wave; a < nt; a += 4) {
    const float2 *ml = (const float2 *)part_ml + ((long long)(t0 + a) * sh.H + h) * splits;
    const float sk = sink[h] * kLog2e;
    float mm = sk;
    for (int s = lane; s < splits; s += 64) mm = fmaxf(mm, ml[s].x);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mm = fmaxf(mm, __shfl_xor(mm, o));
    float den = 0.f;
    for (int s = lane; s < splits; s += 64) den += ml[s].y * fast_exp2(ml[s].x - mm);  // (an empty range: 0 * 0)
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) den += __shfl_xor(den, o);
    const float inv = 1.f / (den + fast_exp2(sk - mm));
    for (int s = lane; s < splits; s += 64) fac[a * splits + s] = fast_exp2(ml[s].x - mm) * inv;
  }
  __syncthreads();
  const int v4 = v_w >> 2;
  for (int i = threadIdx.x; i < nt * v4; i += 256) {
    const int a = i / v4, c = i - a * v4;
    const float *po = part_o + ((long long)(t0 + a) * sh.H + h) * splits * v_w + 4 * c;
    f32x4 sum = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < splits; s0 += 8) {
      f32x4 x[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) x[u] = *(const f32x4 *)(po + (long long)min(s0 + u, splits - 1) * v_w);
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (s0 + u < splits) sum += fac[a * splits + s0 + u] * x[u];
    }
    *(f32x4 *)(lat + a * v_w + 4 * c) = sum;
  }
  __syncthreads();
  const int j1 = min(sh.vdim, ((int)blockIdx.x + 1) * per_wg);
  for (int jj = blockIdx.x * per_wg + wave; jj < j1; jj += 4) {
    const float *wr = uv + ((long long)h * sh.vdim + jj) * sh.kv_rank;
    float s[RT];
#pragma unroll
    for (int a = 0; a < RT; ++a) s[a] = 0.f;
    for (int c0 = lane; c0 < sh.kv_rank; c0 += 64 * 8) {
      float w[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) w[u] = wr[min(c0 + 64 * u, sh.kv_rank - 1)];
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (c0 + 64 * u < sh.kv_rank) {
#pragma unroll
          for (int a = 0; a < RT; ++a) s[a] += w[u] * lat[a * v_w + c0 + 64 * u];
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

hipError_t launch_latent_append(const LatentRows &r, const LatentShape &sh, int T, hipStream_t stream) {
  if (!rows_ok(r, sh, T)) return hipErrorInvalidValue;
  hipLaunchKernelGGL(latent_append_kernel, dim3((unsigned)T), dim3(256), 0, stream, r, sh);
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
  p.key_tile = sh.row_w <= 320 ? 32 : 16;
  const size_t ldr = (size_t)sh.row_w + 4;
  p.lds_bytes = ((16 + p.key_tile) * ldr + (size_t)4 * 16 * 17) * sizeof(float);
  if (p.lds_bytes > kMaxLds) return false;
  p.col_tiles = (T * sh.H + 15) / 16;
  // the most keys a tile of columns walks: the visible ones of its last row and of the rows before it
  const int rows_per_tile = (15 + sh.H) / sh.H + 1;
  long long keys = (long long)start_row + T;
  if (sh.window && keys > sh.window + rows_per_tile) keys = (long long)sh.window + rows_per_tile;
  const int tiles = (int)((keys + p.key_tile - 1) / p.key_tile) + 1;
  static const int target_knob = getenv("SHAINET_HIP_LATENT_WGS") ? atoi(getenv("SHAINET_HIP_LATENT_WGS")) : 0;
  const int target = target_knob > 0 ? target_knob : 256;
  int splits = (target + p.col_tiles - 1) / p.col_tiles;
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
  const int ntw = (slice / 16 + 3) / 4;
#define SHAINET_LAUNCH_ABSORBED(KT_, NTW_)                                                                               \
  do {                                                                                                                   \
    static const hipError_t a_ = hipFuncSetAttribute((const void *)latent_absorbed_kernel<KT_, NTW_>,                           \
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds);                 \
    if (a_ != hipSuccess) return a_;                                                                                    \
    hipLaunchKernelGGL((latent_absorbed_kernel<KT_, NTW_>), grid, dim3(256), p.lds_bytes, stream, q_abs, rows, part_o,  \
                       part_ml, sh, T, start_row, p.splits, p.tiles_per_split, p.v_w);                                  \
  } while (0)
#define SHAINET_LAUNCH_ABSORBED_K(NTW_)  \
  do {                                   \
    if (p.key_tile == 32)                \
      SHAINET_LAUNCH_ABSORBED(32, NTW_); \
    else                                 \
      SHAINET_LAUNCH_ABSORBED(16, NTW_); \
  } while (0)
  if (ntw <= 2)
    SHAINET_LAUNCH_ABSORBED_K(2);
  else if (ntw <= 4)
    SHAINET_LAUNCH_ABSORBED_K(4);
  else if (ntw <= 8)
    SHAINET_LAUNCH_ABSORBED_K(8);
  else
    SHAINET_LAUNCH_ABSORBED_K(16);
#undef SHAINET_LAUNCH_ABSORBED_K
#undef SHAINET_LAUNCH_ABSORBED
  return hipGetLastError();
}

hipError_t launch_latent_out(const float *partials, const float *uv, const float *sink, const LatentRows &r,
                             const LatentShape &sh, int T, const LatentPlan &p, float *out, hipStream_t stream) {
  if (!rows_ok(r, sh, T) || !partials || !uv || !sink || !out || sh.H > 65535) return hipErrorInvalidValue;
  const float *part_ml = partials + (size_t)p.col_tiles * 16 * p.splits * p.v_w;
  const int per_wg = 16;
  const int rt = T == 1 ? 1 : 4;
  const size_t lds = (size_t)rt * (p.v_w + p.splits) * sizeof(float);
  if (lds > 64 * 1024 || (T + rt - 1) / rt > 65535) return hipErrorInvalidValue;
  const dim3 grid((unsigned)((sh.vdim + per_wg - 1) / per_wg), (unsigned)sh.H, (unsigned)((T + rt - 1) / rt));
  if (rt == 1)
    hipLaunchKernelGGL(latent_out_kernel<1>, grid, dim3(256), lds, stream, partials, part_ml, uv, sink, r, sh, T, p.splits,
                       p.v_w, per_wg, out);
  else
    hipLaunchKernelGGL(latent_out_kernel<4>, grid, dim3(256), lds, stream, partials, part_ml, uv, sink, r, sh, T, p.splits,
                       p.v_w, per_wg, out);
  return hipGetLastError();
}

}  // namespace shainet
