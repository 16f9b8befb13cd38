// Launchers of the latent-attention kernels: attention whose cache holds, per position, one row
// that all heads share: an RMS-normed latent vector c of kv_rank values and one rotated key part of
// rot_dim values, [c | rotated key | zeros up to row_w].  Head h's key is (W_uk,h c, rotated part),
// its value W_uv,h c.  Two ways to attend over such rows:
//
//   absorbed   W_uk moves to the query side (q_abs = W_uk,h^T q, rot(q)), scores and weighted sums
//              are taken over the cached rows as they are, and W_uv is applied to the weighted sum of
//              latents: every head reads the same row_w floats per position (decode, few rows);
//   expanded   keys and values of the visible positions are made by one product, and the attention
//              over them costs dim + rot_dim + vdim instead of row_w + kv_rank multiply-adds per
//              position and head (prefill).
//
// Device pointers only; every launcher checks the shapes its kernel assumes.
#pragma once
#include <hip/hip_runtime.h>

namespace shainet {

struct LatentShape {
  int H, dim, rot_dim, vdim, kv_rank;
  int rot_dims;   // the first rot_dims (even) of rot_dim turn; pair (2i, 2i + 1) by position * f_i
  int row_w;      // floats per cached row: kv_rank + rot_dim, padded to a multiple of 16
  int window;     // > 0: position p sees p - window + 1 .. p; 0: 0 .. p
  float scale;    // of the scores
};
inline int latent_row_width(int kv_rank, int rot_dim) { return (kv_rank + rot_dim + 15) / 16 * 16; }

// The input product's rows, [c_q | c | key part | gates | zeros], n_in floats each.
struct LatentRows {
  const float *raw;
  long long stride;
  int kv_off, gate_off;      // first column of c, of the H gates
  const float *kv_norm;      // [kv_rank]
  double eps;
  const float2 *rope_tab;    // [positions][rot_dims / 2] (cos, sin)
  float *rows;               // the sequence's cached rows
  int start_pos;             // position of the first new row
  int start_row;             // its place in `rows`
};

// rows[start_row + t] = [RMS(c) kv_norm | rotated key part | 0] for T new rows; the rotated parts of
// their queries q [T, H (dim + rot_dim)] turn in place (q nullable)
hipError_t launch_latent_append(const LatentRows &r, const LatentShape &sh, int T, float *q, hipStream_t stream);

// q [T, H (dim + rot_dim)] -> q_abs [T, H, row_w] = [W_uk,h^T q_h | rotated q_h | 0] * scale * log2(e),
// and the append of launch_latent_append in the same launch.  uk: [H dim, kv_rank].
hipError_t launch_latent_absorb(const float *q, const float *uk, const LatentRows &r, const LatentShape &sh, int T,
                                float *q_abs, hipStream_t stream);

// Attention of T rows over the cached ones, absorbed: partial results of `splits` key ranges per
// (row, head): part_o [tiles of 16 (row, head)][16][splits][v_w], part_ml the same with (max, sum), log2 units.
struct LatentPlan {
  int key_tile;       // 16 or 32 keys per step
  int col_tiles;      // tiles of 16 (row, head) pairs
  int splits, tiles_per_split;
  int v_w;            // kv_rank padded to a multiple of 16
  int v_slices;       // slices of at most 1024 of them, each a workgroup of its own
  size_t lds_bytes;
  size_t partial_floats;  // o and (max, sum) together
};
bool plan_latent_absorbed(const LatentShape &sh, int T, int start_row, LatentPlan &p);
hipError_t launch_latent_absorbed(const float *q_abs, const float *rows, float *partials, const LatentShape &sh, int T,
                                  int start_row, const LatentPlan &p, hipStream_t stream);

// out [T, H vdim] = sigmoid(gate_h) * W_uv,h (sum over the splits, sink in the denominator).
// uv: [H vdim, kv_rank]; sink: [H], natural units, counted once per row.
hipError_t launch_latent_out(const float *partials, const float *uv, const float *sink, const LatentRows &r,
                             const LatentShape &sh, int T, const LatentPlan &p, float *out, hipStream_t stream);

// Attention of T rows over expanded keys and values (q as launch_latent_append leaves it): kv [key_rows, H dim + H vdim] = the latents of cached rows
// first_row .. first_row + key_rows - 1 (the ones any of the T rows sees) times [W_uk | W_uv].  False: sizes
// that are no multiple of 4, dim + rot_dim above 256 or vdim above 128 (the absorbed form takes those).
struct LatentExpandedPlan {
  int first_row, key_rows;
  int nk, nt;       // instantiation: pieces of 8 query / key dimensions, tiles of 32 value dimensions
  int items;        // blocks of 128 rows
  int splits;       // key chunks per block; > 1 adds the combine kernel
  size_t partial_floats;
  bool pays;        // cheaper than the absorbed form
};
constexpr int kLatentKvSlack = 128;  // floats behind the last row of kv that the kernel may read (and drops)
bool plan_latent_expanded(const LatentShape &sh, int T, int start_row, LatentExpandedPlan &p);
hipError_t launch_latent_expanded(const float *q, const float *kv, const float *sink, const LatentRows &r,
                                  const LatentShape &sh, int T, const LatentExpandedPlan &p, float *partials, float *out,
                                  hipStream_t stream);

}  // namespace shainet
