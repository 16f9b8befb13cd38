// What the handles behind shainet_attn_ctx and shainet_kv_cache hold; shared by capi.hip, which
// implements both, and by the mixers that keep their rows in such a cache (latent_attn.hip).
#pragma once
#include <hip/hip_runtime.h>

#include <vector>

#include "../../include/shainet_hip_attn.h"
#include "attn_kernels.hpp"

namespace shainet {

// Grow-only device buffer.
struct DevBuf {
  float *p = nullptr;
  size_t cap = 0;  // floats
  int reserve(size_t n);
  void release();
};

// Grow-only pinned host buffer: host-pointer calls stage their rows through it, so that each
// copy to or from the device is one asynchronous DMA instead of the runtime's staged copy of
// pageable memory.
struct PinBuf {
  float *p = nullptr;
  size_t cap = 0;  // floats
  int reserve(size_t n);
  void release();
};

}  // namespace shainet

struct shainet_attn_ctx {
  int H, KV, g, hd;
  // A cache of this context holds, per position and kv head, hd floats in its K array and v_hd in
  // its V array.  v_hd = hd for rotated grouped-query attention; 0 for latent attention, whose one row
  // per position (KV = 1; hd = the padded row width) serves as key and as value.
  int v_hd;
  // > 0: a query reaches `window` rows back, its own row included, so a cache may forget older ones
  // (shainet_kv_cache_make_room); 0: all the way to position 0.
  int window = 0;
  // angles of the cos/sin table in fp64, rounded when the table is written (false: the fp32 product
  // position * frequency of llama_block.cr:274-277)
  bool rope_fp64 = false;
  double eps;
  float scale;  // (float)(1.0 / sqrt((double)hd)), llama_block.cr:249
  std::vector<double> inv_freq64;  // rope_fp64 only: the frequencies before rounding
  std::vector<float> inv_freq;
  float *d_q_norm = nullptr, *d_k_norm = nullptr;
  float *d_bq = nullptr, *d_bk = nullptr, *d_bv = nullptr;
  float2 *d_rope = nullptr;
  int rope_positions = 0;
  // DecodeArgs::ahead_* of the next decode launch (shainet_attn_read_ahead); forgotten after it
  const float *ahead_w = nullptr;
  int ahead_k = 0, ahead_n = 0, ahead_wgs = 0;
  hipStream_t stream = nullptr;      // where work is issued
  hipStream_t own_stream = nullptr;  // created with the context, destroyed with it
  shainet::DevBuf q_rot, partials, in_q, in_k, in_v, out;
  shainet::PinBuf pin_in, pin_out;  // host-pointer calls: q | k | v rows on their way in, the result on its way out
  // decode split: a word per partial slot that says when it is complete (zero between launches)
  unsigned *part_flag = nullptr;
  size_t part_flag_cap = 0;
  bool test_lose_marks = false;  // SHAINET_HIP_TEST_LOSE_PARTIAL_MARKS: exercises the give-up path
  // pinned host word this context's kernels set when they give up a bounded wait; `error` is
  // the one in use: the context's own, or the one of the block or model that owns the context
  int *error = nullptr, *own_error = nullptr;
  int last_rows = 0;
  int decode_wgs_override = 0;  // 0 = default workgroup count of the decode split
  int prefill_wgs_per_cu = 0;   // 0 = default occupancy of the prefill kernel
  int prefill_splits_override = 0;  // 0 = default number of key splits of the prefill kernel
  int prefill_groups_override = 0;  // 0 = default number of wavefront groups of the prefill kernel
  bool profiling = false;
  std::vector<hipEvent_t> prof_events;  // start, stop, start, stop, ...
};

// What shainet_attn_decode_step works with: all of it allocated by shainet_kv_cache_lengths_to_device,
// none of it by the step.
struct StepState {
  int *d_len = nullptr;               // [batch] cached rows per slot, as the device counts them
  int *pin_len = nullptr;             // [batch] pinned staging for both directions
  shainet::DecodeDevicePlan *d_plan = nullptr; // rewritten by every step
  float *q_rot = nullptr;             // [batch, H, hd]
  float *partials = nullptr;          // device_plan_slots(batch, KV) slots of g columns
  unsigned *flags = nullptr;          // zero between launches
  int cap = 0;                        // the capacity the buffers above were laid out for
  // Between shainet_kv_cache_lengths_to_device and _from_device the device's lengths are the ones that count
  // (decode steps advance only those): every entry point that reads or writes the host's copy is refused.
  bool lengths_on_device = false;
};

struct shainet_kv_cache {
  shainet_attn_ctx *ctx;
  int batch, cap;
  float *k = nullptr, *v = nullptr;  // v: null when the context's rows have no V half
  std::vector<int> len;              // positions appended so far, per sequence
  // per sequence: the position whose row lies first in the buffers.  0 until a windowed context's
  // rows outgrow the capacity and the ones nobody can see any more are dropped.
  std::vector<int> base;
  StepState step;
};

// A context for a mixer whose cache holds one row of row_width floats per position and no V array:
// num_heads query heads share it.  window: see the struct; the cos/sin table is that of rope_dims
// rotated dimensions, angles in fp64.
int shainet_attn_create_rows(shainet_attn_ctx **out, int num_heads, int row_width, int window, double rope_base,
                             int rope_dims, float scale, int max_positions);

// A context for grouped-query attention without rotation, whose values may have a width of their own.
int shainet_attn_create_unrotated(shainet_attn_ctx **out, int num_heads, int num_kv_heads, int dim, int v_dim, float scale);
// Attention of new_tokens queries (as DistanceBias lays them out) at positions start_pos .. over sequence 0 of
// a cache that holds their rows already.  The cache may be another context's of the same kind; its
// lengths are neither read nor changed.  Asynchronous on c's stream.
int shainet_attn_run_biased(shainet_attn_ctx *c, shainet_kv_cache *kc, const float *q, const shainet::DistanceBias &bias,
                            int start_pos, int new_tokens, float *out);

// Room for new_rows more rows of one sequence: drops rows that no later position can see (windowed
// contexts), else grows the buffers.  keep_back: rows that a later truncate may take back, at most;
// the rows those positions see stay too.
int shainet_kv_cache_make_room(shainet_kv_cache *kc, int seq, int new_rows, int keep_back);

namespace shainet {
// the context's cos/sin table reaches at least `positions` positions afterwards
int ensure_rope_table(shainet_attn_ctx *c, int positions);
}
