// Latent attention as a block's mixer: the queries and the keys and values go through low-rank
// latents, and the cache holds one row per position that all heads share (latent_kernels.hpp).
// One row of the mixer's input x, normed on its way in, becomes
//   [c_q | c | key part | gates] = x [W_dq | W_dkv | W_g]      one product
//   q = RMS(c_q) W_uq                                          the norm rides in the product
//   row = [RMS(c) | rotated key part]                          appended to the cache
//   heads                                                      absorbed or expanded, see below
//   out = (x +) heads W_o
#include "latent_attn.hpp"

#include <stdlib.h>
#include <string.h>

#include <new>
#include <string>

#include "attn_context.hpp"
#include "attn_kernels.hpp"
#include "latent_kernels.hpp"

namespace shainet {

namespace {
int fail(int code, const std::string &msg) { return llama_fail(code, msg); }
constexpr int kInitialCapacity = 256;
// greedy generation looks at its ids every 16 steps and takes the steps after a stop token back:
// the rows those positions see must not have been dropped
constexpr int kTakeBack = 64;
// which form a call takes: the cheaper one, or (SHAINET_HIP_LATENT_PATH=absorbed|expanded, read when a
// mixer is made) one of them wherever its shapes allow
enum { kByCost = 0, kAbsorbed = 1, kExpanded = 2 };
int path_knob() {
  const char *env = getenv("SHAINET_HIP_LATENT_PATH");
  return env && !strcmp(env, "absorbed") ? kAbsorbed : env && !strcmp(env, "expanded") ? kExpanded : kByCost;
}
}  // namespace

struct LatentAttn {
  int d_model = 0;
  shainet_latent_config cfg = {};
  double eps = 1e-6;
  LatentShape sh = {};
  std::shared_ptr<LatentWeights> w;
  shainet_attn_ctx *ctx = nullptr;
  shainet_kv_cache *cache = nullptr, *scratch_cache = nullptr;
  int *shared_error = nullptr;
  Projector proj;
  int path = kByCost;
  DevF raw, q, q_abs, kv, partials, heads;
};

LatentWeights::~LatentWeights() {
  for (float *p : {w_in, w_in_t, dq_norm, dkv_norm, w_uq, w_uq_t, u_kv, w_ukv, sink, w_o, w_o_t})
    if (p) (void)hipFree(p);
}

int latent_attn_create(LatentAttn **out, int d_model, const shainet_latent_config &c, double eps,
                       const LatentAttn *weights_of) {
  *out = nullptr;
  if (d_model < 1 || c.heads < 1 || c.dim < 1 || c.rot_dim < 0 || c.vdim < 1 || c.kv_rank < 1 || c.q_rank < 1 ||
      c.window < 0)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "latent attention: sizes must be positive");
  if (c.rot_dims < 0 || c.rot_dims > c.rot_dim || (c.rot_dims & 1))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "latent attention: rot.dims must be even and at most rot_dim");
  if (c.rot_dims > 0 && !(c.rot_base > 0.0)) return fail(SHAINET_HIP_ERR_ARGUMENT, "latent attention: rot.base must be positive");
  LatentShape sh = {};
  sh.H = c.heads;
  sh.dim = c.dim;
  sh.rot_dim = c.rot_dim;
  sh.vdim = c.vdim;
  sh.kv_rank = c.kv_rank;
  sh.rot_dims = c.rot_dims;
  sh.row_w = latent_row_width(c.kv_rank, c.rot_dim);
  sh.window = c.window;
  sh.scale = (float)c.scale;
  LatentPlan plan;
  if (!plan_latent_absorbed(sh, 1, 0, plan))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "latent attention: kv_rank + rot_dim is too large for a compute unit's LDS (about 1200 floats)");
  if (weights_of && (weights_of->d_model != d_model || memcmp(&weights_of->cfg, &c, sizeof c) != 0 || weights_of->eps != eps))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "latent attention: layers that share weights must have the same mixer");
  LatentAttn *l = new (std::nothrow) LatentAttn();
  if (!l) return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  l->d_model = d_model;
  l->cfg = c;
  l->eps = eps;
  l->sh = sh;
  l->path = path_knob();
  int rc = SHAINET_HIP_OK;
  if (weights_of) {
    l->w = weights_of->w;
  } else {
    l->w = std::make_shared<LatentWeights>();
    LatentWeights &w = *l->w;
    w.n_in = (c.q_rank + c.kv_rank + c.rot_dim + c.heads + 3) / 4 * 4;
    const size_t d = (size_t)d_model, qw = (size_t)c.heads * (c.dim + c.rot_dim), ukv = (size_t)c.heads * (c.dim + c.vdim);
    struct Want {
      float **p;
      size_t n;
    } wants[] = {{&w.w_in, d * w.n_in},          {&w.dq_norm, (size_t)c.q_rank}, {&w.dkv_norm, (size_t)c.kv_rank},
                 {&w.w_uq, (size_t)c.q_rank * qw}, {&w.u_kv, ukv * c.kv_rank},     {&w.w_ukv, ukv * c.kv_rank},
                 {&w.sink, (size_t)c.heads},     {&w.w_o, (size_t)c.heads * c.vdim * d}};
    for (const Want &x : wants)
      if (!rc && hipMalloc((void **)x.p, x.n * sizeof(float)) != hipSuccess) {
        *x.p = nullptr;
        rc = fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
      }
    // (the columns of w_in past the last gate are never filled by a loader)
    if (!rc && hipMemset(w.w_in, 0, d * w.n_in * sizeof(float)) != hipSuccess)
      rc = fail(SHAINET_HIP_ERR_RUNTIME, "hipMemset failed");
  }
  if (!rc) rc = shainet_attn_create_rows(&l->ctx, c.heads, sh.row_w, c.window, c.rot_base, c.rot_dims, sh.scale, kInitialCapacity);
  if (!rc) rc = shainet_kv_cache_create(&l->cache, l->ctx, 1, kInitialCapacity);
  if (rc) {
    latent_attn_destroy(l);
    return rc;
  }
  l->proj.error = shainet_attn_error_word(l->ctx);
  *out = l;
  return SHAINET_HIP_OK;
}

void latent_attn_destroy(LatentAttn *l) {
  if (!l) return;
  if (l->scratch_cache) shainet_kv_cache_destroy(l->scratch_cache);
  if (l->cache) shainet_kv_cache_destroy(l->cache);
  if (l->ctx) shainet_attn_destroy(l->ctx);
  l->proj.release();
  for (DevF *b : {&l->raw, &l->q, &l->q_abs, &l->kv, &l->partials, &l->heads}) b->release();
  delete l;
}

LatentWeights &latent_attn_weights(LatentAttn *l) { return *l->w; }
const shainet_latent_config &latent_attn_config(const LatentAttn *l) { return l->cfg; }
shainet_attn_ctx *latent_attn_context(LatentAttn *l) { return l->ctx; }
shainet_kv_cache *latent_attn_cache(LatentAttn *l) { return l->cache; }
Projector &latent_attn_projector(LatentAttn *l) { return l->proj; }
int latent_attn_reserve(LatentAttn *l, int positions) {
  long long rows = positions;
  // (twice what must stay: rows move to the front of the buffer once per that many positions)
  if (l->sh.window && rows > 2LL * (l->sh.window + kTakeBack)) rows = 2LL * (l->sh.window + kTakeBack);
  if (rows > 0x7fffffffLL) rows = 0x7fffffffLL;
  return shainet_kv_cache_reserve(l->cache, (int)rows);
}
void latent_attn_share_error_word(LatentAttn *l, int *word) {
  l->shared_error = word;
  shainet_attn_adopt_error_word(l->ctx, word);
  l->proj.error = shainet_attn_error_word(l->ctx);
}

int latent_attn_forward(LatentAttn *l, const float *x, int T, float *out, const Fused &pre, const float *residual,
                        bool no_cache) {
  const LatentShape &sh = l->sh;
  LatentWeights &w = *l->w;
  shainet_attn_ctx *ctx = l->ctx;
  hipStream_t stream = ctx->stream;
  const int qw = sh.H * (sh.dim + sh.rot_dim), vw = sh.H * sh.vdim, q_rank = l->cfg.q_rank, d = l->d_model;
  int rc = SHAINET_HIP_OK;
  shainet_kv_cache *cache = l->cache;
  if (no_cache) {
    if (!l->scratch_cache && (rc = shainet_kv_cache_create(&l->scratch_cache, ctx, 1, T > kInitialCapacity ? T : kInitialCapacity)))
      return rc;
    cache = l->scratch_cache;
    if ((rc = shainet_kv_cache_clear(cache, -1))) return rc;
  }
  if ((rc = shainet_kv_cache_make_room(cache, 0, T, no_cache ? 0 : kTakeBack))) return rc;
  const int start_pos = cache->len[0], start_row = start_pos - cache->base[0];
  if ((rc = ensure_rope_table(ctx, start_pos + T))) return rc;
  if (!l->raw.reserve((size_t)T * w.n_in) || !l->q.reserve((size_t)T * qw) || !l->heads.reserve((size_t)T * vw))
    return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");

  // [c_q | c | key part | gates]
  Fused in = pre;
  if (gemvt_takes(T, d, w.n_in, in.epilogue, in.norm)) in.w_t = transposed_twin(&w.w_in_t, &w.w_in_t_stale, w.w_in, d, w.n_in, stream);
  if ((rc = l->proj.project(x, d, w.w_in, l->raw.p, T, d, w.n_in, stream, in))) return rc;
  // q = RMS(c_q) W_uq
  Fused up;
  up.norm = kNormRms;
  up.gamma = w.dq_norm;
  up.eps = l->eps;
  if (gemvt_takes(T, q_rank, qw, up.epilogue, up.norm)) {
    up.w_t = transposed_twin(&w.w_uq_t, &w.w_uq_t_stale, w.w_uq, q_rank, qw, stream, w.dq_norm);
    up.w_t_has_gamma = up.w_t != nullptr;
  }
  if ((rc = l->proj.project(l->raw.p, w.n_in, w.w_uq, l->q.p, T, q_rank, qw, stream, up))) return rc;

  LatentRows r = {};
  r.raw = l->raw.p;
  r.stride = w.n_in;
  r.kv_off = q_rank;
  r.gate_off = q_rank + sh.kv_rank + sh.rot_dim;
  r.kv_norm = w.dkv_norm;
  r.eps = l->eps;
  r.rope_tab = ctx->d_rope;
  r.rows = cache->k;
  r.start_pos = start_pos;
  r.start_row = start_row;
  LatentExpandedPlan ex;
  hipError_t e;
  if (l->path != kAbsorbed && plan_latent_expanded(sh, T, start_row, ex) && (ex.pays || l->path == kExpanded)) {
    const int kvw = sh.H * (sh.dim + sh.vdim);
    if (!l->kv.reserve((size_t)ex.key_rows * kvw + kLatentKvSlack) || !l->partials.reserve(ex.partial_floats))
      return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    e = launch_latent_append(r, sh, T, l->q.p, stream);
    if (e == hipSuccess) {
      // keys and values of every position the new rows see
      if ((rc = l->proj.project(cache->k + (size_t)ex.first_row * sh.row_w, sh.row_w, w.w_ukv, l->kv.p, ex.key_rows,
                                sh.kv_rank, kvw, stream)))
        return rc;
      e = launch_latent_expanded(l->q.p, l->kv.p, w.sink, r, sh, T, ex, l->partials.p, l->heads.p, stream);
    }
  } else {
    LatentPlan plan;
    if (!plan_latent_absorbed(sh, T, start_row, plan)) return fail(SHAINET_HIP_ERR_ARGUMENT, "too many rows in one call");
    if (!l->q_abs.reserve((size_t)T * sh.H * sh.row_w) || !l->partials.reserve(plan.partial_floats))
      return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    e = launch_latent_absorb(l->q.p, w.u_kv, r, sh, T, l->q_abs.p, stream);
    if (e == hipSuccess) e = launch_latent_absorbed(l->q_abs.p, cache->k, l->partials.p, sh, T, start_row, plan, stream);
    if (e == hipSuccess)
      e = launch_latent_out(l->partials.p, w.u_kv + (size_t)sh.H * sh.dim * sh.kv_rank, w.sink, r, sh, T, plan, l->heads.p, stream);
  }
  if (e != hipSuccess) return fail(SHAINET_HIP_ERR_RUNTIME, std::string("latent attention launch: ") + hipGetErrorString(e));
  if (no_cache) {
    if ((rc = shainet_kv_cache_clear(cache, -1))) return rc;
  } else {
    cache->len[0] += T;
  }
  Fused post;
  if (residual) {
    post.epilogue = kGemvResidual;
    post.res = residual;
  }
  if (gemvt_takes(T, vw, d, post.epilogue, post.norm)) post.w_t = transposed_twin(&w.w_o_t, &w.w_o_t_stale, w.w_o, vw, d, stream);
  return l->proj.project(l->heads.p, vw, w.w_o, out, T, vw, d, stream, post);
}

}  // namespace shainet
