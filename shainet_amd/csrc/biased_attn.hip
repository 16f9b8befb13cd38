// Grouped-query attention as a block's mixer, without rotation: positions enter through a table of values by
// head and distance that are added to the scores (DistanceBias in attn_kernels.hpp; the kernels are the
// ones of rotated attention).  Value heads may be wider or narrower than key heads, and a layer may
// attend over another layer's keys and values with queries of its own.
#include "biased_attn.hpp"

#include <math.h>

#include <new>
#include <string>

#include "attn_context.hpp"
#include "attn_kernels.hpp"

namespace shainet {

namespace {
int fail(int code, const std::string &msg) { return llama_fail(code, msg); }
constexpr int kInitialCapacity = 256;
}  // namespace

int allocate_buffers(const WantedBuffer *wants, int count) {
  for (int i = 0; i < count; ++i)
    if (wants[i].n && !*wants[i].p && hipMalloc((void **)wants[i].p, wants[i].n * sizeof(float)) != hipSuccess) {
      *wants[i].p = nullptr;
      return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    }
  return SHAINET_HIP_OK;
}

int distance_bucket(int n, int rows, int bias_max) {
  const int half = rows / 2;
  if (n < half) return n;
  if (n >= bias_max || half < 1 || bias_max <= half) return rows - 1;
  const double x = log((double)n / half) / log((double)bias_max / half) * (rows - half);
  // (a bucket that begins exactly at n must not be missed for the last bit of a logarithm)
  const double near = nearbyint(x);
  const int b = half + (int)(fabs(x - near) < 1e-9 ? near : floor(x));
  return b < rows - 1 ? b : rows - 1;
}

struct BiasedAttn : Mixer {
  int d_model = 0;
  BiasedConfig cfg;
  BiasedWeights w;
  BiasedAttn *from = nullptr;
  shainet_attn_ctx *ctx = nullptr;
  shainet_kv_cache *kv = nullptr, *scratch = nullptr;  // null in a borrowing layer
  int rows = 0;                                        // positions so far
  float *table = nullptr;
  DistanceBias bias = {};
  Projector proj;
  DevF raw, heads;

  ~BiasedAttn() override {
    if (scratch) shainet_kv_cache_destroy(scratch);
    if (kv) shainet_kv_cache_destroy(kv);
    if (ctx) shainet_attn_destroy(ctx);
    proj.release();
    raw.release();
    heads.release();
    for (float *p : {w.w_in, w.w_in_t, w.w_o, w.w_o_t, table})
      if (p) (void)hipFree(p);
  }
  hipStream_t stream() override { return ctx->stream; }
  int set_stream(hipStream_t s) override { return shainet_attn_set_stream(ctx, (void *)s); }
  int *error_word() override { return shainet_attn_error_word(ctx); }
  void share_error_word(int *word) override {
    shainet_attn_adopt_error_word(ctx, word);
    proj.error = shainet_attn_error_word(ctx);
  }
  Projector &projector() override { return proj; }
  int reserve(int positions) override { return kv ? shainet_kv_cache_reserve(kv, positions) : SHAINET_HIP_OK; }
  int clear() override {
    rows = 0;
    return kv ? shainet_kv_cache_clear(kv, -1) : SHAINET_HIP_OK;
  }
  int len() override { return rows; }
  int truncate(int len) override {
    if (len < 0 || len > rows) return fail(SHAINET_HIP_ERR_ARGUMENT, "truncate beyond the cached length");
    rows = len;
    return kv ? shainet_kv_cache_truncate(kv, 0, len) : SHAINET_HIP_OK;
  }
  shainet_kv_cache *cache() override { return kv ? kv : from->kv; }
  BiasedAttn *biased() override { return this; }

  int forward(const float *x, int T, float *out, const Fused &pre, const float *residual, bool no_cache) override {
    const int H = cfg.heads, KV = cfg.kv_heads, dim = cfg.dim, vdim = cfg.vdim, d = d_model, qw = H * dim;
    if (!table) return fail(SHAINET_HIP_ERR_ARGUMENT, "weights not set");
    hipStream_t s = ctx->stream;
    int rc = SHAINET_HIP_OK;
    const int start = no_cache ? 0 : rows;
    BiasedAttn *owner = from ? from : this;
    if (!from && no_cache && !scratch && (rc = shainet_kv_cache_create(&scratch, ctx, 1, T > kInitialCapacity ? T : kInitialCapacity)))
      return rc;
    shainet_kv_cache *cache = no_cache ? owner->scratch : owner->kv;
    if (!from && (rc = no_cache ? shainet_kv_cache_reserve(cache, T) : shainet_kv_cache_make_room(cache, 0, T, 0))) return rc;
    if (from && !no_cache && from->rows != start + T)
      return fail(SHAINET_HIP_ERR_ARGUMENT, "a layer that attends over another layer's keys has to run behind it");
    if (!raw.reserve((size_t)T * w.n_in) || !heads.reserve((size_t)T * H * vdim)) return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    DistanceBias b = bias;
    b.q_stride = w.n_in;
    Fused in = pre;
    const bool fuse = !from && T <= 16 && dim == vdim && (w.n_in & 3) == 0 && dim >= 2 && dim <= 128 && (dim & (dim - 1)) == 0;
    if (fuse) {
      // few rows: key and value heads go to the cache where the product sums them up
      GemvPrep p = {};
      p.q_rot = raw.p;
      p.kc = cache->k;
      p.vc = cache->v;
      p.H = H;
      p.KV = KV;
      p.hd = dim;
      p.cap = cache->cap;
      p.start_pos = start;
      b.q_stride = qw;
      in.epilogue = kGemvQkvPrep;
      in.prep = &p;
      if (gemvt_takes(T, d, w.n_in, in.epilogue, in.norm, &p)) in.w_t = transposed_twin(&w.w_in_t, &w.w_in_t_stale, w.w_in, d, w.n_in, s);
      if ((rc = proj.project(x, d, w.w_in, nullptr, T, d, w.n_in, s, in))) return rc;
    } else {
      if (gemvt_takes(T, d, w.n_in, in.epilogue, in.norm)) in.w_t = transposed_twin(&w.w_in_t, &w.w_in_t_stale, w.w_in, d, w.n_in, s);
      if ((rc = proj.project(x, d, w.w_in, raw.p, T, d, w.n_in, s, in))) return rc;
      if (!from) {
        const hipError_t e = launch_append_rows(raw.p, w.n_in, qw, qw + KV * dim, T, cache->k, cache->v, KV, dim, vdim, cache->cap, start, s);
        if (e != hipSuccess) return fail(SHAINET_HIP_ERR_RUNTIME, std::string("append launch: ") + hipGetErrorString(e));
      }
    }
    if ((rc = shainet_attn_run_biased(ctx, cache, raw.p, b, start, T, heads.p))) return rc;
    if (!no_cache) {
      rows += T;
      if (kv) kv->len[0] = rows;
    }
    Fused post;
    if (residual) {
      post.epilogue = kGemvResidual;
      post.res = residual;
    }
    if (gemvt_takes(T, H * vdim, d, post.epilogue, post.norm)) post.w_t = transposed_twin(&w.w_o_t, &w.w_o_t_stale, w.w_o, H * vdim, d, s);
    return proj.project(heads.p, H * vdim, w.w_o, out, T, H * vdim, d, s, post);
  }
};

int biased_attn_create(Mixer **out, int d_model, const BiasedConfig &c, Mixer *kv_from) {
  *out = nullptr;
  if (d_model < 1 || c.heads < 1 || c.kv_heads < 1 || c.heads % c.kv_heads || c.dim < 1 || c.vdim < 1 || c.bias_max < 1)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "attention: sizes must be positive, and heads a multiple of kv_heads");
  if (c.dim > 8192 || c.vdim > 8192) return fail(SHAINET_HIP_ERR_ARGUMENT, "attention: heads of more than 8192 values are not supported");
  BiasedAttn *from = kv_from ? kv_from->biased() : nullptr;
  if (kv_from && (!from || from->from || from->d_model != d_model || from->cfg.kv_heads != c.kv_heads || from->cfg.dim != c.dim ||
                  from->cfg.vdim != c.vdim))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "attention: keys and values can be borrowed from a layer with the same heads and projections of its own");
  BiasedAttn *l = new (std::nothrow) BiasedAttn();
  if (!l) return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  l->d_model = d_model;
  l->cfg = c;
  l->from = from;
  l->w.n_in = c.heads * c.dim + (from ? 0 : c.kv_heads * (c.dim + c.vdim));
  const WantedBuffer wants[] = {{&l->w.w_in, (size_t)d_model * l->w.n_in}, {&l->w.w_o, (size_t)c.heads * c.vdim * d_model}};
  int rc = allocate_buffers(wants, 2);
  if (!rc) rc = shainet_attn_create_unrotated(&l->ctx, c.heads, c.kv_heads, c.dim, c.vdim, (float)c.scale);
  if (!rc && !from) rc = shainet_kv_cache_create(&l->kv, l->ctx, 1, kInitialCapacity);
  if (rc) {
    delete l;
    return rc;
  }
  l->proj.error = shainet_attn_error_word(l->ctx);
  *out = l;
  return SHAINET_HIP_OK;
}

BiasedWeights &biased_attn_weights(BiasedAttn *l) { return l->w; }

int biased_attn_set_table(BiasedAttn *l, const std::vector<float> &rel, int rows, int max_positions) {
  const int H = l->cfg.heads;
  if (rows < 1 || rel.size() != (size_t)rows * H || max_positions < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "attention: the table by distance has no rows");
  // `reach`: distances that do not use the last row yet (as far as there are any)
  int reach = 0;
  while (reach < max_positions && distance_bucket(reach, rows, l->cfg.bias_max) < rows - 1) ++reach;
  DistanceBias &b = l->bias;
  b.stride = (reach + 2 * kDistancePad + 3) / 4 * 4;
  b.origin = reach + kDistancePad - 1;
  b.reach = reach;
  b.v_hd = l->cfg.vdim;
  std::vector<float> tab((size_t)H * b.stride, 0.f);
  for (int n = 0; n < reach; ++n) {
    const int row = distance_bucket(n, rows, l->cfg.bias_max);
    for (int h = 0; h < H; ++h)
      tab[(size_t)h * b.stride + b.origin - n] =
          (float)(((double)rel[(size_t)row * H + h] - (double)rel[(size_t)(rows - 1) * H + h]) * 1.4426950408889634);
  }
  const int rc = upload_floats(&l->table, tab.data(), tab.size());
  b.tab = l->table;
  return rc;
}

}  // namespace shainet
