// Host mirror of the attention half of SHAInet's LlamaBlock
// (src/shainet/transformer/llama_block.cr): the state the reference keeps per
// block (weights in [in, out] layout, optional biases, QK-norm weights, RoPE
// parameters, the KV cache and @cache_len) and attention_cached_cpu (246-299)
// with every step on the device: Q/K/V projections, bias, QK-norm, RoPE,
// append, causal GQA attention, output projection.  Activations stay in HBM
// between the steps; only x comes in and the [T, d_model] result goes out.
//
// The second half of this file adds what LlamaBlock#forward_cached
// (llama_block.cr:189-196) does around attention: the two RMSNorms, the two
// residual adds and the dense SwiGLU feed-forward, again all on the device.
// A block's parts are parameters: its mixer is the attention above or one of those
// behind the Mixer interface (latent_attn.hip, biased_attn.hip, hgrn2.hip), its norms
// RMSNorm or Dynamic Tanh, its feed-forward another kind (feed_forward.hip) or
// missing, and its weights may be another block's.  A block with norms behind its
// sublayers, too, and convolutions over time in front of them takes a forward pass of
// its own (wrapped_forward_device).
#include <hip/hip_runtime.h>
#include <math.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>

#include <memory>
#include <new>
#include <string>
#include <vector>

#include "../../include/shainet_hip_attn.h"
#include "attn_kernels.hpp"
#include "attn_context.hpp"
#include "block_kernels.hpp"
#include "feed_forward.hpp"
#include "hgrn2.hpp"
#include "latent_attn.hpp"
#include "llama_internal.hpp"
#include "mixer.hpp"
#include "residual_kernels.hpp"
#include "step_kernel.hpp"

using namespace shainet;

namespace {
int fail(int code, const std::string &msg) { return llama_fail(code, msg); }
}  // namespace

struct shainet_llama_attn {
  // llama_block.cr:10-28
  int d_model, num_heads, num_kv_heads, head_dim, q_dim, kv_dim;
  double qk_norm_eps, rope_theta;
  std::vector<float> rope_freqs, q_norm, k_norm, b_q, b_k, b_v;
  bool has_rope_freqs = false, has_q_norm = false, has_k_norm = false, has_bq = false, has_bk = false, has_bv = false;
  bool params_dirty = true;  // setters may run after construction (hf_loader.cr:319-373)
  float *w_qkv = nullptr, *w_o = nullptr;  // device, [in, out]; w_q | w_k | w_v side by side in one matrix
  // w_o once more, transposed ([d_model, q_dim]), for the product of a single row (launch_gemvt):
  // made on the device when such a call first needs it, made again after the weights change
  // (and q | k | v, [q_dim + 2 kv_dim, d_model], for layers without QK-norm)
  float *w_o_t = nullptr, *w_qkv_t = nullptr;
  bool w_o_t_stale = true, w_qkv_t_stale = true;
  // the norm weights multiplied into the rows of w_qkv_t (null: none), and whether any were
  const float *w_qkv_t_gamma = nullptr;
  shainet_attn_ctx *ctx = nullptr;
  shainet_kv_cache *cache = nullptr;
  shainet_kv_cache *scratch_cache = nullptr;  // rows of a no-cache forward call; empty between calls
  int cache_len = 0;  // @cache_len
  int *shared_error = nullptr;  // the error word of the model that owns this block, if one does
  Projector proj;
  DevF x, qkv, attn, out;
  PinnedF x_pin, out_pin;  // host-pointer calls stage their rows here
};

namespace {

constexpr int kInitialCapacity = 256;  // llama_block.cr:500

void drop_context(shainet_llama_attn *l) {
  if (l->scratch_cache) shainet_kv_cache_destroy(l->scratch_cache);
  l->scratch_cache = nullptr;
  if (l->cache) shainet_kv_cache_destroy(l->cache);
  if (l->ctx) shainet_attn_destroy(l->ctx);
  l->cache = nullptr;
  l->ctx = nullptr;
}

// Build (or rebuild after a setter ran) the attention context; the cache is
// cleared by a rebuild, which only happens between conversations in practice.
int ensure_context(shainet_llama_attn *l) {
  if (l->ctx && !l->params_dirty) return SHAINET_HIP_OK;
  drop_context(l);
  l->cache_len = 0;
  int rc = shainet_attn_create(&l->ctx, l->num_heads, l->num_kv_heads, l->head_dim, l->rope_theta,
                               l->has_rope_freqs ? l->rope_freqs.data() : nullptr,
                               l->has_q_norm ? l->q_norm.data() : nullptr, (int)l->q_norm.size(),
                               l->has_k_norm ? l->k_norm.data() : nullptr, (int)l->k_norm.size(), l->qk_norm_eps,
                               kInitialCapacity);
  if (rc) return rc;
  rc = shainet_attn_set_bias(l->ctx, l->has_bq ? l->b_q.data() : nullptr, (int)l->b_q.size(),
                             l->has_bk ? l->b_k.data() : nullptr, (int)l->b_k.size(),
                             l->has_bv ? l->b_v.data() : nullptr, (int)l->b_v.size());
  if (!rc) rc = shainet_kv_cache_create(&l->cache, l->ctx, 1, kInitialCapacity);
  if (rc) {
    drop_context(l);
    return rc;
  }
  l->params_dirty = false;
  if (l->shared_error) shainet_attn_adopt_error_word(l->ctx, l->shared_error);
  l->proj.error = shainet_attn_error_word(l->ctx);
  return SHAINET_HIP_OK;
}

void set_vec(std::vector<float> &v, bool &has, const float *src, int n) {
  has = src != nullptr;
  v.assign(src ? src : nullptr, src ? src + (n > 0 ? n : 0) : nullptr);
}

// attention_cached_cpu (llama_block.cr:246-299) with x and out on the device,
// asynchronous on the layer's stream.  pre: an RMSNorm to apply to x on its way
// into the projections; residual: rows to add to the result of the output
// projection (both are what LlamaBlock#forward_cached does around attention).
//
// no_cache: attention_full_cpu (209-243) instead: the same arithmetic from
// position 0 over the rows of this call alone; they go through a scratch cache
// that is empty again afterwards, and the block's own cache is not touched.
struct AheadRows {  // the transposed gate | up weights ([2 n, k]) the block's next product but one will read
  const float *wt;
  int k, n;
};
int attn_forward_device(shainet_llama_attn *l, const float *x, int T, float *out, const Fused &pre = Fused(),
                        const float *residual = nullptr, bool no_cache = false, const AheadRows *ahead = nullptr) {
  if (!l->w_qkv) return fail(SHAINET_HIP_ERR_ARGUMENT, "weights not set");
  int rc = ensure_context(l);
  if (rc) return rc;
  shainet_kv_cache *cache = l->cache;
  if (no_cache) {
    if (!l->scratch_cache && (rc = shainet_kv_cache_create(&l->scratch_cache, l->ctx, 1, T > kInitialCapacity ? T : kInitialCapacity)))
      return rc;
    cache = l->scratch_cache;
    if ((rc = shainet_kv_cache_clear(cache, -1))) return rc;
  }
  const int total_len = (no_cache ? 0 : l->cache_len) + T;
  const int cap = shainet_kv_cache_capacity(cache);
  if (total_len > cap) {  // ensure_gpu_cache! (llama_block.cr:497-520): grow by doubling, contents stay on the device
    rc = shainet_kv_cache_reserve(cache, total_len > 2 * cap ? total_len : 2 * cap);
    if (rc) return rc;
  }
  const int wide = l->q_dim + 2 * l->kv_dim;
  if (!l->qkv.reserve((size_t)T * wide) || !l->attn.reserve((size_t)T * l->q_dim))
    return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
  hipStream_t stream = (hipStream_t)shainet_attn_stream(l->ctx);
  // q_full, k_new, v_new (llama_block.cr:253-255) as the three column blocks of one product
  const int hd = l->head_dim;
  static const bool fuse_off = getenv("SHAINET_HIP_NO_FUSED_PREP") != nullptr;
  if (!fuse_off && T <= 16 && (wide & 3) == 0 && hd >= 2 && hd <= 128 && (hd & (hd - 1)) == 0) {
    // few rows: bias, QK-norm, RoPE and the cache append (256-286, 332-344) happen where the
    // product's head rows are summed up; the attention kernel follows directly
    GemvPrep where;
    if ((rc = shainet_attn_begin_prepared(l->ctx, cache, T, &where))) return rc;
    Fused qkv = pre;
    qkv.epilogue = kGemvQkvPrep;
    qkv.prep = &where;
    if (gemvt_takes(T, l->d_model, wide, qkv.epilogue, qkv.norm, &where)) {
      // the copy carries the weights of the norm this product follows (a layer used with another
      // norm, or with none, gets its copy made again)
      const float *gamma = qkv.norm ? qkv.gamma : nullptr;
      if (gamma != l->w_qkv_t_gamma) l->w_qkv_t_stale = true;
      qkv.w_t = transposed_twin(&l->w_qkv_t, &l->w_qkv_t_stale, l->w_qkv, l->d_model, wide, stream, gamma);
      l->w_qkv_t_gamma = qkv.w_t ? gamma : nullptr;
      qkv.w_t_has_gamma = qkv.w_t && gamma;
    }
    if ((rc = l->proj.project(x, l->d_model, l->w_qkv, nullptr, T, l->d_model, wide, stream, qkv))) return rc;
    // One row: the attention launch leaves the memory system idle while it waits on its chain of
    // dependent loads, and takes along workgroups that read the first rows of the gate | up
    // weights into the L2s (8 MB: 1134 -> 1120 us per token of the 1B shape; 17 MB and more
    // slow the attention's own chain down by more than the product gains)
    static const int ahead_wgs = getenv("SHAINET_HIP_READ_AHEAD_WGS") ? atoi(getenv("SHAINET_HIP_READ_AHEAD_WGS")) : 128;
    if (ahead && ahead->wt && ahead_wgs > 0 && T == 1) shainet_attn_read_ahead(l->ctx, ahead->wt, ahead->k, ahead->n, ahead_wgs);
    rc = shainet_attn_finish_prepared(l->ctx, cache, T, l->attn.p);  // 287-296
  } else {
    if ((rc = l->proj.project(x, l->d_model, l->w_qkv, l->qkv.p, T, l->d_model, wide, stream, pre))) return rc;
    rc = shainet_attn_forward_strided(l->ctx, cache, nullptr, &T, 1, l->qkv.p, l->qkv.p + l->q_dim,
                                      l->qkv.p + l->q_dim + l->kv_dim, wide, wide, wide, l->attn.p,
                                      SHAINET_HIP_MEM_DEVICE);  // 256-296
  }
  if (rc) return rc;
  if (no_cache) {
    if ((rc = shainet_kv_cache_clear(cache, -1))) return rc;
  } else {
    l->cache_len = total_len;
  }
  Fused post;
  if (residual) {
    post.epilogue = kGemvResidual;
    post.res = residual;
  }
  if (gemvt_takes(T, l->q_dim, l->d_model, post.epilogue, false)) post.w_t = transposed_twin(&l->w_o_t, &l->w_o_t_stale, l->w_o, l->q_dim, l->d_model, stream);
  return l->proj.project(l->attn.p, l->q_dim, l->w_o, out, T, l->q_dim, l->d_model, stream, post);  // 298
}

}  // namespace

extern "C" {

int shainet_llama_attn_create(shainet_llama_attn **out, int d_model, int num_heads, int num_kv_heads, int head_dim,
                              double eps, double rope_theta) {
  if (!out) return fail(SHAINET_HIP_ERR_ARGUMENT, "out is null");
  *out = nullptr;
  // llama_block.cr:80-89
  if (!(num_kv_heads > 0 && num_heads > 0 && num_heads % num_kv_heads == 0))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "num_heads must be divisible by num_kv_heads");
  if (head_dim < 0) return fail(SHAINET_HIP_ERR_ARGUMENT, "head_dim must be positive");
  if (head_dim == 0) {
    if (d_model <= 0 || d_model % num_heads != 0)
      return fail(SHAINET_HIP_ERR_ARGUMENT, "d_model must be divisible by num_heads");
    head_dim = d_model / num_heads;
  }
  shainet_llama_attn *l = new (std::nothrow) shainet_llama_attn();
  if (!l) return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  l->d_model = d_model;
  l->num_heads = num_heads;
  l->num_kv_heads = num_kv_heads;
  l->head_dim = head_dim;
  l->q_dim = num_heads * head_dim;
  l->kv_dim = num_kv_heads * head_dim;
  l->qk_norm_eps = eps;
  l->rope_theta = rope_theta;
  *out = l;
  return SHAINET_HIP_OK;
}

int shainet_llama_attn_destroy(shainet_llama_attn *l) {
  if (!l) return SHAINET_HIP_OK;
  drop_context(l);
  l->proj.release();
  for (float *p : {l->w_qkv, l->w_o, l->w_o_t, l->w_qkv_t})
    if (p) (void)hipFree(p);
  for (DevF *b : {&l->x, &l->qkv, &l->attn, &l->out}) b->release();
  l->x_pin.release();
  l->out_pin.release();
  delete l;
  return SHAINET_HIP_OK;
}

int shainet_llama_attn_set_rope(shainet_llama_attn *l, double rope_theta, const float *rope_freqs) {
  if (!l) return fail(SHAINET_HIP_ERR_ARGUMENT, "layer is null");
  l->rope_theta = rope_theta;
  set_vec(l->rope_freqs, l->has_rope_freqs, rope_freqs, l->head_dim / 2);
  l->params_dirty = true;
  return SHAINET_HIP_OK;
}

int shainet_llama_attn_set_qk_norm(shainet_llama_attn *l, const float *q_norm, int q_len, const float *k_norm,
                                   int k_len) {
  if (!l) return fail(SHAINET_HIP_ERR_ARGUMENT, "layer is null");
  set_vec(l->q_norm, l->has_q_norm, q_norm, q_len);
  set_vec(l->k_norm, l->has_k_norm, k_norm, k_len);
  l->params_dirty = true;
  return SHAINET_HIP_OK;
}

int shainet_llama_attn_set_bias(shainet_llama_attn *l, const float *b_q, int q_len, const float *b_k, int k_len,
                                const float *b_v, int v_len) {
  if (!l) return fail(SHAINET_HIP_ERR_ARGUMENT, "layer is null");
  set_vec(l->b_q, l->has_bq, b_q, q_len);
  set_vec(l->b_k, l->has_bk, b_k, k_len);
  set_vec(l->b_v, l->has_bv, b_v, v_len);
  l->params_dirty = true;
  return SHAINET_HIP_OK;
}

int shainet_llama_attn_set_weights(shainet_llama_attn *l, const float *w_q, const float *w_k, const float *w_v,
                                   const float *w_o) {
  if (!l || !w_q || !w_k || !w_v || !w_o) return fail(SHAINET_HIP_ERR_ARGUMENT, "null argument");
  if (!shainet_hip_available()) return fail(SHAINET_HIP_ERR_RUNTIME, "no gfx950 device available");
  const float *mats[3] = {w_q, w_k, w_v};
  const int widths[3] = {l->q_dim, l->kv_dim, l->kv_dim};
  int rc = upload_side_by_side(&l->w_qkv, mats, widths, 3, l->d_model);
  if (!rc) rc = upload_floats(&l->w_o, w_o, (size_t)l->q_dim * l->d_model);
  l->w_o_t_stale = l->w_qkv_t_stale = true;
  return rc;
}

int shainet_llama_attn_clear_cache(shainet_llama_attn *l) {
  if (!l) return fail(SHAINET_HIP_ERR_ARGUMENT, "layer is null");
  l->cache_len = 0;
  return l->cache ? shainet_kv_cache_clear(l->cache, -1) : SHAINET_HIP_OK;
}

int shainet_llama_attn_cache_len(const shainet_llama_attn *l) { return l ? l->cache_len : -1; }

static int attn_forward_host(shainet_llama_attn *l, const float *x, int new_tokens, float *out, bool no_cache);

int shainet_llama_attn_forward_cached(shainet_llama_attn *l, const float *x, int new_tokens, float *out) {
  return attn_forward_host(l, x, new_tokens, out, false);
}

int shainet_llama_attn_forward_full(shainet_llama_attn *l, const float *x, int seq_len, float *out) {
  return attn_forward_host(l, x, seq_len, out, true);
}

static int attn_forward_host(shainet_llama_attn *l, const float *x, int new_tokens, float *out, bool no_cache) {
  if (!l || !x || !out || new_tokens < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "invalid arguments");
  if (!l->w_qkv) return fail(SHAINET_HIP_ERR_ARGUMENT, "weights not set");
  int rc = ensure_context(l);  // raises what add_bias! / apply_head_rmsnorm! raise (llama_block.cr:587, 618)
  if (rc) return rc;
  const size_t xd = (size_t)new_tokens * l->d_model;
  if (!l->x.reserve(xd) || !l->out.reserve(xd) || !l->x_pin.reserve(xd) || !l->out_pin.reserve(xd))
    return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
  hipStream_t stream = (hipStream_t)shainet_attn_stream(l->ctx);
  memcpy(l->x_pin.p, x, xd * sizeof(float));  // the last call's copies are done: every host-pointer call ends with a wait
  if (hipMemcpyAsync(l->x.p, l->x_pin.p, xd * sizeof(float), hipMemcpyHostToDevice, stream) != hipSuccess)
    return fail(SHAINET_HIP_ERR_RUNTIME, "hipMemcpyAsync(x) failed");
  if ((rc = attn_forward_device(l, l->x.p, new_tokens, l->out.p, Fused(), nullptr, no_cache))) {
    (void)hipStreamSynchronize(stream);  // the copy out of the pinned staging buffer may still run
    return rc;
  }
  if (hipMemcpyAsync(l->out_pin.p, l->out.p, xd * sizeof(float), hipMemcpyDeviceToHost, stream) != hipSuccess ||
      hipStreamSynchronize(stream) != hipSuccess)
    return fail(SHAINET_HIP_ERR_RUNTIME, "copying the result back failed");
  memcpy(out, l->out_pin.p, xd * sizeof(float));
  return check_error_word(shainet_attn_error_word(l->ctx));
}

}  // extern "C"

// ---------------------------------------------------------------------------
// The whole block: LlamaBlock#forward_cached (llama_block.cr:189-196) with a dense
// SwiGLU feed-forward (swiglu_ff.cr:76-91).

// What blocks that use the same weights share.
struct BlockWeights {
  NormWeights norm1, norm2;
  float *gate_up = nullptr, *down = nullptr;        // device [d_model, 2*ff] (gate | up) and [ff, d_model]
  float *gate_up_t = nullptr, *down_t = nullptr;    // the same transposed ([2*ff, d_model], [d_model, ff]), like w_o_t
  bool gate_up_t_stale = true, down_t_stale = true;
  // wrapped blocks: norms behind the sublayers [d_model], convolutions in front of them [taps, d_model], and a
  // feed-forward of another kind (null: none)
  float *post1 = nullptr, *post2 = nullptr, *conv1 = nullptr, *conv2 = nullptr;
  int taps = 0;
  std::unique_ptr<FeedForward> ff;
  ~BlockWeights() {
    for (float *p : {norm1.gamma, norm1.beta, norm2.gamma, norm2.beta, gate_up, down, gate_up_t, down_t, post1, post2, conv1, conv2})
      if (p) (void)hipFree(p);
  }
};

// The latent-attention mixer behind the interface all mixers share.
struct LatentMixer : Mixer {
  LatentAttn *l;
  explicit LatentMixer(LatentAttn *l) : l(l) {}
  ~LatentMixer() override { latent_attn_destroy(l); }
  hipStream_t stream() override { return (hipStream_t)shainet_attn_stream(latent_attn_context(l)); }
  int set_stream(hipStream_t s) override { return shainet_attn_set_stream(latent_attn_context(l), (void *)s); }
  int *error_word() override { return shainet_attn_error_word(latent_attn_context(l)); }
  void share_error_word(int *word) override { latent_attn_share_error_word(l, word); }
  Projector &projector() override { return latent_attn_projector(l); }
  int forward(const float *x, int T, float *out, const Fused &pre, const float *residual, bool no_cache) override {
    return latent_attn_forward(l, x, T, out, pre, residual, no_cache);
  }
  int reserve(int positions) override { return latent_attn_reserve(l, positions); }
  int clear() override { return shainet_kv_cache_clear(cache(), -1); }
  int len() override { return shainet_kv_cache_len(cache(), 0); }
  int truncate(int len) override { return shainet_kv_cache_truncate(cache(), 0, len); }
  shainet_kv_cache *cache() override { return latent_attn_cache(l); }
  LatentAttn *latent() override { return l; }
};

// What a convolution over time in front of a sublayer keeps of its sequence: the sublayer's last taps - 1
// inputs, in two buffers that take turns.
struct ConvState {
  float *rows[2] = {nullptr, nullptr}, *saved = nullptr;
  int cur = 0;
  int allocate(size_t n) {
    const WantedBuffer wants[] = {{&rows[0], n}, {&rows[1], n}, {&saved, n}};
    return allocate_buffers(wants, 3);
  }
  ~ConvState() {
    for (float *p : {rows[0], rows[1], saved})
      if (p) (void)hipFree(p);
  }
};

struct shainet_llama_block {
  shainet_llama_attn *attn = nullptr;  // the mixer: one of the two
  std::unique_ptr<Mixer> mixer;
  bool wrapped = false;  // norms behind the sublayers (and convolutions in front)
  ConvState conv[2];
  int pos = 0, saved_pos = -1;  // wrapped: positions so far, and where the state was saved last
  DevF joined, y, factors;      // wrapped: the residual with the block before joined in; a sublayer's result; scratch
  int d_model = 0, ff_hidden = 0;                   // ff_hidden 0: no feed-forward
  double eps = 1e-6;                                // RMSNorm eps of @norm1 / @norm2 (llama_block.cr:93-94)
  std::shared_ptr<BlockWeights> w = std::make_shared<BlockWeights>();
  DevF x, h, hidden, out;
  PinnedF x_pin, out_pin;  // host-pointer calls stage their rows here
};

namespace {

// the stream the block's work runs on, once its mixer is ready
int block_stream(shainet_llama_block *b, hipStream_t *stream) {
  if (b->mixer) {
    *stream = b->mixer->stream();
    return SHAINET_HIP_OK;
  }
  const int rc = ensure_context(b->attn);
  if (!rc) *stream = (hipStream_t)shainet_attn_stream(b->attn->ctx);
  return rc;
}
int *block_error_word(shainet_llama_block *b) { return b->mixer ? b->mixer->error_word() : shainet_attn_error_word(b->attn->ctx); }

int grouped_only(const shainet_llama_block *b, const char *what) {
  if (b->mixer) return fail(SHAINET_HIP_ERR_ARGUMENT, std::string(what) + ": this block's mixer is not the grouped-query attention of a LLaMA block");
  return SHAINET_HIP_OK;
}

}  // namespace

namespace {

// One residual_kernels.hpp launch: (with y) the result y of a sublayer joins x; (with pre) what the next sublayer
// reads, from conv's state if there is a convolution.
int join(shainet_llama_block *b, const float *x, const float *y, const float *post, float *x_out, const float *pre,
         const float *conv_w, ConvState *conv, float *h, int T, bool no_cache, hipStream_t stream) {
  ResidualArgs a = {};
  a.x = x;
  a.y = y;
  a.post = post;
  a.x_out = x_out;
  a.pre = pre;
  a.h = h;
  a.T = T;
  a.d = b->d_model;
  a.eps = (float)b->eps;
  if (conv_w) {
    a.conv = conv_w;
    a.taps = b->w->taps;
    a.factors = b->factors.p;
    if (a.taps > 1 && !no_cache) {
      a.hist_in = b->pos ? conv->rows[conv->cur] : nullptr;  // (nothing lies before a sequence's first row)
      a.hist_out = conv->rows[conv->cur ^ 1];
      conv->cur ^= 1;
    }
  }
  const hipError_t e = launch_residual(a, stream);
  return e == hipSuccess ? SHAINET_HIP_OK : fail(SHAINET_HIP_ERR_RUNTIME, std::string("residual launch: ") + hipGetErrorString(e));
}

// x <- x + norm1b(mixer(conv1(norm1(x)))), then x <- x + norm2b(ff(conv2(norm2(x)))), where conv(h) = h + the
// convolution.  Each arrow and what the next sublayer reads are one launch; carry takes the last one over
// to the next block (BlockCarry).
int wrapped_forward_device(shainet_llama_block *b, const float *x, int T, float *out, bool no_cache, BlockCarry *carry) {
  BlockWeights &w = *b->w;
  const size_t n = (size_t)T * b->d_model;
  hipStream_t stream = b->mixer->stream();
  if (!w.norm1.gamma || !w.post1) return fail(SHAINET_HIP_ERR_ARGUMENT, "weights not set");
  if (!b->h.reserve(n) || !b->y.reserve(n) || !b->joined.reserve(n) || !b->factors.reserve((size_t)T)) return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
  const bool carried = carry && carry->y;
  int rc = join(b, x, carried ? carry->y : nullptr, carried ? carry->post : nullptr, b->joined.p, w.norm1.gamma, w.conv1, &b->conv[0],
                b->h.p, T, no_cache, stream);
  if (carry) carry->y = nullptr;
  const float *res = carried ? b->joined.p : x;
  if (!rc) rc = b->mixer->forward(b->h.p, T, b->y.p, Fused(), nullptr, no_cache);
  if (!rc && !w.ff) rc = join(b, res, b->y.p, w.post1, out, nullptr, nullptr, nullptr, nullptr, T, no_cache, stream);
  if (!rc && w.ff) {
    rc = join(b, res, b->y.p, w.post1, out, w.norm2.gamma, w.conv2, &b->conv[1], b->h.p, T, no_cache, stream);
    if (!rc) rc = w.ff->forward(b->mixer->projector(), b->h.p, T, b->y.p, stream);
    if (!rc && carry) {
      carry->y = b->y.p;
      carry->post = w.post2;
    } else if (!rc) {
      rc = join(b, out, b->y.p, w.post2, out, nullptr, nullptr, nullptr, nullptr, T, no_cache, stream);
    }
  }
  if (!rc && !no_cache) b->pos += T;
  return rc;
}

// x and out on the device; asynchronous on the block's stream.
int block_forward_device(shainet_llama_block *b, const float *x, int T, float *out, bool no_cache = false, BlockCarry *carry = nullptr) {
  if (b->wrapped) return wrapped_forward_device(b, x, T, out, no_cache, carry);
  if (carry && carry->y) return fail(SHAINET_HIP_ERR_ARGUMENT, "a block without norms behind its sublayers takes no carried result");
  BlockWeights &w = *b->w;
  const int d = b->d_model, ff = b->ff_hidden;
  if (ff && (!w.gate_up || !w.down)) return fail(SHAINET_HIP_ERR_ARGUMENT, "feed-forward weights not set");
  hipStream_t stream = nullptr;
  int rc = block_stream(b, &stream);
  if (rc) return rc;
  Projector &proj = b->mixer ? b->mixer->projector() : b->attn->proj;
  if (ff && (!b->h.reserve((size_t)T * d) || !b->hidden.reserve((size_t)T * ff)))
    return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
  float *h = ff ? b->h.p : out;  // without a feed-forward the mixer's sum is the block's result
  // h = x + attention_cached_cpu(@norm1.forward(x))
  Fused n1;
  w.norm1.apply(n1, b->eps);
  Fused gate;
  w.norm2.apply(gate, b->eps);
  gate.epilogue = kGemvSwiglu;
  if (ff && gemvt_takes(T, d, ff, gate.epilogue, gate.norm)) {
    // (the RMSNorm weights ride in the copy; Dynamic Tanh adds beta behind its own, so they stay outside)
    const float *ride = gate.norm == kNormRms ? gate.gamma : nullptr;
    gate.w_t = transposed_twin(&w.gate_up_t, &w.gate_up_t_stale, w.gate_up, d, 2 * ff, stream, ride);
    gate.w_t_has_gamma = gate.w_t && ride;
  }
  if (b->mixer) {
    rc = b->mixer->forward(x, T, h, n1, x, no_cache);
  } else {
    const AheadRows ahead = {gate.w_t, d, ff};
    rc = attn_forward_device(b->attn, x, T, h, n1, x, no_cache, &ahead);
  }
  if (rc || !ff) return rc;
  // hidden = silu(normed2 * gate_proj) * (normed2 * up_proj), normed2 = @norm2.forward(h)
  if ((rc = proj.project(h, d, w.gate_up, b->hidden.p, T, d, ff, stream, gate))) return rc;
  // out = h + hidden * down_proj
  Fused down;
  down.epilogue = kGemvResidual;
  down.res = h;
  if (gemvt_takes(T, ff, d, down.epilogue, down.norm)) down.w_t = transposed_twin(&w.down_t, &w.down_t_stale, w.down, ff, d, stream);
  return proj.project(b->hidden.p, ff, w.down, out, T, ff, d, stream, down);
}

}  // namespace

// used by the model (llama_model.hip)
int shainet_llama_block_forward_device(shainet_llama_block *b, const float *x, int T, float *out, bool no_cache, BlockCarry *carry) {
  return block_forward_device(b, x, T, out, no_cache, b->wrapped ? carry : nullptr);
}
int shainet_llama_block_join_carry(shainet_llama_block *b, const BlockCarry &carry, float *x, int T) {
  return join(b, x, carry.y, carry.post, x, nullptr, nullptr, nullptr, nullptr, T, true, b->mixer->stream());
}
bool shainet_llama_block_keeps_state(const shainet_llama_block *b) { return b->wrapped; }
int shainet_llama_block_save_state(shainet_llama_block *b) {
  if (!b->wrapped) return SHAINET_HIP_OK;
  b->saved_pos = -1;
  if (int rc = b->mixer->save()) return rc;
  const size_t bytes = (size_t)(b->w->taps > 1 ? b->w->taps - 1 : 0) * b->d_model * sizeof(float);
  for (ConvState &c : b->conv)
    if (b->pos && bytes && c.saved && hipMemcpyAsync(c.saved, c.rows[c.cur], bytes, hipMemcpyDeviceToDevice, b->mixer->stream()) != hipSuccess)
      return fail(SHAINET_HIP_ERR_RUNTIME, "hipMemcpyAsync(state) failed");
  b->saved_pos = b->pos;
  return SHAINET_HIP_OK;
}
int shainet_llama_block_buffers(shainet_llama_block *b, LlamaBlockBuffers *out) {
  shainet_llama_attn *l = b->attn;
  BlockWeights &bw = *b->w;
  const size_t d = (size_t)b->d_model, ff = (size_t)b->ff_hidden;
  const bool tanh_norm = bw.norm1.kind == kNormDynTanh;
  struct Want {
    float **p;
    size_t n;  // 0: this block has no such buffer
  } wants[] = {{l ? &l->w_qkv : nullptr, l ? d * (size_t)(l->q_dim + 2 * l->kv_dim) : 0},
               {l ? &l->w_o : nullptr, l ? (size_t)l->q_dim * d : 0},
               {&bw.gate_up, d * 2 * ff},
               {&bw.down, ff * d},
               {&bw.norm1.gamma, d},
               {&bw.norm2.gamma, ff ? d : 0},
               {&bw.norm1.beta, tanh_norm ? d : 0},
               {&bw.norm2.beta, tanh_norm && ff ? d : 0}};
  for (const Want &w : wants)
    if (w.n && !*w.p && hipMalloc((void **)w.p, w.n * sizeof(float)) != hipSuccess) {
      *w.p = nullptr;
      return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    }
  // (whoever asks for the buffers is about to write the weights: the transposed copies are made again)
  bw.gate_up_t_stale = bw.down_t_stale = true;
  if (l) l->w_o_t_stale = l->w_qkv_t_stale = true;
  *out = LlamaBlockBuffers{l ? l->w_qkv : nullptr, l ? l->w_o : nullptr, bw.gate_up, bw.down,
                           &bw.norm1,  &bw.norm2,  b->d_model,  l ? l->q_dim : 0, l ? l->kv_dim : 0, b->ff_hidden};
  return SHAINET_HIP_OK;
}

int shainet_llama_block_create_latent(shainet_llama_block **out, int d_model, const shainet_latent_config &cfg,
                                      int ff_hidden, int norm_kind, double eps, const shainet_llama_block *weights_of) {
  *out = nullptr;
  if (ff_hidden < 0) return fail(SHAINET_HIP_ERR_ARGUMENT, "ff_hidden must not be negative");
  if (weights_of && (!weights_of->mixer || !weights_of->mixer->latent() || weights_of->d_model != d_model || weights_of->ff_hidden != ff_hidden ||
                     weights_of->w->norm1.kind != norm_kind))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "layers that share weights must have the same mixer, feed-forward and norms");
  LatentAttn *l = nullptr;
  if (int rc = latent_attn_create(&l, d_model, cfg, eps, weights_of ? weights_of->mixer->latent() : nullptr)) return rc;
  shainet_llama_block *b = new (std::nothrow) shainet_llama_block();
  if (!b) {
    latent_attn_destroy(l);
    return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  }
  b->mixer.reset(new LatentMixer(l));
  b->d_model = d_model;
  b->ff_hidden = ff_hidden;
  b->eps = eps;
  if (weights_of)
    b->w = weights_of->w;
  else
    b->w->norm1.kind = b->w->norm2.kind = norm_kind;
  *out = b;
  return SHAINET_HIP_OK;
}
LatentAttn *shainet_llama_block_latent_mixer(shainet_llama_block *b) { return b->mixer ? b->mixer->latent() : nullptr; }

int shainet_llama_block_create_wrapped(shainet_llama_block **out, int d_model, Mixer *mixer, FeedForward *ff, int taps, double eps) {
  *out = nullptr;
  std::unique_ptr<Mixer> owned(mixer);
  std::unique_ptr<FeedForward> owned_ff(ff);
  if (taps < 1 || taps > kMaxConvTaps)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "convolution taps must be in [1, " + std::to_string(kMaxConvTaps) + "]");
  std::unique_ptr<shainet_llama_block> b(new (std::nothrow) shainet_llama_block());
  if (!b) return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  b->mixer = std::move(owned);
  b->wrapped = true;
  b->d_model = d_model;
  b->eps = eps;
  BlockWeights &w = *b->w;
  w.taps = taps;
  w.ff = std::move(owned_ff);
  const size_t d = (size_t)d_model, conv = (size_t)taps * d;
  const WantedBuffer wants[] = {{&w.norm1.gamma, d}, {&w.post1, d}, {&w.conv1, conv}, {&w.norm2.gamma, ff ? d : 0},
                                {&w.post2, ff ? d : 0}, {&w.conv2, ff ? conv : 0}};
  int rc = allocate_buffers(wants, 6);
  if (!rc && taps > 1) rc = b->conv[0].allocate(conv - d);
  if (!rc && taps > 1 && ff) rc = b->conv[1].allocate(conv - d);
  if (rc) return rc;
  *out = b.release();
  return SHAINET_HIP_OK;
}
WrappedBlockBuffers shainet_llama_block_wrapped_buffers(shainet_llama_block *b) {
  BlockWeights &w = *b->w;
  return WrappedBlockBuffers{w.norm1.gamma, w.post1, w.conv1, w.norm2.gamma, w.post2, w.conv2};
}
Mixer *shainet_llama_block_mixer_of(shainet_llama_block *b) { return b->mixer.get(); }

// One decode step of the whole stack in one launch (step_kernel.hip): where this block's weights,
// parameters and cache are, with room for one more row made first (ensure_gpu_cache!,
// llama_block.cr:497-520); *pos = rows cached so far.  The step's kernel appends the row;
// shainet_llama_block_step_commit counts it afterwards.
int shainet_llama_block_step_begin(shainet_llama_block *b, StepLayer *out, int *pos) {
  if (int bad = grouped_only(b, "one-launch decode step")) return bad;
  shainet_llama_attn *l = b->attn;
  const BlockWeights &w = *b->w;
  if (!l->w_qkv || !l->w_o || !w.gate_up || !w.down) return fail(SHAINET_HIP_ERR_ARGUMENT, "weights not set");
  int rc = ensure_context(l);
  if (rc) return rc;
  const int cap = shainet_kv_cache_capacity(l->cache);
  if (l->cache_len + 1 > cap && (rc = shainet_kv_cache_reserve(l->cache, 2 * cap))) return rc;
  GemvPrep where;
  if ((rc = shainet_attn_begin_prepared(l->ctx, l->cache, 1, &where))) return rc;
  out->w_qkv = l->w_qkv;
  out->w_o = l->w_o;
  out->w_gu = w.gate_up;
  out->w_down = w.down;
  out->norm1 = w.norm1.gamma;
  out->norm2 = w.norm2.gamma;
  out->b_q = where.b_q;
  out->b_k = where.b_k;
  out->b_v = where.b_v;
  out->q_norm = where.q_norm;
  out->k_norm = where.k_norm;
  out->rope_tab = where.rope_tab;
  out->kc = where.kc;
  out->vc = where.vc;
  out->cap = where.cap;
  out->pad_ = 0;
  *pos = where.start_pos;
  return SHAINET_HIP_OK;
}
void shainet_llama_block_step_commit(shainet_llama_block *b) {
  shainet_llama_attn *l = b->attn;
  shainet_attn_commit_prepared(l->ctx, l->cache, 1);
  l->cache_len += 1;
}
// The block's geometry, for the planner of the step kernel (false: the kernel does not know this mixer).
bool shainet_llama_block_geometry(const shainet_llama_block *b, int *H, int *KV, int *hd, int *ff, double *qk_eps) {
  if (!b->attn) return false;
  *H = b->attn->num_heads;
  *KV = b->attn->num_kv_heads;
  *hd = b->attn->head_dim;
  *ff = b->ff_hidden;
  *qk_eps = b->attn->qk_norm_eps;
  return true;
}

// Forget the cached rows past `len` (generation that ran ahead of a stop token).
int shainet_llama_block_truncate(shainet_llama_block *b, int len) {
  if (b->wrapped) {
    if (len == b->pos) return SHAINET_HIP_OK;
    if (len == 0) return shainet_llama_block_clear_cache(b);
    if (len != b->saved_pos) return fail(SHAINET_HIP_ERR_ARGUMENT, "a block with state can only go back to where it was saved");
    if (int rc = b->mixer->truncate(len)) return rc;
    const size_t bytes = (size_t)(b->w->taps - 1) * b->d_model * sizeof(float);
    for (ConvState &c : b->conv)
      if (bytes && c.saved && hipMemcpyAsync(c.rows[c.cur], c.saved, bytes, hipMemcpyDeviceToDevice, b->mixer->stream()) != hipSuccess)
        return fail(SHAINET_HIP_ERR_RUNTIME, "hipMemcpyAsync(state) failed");
    b->pos = len;
    return SHAINET_HIP_OK;
  }
  if (b->mixer) return b->mixer->truncate(len);
  shainet_llama_attn *l = b->attn;
  if (len < 0 || len > l->cache_len) return fail(SHAINET_HIP_ERR_ARGUMENT, "truncate beyond the cached length");
  if (l->cache) {
    int rc = shainet_kv_cache_truncate(l->cache, 0, len);
    if (rc) return rc;
  }
  l->cache_len = len;
  return SHAINET_HIP_OK;
}
// The model's kernels and its blocks' report a given-up wait into one word, the model's.
void shainet_llama_block_share_error_word(shainet_llama_block *b, int *word) {
  if (b->mixer) {
    b->mixer->share_error_word(word);
    return;
  }
  shainet_llama_attn *l = b->attn;
  l->shared_error = word;
  if (l->ctx) {
    shainet_attn_adopt_error_word(l->ctx, word);
    l->proj.error = shainet_attn_error_word(l->ctx);
  }
}
int shainet_llama_block_set_stream(shainet_llama_block *b, hipStream_t stream) {
  if (b->mixer) return b->mixer->set_stream(stream);
  const int rc = ensure_context(b->attn);
  return rc ? rc : shainet_attn_set_stream(b->attn->ctx, (void *)stream);
}
// Room for `positions` positions in all, made ahead (a windowed mixer keeps what its window needs).
int shainet_llama_block_reserve(shainet_llama_block *b, int positions) {
  if (b->mixer) return b->mixer->reserve(positions);
  const int rc = ensure_context(b->attn);
  return rc ? rc : shainet_kv_cache_reserve(b->attn->cache, positions);
}

extern "C" {

int shainet_llama_block_create(shainet_llama_block **out, int d_model, int num_heads, int ff_hidden, double eps,
                               double rope_theta, int num_kv_heads, int head_dim) {
  if (!out) return fail(SHAINET_HIP_ERR_ARGUMENT, "out is null");
  *out = nullptr;
  if (ff_hidden < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "ff_hidden must be positive");
  if (num_kv_heads == 0) num_kv_heads = num_heads;  // @num_kv_heads = @num_heads (llama_block.cr:73)
  shainet_llama_attn *a = nullptr;
  int rc = shainet_llama_attn_create(&a, d_model, num_heads, num_kv_heads, head_dim, eps, rope_theta);
  if (rc) return rc;
  shainet_llama_block *b = new (std::nothrow) shainet_llama_block();
  if (!b) {
    shainet_llama_attn_destroy(a);
    return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  }
  b->attn = a;
  b->d_model = d_model;
  b->ff_hidden = ff_hidden;
  b->eps = eps;
  *out = b;
  return SHAINET_HIP_OK;
}

int shainet_llama_block_destroy(shainet_llama_block *b) {
  if (!b) return SHAINET_HIP_OK;
  shainet_llama_attn_destroy(b->attn);
  for (DevF *f : {&b->x, &b->h, &b->hidden, &b->out, &b->joined, &b->y, &b->factors}) f->release();
  b->x_pin.release();
  b->out_pin.release();
  delete b;
  return SHAINET_HIP_OK;
}

shainet_llama_attn *shainet_llama_block_attn(shainet_llama_block *b) { return b ? b->attn : nullptr; }

int shainet_llama_block_set_norms(shainet_llama_block *b, const float *norm1, const float *norm2) {
  if (!b) return fail(SHAINET_HIP_ERR_ARGUMENT, "block is null");
  if (int bad = grouped_only(b, "shainet_llama_block_set_norms")) return bad;
  if (!shainet_hip_available()) return fail(SHAINET_HIP_ERR_RUNTIME, "no gfx950 device available");
  int rc = SHAINET_HIP_OK;
  float **dst[2] = {&b->w->norm1.gamma, &b->w->norm2.gamma};
  const float *src[2] = {norm1, norm2};
  for (int i = 0; i < 2 && !rc; ++i) {
    if (src[i]) {
      rc = upload_floats(dst[i], src[i], (size_t)b->d_model);
    } else if (*dst[i]) {
      (void)hipFree(*dst[i]);
      *dst[i] = nullptr;
    }
  }
  // (the transposed copies of q | k | v and gate | up carry the norm weights)
  b->attn->w_qkv_t_stale = b->w->gate_up_t_stale = true;
  b->attn->w_qkv_t_gamma = nullptr;
  return rc;
}

int shainet_llama_block_set_ffn(shainet_llama_block *b, const float *gate, const float *up, const float *down) {
  if (!b || !gate || !up || !down) return fail(SHAINET_HIP_ERR_ARGUMENT, "null argument");
  if (int bad = grouped_only(b, "shainet_llama_block_set_ffn")) return bad;
  if (!shainet_hip_available()) return fail(SHAINET_HIP_ERR_RUNTIME, "no gfx950 device available");
  const float *mats[2] = {gate, up};
  const int widths[2] = {b->ff_hidden, b->ff_hidden};
  int rc = upload_side_by_side(&b->w->gate_up, mats, widths, 2, b->d_model);
  if (!rc) rc = upload_floats(&b->w->down, down, (size_t)b->ff_hidden * b->d_model);
  b->w->gate_up_t_stale = b->w->down_t_stale = true;
  return rc;
}

int shainet_llama_block_clear_cache(shainet_llama_block *b) {
  if (!b) return fail(SHAINET_HIP_ERR_ARGUMENT, "block is null");
  b->pos = 0;
  b->saved_pos = -1;
  if (b->mixer) return b->mixer->clear();
  return shainet_llama_attn_clear_cache(b->attn);
}

int shainet_llama_block_cache_len(const shainet_llama_block *b) {
  if (b && b->wrapped) return b->pos;
  if (b && b->mixer) return b->mixer->len();
  return b ? b->attn->cache_len : -1;
}

shainet_kv_cache *shainet_llama_block_cache(shainet_llama_block *b) {
  if (!b) return nullptr;
  return b->mixer ? b->mixer->cache() : b->attn->cache;
}

int shainet_llama_block_latent_config(shainet_llama_block *b, shainet_latent_config *cfg) {
  if (!b || !cfg) return fail(SHAINET_HIP_ERR_ARGUMENT, "null argument");
  if (!b->mixer || !b->mixer->latent()) return fail(SHAINET_HIP_ERR_ARGUMENT, "this block's mixer is not latent attention");
  *cfg = latent_attn_config(b->mixer->latent());
  return SHAINET_HIP_OK;
}

int shainet_llama_block_mixer(shainet_llama_block *b) {
  if (!b) return -1;
  return !b->mixer             ? SHAINET_HIP_MIXER_GROUPED
         : b->mixer->latent()  ? SHAINET_HIP_MIXER_LATENT
         : b->mixer->biased()  ? SHAINET_HIP_MIXER_BIASED
                               : SHAINET_HIP_MIXER_HGRN2;
}

int shainet_llama_block_read_state(shainet_llama_block *b, float *out, long long n) {
  if (!b || !out) return fail(SHAINET_HIP_ERR_ARGUMENT, "null argument");
  Hgrn2 *l = b->mixer ? b->mixer->hgrn2() : nullptr;
  if (!l) return fail(SHAINET_HIP_ERR_ARGUMENT, "this block has no recurrent state");
  const Hgrn2Config &c = hgrn2_config(l);
  if (n != (long long)c.heads * c.dim * c.vdim)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "the state holds " + std::to_string((long long)c.heads * c.dim * c.vdim) + " floats");
  if (b->pos == 0) {
    memset(out, 0, (size_t)n * sizeof(float));
    return SHAINET_HIP_OK;
  }
  if (hipStreamSynchronize(b->mixer->stream()) != hipSuccess ||
      hipMemcpy(out, hgrn2_state(l), (size_t)n * sizeof(float), hipMemcpyDeviceToHost) != hipSuccess)
    return fail(SHAINET_HIP_ERR_RUNTIME, "copying the state back failed");
  return SHAINET_HIP_OK;
}

static int block_forward_any(shainet_llama_block *b, const float *x, int new_tokens, float *out, int mem, bool no_cache);

int shainet_llama_block_forward_cached(shainet_llama_block *b, const float *x, int new_tokens, float *out, int mem) {
  return block_forward_any(b, x, new_tokens, out, mem, false);
}

int shainet_llama_block_forward(shainet_llama_block *b, const float *x, int seq_len, float *out, int mem) {
  return block_forward_any(b, x, seq_len, out, mem, true);
}

static int block_forward_any(shainet_llama_block *b, const float *x, int new_tokens, float *out, int mem, bool no_cache) {
  if (!b || !x || !out || new_tokens < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "invalid arguments");
  if (mem != SHAINET_HIP_MEM_HOST && mem != SHAINET_HIP_MEM_DEVICE)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "mem must be SHAINET_HIP_MEM_HOST or SHAINET_HIP_MEM_DEVICE");
  if (mem == SHAINET_HIP_MEM_DEVICE) return block_forward_device(b, x, new_tokens, out, no_cache);
  hipStream_t stream = nullptr;
  int rc = block_stream(b, &stream);
  if (rc) return rc;
  const size_t xd = (size_t)new_tokens * b->d_model;
  if (!b->x.reserve(xd) || !b->out.reserve(xd) || !b->x_pin.reserve(xd) || !b->out_pin.reserve(xd))
    return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
  memcpy(b->x_pin.p, x, xd * sizeof(float));
  if (hipMemcpyAsync(b->x.p, b->x_pin.p, xd * sizeof(float), hipMemcpyHostToDevice, stream) != hipSuccess)
    return fail(SHAINET_HIP_ERR_RUNTIME, "hipMemcpyAsync(x) failed");
  if ((rc = block_forward_device(b, b->x.p, new_tokens, b->out.p, no_cache))) {
    (void)hipStreamSynchronize(stream);  // the copy out of the pinned staging buffer may still run
    return rc;
  }
  if (hipMemcpyAsync(b->out_pin.p, b->out.p, xd * sizeof(float), hipMemcpyDeviceToHost, stream) != hipSuccess ||
      hipStreamSynchronize(stream) != hipSuccess)
    return fail(SHAINET_HIP_ERR_RUNTIME, "copying the result back failed");
  memcpy(out, b->out_pin.p, xd * sizeof(float));
  return check_error_word(block_error_word(b));
}

}  // extern "C"
