// HGRN2 as a block's mixer (what it computes: hgrn2_kernels.hpp).  One product makes the rows q | f | v, the
// kernels take them through the state, one product takes the heads back to the model's width.
#include "hgrn2.hpp"

#include <new>
#include <string>

#include "attn_kernels.hpp"
#include "hgrn2_kernels.hpp"

namespace shainet {

namespace {
int fail(int code, const std::string &msg) { return llama_fail(code, msg); }
}  // namespace

struct Hgrn2 : Mixer {
  int d_model = 0;
  Hgrn2Config cfg;
  double eps = 1e-6;
  Hgrn2Weights w;
  hipStream_t own_stream = nullptr, cur_stream = nullptr;
  int *own_error = nullptr;
  float *state = nullptr, *saved = nullptr;
  int rows = 0, saved_rows = -1;  // positions so far; where `saved` was taken (-1: nowhere)
  Projector proj;
  DevF raw, heads, scratch, other_state;

  ~Hgrn2() override {
    proj.release();
    for (DevF *f : {&raw, &heads, &scratch, &other_state}) f->release();
    for (float *p : {w.w_in, w.w_in_t, w.f_bias, w.lower, w.norm, w.w_o, w.w_o_t, state, saved})
      if (p) (void)hipFree(p);
    if (own_stream) (void)hipStreamDestroy(own_stream);
    free_error_word(own_error);
  }
  size_t state_floats() const { return (size_t)cfg.heads * cfg.dim * cfg.vdim; }
  hipStream_t stream() override { return cur_stream; }
  int set_stream(hipStream_t s) override {
    if (s != cur_stream && hipStreamSynchronize(cur_stream) != hipSuccess) return fail(SHAINET_HIP_ERR_RUNTIME, "hipStreamSynchronize failed");
    cur_stream = s ? s : own_stream;
    return SHAINET_HIP_OK;
  }
  int *error_word() override { return proj.error; }
  void share_error_word(int *word) override { proj.error = word ? word : own_error; }
  Projector &projector() override { return proj; }
  int reserve(int) override { return SHAINET_HIP_OK; }
  int clear() override {
    rows = 0;
    saved_rows = -1;
    return SHAINET_HIP_OK;
  }
  int len() override { return rows; }
  bool keeps_state() override { return true; }
  int save() override {
    saved_rows = -1;
    if (rows && !saved && hipMalloc((void **)&saved, state_floats() * sizeof(float)) != hipSuccess) {
      saved = nullptr;
      return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    }
    if (rows && hipMemcpyAsync(saved, state, state_floats() * sizeof(float), hipMemcpyDeviceToDevice, cur_stream) != hipSuccess)
      return fail(SHAINET_HIP_ERR_RUNTIME, "hipMemcpyAsync(state) failed");
    saved_rows = rows;
    return SHAINET_HIP_OK;
  }
  int truncate(int len) override {
    if (len == rows) return SHAINET_HIP_OK;
    if (len == 0) return clear();
    if (len != saved_rows) return fail(SHAINET_HIP_ERR_ARGUMENT, "a recurrent state can only go back to where it was saved");
    if (hipMemcpyAsync(state, saved, state_floats() * sizeof(float), hipMemcpyDeviceToDevice, cur_stream) != hipSuccess)
      return fail(SHAINET_HIP_ERR_RUNTIME, "hipMemcpyAsync(state) failed");
    rows = len;
    return SHAINET_HIP_OK;
  }
  Hgrn2 *hgrn2() override { return this; }

  int forward(const float *x, int T, float *out, const Fused &pre, const float *residual, bool no_cache) override {
    const int d = d_model, vw = cfg.heads * cfg.vdim;
    Hgrn2Plan plan;
    if (!plan_hgrn2(T, cfg.heads, cfg.dim, cfg.vdim, plan)) return fail(SHAINET_HIP_ERR_ARGUMENT, "too many rows in one call");
    if (!raw.reserve((size_t)T * w.n_in) || !heads.reserve((size_t)T * vw) || !scratch.reserve(plan.scratch_floats) ||
        (no_cache && !other_state.reserve(state_floats())))
      return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    Fused in = pre;
    if (gemvt_takes(T, d, w.n_in, in.epilogue, in.norm)) in.w_t = transposed_twin(&w.w_in_t, &w.w_in_t_stale, w.w_in, d, w.n_in, cur_stream);
    int rc = proj.project(x, d, w.w_in, raw.p, T, d, w.n_in, cur_stream, in);
    if (rc) return rc;
    Hgrn2Args a = {};
    a.raw = raw.p;
    a.stride = w.n_in;
    a.f_bias = w.f_bias;
    a.lower = w.lower;
    a.norm = w.norm;
    a.state = no_cache ? other_state.p : state;
    a.fresh = no_cache || rows == 0;
    a.out = heads.p;
    a.T = T;
    a.H = cfg.heads;
    a.dim = cfg.dim;
    a.vdim = cfg.vdim;
    a.eps = (float)eps;
    const hipError_t e = launch_hgrn2(a, plan, scratch.p, cur_stream);
    if (e != hipSuccess) return fail(SHAINET_HIP_ERR_RUNTIME, std::string("hgrn2 launch: ") + hipGetErrorString(e));
    if (!no_cache) rows += T;
    Fused post;
    if (residual) {
      post.epilogue = kGemvResidual;
      post.res = residual;
    }
    if (gemvt_takes(T, vw, d, post.epilogue, post.norm)) post.w_t = transposed_twin(&w.w_o_t, &w.w_o_t_stale, w.w_o, vw, d, cur_stream);
    return proj.project(heads.p, vw, w.w_o, out, T, vw, d, cur_stream, post);
  }
};

int hgrn2_create(Mixer **out, int d_model, const Hgrn2Config &c, double eps) {
  *out = nullptr;
  Hgrn2Plan plan;
  if (d_model < 1 || c.heads < 1 || c.dim < 1 || c.vdim < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "hgrn2: sizes must be positive");
  if (!plan_hgrn2(1, c.heads, c.dim, c.vdim, plan)) return fail(SHAINET_HIP_ERR_ARGUMENT, "hgrn2: dim above 4096 or vdim above 1024");
  if (!shainet_hip_available()) return fail(SHAINET_HIP_ERR_RUNTIME, "no gfx950 device available");
  Hgrn2 *l = new (std::nothrow) Hgrn2();
  if (!l) return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  l->d_model = d_model;
  l->cfg = c;
  l->eps = eps;
  const size_t d = (size_t)d_model, hd = (size_t)c.heads * c.dim, vw = (size_t)c.heads * c.vdim;
  l->w.n_in = (int)((2 * hd + vw + 3) / 4 * 4);
  const WantedBuffer wants[] = {{&l->w.w_in, d * l->w.n_in}, {&l->w.f_bias, hd}, {&l->w.lower, hd}, {&l->w.norm, (size_t)c.vdim},
                                {&l->w.w_o, vw * d},         {&l->state, l->state_floats()}};
  int rc = allocate_buffers(wants, 6);
  // (the columns of w_in past the last value are never filled by a loader)
  if (!rc && hipMemset(l->w.w_in, 0, d * l->w.n_in * sizeof(float)) != hipSuccess) rc = fail(SHAINET_HIP_ERR_RUNTIME, "hipMemset failed");
  if (!rc && hipStreamCreateWithFlags(&l->own_stream, hipStreamNonBlocking) != hipSuccess) rc = fail(SHAINET_HIP_ERR_RUNTIME, "hipStreamCreate failed");
  l->cur_stream = l->own_stream;
  l->own_error = l->proj.error = alloc_error_word();
  if (!rc && !l->own_error) rc = fail(SHAINET_HIP_ERR_ALLOC, "hipHostMalloc failed");
  if (rc) {
    delete l;
    return rc;
  }
  *out = l;
  return SHAINET_HIP_OK;
}

Hgrn2Weights &hgrn2_weights(Hgrn2 *l) { return l->w; }
const Hgrn2Config &hgrn2_config(Hgrn2 *l) { return l->cfg; }
const float *hgrn2_state(Hgrn2 *l) { return l->state; }

}  // namespace shainet
