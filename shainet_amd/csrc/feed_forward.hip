#include "feed_forward.hpp"

#include <new>
#include <string>

#include "attn_kernels.hpp"
#include "mixer.hpp"

namespace shainet {

namespace {

int fail(int code, const std::string &msg) { return llama_fail(code, msg); }

struct Dense : FeedForward {
  int d = 0, ff = 0;
  DenseWeights w;
  DevF hidden;
  ~Dense() override {
    hidden.release();
    for (float *p : {w.up, w.up_t, w.up_bias, w.down, w.down_t, w.down_bias})
      if (p) (void)hipFree(p);
  }
  int forward(Projector &proj, const float *h, int T, float *y, hipStream_t stream) override {
    if (!hidden.reserve((size_t)T * ff)) return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
    Fused up;
    up.epilogue = kGemvBias;
    up.bias = w.up_bias;
    up.act = w.act;
    if (gemvt_takes(T, d, ff, up.epilogue, up.norm)) up.w_t = transposed_twin(&w.up_t, &w.up_t_stale, w.up, d, ff, stream);
    if (int rc = proj.project(h, d, w.up, hidden.p, T, d, ff, stream, up)) return rc;
    Fused down;
    down.epilogue = kGemvBias;
    down.bias = w.down_bias;
    if (gemvt_takes(T, ff, d, down.epilogue, down.norm)) down.w_t = transposed_twin(&w.down_t, &w.down_t_stale, w.down, ff, d, stream);
    return proj.project(hidden.p, ff, w.down, y, T, ff, d, stream, down);
  }
};

struct Moe : FeedForward {
  MoeShape m = {};
  MoeWeights w;
  DevF scratch, hidden, logits;
  int *counts = nullptr;
  ~Moe() override {
    for (DevF *f : {&scratch, &hidden, &logits}) f->release();
    if (counts) (void)hipFree(counts);
    for (float *p : {w.router, w.router_in, w.correction, w.gate_up, w.down, w.shared_gate_up, w.shared_down, w.shared_gate_up_in,
                     w.shared_down_in})
      if (p) (void)hipFree(p);
  }
  int forward(Projector &proj, const float *h, int T, float *y, hipStream_t stream) override {
    const MoeTensors t = {w.router, w.correction, w.gate_up, w.down, w.shared_gate_up, w.shared_down};
    hipError_t e;
    if (T <= kMoeFewTokens) {
      if (!scratch.reserve(moe_few_floats(m, T))) return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
      e = launch_moe_few(m, t, h, y, T, scratch.p, stream);
      return e == hipSuccess ? SHAINET_HIP_OK : fail(SHAINET_HIP_ERR_RUNTIME, std::string("expert launch: ") + hipGetErrorString(e));
    }
    constexpr int kAtOnce = 8192;  // tokens whose experts' rows are in memory together
    for (int t0 = 0; t0 < T; t0 += kAtOnce) {
      const int n = T - t0 < kAtOnce ? T - t0 : kAtOnce;
      const float *hp = h + (size_t)t0 * m.d;
      float *yp = y + (size_t)t0 * m.d;
      if (m.shared_ff) {
        if (!hidden.reserve((size_t)n * m.shared_ff)) return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
        Fused gate;
        gate.epilogue = kGemvSwiglu;
        if (int rc = proj.project(hp, m.d, w.shared_gate_up_in, hidden.p, n, m.d, m.shared_ff, stream, gate)) return rc;
        if (int rc = proj.project(hidden.p, m.shared_ff, w.shared_down_in, yp, n, m.shared_ff, m.d, stream)) return rc;
      }
      if (!scratch.reserve(moe_many_floats(m, n)) || !logits.reserve((size_t)n * w.n_router))
        return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
      if (int rc = proj.project(hp, m.d, w.router_in, logits.p, n, m.d, w.n_router, stream)) return rc;
      e = launch_moe_many(m, t, hp, logits.p, w.n_router, yp, m.shared_ff > 0, n, scratch.p, counts, stream);
      if (e != hipSuccess) return fail(SHAINET_HIP_ERR_RUNTIME, std::string("expert launch: ") + hipGetErrorString(e));
    }
    return SHAINET_HIP_OK;
  }
};

}  // namespace

int dense_create(FeedForward **out, int d_model, int ff, DenseWeights **weights) {
  *out = nullptr;
  if (d_model < 1 || ff < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "feed-forward: sizes must be positive");
  Dense *f = new (std::nothrow) Dense();
  if (!f) return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  f->d = d_model;
  f->ff = ff;
  const size_t n = (size_t)d_model * ff;
  const WantedBuffer wants[] = {{&f->w.up, n}, {&f->w.up_bias, (size_t)ff}, {&f->w.down, n}, {&f->w.down_bias, (size_t)d_model}};
  if (int rc = allocate_buffers(wants, 4)) {
    delete f;
    return rc;
  }
  *weights = &f->w;
  *out = f;
  return SHAINET_HIP_OK;
}

int moe_create(FeedForward **out, const MoeShape &m, MoeWeights **weights) {
  *out = nullptr;
  if (!moe_shape_ok(m))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "experts: sizes must be positive, at most 1024 router outputs in equal groups, and top at most what the kept groups hold");
  Moe *f = new (std::nothrow) Moe();
  if (!f) return fail(SHAINET_HIP_ERR_ALLOC, "out of host memory");
  f->m = m;
  const size_t d = (size_t)m.d, n = (size_t)m.experts + m.identity, e = (size_t)m.experts * d * m.ff, s = d * m.shared_ff;
  f->w.n_router = (int)((n + 3) / 4 * 4);
  const WantedBuffer wants[] = {{&f->w.router_in, d * f->w.n_router}, {&f->w.router, n * d}, {&f->w.correction, n},  {&f->w.gate_up, 2 * e},
                                {&f->w.down, e},              {&f->w.shared_gate_up, 2 * s}, {&f->w.shared_down, s},
                                {&f->w.shared_gate_up_in, 2 * s}, {&f->w.shared_down_in, s}};
  int rc = allocate_buffers(wants, 9);
  // (the columns past the last output are never filled by a loader)
  if (!rc && hipMemset(f->w.router_in, 0, d * f->w.n_router * sizeof(float)) != hipSuccess) rc = fail(SHAINET_HIP_ERR_RUNTIME, "hipMemset failed");
  if (!rc && hipMalloc((void **)&f->counts, (size_t)m.experts * sizeof(int)) != hipSuccess) {
    f->counts = nullptr;
    rc = fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
  }
  if (!rc && hipMemset(f->counts, 0, (size_t)m.experts * sizeof(int)) != hipSuccess) rc = fail(SHAINET_HIP_ERR_RUNTIME, "hipMemset failed");
  if (rc) {
    delete f;
    return rc;
  }
  *weights = &f->w;
  *out = f;
  return SHAINET_HIP_OK;
}

}  // namespace shainet
