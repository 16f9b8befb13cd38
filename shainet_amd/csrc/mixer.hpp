// What a block asks of its mixer, whatever kind it is.  A mixer owns what its sequence needs of the past:
// rows of a cache, or a state that every token rewrites.
#pragma once
#include <hip/hip_runtime.h>

#include "../../include/shainet_hip_attn.h"
#include "llama_internal.hpp"

namespace shainet {

struct LatentAttn;
struct BiasedAttn;
struct Hgrn2;

struct Mixer {
  virtual ~Mixer() {}
  virtual hipStream_t stream() = 0;
  virtual int set_stream(hipStream_t s) = 0;
  virtual int *error_word() = 0;
  virtual void share_error_word(int *word) = 0;
  virtual Projector &projector() = 0;
  // out = (residual +) mixer(pre(x)), T rows on the device behind the ones before; no_cache: the rows see
  // each other from position 0 and nothing of what is kept changes.  Asynchronous on the stream.
  virtual int forward(const float *x, int T, float *out, const Fused &pre, const float *residual, bool no_cache) = 0;
  virtual int reserve(int positions) = 0;
  virtual int clear() = 0;
  virtual int len() = 0;
  // Back to `len` positions.  A mixer that keeps a state can only go back to where save was called last.
  virtual int truncate(int len) = 0;
  virtual bool keeps_state() { return false; }
  virtual int save() { return SHAINET_HIP_OK; }
  virtual shainet_kv_cache *cache() { return nullptr; }
  virtual LatentAttn *latent() { return nullptr; }
  virtual BiasedAttn *biased() { return nullptr; }
  virtual Hgrn2 *hgrn2() { return nullptr; }
};

// Device buffers that go together: all allocated, or a SHAINET_HIP_ERR_ALLOC.
struct WantedBuffer {
  float **p;
  size_t n;  // floats; 0: none
};
int allocate_buffers(const WantedBuffer *wants, int count);

}  // namespace shainet
