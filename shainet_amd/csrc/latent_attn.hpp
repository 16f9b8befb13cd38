// The latent-attention mixer of a block (latent_attn.hip): weights, cache and forward pass, beside
// the grouped-query one of llama_block.hip.
#pragma once
#include <hip/hip_runtime.h>

#include <memory>

#include "../../include/shainet_hip_attn.h"
#include "llama_internal.hpp"

namespace shainet {

// On the device; shared by the layers that use one layer's weights (each with a cache of its own).
struct LatentWeights {
  // W_dq | W_dkv | W_g side by side, [d_model, n_in], zero columns up to a multiple of 4: what a row of the
  // mixer's input turns into is [c_q | c | key part | gates]
  float *w_in = nullptr, *w_in_t = nullptr;
  float *dq_norm = nullptr, *dkv_norm = nullptr;
  float *w_uq = nullptr, *w_uq_t = nullptr;  // [q_rank, H (dim + rot_dim)]; the transposed copy carries dq_norm
  float *u_kv = nullptr;                     // [H dim + H vdim, kv_rank]: W_uk then W_uv, a row per output
  float *w_ukv = nullptr;                    // the same transposed: [kv_rank, H dim + H vdim]
  float *sink = nullptr;                     // [H]
  float *w_o = nullptr, *w_o_t = nullptr;    // [H vdim, d_model]
  bool w_in_t_stale = true, w_uq_t_stale = true, w_o_t_stale = true;
  int n_in = 0;
  ~LatentWeights();
};

struct LatentAttn;  // the mixer of one layer
// weights_of != null: that mixer's weights (the geometry must be the same); else device buffers are allocated, unset
int latent_attn_create(LatentAttn **out, int d_model, const shainet_latent_config &cfg, double eps,
                       const LatentAttn *weights_of);
void latent_attn_destroy(LatentAttn *l);
LatentWeights &latent_attn_weights(LatentAttn *l);
const shainet_latent_config &latent_attn_config(const LatentAttn *l);
shainet_attn_ctx *latent_attn_context(LatentAttn *l);  // stream, error word
shainet_kv_cache *latent_attn_cache(LatentAttn *l);
Projector &latent_attn_projector(LatentAttn *l);       // for the block's other products
int latent_attn_reserve(LatentAttn *l, int positions);  // rows for that many positions, or what the window needs of them
void latent_attn_share_error_word(LatentAttn *l, int *word);
// out = (residual +) mixer(pre(x)), T rows on the device, appended behind the cached ones; no_cache:
// the rows attend among themselves from position 0 and the cache stays as it is
int latent_attn_forward(LatentAttn *l, const float *x, int T, float *out, const Fused &pre, const float *residual,
                        bool no_cache);

}  // namespace shainet
