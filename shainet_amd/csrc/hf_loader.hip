// HFLoader.load_llama (src/shainet/hf_loader.cr:184-412) for the device: reads
// config.json, builds the model, and moves every tensor from the memory-mapped
// SafeTensors file to the GPU in its stored type (F32, F16, BF16 or F64); a
// kernel there converts it to fp32 and writes it transposed, [out, in] ->
// [in, out] (hf_loader.cr:326-337), straight into the place the decode kernels
// read: q/k/v side by side in one matrix, gate|up in another.  No fp32 copy of a
// weight matrix is ever made on the host.
#include <hip/hip_runtime.h>
#include <math.h>
#include <string.h>
#include <sys/stat.h>

#include <string>
#include <vector>

#include "../../include/shainet_hip_attn.h"
#include "attn_kernels.hpp"
#include "biased_attn.hpp"
#include "feed_forward.hpp"
#include "hgrn2.hpp"
#include "latent_attn.hpp"
#include "llama_internal.hpp"
#include "mini_json.hpp"
#include "residual_kernels.hpp"
#include "safetensors.hpp"

using namespace shainet;

namespace {

int fail(int code, const std::string &msg) { return llama_fail(code, msg); }

enum { kF32 = 0, kF16 = 1, kBF16 = 2, kF64 = 3 };

__device__ __forceinline__ float load_as_f32(const void *src, long long i, int dtype) {
  switch (dtype) {
    case kF32: return ((const float *)src)[i];
    case kF16: return __uint_as_float(f16_bits_to_f32_bits(((const unsigned short *)src)[i]));
    case kBF16: return __uint_as_float(bf16_bits_to_f32_bits(((const unsigned short *)src)[i]));
    default: return (float)((const double *)src)[i];
  }
}

// dst[i] = src[i], n elements
__global__ __launch_bounds__(256) void convert_kernel(const void *__restrict__ src, float *__restrict__ dst, long long n,
                                                      int dtype) {
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i < n) dst[i] = load_as_f32(src, i, dtype);
}

// src [rows, cols] row-major -> dst[c * ld + r] for every (r, c): the transpose, written into a
// matrix whose rows are ld floats long (dst already points at the first column to fill).
// 32 x 32 tiles through LDS so that both the reads and the writes are coalesced.
__global__ __launch_bounds__(256) void convert_transpose_kernel(const void *__restrict__ src, float *__restrict__ dst,
                                                                int rows, int cols, long long ld, int dtype) {
  __shared__ float tile[32][33];
  const int tx = threadIdx.x & 31, ty = threadIdx.x >> 5;  // 32 x 8
  const int r0 = blockIdx.y * 32, c0 = blockIdx.x * 32;
#pragma unroll
  for (int j = 0; j < 32; j += 8) {
    const int r = r0 + ty + j, c = c0 + tx;
    if (r < rows && c < cols) tile[ty + j][tx] = load_as_f32(src, (long long)r * cols + c, dtype);
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < 32; j += 8) {
    const int c = c0 + ty + j, r = r0 + tx;
    if (r < rows && c < cols) dst[(long long)c * ld + r] = tile[tx][ty + j];
  }
}

// dst[c * ld + r] = src[r * cols + c] for fp32 already on the device (tied lm_head = embedding^T)
int dtype_code(const std::string &d) {
  if (d == "F32") return kF32;
  if (d == "F16") return kF16;
  if (d == "BF16") return kBF16;
  if (d == "F64") return kF64;
  return -1;
}

struct Stager {
  void *dev = nullptr;
  size_t cap = 0;
  ~Stager() {
    if (dev) (void)hipFree(dev);
  }
  int put(const StTensor &t) {
    if ((size_t)t.nbytes > cap) {
      if (dev) (void)hipFree(dev);
      dev = nullptr;
      cap = 0;
      if (hipMalloc(&dev, (size_t)t.nbytes) != hipSuccess) return fail(SHAINET_HIP_ERR_ALLOC, "hipMalloc failed");
      cap = (size_t)t.nbytes;
    }
    // pageable (memory-mapped) source: returns when the bytes have left the mapping
    if (hipMemcpy(dev, t.data, (size_t)t.nbytes, hipMemcpyHostToDevice) != hipSuccess)
      return fail(SHAINET_HIP_ERR_RUNTIME, "hipMemcpy of tensor '" + t.name + "' failed");
    return SHAINET_HIP_OK;
  }
};

const StTensor *need(const shainet_safetensors *st, const std::string &name, int &rc) {
  const StTensor *t = st->find(name);
  if (!t) rc = fail(SHAINET_HIP_ERR_ARGUMENT, "Tensor '" + name + "' not found");
  return t;
}

// A [rows, cols] tensor (1-D: one row), checked against the shape the model expects.
int check_matrix(const StTensor &t, long long rows, long long cols, int &dtype) {
  dtype = dtype_code(t.dtype);
  if (dtype < 0) return fail(SHAINET_HIP_ERR_ARGUMENT, "Unsupported dtype " + t.dtype + " for float conversion");
  if (t.shape.size() > 2)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "Cannot read tensor '" + t.name + "' with " + std::to_string(t.shape.size()) +
                                              "D shape as matrix");
  const long long r = t.shape.size() == 2 ? t.shape[0] : 1, c = t.shape.empty() ? 1 : t.shape.back();
  if (r != rows || c != cols || t.nbytes != rows * cols * dtype_size(t.dtype))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "tensor '" + t.name + "' is [" + std::to_string(r) + ", " + std::to_string(c) +
                                              "], the model needs [" + std::to_string(rows) + ", " +
                                              std::to_string(cols) + "]");
  return SHAINET_HIP_OK;
}

// HF [out, in] tensor -> columns [col0, col0 + out) of the device matrix dst [in, ld]
int load_transposed(const shainet_safetensors *st, Stager &stage, const std::string &name, int out_dim, int in_dim,
                    float *dst, long long ld, long long col0) {
  int rc = SHAINET_HIP_OK, dtype;
  const StTensor *t = need(st, name, rc);
  if (!t) return rc;
  if ((rc = check_matrix(*t, out_dim, in_dim, dtype)) || (rc = stage.put(*t))) return rc;
  dim3 grid((unsigned)((in_dim + 31) / 32), (unsigned)((out_dim + 31) / 32));
  hipLaunchKernelGGL(convert_transpose_kernel, grid, dim3(256), 0, nullptr, stage.dev, dst + col0, out_dim, in_dim, ld,
                     dtype);
  if (hipGetLastError() != hipSuccess || hipDeviceSynchronize() != hipSuccess)  // the staging buffer is reused next
    return fail(SHAINET_HIP_ERR_RUNTIME, "converting tensor '" + name + "' failed");
  return SHAINET_HIP_OK;
}

int load_plain(const shainet_safetensors *st, Stager &stage, const std::string &name, long long rows, long long cols,
               float *dst) {
  int rc = SHAINET_HIP_OK, dtype;
  const StTensor *t = need(st, name, rc);
  if (!t) return rc;
  if ((rc = check_matrix(*t, rows, cols, dtype)) || (rc = stage.put(*t))) return rc;
  const long long n = rows * cols;
  hipLaunchKernelGGL(convert_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, nullptr, stage.dev, dst, n, dtype);
  if (hipGetLastError() != hipSuccess || hipDeviceSynchronize() != hipSuccess)
    return fail(SHAINET_HIP_ERR_RUNTIME, "converting tensor '" + name + "' failed");
  return SHAINET_HIP_OK;
}

int read_host_vector(const shainet_safetensors *st, const std::string &name, std::vector<float> &out) {
  const StTensor *t = st->find(name);
  if (!t) return fail(SHAINET_HIP_ERR_ARGUMENT, "Tensor '" + name + "' not found");
  const int es = dtype_size(t->dtype);
  out.resize(es ? (size_t)(t->nbytes / es) : 0);
  return shainet_safetensors_read_f32(st, name.c_str(), out.data(), (long long)out.size());
}

bool as_int(const Json *j, int &v) {
  if (!j || j->kind != Json::kNumber) return false;
  v = (int)j->inum;
  return true;
}
bool as_double(const Json *j, double &v) {
  if (!j || j->kind != Json::kNumber) return false;
  v = j->num;
  return true;
}

// config.json of a model directory, parsed
int read_text(const std::string &path, std::string &out);
int read_config(const char *model_dir, Json &j) {
  std::string text, err;
  if (int rc = read_text(std::string(model_dir) + "/config.json", text)) return rc;
  if (!JsonParser(text.data(), text.size()).parse(j, err) || j.kind != Json::kObject)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + (err.empty() ? std::string("not a JSON object") : err));
  return SHAINET_HIP_OK;
}

int read_text(const std::string &path, std::string &out) {
  FILE *f = fopen(path.c_str(), "rb");
  if (!f) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json not found in " + path.substr(0, path.rfind('/')));
  char buf[4096];
  size_t n;
  out.clear();
  while ((n = fread(buf, 1, sizeof buf, f)) > 0) out.append(buf, n);
  fclose(f);
  return SHAINET_HIP_OK;
}

}  // namespace

extern "C" {

int shainet_hf_read_llama_config(const char *model_dir, shainet_hf_llama_config *cfg) {
  if (!model_dir || !cfg) return fail(SHAINET_HIP_ERR_ARGUMENT, "null argument");
  memset(cfg, 0, sizeof *cfg);
  Json j;
  if (int rc = read_config(model_dir, j)) return rc;
  const Json *mt = j.get("model_type");
  if (!mt || mt->kind != Json::kString) return fail(SHAINET_HIP_ERR_ARGUMENT, "No model_type in config.json");
  strncpy(cfg->model_type, mt->str.c_str(), sizeof cfg->model_type - 1);
  // load_llama_config (hf_loader.cr:215-233)
  if (!as_int(j.get("vocab_size"), cfg->vocab_size) || !as_int(j.get("hidden_size"), cfg->hidden_size) ||
      !as_int(j.get("num_attention_heads"), cfg->num_attention_heads) ||
      !as_int(j.get("num_hidden_layers"), cfg->num_hidden_layers) ||
      !as_int(j.get("intermediate_size"), cfg->intermediate_size) || !as_double(j.get("rms_norm_eps"), cfg->rms_norm_eps))
    return fail(SHAINET_HIP_ERR_ARGUMENT,
                "config.json lacks one of vocab_size, hidden_size, num_attention_heads, num_hidden_layers, "
                "intermediate_size, rms_norm_eps");
  cfg->rope_theta = 10000.0;
  if (!as_double(j.get("rope_theta"), cfg->rope_theta)) {
    const Json *rp = j.get("rope_parameters");
    if (rp) as_double(rp->get("rope_theta"), cfg->rope_theta);
  }
  if (!as_int(j.get("num_key_value_heads"), cfg->num_key_value_heads)) cfg->num_key_value_heads = cfg->num_attention_heads;
  const Json *tie = j.get("tie_word_embeddings");
  cfg->tie_word_embeddings = tie && tie->kind == Json::kBool && tie->b ? 1 : 0;
  as_int(j.get("head_dim"), cfg->head_dim);  // stays 0 when absent or null
  if (!as_int(j.get("num_experts"), cfg->num_experts)) as_int(j.get("num_local_experts"), cfg->num_experts);
  // compute_rope_freqs (235-242): only rope_scaling of type "llama3" changes the frequencies
  const Json *rs = j.get("rope_scaling");
  if (rs && rs->kind == Json::kObject) {
    const Json *ty = rs->get("rope_type");
    if (!ty || ty->kind != Json::kString) ty = rs->get("type");
    if (ty && ty->kind == Json::kString && ty->str == "llama3") {
      int old_ctx = 0;
      if (!as_double(rs->get("factor"), cfg->rope_factor) || !as_double(rs->get("low_freq_factor"), cfg->rope_low_freq_factor) ||
          !as_double(rs->get("high_freq_factor"), cfg->rope_high_freq_factor) ||
          !as_int(rs->get("original_max_position_embeddings"), old_ctx))
        return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: incomplete llama3 rope_scaling");
      cfg->rope_original_max_position_embeddings = old_ctx;
      cfg->rope_llama3 = 1;
    }
  }
  return SHAINET_HIP_OK;
}

int shainet_hf_rope_freqs(const shainet_hf_llama_config *cfg, float *out, int n) {
  if (!cfg || !out) return -fail(SHAINET_HIP_ERR_ARGUMENT, "null argument");
  if (cfg->num_attention_heads < 1) return -fail(SHAINET_HIP_ERR_ARGUMENT, "num_attention_heads must be positive");
  const int head_dim = cfg->head_dim ? cfg->head_dim : cfg->hidden_size / cfg->num_attention_heads;
  if (!cfg->rope_llama3) return 0;  // nil: the block uses theta^(-2i/d)
  if (n != head_dim / 2) return -fail(SHAINET_HIP_ERR_ARGUMENT, "out must hold head_dim / 2 values");
  // hf_loader.cr:244-265, all in fp64, rounded once
  const double theta = cfg->rope_theta, factor = cfg->rope_factor;
  const double old_ctx = (double)cfg->rope_original_max_position_embeddings;
  const double low_freq_wavelen = old_ctx / cfg->rope_low_freq_factor;
  const double high_freq_wavelen = old_ctx / cfg->rope_high_freq_factor;
  for (int i = 0; i < head_dim / 2; ++i) {
    const double inv = 1.0 / pow(theta, 2.0 * i / head_dim);
    const double wavelen = 2.0 * M_PI / inv;
    double new_inv;
    if (wavelen < high_freq_wavelen) {
      new_inv = inv;
    } else if (wavelen > low_freq_wavelen) {
      new_inv = inv / factor;
    } else {
      const double smooth = (old_ctx / wavelen - cfg->rope_low_freq_factor) / (cfg->rope_high_freq_factor - cfg->rope_low_freq_factor);
      new_inv = (1.0 - smooth) * inv / factor + smooth * inv;
    }
    out[i] = (float)new_inv;
  }
  return head_dim / 2;
}

int shainet_hf_load_llama(const char *model_dir, shainet_llama_model **out) {
  if (!out) return fail(SHAINET_HIP_ERR_ARGUMENT, "out is null");
  *out = nullptr;
  shainet_hf_llama_config cfg;
  int rc = shainet_hf_read_llama_config(model_dir, &cfg);
  if (rc) return rc;
  const std::string mt = cfg.model_type;
  if (mt == "qwen3_moe" || cfg.num_experts > 0)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "mixture-of-experts models (" + mt + ") are not covered by this loader");
  if (mt != "llama" && mt != "mistral" && mt != "qwen2" && mt != "qwen3")  // hf_loader.cr:38-45
    return fail(SHAINET_HIP_ERR_ARGUMENT, "Unsupported model_type: '" + mt + "'. Supported: llama, mistral, qwen2, qwen3");
  if (!shainet_hip_available()) return fail(SHAINET_HIP_ERR_RUNTIME, "no gfx950 device available");
  shainet_safetensors *st = nullptr;
  if ((rc = shainet_safetensors_open(model_dir, &st))) return rc;
  shainet_llama_model *m = nullptr;
  rc = shainet_llama_model_create(&m, cfg.vocab_size, cfg.hidden_size, cfg.num_hidden_layers, cfg.num_attention_heads,
                                  cfg.num_key_value_heads, cfg.head_dim, cfg.intermediate_size, cfg.rms_norm_eps,
                                  cfg.rope_theta);
  const int d = cfg.hidden_size, ff = cfg.intermediate_size, V = cfg.vocab_size;
  const int head_dim = cfg.head_dim ? cfg.head_dim : (cfg.num_attention_heads ? d / cfg.num_attention_heads : 0);
  std::vector<float> freqs(head_dim / 2 > 0 ? head_dim / 2 : 1);
  int n_freqs = 0;
  if (!rc) {
    n_freqs = shainet_hf_rope_freqs(&cfg, freqs.data(), head_dim / 2);
    if (n_freqs < 0) rc = -n_freqs;
  }
  Stager stage;
  LlamaModelBuffers mb;
  if (!rc) rc = shainet_llama_model_buffers(m, &mb);
  if (!rc) rc = load_plain(st, stage, "model.embed_tokens.weight", V, d, mb.embedding);  // [vocab, d]
  for (int li = 0; li < cfg.num_hidden_layers && !rc; ++li) {
    shainet_llama_block *b = shainet_llama_model_block(m, li);
    shainet_llama_attn *a = shainet_llama_block_attn(b);
    const std::string p = "model.layers." + std::to_string(li);
    rc = shainet_llama_attn_set_rope(a, cfg.rope_theta, n_freqs > 0 ? freqs.data() : nullptr);
    LlamaBlockBuffers bb;
    if (!rc) rc = shainet_llama_block_buffers(b, &bb);
    if (rc) break;
    const long long wide = bb.q_dim + 2LL * bb.kv_dim;
    // attention weights: HF is [out, in], the products are x * W, so [in, out] (hf_loader.cr:325-329)
    if ((rc = load_transposed(st, stage, p + ".self_attn.q_proj.weight", bb.q_dim, d, bb.w_qkv, wide, 0))) break;
    if ((rc = load_transposed(st, stage, p + ".self_attn.k_proj.weight", bb.kv_dim, d, bb.w_qkv, wide, bb.q_dim))) break;
    if ((rc = load_transposed(st, stage, p + ".self_attn.v_proj.weight", bb.kv_dim, d, bb.w_qkv, wide,
                              bb.q_dim + bb.kv_dim)))
      break;
    if ((rc = load_transposed(st, stage, p + ".self_attn.o_proj.weight", d, bb.q_dim, bb.w_o, d, 0))) break;
    // dense SwiGLU (333-336)
    if ((rc = load_transposed(st, stage, p + ".mlp.gate_proj.weight", ff, d, bb.gate_up, 2LL * ff, 0))) break;
    if ((rc = load_transposed(st, stage, p + ".mlp.up_proj.weight", ff, d, bb.gate_up, 2LL * ff, ff))) break;
    if ((rc = load_transposed(st, stage, p + ".mlp.down_proj.weight", d, ff, bb.down, d, 0))) break;
    // RMSNorm (349-350)
    if ((rc = load_plain(st, stage, p + ".input_layernorm.weight", 1, d, bb.norm1->gamma))) break;
    if ((rc = load_plain(st, stage, p + ".post_attention_layernorm.weight", 1, d, bb.norm2->gamma))) break;
    // optional Q/K/V biases, a complete set or none (352-363)
    const bool hq = st->find(p + ".self_attn.q_proj.bias"), hk = st->find(p + ".self_attn.k_proj.bias"),
               hv = st->find(p + ".self_attn.v_proj.bias");
    if (hq || hk || hv) {
      if (!(hq && hk && hv)) {
        rc = fail(SHAINET_HIP_ERR_ARGUMENT, "Incomplete Q/K/V projection biases for " + p);
        break;
      }
      std::vector<float> bq, bk, bv;
      if ((rc = read_host_vector(st, p + ".self_attn.q_proj.bias", bq)) ||
          (rc = read_host_vector(st, p + ".self_attn.k_proj.bias", bk)) ||
          (rc = read_host_vector(st, p + ".self_attn.v_proj.bias", bv)))
        break;
      if ((rc = shainet_llama_attn_set_bias(a, bq.data(), (int)bq.size(), bk.data(), (int)bk.size(), bv.data(),
                                            (int)bv.size())))
        break;
    }
    // optional Qwen3 QK-norm weights, a complete pair or none (365-375)
    const bool hqn = st->find(p + ".self_attn.q_norm.weight"), hkn = st->find(p + ".self_attn.k_norm.weight");
    if (hqn || hkn) {
      if (!(hqn && hkn)) {
        rc = fail(SHAINET_HIP_ERR_ARGUMENT, "Incomplete QK-norm weights for " + p);
        break;
      }
      std::vector<float> qn, kn;
      if ((rc = read_host_vector(st, p + ".self_attn.q_norm.weight", qn)) ||
          (rc = read_host_vector(st, p + ".self_attn.k_norm.weight", kn)))
        break;
      if ((rc = shainet_llama_attn_set_qk_norm(a, qn.data(), (int)qn.size(), kn.data(), (int)kn.size()))) break;
    }
  }
  // final RMSNorm and the output head (393-404)
  if (!rc) rc = load_plain(st, stage, "model.norm.weight", 1, d, mb.final_norm->gamma);
  if (!rc) {
    if (cfg.tie_word_embeddings) {  // embed.transpose: [d, vocab] from the rows already on the device
      dim3 grid((unsigned)((d + 31) / 32), (unsigned)((V + 31) / 32));
      hipLaunchKernelGGL(convert_transpose_kernel, grid, dim3(256), 0, nullptr, (const void *)mb.embedding, mb.lm_head, V,
                         d, (long long)V, (int)kF32);
      if (hipGetLastError() != hipSuccess || hipDeviceSynchronize() != hipSuccess)
        rc = fail(SHAINET_HIP_ERR_RUNTIME, "transposing the tied embedding failed");
    } else {
      rc = load_transposed(st, stage, "lm_head.weight", V, d, mb.lm_head, V, 0);
    }
  }
  shainet_safetensors_close(st);
  if (rc) {
    shainet_llama_model_destroy(m);
    return rc;
  }
  *out = m;
  return SHAINET_HIP_OK;
}

}  // extern "C"

// ---- designs whose config.json lists their layers one by one ---------------------------------
namespace {

// Numbers of an object that must be there; the first one that is not is named in the error.
struct Fields {
  const Json *obj;
  std::string where, missing;
  int integer(const char *key) {
    int v = 0;
    if (!obj || !as_int(obj->get(key), v) || !obj->get(key)->is_int) note(key);
    return v;
  }
  double real(const char *key) {
    double v = 0.0;
    if (!obj || !as_double(obj->get(key), v)) note(key);
    return v;
  }
  const Json *object(const char *key) {
    const Json *o = obj ? obj->get(key) : nullptr;
    if (!o || o->kind != Json::kObject) note(key);
    return o && o->kind == Json::kObject ? o : nullptr;
  }
  void note(const char *key) {
    if (missing.empty()) missing = where + key;
  }
  int status() const {
    return missing.empty() ? SHAINET_HIP_OK : fail(SHAINET_HIP_ERR_ARGUMENT, "config.json lacks " + missing);
  }
};

struct LayerConfig {
  shainet_latent_config mixer = {};
  int ff = 0;           // 0: no feed-forward
  int weights_of = -1;  // the layer whose weights it uses
};
struct TutilornConfig {
  int vocab = 0, width = 0;
  double eps = 0.0, embedding_scale = 1.0;
  std::vector<LayerConfig> layers;
};

int read_layer(const Json &j, int index, LayerConfig &out) {
  const std::string where = "layers[" + std::to_string(index) + "].";
  const Json *type = j.get("type");
  if (!type || type->kind != Json::kString) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json lacks " + where + "type");
  if (type->str != "latent_attention")
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "type '" + type->str + "' is not a mixer this library has");
  Fields top = {&j, where, ""};
  const Json *mixer = top.object("mixer");
  if (int rc = top.status()) return rc;
  Fields f = {mixer, where + "mixer.", ""};
  shainet_latent_config &m = out.mixer;
  m.heads = f.integer("heads");
  m.dim = f.integer("dim");
  m.rot_dim = f.integer("rot_dim");
  m.vdim = f.integer("vdim");
  m.kv_rank = f.integer("kv_rank");
  m.q_rank = f.integer("q_rank");
  m.scale = f.real("scale");
  Fields rot = {f.object("rot"), where + "mixer.rot.", ""};
  m.rot_dims = rot.integer("dims");
  m.rot_base = rot.real("base");
  const Json *mask = mixer->get("mask");
  Fields win = {mask, where + "mixer.mask.", ""};
  if (mask && !mask->is_null()) {  // without a mask: every position up to its own
    m.window = win.integer("size");
    if (win.missing.empty() && m.window < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + win.where + "size must be positive");
  }
  for (const Fields *x : {&f, &rot, &win})
    if (int rc = x->status()) return rc;
  const Json *mlp = j.get("mlp");
  if (mlp && !mlp->is_null()) {
    const Json *kind = mlp->get("kind");
    if (!kind || kind->kind != Json::kString || kind->str != "dense")
      return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "mlp.kind must be \"dense\"");
    Fields g = {mlp, where + "mlp.", ""};
    out.ff = g.integer("ff");
    if (int rc = g.status()) return rc;
    if (out.ff < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "mlp.ff must be positive");
  }
  const Json *of = j.get("weights_of");
  if (of && !of->is_null() && !as_int(of, out.weights_of)) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "weights_of is not a layer");
  return SHAINET_HIP_OK;
}

int read_tutilorn_config(const Json &j, TutilornConfig &c) {
  Fields f = {&j, "", ""};
  c.vocab = f.integer("vocab");
  c.width = f.integer("width");
  Fields norm = {f.object("norm"), "norm.", ""}, emb = {f.object("embedding"), "embedding.", ""};
  c.eps = norm.real("eps");
  c.embedding_scale = emb.real("scale");
  for (const Fields *x : {&f, &norm, &emb})
    if (int rc = x->status()) return rc;
  if (c.vocab < 1 || c.width < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: vocab and width must be positive");
  const Json *layers = j.get("layers");
  if (!layers || layers->kind != Json::kArray || layers->arr.empty())
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json lacks layers");
  const int n = (int)layers->arr.size();
  c.layers.resize(n);
  for (int i = 0; i < n; ++i)
    if (int rc = read_layer(layers->arr[i], i, c.layers[i])) return rc;
  for (int i = 0; i < n; ++i) {  // a layer that borrows may lend what it borrowed
    int owner = i, steps = 0;
    while (c.layers[owner].weights_of >= 0 && steps++ <= n) {
      owner = c.layers[owner].weights_of;
      if (owner >= n) break;
    }
    if (owner >= n || steps > n)
      return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: layers[" + std::to_string(i) + "].weights_of leads to no layer with weights");
    if (owner != i) {
      const LayerConfig &a = c.layers[i], &b = c.layers[owner];
      const shainet_latent_config &p = a.mixer, &q = b.mixer;
      if (p.heads != q.heads || p.dim != q.dim || p.rot_dim != q.rot_dim || p.vdim != q.vdim || p.kv_rank != q.kv_rank ||
          p.q_rank != q.q_rank || p.window != q.window || p.rot_dims != q.rot_dims || p.rot_base != q.rot_base ||
          p.scale != q.scale || a.ff != b.ff)
        return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: layers[" + std::to_string(i) + "] differs from the layer whose weights it uses");
    }
  }
  for (int i = 0; i < n; ++i)  // (only now: the walk above follows the links as they are written)
    while (c.layers[i].weights_of >= 0 && c.layers[c.layers[i].weights_of].weights_of >= 0)
      c.layers[i].weights_of = c.layers[c.layers[i].weights_of].weights_of;
  return SHAINET_HIP_OK;
}

int load_norm(const shainet_safetensors *st, Stager &stage, const std::string &name, int d, NormWeights &n) {
  int rc = load_plain(st, stage, name, 1, d, n.gamma);
  if (rc || n.kind != kNormDynTanh) return rc;
  if ((rc = load_plain(st, stage, name + ".b", 1, d, n.beta))) return rc;
  std::vector<float> alpha;
  if ((rc = read_host_vector(st, name + ".alpha", alpha))) return rc;
  if (alpha.size() != 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "tensor '" + name + ".alpha' is not a scalar");
  n.alpha = alpha[0];
  return SHAINET_HIP_OK;
}

int load_latent_mixer(const shainet_safetensors *st, Stager &stage, const std::string &p, int d, const shainet_latent_config &c,
                      LatentWeights &w) {
  const int qw = c.heads * (c.dim + c.rot_dim), kw = c.heads * c.dim, vw = c.heads * c.vdim;
  int rc;
  if ((rc = load_transposed(st, stage, p + "dq", c.q_rank, d, w.w_in, w.n_in, 0))) return rc;
  if ((rc = load_transposed(st, stage, p + "dkv", c.kv_rank + c.rot_dim, d, w.w_in, w.n_in, c.q_rank))) return rc;
  if ((rc = load_transposed(st, stage, p + "g", c.heads, d, w.w_in, w.n_in, c.q_rank + c.kv_rank + c.rot_dim))) return rc;
  if ((rc = load_plain(st, stage, p + "dq.norm", 1, c.q_rank, w.dq_norm))) return rc;
  if ((rc = load_plain(st, stage, p + "dkv.norm", 1, c.kv_rank, w.dkv_norm))) return rc;
  if ((rc = load_transposed(st, stage, p + "uq", qw, c.q_rank, w.w_uq, qw, 0))) return rc;
  // W_uk and W_uv twice: a row per output (absorbed), and side by side as a product's matrix (expanded)
  if ((rc = load_plain(st, stage, p + "uk", kw, c.kv_rank, w.u_kv))) return rc;
  if ((rc = load_plain(st, stage, p + "uv", vw, c.kv_rank, w.u_kv + (size_t)kw * c.kv_rank))) return rc;
  if ((rc = load_transposed(st, stage, p + "uk", kw, c.kv_rank, w.w_ukv, kw + vw, 0))) return rc;
  if ((rc = load_transposed(st, stage, p + "uv", vw, c.kv_rank, w.w_ukv, kw + vw, kw))) return rc;
  if ((rc = load_plain(st, stage, p + "sink", 1, c.heads, w.sink))) return rc;
  if ((rc = load_transposed(st, stage, p + "o", d, vw, w.w_o, d, 0))) return rc;
  w.w_in_t_stale = w.w_uq_t_stale = w.w_o_t_stale = true;
  return SHAINET_HIP_OK;
}

// Tutilorn: latent attention with sliding windows, sinks and output gates, Dynamic Tanh norms, dense SwiGLU
// feed-forwards, layers that may use another layer's weights.
int load_tutilorn(const char *model_dir, const Json &j, shainet_llama_model **out) {
  TutilornConfig cfg;
  int rc = read_tutilorn_config(j, cfg);
  if (rc) return rc;
  if (!shainet_hip_available()) return fail(SHAINET_HIP_ERR_RUNTIME, "no gfx950 device available");
  const int d = cfg.width, n = (int)cfg.layers.size();
  shainet_safetensors *st = nullptr;
  if ((rc = shainet_safetensors_open(model_dir, &st))) return rc;
  shainet_llama_model *m = nullptr;
  Stager stage;
  rc = shainet_llama_model_create_empty(&m, cfg.vocab, d, cfg.eps, cfg.embedding_scale, kNormDynTanh);
  std::vector<shainet_llama_block *> blocks(n, nullptr);
  for (int pass = 0; pass < 2; ++pass)  // layers with weights first: the others may come before them
    for (int i = 0; i < n && !rc; ++i) {
      const LayerConfig &lc = cfg.layers[i];
      if ((lc.weights_of >= 0) != (pass == 1)) continue;
      rc = shainet_llama_block_create_latent(&blocks[i], d, lc.mixer, lc.ff, kNormDynTanh, cfg.eps,
                                             pass ? blocks[lc.weights_of] : nullptr);
    }
  for (int i = 0; i < n && !rc; ++i) {
    const LayerConfig &lc = cfg.layers[i];
    if (lc.weights_of >= 0) continue;
    const std::string p = "l" + std::to_string(i) + ".";
    LlamaBlockBuffers bb;
    if ((rc = shainet_llama_block_buffers(blocks[i], &bb))) break;
    if ((rc = load_norm(st, stage, p + "norm1", d, *bb.norm1))) break;
    if ((rc = load_latent_mixer(st, stage, p + "mix.", d, lc.mixer, latent_attn_weights(shainet_llama_block_latent_mixer(blocks[i]))))) break;
    if (!lc.ff) continue;
    if ((rc = load_norm(st, stage, p + "norm2", d, *bb.norm2))) break;
    if ((rc = load_transposed(st, stage, p + "mlp.gate", lc.ff, d, bb.gate_up, 2LL * lc.ff, 0))) break;
    if ((rc = load_transposed(st, stage, p + "mlp.up", lc.ff, d, bb.gate_up, 2LL * lc.ff, lc.ff))) break;
    if ((rc = load_transposed(st, stage, p + "mlp.down", d, lc.ff, bb.down, d, 0))) break;
  }
  // the model owns the blocks from here on, in the order of the layers
  for (int i = 0; i < n; ++i)
    if (blocks[i]) {
      if (m)
        shainet_llama_model_add_block(m, blocks[i]);
      else
        shainet_llama_block_destroy(blocks[i]);
    }
  LlamaModelBuffers mb;
  if (!rc) rc = shainet_llama_model_buffers(m, &mb);
  if (!rc) rc = load_plain(st, stage, "embed", cfg.vocab, d, mb.embedding);
  if (!rc) rc = load_norm(st, stage, "final.norm", d, *mb.final_norm);
  if (!rc) rc = load_transposed(st, stage, "head", cfg.vocab, d, mb.lm_head, cfg.vocab, 0);
  shainet_safetensors_close(st);
  if (rc) {
    shainet_llama_model_destroy(m);
    return rc;
  }
  *out = m;
  return SHAINET_HIP_OK;
}

// Zabutar: layers of HGRN2 or of attention with a bias by distance (which may use another layer's keys and
// values), each sublayer between two RMS norms and behind a short convolution over time, feed-forwards with
// xIELU or of experts, learned positions.
struct ZabutarLayer {
  bool recurrent = false;
  Hgrn2Config hgrn2;
  BiasedConfig attention;
  int kv_from = -1;
  int ff = 0;         // > 0: a dense feed-forward
  MoeShape moe = {};  // experts > 0: a mixture; neither: no feed-forward
};
struct ZabutarConfig {
  int vocab = 0, width = 0, max_positions = 0, taps = 0;
  double eps = 0.0;
  std::vector<ZabutarLayer> layers;
};

bool given(const Json *obj, const char *key) {
  const Json *v = obj ? obj->get(key) : nullptr;
  return v && !v->is_null();
}

int read_zabutar_mlp(const Json &mlp, const std::string &where, int width, ZabutarLayer &out) {
  const Json *kind = mlp.get("kind");
  if (!kind || kind->kind != Json::kString) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json lacks " + where + "kind");
  Fields f = {&mlp, where, ""};
  if (kind->str == "dense") {
    out.ff = f.integer("ff");
    if (int rc = f.status()) return rc;
    return out.ff > 0 ? SHAINET_HIP_OK : fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "ff must be positive");
  }
  if (kind->str != "moe") return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "kind '" + kind->str + "' is not a feed-forward this library has");
  MoeShape &m = out.moe;
  m.d = width;
  m.groups = m.keep = 1;
  m.scale = 1.f;
  Fields expert = {f.object("expert"), where + "expert.", ""}, router = {f.object("router"), where + "router.", ""};
  if (int rc = f.status()) return rc;
  m.ff = expert.integer("ff");
  m.experts = router.integer("experts");
  m.top = router.integer("top");
  if (given(router.obj, "identity")) m.identity = router.integer("identity");
  if (given(router.obj, "scale")) m.scale = (float)router.real("scale");
  Fields groups = {nullptr, where + "router.groups.", ""}, shared = {nullptr, where + "shared.", ""};
  if (given(router.obj, "groups")) {
    groups.obj = router.object("groups");
    m.groups = groups.integer("count");
    m.keep = groups.integer("keep");
  }
  if (given(&mlp, "shared")) {
    shared.obj = f.object("shared");
    m.shared_ff = shared.integer("ff");
    if (shared.missing.empty() && m.shared_ff < 1) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + shared.where + "ff must be positive");
  }
  for (const Fields *x : {&f, &expert, &router, &groups, &shared})
    if (int rc = x->status()) return rc;
  if (!moe_shape_ok(m))
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "router: at most 1024 outputs in equal groups, and top at most what the kept groups hold");
  return SHAINET_HIP_OK;
}

int read_zabutar_layer(const Json &j, int index, int width, ZabutarLayer &out) {
  const std::string where = "layers[" + std::to_string(index) + "].";
  const Json *type = j.get("type");
  if (!type || type->kind != Json::kString) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json lacks " + where + "type");
  out.recurrent = type->str == "hgrn2";
  if (!out.recurrent && type->str != "attention")
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "type '" + type->str + "' is not a mixer this design has");
  Fields top = {&j, where, ""};
  Fields f = {top.object("mixer"), where + "mixer.", ""};
  if (int rc = top.status()) return rc;
  if (out.recurrent) {
    out.hgrn2.heads = f.integer("heads");
    out.hgrn2.dim = f.integer("dim");
    out.hgrn2.vdim = f.integer("vdim");
  } else {
    BiasedConfig &a = out.attention;
    a.heads = f.integer("heads");
    a.kv_heads = f.integer("kv_heads");
    a.dim = f.integer("dim");
    a.vdim = f.integer("vdim");
    a.scale = f.real("scale");
    a.bias_max = f.integer("bias_max");
    if (given(f.obj, "kv_from")) {
      out.kv_from = f.integer("kv_from");
      if (out.kv_from < 0) return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: " + where + "mixer.kv_from is not a layer");
    }
  }
  if (int rc = f.status()) return rc;
  const Json *mlp = j.get("mlp");
  return mlp && !mlp->is_null() ? read_zabutar_mlp(*mlp, where + "mlp.", width, out) : SHAINET_HIP_OK;
}

int read_zabutar_config(const Json &j, ZabutarConfig &c) {
  Fields f = {&j, "", ""};
  c.vocab = f.integer("vocab");
  c.width = f.integer("width");
  c.max_positions = f.integer("max_positions");
  Fields norm = {f.object("norm"), "norm.", ""}, canon = {f.object("canon"), "canon.", ""};
  c.eps = norm.real("eps");
  c.taps = canon.integer("taps");
  for (const Fields *x : {&f, &norm, &canon})
    if (int rc = x->status()) return rc;
  if (c.vocab < 1 || c.width < 1 || c.max_positions < 1)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: vocab, width and max_positions must be positive");
  if (c.taps < 1 || c.taps > kMaxConvTaps)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: canon.taps must be in [1, " + std::to_string(kMaxConvTaps) + "]");
  const Json *layers = j.get("layers");
  if (!layers || layers->kind != Json::kArray || layers->arr.empty())
    return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json lacks layers");
  const int n = (int)layers->arr.size();
  c.layers.resize(n);
  for (int i = 0; i < n; ++i) {
    ZabutarLayer &l = c.layers[i];
    if (int rc = read_zabutar_layer(layers->arr[i], i, c.width, l)) return rc;
    if (l.kv_from < 0) continue;
    const ZabutarLayer *from = l.kv_from < i ? &c.layers[l.kv_from] : nullptr;
    if (!from || from->recurrent || from->kv_from >= 0 || from->attention.kv_heads != l.attention.kv_heads ||
        from->attention.dim != l.attention.dim || from->attention.vdim != l.attention.vdim)
      return fail(SHAINET_HIP_ERR_ARGUMENT, "config.json: layers[" + std::to_string(i) +
                                                "].mixer.kv_from is not an earlier attention layer with projections of its own and the same heads");
  }
  return SHAINET_HIP_OK;
}

// an RMS norm's weight, stored as the distance from 1
int load_centred_norm(const shainet_safetensors *st, Stager &stage, const std::string &name, int d, float *dst) {
  if (int rc = load_plain(st, stage, name, 1, d, dst)) return rc;
  if (launch_add_one(dst, d, nullptr) != hipSuccess || hipDeviceSynchronize() != hipSuccess)
    return fail(SHAINET_HIP_ERR_RUNTIME, "converting tensor '" + name + "' failed");
  return SHAINET_HIP_OK;
}

int load_hgrn2(const shainet_safetensors *st, Stager &stage, const std::string &p, int d, const Hgrn2Config &c, Hgrn2Weights &w) {
  const int qw = c.heads * c.dim, vw = c.heads * c.vdim;
  int rc;
  if ((rc = load_transposed(st, stage, p + "q", qw, d, w.w_in, w.n_in, 0))) return rc;
  if ((rc = load_transposed(st, stage, p + "f", qw, d, w.w_in, w.n_in, qw))) return rc;
  if ((rc = load_transposed(st, stage, p + "v", vw, d, w.w_in, w.n_in, 2 * qw))) return rc;
  if ((rc = load_plain(st, stage, p + "f.b", 1, qw, w.f_bias))) return rc;
  if ((rc = load_plain(st, stage, p + "lower", 1, qw, w.lower))) return rc;
  if ((rc = load_plain(st, stage, p + "norm", 1, c.vdim, w.norm))) return rc;
  return load_transposed(st, stage, p + "o", d, vw, w.w_o, d, 0);
}

int load_biased(const shainet_safetensors *st, Stager &stage, const std::string &p, int d, const ZabutarLayer &l, int max_positions,
                BiasedAttn *mixer) {
  const BiasedConfig &c = l.attention;
  BiasedWeights &w = biased_attn_weights(mixer);
  const int qw = c.heads * c.dim, kw = c.kv_heads * c.dim, vw = c.kv_heads * c.vdim;
  int rc;
  if ((rc = load_transposed(st, stage, p + "q", qw, d, w.w_in, w.n_in, 0))) return rc;
  if (l.kv_from < 0) {
    if ((rc = load_transposed(st, stage, p + "k", kw, d, w.w_in, w.n_in, qw))) return rc;
    if ((rc = load_transposed(st, stage, p + "v", vw, d, w.w_in, w.n_in, qw + kw))) return rc;
  }
  const StTensor *t = need(st, p + "rel", rc);
  if (!t) return rc;
  if (t->shape.size() != 2 || t->shape[0] < 1 || t->shape[1] != c.heads)
    return fail(SHAINET_HIP_ERR_ARGUMENT, "tensor '" + p + "rel' is not [rows, heads]");
  std::vector<float> rel;
  if ((rc = read_host_vector(st, p + "rel", rel))) return rc;
  if ((rc = biased_attn_set_table(mixer, rel, (int)t->shape[0], max_positions))) return rc;
  return load_transposed(st, stage, p + "o", d, c.heads * c.vdim, w.w_o, d, 0);
}

int load_xielu(const shainet_safetensors *st, Stager &stage, const std::string &p, int d, int ff, DenseWeights &w) {
  int rc;
  if ((rc = load_transposed(st, stage, p + "up", ff, d, w.up, ff, 0))) return rc;
  if ((rc = load_plain(st, stage, p + "up.b", 1, ff, w.up_bias))) return rc;
  if ((rc = load_transposed(st, stage, p + "down", d, ff, w.down, d, 0))) return rc;
  if ((rc = load_plain(st, stage, p + "down.b", 1, d, w.down_bias))) return rc;
  std::vector<float> act;
  if ((rc = read_host_vector(st, p + "act", act))) return rc;
  if (act.size() != 2) return fail(SHAINET_HIP_ERR_ARGUMENT, "tensor '" + p + "act' does not hold two numbers");
  auto softplus = [](double z) { return z > 0 ? z + log1p(exp(-z)) : log1p(exp(z)); };
  w.act.kind = kActXielu;
  w.act.pos = (float)softplus(act[0]);
  w.act.neg = (float)(0.5 + softplus(act[1]));
  return SHAINET_HIP_OK;
}

int load_experts(const shainet_safetensors *st, Stager &stage, const std::string &p, const MoeShape &m, MoeWeights &w) {
  const int n = m.experts + m.identity;
  const size_t mat = (size_t)m.ff * m.d;
  int rc;
  if ((rc = load_plain(st, stage, p + "router", n, m.d, w.router))) return rc;
  if ((rc = load_transposed(st, stage, p + "router", n, m.d, w.router_in, w.n_router, 0))) return rc;
  if ((rc = load_plain(st, stage, p + "correction", 1, n, w.correction))) return rc;
  for (int e = 0; e < m.experts; ++e) {
    const std::string pe = p + "e" + std::to_string(e) + ".";
    if ((rc = load_plain(st, stage, pe + "gate", m.ff, m.d, w.gate_up + 2 * e * mat))) return rc;
    if ((rc = load_plain(st, stage, pe + "up", m.ff, m.d, w.gate_up + (2 * e + 1) * mat))) return rc;
    if ((rc = load_plain(st, stage, pe + "down", m.d, m.ff, w.down + e * mat))) return rc;
  }
  if (!m.shared_ff) return SHAINET_HIP_OK;
  const std::string ps = p + "shared.";
  const int ff = m.shared_ff;
  if ((rc = load_plain(st, stage, ps + "gate", ff, m.d, w.shared_gate_up))) return rc;
  if ((rc = load_plain(st, stage, ps + "up", ff, m.d, w.shared_gate_up + (size_t)ff * m.d))) return rc;
  if ((rc = load_plain(st, stage, ps + "down", m.d, ff, w.shared_down))) return rc;
  if ((rc = load_transposed(st, stage, ps + "gate", ff, m.d, w.shared_gate_up_in, 2LL * ff, 0))) return rc;
  if ((rc = load_transposed(st, stage, ps + "up", ff, m.d, w.shared_gate_up_in, 2LL * ff, ff))) return rc;
  return load_transposed(st, stage, ps + "down", m.d, ff, w.shared_down_in, m.d, 0);
}

// One layer: its parts made and filled.
int load_zabutar_layer(const shainet_safetensors *st, Stager &stage, const ZabutarConfig &cfg, int i,
                       const std::vector<shainet_llama_block *> &before, shainet_llama_block **out) {
  const ZabutarLayer &l = cfg.layers[i];
  const int d = cfg.width;
  const std::string p = "l" + std::to_string(i) + ".";
  Mixer *mixer = nullptr;
  FeedForward *ff = nullptr;
  DenseWeights *dense = nullptr;
  MoeWeights *moe = nullptr;
  int rc = l.recurrent ? hgrn2_create(&mixer, d, l.hgrn2, cfg.eps)
                       : biased_attn_create(&mixer, d, l.attention, l.kv_from < 0 ? nullptr : shainet_llama_block_mixer_of(before[l.kv_from]));
  if (!rc && l.ff) rc = dense_create(&ff, d, l.ff, &dense);
  if (!rc && l.moe.experts) rc = moe_create(&ff, l.moe, &moe);
  if (rc) {
    delete mixer;
    return rc;
  }
  if ((rc = shainet_llama_block_create_wrapped(out, d, mixer, ff, cfg.taps, cfg.eps))) return rc;
  const WrappedBlockBuffers b = shainet_llama_block_wrapped_buffers(*out);
  if ((rc = load_centred_norm(st, stage, p + "norm1", d, b.norm1))) return rc;
  if ((rc = load_centred_norm(st, stage, p + "norm1b", d, b.post1))) return rc;
  if ((rc = load_transposed(st, stage, p + "canon1", d, cfg.taps, b.conv1, d, 0))) return rc;
  rc = l.recurrent ? load_hgrn2(st, stage, p + "mix.", d, l.hgrn2, hgrn2_weights(mixer->hgrn2()))
                   : load_biased(st, stage, p + "mix.", d, l, cfg.max_positions, mixer->biased());
  if (rc || !ff) return rc;
  if ((rc = load_centred_norm(st, stage, p + "norm2", d, b.norm2))) return rc;
  if ((rc = load_centred_norm(st, stage, p + "norm2b", d, b.post2))) return rc;
  if ((rc = load_transposed(st, stage, p + "canon2", d, cfg.taps, b.conv2, d, 0))) return rc;
  return dense ? load_xielu(st, stage, p + "mlp.", d, l.ff, *dense) : load_experts(st, stage, p + "mlp.", l.moe, *moe);
}

int load_zabutar(const char *model_dir, const Json &j, shainet_llama_model **out) {
  ZabutarConfig cfg;
  int rc = read_zabutar_config(j, cfg);
  if (rc) return rc;
  if (!shainet_hip_available()) return fail(SHAINET_HIP_ERR_RUNTIME, "no gfx950 device available");
  const int d = cfg.width, n = (int)cfg.layers.size();
  shainet_safetensors *st = nullptr;
  if ((rc = shainet_safetensors_open(model_dir, &st))) return rc;
  shainet_llama_model *m = nullptr;
  Stager stage;
  rc = shainet_llama_model_create_empty(&m, cfg.vocab, d, cfg.eps, 1.0, kNormRms);
  std::vector<shainet_llama_block *> blocks;
  for (int i = 0; i < n && !rc; ++i) {
    shainet_llama_block *b = nullptr;
    rc = load_zabutar_layer(st, stage, cfg, i, blocks, &b);
    if (!b) break;
    blocks.push_back(b);
    shainet_llama_model_add_block(m, b);  // owned by the model from here on
  }
  LlamaModelBuffers mb;
  float *positions = nullptr;
  if (!rc) rc = shainet_llama_model_buffers(m, &mb);
  if (!rc) rc = shainet_llama_model_position_buffer(m, cfg.max_positions, &positions);
  if (!rc) rc = load_plain(st, stage, "embed", cfg.vocab, d, mb.embedding);
  if (!rc) rc = load_plain(st, stage, "pos", cfg.max_positions, d, positions);
  if (!rc) rc = load_centred_norm(st, stage, "final.norm", d, mb.final_norm->gamma);
  if (!rc) rc = load_transposed(st, stage, "head", cfg.vocab, d, mb.lm_head, cfg.vocab, 0);
  shainet_safetensors_close(st);
  if (rc) {
    shainet_llama_model_destroy(m);
    return rc;
  }
  *out = m;
  return SHAINET_HIP_OK;
}

// Designs by the name their config.json gives under "architecture".
struct Design {
  const char *name;
  int (*load)(const char *model_dir, const Json &config, shainet_llama_model **out);
};
constexpr Design kDesigns[] = {{"Tutilorn", load_tutilorn}, {"Zabutar", load_zabutar}};

}  // namespace

extern "C" {

int shainet_hf_load_model(const char *model_dir, shainet_llama_model **out) {
  if (!model_dir || !out) return fail(SHAINET_HIP_ERR_ARGUMENT, "null argument");
  *out = nullptr;
  Json j;
  if (int rc = read_config(model_dir, j)) return rc;
  const Json *arch = j.get("architecture");
  if (!arch || arch->kind != Json::kString) return shainet_hf_load_llama(model_dir, out);  // goes by model_type
  for (const Design &d : kDesigns)
    if (arch->str == d.name) return d.load(model_dir, j, out);
  std::string known;
  for (const Design &d : kDesigns) known += std::string(known.empty() ? "" : ", ") + d.name;
  return fail(SHAINET_HIP_ERR_ARGUMENT, "Unsupported architecture: '" + arch->str + "'. Supported: " + known);
}

}  // extern "C"
