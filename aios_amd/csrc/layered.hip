// LayeredDecoder implementation -- see layered.h.
//
// Per layer, 16-bit engine (weights, activations and cache bf16; residual, norms, scores fp32):
//   1-4 rows    one GEMV over [q | kv down | gate | MLP gate/up] with the RMSNorm in its prologue and the
//               GLU in its epilogue; latent prep; attention; normalise + Wuv + gate; one GEMV over
//               [attention out | MLP down] adding to the residual          -- 5 launches
//   5-64 rows   the same two products through the skinny MFMA GEMM, the RMSNorm split across them
//   more rows   prefill GEMMs; long portions take the expanded attention (latent.h)
// Sequential layers (mixer, then feed-forward, each closed by its residual gate and norms): every product reads a
// bf16 operand that the row operation before it wrote (mixers.h), so a layer is
//   input product (+ residual gate rows) | mixer | output product | close | input product (+ residual gate and
//   router rows, GLU in its epilogue) | experts | down product | close
// Where a sublayer's result is added as it is (no gate, no norm of it), batches up to 64 rows need no row operations: as
// above, the product that reads the residual normalises it and the one before adds to it (layer_fused).
// Mixers that read the same input share the input product and the output product: a layer's attention and linear
// recurrence leave their results side by side in one operand.
// 32-bit engine: the same steps in fp32, absorbed attention for every row.
#include "layered.h"

#include <algorithm>
#include <cmath>
#include <cstdlib>
#include <cstring>
#include <set>

#include "engine.h"

namespace aios {

static int up(int x, int a) { return (x + a - 1) / a * a; }
// rows of a product of its own: whole tiles of the prefill GEMM
static int up_n(int x) { return x <= 1024 ? up(x, 128) : up(x, 256); }
static int env_or(const char* name, int dflt) {
  const char* e = std::getenv(name);
  return e ? std::atoi(e) : dflt;
}
// padded latent widths the attention kernels are built for
static int pad_rank(int r) {
  for (int t : {2, 4, 6, 8, 10, 12, 16, 32})
    if (r <= 64 * t) return 64 * t;
  throw std::runtime_error("latent attention: cached rows above 2048 numbers");
}

LayeredDecoder::LayeredDecoder(Engine& e) : e_(e) {
  const EngineConfig& c = e.cfg_;
  nl_ = (int)c.layers.size();
  d_ = c.d_model;
  dp_ = up(d_, 64);
  v_ = c.vocab_size;
  vp_ = up(v_, 64);
  f32_ = c.compute_f32;
  if (d_ < 1 || v_ < 1 || c.max_positions < 0 || c.max_ctx < 1) throw std::runtime_error("layered model: bad sizes");
  if (c.tp_size > 1) throw std::runtime_error("layered models run on one GPU (no tensor parallelism)");
  if (c.kv_fp8) throw std::runtime_error("layered models: the cache has no fp8 form");
  if (c.loop_times > 0 && !(c.loop_start >= 0 && c.loop_start < c.loop_stop && c.loop_stop <= nl_))
    throw std::runtime_error("layered model: bad loop");
  if (c.bigram_buckets < 0) throw std::runtime_error("layered model: bad pair table");
  seq_ = !c.layers[0].parallel;
  recurrent_ = c.bigram_buckets > 0;
  dims_.resize(nl_);
  owner_.resize(nl_);
  w_.resize(nl_);
  rope_.assign(nl_, nullptr);
  bool all_windowed = true;
  for (int i = 0; i < nl_; ++i) {
    int o = i;
    for (int hop = 0; c.layers[o].weights_of >= 0; ++hop) {
      o = c.layers[o].weights_of;
      if (o >= nl_ || hop > nl_) throw std::runtime_error("layer " + std::to_string(i) + ": weights_of names no layer");
    }
    owner_[i] = o;
    const LayerSpec &s = c.layers[i], &t = c.layers[o];
    const std::string at = "layer " + std::to_string(i) + ": ";
    if (!s.parallel != seq_) throw std::runtime_error(at + "parallel and sequential layers in one model");
    if (s.mixer != t.mixer || s.heads != t.heads || s.dim != t.dim || s.vdim != t.vdim || s.kv_rank != t.kv_rank ||
        s.rot_dim != t.rot_dim || s.out_gate != t.out_gate || s.sink != t.sink || s.width != t.width || s.mlp != t.mlp ||
        s.post_norm != t.post_norm || s.resid_gate != t.resid_gate || s.norm_scalar != t.norm_scalar ||
        s.kv_heads != t.kv_heads || s.attn_bias != t.attn_bias || s.qk_norm != t.qk_norm || s.head_temp != t.head_temp ||
        s.v_mix != t.v_mix || s.mlp_scale != t.mlp_scale || s.act != t.act || s.beside != t.beside || s.lin.heads != t.lin.heads ||
        s.lin.groups != t.lin.groups || s.lin.dim != t.lin.dim || s.lin.vdim != t.lin.vdim || s.lin.conv != t.lin.conv ||
        s.lin.rank != t.lin.rank || s.mixer_scale != t.mixer_scale || s.mlp_bias != t.mlp_bias ||
        (s.mlp != MLP_NONE && (s.ff != t.ff || s.experts != t.experts || s.shared_ff != t.shared_ff || s.correction != t.correction)))
      throw std::runtime_error(at + "sizes differ from the layer whose weights it uses");
    if (s.mlp != MLP_NONE && s.ff < 1) throw std::runtime_error(at + "bad sizes");
    if (s.mlp != MLP_ACT && (s.act == ACT_RELU2 || s.act == ACT_XIELU || s.mlp_scale != 1.f) && s.mlp != MLP_NONE)
      throw std::runtime_error(at + "an activation without a gate, or a scale, in an MLP with one");
    if (s.mlp == MLP_MOE && (s.experts < 1 || s.experts > MOE_MAX_EXPERTS || s.top < 1 || s.top > std::min(s.experts, MOE_MAX_TOP) ||
                             s.shared_ff < 0))
      throw std::runtime_error(at + "bad number of experts");
    if (s.parallel && (s.mixer != MIX_LATENT || s.beside || s.mlp == MLP_MOE || s.mlp == MLP_ACT || s.post_norm || s.resid_gate))
      throw std::runtime_error(at + "a parallel layer is latent attention beside a dense MLP");
    Dims& D = dims_[i];
    std::memset(&D, 0, sizeof(D));
    int n;  // columns of the mixer's input product
    if (s.mixer == MIX_LATENT) {
      if (s.heads < 1 || s.dim < 1 || s.vdim < 1 || s.kv_rank < 1 || s.window < 0) throw std::runtime_error(at + "bad sizes");
      if (s.rot_dim < 0 || s.rot_dim % 2 || s.rot_dims < 0 || s.rot_dims % 2 || s.rot_dims > s.rot_dim)
        throw std::runtime_error(at + "bad rotated dimensions");
      D.H = s.heads;
      D.dk = s.dim;
      D.dv = s.vdim;
      D.rank = s.kv_rank;
      D.rot = s.rot_dim;
      D.qrot = up(D.dk, 8);
      D.roff = up(D.rank, 8);
      D.dkp = up(D.rot ? D.qrot + D.rot : D.dk, 32);
      D.dvp = up(D.dv, 32);
      D.rp = pad_rank(D.rot ? D.roff + D.rot : D.rank);
      D.qn = up(D.H * D.dkp, 64);
      D.gn = up(D.H * D.dvp, 64);
      D.gate_off = D.qn + D.rp;
      n = D.gate_off + (s.out_gate == GATE_ELEMENT ? D.gn : s.out_gate == GATE_HEAD ? up(D.H, 64) : 0);
      if (s.window) max_window_ = std::max(max_window_, s.window);
      else all_windowed = false;
    } else if (s.mixer == MIX_MINGRU) {
      if (s.width < 1) throw std::runtime_error(at + "bad sizes");
      D.wp = up(s.width, 64);
      D.gn = D.wp;
      n = 3 * D.wp;
      recurrent_ = true;
    } else if (s.mixer == MIX_GQA) {
      if (s.heads < 1 || s.kv_heads < 1 || s.heads % s.kv_heads || s.dim < 1 || s.vdim < 1 || s.window < 0 || s.chunk < 0 ||
          s.rot_dims < 0 || s.rot_dims % 2 || s.rot_dims > s.dim || s.out_gate == GATE_ELEMENT)
        throw std::runtime_error(at + "bad sizes");
      if (s.v_mix) {
        if (v_first_layer_ < 0) v_first_layer_ = i;
        const LayerSpec& f = c.layers[v_first_layer_];
        if (s.kv_heads != f.kv_heads || s.vdim != f.vdim)
          throw std::runtime_error(at + "values to mix differ in size from those of layer " + std::to_string(v_first_layer_));
        if (c.loop_times > 0) throw std::runtime_error(at + "mixed values in a looped model");
      }
      D.H = s.heads;
      D.G = s.kv_heads;
      D.dk = s.dim;
      D.dv = s.vdim;
      D.rot = s.rot_dims;
      D.dkp = up(D.dk, 32);
      D.dvp = up(D.dv, 32);
      if (!gqa_supports(D.dkp, D.dvp)) throw std::runtime_error(at + "attention heads above 256 dimensions");
      D.gn = up(D.H * D.dvp, 64);
      D.koff = D.H * D.dk;
      D.voff = D.koff + D.G * D.dk;
      D.gate_off = D.voff + D.G * D.dv;
      n = D.gate_off + (s.out_gate == GATE_HEAD ? D.H : 0);
      const int w = s.window && s.chunk ? std::min(s.window, s.chunk) : s.window + s.chunk;
      if (w) max_window_ = std::max(max_window_, w);
      else all_windowed = false;
    } else if (s.mixer == MIX_MAMBA2 || s.mixer == MIX_GLA || s.mixer == MIX_DELTA) {
      n = 0;
    } else {
      throw std::runtime_error("unknown mixer kind");
    }
    const int lin = s.mixer == MIX_MAMBA2 || s.mixer == MIX_GLA || s.mixer == MIX_DELTA ? s.mixer : s.beside;
    if (s.beside && s.mixer != MIX_GQA) throw std::runtime_error(at + "a second mixer stands beside grouped-query attention only");
    if (lin) {
      const LinSpec& l = s.lin;
      const bool key = lin == MIX_GLA, delta = lin == MIX_DELTA;
      if (lin != MIX_MAMBA2 && !key && !delta) throw std::runtime_error(at + "unknown second mixer");
      if (l.heads < 1 || l.dim < 1 || l.vdim < 1 || !lin_pad_n(l.dim) || l.vdim > 1024 ||
          (key ? l.rank < 1 || l.tau <= 0 : l.groups < 1 || l.heads % l.groups || l.conv < 1 || l.conv > 16) ||
          (lin == MIX_MAMBA2 && (l.norm_groups < 1 || (l.heads * l.vdim) % l.norm_groups)))
        throw std::runtime_error(at + "bad sizes of the linear recurrence");
      D.lin = key ? LIN_KEY : delta ? LIN_DELTA : LIN_HEAD;
      D.lH = l.heads;
      D.lG = key ? l.heads : l.groups;
      D.lN = l.dim;
      D.lnp = lin_pad_n(l.dim);
      D.ldv = l.vdim;
      D.lvp = up(l.vdim, 16);
      D.lin_off = n;
      D.lin_out = D.gn;
      n += key ? D.lH * (2 * D.lN + 2 * D.ldv) + l.rank : 2 * D.lH * D.ldv + 2 * D.lG * D.lN + (delta ? 2 : 1) * D.lH;
      D.gn += up(D.lH * D.ldv, 64);
      recurrent_ = true;
    }
    n = up(n, 64);
    D.ff = s.mlp != MLP_NONE ? s.ff : 0;
    D.fp = up(D.ff, 64);
    if (s.parallel) {
      D.n1 = n;
      D.nin = D.n1 + 2 * D.fp;
      D.kout = D.gn + D.fp;
      continue;
    }
    D.rg_off = n;
    D.n1 = up_n(n + (s.resid_gate ? dp_ : 0));
    D.kout = D.gn;
    D.shf = s.mlp == MLP_MOE ? s.shared_ff : 0;
    D.shp = up(D.shf, 64);
    if (s.mlp == MLP_ACT) D.fp = D.ff > 4096 ? up(D.ff, 512) : up_n(D.ff);  // (the GEMV engine's K: whole 512s)
    D.glu = s.mlp == MLP_MOE ? D.shp : D.fp;
    D.router_off = s.resid_gate ? dp_ : 0;
    D.n2 = up_n(D.router_off + (s.mlp == MLP_MOE ? up(s.experts, 64) : 0));
  }
  if (!all_windowed) max_window_ = 0;
  for (int i = 0; i < nl_; ++i) {
    const bool looped = c.loop_times > 0 && i >= c.loop_start && i < c.loop_stop;
    if (looped && i == c.loop_start)
      for (int t = 0; t < c.loop_times; ++t)
        for (int j = c.loop_start; j < c.loop_stop; ++j) runs_.push_back({j, t, nullptr, nullptr, nullptr});
    if (!looped) runs_.push_back({i, -1, nullptr, nullptr, nullptr});
  }
  if (c.loop_times > 0 && !seq_) throw std::runtime_error("layered model: a loop of parallel layers");
  embd_ = balloc((size_t)v_ * dp_);
  if (c.max_positions) posw_ = balloc((size_t)c.max_positions * dp_);
  if (c.bigram_buckets) pairw_ = balloc((size_t)(c.bigram_buckets + 1) * dp_);
  if (c.loop_times > 0 && !c.loop_add) {
    loopw_ = balloc((size_t)dp_ * 2 * dp_);
    loop_step_ = falloc((size_t)c.loop_times * dp_);
  }
  headw_ = balloc((size_t)vp_ * dp_);
  out_norm_ = falloc(dp_);
  for (int i = 0; i < nl_; ++i)
    if (owner_[i] == i) alloc_layer(i);
  e_.weight_bytes_ = 0;
  list_tensors();
  for (const auto& t : tensors_) e_.weight_bytes_ += (size_t)t.second.first * t.second.second * 2;
}

void LayeredDecoder::alloc_layer(int i) {
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  Weights& w = w_[i];
  w.own = true;
  w.norm = falloc(dp_);
  if (s.mixer == MIX_LATENT) {
    w.kv_norm = falloc(D.rp);
    w.sink = falloc(D.H);
    w.ukv = balloc((size_t)(D.qn + D.gn) * D.rp);
    w.ukT = balloc((size_t)D.H * D.rp * D.dkp);
  } else if (s.mixer == MIX_MINGRU) {
    w.zb = falloc(D.wp);
    w.ub = falloc(D.wp);
  } else if (s.mixer == MIX_GQA) {
    w.sink = falloc(D.H);
    if (s.attn_bias) {
      w.qb = falloc(D.H * D.dk);
      w.kb = falloc(D.G * D.dk);
      w.vb = falloc(D.G * D.dv);
      if (s.attn_bias == 1) w.ob = falloc(dp_);
    }
    if (s.qk_norm) {
      w.qn = falloc(D.H * D.dk);
      w.kn = falloc(D.G * D.dk);
    }
    if (s.head_temp) w.temp = falloc(D.H);
    if (s.v_mix) w.lambda = falloc(1);
  }
  if (D.lin == LIN_HEAD || D.lin == LIN_DELTA) {
    const int C = D.lH * D.ldv + 2 * D.lG * D.lN;
    w.conv_w = falloc((size_t)C * s.lin.conv);
    w.dt_b = falloc(D.lH);
    w.a_log = falloc(D.lH);
    w.lin_norm = falloc(D.lin == LIN_DELTA ? D.ldv : (size_t)D.lH * D.ldv);
    if (D.lin == LIN_HEAD) {
      w.conv_b = falloc(C);
      w.lin_d = falloc(D.lH);
    }
  } else if (D.lin == LIN_KEY) {
    w.a2 = falloc((size_t)D.lH * D.lN * s.lin.rank);
    w.a2_b = falloc((size_t)D.lH * D.lN);
    w.lin_norm = falloc(D.ldv);
  }
  if (s.parallel) {
    w.in = balloc((size_t)D.nin * dp_);
    w.out = balloc((size_t)dp_ * D.kout);
    return;
  }
  w.in = balloc((size_t)D.n1 * dp_);
  w.out = balloc((size_t)dp_ * D.kout);
  if (s.post_norm) w.post = falloc(dp_);
  if (s.resid_gate) w.rgb = falloc(dp_);
  if (s.mlp == MLP_NONE) return;
  w.norm2 = falloc(dp_);
  if (s.post_norm) w.post2 = falloc(dp_);
  if (s.resid_gate) w.rgb2 = falloc(dp_);
  w.in2 = balloc((size_t)(D.n2 + (s.mlp == MLP_ACT ? 1 : 2) * D.glu) * dp_);
  w.act_n.scale = s.mlp_scale;
  if (s.mlp == MLP_ACT && s.mlp_bias) {
    w.upb = falloc(D.fp);
    w.dnb = falloc(dp_);
  }
  if (D.glu) w.out2 = balloc((size_t)dp_ * D.glu);
  if (s.mlp == MLP_MOE) {
    w.corr = falloc(s.experts);
    w.egu = balloc((size_t)s.experts * 2 * D.fp * dp_);
    w.edn = balloc((size_t)s.experts * dp_ * D.fp);
  }
}

LayeredDecoder::~LayeredDecoder() {
  if (h_step_) hipHostFree(h_step_);
}

// zeroed device memory: the padding of every operand stays zero (16 KB of slack behind: tile loaders may
// request whole tiles)
bf16_t* LayeredDecoder::balloc(size_t n) {
  void* p = e_.dmalloc(n * 2 + 16384);
  HIP_CHECK(hipMemset(p, 0, n * 2 + 16384));
  return (bf16_t*)p;
}
float* LayeredDecoder::falloc(size_t n) {
  void* p = e_.dmalloc(n * 4 + 16384);
  HIP_CHECK(hipMemset(p, 0, n * 4 + 16384));
  return (float*)p;
}

// ---- weights ----------------------------------------------------------------------------------------
void LayeredDecoder::place(bf16_t* dst, int dpitch, const bf16_t* src, int spitch, int width, int height, bool device) {
  HIP_CHECK(hipMemcpy2D(dst, (size_t)dpitch * 2, src, (size_t)spitch * 2, (size_t)width * 2, height,
                        device ? hipMemcpyDeviceToDevice : hipMemcpyHostToDevice));
}

static std::vector<float> numbers(const bf16_t* src, int n, bool device) {
  std::vector<bf16_t> h(n);
  std::vector<float> f(n);
  if (device) HIP_CHECK(hipMemcpy(h.data(), src, (size_t)n * 2, hipMemcpyDeviceToHost));
  else std::memcpy(h.data(), src, (size_t)n * 2);
  for (int i = 0; i < n; ++i) {
    const uint32_t u = (uint32_t)h[i] << 16;
    std::memcpy(&f[i], &u, 4);
  }
  return f;
}

// src's n numbers times `mul`, or (spread > 0) its one number that many times
void LayeredDecoder::put_vec(float* dst, int n, const bf16_t* src, bool device, int spread, float mul) {
  std::vector<float> f = numbers(src, n, device);
  for (float& v : f) v *= mul;
  if (spread > 0) f.assign(spread, f[0]);
  HIP_CHECK(hipMemcpy(dst, f.data(), f.size() * 4, hipMemcpyHostToDevice));
}

// every tensor of the model: name, (rows, cols)
void LayeredDecoder::list_tensors() {
  const EngineConfig& c = e_.cfg_;
  auto add = [&](const std::string& n, int r, int cl) {
    tensors_.push_back({n, {r, cl}});
    shape_[n] = {r, cl};
  };
  const int norm_final = c.layers[0].norm_scalar ? 1 : d_;
  add("token_embd.weight", v_, d_);
  if (posw_) add("position_embd.weight", c.max_positions, d_);
  if (pairw_) add("bigram_embd.weight", c.bigram_buckets + 1, d_);
  if (loopw_) {
    add("loop_in.weight", d_, 2 * d_);
    add("loop_step.weight", c.loop_times, d_);
  }
  add("output_norm.weight", 1, norm_final);
  add("output.weight", v_, d_);
  for (int i = 0; i < nl_; ++i) {
    if (owner_[i] != i) continue;
    const Dims& D = dims_[i];
    const LayerSpec& s = c.layers[i];
    const std::string p = "blk." + std::to_string(i) + ".";
    const int nw = s.norm_scalar ? 1 : d_;
    add(p + "attn_norm.weight", 1, nw);
    if (s.mixer == MIX_LATENT) {
      add(p + "attn_q.weight", D.H * (D.dk + D.rot), d_);
      add(p + "attn_kv_a.weight", D.rank + D.rot, d_);
      add(p + "attn_kv_a_norm.weight", 1, D.rank);
      add(p + "attn_k_b.weight", D.H * D.dk, D.rank);
      add(p + "attn_v_b.weight", D.H * D.dv, D.rank);
      if (s.sink) add(p + "attn_sinks.weight", 1, D.H);
      if (s.out_gate) add(p + "attn_gate.weight", s.out_gate == GATE_HEAD ? D.H : D.H * D.dv, d_);
      add(p + "attn_output.weight", d_, D.H * D.dv);
    } else if (s.mixer == MIX_GQA) {
      const struct { const char* n; int rows, cols; } mats[] = {
          {"attn_q", D.H * D.dk, d_}, {"attn_k", D.G * D.dk, d_}, {"attn_v", D.G * D.dv, d_}, {"attn_output", d_, D.H * D.dv}};
      for (const auto& m : mats) {
        add(p + m.n + ".weight", m.rows, m.cols);
        if (s.attn_bias == 1 || (s.attn_bias && &m != &mats[3])) add(p + m.n + ".bias", 1, m.rows);
      }
      if (s.qk_norm) {
        add(p + "attn_q_norm.weight", 1, D.H * D.dk);
        add(p + "attn_k_norm.weight", 1, D.G * D.dk);
      }
      if (s.head_temp) add(p + "attn_temp.weight", 1, D.H);
      if (s.v_mix) add(p + "attn_v_mix.weight", 1, 1);
      if (s.sink == 1) add(p + "attn_sinks.weight", 1, D.H);
      if (s.out_gate) add(p + "attn_gate.weight", D.H, d_);
    } else if (s.mixer == MIX_MINGRU) {
      for (const char* n : {"z", "x"}) {
        add(p + "rnn_" + n + ".weight", s.width, d_);
        add(p + "rnn_" + n + ".bias", 1, s.width);
      }
      add(p + "rnn_gate.weight", s.width, d_);
      add(p + "rnn_output.weight", d_, s.width);
    }
    if (D.lin == LIN_HEAD) {
      const int inner = D.lH * D.ldv, C = inner + 2 * D.lG * D.lN;
      add(p + "ssm_in.weight", inner + C + D.lH, d_);
      add(p + "ssm_conv1d.weight", C, s.lin.conv);
      add(p + "ssm_conv1d.bias", 1, C);
      add(p + "ssm_dt.bias", 1, D.lH);
      add(p + "ssm_a_log.bias", 1, D.lH);
      add(p + "ssm_d.bias", 1, D.lH);
      add(p + "ssm_norm.weight", 1, inner);
      add(p + "ssm_out.weight", d_, inner);
    } else if (D.lin == LIN_DELTA) {
      const int nk = D.lG * D.lN, nv = D.lH * D.ldv;
      for (const char* n : {"q", "k", "v"}) {
        add(p + "delta_" + n + ".weight", *n == 'v' ? nv : nk, d_);
        add(p + "delta_" + n + "_conv1d.weight", *n == 'v' ? nv : nk, s.lin.conv);
      }
      add(p + "delta_b.weight", D.lH, d_);
      add(p + "delta_a.weight", D.lH, d_);
      add(p + "delta_dt.bias", 1, D.lH);
      add(p + "delta_a_log.bias", 1, D.lH);
      add(p + "delta_gate.weight", nv, d_);
      add(p + "delta_norm.weight", 1, D.ldv);
      add(p + "delta_output.weight", d_, nv);
    } else if (D.lin == LIN_KEY) {
      const int nk = D.lH * D.lN, nv = D.lH * D.ldv;
      add(p + "gla_q.weight", nk, d_);
      add(p + "gla_k.weight", nk, d_);
      add(p + "gla_v.weight", nv, d_);
      add(p + "gla_gate.weight", nv, d_);
      add(p + "gla_a1.weight", s.lin.rank, d_);
      add(p + "gla_a2.weight", nk, s.lin.rank);
      add(p + "gla_a2.bias", 1, nk);
      add(p + "gla_norm.weight", 1, D.ldv);
      add(p + "gla_output.weight", d_, nv);
    }
    auto closing = [&](const std::string& sub) {
      if (s.post_norm) add(p + sub + "_post_norm.weight", 1, nw);
      if (s.resid_gate) {
        add(p + sub + "_resid_gate.weight", d_, d_);
        add(p + sub + "_resid_gate.bias", 1, d_);
      }
    };
    if (!s.parallel) closing("attn");
    if (s.mlp == MLP_NONE) continue;
    if (!s.parallel) {
      add(p + "ffn_norm.weight", 1, nw);
      closing("ffn");
    }
    if (s.mlp == MLP_GLU) {
      add(p + "ffn_gate.weight", D.ff, d_);
      add(p + "ffn_up.weight", D.ff, d_);
      add(p + "ffn_down.weight", d_, D.ff);
      continue;
    }
    if (s.mlp == MLP_ACT) {
      add(p + "ffn_up.weight", D.ff, d_);
      add(p + "ffn_down.weight", d_, D.ff);
      if (s.mlp_bias) {
        add(p + "ffn_up.bias", 1, D.ff);
        add(p + "ffn_down.bias", 1, d_);
      }
      if (s.act == ACT_XIELU) add(p + "ffn_act.bias", 1, 2);
      continue;
    }
    add(p + "ffn_gate_inp.weight", s.experts, d_);
    if (s.correction) add(p + "exp_probs_b.bias", 1, s.experts);
    if (s.shared_ff) {
      add(p + "ffn_gate_shexp.weight", D.shf, d_);
      add(p + "ffn_up_shexp.weight", D.shf, d_);
      add(p + "ffn_down_shexp.weight", d_, D.shf);
    }
    for (int x = 0; x < s.experts; ++x) {
      const std::string n = "." + std::to_string(x) + ".weight";
      add(p + "ffn_gate" + n, D.ff, d_);
      add(p + "ffn_up" + n, D.ff, d_);
      add(p + "ffn_down" + n, d_, D.ff);
    }
  }
}

void LayeredDecoder::put(const std::string& name, int rows, int cols, const bf16_t* src, bool device) {
  const EngineConfig& c = e_.cfg_;
  if (name == "token_embd.weight") return place(embd_, dp_, src, cols, cols, rows, device);
  if (name == "position_embd.weight") return place(posw_, dp_, src, cols, cols, rows, device);
  if (name == "bigram_embd.weight") return place(pairw_, dp_, src, cols, cols, rows, device);
  if (name == "output.weight") return place(headw_, dp_, src, cols, cols, rows, device);
  // (the logits' scale goes with the norm before the head)
  if (name == "output_norm.weight") return put_vec(out_norm_, cols, src, device, cols < d_ ? d_ : 0, c.logit_scale);
  if (name == "loop_in.weight") {
    place(loopw_, 2 * dp_, src, cols, d_, rows, device);
    return place(loopw_ + dp_, 2 * dp_, src + d_, cols, d_, rows, device);
  }
  if (name == "loop_step.weight") {
    for (int t = 0; t < rows; ++t) put_vec(loop_step_ + (size_t)t * dp_, cols, src + (size_t)t * cols, device);
    return;
  }
  const size_t dot = name.find('.', 4);
  const int i = std::stoi(name.substr(4, dot - 4));
  const std::string t = name.substr(dot + 1);
  const Dims& D = dims_[i];
  const LayerSpec& s = c.layers[i];
  Weights& w = w_[i];
  // heads of per_head rows each, `take` of them from row `from` spread to pad rows each
  auto heads = [&](bf16_t* dst, int dpitch, int per_head, int pad, int from = 0, int take = -1) {
    for (int h = 0; h < D.H; ++h)
      place(dst + (size_t)h * pad * dpitch, dpitch, src + ((size_t)h * per_head + from) * cols, cols, cols,
            take < 0 ? per_head : take, device);
  };
  auto rows_at = [&](bf16_t* m, int row) { place(m + (size_t)row * dp_, dp_, src, cols, cols, rows, device); };
  auto norm = [&](float* dst) { put_vec(dst, cols, src, device, cols < d_ ? d_ : 0); };
  auto glu = [&](bf16_t* m, int row0, int up_row) {  // gate and up rows interleaved from row0
    place(m + (size_t)(row0 + up_row) * dp_, 2 * dp_, src, cols, cols, rows, device);
  };
  bf16_t* gu = s.parallel ? w.in : w.in2;
  const int gu0 = s.parallel ? D.n1 : D.n2;
  if (t == "attn_norm.weight") norm(w.norm);
  else if (t == "ffn_norm.weight") norm(w.norm2);
  else if (t == "attn_post_norm.weight") norm(w.post);
  else if (t == "ffn_post_norm.weight") norm(w.post2);
  else if (t == "attn_kv_a_norm.weight") put_vec(w.kv_norm, cols, src, device);
  else if (t == "attn_sinks.weight") put_vec(w.sink, cols, src, device);
  else if (s.mixer == MIX_GQA && t == "attn_q.weight") rows_at(w.in, 0);
  else if (s.mixer == MIX_GQA && t == "attn_k.weight") rows_at(w.in, D.koff);
  else if (s.mixer == MIX_GQA && t == "attn_v.weight") rows_at(w.in, D.voff);
  else if (t == "attn_q.bias") put_vec(w.qb, cols, src, device);
  else if (t == "attn_k.bias") put_vec(w.kb, cols, src, device);
  else if (t == "attn_v.bias") put_vec(w.vb, cols, src, device);
  else if (t == "attn_output.bias") put_vec(w.ob, cols, src, device, 0, s.mixer_scale);
  else if (t == "attn_q_norm.weight") put_vec(w.qn, cols, src, device);
  else if (t == "attn_k_norm.weight") put_vec(w.kn, cols, src, device);
  else if (t == "attn_temp.weight") put_vec(w.temp, cols, src, device);
  else if (t == "attn_v_mix.weight") put_vec(w.lambda, cols, src, device);
  else if (t == "delta_v.weight") rows_at(w.in, D.lin_off);  // [v | k | q | gate | strengths | steps], convolved: [v | k | q]
  else if (t == "delta_k.weight") rows_at(w.in, D.lin_off + D.lH * D.ldv);
  else if (t == "delta_q.weight") rows_at(w.in, D.lin_off + D.lH * D.ldv + D.lG * D.lN);
  else if (t == "delta_gate.weight") rows_at(w.in, D.lin_off + D.lH * D.ldv + 2 * D.lG * D.lN);
  else if (t == "delta_b.weight") rows_at(w.in, D.lin_off + 2 * (D.lH * D.ldv + D.lG * D.lN));
  else if (t == "delta_a.weight") rows_at(w.in, D.lin_off + 2 * (D.lH * D.ldv + D.lG * D.lN) + D.lH);
  else if (t == "delta_v_conv1d.weight") put_vec(w.conv_w, rows * cols, src, device);
  else if (t == "delta_k_conv1d.weight") put_vec(w.conv_w + (size_t)D.lH * D.ldv * cols, rows * cols, src, device);
  else if (t == "delta_q_conv1d.weight") put_vec(w.conv_w + (size_t)(D.lH * D.ldv + D.lG * D.lN) * cols, rows * cols, src, device);
  else if (t == "delta_dt.bias") put_vec(w.dt_b, cols, src, device);
  else if (t == "delta_a_log.bias") put_vec(w.a_log, cols, src, device);
  else if (t == "delta_norm.weight") put_vec(w.lin_norm, cols, src, device);
  else if (t == "delta_output.weight") place(w.out + D.lin_out, D.kout, src, cols, cols, rows, device);
  else if (t == "ffn_act.bias") {  // (its two numbers go into softplus)
    const std::vector<float> f = numbers(src, 2, device);
    auto softplus = [](double z) { return std::max(z, 0.0) + std::log1p(std::exp(-std::fabs(z))); };
    w.act_n.pos = (float)softplus(f[0]);
    w.act_n.neg = (float)(0.5 + softplus(f[1]));
  } else if (t == "ssm_in.weight" || t == "gla_q.weight") rows_at(w.in, D.lin_off);
  else if (t == "gla_k.weight") rows_at(w.in, D.lin_off + D.lH * D.lN);
  else if (t == "gla_v.weight") rows_at(w.in, D.lin_off + 2 * D.lH * D.lN);
  else if (t == "gla_gate.weight") rows_at(w.in, D.lin_off + 2 * D.lH * D.lN + D.lH * D.ldv);
  else if (t == "gla_a1.weight") rows_at(w.in, D.lin_off + 2 * D.lH * (D.lN + D.ldv));
  else if (t == "gla_a2.weight") put_vec(w.a2, rows * cols, src, device);
  else if (t == "gla_a2.bias") put_vec(w.a2_b, cols, src, device);
  else if (t == "ssm_conv1d.weight") put_vec(w.conv_w, rows * cols, src, device);
  else if (t == "ssm_conv1d.bias") put_vec(w.conv_b, cols, src, device);
  else if (t == "ssm_dt.bias") put_vec(w.dt_b, cols, src, device);
  else if (t == "ssm_a_log.bias") put_vec(w.a_log, cols, src, device);
  else if (t == "ssm_d.bias") put_vec(w.lin_d, cols, src, device);
  else if (t == "ssm_norm.weight" || t == "gla_norm.weight") put_vec(w.lin_norm, cols, src, device);
  else if (t == "ssm_out.weight" || t == "gla_output.weight") place(w.out + D.lin_out, D.kout, src, cols, cols, rows, device);
  else if (s.mlp == MLP_ACT && t == "ffn_up.weight") rows_at(w.in2, D.n2);
  else if (t == "ffn_up.bias") put_vec(w.upb, cols, src, device);
  else if (t == "ffn_down.bias") put_vec(w.dnb, cols, src, device, 0, s.mlp_scale);
  else if (t == "attn_q.weight") {
    heads(w.in, dp_, D.dk + D.rot, D.dkp, 0, D.dk);
    if (D.rot) heads(w.in + (size_t)D.qrot * dp_, dp_, D.dk + D.rot, D.dkp, D.dk, D.rot);
  } else if (t == "attn_kv_a.weight") {
    place(w.in + (size_t)D.qn * dp_, dp_, src, cols, cols, D.rank, device);
    if (D.rot) place(w.in + (size_t)(D.qn + D.roff) * dp_, dp_, src + (size_t)D.rank * cols, cols, cols, D.rot, device);
  } else if (t == "attn_gate.weight") {
    if (s.out_gate == GATE_HEAD) rows_at(w.in, D.gate_off);
    else heads(w.in + (size_t)D.gate_off * dp_, dp_, D.dv, D.dvp);
  } else if (t == "rnn_z.weight") rows_at(w.in, 0);
  else if (t == "rnn_x.weight") rows_at(w.in, D.wp);
  else if (t == "rnn_gate.weight") rows_at(w.in, 2 * D.wp);
  else if (t == "rnn_z.bias") put_vec(w.zb, cols, src, device);
  else if (t == "rnn_x.bias") put_vec(w.ub, cols, src, device);
  else if (t == "rnn_output.weight") place(w.out, D.kout, src, cols, cols, rows, device);
  else if (t == "attn_resid_gate.weight") rows_at(w.in, D.rg_off);
  else if (t == "ffn_resid_gate.weight") rows_at(w.in2, 0);
  else if (t == "attn_resid_gate.bias") put_vec(w.rgb, cols, src, device);
  else if (t == "ffn_resid_gate.bias") put_vec(w.rgb2, cols, src, device);
  else if (t == "ffn_gate_inp.weight") rows_at(w.in2, D.router_off);
  else if (t == "exp_probs_b.bias") put_vec(w.corr, cols, src, device);
  else if (t == "ffn_gate.weight" || t == "ffn_gate_shexp.weight") glu(gu, gu0, 0);
  else if (t == "ffn_up.weight" || t == "ffn_up_shexp.weight") glu(gu, gu0, 1);
  else if (t == "attn_k_b.weight") heads(w.ukv, D.rp, D.dk, D.dkp);
  else if (t == "attn_v_b.weight") heads(w.ukv + (size_t)D.qn * D.rp, D.rp, D.dv, D.dvp);
  else if (t == "attn_output.weight")
    for (int h = 0; h < D.H; ++h) place(w.out + (size_t)h * D.dvp, D.kout, src + (size_t)h * D.dv, cols, D.dv, rows, device);
  else if (t == "ffn_down.weight" && s.parallel) place(w.out + D.gn, D.kout, src, cols, cols, rows, device);
  else if (t == "ffn_down.weight" || t == "ffn_down_shexp.weight") place(w.out2, D.glu, src, cols, cols, rows, device);
  else if (t.compare(0, 4, "ffn_") == 0 && s.mlp == MLP_MOE) {  // ffn_{gate,up,down}.<expert>.weight
    const size_t d1 = t.find('.');
    const int x = std::stoi(t.substr(d1 + 1));
    const std::string kind = t.substr(0, d1);
    if (kind == "ffn_down") place(w.edn + (size_t)x * dp_ * D.fp, D.fp, src, cols, cols, rows, device);
    else glu(w.egu + (size_t)x * 2 * D.fp * dp_, 0, kind == "ffn_up");
  } else throw std::runtime_error("unknown layer tensor " + name);
}

void LayeredDecoder::set_tensor(const std::string& name, int qt, int rows, int cols, const void* host, size_t nbytes) {
  if (qt != QT_BF16) throw std::runtime_error(name + ": layered models load bf16 tensors");
  if (nbytes != (size_t)rows * cols * 2) throw std::runtime_error(name + ": byte size mismatch");
  const auto t = shape_.find(name);
  if (t == shape_.end()) throw std::runtime_error("unknown tensor " + name);
  if (t->second.first != rows || t->second.second != cols)
    throw std::runtime_error(name + ": shape " + std::to_string(rows) + " x " + std::to_string(cols) + ", expected " +
                             std::to_string(t->second.first) + " x " + std::to_string(t->second.second));
  put(name, rows, cols, (const bf16_t*)host, false);
  have_.insert(name);
}

void LayeredDecoder::init_random(uint64_t seed) {
  uint64_t s = seed * 1000003ULL;
  for (const auto& t : tensors_) {
    const int rows = t.second.first, cols = t.second.second;
    const size_t n = (size_t)rows * cols;
    const bool norm = t.first.find("norm") != std::string::npos || t.first.find("attn_temp") != std::string::npos;
    const bool sink = t.first.find("sinks") != std::string::npos;
    const bool bias = t.first.find(".bias") != std::string::npos;
    bf16_t* tmp = nullptr;
    if (norm || sink || bias) {
      float* f = nullptr;
      HIP_CHECK(hipMalloc(&f, n * 4));
      HIP_CHECK(hipMalloc(&tmp, n * 2 + 16));
      fill_random_f32(f, n, ++s, norm ? 1.f : 0.f, norm ? 0.1f : bias ? 0.05f : 1.f, e_.stream_);
      launch_f32_to_bf16(f, tmp, n, e_.stream_);
      HIP_CHECK(hipStreamSynchronize(e_.stream_));
      HIP_CHECK(hipFree(f));
    } else {
      HIP_CHECK(hipMalloc(&tmp, n * 2));
      fill_random_weight(mat(tmp, rows, cols), ++s, t.first == "token_embd.weight" || t.first == "bigram_embd.weight" ? 1.f : 0.02f, e_.stream_);
      HIP_CHECK(hipStreamSynchronize(e_.stream_));
    }
    put(t.first, rows, cols, tmp, true);
    HIP_CHECK(hipDeviceSynchronize());
    HIP_CHECK(hipFree(tmp));
    have_.insert(t.first);
  }
}

std::vector<std::string> LayeredDecoder::missing() const {
  std::vector<std::string> m;
  for (const auto& t : tensors_)
    if (!have_.count(t.first)) m.push_back(t.first);
  return m;
}

QWeight LayeredDecoder::mat(const bf16_t* p, int rows, int cols) const {
  QWeight w{};
  w.qtype = QT_BF16;
  w.rows = rows;
  w.cols = cols;
  w.p0 = (const uint8_t*)p;
  return w;
}

// ---- workspace ----------------------------------------------------------------------------------------
// (cos, sin) of every position and pair; pairs past `dims` do not turn
std::vector<float> LayeredDecoder::rope_table(int rot, int dims, double base) const {
  const int half = rot / 2, n = e_.cfg_.max_ctx;
  std::vector<float> t((size_t)n * half * 2);
  for (int i = 0; i < half; ++i) {
    const double f = 2 * i < dims ? std::pow(base, -2.0 * i / dims) : 0.0;
    for (int p = 0; p < n; ++p) {
      t[((size_t)p * half + i) * 2] = (float)std::cos(p * f);
      t[((size_t)p * half + i) * 2 + 1] = (float)std::sin(p * f);
    }
  }
  return t;
}

void LayeredDecoder::finalize() {
  const EngineConfig& c = e_.cfg_;
  const int Bm = c.max_batch;
  hipStream_t st = e_.stream_;
  std::map<std::pair<std::pair<int, int>, double>, float2*> ropes;
  for (int i = 0; i < nl_; ++i) {
    const Dims& D = dims_[i];
    const LayerSpec& s = c.layers[i];
    if (!D.H) continue;
    if (D.rot) {
      float2*& t = ropes[{{D.rot, s.rot_dims}, s.rot_base}];
      if (!t) {
        const std::vector<float> h = rope_table(D.rot, s.rot_dims, s.rot_base);
        t = (float2*)e_.dmalloc(h.size() * 4);
        HIP_CHECK(hipMemcpy(t, h.data(), h.size() * 4, hipMemcpyHostToDevice));
      }
      rope_[i] = t;
    }
    if (!w_[i].own || s.mixer != MIX_LATENT) continue;
    if (D.rot) {  // the rotated part of the cached row is a head's rotated key as it is
      std::vector<bf16_t> one((size_t)D.rot * D.rot, 0);
      for (int k = 0; k < D.rot; ++k) one[(size_t)k * D.rot + k] = 0x3f80;
      for (int h = 0; h < D.H; ++h)
        place(w_[i].ukv + ((size_t)h * D.dkp + D.qrot) * D.rp + D.roff, D.rp, one.data(), D.rot, D.rot, D.rot, false);
    }
    launch_transpose_heads(w_[i].ukv, D.H, D.dkp, D.rp, w_[i].ukT, st);
  }
  // a cache pool or a state per run (weights may be shared, what they leave behind is not)
  const int es = f32_ ? 4 : 2;
  e_.kv_bytes_ = 0;
  for (Run& k : runs_) {
    const Dims& D = dims_[k.layer];
    if (const size_t n = state_floats(k.layer)) {
      k.state = falloc((size_t)2 * c.max_slots * n);
      e_.kv_bytes_ += (size_t)2 * c.max_slots * n * 4;
    }
    if (const size_t n = ring_floats(k.layer)) {
      k.ring = falloc((size_t)c.max_slots * n);
      e_.kv_bytes_ += (size_t)c.max_slots * n * 4;
    }
    if (!D.H) continue;
    if (D.G && e_.kvb_ != GQA_BLOCK) throw std::runtime_error("grouped-query attention: cache block size");
    const size_t block = (D.G ? gqa_block_elems(D.G, D.dkp, D.dvp) : (size_t)e_.kvb_ * D.rp) * es, bytes = (size_t)(e_.kv_nblocks_ + 1) * block;
    k.pool = (char*)e_.dmalloc(bytes);
    HIP_CHECK(hipMemset(k.pool, 0, bytes));
    e_.pools_.push_back({k.pool, block});
    e_.kv_bytes_ += bytes;
  }
  int heads = 0;
  for (const LayerSpec& s : c.layers)
    if (s.sink == 2) heads = std::max(heads, s.heads);
  if (heads) zero_sink_ = falloc(heads);
  if (pairw_) last_tok_ = (int*)falloc((size_t)2 * c.max_slots);
  step_rows_ = std::max(Bm, std::min(2048, c.max_slots * c.max_ctx));
  if (const char* v = std::getenv("AIOS_STEP_ROWS")) step_rows_ = std::max(Bm, std::atoi(v));
  const int R = step_rows_;
  int n1 = 0, nin = 0, kout = 0, fp = 0, wp = 0;
  size_t qa = 0, part = 0, kvw = 0, flat = 0;
  size_t e_act = 0, e_gu = 0, pairs = 0;  // experts
  LinWs lw = {0, 0, 0, 0, 0, 0};
  size_t lin_y = 0, lin_seg = 0, lin_seg_dec = 0;
  int rp = 0;
  for (int i = 0; i < nl_; ++i) {
    const Dims& D = dims_[i];
    const LayerSpec& s = c.layers[i];
    n1 = std::max({n1, D.n1, D.n2});
    nin = std::max({nin, D.nin, D.n1, D.n2 + 2 * D.glu});
    if (D.lin) {
      const LinWs l = lin_ws(D.lin, D.lH, D.lG, D.lnp, D.lvp, f32_);
      lw = LinWs{std::max(lw.qo, l.qo), std::max(lw.ko, l.ko), std::max(lw.kr, l.kr),
                 std::max(lw.vo, l.vo), std::max(lw.so, l.so), std::max(lw.dec, l.dec)};
      lin_y = std::max(lin_y, (size_t)R * D.lH * D.ldv);
      lin_seg = std::max(lin_seg, (size_t)LIN_SEGS * D.lH * D.lnp * D.lvp);
      lin_seg_dec = std::max(lin_seg_dec, (size_t)LIN_SEGS * D.lH * D.lnp);
    }
    kout = std::max({kout, D.kout, D.glu});
    fp = std::max(fp, seq_ ? D.glu : D.fp);
    wp = std::max(wp, D.wp);
    if (s.mlp == MLP_MOE) {
      const size_t P = (size_t)R * s.top;
      pairs = std::max(pairs, P);
      e_act = std::max(e_act, P * D.fp);
      e_gu = std::max(e_gu, P * 2 * D.fp);
      moe_max_tiles_ = std::max(moe_max_tiles_, s.experts + (int)(P / 32));
    }
    if (D.G) {
      qa = std::max(qa, (size_t)R * D.H * D.dkp);
      const size_t fl = std::max((size_t)R * D.H, (size_t)16 * 1024);  // (key_split: rows x splits)
      flat = std::max(flat, fl);
      part = std::max(part, fl * D.dvp);
    }
    if (s.mixer != MIX_LATENT) continue;
    rp = std::max(rp, D.rp);
    qa = std::max(qa, (size_t)R * D.H * D.rp);
    const size_t fl = std::max((size_t)R * D.H, (size_t)16 * 1024);  // (key_split: rows x splits)
    flat = std::max(flat, fl);
    part = std::max(part, fl * D.rp);
    kvw = std::max(kvw, (size_t)D.qn + D.gn);
  }
  if (v_first_layer_ >= 0) {
    const size_t n = (size_t)R * dims_[v_first_layer_].G * dims_[v_first_layer_].dv;
    v_first_ = falloc(n);
    e_.ws_bytes_ += n * 4;
  }
  x_ = falloc((size_t)R * dp_);
  xh_ = falloc((size_t)R * dp_);
  qdg_ = falloc((size_t)R * n1);
  opart_ = falloc(part);
  ml_ = falloc(flat * 2);
  e_.ws_bytes_ = ((size_t)R * (2 * dp_ + n1) + part + 2 * flat) * 4;
  pf_max_ctx_ = std::min(c.max_ctx, max_window_ ? std::min(32768, R + max_window_) : 32768);
  auto operand = [&](size_t n) {  // a product's operand: bf16, or fp32 in the 32-bit engine
    e_.ws_bytes_ += n * es;
    return f32_ ? (void*)falloc(n) : (void*)balloc(n);
  };
  max_chunks_ = R / SCAN_CHUNK + c.max_slots + 1;
  if (seq_) {
    y_ = falloc((size_t)R * dp_);
    e_.ws_bytes_ += (size_t)R * dp_ * 4;
    if (loopw_) xin_ = operand((size_t)R * 2 * dp_);
    if (c.loop_times > 1 && c.loop_add) {
      x0_ = falloc((size_t)R * dp_);
      e_.ws_bytes_ += (size_t)R * dp_ * 4;
    }
    if (lin_y) {
      const size_t nb = (size_t)2 * max_chunks_;  // (a chunk is two blocks)
      lin_qo_ = operand(nb * lw.qo);
      lin_ko_ = operand(nb * lw.ko);
      lin_kr_ = operand(nb * lw.kr);
      lin_vo_ = operand(nb * lw.vo);
      lin_so_ = operand(nb * lw.so);
      lin_dec_ = falloc(nb * lw.dec);
      lin_y_ = falloc(lin_y);
      lin_seg_ = falloc(lin_seg);
      lin_seg_dec_ = falloc(lin_seg_dec);
      e_.ws_bytes_ += (nb * lw.dec + lin_y + lin_seg + lin_seg_dec) * 4;
    }
    if (wp) {
      agg_ = falloc((size_t)max_chunks_ * 3 * wp);
      e_.ws_bytes_ += (size_t)max_chunks_ * 3 * wp * 4;
    }
    if (pairs) {
      moe_sel_ = (int*)falloc(pairs);
      moe_pair_ = (int*)falloc(pairs);
      moe_token_ = (int*)falloc(pairs);
      moe_wt_ = falloc(pairs);
      moe_tiles_ = (int4*)falloc((size_t)4 * moe_max_tiles_);
      moe_ntiles_ = (int*)falloc(1);
      moe_act_ = operand(e_act);
      moe_ye_ = operand(pairs * dp_);
      e_.ws_bytes_ += pairs * 16;
      if (f32_) {
        moe_gu32_ = falloc(e_gu);
        e_.ws_bytes_ += e_gu * 4;
      }
    }
  }
  if (f32_) {
    h32_ = falloc((size_t)R * dp_);
    gu32_ = falloc((size_t)R * 2 * std::max(fp, 1));
    cat32_ = falloc((size_t)R * kout);
    qa_ = falloc(qa);
    e_.ws_bytes_ += ((size_t)R * (dp_ + 2 * fp + kout) + qa) * 4;
    pf_min_ = 1 << 30;
  } else {
    h16_ = balloc((size_t)R * dp_);
    cat16_ = balloc((size_t)R * kout);
    qa_ = balloc(qa);
    cfull_ = balloc((size_t)up(pf_max_ctx_, 64) * rp);
    kv_ = balloc((size_t)up(pf_max_ctx_, 64) * kvw);
    e_.ws_bytes_ += ((size_t)R * (dp_ + kout) + qa + (size_t)pf_max_ctx_ * (rp + kvw)) * 2;
    // expanded attention from the portion length where its operations (key and value projections of the
    // whole context + dim + vdim per pair) drop below the absorbed form's (2 x rank per pair)
    pf_min_ = rp ? 0 : 1 << 30;
    for (const Dims& D : dims_) {
      if (!D.H || D.G) continue;
      const double s = D.dkp + D.dvp, gain = 2.0 * D.rp - s;
      const int t = gain > 0 ? (int)std::min(256.0, std::max(64.0, D.rp * s / gain)) : 256;
      pf_min_ = std::max(pf_min_, t);
    }
    if (const char* v = std::getenv("AIOS_LATENT_PF_MIN"))
      if (rp) pf_min_ = std::max(1, std::atoi(v));
    // grouped-query attention: the flash kernel's 128-row blocks from half a block on
    for (const Dims& D : dims_)
      if (D.G) pf_min_ = rp ? std::max(pf_min_, 64) : env_or("AIOS_GQA_PF_MIN", 64);
    if (!rp) pf_max_ctx_ = 1 << 30;  // (no context is expanded)
    for (const Dims& D : dims_)
      if (D.H && !mha_prefill_supports(D.dkp, D.dvp)) pf_min_ = 1 << 30;
    // the skinny GEMM's split-K workspace (shared with the engine's other users of gemm())
    const int maxN = std::max({nin, dp_, vp_, (int)kvw});
    e_.gk_ws_bytes_ = gemm_skinny_ws_bytes(64, maxN);
    e_.gk_ws_ = falloc(e_.gk_ws_bytes_ / 4 + 1);
    e_.gk_cnt_len_ = gemm_skinny_cnt_len(maxN);
    e_.gk_cnt_ = (int*)falloc(e_.gk_cnt_len_);
    plain_ = seq_ && !loopw_ && dp_ == d_;
    for (const LayerSpec& l : c.layers)
      if (l.parallel || l.post_norm || l.resid_gate || (l.mlp != MLP_ACT && l.mlp != MLP_NONE)) plain_ = false;
    if ((!seq_ || plain_) && dp_ == d_ && d_ % 128 == 0 && env_or("AIOS_GEMM_NORM_FUSE", 1)) {
      GemmQArgs p;
      std::memset(&p, 0, sizeof(p));
      p.M = 64; p.N = dp_; p.K = dims_[0].kout; p.nseg = 1; p.seg[0] = mat(w_[owner_[0]].out, dp_, dims_[0].kout);
      const int parts = gemm_skinny_ntile(p);
      if (parts > 0 && parts % 4 == 0 && parts <= 64) {
        nparts_ = parts;
        xn16_ = balloc((size_t)64 * dp_);
        npart_ = falloc((size_t)64 * parts);
      }
    }
  }
  // step parameters
  std::set<int> hs;  // rows of a token that read the same keys
  for (const Dims& D : dims_)
    if (D.H) hs.insert(D.G ? D.H / D.G : D.H);
  size_t tiles = 0;
  for (int h : hs) tiles += (size_t)R * ((h + 15) / 16) + R;
  const size_t chunk_ints = (size_t)max_chunks_ * (sizeof(ScanChunk) / 4);
  const size_t seq_ints = (size_t)std::min(R, max_chunks_) * (sizeof(ScanSeq) / 4);
  step_ints_ = (size_t)5 * R + chunk_ints + seq_ints + 1 + 2 * tiles;
  HIP_CHECK(hipHostMalloc((void**)&h_step_, step_ints_ * 4, hipHostMallocDefault));
  d_step_ = (int*)falloc(step_ints_);
  st_tokens_ = d_step_;
  st_pos_ = st_tokens_ + R;
  st_slot_ = st_pos_ + R;
  st_want_ = st_slot_ + R;
  st_run_ = st_want_ + R;
  st_chunks_ = (ScanChunk*)(st_run_ + R);
  st_seqs_ = (ScanSeq*)(st_run_ + R + chunk_ints);
  st_tiles_ = (LatentTile*)(st_run_ + R + chunk_ints + seq_ints);
  gemv_ok_.assign(5, 0);
  for (int b = 1; b <= 4 && !f32_; ++b) {
    bool ok = (!seq_ || plain_) && dp_ == d_ && env_or("AIOS_LAYERED_GEMV", 1);
    for (int i = 0; i < nl_ && ok; ++i) ok = gemv_fits(i, b);
    gemv_ok_[b] = ok;
  }
  HIP_CHECK(hipStreamSynchronize(st));
  if (!f32_) tune();
}

bool LayeredDecoder::gemv_fits(int i, int B) {
  const Dims& D = dims_[i];
  const Weights& w = w_[owner_[i]];
  auto fits = [&](const bf16_t* m, int N, int K, const float* norm) {
    GemvArgs a = e_.gemv_args({}, N, K, B, x_, K, norm, qdg_, N, EPI_STORE, 0);
    a.nseg = 1;
    a.seg[0] = mat(m, N, K);
    return gemv_bf16_engine_fits(a);
  };
  return fits(w.in, seq_ ? D.n1 : D.nin, dp_, w.norm) && fits(w.out, dp_, D.kout, nullptr) &&
         (!seq_ || !D.glu || (fits(w.in2, D.glu, dp_, w.norm2) && fits(w.out2, dp_, D.glu, nullptr)));
}

// measured prefill-GEMM plans for the layers' shapes (as Engine::tune_prefill_gemm)
void LayeredDecoder::tune() {
  if (!env_or("AIOS_GEMM_PF_TUNE", 1) || nl_ == 0) return;
  float* tmp = nullptr;
  HIP_CHECK(hipMalloc(&tmp, (size_t)step_rows_ * dp_ * 4));
  fill_random_f32(tmp, (size_t)step_rows_ * dp_, 0x7u, 0.f, 1.f, e_.stream_);
  launch_f32_to_bf16(tmp, h16_, (size_t)step_rows_ * dp_, e_.stream_);
  for (int M = 64; M <= step_rows_; M *= 2) {
    auto go = [&](const bf16_t* A, int lda, const bf16_t* wt, int N, int K, int epi, float* C, int ldc, bf16_t* C16, int act) {
      GemmQArgs g;
      std::memset(&g, 0, sizeof(g));
      g.A = A; g.lda = lda; g.M = M; g.N = N; g.K = K; g.nseg = 1; g.seg[0] = mat(wt, N, K);
      g.C = C; g.C16 = C16; g.ldc = ldc; g.epi = epi; g.act = act;
      gemm_pf_autotune(g, e_.stream_);
    };
    if (loopw_) go((const bf16_t*)xin_, 2 * dp_, loopw_, dp_, 2 * dp_, GEPI_STORE, y_, dp_, nullptr, 0);
    for (int i = 0; i < nl_; ++i) {
      if (owner_[i] != i) continue;
      const Dims& D = dims_[i];
      const Weights& w = w_[i];
      const int act = e_.cfg_.layers[i].act;
      go(h16_, dp_, w.in, D.n1, dp_, GEPI_STORE, qdg_, D.n1, nullptr, act);
      if (seq_) {
        go(cat16_, D.kout, w.out, dp_, D.kout, GEPI_STORE, y_, dp_, nullptr, act);
        if (w.in2 && D.n2) go(h16_, dp_, w.in2, D.n2, dp_, GEPI_STORE, qdg_, D.n2, nullptr, act);
        if (D.glu && e_.cfg_.layers[i].mlp == MLP_ACT) {
          go(h16_, dp_, w.in2 + (size_t)D.n2 * dp_, D.glu, dp_, GEPI_STORE16, nullptr, D.glu, cat16_, 0);
          go(cat16_, D.glu, w.out2, dp_, D.glu, GEPI_STORE, y_, dp_, nullptr, act);
        } else if (D.glu) {
          go(h16_, dp_, w.in2 + (size_t)D.n2 * dp_, 2 * D.glu, dp_, GEPI_SWIGLU_BF16, nullptr, D.glu, cat16_, act);
          go(cat16_, D.glu, w.out2, dp_, D.glu, GEPI_STORE, y_, dp_, nullptr, act);
        }
      } else {
        if (D.fp) go(h16_, dp_, w.in + (size_t)D.n1 * dp_, 2 * D.fp, dp_, GEPI_SWIGLU_BF16, nullptr, D.kout, cat16_ + D.gn, act);
        go(cat16_, D.kout, w.out, dp_, D.kout, GEPI_ACCUM, x_, dp_, nullptr, act);
      }
      if (D.rp && M <= pf_max_ctx_) go(cfull_, D.rp, w.ukv, D.qn + D.gn, D.rp, GEPI_STORE16, nullptr, D.qn + D.gn, kv_, act);
    }
  }
  HIP_CHECK(hipMemsetAsync(h16_, 0, (size_t)step_rows_ * dp_ * 2, e_.stream_));
  HIP_CHECK(hipStreamSynchronize(e_.stream_));
  HIP_CHECK(hipFree(tmp));
}

// ---- forward ----------------------------------------------------------------------------------------
void LayeredDecoder::gemm16(const bf16_t* A, int lda, const bf16_t* w, int M, int N, int K, int epi, float* C, int ldc,
                            bf16_t* C16, int act) {
  GemmQArgs g;
  std::memset(&g, 0, sizeof(g));
  g.A = A; g.lda = lda; g.M = M; g.N = N; g.K = K; g.nseg = 1; g.seg[0] = mat(w, N, K);
  g.C = C; g.C16 = C16; g.ldc = ldc; g.epi = epi; g.act = act;
  e_.gemm(g);
}

// key splits of an absorbed attention launch: one round of workgroups (two per CU), at least two 32-key tiles
// each (one for a token or two); rows x splits stays below rows + 16 x 512, which bounds the partial sums' buffer
int LayeredDecoder::key_split(int tiles, int max_len) const {
  const int want = (512 + tiles - 1) / std::max(tiles, 1);
  const int keys = tiles <= 4 ? 32 : 64;
  return std::max(1, std::min({want, (max_len + keys - 1) / keys, max_len <= 4096 ? 32 : 64}));
}

LatentAttnArgs LayeredDecoder::latent_args(int k, const RowSet& r) {
  const int i = runs_[k].layer;
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  LatentAttnArgs a;
  std::memset(&a, 0, sizeof(a));
  a.n = r.n_abs;
  a.H = D.H; a.dk = D.dk; a.dkp = D.dkp; a.dvp = D.dvp; a.rank = D.rank; a.rp = D.rp;
  a.rot = D.rot; a.roff = D.roff; a.qrot = D.qrot; a.rope = rope_[i];
  a.window = s.window;
  a.head_gate = s.out_gate == GATE_HEAD;
  a.scale = s.scale;
  a.eps = e_.cfg_.norm_eps;
  a.norm_w = w.kv_norm;
  a.sink = s.sink ? w.sink : nullptr;
  a.qdg = qdg_; a.ld = D.n1; a.dkv_off = D.qn; a.g_off = s.out_gate ? D.gate_off : -1;
  a.pos = r.pos; a.slot = r.slot;
  a.pool = runs_[k].pool;
  a.bt = e_.d_bt_; a.maxb = e_.kv_maxb_; a.kvb = e_.kvb_; a.f32 = f32_;
  a.wukT = w.ukT;
  a.wuv = w.ukv + (size_t)D.qn * D.rp;
  a.qa = qa_;
  if (r.decode) {
    a.n_tiles = r.n * ((D.H + 15) / 16);
  } else {
    const auto t = r.tiles.at(D.H);
    a.tiles = st_tiles_ + t.first;
    a.n_tiles = t.second;
  }
  // (a tile's window reaches from its first row's first key to its last row: at most 15 tokens more)
  const int keys = s.window ? std::min(r.max_len, s.window + 15) : r.max_len;
  a.nsplit = f32_ || !latent_attn_mfma(D.rp) ? 1 : key_split(a.n_tiles, keys);
  a.opart = opart_; a.ml = ml_;
  a.out = f32_ ? (void*)cat32_ : (void*)cat16_;
  a.ldo = D.kout;
  return a;
}

void LayeredDecoder::attention(int k, const RowSet& r) {
  const int i = runs_[k].layer;
  const Dims& D = dims_[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  const LatentAttnArgs a = latent_args(k, r);
  launch_latent_prep(a, r.n, st);
  if (a.n > 0) {
    launch_latent_attn(a, st);
    launch_latent_out(a, st);
  }
  for (const auto& pf : r.pf) {
    const Piece& p = pf.second;
    const int row0 = pf.first, k0 = a.window ? std::max(0, p.start - a.window + 1) : 0;
    const int S = p.start + p.n - k0, nkv = D.qn + D.gn;
    launch_latent_gather((const bf16_t*)a.pool, e_.d_bt_, e_.kv_maxb_, e_.kvb_, p.slot, k0, S, D.rp, cfull_, st);
    gemm16(cfull_, D.rp, w.ukv, S, nkv, D.rp, GEPI_STORE16, nullptr, nkv, kv_);
    MhaPrefillArgs m;
    std::memset(&m, 0, sizeof(m));
    m.q = qdg_ + (size_t)row0 * D.n1; m.ldq = D.n1;
    m.k = kv_; m.v = kv_ + D.qn; m.ldkv = nkv;
    m.H = D.H; m.dkp = D.dkp; m.dvp = D.dvp; m.start = p.start - k0; m.T = p.n;
    m.window = a.window; m.rot = a.rot; m.qrot = a.qrot; m.pos0 = p.start; m.rope = a.rope;
    m.scale = a.scale; m.sink = a.sink;
    m.gate = a.g_off >= 0 ? qdg_ + (size_t)row0 * D.n1 + a.g_off : nullptr;
    m.head_gate = a.head_gate;
    m.out = cat16_ + (size_t)row0 * D.kout; m.ldo = D.kout;
    launch_mha_prefill(m, st);
  }
}

void LayeredDecoder::recurrence(int k, const RowSet& r) {
  const int i = runs_[k].layer;
  const Dims& D = dims_[i];
  const Weights& w = w_[owner_[i]];
  MinGruArgs a;
  std::memset(&a, 0, sizeof(a));
  a.in = qdg_; a.ld = D.n1; a.z_off = 0; a.u_off = D.wp; a.g_off = 2 * D.wp;
  a.zb = w.zb; a.ub = w.ub;
  a.w = D.wp;
  a.state = runs_[k].state;
  a.slots = e_.cfg_.max_slots;
  a.chunks = r.decode ? nullptr : st_chunks_;
  a.pos = r.pos; a.slot = r.slot;
  a.n = r.decode ? r.n : r.n_chunks;
  a.split = r.decode ? 0 : r.split;
  a.agg = agg_;
  a.out = f32_ ? (void*)cat32_ : (void*)cat16_;
  a.ldo = D.kout;
  a.f32 = f32_;
  launch_mingru(a, e_.stream_);
}

size_t LayeredDecoder::state_floats(int i) const {
  const Dims& D = dims_[i];
  return (size_t)D.wp + (D.lin ? (size_t)D.lH * D.lnp * D.lvp : 0);
}
size_t LayeredDecoder::ring_floats(int i) const {
  const Dims& D = dims_[i];
  return D.lin == LIN_HEAD || D.lin == LIN_DELTA ? (size_t)e_.cfg_.layers[i].lin.conv * (D.lH * D.ldv + 2 * D.lG * D.lN) : 0;
}

void LayeredDecoder::linear(int k, const RowSet& r) {
  const int i = runs_[k].layer;
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  const int nk = D.lH * D.lN, nv = D.lH * D.ldv, c0 = D.lin_off;
  LinScanArgs a;
  std::memset(&a, 0, sizeof(a));
  a.kind = D.lin;
  a.H = D.lH; a.G = D.lG; a.N = D.lN; a.np = D.lnp; a.dv = D.ldv; a.vp = D.lvp;
  a.in = qdg_; a.ld = D.n1;
  if (D.lin == LIN_HEAD) {  // [z | x | B | C | dt]
    a.z_off = c0;
    a.x_off = c0 + nv;
    a.dt_off = c0 + 2 * nv + 2 * D.lG * D.lN;
    a.taps = s.lin.conv;
    a.norm_parts = s.lin.norm_groups;
  } else if (D.lin == LIN_DELTA) {  // [v | k | q | gate | strengths | steps]
    a.x_off = c0;
    a.z_off = c0 + nv + 2 * D.lG * D.lN;
    a.b_off = a.z_off + nv;
    a.dt_off = a.b_off + D.lH;
    a.taps = s.lin.conv;
    a.q_scale = (float)(1.0 / std::sqrt((double)D.lN));
  } else {  // [q | k | v | gate | a]
    a.q_off = c0;
    a.k_off = c0 + nk;
    a.v_off = c0 + 2 * nk;
    a.z_off = c0 + 2 * nk + nv;
    a.a_off = c0 + 2 * nk + 2 * nv;
    a.rank = s.lin.rank;
    a.q_scale = (float)(1.0 / std::sqrt((double)D.lN));
    a.inv_tau = (float)(1.0 / s.lin.tau);
  }
  a.conv_w = w.conv_w; a.conv_b = w.conv_b; a.dt_b = w.dt_b; a.a_log = w.a_log; a.D = w.lin_d;
  a.a2 = w.a2; a.a2_b = w.a2_b;
  a.ring = runs_[k].ring;
  a.state = runs_[k].state; a.slots = e_.cfg_.max_slots;
  if (!r.decode) {
    a.seqs = st_seqs_; a.n_seqs = r.n_seqs;
    a.chunks = st_chunks_; a.n_chunks = r.n_chunks;
    a.nseg = lin_segments(D.lin, D.lH, D.lnp, D.lvp, r.n_seqs, (r.longest + LIN_T - 1) / LIN_T);
    a.seg = lin_seg_; a.seg_dec = lin_seg_dec_;
  }
  a.pos = r.pos; a.slot = r.slot; a.n = a.rows = r.n;
  a.qo = lin_qo_; a.ko = lin_ko_; a.kr = lin_kr_; a.vo = lin_vo_; a.so = lin_so_; a.dec = lin_dec_;
  a.y = lin_y_;
  a.norm_w = w.lin_norm;
  a.eps = e_.cfg_.norm_eps;
  a.out_scale = s.beside ? s.beside_scale : s.mixer_scale;
  a.out = f32_ ? (void*)(cat32_ + D.lin_out) : (void*)(cat16_ + D.lin_out);
  a.ldo = D.kout;
  a.f32 = f32_;
  launch_lin_scan(a, e_.stream_);
}

void LayeredDecoder::grouped_attention(int k, const RowSet& r) {
  const int i = runs_[k].layer;
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  GqaArgs a;
  std::memset(&a, 0, sizeof(a));
  a.rows = r.n; a.n = f32_ ? r.n : r.n_abs;
  a.H = D.H; a.G = D.G; a.dk = D.dk; a.dkp = D.dkp; a.dv = D.dv; a.dvp = D.dvp;
  a.rot = D.rot; a.rope = rope_[i];
  a.window = s.window; a.chunk = s.chunk;
  a.scale = s.scale; a.softcap = s.softcap;
  a.sink = s.sink == 2 ? zero_sink_ : s.sink ? w.sink : nullptr;
  a.qn = w.qn; a.kn = w.kn; a.temp = w.temp;
  a.v_norm = s.v_norm;
  a.eps = e_.cfg_.norm_eps;
  if (s.v_mix) a.first = v_first_;
  a.lambda = s.v_mix && i != v_first_layer_ ? w.lambda : nullptr;
  a.qb = w.qb; a.kb = w.kb; a.vb = w.vb;
  a.in = qdg_; a.ld = D.n1; a.k_off = D.koff; a.v_off = D.voff; a.g_off = s.out_gate == GATE_HEAD ? D.gate_off : -1;
  a.out_scale = s.mixer_scale;
  a.pos = r.pos; a.slot = r.slot;
  a.pool = runs_[k].pool; a.bt = e_.d_bt_; a.maxb = e_.kv_maxb_; a.f32 = f32_;
  a.q = qa_;
  const int rep = D.H / D.G;
  if (r.decode) {
    a.n_tiles = r.n * ((rep + 15) / 16);
  } else {
    const auto t = r.tiles.at(rep);
    a.tiles = st_tiles_ + t.first;
    a.n_tiles = t.second;
  }
  // (a tile's keys reach from its first row's first one to its last row: at most 15 tokens more)
  const int w1 = s.window ? s.window : 1 << 30, w2 = s.chunk ? s.chunk : 1 << 30;
  const int keys = std::min(r.max_len, std::min(w1, w2) + 15);
  a.nsplit = f32_ ? 1 : std::min(64, key_split(a.n_tiles * D.G, (keys + 3) / 4));  // (four waves share a split's keys)
  a.opart = opart_; a.ml = ml_;
  a.out = f32_ ? (void*)cat32_ : (void*)cat16_;
  a.ldo = D.kout;
  launch_gqa_prep(a, st);
  if (a.n > 0) launch_gqa_attn(a, st);
  for (const auto& pf : r.pf) {
    if (f32_) break;
    const Piece& p = pf.second;
    const int row0 = pf.first;
    MhaPrefillArgs m;
    std::memset(&m, 0, sizeof(m));
    m.q16 = (const bf16_t*)qa_ + (size_t)row0 * D.H * D.dkp;
    m.pool = (const bf16_t*)a.pool;
    m.bt = e_.d_bt_ + (size_t)p.slot * e_.kv_maxb_;
    m.G = D.G; m.H = D.H; m.dkp = D.dkp; m.dvp = D.dvp;
    m.start = p.start; m.T = p.n;
    m.window = s.window; m.chunk = s.chunk;
    m.softcap = s.softcap; m.out_scale = s.mixer_scale;
    m.sink = a.sink;
    m.gate = a.g_off >= 0 ? qdg_ + (size_t)row0 * D.n1 + a.g_off : nullptr;
    m.ldq = D.n1; m.head_gate = 1;
    m.out = cat16_ + (size_t)row0 * D.kout; m.ldo = D.kout;
    launch_mha_prefill(m, st);
  }
}

bool LayeredDecoder::enters_pass(int k) const {
  return x0_ && k < runs_to_do() && runs_[k].pass > 0 && runs_[k].layer == e_.cfg_.loop_start;
}

// ---- sequential layers --------------------------------------------------------------------------------
void LayeredDecoder::project(const void* a, int lda, const bf16_t* w, int n, int N, int K, float* y, int ldy) {
  if (f32_) return launch_gemm_f32((const float*)a, lda, w, K, n, N, K, y, ldy, 0, e_.stream_);
  if (n <= 4) {
    GemvArgs g = e_.gemv_args({}, N, K, n, nullptr, lda, nullptr, y, ldy, EPI_STORE, 0);
    g.nseg = 1;
    g.seg[0] = mat(w, N, K);
    g.x16 = (const bf16_t*)a;
    if (gemv_bf16_engine_fits(g)) return launch_gemv(g, e_.stream_);
  }
  gemm16((const bf16_t*)a, lda, w, n, N, K, GEPI_STORE, y, ldy, nullptr);
}

NextArgs LayeredDecoder::next_of(int k, bool decode) {
  NextArgs x;
  if (k >= (int)runs_.size()) {
    if (!decode) return x;  // (a step's head gathers and normalises the rows it is asked for)
    x.kind = NEXT_NORM;
    x.g = out_norm_;
  } else if (loopw_ && runs_[k].pass >= 0 && runs_[k].layer == e_.cfg_.loop_start) {
    x.kind = NEXT_RAW;
    x.out = xin_;
    x.ldo = 2 * dp_;
    return x;
  } else {
    x.kind = NEXT_NORM;
    x.g = w_[owner_[runs_[k].layer]].norm;
  }
  x.out = f32_ ? (void*)h32_ : (void*)h16_;
  x.ldo = dp_;
  return x;
}

RowCloseArgs LayeredDecoder::close_args() const {
  RowCloseArgs c;
  std::memset((void*)&c, 0, sizeof(c));
  c.x = x_;
  c.dp = dp_; c.d = d_;
  c.eps = e_.cfg_.norm_eps;
  c.y = y_;
  c.f32 = f32_;
  return c;
}

// the second sublayer's products up to its result: c.y, or c.y and the experts' rows
void LayeredDecoder::feed_forward(int k, const RowSet& r, RowCloseArgs& c) {
  const int i = runs_[k].layer, n = r.n;
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  const void* h = f32_ ? (const void*)h32_ : (const void*)h16_;
  void* act = f32_ ? (void*)cat32_ : (void*)cat16_;
  const bf16_t* wglu = w.in2 + (size_t)D.n2 * dp_;
  bool done = false;
  if (s.mlp == MLP_ACT) {
    if (D.n2) project(h, dp_, w.in2, n, D.n2, dp_, qdg_, D.n2);
    if (f32_) {
      launch_gemm_f32(h32_, dp_, wglu, dp_, n, D.fp, dp_, gu32_, D.fp, 0, e_.stream_);
      launch_bias_act_f32(gu32_, D.fp, w.upb, cat32_, D.fp, n, D.fp, s.act, w.act_n, e_.stream_);
    } else {
      if (n <= 4) {
        GemvArgs a = e_.gemv_args({}, D.fp, dp_, n, nullptr, dp_, nullptr, nullptr, D.fp, EPI_ACT16, 0);
        a.nseg = 1;
        a.seg[0] = mat(wglu, D.fp, dp_);
        a.x16 = h16_;
        a.act = s.act;
        a.act_n = w.act_n;
        a.bias = w.upb;
        a.y16 = cat16_;
        a.ldy16 = D.fp;
        done = gemv_bf16_engine_fits(a);
        if (done) launch_gemv(a, e_.stream_);
      }
      if (!done) {
        GemmQArgs g;
        std::memset(&g, 0, sizeof(g));
        g.A = h16_; g.lda = dp_; g.M = n; g.N = D.fp; g.K = dp_; g.nseg = 1; g.seg[0] = mat(wglu, D.fp, dp_);
        g.C16 = cat16_; g.ldc = D.fp; g.epi = GEPI_STORE16;
        g.bias16 = w.upb; g.unary = 1 + s.act; g.act_n = w.act_n;
        e_.gemm(g);
      }
    }
    project(act, D.fp, w.out2, n, dp_, D.fp, y_, dp_);
    c.y = y_;
    c.y_bias = w.dnb;
    return;
  }
  if (!f32_ && D.glu && n <= 64) {  // one launch over all rows of in2
    const int N = D.n2 + 2 * D.glu;
    if (n <= 4) {
      GemvArgs a = e_.gemv_args({}, N, dp_, n, nullptr, dp_, nullptr, qdg_, D.n2, EPI_STORE_GLU, 0);
      a.nseg = 1;
      a.seg[0] = mat(w.in2, N, dp_);
      a.x16 = h16_;
      a.act = s.act;
      a.glu_row0 = D.n2;
      a.y16 = cat16_;
      a.ldy16 = D.glu;
      done = gemv_bf16_engine_fits(a);
      if (done) launch_gemv(a, e_.stream_);
    }
    if (!done && D.n2) {
      GemmQArgs g;
      std::memset(&g, 0, sizeof(g));
      g.A = h16_; g.lda = dp_; g.M = n; g.N = N; g.K = dp_; g.nseg = 1; g.seg[0] = mat(w.in2, N, dp_);
      g.C = qdg_; g.ldc = D.n2; g.epi = GEPI_STORE_GLU; g.act = s.act;
      g.glu_n0 = D.n2; g.C16 = cat16_; g.ldc16 = D.glu;
      e_.gemm(g);
      done = true;
    }
  }
  if (!done) {
    if (D.n2) project(h, dp_, w.in2, n, D.n2, dp_, qdg_, D.n2);
    if (D.glu && f32_) {
      launch_gemm_f32(h32_, dp_, wglu, dp_, n, 2 * D.glu, dp_, gu32_, 2 * D.glu, 0, e_.stream_);
      launch_glu_f32(gu32_, 2 * D.glu, cat32_, D.glu, n, D.glu, s.act, e_.stream_);
    } else if (D.glu) {
      gemm16(h16_, dp_, wglu, n, 2 * D.glu, dp_, GEPI_SWIGLU_BF16, nullptr, D.glu, cat16_, s.act);
    }
  }
  c.y = D.glu || s.mlp == MLP_GLU ? y_ : nullptr;
  if (s.mlp == MLP_MOE) {
    MoeArgs m;
    std::memset(&m, 0, sizeof(m));
    m.n = n; m.experts = s.experts; m.top = s.top; m.scale = s.router_scale;
    m.logits = qdg_ + D.router_off; m.ldl = D.n2;
    m.corr = s.correction ? w.corr : nullptr;
    m.dp = dp_; m.ff = D.fp; m.act = s.act;
    m.h = h; m.ldh = dp_;
    m.wgu = w.egu; m.wdn = w.edn;
    m.sel = moe_sel_; m.wt = moe_wt_; m.pair = moe_pair_; m.token = moe_token_;
    m.tiles = moe_tiles_; m.n_tiles = moe_ntiles_; m.max_tiles = moe_max_tiles_;
    m.act_out = moe_act_; m.ye = moe_ye_; m.gu32 = moe_gu32_;
    m.f32 = f32_;
    if (D.glu) { m.sh_act = cat16_; m.ld_sh = D.glu; m.sh_ff = D.glu; m.sh_dn = w.out2; }
    m.y = y_;
    if (moe_few_fits(m)) {
      c.y = y_;
      return launch_moe_few(m, e_.stream_);
    }
    launch_moe_grouped(m, e_.stream_);
    c.ye = moe_ye_; c.pair = moe_pair_; c.wt = moe_wt_; c.top = s.top;
  }
  if (D.glu) project(act, D.glu, w.out2, n, dp_, D.glu, y_, dp_);
}

void LayeredDecoder::layer_seq(int k, const RowSet& r) {
  const int i = runs_[k].layer, n = r.n;
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  const void* h = f32_ ? (const void*)h32_ : (const void*)h16_;
  void* cat = f32_ ? (void*)cat32_ : (void*)cat16_;
  if (loopw_ && runs_[k].pass >= 0 && i == e_.cfg_.loop_start) {  // a pass begins: x = W [x; x0] + step
    project(xin_, 2 * dp_, loopw_, n, dp_, 2 * dp_, y_, dp_);
    RowCloseArgs c = close_args();
    c.replace = 1;
    c.add = loop_step_ + (size_t)runs_[k].pass * dp_;
    c.next.kind = NEXT_NORM;
    c.next.g = w.norm;
    c.next.out = f32_ ? (void*)h32_ : (void*)h16_;
    c.next.ldo = dp_;
    launch_row_close(c, n, st);
  }
  project(h, dp_, w.in, n, D.n1, dp_, qdg_, D.n1);
  if (s.mixer == MIX_MINGRU) recurrence(k, r);
  else if (s.mixer == MIX_GQA) grouped_attention(k, r);
  else if (s.mixer == MIX_LATENT) attention(k, r);
  if (D.lin) linear(k, r);
  project(cat, D.kout, w.out, n, dp_, D.kout, y_, dp_);
  RowCloseArgs c = close_args();
  if (s.resid_gate) { c.gate = qdg_ + D.rg_off; c.ldg = D.n1; c.gate_bias = w.rgb; }
  if (s.post_norm) c.post = w.post;
  c.y_bias = w.ob;
  if (s.mlp == MLP_NONE) {
    if (enters_pass(k + 1)) c.extra = x0_;
    c.next = next_of(k + 1, r.decode);
    return launch_row_close(c, n, st);
  }
  c.next.kind = NEXT_NORM;
  c.next.g = w.norm2;
  c.next.out = f32_ ? (void*)h32_ : (void*)h16_;
  c.next.ldo = dp_;
  launch_row_close(c, n, st);
  RowCloseArgs f = close_args();
  feed_forward(k, r, f);
  if (s.resid_gate) { f.gate = qdg_; f.ldg = D.n2; f.gate_bias = w.rgb2; }
  if (s.post_norm) f.post = w.post2;
  if (enters_pass(k + 1)) f.extra = x0_;
  f.next = next_of(k + 1, r.decode);
  launch_row_close(f, n, st);
}

void LayeredDecoder::layer16(int k, const RowSet& r) {
  const int i = runs_[k].layer;
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  const float eps = e_.cfg_.norm_eps;
  const int n = r.n;
  if (n <= 4 && gemv_ok_[n]) {
    GemvArgs a = e_.gemv_args({}, D.nin, dp_, n, x_, dp_, w.norm, qdg_, D.n1, D.fp ? EPI_STORE_GLU : EPI_STORE, 0);
    a.nseg = 1;
    a.seg[0] = mat(w.in, D.nin, dp_);
    a.act = s.act;
    a.glu_row0 = D.n1;
    a.y16 = D.fp ? cat16_ + D.gn : nullptr;
    a.ldy16 = D.kout;
    launch_gemv(a, st);
    attention(k, r);
    GemvArgs b = e_.gemv_args({}, dp_, D.kout, n, nullptr, D.kout, nullptr, x_, dp_, EPI_RESID, 0);
    b.nseg = 1;
    b.seg[0] = mat(w.out, dp_, D.kout);
    b.x16 = cat16_;
    launch_gemv(b, st);
    return;
  }
  const bool fuse = nparts_ > 0 && n <= 64;
  if (!norm_ready_) launch_rmsnorm_bf16(x_, dp_, w.norm, h16_, dp_, n, d_, eps, st);
  if (n <= 64) {
    GemmQArgs g;
    std::memset(&g, 0, sizeof(g));
    g.A = h16_; g.lda = dp_; g.M = n; g.N = D.nin; g.K = dp_; g.nseg = 1; g.seg[0] = mat(w.in, D.nin, dp_);
    g.C = qdg_; g.ldc = D.n1; g.epi = D.fp ? GEPI_STORE_GLU : GEPI_STORE; g.act = s.act;
    g.glu_n0 = D.n1; g.C16 = cat16_ + D.gn; g.ldc16 = D.kout;
    if (norm_ready_) { g.A = xn16_; g.nrm_in = npart_; g.nrm_parts = nparts_; g.nrm_eps = eps; }
    e_.gemm(g);
  } else {
    gemm16(h16_, dp_, w.in, n, D.n1, dp_, GEPI_STORE, qdg_, D.n1, nullptr);
    if (D.fp)
      gemm16(h16_, dp_, w.in + (size_t)D.n1 * dp_, n, 2 * D.fp, dp_, GEPI_SWIGLU_BF16, nullptr, D.kout, cat16_ + D.gn, s.act);
  }
  attention(k, r);
  GemmQArgs g;
  std::memset(&g, 0, sizeof(g));
  g.A = cat16_; g.lda = D.kout; g.M = n; g.N = dp_; g.K = D.kout; g.nseg = 1; g.seg[0] = mat(w.out, dp_, D.kout);
  g.C = x_; g.ldc = dp_; g.epi = GEPI_ACCUM;
  if (fuse) {
    g.epi = GEPI_ACCUM_NORM;
    g.nrm_g = i + 1 < nl_ ? w_[owner_[i + 1]].norm : out_norm_;
    g.nrm_out16 = xn16_; g.nrm_part = npart_; g.nrm_parts = nparts_;
  }
  e_.gemm(g);
  norm_ready_ = fuse;
}

void LayeredDecoder::layer32(int k, const RowSet& r) {
  const int i = runs_[k].layer;
  const Dims& D = dims_[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  launch_rmsnorm(x_, dp_, w.norm, h32_, dp_, r.n, d_, e_.cfg_.norm_eps, st);
  launch_gemm_f32(h32_, dp_, w.in, dp_, r.n, D.n1, dp_, qdg_, D.n1, 0, st);
  if (D.fp) {
    launch_gemm_f32(h32_, dp_, w.in + (size_t)D.n1 * dp_, dp_, r.n, 2 * D.fp, dp_, gu32_, 2 * D.fp, 0, st);
    launch_glu_f32(gu32_, 2 * D.fp, cat32_ + D.gn, D.kout, r.n, D.fp, e_.cfg_.layers[i].act, st);
  }
  attention(k, r);
  launch_gemm_f32(cat32_, D.kout, w.out, D.kout, r.n, dp_, D.kout, x_, dp_, 1, st);
}

void LayeredDecoder::layer_fused(int k, const RowSet& r) {
  const int i = runs_[k].layer, n = r.n;
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  const float eps = e_.cfg_.norm_eps;
  const bool few = n <= 4;
  // y = W norm(x) in fp32, or (y16) act(W norm(x) + bias)
  auto from_residual = [&](const bf16_t* m, int N, const float* g, float* y, bf16_t* y16, const float* bias) {
    if (few) {
      GemvArgs a = e_.gemv_args({}, N, dp_, n, x_, dp_, g, y, N, y16 ? EPI_ACT16 : EPI_STORE, 0);
      a.nseg = 1;
      a.seg[0] = mat(m, N, dp_);
      a.act = s.act;
      a.act_n = w.act_n;
      a.bias = bias;
      a.y16 = y16;
      a.ldy16 = N;
      return launch_gemv(a, st);
    }
    GemmQArgs a;
    std::memset(&a, 0, sizeof(a));
    a.A = h16_; a.lda = dp_; a.M = n; a.N = N; a.K = dp_; a.nseg = 1; a.seg[0] = mat(m, N, dp_);
    a.C = y; a.C16 = y16; a.ldc = N; a.epi = y16 ? GEPI_STORE16 : GEPI_STORE;
    a.bias16 = bias;
    if (y16) a.unary = 1 + s.act;
    a.act_n = w.act_n;
    if (norm_ready_) { a.A = xn16_; a.nrm_in = npart_; a.nrm_parts = nparts_; a.nrm_eps = eps; }
    e_.gemm(a);
  };
  // x += W cat + bias; g: weight of the norm that reads it next; enter: the loop's embedding joins
  auto to_residual = [&](const bf16_t* m, int K, const float* bias, const float* g, bool enter) {
    if (few) {
      GemvArgs a = e_.gemv_args({}, dp_, K, n, nullptr, K, nullptr, x_, dp_, bias ? EPI_RESID_BIAS : EPI_RESID, 0);
      a.nseg = 1;
      a.seg[0] = mat(m, dp_, K);
      a.x16 = cat16_;
      a.bias = bias;
      launch_gemv(a, st);
      if (!enter) return;
    } else if (!enter) {
      GemmQArgs a;
      std::memset(&a, 0, sizeof(a));
      a.A = cat16_; a.lda = K; a.M = n; a.N = dp_; a.K = K; a.nseg = 1; a.seg[0] = mat(m, dp_, K);
      a.C = x_; a.ldc = dp_; a.epi = GEPI_ACCUM_NORM;
      a.bias16 = bias;
      a.nrm_g = g; a.nrm_out16 = xn16_; a.nrm_part = npart_; a.nrm_parts = nparts_;
      e_.gemm(a);
      norm_ready_ = true;
      return;
    }
    RowCloseArgs c = close_args();
    c.extra = x0_;
    if (!few) {
      project(cat16_, K, m, n, dp_, K, y_, dp_);
      c.y = y_;
      c.y_bias = bias;
      c.next = next_of(k + 1, r.decode);
      norm_ready_ = false;
    }
    launch_row_close(c, n, st);
  };
  from_residual(w.in, D.n1, w.norm, qdg_, nullptr, nullptr);
  if (s.mixer == MIX_MINGRU) recurrence(k, r);
  else if (s.mixer == MIX_GQA) grouped_attention(k, r);
  else if (s.mixer == MIX_LATENT) attention(k, r);
  if (D.lin) linear(k, r);
  const float* after = k + 1 < runs_to_do() ? w_[owner_[runs_[k + 1].layer]].norm : out_norm_;
  to_residual(w.out, D.kout, w.ob, D.glu ? w.norm2 : after, !D.glu && enters_pass(k + 1));
  if (!D.glu) return;
  from_residual(w.in2, D.glu, w.norm2, nullptr, cat16_, w.upb);
  to_residual(w.out2, D.glu, w.dnb, after, enters_pass(k + 1));
}

void LayeredDecoder::run(const RowSet& r) {
  const EngineConfig& c = e_.cfg_;
  EmbedArgs e;
  std::memset((void*)&e, 0, sizeof(e));
  e.table = embd_; e.scale = c.embed_scale; e.pos_table = posw_;
  e.pair_table = pairw_; e.buckets = c.bigram_buckets; e.mul_prev = c.bigram_prev; e.mul_cur = c.bigram_cur;
  e.tokens = r.tokens; e.pos = r.pos; e.slot = r.slot; e.run = r.run;
  e.last = last_tok_; e.slots = c.max_slots;
  e.dp = dp_; e.d = d_; e.eps = c.norm_eps;
  e.x = x_;
  if (xin_) {
    e.keep = f32_ ? (void*)((float*)xin_ + dp_) : (void*)((bf16_t*)xin_ + dp_);
    e.ld_keep = 2 * dp_;
  }
  e.keep32 = x0_;
  e.f32 = f32_;
  const bool few = fused(r.n);
  if (seq_ && !(few && r.n <= 4)) e.next = next_of(0, r.decode);
  launch_embed_rows(e, r.n, e_.stream_);
  norm_ready_ = false;
  const int n = runs_to_do();
  for (int k = 0; k < n; ++k) {
    if (few) layer_fused(k, r);
    else if (seq_) layer_seq(k, r);
    else if (f32_) layer32(k, r);
    else layer16(k, r);
  }
}

void LayeredDecoder::decode_forward(int B) {
  RowSet r;
  r.tokens = e_.d_tokens_; r.pos = e_.d_pos_; r.slot = e_.d_slot_; r.run = nullptr;
  r.n_chunks = r.split = r.n_seqs = r.longest = 0;
  r.n = r.n_abs = B;
  r.decode = true;
  r.max_len = e_.cfg_.max_ctx;
  run(r);
  head_ready_ = seq_ && !fused(B);  // (the last layer left the head's operand)
  // (the head reads the residual in place: the decode rows are x rows 0 .. B-1)
  std::swap(x_, xh_);
  head(B);
  std::swap(x_, xh_);
}

int LayeredDecoder::span(const Piece& p) const {
  return max_window_ ? std::min(p.start + p.n, p.n + max_window_ - 1) : p.start + p.n;
}

void LayeredDecoder::forward(const std::vector<Piece>& pieces, std::vector<int>& first_row) {
  const int R = step_rows_;
  std::vector<int> order;  // absorbed pieces first
  RowSet r;
  r.decode = false;
  r.n = r.n_abs = r.max_len = 0;
  for (int p = 0; p < (int)pieces.size(); ++p) {
    const Piece& q = pieces[p];
    r.n += q.n;
    if (q.n < pf_min_ || span(q) > pf_max_ctx_) {
      order.push_back(p);
      r.n_abs += q.n;
      r.max_len = std::max(r.max_len, q.start + q.n);
    }
  }
  if (r.n < 1 || r.n > R) throw std::runtime_error("layered forward: too many rows");
  const int n_small = (int)order.size();
  for (int p = 0; p < (int)pieces.size(); ++p)
    if (std::find(order.begin(), order.begin() + n_small, p) == order.begin() + n_small) order.push_back(p);
  first_row.assign(pieces.size(), 0);
  int *ht = h_step_, *hp = ht + R, *hs = hp + R, *hr = hs + 2 * R;
  ScanChunk* chunks = (ScanChunk*)(hr + R);
  ScanSeq* seqs = (ScanSeq*)(h_step_ + ((const int*)st_seqs_ - d_step_));
  LatentTile* tiles = (LatentTile*)(h_step_ + ((const int*)st_tiles_ - d_step_));
  r.n_chunks = r.split = r.n_seqs = r.longest = 0;
  int row = 0, nt = 0;
  for (int o = 0; o < (int)order.size(); ++o) {
    const Piece& q = pieces[order[o]];
    first_row[order[o]] = row;
    for (int k = 0; k < q.n; ++k) {
      ht[row + k] = q.tokens[k];
      hp[row + k] = q.start + k;
      hs[row + k] = q.slot;
      hr[row + k] = k ? 0 : q.n;
    }
    const int c0 = r.n_chunks;
    r.longest = std::max(r.longest, q.n);
    seqs[r.n_seqs++] = ScanSeq{row, q.n, q.slot, q.start, 2 * c0};
    if (c0 + (q.n + SCAN_CHUNK - 1) / SCAN_CHUNK > max_chunks_) throw std::runtime_error("layered forward: too many pieces");
    for (int k = 0; k < q.n; k += SCAN_CHUNK)
      chunks[r.n_chunks++] = ScanChunk{row + k, std::min(SCAN_CHUNK, q.n - k), q.slot, q.start + k, c0, k + SCAN_CHUNK >= q.n};
    if (q.n > SCAN_CHUNK) r.split = 1;
    if (o >= n_small) r.pf.push_back({row, q});
    row += q.n;
  }
  for (const Dims& D : dims_) {
    const int rep = D.G ? D.H / D.G : D.H;  // rows of a token that read the same keys
    if (!D.H || r.tiles.count(rep)) continue;
    const int t0 = nt;
    for (int o = 0; o < n_small; ++o) {
      const int f0 = first_row[order[o]] * rep, f1 = f0 + pieces[order[o]].n * rep;
      for (int f = f0; f < f1; f += 16) tiles[nt++] = LatentTile{f, std::min(16, f1 - f)};
    }
    r.tiles[rep] = {t0, nt - t0};
  }
  r.tokens = st_tokens_; r.pos = st_pos_; r.slot = st_slot_; r.run = st_run_;
  const size_t ints = (size_t)((const int*)st_tiles_ - d_step_) + 2 * (size_t)nt;
  HIP_CHECK(hipMemcpyAsync(d_step_, h_step_, ints * 4, hipMemcpyHostToDevice, e_.stream_));
  run(r);
  head_ready_ = false;
  norm_ready_ = false;  // (the head normalises the rows it is asked for)
}

void LayeredDecoder::collect(const std::vector<int>& rows, int at) {
  if (rows.empty()) return;
  if (at + (int)rows.size() > step_rows_) throw std::runtime_error("layered forward: too many rows asked for");
  int* hw = h_step_ + (st_want_ - d_step_);
  std::copy(rows.begin(), rows.end(), hw + at);
  HIP_CHECK(hipMemcpyAsync(st_want_ + at, hw + at, rows.size() * 4, hipMemcpyHostToDevice, e_.stream_));
  launch_gather_rows(x_, dp_, st_want_ + at, (int)rows.size(), xh_ + (size_t)at * dp_, e_.stream_);
}

// logits rows [0, B) = head(norm(head input rows [from, from + B)))
void LayeredDecoder::head(int B, int from) {
  const float* x = xh_ + (size_t)from * dp_;
  hipStream_t st = e_.stream_;
  const float eps = e_.cfg_.norm_eps;
  float* y = e_.logits_;
  if (f32_) {
    if (!head_ready_) launch_rmsnorm(x, dp_, out_norm_, h32_, dp_, B, d_, eps, st);
    head_ready_ = false;
    launch_gemm_f32(h32_, dp_, headw_, dp_, B, vp_, dp_, y, vp_, 0, st);
    return;
  }
  if (head_ready_) {
    head_ready_ = false;
    return project(h16_, dp_, headw_, B, vp_, dp_, y, vp_);
  }
  if (B <= 4 && dp_ == d_ && !norm_ready_) {
    GemvArgs a = e_.gemv_args({}, vp_, dp_, B, x, dp_, out_norm_, y, vp_, EPI_STORE, 0);
    a.nseg = 1;
    a.seg[0] = mat(headw_, vp_, dp_);
    if (gemv_bf16_engine_fits(a)) {
      launch_gemv(a, st);
      return;
    }
  }
  GemmQArgs g;
  std::memset(&g, 0, sizeof(g));
  g.A = h16_; g.lda = dp_; g.M = B; g.N = vp_; g.K = dp_; g.nseg = 1; g.seg[0] = mat(headw_, vp_, dp_);
  g.C = y; g.ldc = vp_; g.epi = GEPI_STORE;
  if (norm_ready_) {
    g.A = xn16_; g.nrm_in = npart_; g.nrm_parts = nparts_; g.nrm_eps = eps;
    norm_ready_ = false;
  } else {
    launch_rmsnorm_bf16(x, dp_, out_norm_, h16_, dp_, B, d_, eps, st);
  }
  e_.gemm(g);
}

void LayeredDecoder::copy_state(int src, int dst) {
  const int slots = e_.cfg_.max_slots;
  auto copy = [&](void* base, size_t row) {
    for (int p = 0; p < 2; ++p)
      HIP_CHECK(hipMemcpyAsync((char*)base + ((size_t)p * slots + dst) * row, (char*)base + ((size_t)p * slots + src) * row, row,
                               hipMemcpyDeviceToDevice, e_.stream_));
  };
  for (const Run& k : runs_) {
    if (k.state) copy(k.state, state_floats(k.layer) * 4);
    if (k.ring)
      HIP_CHECK(hipMemcpyAsync(k.ring + dst * ring_floats(k.layer), k.ring + src * ring_floats(k.layer), ring_floats(k.layer) * 4,
                               hipMemcpyDeviceToDevice, e_.stream_));
  }
  if (last_tok_) copy(last_tok_, 4);
}

std::vector<float> LayeredDecoder::residual(int rows) {
  std::vector<float> out((size_t)rows * d_);
  HIP_CHECK(hipStreamSynchronize(e_.stream_));
  HIP_CHECK(hipMemcpy2D(out.data(), (size_t)d_ * 4, x_, (size_t)dp_ * 4, (size_t)d_ * 4, rows, hipMemcpyDeviceToHost));
  return out;
}

}  // namespace aios
