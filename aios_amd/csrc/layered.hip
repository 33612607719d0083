// LayeredDecoder implementation -- see layered.h.
//
// Per layer, 16-bit engine (weights, activations and cache bf16; residual, norms, scores fp32):
//   1-4 rows    one GEMV over [q | kv down | gate | MLP gate/up] with the RMSNorm in its prologue and the
//               GLU in its epilogue; latent prep; attention; normalise + Wuv + gate; one GEMV over
//               [attention out | MLP down] adding to the residual          -- 5 launches
//   5-64 rows   the same two products through the skinny MFMA GEMM, the RMSNorm split across them
//   more rows   prefill GEMMs; long portions take the expanded attention (latent.h)
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
static int env_or(const char* name, int dflt) {
  const char* e = std::getenv(name);
  return e ? std::atoi(e) : dflt;
}
// padded latent widths the attention kernels are built for
static int pad_rank(int r) {
  for (int t : {2, 4, 6, 8, 12, 16, 32})
    if (r <= 64 * t) return 64 * t;
  throw std::runtime_error("latent attention: kv_rank above 2048");
}

LayeredDecoder::LayeredDecoder(Engine& e) : e_(e) {
  const EngineConfig& c = e.cfg_;
  nl_ = (int)c.layers.size();
  d_ = c.d_model;
  dp_ = up(d_, 64);
  v_ = c.vocab_size;
  vp_ = up(v_, 64);
  f32_ = c.compute_f32;
  if (d_ < 1 || v_ < 1 || c.max_positions < 1) throw std::runtime_error("layered model: bad sizes");
  if (c.tp_size > 1) throw std::runtime_error("layered models run on one GPU (no tensor parallelism)");
  if (c.kv_fp8) throw std::runtime_error("layered models: the latent cache has no fp8 form");
  dims_.resize(nl_);
  owner_.resize(nl_);
  w_.resize(nl_);
  for (int i = 0; i < nl_; ++i) {
    int o = i;
    for (int hop = 0; c.layers[o].weights_of >= 0; ++hop) {
      o = c.layers[o].weights_of;
      if (o >= nl_ || hop > nl_) throw std::runtime_error("layer " + std::to_string(i) + ": weights_of names no layer");
    }
    owner_[i] = o;
    const LayerSpec &s = c.layers[i], &t = c.layers[o];
    if (s.mixer != MIX_LATENT) throw std::runtime_error("unknown mixer kind");
    if (s.heads != t.heads || s.dim != t.dim || s.vdim != t.vdim || s.kv_rank != t.kv_rank || s.mlp != t.mlp ||
        (s.mlp != MLP_NONE && s.ff != t.ff))
      throw std::runtime_error("layer " + std::to_string(i) + ": sizes differ from the layer whose weights it uses");
    if (s.heads < 1 || s.dim < 1 || s.vdim < 1 || s.kv_rank < 1 || (s.mlp != MLP_NONE && s.ff < 1))
      throw std::runtime_error("layer " + std::to_string(i) + ": bad sizes");
    Dims& D = dims_[i];
    D.H = s.heads;
    D.dk = s.dim;
    D.dv = s.vdim;
    D.rank = s.kv_rank;
    D.ff = s.mlp != MLP_NONE ? s.ff : 0;
    D.dkp = up(D.dk, 32);
    D.dvp = up(D.dv, 32);
    D.rp = pad_rank(D.rank);
    D.qn = up(D.H * D.dkp, 64);
    D.gn = up(D.H * D.dvp, 64);
    D.fp = up(D.ff, 64);
    D.n1 = D.qn + D.rp + D.gn;
    D.nin = D.n1 + 2 * D.fp;
    D.kout = D.gn + D.fp;
  }
  embd_ = balloc((size_t)v_ * dp_);
  posw_ = balloc((size_t)c.max_positions * dp_);
  headw_ = balloc((size_t)vp_ * dp_);
  out_norm_ = falloc(dp_);
  for (int i = 0; i < nl_; ++i) {
    if (owner_[i] != i) continue;
    const Dims& D = dims_[i];
    Weights& w = w_[i];
    w.own = true;
    w.norm = falloc(dp_);
    w.kv_norm = falloc(D.rp);
    w.sink = falloc(D.H);
    w.in = balloc((size_t)D.nin * dp_);
    w.out = balloc((size_t)dp_ * D.kout);
    w.ukv = balloc((size_t)(D.qn + D.gn) * D.rp);
    w.ukT = balloc((size_t)D.H * D.rp * D.dkp);
  }
  e_.weight_bytes_ = 0;
  for (const auto& t : tensor_list()) e_.weight_bytes_ += (size_t)t.second.first * t.second.second * 2;
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

void LayeredDecoder::put_vec(float* dst, int n, const bf16_t* src, bool device) {
  std::vector<bf16_t> h(n);
  std::vector<float> f(n);
  if (device) HIP_CHECK(hipMemcpy(h.data(), src, (size_t)n * 2, hipMemcpyDeviceToHost));
  else std::memcpy(h.data(), src, (size_t)n * 2);
  for (int i = 0; i < n; ++i) {
    const uint32_t u = (uint32_t)h[i] << 16;
    std::memcpy(&f[i], &u, 4);
  }
  HIP_CHECK(hipMemcpy(dst, f.data(), (size_t)n * 4, hipMemcpyHostToDevice));
}

// every tensor of the model: name, (rows, cols)
std::vector<std::pair<std::string, std::pair<int, int>>> LayeredDecoder::tensor_list() const {
  std::vector<std::pair<std::string, std::pair<int, int>>> t;
  auto add = [&](const std::string& n, int r, int c) { t.push_back({n, {r, c}}); };
  add("token_embd.weight", v_, d_);
  add("position_embd.weight", e_.cfg_.max_positions, d_);
  add("output_norm.weight", 1, d_);
  add("output.weight", v_, d_);
  for (int i = 0; i < nl_; ++i) {
    if (owner_[i] != i) continue;
    const Dims& D = dims_[i];
    const LayerSpec& s = e_.cfg_.layers[i];
    const std::string p = "blk." + std::to_string(i) + ".";
    add(p + "attn_norm.weight", 1, d_);
    add(p + "attn_q.weight", D.H * D.dk, d_);
    add(p + "attn_kv_a.weight", D.rank, d_);
    add(p + "attn_kv_a_norm.weight", 1, D.rank);
    add(p + "attn_k_b.weight", D.H * D.dk, D.rank);
    add(p + "attn_v_b.weight", D.H * D.dv, D.rank);
    if (s.sink) add(p + "attn_sinks.weight", 1, D.H);
    if (s.out_gate) add(p + "attn_gate.weight", D.H * D.dv, d_);
    add(p + "attn_output.weight", d_, D.H * D.dv);
    if (D.ff) {
      add(p + "ffn_gate.weight", D.ff, d_);
      add(p + "ffn_up.weight", D.ff, d_);
      add(p + "ffn_down.weight", d_, D.ff);
    }
  }
  return t;
}

void LayeredDecoder::put(const std::string& name, int rows, int cols, const bf16_t* src, bool device) {
  if (name == "token_embd.weight") return place(embd_, dp_, src, cols, cols, rows, device);
  if (name == "position_embd.weight") return place(posw_, dp_, src, cols, cols, rows, device);
  if (name == "output.weight") return place(headw_, dp_, src, cols, cols, rows, device);
  if (name == "output_norm.weight") return put_vec(out_norm_, cols, src, device);
  const size_t dot = name.find('.', 4);
  const int i = std::stoi(name.substr(4, dot - 4));
  const std::string t = name.substr(dot + 1);
  const Dims& D = dims_[i];
  Weights& w = w_[i];
  // heads of per_head rows each, spread to pad rows each
  auto heads = [&](bf16_t* dst, int dpitch, int per_head, int pad) {
    for (int h = 0; h < D.H; ++h)
      place(dst + (size_t)h * pad * dpitch, dpitch, src + (size_t)h * per_head * cols, cols, cols, per_head, device);
  };
  if (t == "attn_norm.weight") put_vec(w.norm, cols, src, device);
  else if (t == "attn_kv_a_norm.weight") put_vec(w.kv_norm, cols, src, device);
  else if (t == "attn_sinks.weight") put_vec(w.sink, cols, src, device);
  else if (t == "attn_q.weight") heads(w.in, dp_, D.dk, D.dkp);
  else if (t == "attn_kv_a.weight") place(w.in + (size_t)D.qn * dp_, dp_, src, cols, cols, rows, device);
  else if (t == "attn_gate.weight") heads(w.in + (size_t)(D.qn + D.rp) * dp_, dp_, D.dv, D.dvp);
  else if (t == "ffn_gate.weight") place(w.in + (size_t)D.n1 * dp_, 2 * dp_, src, cols, cols, rows, device);
  else if (t == "ffn_up.weight") place(w.in + (size_t)(D.n1 + 1) * dp_, 2 * dp_, src, cols, cols, rows, device);
  else if (t == "attn_k_b.weight") heads(w.ukv, D.rp, D.dk, D.dkp);
  else if (t == "attn_v_b.weight") heads(w.ukv + (size_t)D.qn * D.rp, D.rp, D.dv, D.dvp);
  else if (t == "attn_output.weight")
    for (int h = 0; h < D.H; ++h) place(w.out + (size_t)h * D.dvp, D.kout, src + (size_t)h * D.dv, cols, D.dv, rows, device);
  else if (t == "ffn_down.weight") place(w.out + D.gn, D.kout, src, cols, cols, rows, device);
  else throw std::runtime_error("unknown layer tensor " + name);
}

void LayeredDecoder::set_tensor(const std::string& name, int qt, int rows, int cols, const void* host, size_t nbytes) {
  if (qt != QT_BF16) throw std::runtime_error(name + ": layered models load bf16 tensors");
  if (nbytes != (size_t)rows * cols * 2) throw std::runtime_error(name + ": byte size mismatch");
  for (const auto& t : tensor_list())
    if (t.first == name) {
      if (t.second.first != rows || t.second.second != cols)
        throw std::runtime_error(name + ": shape " + std::to_string(rows) + " x " + std::to_string(cols) + ", expected " +
                                 std::to_string(t.second.first) + " x " + std::to_string(t.second.second));
      put(name, rows, cols, (const bf16_t*)host, false);
      have_.insert(name);
      return;
    }
  throw std::runtime_error("unknown tensor " + name);
}

void LayeredDecoder::init_random(uint64_t seed) {
  uint64_t s = seed * 1000003ULL;
  for (const auto& t : tensor_list()) {
    const int rows = t.second.first, cols = t.second.second;
    const size_t n = (size_t)rows * cols;
    const bool norm = t.first.find("norm") != std::string::npos, sink = t.first.find("sinks") != std::string::npos;
    bf16_t* tmp = nullptr;
    if (norm || sink) {
      float* f = nullptr;
      HIP_CHECK(hipMalloc(&f, n * 4));
      HIP_CHECK(hipMalloc(&tmp, n * 2 + 16));
      fill_random_f32(f, n, ++s, norm ? 1.f : 0.f, norm ? 0.1f : 1.f, e_.stream_);
      launch_f32_to_bf16(f, tmp, n, e_.stream_);
      HIP_CHECK(hipStreamSynchronize(e_.stream_));
      HIP_CHECK(hipFree(f));
    } else {
      HIP_CHECK(hipMalloc(&tmp, n * 2));
      fill_random_weight(mat(tmp, rows, cols), ++s, t.first == "token_embd.weight" ? 1.f : 0.02f, e_.stream_);
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
  for (const auto& t : tensor_list())
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
void LayeredDecoder::finalize() {
  const EngineConfig& c = e_.cfg_;
  const int Bm = c.max_batch;
  hipStream_t st = e_.stream_;
  for (int i = 0; i < nl_; ++i)
    if (w_[i].own) launch_transpose_heads(w_[i].ukv, dims_[i].H, dims_[i].dkp, dims_[i].rp, w_[i].ukT, st);
  // cache pools: one per layer (weights may be shared, the cached vectors are not)
  const int es = f32_ ? 4 : 2;
  pool_.resize(nl_);
  e_.kv_bytes_ = 0;
  for (int i = 0; i < nl_; ++i) {
    const size_t block = (size_t)e_.kvb_ * dims_[i].rp * es, bytes = (size_t)(e_.kv_nblocks_ + 1) * block;
    pool_[i] = (char*)e_.dmalloc(bytes);
    HIP_CHECK(hipMemset(pool_[i], 0, bytes));
    e_.pools_.push_back({pool_[i], block});
    e_.kv_bytes_ += bytes;
  }
  step_rows_ = std::max(Bm, std::min(2048, c.max_slots * c.max_ctx));
  if (const char* v = std::getenv("AIOS_STEP_ROWS")) step_rows_ = std::max(Bm, std::atoi(v));
  const int R = step_rows_;
  int n1 = 0, nin = 0, kout = 0, fp = 0, maxH = 0;
  size_t qa = 0, part = 0, kvw = 0, flat = 0;
  int rp = 0;
  for (const Dims& D : dims_) {
    n1 = std::max(n1, D.n1);
    nin = std::max(nin, D.nin);
    kout = std::max(kout, D.kout);
    fp = std::max(fp, D.fp);
    maxH = std::max(maxH, D.H);
    rp = std::max(rp, D.rp);
    qa = std::max(qa, (size_t)R * D.H * D.rp);
    const size_t fl = std::max((size_t)R * D.H, (size_t)16 * 1024);  // (key_split: rows x splits)
    flat = std::max(flat, fl);
    part = std::max(part, fl * D.rp);
    kvw = std::max(kvw, (size_t)D.qn + D.gn);
  }
  x_ = falloc((size_t)R * dp_);
  xh_ = falloc((size_t)R * dp_);
  qdg_ = falloc((size_t)R * n1);
  opart_ = falloc(part);
  ml_ = falloc(flat * 2);
  e_.ws_bytes_ = ((size_t)R * (2 * dp_ + n1) + part + 2 * flat) * 4;
  pf_max_ctx_ = std::min(c.max_ctx, 32768);
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
    pf_min_ = 0;
    for (const Dims& D : dims_) {
      const double s = D.dkp + D.dvp, gain = 2.0 * D.rp - s;
      const int t = gain > 0 ? (int)std::min(256.0, std::max(64.0, D.rp * s / gain)) : 256;
      pf_min_ = std::max(pf_min_, t);
      if (!mha_prefill_supports(D.dkp, D.dvp)) pf_min_ = 1 << 30;
    }
    if (const char* v = std::getenv("AIOS_LATENT_PF_MIN")) pf_min_ = std::max(1, std::atoi(v));
    for (const Dims& D : dims_)
      if (!mha_prefill_supports(D.dkp, D.dvp)) pf_min_ = 1 << 30;
    // the skinny GEMM's split-K workspace (shared with the engine's other users of gemm())
    const int maxN = std::max({nin, dp_, vp_, (int)kvw});
    e_.gk_ws_bytes_ = gemm_skinny_ws_bytes(64, maxN);
    e_.gk_ws_ = falloc(e_.gk_ws_bytes_ / 4 + 1);
    e_.gk_cnt_len_ = gemm_skinny_cnt_len(maxN);
    e_.gk_cnt_ = (int*)falloc(e_.gk_cnt_len_);
    if (nl_ > 0 && dp_ == d_ && d_ % 128 == 0 && env_or("AIOS_GEMM_NORM_FUSE", 1)) {
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
  std::set<int> hs;
  for (const Dims& D : dims_) hs.insert(D.H);
  size_t tiles = 0;
  for (int h : hs) tiles += (size_t)R * ((h + 15) / 16) + R;
  step_ints_ = (size_t)4 * R + 2 * tiles;
  HIP_CHECK(hipHostMalloc((void**)&h_step_, step_ints_ * 4, hipHostMallocDefault));
  d_step_ = (int*)falloc(step_ints_);
  st_tokens_ = d_step_;
  st_pos_ = st_tokens_ + R;
  st_slot_ = st_pos_ + R;
  st_want_ = st_slot_ + R;
  st_tiles_ = (LatentTile*)(st_want_ + R);
  gemv_ok_.assign(5, 0);
  for (int b = 1; b <= 4 && !f32_; ++b) {
    bool ok = dp_ == d_ && env_or("AIOS_LAYERED_GEMV", 1);
    for (int i = 0; i < nl_ && ok; ++i) ok = gemv_fits(i, b);
    gemv_ok_[b] = ok;
  }
  HIP_CHECK(hipStreamSynchronize(st));
  if (!f32_) tune();
}

bool LayeredDecoder::gemv_fits(int i, int B) {
  const Dims& D = dims_[i];
  const Weights& w = w_[owner_[i]];
  GemvArgs a = e_.gemv_args({}, D.nin, dp_, B, x_, dp_, w.norm, qdg_, D.n1, EPI_STORE, 0);
  a.nseg = 1;
  a.seg[0] = mat(w.in, D.nin, dp_);
  if (!gemv_bf16_engine_fits(a)) return false;
  a.seg[0] = mat(w.out, dp_, D.kout);
  a.N = dp_;
  a.K = D.kout;
  a.ldx = D.kout;
  return gemv_bf16_engine_fits(a);
}

// measured prefill-GEMM plans for the layers' shapes (as Engine::tune_prefill_gemm)
void LayeredDecoder::tune() {
  if (!env_or("AIOS_GEMM_PF_TUNE", 1) || nl_ == 0) return;
  float* tmp = nullptr;
  const size_t n = (size_t)step_rows_ * std::max({dp_, dims_[0].kout, 64});
  HIP_CHECK(hipMalloc(&tmp, n * 4));
  fill_random_f32(tmp, n, 0x7u, 0.f, 1.f, e_.stream_);
  launch_f32_to_bf16(tmp, h16_, (size_t)step_rows_ * dp_, e_.stream_);
  for (int M = 64; M <= step_rows_; M *= 2)
    for (int i = 0; i < nl_; ++i) {
      if (owner_[i] != i) continue;
      const Dims& D = dims_[i];
      const Weights& w = w_[i];
      auto go = [&](const bf16_t* A, int lda, const bf16_t* wt, int N, int K, int epi, float* C, int ldc, bf16_t* C16) {
        GemmQArgs g;
        std::memset(&g, 0, sizeof(g));
        g.A = A; g.lda = lda; g.M = M; g.N = N; g.K = K; g.nseg = 1; g.seg[0] = mat(wt, N, K);
        g.C = C; g.C16 = C16; g.ldc = ldc; g.epi = epi; g.act = e_.cfg_.layers[i].act;
        gemm_pf_autotune(g, e_.stream_);
      };
      go(h16_, dp_, w.in, D.n1, dp_, GEPI_STORE, qdg_, D.n1, nullptr);
      if (D.fp) go(h16_, dp_, w.in + (size_t)D.n1 * dp_, 2 * D.fp, dp_, GEPI_SWIGLU_BF16, nullptr, D.kout, cat16_ + D.gn);
      go(cat16_, D.kout, w.out, dp_, D.kout, GEPI_ACCUM, x_, dp_, nullptr);
      if (M <= pf_max_ctx_) go(cfull_, D.rp, w.ukv, D.qn + D.gn, D.rp, GEPI_STORE16, nullptr, D.qn + D.gn, kv_);
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

LatentAttnArgs LayeredDecoder::latent_args(int i, const RowSet& r) {
  const Dims& D = dims_[i];
  const LayerSpec& s = e_.cfg_.layers[i];
  const Weights& w = w_[owner_[i]];
  LatentAttnArgs a;
  std::memset(&a, 0, sizeof(a));
  a.n = r.n_abs;
  a.H = D.H; a.dk = D.dk; a.dkp = D.dkp; a.dvp = D.dvp; a.rank = D.rank; a.rp = D.rp;
  a.scale = s.scale;
  a.eps = e_.cfg_.norm_eps;
  a.norm_w = w.kv_norm;
  a.sink = s.sink ? w.sink : nullptr;
  a.qdg = qdg_; a.ld = D.n1; a.dkv_off = D.qn; a.g_off = s.out_gate ? D.qn + D.rp : -1;
  a.pos = r.pos; a.slot = r.slot;
  a.pool = pool_[i];
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
  a.nsplit = f32_ || !latent_attn_mfma(D.rp) ? 1 : key_split(a.n_tiles, r.max_len);
  a.opart = opart_; a.ml = ml_;
  a.out = f32_ ? (void*)cat32_ : (void*)cat16_;
  a.ldo = D.kout;
  return a;
}

void LayeredDecoder::attention(int i, const RowSet& r) {
  const Dims& D = dims_[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  const LatentAttnArgs a = latent_args(i, r);
  launch_latent_prep(a, r.n, st);
  if (a.n > 0) {
    launch_latent_attn(a, st);
    launch_latent_out(a, st);
  }
  for (const auto& pf : r.pf) {
    const Piece& p = pf.second;
    const int row0 = pf.first, S = p.start + p.n, nkv = D.qn + D.gn;
    launch_latent_gather((const bf16_t*)pool_[i], e_.d_bt_, e_.kv_maxb_, e_.kvb_, p.slot, S, D.rp, cfull_, st);
    gemm16(cfull_, D.rp, w.ukv, S, nkv, D.rp, GEPI_STORE16, nullptr, nkv, kv_);
    MhaPrefillArgs m;
    m.q = qdg_ + (size_t)row0 * D.n1; m.ldq = D.n1;
    m.k = kv_; m.v = kv_ + D.qn; m.ldkv = nkv;
    m.H = D.H; m.dkp = D.dkp; m.dvp = D.dvp; m.start = p.start; m.T = p.n;
    m.scale = a.scale; m.sink = a.sink;
    m.gate = a.g_off >= 0 ? qdg_ + (size_t)row0 * D.n1 + a.g_off : nullptr;
    m.out = cat16_ + (size_t)row0 * D.kout; m.ldo = D.kout;
    launch_mha_prefill(m, st);
  }
}

void LayeredDecoder::layer16(int i, const RowSet& r) {
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
    attention(i, r);
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
  attention(i, r);
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

void LayeredDecoder::layer32(int i, const RowSet& r) {
  const Dims& D = dims_[i];
  const Weights& w = w_[owner_[i]];
  hipStream_t st = e_.stream_;
  launch_rmsnorm(x_, dp_, w.norm, h32_, dp_, r.n, d_, e_.cfg_.norm_eps, st);
  launch_gemm_f32(h32_, dp_, w.in, dp_, r.n, D.n1, dp_, qdg_, D.n1, 0, st);
  if (D.fp) {
    launch_gemm_f32(h32_, dp_, w.in + (size_t)D.n1 * dp_, dp_, r.n, 2 * D.fp, dp_, gu32_, 2 * D.fp, 0, st);
    launch_glu_f32(gu32_, 2 * D.fp, cat32_ + D.gn, D.kout, r.n, D.fp, e_.cfg_.layers[i].act, st);
  }
  attention(i, r);
  launch_gemm_f32(cat32_, D.kout, w.out, D.kout, r.n, dp_, D.kout, x_, dp_, 1, st);
}

void LayeredDecoder::run(const RowSet& r) {
  launch_embed_pos(embd_, posw_, r.tokens, r.pos, r.n, dp_, x_, e_.stream_);
  norm_ready_ = false;
  for (int i = 0; i < nl_; ++i) {
    if (f32_) layer32(i, r);
    else layer16(i, r);
  }
}

void LayeredDecoder::decode_forward(int B) {
  RowSet r;
  r.tokens = e_.d_tokens_; r.pos = e_.d_pos_; r.slot = e_.d_slot_;
  r.n = r.n_abs = B;
  r.decode = true;
  r.max_len = e_.cfg_.max_ctx;
  run(r);
  // (the head reads the residual in place: the decode rows are x rows 0 .. B-1)
  std::swap(x_, xh_);
  head(B);
  std::swap(x_, xh_);
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
    if (q.n < pf_min_ || q.start + q.n > pf_max_ctx_) {
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
  int *ht = h_step_, *hp = ht + R, *hs = hp + R;
  LatentTile* tiles = (LatentTile*)(hs + 2 * R);
  int row = 0, nt = 0;
  for (int o = 0; o < (int)order.size(); ++o) {
    const Piece& q = pieces[order[o]];
    first_row[order[o]] = row;
    for (int k = 0; k < q.n; ++k) {
      ht[row + k] = q.tokens[k];
      hp[row + k] = q.start + k;
      hs[row + k] = q.slot;
    }
    if (o >= n_small) r.pf.push_back({row, q});
    row += q.n;
  }
  for (const Dims& D : dims_) {
    if (r.tiles.count(D.H)) continue;
    const int t0 = nt;
    for (int o = 0; o < n_small; ++o) {
      const int f0 = first_row[order[o]] * D.H, f1 = f0 + pieces[order[o]].n * D.H;
      for (int f = f0; f < f1; f += 16) tiles[nt++] = LatentTile{f, std::min(16, f1 - f)};
    }
    r.tiles[D.H] = {t0, nt - t0};
  }
  r.tokens = st_tokens_; r.pos = st_pos_; r.slot = st_slot_;
  HIP_CHECK(hipMemcpyAsync(d_step_, h_step_, ((size_t)4 * R + 2 * (size_t)nt) * 4, hipMemcpyHostToDevice, e_.stream_));
  run(r);
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
    launch_rmsnorm(x, dp_, out_norm_, h32_, dp_, B, d_, eps, st);
    launch_gemm_f32(h32_, dp_, headw_, dp_, B, vp_, dp_, y, vp_, 0, st);
    return;
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

std::vector<float> LayeredDecoder::residual(int rows) {
  std::vector<float> out((size_t)rows * d_);
  HIP_CHECK(hipStreamSynchronize(e_.stream_));
  HIP_CHECK(hipMemcpy2D(out.data(), (size_t)d_ * 4, x_, (size_t)dp_ * 4, (size_t)d_ * 4, rows, hipMemcpyDeviceToHost));
  return out;
}

}  // namespace aios
