// Decoders described layer by layer (EngineConfig::layers) instead of by one set of llama sizes.
//
// The Engine keeps what every model shares -- slots, the paged cache's tables and reference counts, the
// captured decode graphs, sampling, the step and decode entry points; a LayeredDecoder holds the
// layers' weights and cache pools and enqueues the forward pass of a set of rows.  A row is one token of
// one slot at one position, so a batch may mix portions of prompts and single decoded tokens.
#pragma once
#include <map>
#include <set>
#include <string>
#include <vector>

#include "common.h"
#include "latent.h"
#include "ops.h"

namespace aios {

enum MixerKind : int { MIX_LATENT = 1 };
enum MlpKind : int { MLP_NONE = 0, MLP_GLU = 1 };

// One layer: a mixer and a feed-forward that read the same normalised input and are added to the
// residual together (x += mixer(norm(x)) + mlp(norm(x))).
struct LayerSpec {
  int mixer = MIX_LATENT;
  int heads = 1, dim = 64, vdim = 64;  // query-key and value dimensions per head
  int kv_rank = 64;                    // latent width (MIX_LATENT)
  float scale = 0.125f;                // of q . k
  int sink = 1;                        // a learned logit per head joins the softmax's denominator
  int out_gate = 1;                    // head outputs times sigmoid(Wg h)
  int mlp = MLP_GLU;
  int ff = 256;
  int act = ACT_GELU_TANH;             // GluAct of the gate
  int weights_of = -1;                 // layer whose weights this one uses (its cache is its own), or -1
};

class Engine;

class LayeredDecoder {
 public:
  explicit LayeredDecoder(Engine& e);
  ~LayeredDecoder();

  void set_tensor(const std::string& name, int qt, int rows, int cols, const void* host, size_t nbytes);
  void init_random(uint64_t seed);
  std::vector<std::string> missing() const;
  void finalize();

  int logits_ld() const { return vp_; }
  int step_rows() const { return step_rows_; }
  // enqueue the forward of the decode batch's B rows (device parameter arrays; capturable) to the logits
  void decode_forward(int B);

  // rows of one forward pass: entry e's tokens at positions [start, start + n) of its slot
  struct Piece {
    int slot, start, n;
    const int* tokens;  // host
  };
  // enqueue the forward of these pieces (at most step_rows() rows together); x row of piece p's i-th token
  // is first_row[p] + i afterwards
  void forward(const std::vector<Piece>& pieces, std::vector<int>& first_row);
  // logits of x rows `rows` (<= max_batch) into logits rows [0, rows.size()); keep: rows gathered earlier
  // by collect() instead
  void collect(const std::vector<int>& rows, int at);  // x rows -> head input rows [at, ...)
  void head(int B, int from = 0);                      // logits of head input rows [from, from + B)
  std::vector<float> residual(int rows);               // host copy of x rows [0, rows), width columns

 private:
  struct Dims {
    int H, dk, dv, rank, ff;
    int dkp, dvp, rp, qn, gn, fp;  // padded; qn / gn: rows of all heads' queries / values
    int n1, nin, kout;             // input projections without / with gate and up; columns of the output matrix
  };
  struct Weights {
    bool own = false;
    float *norm = nullptr, *kv_norm = nullptr, *sink = nullptr;
    bf16_t *in = nullptr;    // [nin][dp]: q | kv down | output gate | gate / up interleaved
    bf16_t *out = nullptr;   // [dp][kout]: attention output | MLP down
    bf16_t *ukv = nullptr;   // [qn + gn][rp]: key | value up-projections
    bf16_t *ukT = nullptr;   // [H][rp][dkp]
  };
  struct RowSet {
    const int *tokens, *pos, *slot;
    int n, n_abs;                         // rows, rows on the absorbed path (they come first)
    bool decode;
    std::map<int, std::pair<int, int>> tiles;  // step batches: heads -> (first tile, count)
    int max_len;                          // of the absorbed rows
    std::vector<std::pair<int, Piece>> pf;  // expanded path: first row, piece
  };
  void layer(int i, const RowSet& r);
  void layer16(int i, const RowSet& r);
  void layer32(int i, const RowSet& r);
  void attention(int i, const RowSet& r);
  void run(const RowSet& r);
  LatentAttnArgs latent_args(int i, const RowSet& r);
  QWeight mat(const bf16_t* p, int rows, int cols) const;
  void gemm16(const bf16_t* A, int lda, const bf16_t* w, int M, int N, int K, int epi, float* C, int ldc, bf16_t* C16,
              int act = 0);
  bool gemv_fits(int i, int B);
  int key_split(int tiles, int max_len) const;
  bf16_t* balloc(size_t n);
  float* falloc(size_t n);
  void place(bf16_t* dst, int dpitch, const bf16_t* src, int spitch, int width, int height, bool device);
  void put(const std::string& name, int rows, int cols, const bf16_t* src, bool device);
  void put_vec(float* dst, int n, const bf16_t* src, bool device);
  std::vector<std::pair<std::string, std::pair<int, int>>> tensor_list() const;
  void tune();

  Engine& e_;
  int nl_, d_, dp_, v_, vp_, f32_;
  std::vector<Dims> dims_;
  std::vector<int> owner_;
  std::vector<Weights> w_;
  std::vector<char*> pool_;
  bf16_t *embd_ = nullptr, *posw_ = nullptr, *headw_ = nullptr;
  float* out_norm_ = nullptr;
  std::set<std::string> have_;

  int step_rows_ = 0, pf_min_ = 0, pf_max_ctx_ = 0;
  std::vector<char> gemv_ok_;  // [5]: batch b goes through the GEMV engine
  float *x_ = nullptr, *xh_ = nullptr, *qdg_ = nullptr, *opart_ = nullptr, *ml_ = nullptr, *h32_ = nullptr, *gu32_ = nullptr,
        *cat32_ = nullptr;
  bf16_t *h16_ = nullptr, *cat16_ = nullptr, *cfull_ = nullptr, *kv_ = nullptr;
  void* qa_ = nullptr;
  // RMSNorm split across the short GEMMs (GemmQArgs nrm_*): set when the residual in x_ already went
  // through bf16(x * g_next) and per-tile sums
  bf16_t* xn16_ = nullptr;
  float* npart_ = nullptr;
  int nparts_ = 0;
  bool norm_ready_ = false;
  // step parameters: one pinned block, one copy
  int *h_step_ = nullptr, *d_step_ = nullptr;
  size_t step_ints_ = 0;
  int *st_tokens_ = nullptr, *st_pos_ = nullptr, *st_slot_ = nullptr, *st_want_ = nullptr;
  LatentTile* st_tiles_ = nullptr;
};

}  // namespace aios
