// Decoders described layer by layer (EngineConfig::layers) instead of by one set of llama sizes.
//
// The Engine keeps what every model shares -- slots, the paged cache's tables and reference counts, the
// captured decode graphs, sampling, the step and decode entry points; a LayeredDecoder holds the
// layers' weights and cache pools and enqueues the forward pass of a set of rows.  A row is one token of
// one slot at one position, so a batch may mix portions of prompts and single decoded tokens.
#pragma once
#include <algorithm>
#include <map>
#include <set>
#include <string>
#include <vector>

#include "common.h"
#include "latent.h"
#include "mixers.h"
#include "ops.h"

namespace aios {

enum MixerKind : int { MIX_NONE = 0, MIX_LATENT = 1, MIX_MINGRU = 2, MIX_GQA = 3, MIX_MAMBA2 = 4, MIX_GLA = 5, MIX_DELTA = 6 };
enum MlpKind : int { MLP_NONE = 0, MLP_GLU = 1, MLP_MOE = 2, MLP_ACT = 3 };
enum OutGate : int { GATE_NONE = 0, GATE_ELEMENT = 1, GATE_HEAD = 2 };

// One layer: a mixer and a feed-forward.  Parallel: both read the same normalised input and are added to the
// residual together (x += mixer(norm(x)) + mlp(norm(x))).  Otherwise one after the other, each
//   x += post( f(h) * sigmoid(Wr h + br) ),  h = norm(x)
// with the gate (resid_gate) and the norm of the result (post_norm) where the layer has them.

// A linear recurrence (mixers.h LinScanArgs).
struct LinSpec {
  int heads = 1, groups = 1;           // groups: heads that share B and C (MIX_MAMBA2) or a query and a key (MIX_DELTA)
  int dim = 64, vdim = 64;             // state rows (key channels) and columns per head
  int conv = 4;                        // MIX_MAMBA2, MIX_DELTA: taps
  int norm_groups = 1;                 // MIX_MAMBA2: parts of the gated norm
  int rank = 8;                        // MIX_GLA: width of the decay's first projection
  double tau = 1.0;                    // MIX_GLA
};
struct LayerSpec {
  int mixer = MIX_LATENT;
  int parallel = 1;
  int norm_scalar = 0;                 // norms of the sublayers: one number instead of one per column
  int post_norm = 0, resid_gate = 0;
  // MIX_LATENT
  int heads = 1, dim = 64, vdim = 64;  // (unrotated) query-key and value dimensions per head
  int kv_rank = 64;                    // latent width
  int rot_dim = 0, rot_dims = 0;       // rotated query-key dimensions (0: none), the first rot_dims of which turn
  double rot_base = 10000.0;
  int window = 0;                      // keys a token sees, itself included (0: all before it)
  float scale = 0.125f;                // of q . k
  int sink = 1;                        // 1: a learned logit per head joins the softmax's denominator; 2 (MIX_GQA): the logit 0
  int out_gate = GATE_ELEMENT;         // head outputs times sigmoid(Wg h): a number each, or one per head
  // MIX_GQA: heads, dim, vdim, the first rot_dims dimensions turn (in halves), window, scale, sink, out_gate, and
  int kv_heads = 1;
  int chunk = 0;                       // keys before a token's chunk of so many positions are out (0: no chunks)
  float softcap = 0.f;                 // of the scores (0: none)
  int attn_bias = 0;                   // 1: biases of q, k, v and the output projection; 2: of q, k, v
  int qk_norm = 0;                     // RMS norm of all queries of a token at once, and of all keys, with weights
  int v_norm = 0;                      // RMS norm of every head's value, without weights
  int head_temp = 0;                   // a learned number per query head multiplies its scores
  // from the second layer with v_mix on: values (1 - lambda) v + lambda v_first, lambda learned, v_first the values of the
  // first such layer
  int v_mix = 0;
  // MIX_MINGRU
  int width = 64;                      // of the state
  // MIX_MAMBA2, MIX_GLA, MIX_DELTA
  LinSpec lin;
  // a second mixer that reads the same input (MIX_MAMBA2, MIX_GLA or MIX_DELTA, sizes in lin): mixer_scale * first + beside_scale *
  // second
  int beside = MIX_NONE;
  float mixer_scale = 1.f, beside_scale = 1.f;
  int mlp = MLP_GLU;
  int ff = 256;                        // MLP_GLU, MLP_ACT: hidden width; MLP_MOE: of every expert
  int act = ACT_GELU_TANH;             // GluAct of the gate; MLP_ACT: of the hidden layer
  int mlp_bias = 0;                    // MLP_ACT
  float mlp_scale = 1.f;               // MLP_ACT: of the result
  int experts = 0, top = 0;            // MLP_MOE
  int shared_ff = 0;                   // hidden width of the expert that runs for every token (0: none)
  int correction = 0;                  // a learned number per expert joins the choice, not the weights
  float router_scale = 1.f;
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
  bool recurrent() const { return recurrent_; }        // a slot's state is more than its cached tokens
  void copy_state(int src, int dst);                   // recurrent state and last tokens of a slot
  int layer_runs() const { return (int)runs_.size(); }
  void set_run_limit(int n) { run_limit_ = n; }        // stop after n layer runs (n < 0: all)

 private:
  struct Dims {
    // latent attention; padded: dkp, dvp, rp.  A head's query is [dk | rotated at qrot], the cached row
    // [latent | rotated at roff]; qn / gn: rows of all heads' queries / values (gn: columns the mixer leaves)
    int H, dk, dv, rank, rot, qrot, roff, dkp, dvp, rp, qn, gn;
    int wp;                   // minGRU: padded width
    int G, koff, voff;        // grouped-query attention: key / value heads, their columns (q at 0)
    // linear recurrence: kind (0: none), heads, groups, state rows and columns (padded: np, vp), its columns in the
    // input product and in the joint output matrix
    int lin, lH, lG, lN, lnp, ldv, lvp, lin_off, lin_out;
    int ff, fp, shf, shp;     // feed-forward and shared expert, padded
    int gate_off, rg_off;     // columns of the output gate and of the residual gate in the input product
    int n1;                   // input product without gate / up
    int nin, kout;            // parallel: with gate / up; columns of the joint output matrix
    int n2, router_off, glu;  // sequential: the feed-forward's input product [residual gate | router], GLU width (padded)
  };
  struct Weights {
    bool own = false;
    float *norm = nullptr, *norm2 = nullptr, *post = nullptr, *post2 = nullptr, *kv_norm = nullptr, *sink = nullptr;
    float *rgb = nullptr, *rgb2 = nullptr, *zb = nullptr, *ub = nullptr, *corr = nullptr;
    bf16_t *in = nullptr;    // parallel [nin][dp]: q | kv down | output gate | gate / up interleaved
                             // sequential [n1][dp]: q | kv down | output gate | residual gate, or z | u | g | residual gate
    bf16_t *out = nullptr;   // [dp][kout]: attention output | MLP down; sequential [dp][gn]
    bf16_t *in2 = nullptr;   // [n2 + 2 glu][dp]: residual gate | router | gate / up interleaved
    bf16_t *out2 = nullptr;  // [dp][glu]
    bf16_t *egu = nullptr;   // [experts][2 fp][dp] gate / up interleaved
    bf16_t *edn = nullptr;   // [experts][dp][fp]
    bf16_t *ukv = nullptr;   // [qn + gn][rp]: key | value up-projections
    bf16_t *ukT = nullptr;   // [H][rp][dkp]
    // biases: q, k, v, output projection (times mixer_scale), MLP up and down
    float *qb = nullptr, *kb = nullptr, *vb = nullptr, *ob = nullptr, *upb = nullptr, *dnb = nullptr;
    // linear recurrence (mixers.h LinScanArgs)
    float *qn = nullptr, *kn = nullptr, *temp = nullptr, *lambda = nullptr;  // grouped-query attention's norms and numbers
    ActNum act_n{0.f, 0.f, 1.f};
    float *conv_w = nullptr, *conv_b = nullptr, *dt_b = nullptr, *a_log = nullptr, *lin_d = nullptr, *lin_norm = nullptr,
          *a2 = nullptr, *a2_b = nullptr;
  };
  // one pass of one layer; a looped layer has a cache or state per pass
  struct Run {
    int layer, pass;         // pass: -1 outside the loop
    char* pool;              // cache (attention)
    float* state;            // [2][slots][state numbers]
    float* ring;             // [slots][taps][columns]: the convolution's last inputs
  };
  struct RowSet {
    const int *tokens, *pos, *slot, *run;  // run: rows of the sequence from its first row (null: one each)
    int n, n_abs;                         // rows, rows on the absorbed path (they come first)
    bool decode;
    std::map<int, std::pair<int, int>> tiles;  // step batches: heads -> (first tile, count)
    int max_len;                          // of the absorbed rows
    std::vector<std::pair<int, Piece>> pf;  // expanded path: first row, piece
    int n_chunks, split, n_seqs;          // step batches: chunks of the recurrences, pieces
    int longest;                          // tokens of the longest piece
  };
  void layer16(int k, const RowSet& r);  // k: run
  void layer32(int k, const RowSet& r);
  void layer_seq(int k, const RowSet& r);
  // few rows: norms in the products that read the residual, sums and biases in those that add to it
  void layer_fused(int k, const RowSet& r);
  bool fused(int n) const { return plain_ && (n <= 4 ? (bool)gemv_ok_[n] : n <= 64 && nparts_ > 0); }
  const Weights& weights(int k) const { return w_[owner_[runs_[k].layer]]; }
  void feed_forward(int k, const RowSet& r, RowCloseArgs& c);
  void recurrence(int k, const RowSet& r);
  void linear(int k, const RowSet& r);
  void grouped_attention(int k, const RowSet& r);
  size_t state_floats(int i) const;      // of one slot and parity
  size_t ring_floats(int i) const;       // of one slot
  bool enters_pass(int k) const;         // run k begins a pass but the first, entered by adding the embedding
  void attention(int k, const RowSet& r);
  void run(const RowSet& r);
  NextArgs next_of(int k, bool decode);  // what the residual becomes before run k (the head's input after the last)
  RowCloseArgs close_args() const;
  LatentAttnArgs latent_args(int k, const RowSet& r);
  int runs_to_do() const { return run_limit_ < 0 ? (int)runs_.size() : std::min(run_limit_, (int)runs_.size()); }
  // y[n][N] (ldy) = operand rows x w^T, through the GEMV, the short or the prefill GEMM
  void project(const void* a, int lda, const bf16_t* w, int n, int N, int K, float* y, int ldy);
  void alloc_layer(int i);
  std::vector<float> rope_table(int rot, int dims, double base) const;
  int span(const Piece& p) const;        // keys the expanded path of a piece needs at most
  QWeight mat(const bf16_t* p, int rows, int cols) const;
  void gemm16(const bf16_t* A, int lda, const bf16_t* w, int M, int N, int K, int epi, float* C, int ldc, bf16_t* C16,
              int act = 0);
  bool gemv_fits(int i, int B);
  int key_split(int tiles, int max_len) const;
  bf16_t* balloc(size_t n);
  float* falloc(size_t n);
  void place(bf16_t* dst, int dpitch, const bf16_t* src, int spitch, int width, int height, bool device);
  void put(const std::string& name, int rows, int cols, const bf16_t* src, bool device);
  void put_vec(float* dst, int n, const bf16_t* src, bool device, int spread = 0, float mul = 1.f);
  void list_tensors();
  void tune();

  Engine& e_;
  int nl_, d_, dp_, v_, vp_, f32_;
  std::vector<Dims> dims_;
  std::vector<int> owner_;
  std::vector<Weights> w_;
  std::vector<Run> runs_;
  bool plain_ = false;  // 16-bit sequential layers that add a sublayer's result as it is
  bool seq_ = false, recurrent_ = false, head_ready_ = false;
  int run_limit_ = -1, max_window_ = 0;  // max_window_: largest window, 0 if a layer has none
  bf16_t *embd_ = nullptr, *posw_ = nullptr, *headw_ = nullptr, *pairw_ = nullptr, *loopw_ = nullptr;
  float *out_norm_ = nullptr, *loop_step_ = nullptr, *x0_ = nullptr;  // x0_: embedding rows (loops that add them)
  std::vector<float2*> rope_;            // per layer
  float* v_first_ = nullptr;             // [rows][G dv] values of the first layer that mixes them (v_first_layer_; -1: none)
  int v_first_layer_ = -1;
  const float* zero_sink_ = nullptr;     // [heads] zeros
  int* last_tok_ = nullptr;              // [2][slots]
  std::vector<std::pair<std::string, std::pair<int, int>>> tensors_;  // name, (rows, columns)
  std::map<std::string, std::pair<int, int>> shape_;
  std::set<std::string> have_;

  int step_rows_ = 0, pf_min_ = 0, pf_max_ctx_ = 0;
  std::vector<char> gemv_ok_;  // [5]: batch b goes through the GEMV engine
  float *x_ = nullptr, *xh_ = nullptr, *qdg_ = nullptr, *opart_ = nullptr, *ml_ = nullptr, *h32_ = nullptr, *gu32_ = nullptr,
        *cat32_ = nullptr;
  bf16_t *h16_ = nullptr, *cat16_ = nullptr, *cfull_ = nullptr, *kv_ = nullptr;
  void* qa_ = nullptr;
  // sequential layers: sublayer result, loop entry operand [rows][2 dp], recurrences' chunk transitions, experts
  float *y_ = nullptr, *agg_ = nullptr, *moe_wt_ = nullptr, *moe_gu32_ = nullptr;
  void *xin_ = nullptr, *moe_act_ = nullptr, *moe_ye_ = nullptr;
  int *moe_sel_ = nullptr, *moe_pair_ = nullptr, *moe_token_ = nullptr, *moe_ntiles_ = nullptr;
  int4* moe_tiles_ = nullptr;
  // linear recurrences: operands of the blocks, outputs before the norm
  void *lin_qo_ = nullptr, *lin_ko_ = nullptr, *lin_kr_ = nullptr, *lin_vo_ = nullptr, *lin_so_ = nullptr;
  float *lin_dec_ = nullptr, *lin_y_ = nullptr, *lin_seg_ = nullptr, *lin_seg_dec_ = nullptr;
  int moe_max_tiles_ = 0;
  // RMSNorm split across the short GEMMs (GemmQArgs nrm_*): set when the residual in x_ already went
  // through bf16(x * g_next) and per-tile sums
  bf16_t* xn16_ = nullptr;
  float* npart_ = nullptr;
  int nparts_ = 0;
  bool norm_ready_ = false;
  // step parameters: one pinned block, one copy
  int *h_step_ = nullptr, *d_step_ = nullptr;
  size_t step_ints_ = 0;
  int *st_tokens_ = nullptr, *st_pos_ = nullptr, *st_slot_ = nullptr, *st_want_ = nullptr, *st_run_ = nullptr;
  ScanChunk* st_chunks_ = nullptr;
  ScanSeq* st_seqs_ = nullptr;
  int max_chunks_ = 0;
  LatentTile* st_tiles_ = nullptr;
};

}  // namespace aios
