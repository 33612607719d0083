// Launchers of the layered decoders' mechanisms beside latent attention (latent.h): embedding rows, the
// closing of a sublayer, gated recurrences, mixtures of experts.  Rows are tokens of any sequences; all
// row lengths are padded with zeros to whole 64-column tiles, norms divide by the true width.
#pragma once
#include "latent.h"
#include "ops.h"

namespace aios {

// ---- row operations (kernels/rowops.hip) ----------------------------------------------------------
// What a row's new residual becomes for the next product: its RMS norm, or the residual itself.
enum NextOperand : int { NEXT_NONE = 0, NEXT_NORM = 1, NEXT_RAW = 2 };
struct NextArgs {
  int kind = NEXT_NONE;
  const float* g = nullptr;  // [dp] norm weight (NEXT_NORM)
  void* out = nullptr;       // [rows][ldo], bf16 or fp32
  int ldo = 0;
};

struct EmbedArgs {
  const bf16_t* table;        // [vocab][dp]
  float scale;                // of the token embedding
  const bf16_t* pos_table;    // [positions][dp] or null
  const bf16_t* pair_table;   // [buckets + 1][dp] or null: row (previous * mul_prev + token * mul_cur) mod buckets,
  int buckets;                //   the last row for a sequence's first token
  long long mul_prev, mul_cur;
  const int *tokens, *pos, *slot;  // [rows]
  // rows of one sequence are consecutive: run[i] > 0 marks its first row and counts its rows; null: one row each
  const int* run;
  // last token of every slot, by parity of its position [2][slots]: a step that is run again (same position)
  // still finds its predecessor
  int* last;
  int slots;
  int dp, d;
  float eps;
  float* x;                   // [rows][dp]
  void* keep;                 // the embedding for later passes, bf16 or fp32, or null
  int ld_keep;
  float* keep32;              // the same in fp32 [rows][dp], or null
  int f32;
  NextArgs next;
};
void launch_embed_rows(const EmbedArgs& a, int rows, hipStream_t st);

// Closes a sublayer: v = y + y_bias (+ the weighted expert rows); v *= sigmoid(gate + bias); v = rms(v) * post;
// x += v (+ rows of its own, extra) -- or, replacing the residual (loop entry), x = y + add -- and the next
// operand, in one pass.
struct RowCloseArgs {
  float* x;                   // [rows][dp]
  int dp, d;
  float eps;
  const float* y;             // [rows][dp] or null
  const float* y_bias;        // [dp] or null
  const float* extra;         // [rows][dp] or null: added to the new residual
  const void* ye;             // [pairs][dp] expert outputs (bf16 or fp32) or null
  const int* pair;            // [rows][top] row in ye
  const float* wt;            // [rows][top] weight
  int top;
  const float* gate;          // [rows][ldg] pre-activation or null
  int ldg;
  const float* gate_bias;     // [dp] or null
  const float* post;          // [dp] norm weight or null (no norm)
  int replace;
  const float* add;           // [dp] (replace)
  int f32;                    // operands (ye, next.out) in fp32
  NextArgs next;
};
void launch_row_close(const RowCloseArgs& a, int rows, hipStream_t st);

// ---- minGRU (kernels/recurrent.hip) ---------------------------------------------------------------
// S_t = (1 - f) S_{t-1} + f c with f = sigmoid(z_t), c = u_t + 1/2 (u_t >= 0) or sigmoid(u_t) (u_t < 0), element
// by element in fp32; out_t = S_t * silu(g_t).  Portions are scanned in chunks of SCAN_CHUNK tokens side by
// side.  The state is kept twice, by parity of the position it was left at: a single token that is run again
// at the same position reads the same state.
constexpr int SCAN_CHUNK = 32;
struct ScanChunk {
  int row0, n;      // rows of the step
  int slot, pos0;   // position of row0
  int first;        // index of the sequence's first chunk
  int last;         // 1: leaves the state
};
struct MinGruArgs {
  const float* in;            // [rows][ld]: z, u, g at their offsets
  int ld, z_off, u_off, g_off;
  const float *zb, *ub;       // [w] biases
  int w;                      // width (a multiple of 64)
  float* state;               // [2][slots][w]
  int slots;
  const ScanChunk* chunks;    // null: row i is one token of slot[i] at pos[i]
  const int *pos, *slot;
  int n;                      // chunks (or rows)
  int split;                  // some sequence has more than one chunk
  float* agg;                 // [chunks][3][w] (split)
  void* out;                  // [rows][ldo] bf16 or fp32
  int ldo, f32;
};
void launch_mingru(const MinGruArgs& a, hipStream_t st);

// ---- grouped-query attention (kernels/gqa.hip) ------------------------------------------------------
// Query head h reads key / value head h / (H / G).  Keys and values are cached per block of GQA_BLOCK tokens as
// [G][block][dkp] keys, then [G][block][dvp] values.  Head sizes are padded to dkp / dvp (multiples of 32) there and in
// q; the input product's columns are not.  Rotation turns the pairs (i, i + rot / 2) of a head's first rot dimensions.
//   s = q . k * scale * temp_h;  s = softcap tanh(s / softcap) (softcap > 0);  weights exp(s) / (exp(sink_h) + sum exp(s)) over
//   the visible keys;  out_h = out_scale * sigmoid(gate_h) * sum weights v
// Before the rotation q and k may be divided by the root mean square of all their heads' columns together and multiplied by
// weights (qn, kn); v may be divided, head by head, by its own (v_norm), and then mixed with another layer's values of the
// same token (lambda).
// A query at position i sees keys j <= i with j > i - window (window > 0) and floor(j / chunk) = floor(i / chunk)
// (chunk > 0).
constexpr int GQA_BLOCK = 64;
struct GqaArgs {
  int rows;                   // rows of the step
  int n;                      // rows [0, n) take launch_gqa_attn
  int H, G, dk, dkp, dv, dvp;
  int rot;                    // even; (cos, sin) of pair i at position p: rope[p * rot / 2 + i]
  const float2* rope;
  int window, chunk;
  float scale, softcap;
  const float* sink;          // [H] or null
  const float *qb, *kb, *vb;  // biases of q [H dk], k [G dk], v [G dv], or null
  const float *qn, *kn;       // [H dk], [G dk] norm weights, or null
  const float* temp;          // [H] or null
  int v_norm;
  float eps;                  // of these norms
  float* first;               // [rows][G dv] or null: values kept for later layers, or (lambda set) those of that layer
  const float* lambda;        // one number or null: v = (1 - lambda) v + lambda first
  const float* in;            // [rows][ld]: q, k, v at their offsets, gates at g_off + h (g_off -1: none)
  int ld, q_off, k_off, v_off, g_off;
  float out_scale;
  const int *pos, *slot;      // [rows]
  void* pool;                 // bf16 or fp32 (f32)
  const int* bt;              // [slots][maxb]
  int maxb, f32;
  void* q;                    // [rows][H dkp]: rotated queries; bf16 (the score's factor folded in) or fp32
  // flat rows [f0, f0 + nv) of the [row][query head of one kv head] space, one sequence each; null: every row its own
  const LatentTile* tiles;
  int n_tiles, nsplit;        // key splits (at most 64)
  float* opart;               // [nsplit][n * H][dvp]
  float* ml;                  // [nsplit][n * H][2]
  void* out;                  // [rows][ldo], head h at h * dvp, bf16 or fp32
  int ldo;
};
inline size_t gqa_block_elems(int G, int dkp, int dvp) { return (size_t)G * GQA_BLOCK * (dkp + dvp); }
// factor of q . k folded into the bf16 queries
float gqa_q_factor(float scale, float softcap);
void launch_gqa_prep(const GqaArgs& a, hipStream_t st);  // queries; keys and values into the cache
void launch_gqa_attn(const GqaArgs& a, hipStream_t st);
bool gqa_supports(int dkp, int dvp);

// ---- linear recurrences with a matrix state (kernels/linear_scan.hip) ----------------------------------
// Per head, S [N][dv] in fp32:  S_t = d_t S_{t-1} + k_t v_t^T,  o_t = S_t^T q_t.
//   LIN_HEAD  d_t one number per head (state-space duality).  x, B, C: a causal convolution per channel and SiLU of the
//             input columns [x: H dv | B: G N | C: G N];  dt = softplus(in + dt_b);  d = exp(-exp(a_log) dt),
//             k = dt B, q = C (group h / (H / G)), v = x;  y = o + D x.  out = rms over norm_parts equal parts of
//             (y silu(z)) * norm_w [H dv].
//   LIN_KEY   d_t one number per key channel (gated linear attention): d = sigmoid(a2 a + a2_b)^(1 / tau), k and v
//             the input columns, q times q_scale (G = H).  out = rms(o) per head * norm_w [dv] * silu(z).
//   LIN_DELTA d_t one number per head, as LIN_HEAD's; the convolved columns are v, k, q (group h / (H / G)), k and q made
//             unit vectors, q times q_scale.  b_t = sigmoid(in), and instead of v_t the state takes
//             u_t = b_t (v_t - d_t S_{t-1}^T k_t).  out as LIN_KEY's.
// Portions run in blocks of LIN_T tokens: what a block needs besides the state it starts from (operands, decays,
// scores between its own tokens) is prepared for all blocks side by side; then one wave per head and 16 columns of
// v walks the blocks with its part of S in registers, long portions in segments side by side.  The state is kept twice, by parity of the position it was left
// at, and the convolution's inputs in a ring of `taps` positions, so that a single token that is run again at the
// same position finds what it started from.
enum LinKind : int { LIN_HEAD = 1, LIN_KEY = 2, LIN_DELTA = 3 };
constexpr float LIN_UNIT_EPS = 1e-6f;  // of the unit vectors, beside the sum of squares
constexpr int LIN_T = 16;
constexpr int LIN_SEGS = 16, LIN_SEG_MIN = 8;  // segments of a step at most; blocks of a segment at least
struct ScanSeq {
  int row0, n, slot, pos0;
  int b0;           // index of its first block in the operand buffers
};
struct LinScanArgs {
  int kind;
  int H, G, N, np, dv, vp;    // np, vp: N and dv padded (lin_pad_n, multiple of 16)
  const float* in;            // [rows][ld] input product
  int ld, z_off;              // output gate [H dv]
  int x_off, taps, dt_off;    // LIN_HEAD, LIN_DELTA: convolved columns, step sizes [H]
  int b_off;                  // LIN_DELTA: strengths [H]
  const float *conv_w, *conv_b;        // [H dv + 2 G N][taps], last tap the current token's; bias or null
  const float *dt_b, *a_log, *D;       // [H]
  float* ring;                // [slots][taps][H dv + 2 G N]
  int q_off, k_off, v_off, a_off, rank;  // LIN_KEY
  float q_scale, inv_tau;
  const float *a2, *a2_b;     // [H N][rank], [H N]
  float* state;               // [2][slots][H][np][vp]
  int slots;
  // portions (seqs, and chunks: the same tokens in SCAN_CHUNK pieces); or n single tokens (pos, slot)
  const ScanSeq* seqs;
  int n_seqs;
  const ScanChunk* chunks;
  int n_chunks;
  const int *pos, *slot;
  int n;
  // operands of the blocks (bf16 or fp32), see lin_ws
  void *qo, *ko, *kr, *vo, *so;
  float* dec;
  int nseg;                   // segments a portion is walked in (lin_segments); more than 1: the states and decays at
  float *seg, *seg_dec;       // their borders, [n_seqs][nseg][H] x [np][vp] and x [np]
  float* y;                   // [rows][H dv]
  const float* norm_w;
  int norm_parts;
  float eps, out_scale;
  int rows;
  void* out;                  // [rows][ldo], bf16 or fp32
  int ldo, f32;
};
int lin_pad_n(int n);                                // 0: not served
struct LinWs { size_t qo, ko, kr, vo, so, dec; };    // numbers per block
int lin_segments(int kind, int H, int np, int vp, int n_seqs, int blocks);  // blocks: of the longest portion
LinWs lin_ws(int kind, int H, int G, int np, int vp, bool f32);
void launch_lin_scan(const LinScanArgs& a, hipStream_t st);

// y[r][i] = act(x[r][i] + bias[i]) in fp32
void launch_bias_act_f32(const float* x, int ldx, const float* bias, float* y, int ldy, int rows, int n, int act, const ActNum& num,
                         hipStream_t st);

// ---- mixture of experts (kernels/moe.hip) -----------------------------------------------------------
// Router: s = softmax(logits), the `top` largest of s + correction, weights s * scale.  The (token, expert) pairs
// are ordered by expert and every expert's rows go through its gate / up and down matrices; sums over a
// token's experts are taken in launch_row_close (or, for few tokens, in launch_moe_few).
constexpr int MOE_MAX_EXPERTS = 1024, MOE_MAX_TOP = 32;
struct MoeArgs {
  int n;                      // tokens
  int experts, top;
  float scale;
  const float* logits;        // [n][ldl]
  int ldl;
  const float* corr;          // [experts] or null
  int dp, ff, act;            // width, expert width (multiples of 64), gate activation
  const void* h;              // [n][ldh] normalised input, bf16 or fp32
  int ldh;
  const bf16_t* wgu;          // [experts][2 ff][dp] gate / up interleaved
  const bf16_t* wdn;          // [experts][dp][ff]
  int* sel;                   // [n][top]
  float* wt;                  // [n][top]
  int* pair;                  // [n][top] row in expert order
  int* token;                 // [n * top] token of that row
  int4* tiles;                // {expert, first row, rows, first tile of the expert | tiles of it << 16}; count in n_tiles
  int* n_tiles;
  int max_tiles;
  void* act_out;              // [n * top][ff] bf16 or fp32
  void* ye;                   // [n * top][dp] bf16 or fp32
  float* gu32;                // [n * top][2 ff] (f32)
  int f32;
  // launch_moe_few: a shared expert's activation and down matrix [dp][sh_ff] join the sum (or null)
  const bf16_t* sh_act;
  int ld_sh, sh_ff;
  const bf16_t* sh_dn;
  float* y;                   // [n][dp]
};
constexpr int MOE_FEW = 4;    // tokens up to which every (token, expert) pair is its own product
bool moe_few_fits(const MoeArgs& a);                 // launch_moe_few takes these
int moe_tile_rows(int n, int top, int experts);      // rows per tile the grouped path uses
int moe_max_tiles(int n, int top, int experts);      // bound of the tile count
void launch_moe_grouped(const MoeArgs& a, hipStream_t st);  // routing, grouping, experts -> ye
void launch_moe_few(const MoeArgs& a, hipStream_t st);      // few tokens, bf16: routing, experts, weighted sum -> y

}  // namespace aios
