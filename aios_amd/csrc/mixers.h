// Launchers of the layered decoders' mechanisms beside latent attention (latent.h): embedding rows, the
// closing of a sublayer, gated recurrences, mixtures of experts.  Rows are tokens of any sequences; all
// row lengths are padded with zeros to whole 64-column tiles, norms divide by the true width.
#pragma once
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
  int f32;
  NextArgs next;
};
void launch_embed_rows(const EmbedArgs& a, int rows, hipStream_t st);

// Closes a sublayer: v = y (+ the weighted expert rows); v *= sigmoid(gate + bias); v = rms(v) * post;
// x += v -- or, replacing the residual (loop entry), x = y + add -- and the next operand, in one pass.
struct RowCloseArgs {
  float* x;                   // [rows][dp]
  int dp, d;
  float eps;
  const float* y;             // [rows][dp] or null
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
