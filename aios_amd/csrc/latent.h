// Launchers of the latent-attention kernels (kernels/latent.hip, kernels/attention_mha.hip) and of the
// 32-bit matrix product (kernels/gemm_f32.hip).
//
// Latent attention caches one vector c per token (its normalised down-projection, `rank` numbers)
// instead of keys and values: k_h = Wuk_h c and v_h = Wuv_h c for every head h.  Two equivalent forms:
//   absorbed  score = (Wuk_h^T q_h) . c and o_h = Wuv_h (sum_s p_s c_s): reads only c, for rows with few
//             new tokens per sequence (decode, short portions);
//   expanded  k and v of the whole context are computed once per call and a flash attention runs on
//             them: fewer operations per (query, key) pair, for long portions of a prompt.
// A key may have a second, rotated part that all heads share (rot numbers per token, cached beside c).  The cached
// row is then [c | rotated part] and a head's query [unrotated | rotated]: with the identity as the rotated
// rows of Wuk, both forms serve it as a longer latent, and the value product has zeros there.
// Every head dimension is padded with zeros: dkp / dvp (query-key / value) to multiples of 32, the cached
// row to rp, a multiple of 128, so the kernels have no ragged dimension.
#pragma once
#include "ops.h"

namespace aios {

// query rows (a row = one head of one token) of one sequence: flat rows [f0, f0 + nv) of the flattened
// [token][head] row space, nv <= 16
struct LatentTile {
  int f0, nv;
};

struct LatentAttnArgs {
  int n;                       // tokens on the absorbed path: rows [0, n) of the step
  int H, dk, dkp, dvp, rank, rp;
  // rotated part: rot numbers (even; 0: none) at column roff of the cached row and of the kv down-projection, and at
  // qrot of a head's query (both multiples of 8); pairs (2 i, 2 i + 1) turn by the angle whose (cos, sin) is
  // rope[pos * rot / 2 + i]
  int rot, roff, qrot;
  const float2* rope;
  int window;                  // keys a query sees, itself included (0: all before it)
  int head_gate;               // the output gate has one number per head (column g_off + head)
  float scale;                 // of q . k
  float eps;                   // of the latent's RMS norm
  const float* norm_w;         // [rp] weight of the latent's RMS norm (zero beyond rank)
  const float* sink;           // [H] logit that only joins the softmax's denominator, or null
  const float* qdg;            // [rows][ld]: q at column 0 (H x dkp), dkv at dkv_off, output gate at g_off (-1: none)
  int ld, dkv_off, g_off;
  const int *pos, *slot;       // [rows]
  // paged cache of c: [blocks][kvb][rp], bf16 or fp32 (f32); table [slots][maxb]
  void* pool;
  const int* bt;
  int maxb, kvb, f32;
  const bf16_t* wukT;          // [H][rp][dkp]
  const bf16_t* wuv;           // [H][dvp][rp]
  void* qa;                    // absorbed queries [n][H][rp], bf16 or fp32
  const LatentTile* tiles;     // null: every token is its own sequence (decode)
  int n_tiles, nsplit;
  float* opart;                // [nsplit][n * H][rp] unnormalised partial sums
  float* ml;                   // [nsplit][n * H][2]: running maximum (log2 domain) and sum
  void* out;                   // [rows][ldo] head outputs (gated), bf16 or fp32
  int ldo;
};
// c of every row of the step into the cache (rows [0, rows)), and the absorbed queries of rows [0, n)
void launch_latent_prep(const LatentAttnArgs& a, int rows, hipStream_t st);
// attention of the absorbed rows over their cached context, split over the keys
void launch_latent_attn(const LatentAttnArgs& a, hipStream_t st);
// partial sums -> softmax normalisation with the sink, Wuv, output gate
void launch_latent_out(const LatentAttnArgs& a, hipStream_t st);
bool latent_attn_mfma(int rp);  // the matrix-core kernels serve this padded rank (else the plain one, rank <= 2048)

// S cached vectors of a slot from position k0, contiguous: out [S][rp] (bf16 cache)
void launch_latent_gather(const bf16_t* pool, const int* bt, int maxb, int kvb, int slot, int k0, int S, int rp, bf16_t* out,
                          hipStream_t st);

// causal flash attention of one sequence's T new tokens at positions [start, start + T) over contiguous
// per-head keys and values [0, start + T), with a sink and an output gate
// paged (pool set): keys and values from the blocks of grouped-query attention's cache (mixers.h GqaArgs), whose
// positions are the sequence's; queries q16 with the score's factor folded in
struct MhaPrefillArgs {
  const float* q;        // [T][ldq], head h at h * dkp
  const bf16_t* q16;     // paged: [T][H dkp]
  const bf16_t* pool;
  const int* bt;         // paged: block table of the sequence
  int G;                 // paged: key / value heads
  int chunk;             // paged: keys before the query's chunk of this many positions are out (0: none)
  float softcap, out_scale;  // paged
  int ldq;
  const bf16_t *k, *v;   // [S][ldkv]: key of head h at k + h * dkp, value at v + h * dvp
  int ldkv;
  int H, dkp, dvp;
  int start, T;
  int window;            // keys a query sees, itself included (0: all before it)
  int rot, qrot, pos0;   // rotated part of the queries (LatentAttnArgs); position of the first new token
  const float2* rope;
  float scale;
  const float* sink;     // [H] or null
  const float* gate;     // [T][ldq] (paged: ldq of the gate alone), head h at h * dvp (head_gate: at h): the output times sigmoid(gate); or null
  int head_gate;
  bf16_t* out;           // [T][ldo], head h at h * dvp
  int ldo;
};
bool mha_prefill_supports(int dkp, int dvp);
void launch_mha_prefill(const MhaPrefillArgs& a, hipStream_t st);

// ---- shared by the layered decoders (and mixers.h) ----------------------------------------------
// y[i] = x[rows[i]], d columns (d % 4 == 0)
void launch_gather_rows(const float* x, int d, const int* rows, int n, float* y, hipStream_t st);
// heads of w [H][rows][cols] transposed: out [H][cols][rows]
void launch_transpose_heads(const bf16_t* w, int H, int rows, int cols, bf16_t* out, hipStream_t st);
// C[M][ldc] (+)= A[M][lda] x W[N][ldw]^T with fp32 A, C and products (bf16 weights widened); K % 16 == 0
void launch_gemm_f32(const float* A, int lda, const bf16_t* W, int ldw, int M, int N, int K, float* C, int ldc,
                     int accumulate, hipStream_t st);
// the same over the tiles of a grouped product {group, first row, rows, -} (at most 64 rows each): C[row][N] =
// A[token[row]] (token null: A[row]) x W[group]^T, W [groups][N][K], C rows of N columns
void launch_gemm_f32_grouped(const float* A, int lda, const int* token, const bf16_t* W, const int4* tiles, const int* n_tiles,
                             int max_tiles, int N, int K, float* C, hipStream_t st);
// out[m][i] = act(gu[m][2 i]) * gu[m][2 i + 1] in fp32 (accurate exponential)
void launch_glu_f32(const float* gu, int ldg, float* out, int ldo, int rows, int n, int act, hipStream_t st);

}  // namespace aios
