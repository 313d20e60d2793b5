// Weight-streaming matrix product for few rows (decode): C[M,N] = A[M,K] * W[N,K]^T,
// bfloat16 in and out, float32 accumulate on the matrix cores, M <= 16 (<= 32 for the
// gated and the rotary product).
//
// At these sizes the product is bound by reading W once from HBM.  A block owns 8 to 64
// output features and all of K: its 8 waves each stream one eighth of every one of its
// weight rows (MFMA 16x16x32 with the weights as the A operand and the activations,
// transposed, as the B operand), then add their partial tiles through LDS in a fixed order,
// so the result does not depend on timing.  Activations are small and come from the cache
// hierarchy.  How the weight rows are read decides the kernel's speed: in whole cache lines
// with non-temporal loads where the matrix lies so that they can be (LINES; common.h says
// how and what was measured), else 16 contiguous bytes per lane and k-step.
//
// What follows a product in a decoder layer is folded into its last step where that saves a
// launch: the SiLU-gated product, the rotary encoding with the cache write, the residual
// add with the beginning of the norm (EPI_*).
//
// This stands where the reference's engine calls the vendor BLAS
// (distributed/linear.py:167); that library's kernels reach about half of the HBM
// rate at these shapes.
#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8_t;
typedef __attribute__((__vector_size__(4 * sizeof(__bf16)))) __bf16 bf16x4_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float f32x4_t;

#define SK_WAVES 8

// LINES: the weights are read in whole cache lines (lines_to_operands in common.h), where
// the matrix lies so that they can be.  RT = tiles of 16 rows (tokens) a wave keeps sums for.
// NT = 16-feature tiles of the OUTPUT per block (the activations a wave loads are used
// for every weight tile of the block), U = k-steps whose loads are issued together
// before their products run.  Register use is kept low on purpose: many resident waves,
// each with U*(tiles+1) loads in flight, hide the memory latency better than a deeper
// pipeline in fewer waves.
//
// What the last step does with the products (each folds a neighbouring launch of a
// decoder layer into this one):
//   EPI_STORE  c = bf16(product).
//   EPI_STORE_F32  c (float32) = float(bf16(product)): the output head's logits, which are
//              wanted in float32 (no cast launch after the product).  Rounded to bfloat16 on the
//              way like every product of this path, so that a position's logits are the same
//              numbers whether its step had few rows (this kernel) or many (the vendor
//              library's bfloat16 product, widened afterwards).
//   EPI_GELU_TABLE  c = bf16(gelu_tanh(bf16(product)) * table[ids[row], col0 + feature]): a gate that
//              multiplies a slice of a per-token table row (a side input that depends on the
//              token's identity); the values are those of the product followed by gated_table_rows.
//   EPI_GRU    W holds three stacked matrices [z; x; g] of n rows each, every row of `a` is the ONE
//              token its request brings to the step, and the output is a step of the gated
//              recurrence: S = (1 - sig(z + bz)) S + sig(z + bz) cand(x + bx), out = S silu(g),
//              with S read from and written to the request's float32 state row (the values
//              of the product followed by the recurrence kernel, bit for bit).
//   EPI_GATED  W holds two stacked matrices [gate; up] of n rows each and the output is
//              silu(gate . a) * (up . a): a block computes both halves of its features,
//              so the [m, 2n] intermediate is never written.
//   EPI_ROPE   W is the stacked q|k|v projection of an attention layer with half-paired
//              rotary encoding over the whole head: a block computes some dims of a
//              head's first half and their partners, rotates them, and writes queries
//              to c[m, q_heads*head_dim] and keys and values straight into their cache
//              slots.
//   EPI_ADDNORM  the product is a layer's contribution to the residual stream and the next
//              thing to happen is an RMS norm: residual += bf16(product) (float32, stored), and
//              c = bf16(residual * norm_weight), the norm's output but for the row's factor
//              rsqrt(mean(residual^2) + eps).  That factor needs the whole row, which no block
//              has: every block leaves the sum of squares of its features per row in
//              sumsq[block][row], and the product that consumes c (PRO_SCALED) adds them up
//              and multiplies its own sums with the factor, which commutes with the product.
//              The norm's launch between two products is saved.
//   EPI_LAYER_IN  W is the stacked input projection of a whole layer whose sublayers read one norm:
//              [q | k | v | head gates | ff gate | ff up] (k and v absent where the layer reads another's, the
//              last two where its feed-forward is made elsewhere).  A block computes PAIRS of features as in
//              EPI_ROPE: rotated dims with their partners, dims that pass with dims that pass, value dims
//              with value dims, gates with gates, a feed-forward's gate feature with its up feature.
//              Biases are added to q, k and v; queries go to c[m, q_heads*head_dim], keys and values to
//              their slots, head gates (not activated) to their own rows, the feed-forward's
//              activation to its own rows.
// In every case the sums are rounded to bfloat16 before the activation or rotation,
// exactly as when the product and the second step run as two kernels.
enum { EPI_STORE = 0, EPI_GATED = 1, EPI_ROPE = 2, EPI_ADDNORM = 3, EPI_STORE_F32 = 4, EPI_GELU_TABLE = 5, EPI_GRU = 6,
       EPI_GATED_CLAMPED = 7, EPI_GATED_GELU = 8, EPI_LAYER_IN = 9 };
// Where the activations come from: a matrix in memory, or (PRO_ATTN, few rows) the
// uncombined key ranges of attn_mfma: each wave first combines its own columns of the
// attention output (what attn_reduce would have written) into LDS, so the combining launch
// between the attention and its output projection is saved at the smallest batches.
// PRO_SCALED: rows whose norm factor is still apart (what EPI_ADDNORM leaves): the sums are
// multiplied with rsqrt(sum of the pieces' squares / width + eps) of their row before rounding.
enum { PRO_NONE = 0, PRO_ATTN = 1, PRO_SCALED = 2 };
#define SK_SCALE_PARTS 32  // threads per row that add up the pieces of a row's sum of squares
#define SK_SCALE_PIECES 8  // pieces per such thread: 256 pieces at most
#define SK_PRO_VALUES 4096  // activations a wave makes and holds: rows * (K / 8 waves) at most

struct FoldArgs {  // what the folded neighbours of a product need
  // EPI_ROPE:
  const float* cos_t;  // [m, head_dim/2]
  const float* sin_t;
  const int* slot_mapping;  // [m]: page * page_size + offset, negative: write nothing
  bf16_t* k_pages;  // [pages][kv_heads][page_size][head_dim]
  bf16_t* v_pages;  // the same, or [pages][kv_heads][head_dim][page_size] if v_transposed
  int q_heads, kv_heads, head_dim, page_size, v_transposed;
  // PRO_ATTN: partial accumulators [row][head][split][head_dim], (max in natural-log units,
  // sum) pairs [row][head][split][2], as attn_mfma leaves them; K = attn_heads * attn_head_dim
  const float* part_acc;
  const float* part_ml;
  int num_splits, attn_heads, attn_head_dim;
  // EPI_ADDNORM: the float32 residual rows [m, n] the product is added to, the norm's weight [n],
  // where the block's sums of squares go ([blocks][m])
  float* residual;
  int64_t ld_residual;
  const bf16_t* norm_weight;
  float* sumsq_out;
  // EPI_GRU: state rows [slots + 1][stride] (a slot outside 0..num_slots-1 means the spare row at
  // num_slots), the slot of each activation row, the two gate biases [n]
  float* gru_state;
  int64_t gru_state_stride;
  const int* gru_slots;
  int gru_num_slots;
  const float* gru_bz;
  const float* gru_bx;
  // EPI_GELU_TABLE: the table [rows][ld_table], the table row of each activation row, the first column
  const bf16_t* table;
  int64_t ld_table;
  const int* table_ids;
  int table_col;
  // EPI_LAYER_IN (beside the fields of EPI_ROPE, cos/sin [m, rot_half]): rotated pairs a head, value heads'
  // width, rows of W the head gates take (q_heads of them count), features of the feed-forward; biases
  // float32 [q | k | v] or null; where gates [m, q_heads] and activations [m, ff] go.  The feed-forward
  // ends as EPI_GATED_CLAMPED does (glu_limit > 0, no biases) or with silu(g) * u (glu_limit 0)
  int rot_half, v_dim, gate_rows, ff;
  const float* qkv_bias;
  bf16_t* gate_out;
  int64_t ld_gate;
  bf16_t* act_out;
  int64_t ld_act;
  // EPI_STORE_F32: the rounded products are multiplied by this
  float out_scale;
  // EPI_GATED_CLAMPED: float32 [2n] biases of gate and up (or null),
  // out = g * logistic(slope * g) * (u + 1), g = min(gate + bias, limit), u = clamp(up + bias, -limit, limit)
  const float* glu_bias;
  float glu_limit, glu_slope;
  // PRO_SCALED: the pieces of the rows' sums of squares [pieces][m], the norm's eps and width
  const float* sumsq_in;
  int sumsq_pieces;
  float norm_eps;
  int norm_width;
};

template <int NT, int U, int EPI, int PRO = PRO_NONE, bool LINES = false, int RT = 1>
__global__ __launch_bounds__(64 * SK_WAVES) void gemm_skinny_bf16_kernel(
    const bf16_t* __restrict__ a, int64_t lda, const bf16_t* __restrict__ w, int64_t ldw,
    bf16_t* __restrict__ c, int64_t ldc, int m, int n, int k, int features_per_block, const FoldArgs fold) {
  constexpr bool GATED = EPI == EPI_GATED || EPI == EPI_GATED_CLAMPED || EPI == EPI_GATED_GELU;
  constexpr bool ROPE = EPI == EPI_ROPE;
  constexpr bool LAYER_IN = EPI == EPI_LAYER_IN;
  constexpr bool ADDNORM = EPI == EPI_ADDNORM;
  constexpr bool SCALED = PRO == PRO_SCALED;
  static_assert(!ROPE || NT == 1, "the rotary epilogue takes one tile of dims and its partner tile");
  static_assert(!LINES || U % 2 == 0, "whole lines are read for pairs of k-steps");
  // RT = tiles of 16 ROWS (tokens): a weight operand once in registers is used for every row tile
  static_assert(RT == 1 || (PRO == PRO_NONE && !ADDNORM), "more than 16 rows: plain activations, no folded norm");
  constexpr bool GRU = EPI == EPI_GRU;
  constexpr int WT = GRU ? 3 * NT : (GATED || ROPE || LAYER_IN) ? 2 * NT : NT;  // weight tiles per block
  __shared__ float red[SK_WAVES][WT][256];

  // (with LINES made uniform for the compiler: the wave's range of K and with it the loop and
  // the base address of every load are scalar)
  const int wave = LINES ? __builtin_amdgcn_readfirstlane(threadIdx.x / MI_WAVE) : threadIdx.x / MI_WAVE;
  const int lane = threadIdx.x % MI_WAVE;
  const int col = lane % 16;
  const int quad = lane / 16;
  // the block's features [n0, n_end): up to 16*NT, a multiple of 4 chosen by the host so
  // that the blocks spread evenly over the CUs (rows past n_end repeat the last one)
  // Rotary epilogue: the unit of work is a PAIR (a dim of a head's first half and its
  // partner half a head further on); pairs are numbered through all heads and a block
  // takes `features_per_block` (a multiple of 4, at most 16) consecutive ones, which may
  // lie in two heads: tile 0 holds the pairs' first dims, tile 1 their partners.
  const int half = ROPE ? fold.head_dim / 2 : 0;
  const int total_pairs = ROPE ? (fold.q_heads + 2 * fold.kv_heads) * half : 0;
  const int pair0 = ROPE ? blockIdx.x * features_per_block : 0;
  const int pair_end = ROPE ? min(pair0 + features_per_block, total_pairs) : 0;
  const int n0 = blockIdx.x * features_per_block;
  const int n_end = min(n0 + features_per_block, n);  // (EPI_LAYER_IN: n and these count pairs)
  // EPI_LAYER_IN: pairs of queries and keys, of values, of head gates; first rows of values, gates, feed-forward
  const int qk_half = LAYER_IN ? fold.head_dim / 2 : 1, v_half = LAYER_IN ? fold.v_dim / 2 : 1;
  const int qk_pairs = LAYER_IN ? (fold.q_heads + fold.kv_heads) * qk_half : 0;
  const int v_pairs = LAYER_IN ? fold.kv_heads * v_half : 0;
  const int gate_pairs = LAYER_IN ? fold.gate_rows / 2 : 0;
  const int v_row0 = 2 * qk_pairs, gate_row0 = v_row0 + 2 * v_pairs, ff_row0 = gate_row0 + 2 * gate_pairs;

  const int ksteps = k / 32;
  const int per_wave = (ksteps + SK_WAVES - 1) / SK_WAVES;
  const int s_begin = min(wave * per_wave, ksteps);
  const int s_end = min(s_begin + per_wave, ksteps);

  // weights: lane reads feature n0 + 16*nt + col (and its twin n rows further down when
  // gated), 8 consecutive k
  auto weight_row = [&](int t, int c) -> int {  // the matrix row behind row c of weight tile t
    if (ROPE) {
      const int pair = min(pair0 + c, pair_end - 1);
      return (pair / half) * fold.head_dim + pair % half + t * half;
    }
    if (LAYER_IN) {
      int pair = min(n0 + (t % NT) * 16 + c, n_end - 1);
      const int partner = t / NT;
      if (pair < qk_pairs) {
        const int head_row = pair / qk_half * fold.head_dim, j = pair % qk_half;
        return j < fold.rot_half ? head_row + j + partner * fold.rot_half
                                 : head_row + fold.rot_half + j + partner * (qk_half - fold.rot_half);
      }
      pair -= qk_pairs;
      if (pair < v_pairs) return v_row0 + pair / v_half * fold.v_dim + pair % v_half + partner * v_half;
      pair -= v_pairs;
      if (pair < gate_pairs) return gate_row0 + pair + partner * gate_pairs;
      return ff_row0 + (pair - gate_pairs) + partner * fold.ff;
    }
    return min(n0 + (t % NT) * 16 + c, n_end - 1) + (t / NT) * n;
  };
  const bf16_t* wp[LINES ? 1 : WT];
  // LINES: byte offsets of this lane's 16 bytes in the tile's lower and upper 8 rows
  uint32_t line_lo[LINES ? WT : 1], line_hi[LINES ? WT : 1];
#pragma unroll
  for (int t = 0; t < WT; ++t) {
    if constexpr (LINES) {
      const uint32_t chunk = line_chunk_of_lane(lane);
      line_lo[t] = (uint32_t)weight_row(t, line_row_of_lane(lane)) * (uint32_t)(ldw * 2) + chunk;
      line_hi[t] = (uint32_t)weight_row(t, 8 + line_row_of_lane(lane)) * (uint32_t)(ldw * 2) + chunk;
    } else {
      wp[t] = w + (int64_t)weight_row(t, col) * ldw + quad * 8;
    }
  }
  // the lane's operands of the k-steps first, first + 1 of weight tile t (LINES)
  auto load_lines = [&](int t, int first, bf16x8_t& even_step, bf16x8_t& odd_step) {
    load_line_pair(w, first, line_lo[LINES ? t : 0], line_hi[LINES ? t : 0], even_step, odd_step);
  };
  // activations: lane reads token `col`; lanes past M re-read the last token (the same
  // cache lines as its own lane, so no extra traffic) and their columns are never stored
  const bf16_t* ap[RT];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) ap[rt] = a + (int64_t)min(rt * 16 + col, m - 1) * lda + quad * 8;
  __shared__ __attribute__((aligned(16))) bf16_t a_own[PRO == PRO_ATTN ? SK_WAVES : 1][PRO == PRO_ATTN ? SK_PRO_VALUES : 8];
  const int own_stride = per_wave * 32;  // elements from one row of this wave's columns to the next
  // PRO_ATTN: the weights of the first U k-steps are requested before the activations are
  // made, so that the trips to the key ranges' results hide behind the first trip to memory
  bf16x8_t w_first[PRO == PRO_ATTN ? U : 1][WT];
  const bool first_ahead = PRO == PRO_ATTN && s_begin + U <= s_end;
  if constexpr (PRO == PRO_ATTN) {
    if (first_ahead) {
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int t = 0; t < WT; ++t) {
          if constexpr (LINES) {
            if (u % 2 == 0) load_lines(t, s_begin + u, w_first[u][t], w_first[u + 1][t]);
          } else {
            w_first[u][t] = *reinterpret_cast<const bf16x8_t*>(wp[LINES ? 0 : t] + (int64_t)(s_begin + u) * 32);
          }
        }
    }
  }
  if constexpr (PRO == PRO_ATTN) {
    // this wave's columns [32*s_begin, 32*s_end) of the attention output, 8 at a time per
    // lane: the key ranges' accumulators weighted by exp(max - overall max), added in range
    // order, divided by the weighted sum of their sums (the arithmetic of attn_reduce_kernel)
    const int chunks = (s_end - s_begin) * 4;
    const int head_dim = fold.attn_head_dim, splits = fold.num_splits;
    for (int idx = lane; idx < m * chunks; idx += MI_WAVE) {
      const int row = idx / chunks, chunk = idx % chunks;
      const int k0 = s_begin * 32 + chunk * 8;
      const int head = k0 / head_dim, dim = k0 % head_dim;
      const int64_t base = ((int64_t)row * fold.attn_heads + head) * splits;
      const float* ml = fold.part_ml + base * 2;
      const float* pa = fold.part_acc + base * head_dim + dim;
      // (requesting every range's values before the first use measured slower than this loop)
      float m_all = -INFINITY;
#pragma unroll 8
      for (int sp = 0; sp < splits; ++sp) m_all = fmaxf(m_all, ml[sp * 2]);
      float o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      float l_all = 0.f;
#pragma unroll 4
      for (int sp = 0; sp < splits; ++sp) {
        const float weight = expf(ml[sp * 2] - m_all);
        l_all += ml[sp * 2 + 1] * weight;
        const f32x4_t lo = *reinterpret_cast<const f32x4_t*>(pa + (int64_t)sp * head_dim);
        const f32x4_t hi = *reinterpret_cast<const f32x4_t*>(pa + (int64_t)sp * head_dim + 4);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          o[j] += lo[j] * weight;
          o[4 + j] += hi[j] * weight;
        }
      }
      const float inv = 1.f / l_all;
      bf16x8_t packed;
#pragma unroll
      for (int j = 0; j < 8; ++j) packed[j] = (bf16_t)(o[j] * inv);
      *reinterpret_cast<bf16x8_t*>(&a_own[wave][row * own_stride + chunk * 8]) = packed;
    }
    __syncthreads();
  }
  const bf16_t* own = &a_own[PRO == PRO_ATTN ? wave : 0][(PRO == PRO_ATTN ? min(col, m - 1) * own_stride : 0) + quad * 8];

  __shared__ float scale_part[SCALED ? SK_SCALE_PARTS : 1][16];
  // EPI_ADDNORM: the residual values and norm weights of the thread's four outputs, asked for
  // now, so that the last step does not begin with a trip to memory
  f32x4_t res_old = {0.f, 0.f, 0.f, 0.f};
  float norm_w4[4] = {0.f, 0.f, 0.f, 0.f};
  if constexpr (ADDNORM) {
    const int item = threadIdx.x;
    const int token = (item % 64) % 16, feature = n0 + (item / 64) * 16 + ((item % 64) / 16) * 4;
    if (item < NT * 64 && token < m) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (feature + r < n_end) {
          res_old[r] = fold.residual[(int64_t)token * fold.ld_residual + feature + r];
          norm_w4[r] = (float)fold.norm_weight[feature + r];
        }
      }
    }
  }

  // PRO_SCALED: SK_SCALE_PARTS threads per row each add up every SK_SCALE_PARTS-th piece of the
  // row's sum of squares, in a fixed order.  Where the loop below leaves registers to spare the
  // pieces are asked for before it, so that the trip to them is over when it ends (whole decode
  // steps 0.9-1.3 % faster); with four weight tiles they would cost the registers of a resident
  // block per CU (measured: 16 % slower), and are asked for after it.  (Capping the registers
  // of the variants just above 80 at 80 measured 0.8-1.4 % slower.)
  constexpr bool SCALE_EARLY = SCALED && WT <= 2;
  float scale_piece[SCALED ? SK_SCALE_PIECES : 1];
  auto load_scale_pieces = [&]() {
    const int row = threadIdx.x % 16, part = threadIdx.x / 16;
#pragma unroll
    for (int i = 0; i < SK_SCALE_PIECES; ++i) {
      const int piece = part + i * SK_SCALE_PARTS;
      scale_piece[SCALED ? i : 0] = (row < m && piece < fold.sumsq_pieces) ? fold.sumsq_in[(int64_t)piece * m + row] : 0.f;
    }
  };
  if constexpr (SCALE_EARLY) load_scale_pieces();

  f32x4_t acc[RT][WT];
#pragma unroll
  for (int rt = 0; rt < RT; ++rt)
#pragma unroll
    for (int t = 0; t < WT; ++t) acc[rt][t] = (f32x4_t){0.f, 0.f, 0.f, 0.f};

  int s = s_begin;
  for (; s + U <= s_end; s += U) {
    bf16x8_t w_reg[U][WT];
    bf16x8_t a_reg[RT][U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
#pragma unroll
      for (int t = 0; t < WT; ++t) {
        if constexpr (LINES) {
          if (u % 2 == 0) {
            if (PRO == PRO_ATTN && first_ahead && s == s_begin) {
              w_reg[u][t] = w_first[PRO == PRO_ATTN ? u : 0][t];
              w_reg[u + 1][t] = w_first[PRO == PRO_ATTN ? u + 1 : 0][t];
            } else {
              load_lines(t, s + u, w_reg[u][t], w_reg[u + 1][t]);
            }
          }
        } else {
          if (PRO == PRO_ATTN && first_ahead && s == s_begin) w_reg[u][t] = w_first[PRO == PRO_ATTN ? u : 0][t];
          else w_reg[u][t] = *reinterpret_cast<const bf16x8_t*>(wp[LINES ? 0 : t] + (int64_t)(s + u) * 32);
        }
      }
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) {
        if constexpr (PRO == PRO_ATTN) a_reg[rt][u] = *reinterpret_cast<const bf16x8_t*>(own + (s + u - s_begin) * 32);
        else a_reg[rt][u] = *reinterpret_cast<const bf16x8_t*>(ap[rt] + (int64_t)(s + u) * 32);
      }
    }
    if constexpr (LINES) {
#pragma unroll
      for (int u = 0; u < U; u += 2)
#pragma unroll
        for (int t = 0; t < WT; ++t) lines_to_operands(w_reg[u][t], w_reg[u + 1][t]);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int t = 0; t < WT; ++t)
#pragma unroll
        for (int rt = 0; rt < RT; ++rt)
          acc[rt][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w_reg[u][t], a_reg[rt][u], acc[rt][t], 0, 0, 0);
  }
  if constexpr (LINES) {
    for (; s + 2 <= s_end; s += 2) {  // fewer than U k-steps left: pair by pair (their number is even)
      bf16x8_t a_even[RT], a_odd[RT];
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) {
        a_even[rt] = PRO == PRO_ATTN ? *reinterpret_cast<const bf16x8_t*>(own + (s - s_begin) * 32)
                                     : *reinterpret_cast<const bf16x8_t*>(ap[rt] + (int64_t)s * 32);
        a_odd[rt] = PRO == PRO_ATTN ? *reinterpret_cast<const bf16x8_t*>(own + (s + 1 - s_begin) * 32)
                                    : *reinterpret_cast<const bf16x8_t*>(ap[rt] + (int64_t)(s + 1) * 32);
      }
#pragma unroll
      for (int t = 0; t < WT; ++t) {
        bf16x8_t w_even, w_odd;
        load_lines(t, s, w_even, w_odd);
        lines_to_operands(w_even, w_odd);
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) {
          acc[rt][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w_even, a_even[rt], acc[rt][t], 0, 0, 0);
          acc[rt][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w_odd, a_odd[rt], acc[rt][t], 0, 0, 0);
        }
      }
    }
  }
  for (; !LINES && s < s_end; ++s) {  // fewer than U k-steps left
    bf16x8_t a_tail[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt)
      a_tail[rt] = PRO == PRO_ATTN ? *reinterpret_cast<const bf16x8_t*>(own + (s - s_begin) * 32)
                                   : *reinterpret_cast<const bf16x8_t*>(ap[rt] + (int64_t)s * 32);
#pragma unroll
    for (int t = 0; t < WT; ++t) {
      const bf16x8_t w_tail = *reinterpret_cast<const bf16x8_t*>(wp[LINES ? 0 : t] + (int64_t)s * 32);
#pragma unroll
      for (int rt = 0; rt < RT; ++rt)
        acc[rt][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w_tail, a_tail[rt], acc[rt][t], 0, 0, 0);
    }
  }

  if constexpr (SCALED && !SCALE_EARLY) load_scale_pieces();
  __shared__ float squares[ADDNORM ? NT * 4 : 1][16];  // EPI_ADDNORM: per (4 features, row) of the block
  // acc[rt][t][r] = C^T[feature n0 + 16*(t % NT) + 4*quad + r][token 16*rt + col]; add the 8 waves
  // in order, one row tile after the other through the same LDS
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
  if (rt > 0) __syncthreads();
#pragma unroll
  for (int t = 0; t < WT; ++t) {
#pragma unroll
    for (int r = 0; r < 4; ++r) red[wave][t][(quad * 4 + r) * 16 + col] = acc[rt][t][r];
  }
  if constexpr (SCALED) {
    float scale_mine = 0.f;
#pragma unroll
    for (int i = 0; i < SK_SCALE_PIECES; ++i) scale_mine += scale_piece[i];
    scale_part[threadIdx.x / 16][threadIdx.x % 16] = scale_mine;
  }
  __syncthreads();
  // 256*NT outputs, each a sum of 8 (two such when gated): a thread takes 4 consecutive
  // features of one token
  for (int item = threadIdx.x; item < NT * 64; item += 64 * SK_WAVES) {
    const int nt = item / 64;
    const int token_in_tile = (item % 64) % 16;
    const int token = rt * 16 + token_in_tile;
    const int fq = (item % 64) / 16;
    if (token >= m) continue;
    float sum[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int wv = 0; wv < SK_WAVES; ++wv)
#pragma unroll
      for (int r = 0; r < 4; ++r) sum[r] += red[wv][nt][(fq * 4 + r) * 16 + token_in_tile];
    float up[4] = {0.f, 0.f, 0.f, 0.f};  // the twin tile's sums: the up half (gated), the partner dims (rotary)
    if (GATED || ROPE || GRU || LAYER_IN) {
#pragma unroll
      for (int wv = 0; wv < SK_WAVES; ++wv)
#pragma unroll
        for (int r = 0; r < 4; ++r) up[r] += red[wv][NT + nt][(fq * 4 + r) * 16 + token_in_tile];
    }
    if constexpr (GRU) {
      float gate[4] = {0.f, 0.f, 0.f, 0.f};  // the third stacked matrix's sums
#pragma unroll
      for (int wv = 0; wv < SK_WAVES; ++wv)
#pragma unroll
        for (int r = 0; r < 4; ++r) gate[r] += red[wv][2 * NT + nt][(fq * 4 + r) * 16 + token_in_tile];
      const int feature = n0 + nt * 16 + fq * 4;
      const int slot = fold.gru_slots[token];
      float* state = fold.gru_state +
                     (int64_t)((slot < 0 || slot >= fold.gru_num_slots) ? fold.gru_num_slots : slot) * fold.gru_state_stride;
      bf16_t* dst = c + (int64_t)token * ldc + feature;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (feature + r < n_end) {  // (rows past n_end repeat the last feature: its state is advanced once)
          const float z = mi_logistic((float)(bf16_t)sum[r] + fold.gru_bz[feature + r]);
          const float u = (float)(bf16_t)up[r] + fold.gru_bx[feature + r];
          const float cand = u >= 0.f ? u + 0.5f : mi_logistic(u);
          const float g = (float)(bf16_t)gate[r];
          const float keep = 1.f - z, add = z * cand;
          const float s = __builtin_fmaf(keep, state[feature + r], add);  // (as the recurrence kernel spells it)
          state[feature + r] = s;
          dst[r] = (bf16_t)(s * (g * mi_logistic(g)));
        }
      }
      continue;
    }
    if constexpr (SCALED) {
      float total = 0.f;
#pragma unroll
      for (int part = 0; part < SK_SCALE_PARTS; ++part) total += scale_part[part][token];
      const float inv = rsqrtf(total / (float)fold.norm_width + fold.norm_eps);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        sum[r] *= inv;
        up[r] *= inv;
      }
    }
    if (GATED) {
      if constexpr (EPI == EPI_GATED_CLAMPED) {  // (the arithmetic of clamped_glu on the rounded products, bit for bit)
        const int feature = n0 + nt * 16 + fq * 4;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int at = min(feature + r, n - 1);
          const float bias_g = fold.glu_bias ? fold.glu_bias[at] : 0.f, bias_u = fold.glu_bias ? fold.glu_bias[n + at] : 0.f;
          const float g = fminf((float)(bf16_t)sum[r] + bias_g, fold.glu_limit);
          const float u = fminf(fmaxf((float)(bf16_t)up[r] + bias_u, -fold.glu_limit), fold.glu_limit);
          sum[r] = g * mi_logistic(fold.glu_slope * g) * (u + 1.f);
        }
      } else if constexpr (EPI == EPI_GATED_GELU) {  // (the tanh form of gelu, as gated_mul spells it)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float g = (float)(bf16_t)sum[r];
          const float f = 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
          sum[r] = f * (float)(bf16_t)up[r];
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float g = (float)(bf16_t)sum[r];
          sum[r] = g / (1.f + expf(-g)) * (float)(bf16_t)up[r];
        }
      }
    }
    if constexpr (ADDNORM) {
      const int feature = n0 + nt * 16 + fq * 4;
      float* res = fold.residual + (int64_t)token * fold.ld_residual + feature;
      bf16_t* dst = c + (int64_t)token * ldc + feature;
      float sq = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (feature + r < n_end) {  // (rows past n_end repeat the last feature: not counted twice)
          const float x = res_old[r] + (float)(bf16_t)sum[r];
          res[r] = x;
          dst[r] = (bf16_t)(x * norm_w4[r]);
          sq += x * x;
        }
      }
      squares[nt * 4 + fq][token] = sq;
      continue;
    }
    if (ROPE) {
      // this thread: four consecutive pairs (never across a head: half is a multiple of 4), one token
      const int pair = pair0 + fq * 4;
      if (pair >= pair_end) continue;
      const int rope_head = pair / half, j = pair % half;
      const int q_heads = fold.q_heads, kv_heads = fold.kv_heads, hd = fold.head_dim;
      float lo[4], hi[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        lo[r] = (float)(bf16_t)sum[r];
        hi[r] = (float)(bf16_t)up[r];
      }
      if (rope_head < q_heads + kv_heads) {  // queries and keys are rotated (formula: models/blocks/fold.py:411-431)
        const f32x4_t cs = *reinterpret_cast<const f32x4_t*>(fold.cos_t + (int64_t)token * half + j);
        const f32x4_t sn = *reinterpret_cast<const f32x4_t*>(fold.sin_t + (int64_t)token * half + j);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float x0 = lo[r], x1 = hi[r];
          lo[r] = x0 * cs[r] - x1 * sn[r];
          hi[r] = x1 * cs[r] + x0 * sn[r];
        }
      }
      bf16x4_t lo_b, hi_b;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        lo_b[r] = (bf16_t)lo[r];
        hi_b[r] = (bf16_t)hi[r];
      }
      if (rope_head < q_heads) {
        bf16_t* dst = c + (int64_t)token * ldc + (int64_t)rope_head * hd + j;
        *reinterpret_cast<bf16x4_t*>(dst) = lo_b;
        *reinterpret_cast<bf16x4_t*>(dst + half) = hi_b;
      } else {
        const int slot = fold.slot_mapping[token];
        if (slot >= 0) {  // padding rows of a replayed step write nothing
          const int page = slot / fold.page_size, off = slot % fold.page_size;
          const bool is_key = rope_head < q_heads + kv_heads;
          const int h = rope_head - q_heads - (is_key ? 0 : kv_heads);
          const int64_t chunk = ((int64_t)page * kv_heads + h) * fold.page_size * hd;
          if (is_key || !fold.v_transposed) {
            bf16_t* dst = (is_key ? fold.k_pages : fold.v_pages) + chunk + (int64_t)off * hd + j;
            *reinterpret_cast<bf16x4_t*>(dst) = lo_b;
            *reinterpret_cast<bf16x4_t*>(dst + half) = hi_b;
          } else {
            bf16_t* dst = fold.v_pages + chunk + off;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              dst[(int64_t)(j + r) * fold.page_size] = lo_b[r];
              dst[(int64_t)(half + j + r) * fold.page_size] = hi_b[r];
            }
          }
        }
      }
      continue;
    }
    if constexpr (LAYER_IN) {
      // this thread: four consecutive pairs of one kind (and of one head: all widths are multiples of 8), one token
      int pair = n0 + nt * 16 + fq * 4;
      if (pair >= n_end) continue;
      float lo[4], hi[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        lo[r] = (float)(bf16_t)sum[r];
        hi[r] = (float)(bf16_t)up[r];
      }
      bf16x4_t lo_b, hi_b;
      auto round_both = [&]() {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          lo_b[r] = (bf16_t)lo[r];
          hi_b[r] = (bf16_t)hi[r];
        }
      };
      auto add_bias = [&](int lo_row, int hi_row) {
        if (fold.qkv_bias == nullptr) return;
        const f32x4_t bl = *reinterpret_cast<const f32x4_t*>(fold.qkv_bias + lo_row);
        const f32x4_t bh = *reinterpret_cast<const f32x4_t*>(fold.qkv_bias + hi_row);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          lo[r] += bl[r];
          hi[r] += bh[r];
        }
      };
      const int hd = fold.head_dim, kv_heads = fold.kv_heads, rot_half = fold.rot_half;
      if (pair < qk_pairs) {
        const int head = pair / qk_half, j = pair % qk_half;
        const bool turned = j < rot_half;
        const int lo_dim = turned ? j : rot_half + j, hi_dim = lo_dim + (turned ? rot_half : qk_half - rot_half);
        add_bias(head * hd + lo_dim, head * hd + hi_dim);
        if (turned) {
          const f32x4_t cs = *reinterpret_cast<const f32x4_t*>(fold.cos_t + (int64_t)token * rot_half + j);
          const f32x4_t sn = *reinterpret_cast<const f32x4_t*>(fold.sin_t + (int64_t)token * rot_half + j);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float x0 = lo[r], x1 = hi[r];
            lo[r] = x0 * cs[r] - x1 * sn[r];
            hi[r] = x1 * cs[r] + x0 * sn[r];
          }
        }
        round_both();
        bf16_t* dst = nullptr;
        if (head < fold.q_heads) {
          dst = c + (int64_t)token * ldc + (int64_t)head * hd;
        } else {
          const int slot = fold.slot_mapping[token];
          if (slot >= 0) {  // padding rows of a replayed step write nothing
            const int page = slot / fold.page_size, off = slot % fold.page_size;
            dst = fold.k_pages + (((int64_t)page * kv_heads + head - fold.q_heads) * fold.page_size + off) * hd;
          }
        }
        if (dst != nullptr) {
          *reinterpret_cast<bf16x4_t*>(dst + lo_dim) = lo_b;
          *reinterpret_cast<bf16x4_t*>(dst + hi_dim) = hi_b;
        }
        continue;
      }
      pair -= qk_pairs;
      if (pair < v_pairs) {
        const int head = pair / v_half, j = pair % v_half, vd = fold.v_dim;
        add_bias(v_row0 + head * vd + j, v_row0 + head * vd + v_half + j);
        round_both();
        const int slot = fold.slot_mapping[token];
        if (slot >= 0) {
          const int page = slot / fold.page_size, off = slot % fold.page_size;
          bf16_t* chunk = fold.v_pages + ((int64_t)page * kv_heads + head) * fold.page_size * vd;
          if (fold.v_transposed) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              chunk[(int64_t)(j + r) * fold.page_size + off] = lo_b[r];
              chunk[(int64_t)(v_half + j + r) * fold.page_size + off] = hi_b[r];
            }
          } else {
            *reinterpret_cast<bf16x4_t*>(chunk + (int64_t)off * vd + j) = lo_b;
            *reinterpret_cast<bf16x4_t*>(chunk + (int64_t)off * vd + v_half + j) = hi_b;
          }
        }
        continue;
      }
      pair -= v_pairs;
      if (pair < gate_pairs) {
        bf16_t* dst = fold.gate_out + (int64_t)token * fold.ld_gate;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (pair + r < fold.q_heads) dst[pair + r] = (bf16_t)lo[r];
          if (pair + gate_pairs + r < fold.q_heads) dst[pair + gate_pairs + r] = (bf16_t)hi[r];
        }
        continue;
      }
      pair -= gate_pairs;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (fold.glu_limit > 0.f) {
          const float g = fminf(lo[r], fold.glu_limit);
          const float u = fminf(fmaxf(hi[r], -fold.glu_limit), fold.glu_limit);
          lo_b[r] = (bf16_t)(g * mi_logistic(fold.glu_slope * g) * (u + 1.f));
        } else {
          lo_b[r] = (bf16_t)(lo[r] / (1.f + expf(-lo[r])) * hi[r]);
        }
      }
      *reinterpret_cast<bf16x4_t*>(fold.act_out + (int64_t)token * fold.ld_act + pair) = lo_b;
      continue;
    }
    const int feature = n0 + nt * 16 + fq * 4;
    if constexpr (EPI == EPI_STORE_F32) {
      float* dst32 = reinterpret_cast<float*>(c) + (int64_t)token * ldc + feature;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (feature + r < n_end) dst32[r] = (float)(bf16_t)sum[r] * fold.out_scale;  // (times 1 changes nothing)
      continue;
    }
    if constexpr (EPI == EPI_GELU_TABLE) {
      const bf16_t* slice = fold.table + (int64_t)fold.table_ids[token] * fold.ld_table + fold.table_col + feature;
      bf16_t* gated = c + (int64_t)token * ldc + feature;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (feature + r < n_end) {
          const float z = (float)(bf16_t)sum[r];
          const float act = 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
          gated[r] = (bf16_t)(act * (float)slice[r]);
        }
      }
      continue;
    }
    bf16_t* dst = c + (int64_t)token * ldc + feature;
    if (feature + 3 < n_end && (ldc % 4 == 0)) {
      bf16x4_t packed;
#pragma unroll
      for (int r = 0; r < 4; ++r) packed[r] = (bf16_t)sum[r];
      *reinterpret_cast<bf16x4_t*>(dst) = packed;
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (feature + r < n_end) dst[r] = (bf16_t)sum[r];
    }
  }
  }  // row tiles
  if constexpr (ADDNORM) {
    __syncthreads();
    if ((int)threadIdx.x < m) {
      float total = 0.f;
#pragma unroll
      for (int i = 0; i < NT * 4; ++i) total += squares[i][threadIdx.x];
      fold.sumsq_out[(int64_t)blockIdx.x * m + threadIdx.x] = total;
    }
  }
}

// Rows.  The gated and the rotary product take two row tiles (17-32 rows: measured against the
// vendor product followed by silu_mul / rope_kv_write, microseconds at 24 / 32 rows: gate|up
// 2x14336x4096 42.9 / 46.2 against 54.6 / 54.6, q|k|v 6144x4096 17.0 / 17.2 against 20.2 / 19.5,
// gate|up 2x8192x3072 22.4 / 23.3 against 23.8 / 23.9, q|k|v 5120x3072 13.9 / 14.6 against
// 17.8 / 16.4; with four row tiles, 48 / 64 rows, they are level or slower: every block reads
// all the rows' activations).  Everything else takes one.
#define SK_MAX_ROWS 16
#define SK_WIDE_MAX_ROWS 32

// Compute units of the current device (asked once per device).
static int compute_units() {
  static int cached[64] = {0};
  int device = 0;
  if (hipGetDevice(&device) != hipSuccess || device < 0 || device >= 64) return 0;
  if (cached[device] == 0) {
    int count = 0;
    if (hipDeviceGetAttribute(&count, hipDeviceAttributeMultiprocessorCount, device) != hipSuccess) return 0;
    cached[device] = count;
  }
  return cached[device];
}

static bool skinny_takes(int m, int n, int k, int64_t lda, int64_t ldw, int max_rows) {
  return m >= 1 && m <= max_rows && n >= 1 && k >= 32 && k % 32 == 0 && lda % 8 == 0 && ldw % 8 == 0;
}

extern "C" int mi_gemm_skinny_bf16_supported(int m, int n, int k, int64_t lda, int64_t ldw) {
  return skinny_takes(m, n, k, lda, ldw, SK_MAX_ROWS) ? 1 : 0;
}

// the gated and the rotary product (mi_gemm_skinny_swiglu_bf16, mi_gemm_skinny_rope_bf16)
extern "C" int mi_gemm_skinny_wide_bf16_supported(int m, int n, int k, int64_t lda, int64_t ldw) {
  return skinny_takes(m, n, k, lda, ldw, SK_WIDE_MAX_ROWS) ? 1 : 0;
}

// Features per block: as even a share of the output as a multiple of 4 allows, in
// whole rounds over the CUs (an HBM-bound kernel ends when its most loaded CU does),
// at most 16*max_tiles.  Measured on MI355X at Llama-8B sizes, batch 8: 6144 features
// run 10% faster as 256 blocks of 24 than as 192 of 32; 28672 as 512 blocks of 56
// rather than 448 of 64.
static int features_per_block_for(int n, int cus, int max_tiles) {
  const int rounds = ceil_div(n, cus * 16 * max_tiles);
  const int fpb = ceil_div(ceil_div(n, cus * rounds), 4) * 4;
  return fpb < 8 ? 8 : fpb;
}

// Whether a weight matrix of `rows` rows can be read in whole cache lines (LINES): its rows
// begin on 128-byte boundaries, every wave gets an even number of k-steps, and byte offsets
// into it fit 32 bits.
static bool whole_lines(const void* w, int64_t ldw, int64_t rows, int k) {
  return (uintptr_t)w % 128 == 0 && ldw % 64 == 0 && (k / 32) % (2 * SK_WAVES) == 0 &&
         rows * ldw * 2 < ((int64_t)1 << 32);
}

// `epi`: EPI_STORE, EPI_STORE_F32 (c is float32 [m, ldc]) or EPI_GELU_TABLE (with its fields of `fold`).
static int skinny_plain(const void* a, int64_t lda, const void* w, int64_t ldw, void* c, int64_t ldc, int m, int n,
                        int k, int epi, hipStream_t stream, const FoldArgs nothing_folded = {}) {
  MI_REQUIRE(mi_gemm_skinny_bf16_supported(m, n, k, lda, ldw),
             "gemm_skinny_bf16: takes 1 <= m <= 16, k a multiple of 32, rows aligned to 16 bytes; "
             "got m=%d n=%d k=%d lda=%lld ldw=%lld", m, n, k, (long long)lda, (long long)ldw);
  MI_REQUIRE(lda >= k && ldw >= k && ldc >= n, "gemm_skinny_bf16: a row stride is shorter than its row");
  const bf16_t* ap = (const bf16_t*)a;
  const bf16_t* wp = (const bf16_t*)w;
  bf16_t* cp = (bf16_t*)c;
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "gemm_skinny_bf16: cannot read the device's compute unit count");
  const int fpb = features_per_block_for(n, cus, 4);
  const int blocks = ceil_div(n, fpb);
  const int threads = 64 * SK_WAVES;
  const bool lines = whole_lines(w, ldw, n, k);
#define SK_PLAIN_AS(NT_, U_, EPI_)                                                                                 \
  if (lines)                                                                                                       \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_, PRO_NONE, true><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldc, m, n, k, fpb, nothing_folded); \
  else                                                                                                             \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldc, m, n, k, fpb, nothing_folded)
#define SK_PLAIN(NT_, U_)                                                \
  if (epi == EPI_STORE_F32) { SK_PLAIN_AS(NT_, U_, EPI_STORE_F32); }       \
  else if (epi == EPI_GELU_TABLE) { SK_PLAIN_AS(NT_, U_, EPI_GELU_TABLE); } \
  else { SK_PLAIN_AS(NT_, U_, EPI_STORE); }
  switch (ceil_div(fpb, 16)) {
    case 1: SK_PLAIN(1, 8); break;
    case 2: SK_PLAIN(2, 8); break;
    case 3: SK_PLAIN(3, 4); break;
    default: SK_PLAIN(4, 2); break;
  }
#undef SK_PLAIN
#undef SK_PLAIN_AS
  MI_CHECK_LAUNCH("gemm_skinny_bf16");
  return MI_OK;
}

extern "C" int mi_gemm_skinny_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, void* c,
                                   int64_t ldc, int m, int n, int k, hipStream_t stream) {
  return skinny_plain(a, lda, w, ldw, c, ldc, m, n, k, EPI_STORE, stream);
}

// The same product, the same values times `scale`, written as float32 [m, ldc].
extern "C" int mi_gemm_skinny_f32out_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, float* c,
                                          int64_t ldc, int m, int n, int k, float scale, hipStream_t stream) {
  FoldArgs fold = {};
  fold.out_scale = scale;
  return skinny_plain(a, lda, w, ldw, c, ldc, m, n, k, EPI_STORE_F32, stream, fold);
}

// c[m, n] = gelu_tanh(a . w^T) * table[ids[row], col0 : col0 + n], bfloat16 (EPI_GELU_TABLE).
extern "C" int mi_gemm_skinny_gelu_table_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, const void* table,
                                              int64_t ld_table, const int* ids, int col0, int table_rows, void* c,
                                              int64_t ldc, int m, int n, int k, hipStream_t stream) {
  MI_REQUIRE(table != nullptr && ids != nullptr && col0 >= 0 && table_rows > 0 && ld_table >= (int64_t)col0 + n,
             "gemm_skinny_gelu_table_bf16: columns %d..%d of a table row of %lld", col0, col0 + n, (long long)ld_table);
  FoldArgs fold = {};
  fold.table = (const bf16_t*)table;
  fold.ld_table = ld_table;
  fold.table_ids = ids;
  fold.table_col = col0;
  return skinny_plain(a, lda, w, ldw, c, ldc, m, n, k, EPI_GELU_TABLE, stream, fold);
}

// c[m, n] = attention output [m, heads*head_dim] . w^T, the attention output still lying in
// attn_mfma's uncombined key ranges (part_acc, part_ml as that kernel leaves them, rows
// 0..m-1): few rows, m * heads*head_dim at most 32768 (8 rows of 4096; see
// mi_gemm_skinny_attn_bf16_supported).
extern "C" int mi_gemm_skinny_attn_bf16_supported(int m, int heads, int head_dim) {
  if (m < 1 || m > SK_MAX_ROWS || heads < 1 || head_dim < 32 || head_dim % 32 != 0) return 0;
  const int k = heads * head_dim;
  return m * ceil_div(k / 32, SK_WAVES) * 32 <= SK_PRO_VALUES ? 1 : 0;
}

extern "C" int mi_gemm_skinny_attn_bf16(const float* part_acc, const float* part_ml, int num_splits, int heads,
                                        int head_dim, const void* w, int64_t ldw, void* c, int64_t ldc, int m,
                                        int n, hipStream_t stream) {
  MI_REQUIRE(part_acc && part_ml && num_splits >= 1 && num_splits <= 64,
             "gemm_skinny_attn_bf16: needs the partial buffers of 1..64 key ranges, got %d", num_splits);
  MI_REQUIRE(heads >= 1 && head_dim >= 32 && head_dim % 32 == 0,
             "gemm_skinny_attn_bf16: takes head_dim a multiple of 32; got heads=%d head_dim=%d", heads, head_dim);
  const int k = heads * head_dim;
  MI_REQUIRE(n >= 1 && ldw % 8 == 0 && ldw >= k && ldc >= n,
             "gemm_skinny_attn_bf16: weight rows must be aligned to 16 bytes; got n=%d k=%d ldw=%lld", n, k,
             (long long)ldw);
  MI_REQUIRE(mi_gemm_skinny_attn_bf16_supported(m, heads, head_dim),
             "gemm_skinny_attn_bf16: rows x (heads*head_dim / 8) must be at most %d; got m=%d k=%d", SK_PRO_VALUES, m, k);
  const bf16_t* ap = (const bf16_t*)w;  // never read: the activations are made in the kernel
  const int64_t lda = ldw;
  const bf16_t* wp = (const bf16_t*)w;
  bf16_t* cp = (bf16_t*)c;
  FoldArgs args = {};
  args.part_acc = part_acc;
  args.part_ml = part_ml;
  args.num_splits = num_splits;
  args.attn_heads = heads;
  args.attn_head_dim = head_dim;
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "gemm_skinny_attn_bf16: cannot read the device's compute unit count");
  const int fpb = features_per_block_for(n, cus, 4);
  const int blocks = ceil_div(n, fpb);
  const int threads = 64 * SK_WAVES;
  const bool lines = whole_lines(w, ldw, n, k);
#define SK_ATTN(NT_, U_)                                                                                          \
  if (lines)                                                                                                      \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_STORE, PRO_ATTN, true><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldc, m, n, k, fpb, args); \
  else                                                                                                            \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_STORE, PRO_ATTN><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldc, m, n, k, fpb, args)
  switch (ceil_div(fpb, 16)) {
    case 1: SK_ATTN(1, 8); break;
    case 2: SK_ATTN(2, 8); break;
    case 3: SK_ATTN(3, 4); break;
    default: SK_ATTN(4, 2); break;
  }
#undef SK_ATTN
  MI_CHECK_LAUNCH("gemm_skinny_attn_bf16");
  return MI_OK;
}

// The product as a layer's contribution to the residual stream, with the following RMS norm but
// for its row factor (EPI_ADDNORM): residual[m, n] += bf16(a . w^T); values[m, n] =
// bf16(residual * norm_weight); sumsq[pieces][m] = each block's sums of squares, where
// pieces = mi_gemm_skinny_addnorm_pieces(n).  With part_acc the activations are the
// uncombined key ranges of attn_mfma (as in mi_gemm_skinny_attn_bf16; a, lda unused).
extern "C" int mi_gemm_skinny_addnorm_pieces(int n) {
  const int cus = compute_units();
  if (cus <= 0 || n < 1) return 0;
  return ceil_div(n, features_per_block_for(n, cus, 4));
}

extern "C" int mi_gemm_skinny_addnorm_bf16(const void* a, int64_t lda, const float* part_acc, const float* part_ml,
                                           int num_splits, int heads, int head_dim, const void* w, int64_t ldw,
                                           float* residual, int64_t ld_residual, const void* norm_weight,
                                           void* values, int64_t ldv, float* sumsq, int m, int n, int k,
                                           hipStream_t stream) {
  const bool from_attention = part_acc != nullptr;
  if (from_attention) {
    MI_REQUIRE(part_ml && num_splits >= 1 && num_splits <= 64 && heads * head_dim == k,
               "gemm_skinny_addnorm_bf16: needs the partial buffers of 1..64 key ranges over k = heads*head_dim; "
               "got splits=%d heads=%d head_dim=%d k=%d", num_splits, heads, head_dim, k);
    MI_REQUIRE(mi_gemm_skinny_attn_bf16_supported(m, heads, head_dim) && ldw % 8 == 0,
               "gemm_skinny_addnorm_bf16: rows x (heads*head_dim / 8) must be at most %d, head_dim a multiple of 32; "
               "got m=%d heads=%d head_dim=%d", SK_PRO_VALUES, m, heads, head_dim);
  } else {
    MI_REQUIRE(mi_gemm_skinny_bf16_supported(m, n, k, lda, ldw) && lda >= k,
               "gemm_skinny_addnorm_bf16: takes 1 <= m <= 16, k a multiple of 32, rows aligned to 16 bytes; "
               "got m=%d n=%d k=%d lda=%lld ldw=%lld", m, n, k, (long long)lda, (long long)ldw);
  }
  MI_REQUIRE(n >= 1 && ldw >= k && ldv >= n && ld_residual >= n, "gemm_skinny_addnorm_bf16: a row stride is shorter than its row");
  MI_REQUIRE(residual && norm_weight && values && sumsq, "gemm_skinny_addnorm_bf16: needs residual, norm weight and both outputs");
  FoldArgs args = {};
  args.part_acc = part_acc;
  args.part_ml = part_ml;
  args.num_splits = num_splits;
  args.attn_heads = heads;
  args.attn_head_dim = head_dim;
  args.residual = residual;
  args.ld_residual = ld_residual;
  args.norm_weight = (const bf16_t*)norm_weight;
  args.sumsq_out = sumsq;
  const bf16_t* wp = (const bf16_t*)w;
  const bf16_t* ap = from_attention ? wp : (const bf16_t*)a;  // (never read when the activations are made in the kernel)
  if (from_attention) lda = ldw;
  bf16_t* cp = (bf16_t*)values;
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "gemm_skinny_addnorm_bf16: cannot read the device's compute unit count");
  const int fpb = features_per_block_for(n, cus, 4);
  const int blocks = ceil_div(n, fpb);
  const int threads = 64 * SK_WAVES;
  const bool lines = whole_lines(w, ldw, n, k);
#define SK_ADDNORM(NT_, U_)                                                                                        \
  if (from_attention && lines)                                                                                     \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_ADDNORM, PRO_ATTN, true><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldv, m, n, k, fpb, args); \
  else if (from_attention)                                                                                         \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_ADDNORM, PRO_ATTN><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldv, m, n, k, fpb, args); \
  else if (lines)                                                                                                  \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_ADDNORM, PRO_NONE, true><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldv, m, n, k, fpb, args); \
  else                                                                                                             \
    gemm_skinny_bf16_kernel<NT_, U_, EPI_ADDNORM><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldv, m, n, k, fpb, args)
  switch (ceil_div(fpb, 16)) {
    case 1: SK_ADDNORM(1, 8); break;
    case 2: SK_ADDNORM(2, 8); break;
    case 3: SK_ADDNORM(3, 4); break;
    default: SK_ADDNORM(4, 2); break;
  }
#undef SK_ADDNORM
  MI_CHECK_LAUNCH("gemm_skinny_addnorm_bf16");
  return MI_OK;
}

// The gated product on rows whose norm factor is still apart (PRO_SCALED): a = the values of
// mi_gemm_skinny_addnorm_bf16, sumsq[pieces][m] its sums of squares; out[m, n] =
// silu(f * a . gate^T) * (f * a . up^T) with f = rsqrt(sum of the row's pieces / k + eps).
extern "C" int mi_gemm_skinny_swiglu_scaled_bf16(const void* a, int64_t lda, const float* sumsq, int pieces, float eps,
                                                 const void* w, int64_t ldw, void* out, int64_t ldo, int m, int n,
                                                 int k, hipStream_t stream) {
  MI_REQUIRE(mi_gemm_skinny_bf16_supported(m, n, k, lda, ldw),
             "gemm_skinny_swiglu_scaled_bf16: takes 1 <= m <= 16, k a multiple of 32, rows aligned to 16 bytes; "
             "got m=%d n=%d k=%d lda=%lld ldw=%lld", m, n, k, (long long)lda, (long long)ldw);
  MI_REQUIRE(lda >= k && ldw >= k && ldo >= n, "gemm_skinny_swiglu_scaled_bf16: a row stride is shorter than its row");
  MI_REQUIRE(sumsq && pieces >= 1 && pieces <= SK_SCALE_PARTS * SK_SCALE_PIECES && eps >= 0.f,
             "gemm_skinny_swiglu_scaled_bf16: needs the rows' sums of squares in 1..%d pieces, got %d",
             SK_SCALE_PARTS * SK_SCALE_PIECES, pieces);
  FoldArgs args = {};
  args.sumsq_in = sumsq;
  args.sumsq_pieces = pieces;
  args.norm_eps = eps;
  args.norm_width = k;
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "gemm_skinny_swiglu_scaled_bf16: cannot read the device's compute unit count");
  const int fpb = features_per_block_for(n, cus, 2);
  const int blocks = ceil_div(n, fpb);
  const int threads = 64 * SK_WAVES;
  const bool lines = whole_lines(w, ldw, 2 * (int64_t)n, k);
#define SK_SCALED(NT_, U_, LINES_)                                                          \
  gemm_skinny_bf16_kernel<NT_, U_, EPI_GATED, PRO_SCALED, LINES_><<<blocks, threads, 0, stream>>>( \
      (const bf16_t*)a, lda, (const bf16_t*)w, ldw, (bf16_t*)out, ldo, m, n, k, fpb, args)
  if (fpb <= 16) {
    if (lines) SK_SCALED(1, 4, true); else SK_SCALED(1, 4, false);
  } else {
    if (lines) SK_SCALED(2, 4, true); else SK_SCALED(2, 2, false);
  }
#undef SK_SCALED
  MI_CHECK_LAUNCH("gemm_skinny_swiglu_scaled_bf16");
  return MI_OK;
}

template <int EPI>
static int skinny_gated(const void* a, int64_t lda, const void* w, int64_t ldw, void* out, int64_t ldo, int m, int n,
                        int k, const FoldArgs& nothing_folded, hipStream_t stream);

// out[m, n] = silu(a . gate^T) * (a . up^T) with w = [gate; up] stacked, [2n, k].
extern "C" int mi_gemm_skinny_swiglu_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, void* out,
                                          int64_t ldo, int m, int n, int k, hipStream_t stream) {
  const FoldArgs nothing_folded = {};
  return skinny_gated<EPI_GATED>(a, lda, w, ldw, out, ldo, m, n, k, nothing_folded, stream);
}

// out[m, n] = gelu_tanh(a . gate^T) * (a . up^T) with w = [gate; up] stacked, [2n, k].
extern "C" int mi_gemm_skinny_geglu_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, void* out,
                                         int64_t ldo, int m, int n, int k, hipStream_t stream) {
  const FoldArgs nothing_folded = {};
  return skinny_gated<EPI_GATED_GELU>(a, lda, w, ldw, out, ldo, m, n, k, nothing_folded, stream);
}

// out[m, n] = g * logistic(slope * g) * (u + 1), g = min(a . gate^T + bias[:n], limit), u = clamp(a . up^T +
// bias[n:], -limit, limit), with w = [gate; up] stacked, [2n, k], and bias float32 [2n] or null (none).
extern "C" int mi_gemm_skinny_clamped_glu_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, const float* bias,
                                               float limit, float slope, void* out, int64_t ldo, int m, int n, int k,
                                               hipStream_t stream) {
  MI_REQUIRE(limit > 0.f, "gemm_skinny_clamped_glu_bf16: needs a positive limit");
  FoldArgs fold = {};
  fold.glu_bias = bias;
  fold.glu_limit = limit;
  fold.glu_slope = slope;
  return skinny_gated<EPI_GATED_CLAMPED>(a, lda, w, ldw, out, ldo, m, n, k, fold, stream);
}

template <int EPI>
static int skinny_gated(const void* a, int64_t lda, const void* w, int64_t ldw, void* out, int64_t ldo, int m, int n,
                        int k, const FoldArgs& nothing_folded, hipStream_t stream) {
  MI_REQUIRE(mi_gemm_skinny_wide_bf16_supported(m, n, k, lda, ldw),
             "gemm_skinny_swiglu_bf16: takes 1 <= m <= 32, k a multiple of 32, rows aligned to 16 bytes; "
             "got m=%d n=%d k=%d lda=%lld ldw=%lld", m, n, k, (long long)lda, (long long)ldw);
  MI_REQUIRE(lda >= k && ldw >= k && ldo >= n, "gemm_skinny_swiglu_bf16: a row stride is shorter than its row");
  const bf16_t* ap = (const bf16_t*)a;
  const bf16_t* wp = (const bf16_t*)w;
  bf16_t* cp = (bf16_t*)out;
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "gemm_skinny_swiglu_bf16: cannot read the device's compute unit count");
  const int fpb = features_per_block_for(n, cus, 2);  // two output tiles = four weight tiles
  const int blocks = ceil_div(n, fpb);
  const int threads = 64 * SK_WAVES;
  const bool lines = whole_lines(w, ldw, 2 * (int64_t)n, k);
#define SK_GATED(NT_, U_, LINES_, RT_) \
  gemm_skinny_bf16_kernel<NT_, U_, EPI, PRO_NONE, LINES_, RT_><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldo, m, n, k, fpb, nothing_folded)
  if (m <= 16) {
    if (fpb <= 16) {
      if (lines) SK_GATED(1, 4, true, 1); else SK_GATED(1, 4, false, 1);
    } else {
      if (lines) SK_GATED(2, 4, true, 1); else SK_GATED(2, 2, false, 1);
    }
  } else {  // (two row tiles: fewer k-steps in flight, the registers hold both tiles' sums)
    if (fpb <= 16) {
      if (lines) SK_GATED(1, 4, true, 2); else SK_GATED(1, 4, false, 2);
    } else {
      if (lines) SK_GATED(2, 2, true, 2); else SK_GATED(2, 2, false, 2);
    }
  }
#undef SK_GATED
  MI_CHECK_LAUNCH("gemm_skinny_swiglu_bf16");
  return MI_OK;
}

// The stacked q|k|v projection of an attention layer with the rotary encoding and the
// cache write in its last step: q_out[m, q_heads*head_dim] gets the rotated queries, the
// rotated keys and the values go to their slots (slot_mapping[m]; kv_heads = 0: queries only,
// w then holds the query rows alone).  Half-paired rotation over the whole head,
// cos/sin [m, head_dim/2] float32.  With `sumsq` the rows are a norm's output but for the
// rows' factors (PRO_SCALED, as in mi_gemm_skinny_swiglu_scaled_bf16).
// out[m, n] = one step of the gated recurrence per row from the stacked projection [z; x; g]
// (EPI_GRU): at most 16 rows, each the only token of its request in this step.
extern "C" int mi_gemm_skinny_gru_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, const float* bz,
                                       const float* bx, float* state, int64_t state_stride, const int* slots,
                                       int num_slots, void* out, int64_t ldo, int m, int n, int k, hipStream_t stream) {
  MI_REQUIRE(mi_gemm_skinny_bf16_supported(m, n, k, lda, ldw),
             "gemm_skinny_gru_bf16: takes 1 <= m <= 16, k a multiple of 32, rows aligned to 16 bytes; "
             "got m=%d n=%d k=%d lda=%lld ldw=%lld", m, n, k, (long long)lda, (long long)ldw);
  MI_REQUIRE(lda >= k && ldw >= k && ldo >= n && state_stride >= n && num_slots >= 0 && bz && bx && state && slots,
             "gemm_skinny_gru_bf16: a row stride is shorter than its row, or an argument is missing");
  const bf16_t* ap = (const bf16_t*)a;
  const bf16_t* wp = (const bf16_t*)w;
  bf16_t* cp = (bf16_t*)out;
  FoldArgs fold = {};
  fold.gru_state = state;
  fold.gru_state_stride = state_stride;
  fold.gru_slots = slots;
  fold.gru_num_slots = num_slots;
  fold.gru_bz = bz;
  fold.gru_bx = bx;
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "gemm_skinny_gru_bf16: cannot read the device's compute unit count");
  const int fpb = features_per_block_for(n, cus, 1);  // one output tile = three weight tiles
  const int blocks = ceil_div(n, fpb);
  const int threads = 64 * SK_WAVES;
  if (whole_lines(w, ldw, 3 * (int64_t)n, k)) {
    gemm_skinny_bf16_kernel<1, 4, EPI_GRU, PRO_NONE, true><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldo, m, n, k,
                                                                                           fpb, fold);
  } else {
    gemm_skinny_bf16_kernel<1, 4, EPI_GRU><<<blocks, threads, 0, stream>>>(ap, lda, wp, ldw, cp, ldo, m, n, k, fpb, fold);
  }
  MI_CHECK_LAUNCH("gemm_skinny_gru_bf16");
  return MI_OK;
}

static int rope_product(const char* name, const void* a, int64_t lda, const float* sumsq, int pieces, float eps,
                        const void* w, int64_t ldw, void* q_out, int64_t ldq, const float* cos_t,
                        const float* sin_t, const int* slot_mapping, void* k_pages, void* v_pages, int m, int k,
                        int q_heads, int kv_heads, int head_dim, int page_size, int num_pages, int v_transposed,
                        hipStream_t stream) {
  MI_REQUIRE(q_heads >= 1 && kv_heads >= 0 && head_dim >= 32 && head_dim % 32 == 0,
             "%s: takes head_dim a multiple of 32; got q_heads=%d kv_heads=%d head_dim=%d", name, q_heads, kv_heads,
             head_dim);
  const int n = (q_heads + 2 * kv_heads) * head_dim;
  MI_REQUIRE(mi_gemm_skinny_wide_bf16_supported(m, n, k, lda, ldw),
             "%s: takes 1 <= m <= 32, k a multiple of 32, rows aligned to 16 bytes; "
             "got m=%d n=%d k=%d lda=%lld ldw=%lld", name, m, n, k, (long long)lda, (long long)ldw);
  MI_REQUIRE(lda >= k && ldw >= k && ldq >= (int64_t)q_heads * head_dim && ldq % 4 == 0,
             "%s: a row stride is shorter than its row or not 8-byte aligned", name);
  MI_REQUIRE(cos_t && sin_t, "%s: needs the rotation tables", name);
  MI_REQUIRE(kv_heads == 0 || (slot_mapping && k_pages && v_pages && page_size > 0 && num_pages > 0),
             "%s: pages and slots are needed to write keys and values", name);
  MI_REQUIRE(!sumsq || (pieces >= 1 && pieces <= SK_SCALE_PARTS * SK_SCALE_PIECES && eps >= 0.f),
             "%s: needs the rows' sums of squares in 1..%d pieces, got %d", name, SK_SCALE_PARTS * SK_SCALE_PIECES,
             pieces);
  FoldArgs fold = {};
  fold.cos_t = cos_t;
  fold.sin_t = sin_t;
  fold.slot_mapping = slot_mapping;
  fold.k_pages = (bf16_t*)k_pages;
  fold.v_pages = (bf16_t*)v_pages;
  fold.q_heads = q_heads;
  fold.kv_heads = kv_heads;
  fold.head_dim = head_dim;
  fold.page_size = page_size;
  fold.v_transposed = v_transposed;
  fold.sumsq_in = sumsq;
  fold.sumsq_pieces = pieces;
  fold.norm_eps = eps;
  fold.norm_width = k;
  // pairs per block: an even share over the CUs in whole rounds, as for the plain product
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "%s: cannot read the device's compute unit count", name);
  const int total_pairs = n / 2;
  const int rounds = ceil_div(total_pairs, cus * 16);
  int pairs_per_block = ceil_div(ceil_div(total_pairs, cus * rounds), 4) * 4;
  if (pairs_per_block > 16) pairs_per_block = 16;
  const int blocks = ceil_div(total_pairs, pairs_per_block);
  const bool lines = whole_lines(w, ldw, n, k);
#define SK_ROPE(U_, PRO_, LINES_, RT_)                                                                \
  gemm_skinny_bf16_kernel<1, U_, EPI_ROPE, PRO_, LINES_, RT_><<<blocks, 64 * SK_WAVES, 0, stream>>>( \
      (const bf16_t*)a, lda, (const bf16_t*)w, ldw, (bf16_t*)q_out, ldq, m, n, k, pairs_per_block, fold)
  if (sumsq) {
    MI_REQUIRE(m <= SK_MAX_ROWS, "%s: rows with their norm factor apart come 16 at most, got %d", name, m);
    if (lines) SK_ROPE(8, PRO_SCALED, true, 1); else SK_ROPE(8, PRO_SCALED, false, 1);
  } else if (m <= 16) {
    if (lines) SK_ROPE(8, PRO_NONE, true, 1); else SK_ROPE(8, PRO_NONE, false, 1);
  } else {
    if (lines) SK_ROPE(4, PRO_NONE, true, 2); else SK_ROPE(4, PRO_NONE, false, 2);
  }
#undef SK_ROPE
  MI_CHECK_LAUNCH(name);
  return MI_OK;
}

extern "C" int mi_gemm_skinny_rope_bf16(const void* a, int64_t lda, const void* w, int64_t ldw, void* q_out,
                                        int64_t ldq, const float* cos_t, const float* sin_t,
                                        const int* slot_mapping, void* k_pages, void* v_pages, int m, int k,
                                        int q_heads, int kv_heads, int head_dim, int page_size, int num_pages,
                                        int v_transposed, hipStream_t stream) {
  return rope_product("gemm_skinny_rope_bf16", a, lda, nullptr, 0, 0.f, w, ldw, q_out, ldq, cos_t, sin_t, slot_mapping,
                      k_pages, v_pages, m, k, q_heads, kv_heads, head_dim, page_size, num_pages, v_transposed, stream);
}

// The same on rows whose norm factor is still apart: a = the values of mi_gemm_skinny_addnorm_bf16,
// sumsq[pieces][m] its sums of squares; the products are multiplied with
// rsqrt(sum of the row's pieces / k + eps) before they are rounded and rotated.
extern "C" int mi_gemm_skinny_rope_scaled_bf16(const void* a, int64_t lda, const float* sumsq, int pieces, float eps,
                                               const void* w, int64_t ldw, void* q_out, int64_t ldq,
                                               const float* cos_t, const float* sin_t, const int* slot_mapping,
                                               void* k_pages, void* v_pages, int m, int k, int q_heads,
                                               int kv_heads, int head_dim, int page_size, int num_pages,
                                               int v_transposed, hipStream_t stream) {
  MI_REQUIRE(sumsq, "gemm_skinny_rope_scaled_bf16: needs the rows' sums of squares");
  return rope_product("gemm_skinny_rope_scaled_bf16", a, lda, sumsq, pieces, eps, w, ldw, q_out, ldq, cos_t, sin_t,
                      slot_mapping, k_pages, v_pages, m, k, q_heads, kv_heads, head_dim, page_size, num_pages,
                      v_transposed, stream);
}

// The stacked input projection of a layer whose sublayers read one norm (EPI_LAYER_IN), for at most 32
// rows.  w: [q heads | k heads | v heads | gate_rows | ff | ff] rows of k; kv_heads = 0: no keys and values;
// ff = 0: no feed-forward; gate_rows = 0: no head gates (else at least q_heads, a multiple of 8).  head_dim,
// v_dim and 2 * rot_half are multiples of 8, ff of 4.  q_out [m, q_heads*head_dim] gets the rotated queries
// (cos/sin float32 [m, rot_half]; the dims past 2 * rot_half pass), keys and values go to their
// slots, gates to gate_out [m, q_heads], the feed-forward's activation to act_out [m, ff]:
// limit > 0: min(g, limit) * logistic(slope * min(g, limit)) * (clamp(u, -limit, limit) + 1), else silu(g) * u.
// qkv_bias: float32 [q | k | v] or null.  With `sumsq` the rows are a norm's output but for their factors, as
// in mi_gemm_skinny_rope_scaled_bf16 (16 rows at most).
extern "C" int mi_gemm_skinny_layer_in_bf16(const void* a, int64_t lda, const float* sumsq, int pieces, float eps,
                                            const void* w, int64_t ldw, void* q_out, int64_t ldq, const float* cos_t,
                                            const float* sin_t, const int* slot_mapping, void* k_pages, void* v_pages,
                                            const float* qkv_bias, void* gate_out, int64_t ld_gate, void* act_out,
                                            int64_t ld_act, int m, int k, int q_heads, int kv_heads, int head_dim,
                                            int v_dim, int rot_half, int gate_rows, int ff, float limit, float slope,
                                            int page_size, int num_pages, int v_transposed, hipStream_t stream) {
  MI_REQUIRE(q_heads >= 1 && kv_heads >= 0 && head_dim >= 8 && head_dim % 8 == 0 && v_dim >= 8 && v_dim % 8 == 0 &&
                 rot_half >= 0 && rot_half % 4 == 0 && 2 * rot_half <= head_dim && ff >= 0 && ff % 4 == 0 &&
                 gate_rows >= 0 && gate_rows % 8 == 0 && (gate_rows == 0 || gate_rows >= q_heads),
             "gemm_skinny_layer_in_bf16: q_heads=%d kv_heads=%d head_dim=%d v_dim=%d rot_half=%d gate_rows=%d ff=%d not taken",
             q_heads, kv_heads, head_dim, v_dim, rot_half, gate_rows, ff);
  const int64_t rows = (int64_t)(q_heads + kv_heads) * head_dim + (int64_t)kv_heads * v_dim + gate_rows + 2 * (int64_t)ff;
  MI_REQUIRE(rows < (1ll << 31) && mi_gemm_skinny_wide_bf16_supported(m, (int)rows, k, lda, ldw),
             "gemm_skinny_layer_in_bf16: takes 1 <= m <= 32, k a multiple of 32, rows aligned to 16 bytes; "
             "got m=%d k=%d lda=%lld ldw=%lld", m, k, (long long)lda, (long long)ldw);
  MI_REQUIRE(lda >= k && ldw >= k && ldq >= (int64_t)q_heads * head_dim && ldq % 4 == 0,
             "gemm_skinny_layer_in_bf16: a row stride is shorter than its row or not 8-byte aligned");
  MI_REQUIRE(rot_half == 0 || (cos_t && sin_t), "gemm_skinny_layer_in_bf16: needs the rotation tables");
  MI_REQUIRE(kv_heads == 0 || (slot_mapping && k_pages && v_pages && page_size > 0 && num_pages > 0),
             "gemm_skinny_layer_in_bf16: pages and slots are needed to write keys and values");
  MI_REQUIRE(gate_rows == 0 || (gate_out && ld_gate >= q_heads), "gemm_skinny_layer_in_bf16: the head gates have no place to go");
  MI_REQUIRE(ff == 0 || (act_out && ld_act >= ff && ld_act % 4 == 0 && (uintptr_t)act_out % 8 == 0),
             "gemm_skinny_layer_in_bf16: the feed-forward's activation has no place to go, or one not aligned to 8 bytes");
  MI_REQUIRE((uintptr_t)q_out % 8 == 0 && (uintptr_t)cos_t % 16 == 0 && (uintptr_t)sin_t % 16 == 0 && (uintptr_t)qkv_bias % 16 == 0,
             "gemm_skinny_layer_in_bf16: outputs, tables and biases must be aligned to their vector accesses");
  MI_REQUIRE(!sumsq || (m <= SK_MAX_ROWS && pieces >= 1 && pieces <= SK_SCALE_PARTS * SK_SCALE_PIECES && eps >= 0.f),
             "gemm_skinny_layer_in_bf16: rows with their norm factor apart come 16 at most and in 1..%d pieces, got %d and %d",
             SK_SCALE_PARTS * SK_SCALE_PIECES, m, pieces);
  FoldArgs fold = {};
  fold.cos_t = cos_t;
  fold.sin_t = sin_t;
  fold.slot_mapping = slot_mapping;
  fold.k_pages = (bf16_t*)k_pages;
  fold.v_pages = (bf16_t*)v_pages;
  fold.q_heads = q_heads;
  fold.kv_heads = kv_heads;
  fold.head_dim = head_dim;
  fold.page_size = page_size;
  fold.v_transposed = v_transposed;
  fold.rot_half = rot_half;
  fold.v_dim = v_dim;
  fold.gate_rows = gate_rows;
  fold.ff = ff;
  fold.qkv_bias = qkv_bias;
  fold.gate_out = (bf16_t*)gate_out;
  fold.ld_gate = ld_gate;
  fold.act_out = (bf16_t*)act_out;
  fold.ld_act = ld_act;
  fold.glu_limit = limit;
  fold.glu_slope = slope;
  fold.sumsq_in = sumsq;
  fold.sumsq_pieces = pieces;
  fold.norm_eps = eps;
  fold.norm_width = k;
  const int cus = compute_units();
  MI_REQUIRE(cus > 0, "gemm_skinny_layer_in_bf16: cannot read the device's compute unit count");
  const int n = (int)(rows / 2);  // pairs
  const int fpb = features_per_block_for(n, cus, 2);
  const int blocks = ceil_div(n, fpb);
  const bool lines = whole_lines(w, ldw, rows, k);
#define SK_LAYER_IN(NT_, U_, PRO_, LINES_, RT_)                                                               \
  gemm_skinny_bf16_kernel<NT_, U_, EPI_LAYER_IN, PRO_, LINES_, RT_><<<blocks, 64 * SK_WAVES, 0, stream>>>( \
      (const bf16_t*)a, lda, (const bf16_t*)w, ldw, (bf16_t*)q_out, ldq, m, n, k, fpb, fold)
  if (fpb <= 16) {
    if (sumsq) { if (lines) SK_LAYER_IN(1, 8, PRO_SCALED, true, 1); else SK_LAYER_IN(1, 8, PRO_SCALED, false, 1); }
    else if (m <= 16) { if (lines) SK_LAYER_IN(1, 8, PRO_NONE, true, 1); else SK_LAYER_IN(1, 8, PRO_NONE, false, 1); }
    else { if (lines) SK_LAYER_IN(1, 4, PRO_NONE, true, 2); else SK_LAYER_IN(1, 4, PRO_NONE, false, 2); }
  } else {
    if (sumsq) { if (lines) SK_LAYER_IN(2, 4, PRO_SCALED, true, 1); else SK_LAYER_IN(2, 2, PRO_SCALED, false, 1); }
    else if (m <= 16) { if (lines) SK_LAYER_IN(2, 4, PRO_NONE, true, 1); else SK_LAYER_IN(2, 2, PRO_NONE, false, 1); }
    else { if (lines) SK_LAYER_IN(2, 2, PRO_NONE, true, 2); else SK_LAYER_IN(2, 2, PRO_NONE, false, 2); }
  }
#undef SK_LAYER_IN
  MI_CHECK_LAUNCH("gemm_skinny_layer_in_bf16");
  return MI_OK;
}
