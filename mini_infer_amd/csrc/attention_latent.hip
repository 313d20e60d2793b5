// Attention over latent rows on the matrix cores: one key row [c | r] per token for all heads, whose front
// part c is the value as well, read in place from the pages (bfloat16).  Decoded tokens and portions of
// prompts alike.
//
// The heads of a request's tokens are the rows of one tall query matrix (row = token * heads + head): every
// row meets the same keys, so a key tile read once serves all of them.  A wave owns 16 rows, their
// queries and their accumulators in registers; a block's waves (1, 2 or 4) share key tiles of 32, which come
// straight from memory into LDS, two buffers: while one is worked on, the next is on its way.  The operands'
// LDS reads are asked for a batch ahead of the MFMAs that use them: at these register counts a wave has its SIMD
// to itself and nobody else hides their latency (two waves a SIMD with half the registers each measured
// slower: 547 against 323 us for 512 tokens over 4,096 keys, 32 heads of 512 + 64).
//
//   scores        S^T = K Q^T   (MFMA 16x16x32, keys first operand, rows second): a lane ends with keys
//                 4 * quad .. + 3 of both 16-key halves for row lane % 16
//   softmax       online, per row: the lane's eight scores, then the other three quads by two exchanges
//   values        O^T = C^T P^T: the lane's eight probabilities are the second operand as they lie (k-slot
//                 (quad, j) is key 4 * quad + j % 4 of half j / 4), and ds_read_b64_tr_b16 fetches the same
//                 keys of 16 latent columns transposed, so neither P nor C is ever rewritten
//
// In LDS a row is padded to whole groups of eight 16-byte chunks; chunk c of key k lies at place
// c ^ f(k), f(k) = ((k % 4) * 2) | (k / 4 % 2): eight keys' pieces of one chunk, and four keys' pieces of two
// neighbouring chunks, lie in different banks.
//
// Keys are cut into `splits` ranges (blockIdx.y); a range leaves its accumulators, maximum (natural log
// units) and sum, and `latent_combine` puts the ranges of a (token, head) together: four groups of lanes take
// every fourth range each, four columns a lane, all their loads asked for at once, and meet in LDS in
// group order.
#include "common.h"

#include <math.h>

namespace {

typedef float f32x4_l __attribute__((ext_vector_type(4)));
typedef short s16x4_l __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) void lds_void;
typedef const __attribute__((address_space(1))) void global_void;

#define KEY_TILE 32

struct LatentShape {
  const int* block_table;
  const int* cu;
  const int* positions;
  const float* sinks;
  int64_t q_stride, out_stride;
  int max_blocks, num_requests, heads, rank, width, page_size, window, splits, single;
  float scale_log2;  // scale * log2(e)
};

__device__ __forceinline__ int swizzle_of(int key) { return ((key & 3) << 1) | ((key >> 2) & 1); }

// Which rows this block works on: request, its first token in the step, its tokens, first row.  False: past the
// last tile.  The same answer in all threads.
__device__ __forceinline__ bool find_rows(const LatentShape& s, int rows_a_block, int tile, int& request, int& token0,
                                          int& tokens, int& row0) {
  if (s.single) {
    const int per = (s.heads + rows_a_block - 1) / rows_a_block;
    request = tile / per;
    if (request >= s.num_requests) return false;
    token0 = request, tokens = 1, row0 = (tile % per) * rows_a_block;
    return true;
  }
  const int lane = threadIdx.x % MI_WAVE;
  int before = 0;
  for (int base = 0; base < s.num_requests; base += MI_WAVE) {
    const int b = base + lane;
    const int n = b < s.num_requests ? s.cu[b + 1] - s.cu[b] : 0;
    const int tiles = n > 0 ? (n * s.heads + rows_a_block - 1) / rows_a_block : 0;
    int upto = tiles;
#pragma unroll
    for (int off = 1; off < MI_WAVE; off <<= 1) {
      const int other = __shfl_up(upto, off, MI_WAVE);
      if (lane >= off) upto += other;
    }
    const uint64_t past = __ballot(before + upto > tile);
    if (past != 0) {
      const int at = __builtin_ctzll(past);
      const int start = before + __shfl(upto, at, MI_WAVE) - __shfl(tiles, at, MI_WAVE);
      request = base + at;
      token0 = s.cu[request];
      tokens = s.cu[request + 1] - token0;
      row0 = (tile - start) * rows_a_block;
      return true;
    }
    before += __shfl(upto, MI_WAVE - 1, MI_WAVE);
  }
  return false;
}

// KS: steps of 32 elements of a key row, VT: tiles of 16 latent columns (EXACT: these, else at most these)
template <int KS, int VT, bool EXACT, int WAVES>
__global__ __launch_bounds__(WAVES * MI_WAVE, 1) void attn_latent_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ k_pages, bf16_t* __restrict__ out,
    float* __restrict__ part_acc, float* __restrict__ part_ml, LatentShape s) {
  constexpr int MAX_GROUPS = (KS + 1) / 2;
  // (an array of its own for each buffer: the compiler then sees that what is fetched into one does not touch
  // what is read from the other, and waits for nothing between)
  __shared__ __align__(16) unsigned char tile_even[KEY_TILE * MAX_GROUPS * 128];
  __shared__ __align__(16) unsigned char tile_odd[KEY_TILE * MAX_GROUPS * 128];
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / MI_WAVE), lane = threadIdx.x % MI_WAVE;
  const int col = lane % 16, quad = lane / 16;
  int request, token0, tokens, block_row0;
  if (!find_rows(s, 16 * WAVES, blockIdx.x, request, token0, tokens, block_row0)) return;
  const int rows = tokens * s.heads;

  // this lane's row
  const int row = block_row0 + wave * 16 + col;
  const bool real = row < rows;
  const int token = token0 + min(row, rows - 1) / s.heads, head = min(row, rows - 1) % s.heads;
  const int pos = s.positions[token];
  const int low = s.window > 0 ? max(0, pos - s.window + 1) : 0;

  // the block's keys, and this range's tiles of them
  const int first_pos = s.positions[token0 + block_row0 / s.heads];
  const int last_pos = s.positions[token0 + (min(block_row0 + 16 * WAVES, rows) - 1) / s.heads];
  const int keys = last_pos + 1;
  const int key0 = s.window > 0 ? max(0, first_pos - s.window + 1) / KEY_TILE * KEY_TILE : 0;
  const int all = (keys - key0 + KEY_TILE - 1) / KEY_TILE;
  const int per = (all + s.splits - 1) / s.splits;
  const int t_begin = blockIdx.y * per, t_end = min(all, t_begin + per);

  const int groups = EXACT ? MAX_GROUPS : (s.width / 8 + 7) / 8;  // groups of eight chunks a row has in LDS
  const int pitch = groups * 128;            // bytes of a row
  const int ksteps = EXACT ? KS : (s.width + 31) / 32, vtiles = EXACT ? VT : s.rank / 16;
  const int* table = s.block_table + (int64_t)request * s.max_blocks;

  // the rows' queries: operand lane (quad, col) holds elements 32 * step + 8 * quad .. + 7 of row col
  bf16x8_t queries[KS];
  {
    const bf16_t* mine = q + (int64_t)token * s.q_stride + (int64_t)head * s.width + quad * 8;
#pragma unroll
    for (int i = 0; i < KS; ++i) {
      const bf16x8_t nothing = {};
      queries[i] = (i * 32 + quad * 8 < s.width) ? *reinterpret_cast<const bf16x8_t*>(mine + i * 32) : nothing;
    }
  }

  // key `lane % 32` of a tile (past the last one: the last) and its page as the table has it; the slot is made of
  // them where the tile is fetched, so that nothing waits for the table meanwhile (a page that a window has
  // passed: page 0, whose keys the mask leaves out)
  struct Where {
    int page, offset;
  };
  auto look_up = [&](int t) {
    const int key = min(key0 + t * KEY_TILE + (lane & (KEY_TILE - 1)), keys - 1);
    const int n = key / s.page_size;
    return Where{table[min(n, s.max_blocks - 1)], key - n * s.page_size};
  };
  const int loads = KEY_TILE / 8 * groups;       // wave-wide loads a tile takes: eight groups each
  const unsigned inverse = 65536u / groups + 1;  // g / groups for g < 512 is (g * inverse) >> 16
  auto fetch = [&](unsigned char* tile, Where where) {
    const int slot = max(where.page, 0) * s.page_size + where.offset;
    constexpr int EACH = (KEY_TILE / 8 * MAX_GROUPS + WAVES - 1) / WAVES;
#pragma unroll
    for (int n = 0; n < EACH; ++n) {
      const int i = n * WAVES + wave;
      if ((EXACT && (KEY_TILE / 8 * MAX_GROUPS) % WAVES == 0) || i < loads) {
        const unsigned g = i * 8 + lane / 8;
        const int r = (int)((g * inverse) >> 16);
        const int chunk = (int)(g - r * groups) * 8 + ((lane % 8) ^ swizzle_of(r));
        const int from = __shfl(slot, r, MI_WAVE);
        const bf16_t* src = k_pages + (int64_t)from * s.width + (chunk * 8 < s.width ? chunk * 8 : 0);
        __builtin_amdgcn_global_load_lds((global_void*)src, (lds_void*)(tile + i * 1024), 16, 0, 0);
      }
    }
  };

  f32x4_l acc[VT];
#pragma unroll
  for (int v = 0; v < VT; ++v) acc[v] = f32x4_l{0.f, 0.f, 0.f, 0.f};
  float top = -INFINITY, sum = 0.f;

  // where this lane's pieces lie in a tile
  uint32_t key_at[2], value_at[4];
#pragma unroll
  for (int odd = 0; odd < 2; ++odd) key_at[odd] = col * pitch + (((odd * 4 + quad) ^ swizzle_of(col)) * 16);
#pragma unroll
  for (int j = 0; j < 4; ++j)
    value_at[j] = (4 * quad + col / 4) * pitch + (((j * 2 + (col % 4) / 2) ^ swizzle_of(4 * quad + col / 4)) * 16) + (col & 1) * 8;

  auto work = [&](const unsigned char* tile, int t) {
    f32x4_l score[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    constexpr int SB = 3, S_BATCHES = (KS + SB - 1) / SB;
    bf16x8_t lower[2][SB], upper[2][SB];
    auto read_keys = [&](int batch) {
#pragma unroll
      for (int j = 0; j < SB; ++j) {
        const int i = batch * SB + j;
        if (i < KS && i < ksteps) {
          const unsigned char* at = tile + key_at[i & 1] + (i / 2) * 128;
          lower[batch & 1][j] = *reinterpret_cast<const bf16x8_t*>(at);
          upper[batch & 1][j] = *reinterpret_cast<const bf16x8_t*>(at + 16 * pitch);
        }
      }
    };
    read_keys(0);
#pragma unroll
    for (int batch = 0; batch < S_BATCHES; ++batch) {
      if (batch + 1 < S_BATCHES) read_keys(batch + 1);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int j = 0; j < SB; ++j) {
        const int i = batch * SB + j;
        if (i < KS && i < ksteps) {
          score[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lower[batch & 1][j], queries[i], score[0], 0, 0, 0);
          score[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(upper[batch & 1][j], queries[i], score[1], 0, 0, 0);
        }
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    // (the first values are asked for before the softmax that they wait for)
    constexpr int VB = 4, V_BATCHES = (VT + VB - 1) / VB;
    bf16x8_t values[2][VB];
    auto read_values = [&](int batch) {
      typedef __attribute__((address_space(3))) s16x4_l lds_s16x4;
      typedef short s16x8_l __attribute__((ext_vector_type(8)));
#pragma unroll
      for (int j = 0; j < VB; ++j) {
        const int v = batch * VB + j;
        if (v < vtiles) {
          const unsigned char* at = tile + value_at[v & 3] + (v / 4) * 128;
          const s16x4_l first = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)at);
          const s16x4_l second = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(at + 16 * pitch));
          const s16x8_l both = __builtin_shufflevector(first, second, 0, 1, 2, 3, 4, 5, 6, 7);
          values[batch & 1][j] = __builtin_bit_cast(bf16x8_t, both);
        }
      }
    };
    read_values(0);
    const int base_key = key0 + t * KEY_TILE + 4 * quad;
    float highest = -INFINITY;
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = base_key + 16 * half + j;
        const float v = (key <= pos && key >= low) ? score[half][j] * s.scale_log2 : -INFINITY;
        score[half][j] = v;
        highest = fmaxf(highest, v);
      }
    highest = fmaxf(highest, __shfl_xor(highest, 16, MI_WAVE));
    highest = fmaxf(highest, __shfl_xor(highest, 32, MI_WAVE));
    const float now = fmaxf(top, highest);
    const float reference = now == -INFINITY ? 0.f : now;
    if (__ballot(now > top) != 0) {  // some row's maximum rose: what has been added up is scaled down
      const float shrink = __builtin_amdgcn_exp2f(top - reference);
      sum *= shrink;
#pragma unroll
      for (int v = 0; v < VT; ++v) acc[v] *= shrink;
      top = now;
    }
    bf16x8_t p;
    float added = 0.f;
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float e = __builtin_amdgcn_exp2f(score[half][j] - reference);
        p[half * 4 + j] = (bf16_t)e;
        added += e;
      }
    sum += added;  // (this lane's keys; the quads meet at the end)
#pragma unroll
    for (int batch = 0; batch < V_BATCHES; ++batch) {
      if (batch + 1 < V_BATCHES) read_values(batch + 1);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int j = 0; j < VB; ++j) {
        const int v = batch * VB + j;
        if (v < VT && v < vtiles) acc[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(values[batch & 1][j], p, acc[v], 0, 0, 0);
      }
      __builtin_amdgcn_sched_barrier(0);
    }
  };
  auto whole = [&]() {  // the tile asked for last is there, for all waves, and nobody reads the other buffer any more
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
  };

  Where next = {0, 0};
  if (t_begin < t_end) {
    fetch(tile_even, look_up(t_begin));
    if (t_begin + 1 < t_end) next = look_up(t_begin + 1);
  }
  for (int t = t_begin; t < t_end; t += 2) {
    whole();
    if (t + 1 < t_end) {
      fetch(tile_odd, next);
      if (t + 2 < t_end) next = look_up(t + 2);
    }
    work(tile_even, t);
    if (t + 1 >= t_end) break;
    whole();
    if (t + 2 < t_end) {
      fetch(tile_even, next);
      if (t + 3 < t_end) next = look_up(t + 3);
    }
    work(tile_odd, t + 1);
  }
  sum += __shfl_xor(sum, 16, MI_WAVE);
  sum += __shfl_xor(sum, 32, MI_WAVE);
  if (!real) return;
  if (s.splits == 1) {
    if (s.sinks != nullptr) sum += __builtin_amdgcn_exp2f(s.sinks[head] * 1.4426950408889634f - top);
    const float inv = 1.0f / sum;
    bf16_t* o = out + (int64_t)token * s.out_stride + (int64_t)head * s.rank + 4 * quad;
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      if (v < vtiles) {
        float r[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) r[j] = acc[v][j] * inv;
        mi_store_cols<bf16_t, 4>(o + v * 16, r);
      }
    }
  } else {
    const int64_t piece = ((int64_t)token * s.heads + head) * s.splits + blockIdx.y;
    float* o = part_acc + piece * s.rank + 4 * quad;
#pragma unroll
    for (int v = 0; v < VT; ++v)
      if (v < vtiles) *reinterpret_cast<f32x4_l*>(o + v * 16) = acc[v];
    if (quad == 0) {
      part_ml[piece * 2] = top * 0.6931471805599453f;
      part_ml[piece * 2 + 1] = sum;
    }
  }
}

// lane s's value, s the same in all lanes: a register move
__device__ __forceinline__ float of_lane(float v, int s) {
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), s));
}

// EACH: ranges a group takes, at most (4 * EACH >= splits)
template <int EACH>
__global__ __launch_bounds__(512) void latent_combine_kernel(const float* __restrict__ part_acc,
                                                             const float* __restrict__ part_ml, bf16_t* __restrict__ out,
                                                             int64_t out_stride, int heads, int rank, int splits,
                                                             const float* __restrict__ sinks) {
  __shared__ f32x4_l meet[3][128];
  const int t = blockIdx.x, h = blockIdx.y;
  const int lanes = blockDim.x / 4;  // of a group: whole waves
  const int group = __builtin_amdgcn_readfirstlane(threadIdx.x / lanes), place = threadIdx.x % lanes, lane = threadIdx.x % MI_WAVE;
  const int64_t base = ((int64_t)t * heads + h) * splits;
  const bool active = place * 4 < rank;
  const float* src = part_acc + base * rank + (active ? place * 4 : 0);
  f32x4_l v[EACH];
#pragma unroll
  for (int i = 0; i < EACH; ++i)  // (past the last range: that one again, not counted)
    v[i] = *reinterpret_cast<const f32x4_l*>(src + (int64_t)min(group + 4 * i, splits - 1) * rank);
  const float m_s = lane < splits ? part_ml[(base + lane) * 2] : -INFINITY;
  const float l_s = lane < splits ? part_ml[(base + lane) * 2 + 1] : 0.f;
  const float top = wave_max(m_s);
  const float w_s = lane < splits ? expf(m_s - top) : 0.f;
  float all = wave_sum(l_s * w_s);
  if (sinks != nullptr) all += expf(sinks[h] - top);
  f32x4_l sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < EACH; ++i)
    if (group + 4 * i < splits) sum += v[i] * of_lane(w_s, group + 4 * i);
  if (group > 0) meet[group - 1][place] = sum;
  __syncthreads();
  if (group > 0 || !active) return;
#pragma unroll
  for (int g = 0; g < 3; ++g) sum += meet[g][place];
  const float inv = 1.0f / all;
  float r[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) r[j] = sum[j] * inv;
  mi_store_cols<bf16_t, 4>(out + (int64_t)t * out_stride + (int64_t)h * rank + place * 4, r);
}

}  // namespace

// Whether cached rows of rank + rot columns (bfloat16) are taken.
extern "C" int mi_attn_latent_takes(int rank, int rot) {
  return rank > 0 && rank % 16 == 0 && rank <= 512 && rot >= 0 && rot <= 64 && (rank + rot) % 8 == 0;
}

// Waves of a block for steps whose rows (tokens x heads) are `rows` a request at most.
extern "C" int mi_attn_latent_waves(int rows) { return rows <= 16 ? 1 : (rows <= 32 ? 2 : 4); }

// q [tokens, heads * width] (row stride), head by head, width = rank + rot; k_pages [pages * page_size, width]; out [tokens,
// heads * rank] (row stride).  num_tiles blocks of 16 * waves rows: with `single` (every request brings one token)
// requests * ceil(heads / (16 * waves)), else at least sum over requests of ceil(tokens * heads / (16 * waves)).
// part_acc [tokens * heads * splits * rank], part_ml [.. * 2] floats, or null with one split.  window 0: none; sinks
// float32 [heads] or null.
extern "C" int mi_attn_latent(const void* q, int64_t q_stride, const void* k_pages, const int* block_table, int max_blocks,
                              const int* cu, const int* positions, int num_requests, int num_tokens, int num_tiles, int waves,
                              void* out, int64_t out_stride, float* part_acc, float* part_ml, int heads, int rank, int rot,
                              int page_size, float scale, int window, int splits, int single, const float* sinks,
                              hipStream_t stream) {
  const int width = rank + rot;
  MI_REQUIRE(mi_attn_latent_takes(rank, rot), "attn_latent: rows of %d + %d are not taken", rank, rot);
  MI_REQUIRE(num_tokens >= 0 && num_requests >= 0 && heads > 0 && page_size > 0 && max_blocks > 0 && num_tiles >= 0,
             "attn_latent: bad sizes tokens=%d heads=%d page_size=%d", num_tokens, heads, page_size);
  MI_REQUIRE(waves == 1 || waves == 2 || waves == 4, "attn_latent: %d waves a block", waves);
  MI_REQUIRE(q_stride >= (int64_t)heads * width && q_stride % 8 == 0 && out_stride >= (int64_t)heads * rank && out_stride % 4 == 0 &&
                 ((uintptr_t)q | (uintptr_t)k_pages) % 16 == 0 && (uintptr_t)out % 8 == 0,
             "attn_latent: rows are read 16 bytes at a time");
  MI_REQUIRE(splits >= 1 && splits <= 64 && (splits == 1 || (part_acc != nullptr && part_ml != nullptr)), "attn_latent: %d key ranges", splits);
  MI_REQUIRE(window >= 0 && (!single || num_tokens == num_requests), "attn_latent: bad window or step");
  if (num_tokens == 0 || num_requests == 0 || num_tiles == 0) return MI_OK;
  const LatentShape s = {block_table, cu, positions, sinks, q_stride, out_stride, max_blocks, num_requests, heads, rank, width,
                         page_size, window, splits, single, scale * 1.4426950408889634f};
  dim3 grid(num_tiles, splits);
#define MI_LATENT_W(KS, VT, EXACT, WAVES)                                                                      \
  attn_latent_kernel<KS, VT, EXACT, WAVES><<<grid, WAVES * MI_WAVE, 0, stream>>>(                              \
      (const bf16_t*)q, (const bf16_t*)k_pages, (bf16_t*)out, part_acc, part_ml, s)
#define MI_LATENT(KS, VT, EXACT)                        \
  do {                                                  \
    if (waves == 1) MI_LATENT_W(KS, VT, EXACT, 1);      \
    else if (waves == 2) MI_LATENT_W(KS, VT, EXACT, 2); \
    else MI_LATENT_W(KS, VT, EXACT, 4);                 \
  } while (0)
  const int ksteps = (width + 31) / 32;
  if (rank == 512 && width / 8 == 72) MI_LATENT(18, 32, true);
  else if (rank == 256 && width / 8 == 36) MI_LATENT(9, 16, true);
  else if (rank <= 128 && ksteps <= 6) MI_LATENT(6, 8, false);
  else if (rank <= 256 && ksteps <= 10) MI_LATENT(10, 16, false);
  else MI_LATENT(18, 32, false);
#undef MI_LATENT
#undef MI_LATENT_W
  MI_CHECK_LAUNCH("attn_latent");
  if (splits > 1) {
    MI_REQUIRE(heads <= 65535, "attn_latent: too many heads (%d)", heads);
    dim3 cgrid(num_tokens, heads);
    const int threads = 4 * (rank <= 256 ? 64 : 128);
#define MI_COMBINE(EACH) \
  latent_combine_kernel<EACH><<<cgrid, threads, 0, stream>>>(part_acc, part_ml, (bf16_t*)out, out_stride, heads, rank, splits, sinks)
    if (splits <= 4) MI_COMBINE(1);
    else if (splits <= 8) MI_COMBINE(2);
    else if (splits <= 16) MI_COMBINE(4);
    else if (splits <= 32) MI_COMBINE(8);
    else MI_COMBINE(16);
#undef MI_COMBINE
    MI_CHECK_LAUNCH("latent_combine");
  }
  return MI_OK;
}
