// Routed experts for many rows (prompts): the two products of every chosen expert as one launch each over
// tiles of BM of the expert's (token, choice) pairs x BN of its output features on the matrix cores, with
// nothing the host has to know: the pairs are listed expert by expert on the device (`expert_sort`),
// and a block finds its tile in that list.
//
// Both operands pass through LDS, 64 elements of K at a time, two buffers: while one is worked on, the next
// is on its way straight from memory into LDS (no registers between).  A row of a buffer is 128 bytes, eight
// chunks of 16; chunk c of row r lies at place c ^ (r % 8), so that the eight lanes that are served together
// find their 16-byte pieces in different banks.  The waves stand 2 x 2 over the tile; MFMA 16x16x32 with
// weight rows as the first operand and pairs as the second, so a lane ends with four consecutive features of
// a pair.
//
// Tiles are numbered expert by expert, within an expert feature tile by feature tile with the row tiles of one
// feature tile side by side; each of the 8 XCDs takes one stretch of these numbers (workgroups are dealt
// to the XCDs in turn), so the row tiles that read the same weights run at the same time behind one
// L2, and an expert's rows stay in it.
//
// MODE as in routed_experts.hip: 0 plain, 1 silu(gate) * up (a block then makes BN / 2 features: gate and up rows
// side by side in its tile), 2 relu(weight * z)^2.
#include "common.h"

namespace {

typedef float f32x4_e __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) void lds_void;
typedef const __attribute__((address_space(1))) void global_void;

#define TILE_K 64

// Which tile this block works on: expert, first pair of the row tile (an index into `listed`), feature tile.
// False: past the last tile.  All threads of the block get the same answer.
__device__ __forceinline__ bool find_tile(const int* __restrict__ first, int experts, int feature_tiles, int bm, int id,
                                          int& expert, int& row0, int& feature_tile) {
  const int lane = threadIdx.x % MI_WAVE;
  // row tiles in all
  int total = 0;
  for (int base = 0; base < experts; base += MI_WAVE) {
    const int e = base + lane;
    int tiles = e < experts ? (first[e + 1] - first[e] + bm - 1) / bm : 0;
#pragma unroll
    for (int off = MI_WAVE / 2; off > 0; off >>= 1) tiles += __shfl_xor(tiles, off, MI_WAVE);
    total += tiles;
  }
  total *= feature_tiles;
  const int per = (total + 7) / 8;
  const int place = (id % 8) * per + id / 8;
  if (id / 8 >= per || place >= total) return false;
  int before = 0;
  for (int base = 0; base < experts; base += MI_WAVE) {
    const int e = base + lane;
    const int tiles = e < experts ? (first[e + 1] - first[e] + bm - 1) / bm : 0;
    int upto = tiles;  // row tiles of the experts up to and including this lane's
#pragma unroll
    for (int off = 1; off < MI_WAVE; off <<= 1) {
      const int other = __shfl_up(upto, off, MI_WAVE);
      if (lane >= off) upto += other;
    }
    const uint64_t past = __ballot((before + upto) * feature_tiles > place);
    if (past != 0) {
      const int at = __builtin_ctzll(past);
      const int mine = __shfl(tiles, at, MI_WAVE), start = before + __shfl(upto, at, MI_WAVE) - mine;
      const int rest = place - start * feature_tiles;
      expert = base + at;
      row0 = first[expert] + (rest % mine) * bm;
      feature_tile = rest / mine;
      return true;
    }
    before += __shfl(upto, MI_WAVE - 1, MI_WAVE);
  }
  return false;
}

// (two blocks to a CU: without the bound the compiler spreads over more registers than two leave each)
template <int MODE, int BM, int BN>
__global__ __launch_bounds__(256, 2) void expert_tiles_lds_kernel(
    const bf16_t* __restrict__ src, int64_t src_stride, int src_div, const bf16_t* __restrict__ weight,
    int64_t expert_stride, const int* __restrict__ listed, const int* __restrict__ first,
    const float* __restrict__ pair_weight, bf16_t* __restrict__ out, int64_t out_stride, int experts, int k_dim,
    int features, int feature_tiles) {
  constexpr bool GATED = MODE == 1;
  constexpr int WM = BM / 2, WN = BN / 2;     // a wave's share of the tile: pairs, weight rows
  constexpr int MT = WM / 16, NT = WN / 16;   // in tiles of 16
  constexpr int ROW = TILE_K;                 // elements of a row in LDS
  constexpr int A_LOADS = BM / 32, B_LOADS = BN / 32;  // 8-row loads a wave makes for each operand
  // (an array of its own for each buffer: the compiler then sees that what is fetched into one does not touch
  // what is read from the other, and waits for nothing between)
  __shared__ __align__(16) bf16_t pairs_even[BM * ROW], pairs_odd[BM * ROW];
  __shared__ __align__(16) bf16_t rows_even[BN * ROW], rows_odd[BN * ROW];

  int expert, row0, feature_tile;
  if (!find_tile(first, experts, feature_tiles, BM, blockIdx.x, expert, row0, feature_tile)) return;
  const int end = first[expert + 1];
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE;
  const int col = lane % 16, quad = lane / 16;
  // a block's features: BN of them, or where they come in pairs BN / 2 (the tile's lower half of weight rows
  // their gate rows, its upper half their up rows)
  constexpr int FEATURES = GATED ? BN / 2 : BN;
  const int f0 = feature_tile * FEATURES;

  // what this lane fetches: 16 bytes of row 8 * load + lane / 8, chunk (lane % 8) ^ (lane / 8), of every load
  const int chunk = (lane % 8) ^ (lane / 8);
  const bf16_t* a_src[A_LOADS];
  const bf16_t* b_src[B_LOADS];
#pragma unroll
  for (int i = 0; i < A_LOADS; ++i) {
    const int r = (wave * A_LOADS + i) * 8 + lane / 8;
    const int pair = listed[min(row0 + r, end - 1)];  // (past the expert's last pair: that one again, not written)
    a_src[i] = src + (int64_t)(pair / src_div) * src_stride + chunk * 8;
  }
  const bf16_t* w = weight + (int64_t)expert * expert_stride;
#pragma unroll
  for (int i = 0; i < B_LOADS; ++i) {
    const int r = (wave * B_LOADS + i) * 8 + lane / 8;
    int row;
    if constexpr (GATED) row = min(f0 + (r % FEATURES), features - 1) + (r / FEATURES) * features;
    else row = min(f0 + r, features - 1);
    b_src[i] = w + (int64_t)row * k_dim + chunk * 8;
  }
  auto fetch = [&](bf16_t* pairs_lds, bf16_t* rows_lds, int k) {
#pragma unroll
    for (int i = 0; i < A_LOADS; ++i)
      __builtin_amdgcn_global_load_lds((global_void*)(a_src[i] + k),
                                       (lds_void*)(&pairs_lds[(wave * A_LOADS + i) * 8 * ROW]), 16, 0, 0);
#pragma unroll
    for (int i = 0; i < B_LOADS; ++i)
      __builtin_amdgcn_global_load_lds((global_void*)(b_src[i] + k),
                                       (lds_void*)(&rows_lds[(wave * B_LOADS + i) * 8 * ROW]), 16, 0, 0);
  };

  const int m_half = wave / 2, n_half = wave % 2;
  f32x4_e acc[NT][MT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[n][m] = f32x4_e{0.f, 0.f, 0.f, 0.f};

  // weight-row tile n of this wave: gated, its first half are gate rows and its second the up rows of the same features
  auto row_tile = [&](int n) {
    if constexpr (GATED) return (n < NT / 2 ? n_half * (NT / 2) + n : NT + n_half * (NT / 2) + (n - NT / 2)) * 16;
    else return (n_half * NT + n) * 16;
  };

  auto work = [&](const bf16_t* pairs_lds, const bf16_t* rows_lds) {
#pragma unroll
    for (int s = 0; s < TILE_K / 32; ++s) {
      bf16x8_t a[NT], b[MT];
      const int place = ((s * 4 + quad) ^ (col % 8)) * 8;
#pragma unroll
      for (int n = 0; n < NT; ++n) a[n] = *reinterpret_cast<const bf16x8_t*>(&rows_lds[(row_tile(n) + col) * ROW + place]);
#pragma unroll
      for (int m = 0; m < MT; ++m)
        b[m] = *reinterpret_cast<const bf16x8_t*>(&pairs_lds[(m_half * WM + m * 16 + col) * ROW + place]);
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[n][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[n], b[m], acc[n][m], 0, 0, 0);
    }
  };
  auto whole = [&]() {  // what was asked for last is there, for all waves, and nobody reads the other buffer any more
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
  };

  fetch(pairs_even, rows_even, 0);
  const int steps = k_dim / TILE_K;
  for (int step = 0; step < steps; step += 2) {
    whole();
    if (step + 1 < steps) fetch(pairs_odd, rows_odd, (step + 1) * TILE_K);
    work(pairs_even, rows_even);
    if (step + 1 >= steps) break;
    whole();
    if (step + 2 < steps) fetch(pairs_even, rows_even, (step + 2) * TILE_K);
    work(pairs_odd, rows_odd);
  }

#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int r = row0 + m_half * WM + m * 16 + col;
    if (r >= end) continue;
    const int pair = listed[r];
    bf16_t* o = out + (int64_t)pair * out_stride;
    const float pw = MODE == 2 && pair_weight != nullptr ? pair_weight[pair] : 1.f;
#pragma unroll
    for (int n = 0; n < (GATED ? NT / 2 : NT); ++n) {
      const int f = f0 + (GATED ? (n_half * (NT / 2) + n) * 16 : (n_half * NT + n) * 16) + 4 * quad;
      float v[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if constexpr (GATED) {
          // the two products as the element type holds them, then silu(gate) * up
          const float g = to_f32(from_f32<bf16_t>(acc[n][m][j])), u = to_f32(from_f32<bf16_t>(acc[n + NT / 2][m][j]));
          v[j] = g / (1.f + expf(-g)) * u;
        } else if constexpr (MODE == 2) {
          const float z = fmaxf(pw * acc[n][m][j], 0.f);
          v[j] = z * z;
        } else {
          v[j] = acc[n][m][j];
        }
      }
      if (f + 4 <= features && out_stride % 4 == 0) {
        mi_store_cols<bf16_t, 4>(o + f, v);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (f + j < features) o[f + j] = from_f32<bf16_t>(v[j]);
      }
    }
  }
}

template <int MODE, int BM, int BN>
void launch_tiles(const void* src, int64_t src_stride, int src_div, const void* weight, const int* listed, const int* first,
                  const float* pair_weight, void* out, int64_t out_stride, int pairs, int experts, int k_dim, int features,
                  hipStream_t stream) {
  const int feature_tiles = ceil_div(features, MODE == 1 ? BN / 2 : BN);
  const int most = feature_tiles * (pairs / BM + min(experts, pairs));  // (an expert's last tile may be a short one)
  expert_tiles_lds_kernel<MODE, BM, BN><<<ceil_div(most, 8) * 8, 256, 0, stream>>>(
      (const bf16_t*)src, src_stride, src_div, (const bf16_t*)weight, (int64_t)(MODE == 1 ? 2 : 1) * features * k_dim, listed,
      first, pair_weight, (bf16_t*)out, out_stride, experts, k_dim, features, feature_tiles);
}

}  // namespace

// Whether rows of k_dim bfloat16 elements are taken.
extern "C" int mi_expert_tiles_take(int k_dim) { return k_dim > 0 && k_dim % TILE_K == 0; }

// Arguments as mi_expert_rows (bfloat16 only), with the number of listed pairs.
extern "C" int mi_expert_tiles(int mode, const void* src, int64_t src_stride, int src_div, const void* weight,
                               const int* listed, const int* first, const float* pair_weight, void* out,
                               int64_t out_stride, int pairs, int experts, int k_dim, int features, hipStream_t stream) {
  MI_REQUIRE(pairs >= 0 && experts > 0 && features > 0 && src_div > 0 && src_stride >= k_dim && out_stride >= features,
             "expert_tiles: bad sizes pairs=%d experts=%d k=%d features=%d", pairs, experts, k_dim, features);
  MI_REQUIRE(mi_expert_tiles_take(k_dim) && src_stride % 8 == 0 && ((uintptr_t)src | (uintptr_t)weight) % 16 == 0 && (uintptr_t)out % 8 == 0,
             "expert_tiles: rows of %d elements are not taken %d at a time", k_dim, TILE_K);
  MI_REQUIRE(mode >= 0 && mode <= 2, "expert_tiles: mode %d", mode);
  MI_REQUIRE((int64_t)ceil_div(features, 64) * ((int64_t)pairs / 128 + experts) < (1 << 30), "expert_tiles: too many tiles");
  if (pairs == 0) return MI_OK;
#define MI_TILES(MODE) \
  launch_tiles<MODE, 128, 128>(src, src_stride, src_div, weight, listed, first, pair_weight, out, out_stride, pairs, experts, k_dim, features, stream)
  if (mode == 1) MI_TILES(1);
  else if (mode == 2) MI_TILES(2);
  else MI_TILES(0);
#undef MI_TILES
  MI_CHECK_LAUNCH("expert_tiles");
  return MI_OK;
}
