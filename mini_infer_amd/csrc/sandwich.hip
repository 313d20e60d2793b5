// Row kernel of a stack whose sublayers stand between two norms.
//
//   gated_update_norm   y[t] = sum of the token's `pieces` rows of the sublayer's result
//                       v    = y * logistic(gate[t] + bias)        (no gate: v = y)
//                       x[t] += v / sqrt(mean(v^2) + eps_out) * out_weight       (float32 stream, in place)
//                       h[t] = x / sqrt(mean(x^2) + eps) * norm_weight           (element type)
//                       and, where every request brings exactly one token, the causal convolution
//                       on what the next sublayer reads: u[t] = h + sum_j w[c, j] * (h, taps-1-j tokens
//                       ago), the earlier h from the request's tail, which is moved on by one.
//                       One launch stands between two sublayers.
//
// Sums and statistics are float32 for bfloat16 rows and 64-bit for float32 rows (rounded once).
#include "common.h"

#include <math.h>

#define SANDWICH_MAX_TAPS 16

namespace {

template <typename T>
struct WideOf {
  using type = float;
};
template <>
struct WideOf<float> {
  using type = double;
};

__device__ __forceinline__ float lane_add(float v, int off) { return v + __shfl_xor(v, off, MI_WAVE); }
__device__ __forceinline__ double lane_add(double v, int off) { return v + __shfl_xor(v, off, MI_WAVE); }

// sum over a block in a fixed order: lanes by butterfly, waves one after another
template <typename A>
__device__ __forceinline__ A block_add(A v, A* scratch) {
#pragma unroll
  for (int off = MI_WAVE / 2; off > 0; off >>= 1) v = lane_add(v, off);
  const int wave = threadIdx.x / MI_WAVE, lane = threadIdx.x % MI_WAVE;
  const int n_waves = (blockDim.x + MI_WAVE - 1) / MI_WAVE;
  __syncthreads();
  if (lane == 0) scratch[wave] = v;
  __syncthreads();
  A total = 0;
  for (int w = 0; w < n_waves; ++w) total += scratch[w];
  return total;
}

__device__ __forceinline__ float inv_root_of(float mean_sq, float eps) { return 1.0f / sqrtf(mean_sq + eps); }
__device__ __forceinline__ double inv_root_of(double mean_sq, double eps) { return 1.0 / sqrt(mean_sq + eps); }

__device__ __forceinline__ float gate_of(float z) { return mi_logistic(z); }
__device__ __forceinline__ double gate_of(double z) { return 1.0 / (1.0 + exp(-z)); }

inline bool is_aligned16(const void* p) { return ((uintptr_t)p % 16) == 0; }

// Columns of a row a thread keeps in registers between the passes (`KEPT` turns of VEC); what lies
// beyond is made again from the inputs.
constexpr int KEPT = 4;

template <typename T, int VEC>
__global__ __launch_bounds__(1024) void gated_update_norm_kernel(
    float* __restrict__ stream, const T* __restrict__ y, int64_t y_stride, int pieces, const T* __restrict__ gate,
    int64_t gate_stride, const float* __restrict__ bias, const T* __restrict__ out_weight,
    const T* __restrict__ norm_weight, const int* __restrict__ rows, T* __restrict__ h, int hidden, float eps_out,
    float eps, const float* __restrict__ conv_weight, int taps, T* __restrict__ tail, int64_t tail_stride,
    const int* __restrict__ slots, int num_slots, T* __restrict__ u) {
  using A = typename WideOf<T>::type;
  __shared__ A scratch[16];
  const int t = rows != nullptr ? rows[blockIdx.x] : blockIdx.x;
  float* x = stream + (int64_t)t * hidden;
  const T* first = y != nullptr ? y + (int64_t)t * pieces * y_stride : nullptr;
  const T* g = gate != nullptr ? gate + (int64_t)t * gate_stride : nullptr;

  auto gated = [&](int c, A (&v)[VEC]) {  // the sublayer's gated result
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] = 0;
    for (int p = 0; p < pieces; ++p) {
      float got[VEC];
      mi_load_cols<T, VEC>(first + (int64_t)p * y_stride + c, got);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += (A)got[j];
    }
    if (g != nullptr) {
      float z[VEC], b[VEC];
      mi_load_cols<T, VEC>(g + c, z);
      mi_load_cols<float, VEC>(bias + c, b);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] *= gate_of((A)z[j] + (A)b[j]);
    }
  };

  A kept[KEPT][VEC];
  A inv_out = 0;
  if (first != nullptr) {
    A squares = 0;
    int turn = 0;
    for (int c = threadIdx.x * VEC; c < hidden; c += blockDim.x * VEC, ++turn) {
      A v[VEC];
      gated(c, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        squares += v[j] * v[j];
        if (turn < KEPT) kept[turn][j] = v[j];
      }
    }
    inv_out = inv_root_of(block_add<A>(squares, scratch) / (A)hidden, (A)eps_out);
  }

  auto fresh = [&](int c, int turn, float (&now)[VEC]) {  // the stream's new values
    mi_load_cols<float, VEC>(x + c, now);
    if (first == nullptr) return;
    A v[VEC];
    if (turn < KEPT) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = kept[turn][j];
    } else {
      gated(c, v);
    }
    float w[VEC];
    mi_load_cols<T, VEC>(out_weight + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) now[j] = (float)((A)now[j] + (v[j] * inv_out) * (A)w[j]);
  };

  A squares = 0;
  int turn = 0;
  for (int c = threadIdx.x * VEC; c < hidden; c += blockDim.x * VEC, ++turn) {
    float now[VEC];
    fresh(c, turn, now);
    if (rows == nullptr && first != nullptr) mi_store_cols<float, VEC>(x + c, now);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      squares += (A)now[j] * (A)now[j];
      if (turn < KEPT) kept[turn][j] = (A)now[j];
    }
  }
  if (norm_weight == nullptr) return;
  const A inv = inv_root_of(block_add<A>(squares, scratch) / (A)hidden, (A)eps);

  T* mine = nullptr;
  if (u != nullptr && taps > 1) {
    const int slot = slots[t];  // (row t is request t's only token)
    mine = tail + (int64_t)((slot < 0 || slot >= num_slots) ? num_slots : slot) * tail_stride;
  }
  T* out = h + (int64_t)blockIdx.x * hidden;
  turn = 0;
  for (int c = threadIdx.x * VEC; c < hidden; c += blockDim.x * VEC, ++turn) {
    float now[VEC], w[VEC], r[VEC];
    if (turn < KEPT) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) now[j] = (float)kept[turn][j];
    } else if (rows == nullptr) {
      mi_load_cols<float, VEC>(x + c, now);  // (written above by this same thread)
    } else {
      fresh(c, turn, now);
    }
    mi_load_cols<T, VEC>(norm_weight + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) r[j] = to_f32(from_f32<T>((float)(((A)now[j] * inv) * (A)w[j])));
    mi_store_cols<T, VEC>(out + c, r);
    if (u == nullptr) continue;
    // the convolution on the rounded row, oldest input first (the order of the convolution's own kernels)
    const int back = taps - 1;
    A sum[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) sum[j] = 0;
    for (int k = 0; k < back; ++k) {
      float before[VEC], next[VEC];
      mi_load_cols<T, VEC>(mine + (int64_t)k * hidden + c, before);
      if (k + 1 < back) {
        mi_load_cols<T, VEC>(mine + (int64_t)(k + 1) * hidden + c, next);
      } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) next[j] = r[j];
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) sum[j] = fma((A)conv_weight[(int64_t)k * hidden + c + j], (A)before[j], sum[j]);
      mi_store_cols<T, VEC>(mine + (int64_t)k * hidden + c, next);
    }
    float made[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      sum[j] = fma((A)conv_weight[(int64_t)back * hidden + c + j], (A)r[j], sum[j]);
      made[j] = (float)((A)r[j] + sum[j]);
    }
    mi_store_cols<T, VEC>(u + (int64_t)t * hidden + c, made);
  }
}

// The same where a thread has one turn of four columns, at most four pieces and at most four taps (few rows, the
// usual widths): everything the row needs is asked for at once, so the launch waits for memory once and
// not before each of its three passes (8 rows of 4,096: 15 us one after the other).
template <typename T>
__global__ __launch_bounds__(1024) void gated_update_norm_early_kernel(
    float* __restrict__ stream, const T* __restrict__ y, int64_t y_stride, int pieces, const T* __restrict__ gate,
    int64_t gate_stride, const float* __restrict__ bias, const T* __restrict__ out_weight,
    const T* __restrict__ norm_weight, const int* __restrict__ rows, T* __restrict__ h, int hidden, float eps_out,
    float eps, const float* __restrict__ conv_weight, int taps, T* __restrict__ tail, int64_t tail_stride,
    const int* __restrict__ slots, int num_slots, T* __restrict__ u) {
  using A = typename WideOf<T>::type;
  constexpr int MOST = 4;
  __shared__ A scratch_out[16], scratch[16];
  const int t = rows != nullptr ? rows[blockIdx.x] : blockIdx.x;
  const int c = threadIdx.x * 4;
  const bool mine_too = c < hidden;
  const int at = mine_too ? c : 0;  // (threads past the row read its first columns, and count and write nothing)
  float* x = stream + (int64_t)t * hidden;
  const int back = taps - 1;
  float part[MOST][4], z[4], b[4], wo[4], now[4], w[4], before[MOST - 1][4], wc[MOST][4];
  mi_load_cols<float, 4>(x + at, now);
  mi_load_cols<T, 4>(norm_weight + at, w);
  if (y != nullptr) {
#pragma unroll
    for (int p = 0; p < MOST; ++p)
      if (p < pieces) mi_load_cols<T, 4>(y + ((int64_t)t * pieces + p) * y_stride + at, part[p]);
    if (gate != nullptr) {
      mi_load_cols<T, 4>(gate + (int64_t)t * gate_stride + at, z);
      mi_load_cols<float, 4>(bias + at, b);
    }
    mi_load_cols<T, 4>(out_weight + at, wo);
  }
  T* kept = nullptr;
  if (u != nullptr) {
    if (taps > 1) {
      const int slot = slots[t];  // (row t is request t's only token)
      kept = tail + (int64_t)((slot < 0 || slot >= num_slots) ? num_slots : slot) * tail_stride;
    }
#pragma unroll
    for (int k = 0; k < MOST - 1; ++k)
      if (k < back) mi_load_cols<T, 4>(kept + (int64_t)k * hidden + at, before[k]);
#pragma unroll
    for (int k = 0; k < MOST; ++k)
      if (k < taps) mi_load_cols<float, 4>(conv_weight + (int64_t)k * hidden + at, wc[k]);
  }

  if (y != nullptr) {
    A v[4], squares = 0;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[j] = 0;
#pragma unroll
      for (int p = 0; p < MOST; ++p)
        if (p < pieces) v[j] += (A)part[p][j];
      if (gate != nullptr) v[j] *= gate_of((A)z[j] + (A)b[j]);
      squares += v[j] * v[j];
    }
    const A inv_out = inv_root_of(block_add<A>(mine_too ? squares : (A)0, scratch_out) / (A)hidden, (A)eps_out);
#pragma unroll
    for (int j = 0; j < 4; ++j) now[j] = (float)((A)now[j] + (v[j] * inv_out) * (A)wo[j]);
    if (rows == nullptr && mine_too) mi_store_cols<float, 4>(x + c, now);
  }
  A squares = 0;
#pragma unroll
  for (int j = 0; j < 4; ++j) squares += (A)now[j] * (A)now[j];
  const A inv = inv_root_of(block_add<A>(mine_too ? squares : (A)0, scratch) / (A)hidden, (A)eps);
  if (!mine_too) return;
  float r[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) r[j] = to_f32(from_f32<T>((float)(((A)now[j] * inv) * (A)w[j])));
  mi_store_cols<T, 4>(h + (int64_t)blockIdx.x * hidden + c, r);
  if (u == nullptr) return;
  A sum[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    sum[j] = 0;
#pragma unroll
    for (int k = 0; k < MOST - 1; ++k)
      if (k < back) sum[j] = fma((A)wc[k][j], (A)before[k][j], sum[j]);
    A last = 0;
#pragma unroll
    for (int k = 0; k < MOST; ++k)
      if (k == back) last = (A)wc[k][j];
    sum[j] = fma(last, (A)r[j], sum[j]);
  }
#pragma unroll
  for (int k = 0; k < MOST - 1; ++k) {
    if (k + 1 < back) mi_store_cols<T, 4>(kept + (int64_t)k * hidden + c, before[k + 1 < MOST - 1 ? k + 1 : k]);
    else if (k + 1 == back) mi_store_cols<T, 4>(kept + (int64_t)k * hidden + c, r);
  }
  float made[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) made[j] = (float)((A)r[j] + sum[j]);
  mi_store_cols<T, 4>(u + (int64_t)t * hidden + c, made);
}

}  // namespace

// y: [tokens * pieces, hidden] (row stride) or null (the norm alone); gate [tokens, hidden] (row stride) with
// bias float32 [hidden], or null; out_weight [hidden]; norm_weight [hidden] or null (the update alone); rows
// (may be null) lists the rows to norm: the stream is then left as it is and h gets the rows in list order.
// With u [tokens, hidden]: conv_weight float32 [taps, hidden] (a tap's weights side by side), tail [slots + 1, (taps - 1) * hidden] (row
// stride), every token the only one of its request: row t is request t's (slots).
extern "C" int mi_gated_update_norm(int dtype, float* stream_rows, const void* y, int64_t y_stride, int pieces,
                                    const void* gate, int64_t gate_stride, const float* bias, const void* out_weight,
                                    const void* norm_weight, const int* rows, void* h, int num_rows, int hidden,
                                    float eps_out, float eps, const float* conv_weight, int taps, void* tail,
                                    int64_t tail_stride, const int* slots, int num_slots,
                                    void* u, hipStream_t stream) {
  MI_REQUIRE(num_rows >= 0 && hidden > 0 && pieces >= 1 && (y == nullptr || y_stride >= hidden) &&
                 (gate == nullptr || gate_stride >= hidden),
             "gated_update_norm: bad sizes rows=%d hidden=%d pieces=%d", num_rows, hidden, pieces);
  MI_REQUIRE(stream_rows != nullptr && (y == nullptr || out_weight != nullptr) && (gate == nullptr || (bias != nullptr && y != nullptr)),
             "gated_update_norm: an update comes with its norm's weight, a gate with its bias");
  MI_REQUIRE(norm_weight == nullptr || h != nullptr, "gated_update_norm: the normed rows need a place to go");
  MI_REQUIRE(rows == nullptr || norm_weight != nullptr, "gated_update_norm: a row list only goes with a norm");
  MI_REQUIRE(u == nullptr || (rows == nullptr && norm_weight != nullptr && conv_weight != nullptr && taps >= 1 && taps <= SANDWICH_MAX_TAPS),
             "gated_update_norm: the convolution goes with the norm of all rows and 1..%d taps, got %d", SANDWICH_MAX_TAPS, taps);
  MI_REQUIRE(u == nullptr || taps == 1 ||
                 (tail != nullptr && tail_stride >= (int64_t)(taps - 1) * hidden && slots != nullptr && num_slots >= 1),
             "gated_update_norm: the convolution needs its requests' tails");
  MI_REQUIRE(eps > 0.f && eps_out > 0.f, "gated_update_norm: eps must be positive");
  MI_REQUIRE(dtype == MI_F32 || dtype == MI_BF16, "gated_update_norm: unknown dtype %d", dtype);
  if (num_rows == 0) return MI_OK;
  const bool vec = hidden % 4 == 0 && y_stride % 4 == 0 && gate_stride % 4 == 0 && tail_stride % 4 == 0 &&
                   is_aligned16(stream_rows) && is_aligned16(y) && is_aligned16(gate) && is_aligned16(bias) && is_aligned16(out_weight) &&
                   is_aligned16(norm_weight) && is_aligned16(h) && is_aligned16(tail) && is_aligned16(u) && is_aligned16(conv_weight);
  const int items = vec ? ceil_div(hidden, 4) : hidden;
  // few rows: a turn of the whole row at once; many rows: four waves a row, several rows to a CU
  const int threads = num_rows < 256 ? min(1024, ceil_div(items, MI_WAVE) * MI_WAVE) : 256;
  if (vec && items <= threads && pieces <= 4 && norm_weight != nullptr && (u == nullptr || taps <= 4)) {
#define MI_SANDWICH_EARLY(T)                                                                                              \
  gated_update_norm_early_kernel<T><<<num_rows, threads, 0, stream>>>(                                                    \
      stream_rows, (const T*)y, y_stride, pieces, (const T*)gate, gate_stride, bias, (const T*)out_weight,                \
      (const T*)norm_weight, rows, (T*)h, hidden, eps_out, eps, conv_weight, taps, (T*)tail, tail_stride, slots, \
      num_slots, (T*)u)
    if (dtype == MI_F32) MI_SANDWICH_EARLY(float);
    else MI_SANDWICH_EARLY(bf16_t);
#undef MI_SANDWICH_EARLY
    MI_CHECK_LAUNCH("gated_update_norm_early");
    return MI_OK;
  }
#define MI_SANDWICH(T, VEC)                                                                                             \
  gated_update_norm_kernel<T, VEC><<<num_rows, threads, 0, stream>>>(                                                   \
      stream_rows, (const T*)y, y_stride, pieces, (const T*)gate, gate_stride, bias, (const T*)out_weight,              \
      (const T*)norm_weight, rows, (T*)h, hidden, eps_out, eps, conv_weight, taps, (T*)tail, tail_stride, slots, \
      num_slots, (T*)u)
  if (dtype == MI_F32) {
    if (vec) MI_SANDWICH(float, 4);
    else MI_SANDWICH(float, 1);
  } else {
    if (vec) MI_SANDWICH(bf16_t, 4);
    else MI_SANDWICH(bf16_t, 1);
  }
#undef MI_SANDWICH
  MI_CHECK_LAUNCH("gated_update_norm");
  return MI_OK;
}
