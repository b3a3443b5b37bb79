// What stands between a mixer's per-head results and its output product when each head is normed by itself:
//   o[t, h, :]   = a[t, h, :]                                            one result a head, or
//                = a[t, first(h), :] - lambda * a[t, second(h), :]      two maps of attention a head, combined
//   out[t, h, e] = o[e] / sqrt(mean(o^2) + eps) * weight[h * dv + e] * mult * f(gate[t, h * dv + e])
// f is the sigmoid (gate_kind 0) or z * sigmoid(z) (gate_kind 1); weight and gate are optional (null: 1).  With gate_first
// the gate joins before the norm: o[e] is a[e] * f(gate[e]) (one result a head only).  Everything is float; `a` holds floats, the gate is read from a
// product's columns (any type, possibly partial sums), out is in the activation type.
//
// Two maps: `a` then holds 2 * heads results a token in the order in which the attention kernel wants its
// query heads, those of one key head side by side: with r = heads / (key/value groups), head h = g * r + i has
// its first map at (2 g) * r + i and its second at (2 g + 1) * r + i.  A map's result may also come in `parts`
// pieces of dv / parts dims each (the attention kernel on the matrix cores takes value heads wider than the keys as
// several heads of the keys' size): piece p of the map of key head k = 2 g + m lies at ((k * parts + p) * r + i).
#include "common.h"

namespace tlie {

template <typename D, typename W, typename A>
__global__ void __launch_bounds__(256)
head_combine_kernel(const float* __restrict__ a, int heads, int dv, int pair_group, int parts, float lambda, float eps,
                    const W* __restrict__ weight, float mult, const D* __restrict__ gate, int gate_nsplit,
                    size_t gate_split_stride, int gate_row, int gate_col, int gate_kind, int gate_first, A* __restrict__ out) {
  const int t = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int h = blockIdx.y * 4 + wave;
  if (h >= heads) return;                              // (a whole wave; no barrier follows)
  // where dim e of the head's first (and second) result lies: with two maps, a map's result may come in `parts`
  // pieces of dv / parts dims, the pieces of one key head's query heads piece by piece
  const int piece = dv / parts;
  const int g = pair_group > 0 ? h / pair_group : 0, i = pair_group > 0 ? h - g * pair_group : 0;
  const float* row = a + static_cast<size_t>(t) * (pair_group > 0 ? 2 : 1) * heads * dv;
  auto gate_value = [&](int e) {
    const float z = sum_splits(gate + static_cast<size_t>(t) * gate_row + gate_col + h * dv + e, gate_nsplit, gate_split_stride);
    return (gate_kind == 1 ? z : 1.f) / (1.f + expf(-z));
  };
  auto value = [&](int e) {
    if (pair_group <= 0) {
      const float o = row[static_cast<size_t>(h) * dv + e];
      return gate_first ? o * gate_value(e) : o;
    }
    const int p = e / piece, inside = e - p * piece;
    const float first = row[((static_cast<size_t>(2 * g) * parts + p) * pair_group + i) * piece + inside];
    const float second = row[((static_cast<size_t>(2 * g + 1) * parts + p) * pair_group + i) * piece + inside];
    return first - lambda * second;
  };
  auto emit = [&](int e, float normed) {
    const int c = h * dv + e;
    float v = normed * mult;
    if (weight != nullptr) v *= to_float(weight[c]);
    if (gate != nullptr && !gate_first) v *= gate_value(e);
    out[static_cast<size_t>(t) * heads * dv + c] = from_float<A>(v);
  };
  // a lane's dims (lane, lane + 64, ...) are read once and kept, up to 512 dims a head; beyond, read again
  constexpr int kKept = 8;
  const bool fits = dv <= 64 * kKept;
  float kept[kKept];
  float squares = 0.f;
#pragma unroll
  for (int i = 0; i < kKept; ++i) {
    const int e = lane + 64 * i;
    kept[i] = fits && e < dv ? value(e) : 0.f;
    squares += kept[i] * kept[i];
  }
  if (!fits) {
    for (int e = lane; e < dv; e += 64) {
      const float o = value(e);
      squares += o * o;
    }
  }
  const float r = 1.f / sqrtf(wave_sum(squares) / static_cast<float>(dv) + eps);
#pragma unroll
  for (int i = 0; i < kKept; ++i) {
    const int e = lane + 64 * i;
    if (fits && e < dv) emit(e, kept[i] * r);
  }
  if (fits) return;
  for (int e = lane; e < dv; e += 64) emit(e, value(e) * r);
}

// The same for one result a head that is too wide for a wave (more than 512 dims: all heads of a mixer normed together
// are one head here): a workgroup a head, eight dims a thread and access, a thread's first kKept groups kept between the
// sum of squares and the output.  dv a multiple of 8, rows of `a`, weight, gate and out at multiples of 32 bytes, the
// gate's parts a multiple of 8 apart.
template <typename D, typename W, typename A>
__global__ void __launch_bounds__(256)
head_combine_wide_kernel(const float* __restrict__ a, int heads, int dv, float eps, const W* __restrict__ weight, float mult,
                         const D* __restrict__ gate, int gate_nsplit, size_t gate_split_stride, int gate_row, int gate_col,
                         int gate_kind, int gate_first, A* __restrict__ out) {
  __shared__ float scratch[16];
  constexpr int kKept = 2;
  const int t = blockIdx.x, h = blockIdx.y;
  const size_t base = (static_cast<size_t>(t) * heads + h) * dv;
  float kept[kKept][8];
  float squares = 0.f;
  auto gates = [&](int e, float (&v)[8]) {             // v *= f(gate) of dims e .. e + 7
    float z[8];
    const D* from = gate + static_cast<size_t>(t) * gate_row + gate_col + h * dv + e;
    load8(from, z);
    for (int s = 1; s < gate_nsplit; ++s) {
      float more[8];
      load8(from + s * gate_split_stride, more);
#pragma unroll
      for (int j = 0; j < 8; ++j) z[j] += more[j];
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] *= (gate_kind == 1 ? z[j] : 1.f) / (1.f + expf(-z[j]));
  };
  auto result = [&](int e, float (&v)[8]) {
    load8(a + base + e, v);
    if (gate_first) gates(e, v);
  };
#pragma unroll
  for (int i = 0; i < kKept; ++i) {
    const int e = (threadIdx.x + i * blockDim.x) * 8;
    if (e < dv) {
      result(e, kept[i]);
#pragma unroll
      for (int j = 0; j < 8; ++j) squares += kept[i][j] * kept[i][j];
    }
  }
  for (int e = (threadIdx.x + kKept * blockDim.x) * 8; e < dv; e += blockDim.x * 8) {
    float v[8];
    result(e, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) squares += v[j] * v[j];
  }
  const float r = mult / sqrtf(block_sum(squares, scratch) / static_cast<float>(dv) + eps);
  auto emit = [&](int e, float (&v)[8]) {
    const int c = h * dv + e;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] *= r;
    if (weight != nullptr) {
      float w[8];
      load8(weight + c, w);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] *= w[j];
    }
    if (gate != nullptr && !gate_first) gates(e, v);
    store8(out + base + e, v);
  };
#pragma unroll
  for (int i = 0; i < kKept; ++i) {
    const int e = (threadIdx.x + i * blockDim.x) * 8;
    if (e < dv) emit(e, kept[i]);
  }
  for (int e = (threadIdx.x + kKept * blockDim.x) * 8; e < dv; e += blockDim.x * 8) {
    float v[8];
    result(e, v);
    emit(e, v);
  }
}

}  // namespace tlie

using namespace tlie;

// a: float [tokens, (pair_group > 0 ? 2 : 1) * heads, dv]; weight (or null): [heads * dv] of weight_dtype; gate (or null):
// a product [nsplit][tokens][gate_row] of gate_dtype whose columns gate_col .. gate_col + heads * dv - 1 are read.
extern "C" int tlie_head_combine(const float* a, int tokens, int heads, int dv, int pair_group, int parts, float lambda, float eps,
                                 const void* weight, int weight_dtype, float mult, const void* gate, int gate_dtype,
                                 int gate_nsplit, long long gate_split_stride, int gate_row, int gate_col, int gate_kind,
                                 int gate_first, void* out, int out_dtype, void* stream) {
  if (tokens <= 0 || heads <= 0 || dv <= 0 || pair_group < 0 || (pair_group > 0 && heads % pair_group != 0)) return kBadArgument;
  if (parts < 1 || dv % parts != 0 || (parts > 1 && pair_group <= 0) || gate_kind < 0 || gate_kind > 1) return kBadArgument;
  if (gate != nullptr && (gate_nsplit < 1 || gate_col < 0 || gate_row < gate_col + heads * dv)) return kBadArgument;
  if (gate_first && (gate == nullptr || pair_group > 0)) return kBadArgument;
  if (heads > 4 * 65535) return kBadArgument;
  const dim3 grid(tokens, (heads + 3) / 4);
  hipStream_t s = (hipStream_t)stream;
  const bool wide = pair_group == 0 && dv > 512 && dv % 8 == 0 && heads <= 65535 && gate_row % 8 == 0 && gate_col % 8 == 0 &&
                    (gate_nsplit <= 1 || gate_split_stride % 8 == 0) &&
                    ((reinterpret_cast<uintptr_t>(a) | reinterpret_cast<uintptr_t>(weight) | reinterpret_cast<uintptr_t>(gate) |
                      reinterpret_cast<uintptr_t>(out)) & 31) == 0;
#define TLIE_CASE(GC, D, WC, W, AC, A)                                                                                   \
  if (gate_dtype == GC && weight_dtype == WC && out_dtype == AC) {                                                       \
    if (wide) {                                                                                                          \
      hipLaunchKernelGGL((head_combine_wide_kernel<D, W, A>), dim3(tokens, heads), dim3(256), 0, s, a, heads, dv, eps,    \
                         (const W*)weight, mult, (const D*)gate, gate_nsplit, (size_t)gate_split_stride, gate_row,       \
                         gate_col, gate_kind, gate_first, (A*)out);                                                                  \
      return launch_status();                                                                                            \
    }                                                                                                                    \
    hipLaunchKernelGGL((head_combine_kernel<D, W, A>), grid, dim3(256), 0, s, a, heads, dv, pair_group, parts, lambda, eps,     \
                       (const W*)weight, mult, (const D*)gate, gate_nsplit, (size_t)gate_split_stride, gate_row, gate_col, \
                       gate_kind, gate_first, (A*)out);                                                                                          \
    return launch_status();                                                                                              \
  }
  TLIE_CASE(kF32, float, kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kF32, float, kBF16, bf16)
  TLIE_CASE(kF32, float, kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kF32, float, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}
