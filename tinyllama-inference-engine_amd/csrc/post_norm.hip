// What joins a residual that nothing norms on its way into a sublayer: a sublayer's result is normed, and only then added.
//
//   y = s1 * delta1 + s2 * delta2 (the second optional), or, for a mixer of two sides whose results are normed each by
//       itself:  y = mult * (delta1 / rms(delta1) * side1 + delta2 / rms(delta2) * side2)
//   z = (y - mean) / sqrt(var + eps) * w (+ b), or, not centred, y / sqrt(mean(y^2) + eps) * w (+ b)
//   residual += z
//   out = the new residual in another type (what the next sublayer's products read), or its norm (the model's last)
//
// Sums, means, variances and the residual are float.  One workgroup a row.
#include "common.h"

namespace tlie {

struct PostNormArgs {
  float* residual;
  const void* d1;
  const void* d2;
  int n1, n2;
  size_t stride1, stride2;
  float s1, s2;
  const void* side1;         // weights of the two sides' own norms, or null: the plain sum
  const void* side2;
  float side_eps, mult;
  const void* weight;        // of the norm; null: nothing joins the residual (out is made of it as it is)
  const void* bias;
  float eps;
  int centred;
  const void* last_weight;   // the norm of the new residual, or null: out is the residual itself
  const void* last_bias;
  float last_eps;
  int last_centred;
  void* out;                 // or null
  const int* rows;           // or null: all rows; else those rows alone, and the residual is left as it was
  int hidden;
};

// V elements a thread at a time (8: rows at multiples of 32 bytes, hidden % 8 == 0).
template <typename T, int V>
__device__ __forceinline__ void read_row(const T* p, float (&v)[V]) {
  if constexpr (V == 8) load8(p, v);
  else v[0] = to_float(p[0]);
}
template <typename T, int V>
__device__ __forceinline__ void write_row(T* p, const float (&v)[V]) {
  if constexpr (V == 8) store8(p, v);
  else p[0] = from_float<T>(v[0]);
}
template <typename D, int V>
__device__ __forceinline__ void read_sum(const D* p, int nsplit, size_t stride, float (&v)[V]) {
  read_row<D, V>(p, v);
  for (int s = 1; s < nsplit; ++s) {
    float more[V];
    read_row<D, V>(p + s * stride, more);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] += more[j];
  }
}

// The row in `values` (a thread reads back only what it wrote itself) -> (value - mean) * r.
template <int V>
__device__ __forceinline__ void row_norm(const float* values, int hidden, int centred, float eps, float sum, float* scratch,
                                         float& mean, float& r) {
  // sum: this thread's share of the row's sum, or (not centred) of its squares
  mean = block_sum(sum, scratch) / static_cast<float>(hidden);
  float mean_square = mean;
  if (centred) {
    float squares = 0.f;
    for (int c = threadIdx.x * V; c < hidden; c += 256 * V) {
#pragma unroll
      for (int j = 0; j < V; ++j) squares += (values[c + j] - mean) * (values[c + j] - mean);
    }
    mean_square = block_sum(squares, scratch) / static_cast<float>(hidden);
  } else {
    mean = 0.f;
  }
  r = 1.f / sqrtf(mean_square + eps);
}

template <typename D1, typename D2, typename W, typename O, int V>
__global__ void __launch_bounds__(256)
post_norm_kernel(const PostNormArgs a) {
  extern __shared__ __attribute__((aligned(16))) float values[];       // [hidden], and with two sides again [hidden]
  __shared__ float scratch[16];
  const int hidden = a.hidden, t = a.rows != nullptr ? a.rows[blockIdx.x] : blockIdx.x;
  const size_t at = static_cast<size_t>(t) * hidden;
  const D1* d1 = static_cast<const D1*>(a.d1);
  const D2* d2 = static_cast<const D2*>(a.d2);
  const W* weight = static_cast<const W*>(a.weight);
  float mean = 0.f, r = 0.f, sum = 0.f;
  if (weight != nullptr) {
    if (a.side1 != nullptr) {
      float q1 = 0.f, q2 = 0.f;
      float* other = values + hidden;
      for (int c = threadIdx.x * V; c < hidden; c += 256 * V) {
        float x[V], y[V];
        read_sum<D1, V>(d1 + at + c, a.n1, a.stride1, x);
        read_sum<D2, V>(d2 + at + c, a.n2, a.stride2, y);
#pragma unroll
        for (int j = 0; j < V; ++j) q1 += x[j] * x[j], q2 += y[j] * y[j], values[c + j] = x[j], other[c + j] = y[j];
      }
      const float r1 = a.mult / sqrtf(block_sum(q1, scratch) / static_cast<float>(hidden) + a.side_eps);
      const float r2 = a.mult / sqrtf(block_sum(q2, scratch) / static_cast<float>(hidden) + a.side_eps);
      for (int c = threadIdx.x * V; c < hidden; c += 256 * V) {
        float w1[V], w2[V];
        read_row<W, V>(static_cast<const W*>(a.side1) + c, w1);
        read_row<W, V>(static_cast<const W*>(a.side2) + c, w2);
#pragma unroll
        for (int j = 0; j < V; ++j) {
          const float y = values[c + j] * r1 * w1[j] + other[c + j] * r2 * w2[j];
          values[c + j] = y;
          sum += a.centred ? y : y * y;
        }
      }
    } else {
      for (int c = threadIdx.x * V; c < hidden; c += 256 * V) {
        float x[V];
        read_sum<D1, V>(d1 + at + c, a.n1, a.stride1, x);
#pragma unroll
        for (int j = 0; j < V; ++j) x[j] *= a.s1;
        if (d2 != nullptr) {
          float y[V];
          read_sum<D2, V>(d2 + at + c, a.n2, a.stride2, y);
#pragma unroll
          for (int j = 0; j < V; ++j) x[j] += a.s2 * y[j];
        }
#pragma unroll
        for (int j = 0; j < V; ++j) {
          values[c + j] = x[j];
          sum += a.centred ? x[j] : x[j] * x[j];
        }
      }
    }
    row_norm<V>(values, hidden, a.centred, a.eps, sum, scratch, mean, r);
  }
  sum = 0.f;
  O* out = a.out != nullptr ? static_cast<O*>(a.out) + static_cast<size_t>(blockIdx.x) * hidden : nullptr;
  for (int c = threadIdx.x * V; c < hidden; c += 256 * V) {
    float x[V];
    read_row<float, V>(a.residual + at + c, x);
    if (weight != nullptr) {
      float w[V];
      read_row<W, V>(weight + c, w);
#pragma unroll
      for (int j = 0; j < V; ++j) w[j] *= (values[c + j] - mean) * r;
      if (a.bias != nullptr) {
        float b[V];
        read_row<W, V>(static_cast<const W*>(a.bias) + c, b);
#pragma unroll
        for (int j = 0; j < V; ++j) w[j] += b[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] += w[j];
      if (a.rows == nullptr) write_row<float, V>(a.residual + at + c, x);
    }
    if (out == nullptr) continue;
    if (a.last_weight == nullptr) {
      write_row<O, V>(out + c, x);
      continue;
    }
#pragma unroll
    for (int j = 0; j < V; ++j) {
      values[c + j] = x[j];
      sum += a.last_centred ? x[j] : x[j] * x[j];
    }
  }
  if (out == nullptr || a.last_weight == nullptr) return;
  row_norm<V>(values, hidden, a.last_centred, a.last_eps, sum, scratch, mean, r);
  for (int c = threadIdx.x * V; c < hidden; c += 256 * V) {
    float w[V];
    read_row<W, V>(static_cast<const W*>(a.last_weight) + c, w);
#pragma unroll
    for (int j = 0; j < V; ++j) w[j] *= (values[c + j] - mean) * r;
    if (a.last_bias != nullptr) {
      float b[V];
      read_row<W, V>(static_cast<const W*>(a.last_bias) + c, b);
#pragma unroll
      for (int j = 0; j < V; ++j) w[j] += b[j];
    }
    write_row<O, V>(out + c, w);
  }
}

}  // namespace tlie

using namespace tlie;

// residual: float [tokens, hidden]; d1, d2: products [nsplit][tokens][hidden] of their types (d2 or null); side1, side2
// (both or none), weight, bias, last_weight, last_bias: [hidden] of w_dtype; out (or null): [count, hidden] of out_dtype.
// count: how many rows (all tokens, or the entries of `rows`).
extern "C" int tlie_post_norm(float* residual, const void* d1, int d1_dtype, int n1, long long stride1, float s1, const void* d2,
                              int d2_dtype, int n2, long long stride2, float s2, const void* side1, const void* side2,
                              float side_eps, float mult, const void* weight, const void* bias, float eps, int centred,
                              const void* last_weight, const void* last_bias, float last_eps, int last_centred, int w_dtype,
                              void* out, int out_dtype, const int* rows, int count, int hidden, void* stream) {
  if (count <= 0 || hidden <= 0 || n1 < 1 || n2 < 1 || residual == nullptr) return kBadArgument;
  if (weight != nullptr && (d1 == nullptr || !(eps > 0.f))) return kBadArgument;
  if ((side1 == nullptr) != (side2 == nullptr) || (side1 != nullptr && (weight == nullptr || d2 == nullptr || !(side_eps > 0.f)))) return kBadArgument;
  if (last_weight != nullptr && (out == nullptr || !(last_eps > 0.f))) return kBadArgument;
  const size_t lds = static_cast<size_t>(hidden) * (side1 != nullptr ? 2 : 1) * sizeof(float);
  if (lds > 128000) return kBadArgument;
  const bool wide = (hidden & 7) == 0 && (n1 == 1 || stride1 % 8 == 0) && (n2 == 1 || stride2 % 8 == 0) &&
                    ((reinterpret_cast<uintptr_t>(residual) | reinterpret_cast<uintptr_t>(d1) | reinterpret_cast<uintptr_t>(d2) |
                      reinterpret_cast<uintptr_t>(side1) | reinterpret_cast<uintptr_t>(side2) | reinterpret_cast<uintptr_t>(weight) |
                      reinterpret_cast<uintptr_t>(bias) | reinterpret_cast<uintptr_t>(last_weight) |
                      reinterpret_cast<uintptr_t>(last_bias) | reinterpret_cast<uintptr_t>(out)) & 31) == 0;
  const PostNormArgs a{residual, d1, d2, n1, n2, (size_t)stride1, (size_t)stride2, s1, s2, side1, side2, side_eps, mult, weight, bias,
                       eps, centred, last_weight, last_bias, last_eps, last_centred, out, rows, hidden};
  hipStream_t s = (hipStream_t)stream;
#define TLIE_CASE(AC, A, BC, B, WC, W, OC, O)                                                                     \
  if (d1_dtype == AC && d2_dtype == BC && w_dtype == WC && out_dtype == OC) {                                     \
    if (wide) hipLaunchKernelGGL((post_norm_kernel<A, B, W, O, 8>), dim3(count), dim3(256), lds, s, a);           \
    else hipLaunchKernelGGL((post_norm_kernel<A, B, W, O, 1>), dim3(count), dim3(256), lds, s, a);                \
    return launch_status();                                                                                       \
  }
  TLIE_CASE(kF32, float, kF32, float, kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kF32, float, kBF16, bf16, kF32, float)
  TLIE_CASE(kF32, float, kF32, float, kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kF32, float, kBF16, bf16, kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kF32, float, kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kBF16, bf16, kF32, float)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kF32, float, kBF16, bf16)
  TLIE_CASE(kF32, float, kF32, float, kF32, float, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}
