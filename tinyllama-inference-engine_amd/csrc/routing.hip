// Products with a handful of outputs whose sums are float whatever the types (a router's logits, the gates of a
// recurrence), and what a routed feed-forward does with a router's scores.
//
//   few_outputs      out[t, n] = bias[n] + sum_k x[t, k] w[n, k]                          float out
//   ... as a router  s = sigmoid(out[t, :]); the `top` largest s (the lower index wins a tie) keep their s,
//                    all others become 0: scale[t, n]                                      float out
//   ... mode 1       the `top` largest sums themselves are picked, and keep their softmax over the picked ones only
//   ... extra        the last `extra` outputs stand outside the choice: each becomes its own sigmoid (a gate
//                    of something that every token uses)
//   routed_gate      hidden[t, c] = act(s g) * (s u), s = scale[t, c / block] for the first experts * block
//                    columns and 1 for the rest (a shared expert's), g and u side by side in gate_up[t, 2c], [2c + 1]
//   ... weigh 1      hidden[t, c] = s * act(g, u): the score weighs the expert's result (the second product is
//                    linear, so its input is weighed in the result's place); shared_scaled: the shared expert's
//                    columns take scale[t, experts] instead of 1; the experts' and the shared expert's gates have
//                    their own limits
//   grouped_router   s = softmax(out[t, :]); the `top` largest s + correction are picked, among the outputs of the `keep`
//                    groups of neighbours whose best s + correction is largest; the picked ones' s divided by their sum
//                    are the weights: scale[t, n], 0 for the others; trailing outputs that stand for the identity (no
//                    expert of their own) share one last column, the sum of their weights
//   relu_squared     hidden[t, c] = s * max(up[t, c], 0)^2, s = scale[t, c / block], or 1 without scales
//
// A token is a workgroup's: wave w of its four takes outputs w, w + 4, ..., lane l the inner indices l, l + 64,
// ...: the order of a sum depends on the sizes alone.
#include "common.h"

namespace tlie {

// The float sum over the inner index of one token's row times one output's weights, in every lane of the wave.
// wide: eight inner indices a lane and load (a wave then asks for a kilobyte or two at once, and a sum of 2048 terms waits
// for memory four times, not sixteen); inner % 8 == 0 and rows at multiples of 32 bytes.
template <typename X, typename W>
__device__ __forceinline__ float few_sum(const X* __restrict__ row, const W* __restrict__ weights, int inner, bool wide, int lane) {
  float a = 0.f, b = 0.f;
  if (wide) {
#pragma unroll 2
    for (int k = lane * 8; k < inner; k += 512) {
      float xv[8], wv[8];
      load8(row + k, xv);
      load8(weights + k, wv);
      a += xv[0] * wv[0];
      b += xv[1] * wv[1];
      a += xv[2] * wv[2];
      b += xv[3] * wv[3];
      a += xv[4] * wv[4];
      b += xv[5] * wv[5];
      a += xv[6] * wv[6];
      b += xv[7] * wv[7];
    }
  } else {
    int k = lane;
    for (; k + 64 < inner; k += 128) {
      a += to_float(row[k]) * to_float(weights[k]);
      b += to_float(row[k + 64]) * to_float(weights[k + 64]);
    }
    if (k < inner) a += to_float(row[k]) * to_float(weights[k]);
  }
  return wave_sum(a + b);
}

template <typename X, typename W>
__device__ __forceinline__ bool few_wide(const X* x, const W* w, int inner) {
  return (inner & 7) == 0 && ((reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(w)) & 31) == 0;
}

// The largest of a value a lane, and where it is: the lower index of equals; in every lane.
__device__ __forceinline__ void wave_best(float& best, int& where) {
#pragma unroll
  for (int offset = 32; offset > 0; offset >>= 1) {
    const float other = __shfl_xor(best, offset, 64);
    const int other_where = __shfl_xor(where, offset, 64);
    if (other > best || (other == best && other_where < where)) best = other, where = other_where;
  }
}

// What one lane of a wave wrote to LDS is there for the others' next reads (one wave: its LDS operations complete in order).
__device__ __forceinline__ void wave_lds_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

template <typename X, typename W>
__global__ void __launch_bounds__(256)
few_outputs_kernel(const X* __restrict__ x, const W* __restrict__ w, const W* __restrict__ bias, float* __restrict__ out,
                   int inner, int outputs, int top, int mode, int extra) {
  extern __shared__ float sums[];                      // outputs
  const int t = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const X* row = x + static_cast<size_t>(t) * inner;
  const bool wide = few_wide(x, w, inner);
  for (int n = wave; n < outputs; n += 4) {
    float total = few_sum(row, w + static_cast<size_t>(n) * inner, inner, wide, lane);
    if (bias != nullptr) total += to_float(bias[n]);
    if (top <= 0) {
      if (lane == 0) out[static_cast<size_t>(t) * outputs + n] = total;
    } else if (lane == 0) {
      sums[n] = (mode == 0 || n >= outputs - extra) ? 1.f / (1.f + expf(-total)) : total;
    }
  }
  if (top <= 0) return;
  __syncthreads();
  if (wave != 0) return;
  // the first wave picks: `top` times the largest score that is left, the lower index on a tie
  float* picked_out = out + static_cast<size_t>(t) * outputs;
  const int choices = outputs - extra;
  for (int n = lane; n < outputs; n += 64) picked_out[n] = n < choices ? 0.f : sums[n];
  const float gone = mode == 0 ? -2.f : -INFINITY;      // (below every score that is left)
  float first = 0.f, denominator = 0.f;                // mode 1: the largest picked sum, and the sum of the picked ones' exponentials
  int my_where = -1;
  float my_weight = 0.f;
  for (int round = 0; round < top; ++round) {
    float best = mode == 0 ? -1.f : -INFINITY;
    int where = 1 << 30;
    for (int n = lane; n < choices; n += 64) {
      const float s = sums[n];
      if (s > best) best = s, where = n;               // (ascending n: the first of equals stays)
    }
    wave_best(best, where);
    if (where >= choices) break;                       // fewer outputs than `top` (or sums that are not finite)
    if (round == 0) first = best;
    const float weight = mode == 0 ? best : expf(best - first);
    denominator += weight;
    if (mode == 1 && lane == round) my_where = where, my_weight = weight;      // (every lane holds the round's pick; lane `round` keeps it)
    if (lane == 0) {
      if (mode == 0) picked_out[where] = weight;
      sums[where] = gone;
    }
    wave_lds_fence();                                  // lane 0's writes come before the other lanes' next reads of sums[]
  }
  if (mode == 1 && my_where >= 0) picked_out[my_where] = my_weight / denominator;   // (at most 64 picks: one a lane)
}

// outputs: experts and, after them, identities; groups: equal groups of neighbours over all outputs.  correction: float
// [outputs] or null.  scale: [tokens, columns], columns = experts + (identities > 0).
template <typename X, typename W>
__global__ void __launch_bounds__(256)
grouped_router_kernel(const X* __restrict__ x, const W* __restrict__ w, const float* __restrict__ correction,
                      float* __restrict__ scale, int inner, int outputs, int identities, int top, int groups, int keep) {
  extern __shared__ float lds[];
  float* scores = lds;                                 // outputs: the sums, then their softmax
  float* choice = scores + outputs;                    // outputs: what the choice goes by; -infinity: not to be picked (any more)
  float* weights = choice + outputs;                   // outputs: a picked one's score, else 0
  float* best_of = weights + outputs;                  // groups: a group's best choice score
  const int t = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const X* row = x + static_cast<size_t>(t) * inner;
  const bool wide = few_wide(x, w, inner);
  for (int n = wave; n < outputs; n += 4) {
    const float total = few_sum(row, w + static_cast<size_t>(n) * inner, inner, wide, lane);
    if (lane == 0) scores[n] = total;
  }
  __syncthreads();
  if (wave != 0) return;
  float largest = -INFINITY, sum = 0.f;
  for (int n = lane; n < outputs; n += 64) largest = fmaxf(largest, scores[n]);
  largest = wave_max(largest);
  for (int n = lane; n < outputs; n += 64) sum += expf(scores[n] - largest);
  sum = wave_sum(sum);
  for (int n = lane; n < outputs; n += 64) {
    const float s = expf(scores[n] - largest) / sum;
    scores[n] = s;
    choice[n] = correction != nullptr ? s + correction[n] : s;
    weights[n] = 0.f;
  }
  wave_lds_fence();
  if (keep < groups) {
    const int size = outputs / groups;
    for (int g = lane; g < groups; g += 64) {
      float best = -INFINITY;
      for (int i = 0; i < size; ++i) best = fmaxf(best, choice[g * size + i]);
      best_of[g] = best;
    }
    wave_lds_fence();
    // a group stays when fewer than `keep` groups are better (of equals, the lower one is)
    for (int g = lane; g < groups; g += 64) {
      const float mine = best_of[g];
      int better = 0;
      for (int o = 0; o < groups; ++o) better += best_of[o] > mine || (best_of[o] == mine && o < g);
      if (better >= keep)
        for (int i = 0; i < size; ++i) choice[g * size + i] = -INFINITY;
    }
    wave_lds_fence();
  }
  float denominator = 0.f;
  for (int round = 0; round < top; ++round) {
    float best = -INFINITY;
    int where = 1 << 30;
    for (int n = lane; n < outputs; n += 64)
      if (choice[n] > best) best = choice[n], where = n;       // (ascending n: the first of equals stays)
    wave_best(best, where);
    if (where >= outputs) break;                       // (nothing left that can be picked, or sums that are not finite)
    denominator += scores[where];
    if (lane == 0) weights[where] = scores[where], choice[where] = -INFINITY;
    wave_lds_fence();
  }
  const int experts = outputs - identities, columns = experts + (identities > 0 ? 1 : 0);
  const float share = 1.f / (denominator + 1e-20f);
  float* to = scale + static_cast<size_t>(t) * columns;
  for (int n = lane; n < experts; n += 64) to[n] = weights[n] * share;
  if (identities > 0) {
    float mine = 0.f;
    for (int n = experts + lane; n < outputs; n += 64) mine += weights[n];
    mine = wave_sum(mine);
    if (lane == 0) to[experts] = mine * share;
  }
}

__device__ __forceinline__ float relu_squared(float z) {
  z = fmaxf(z, 0.f);
  return z * z;
}

// scale (or null): float, of which token t's number for column c is scale[t * scale_cols + c / block].  V columns a thread
// (8: inter and block multiples of 8, no partial sums, rows at multiples of 32 bytes).
template <typename D, typename A, int V>
__global__ void __launch_bounds__(256)
relu_squared_kernel(const D* __restrict__ up, int nsplit, size_t split_stride, const float* __restrict__ scale, int scale_cols,
                    int block, A* __restrict__ out, int inter) {
  const int t = blockIdx.x;
  const D* row = up + static_cast<size_t>(t) * inter;
  A* to = out + static_cast<size_t>(t) * inter;
  for (int c = (blockIdx.y * 256 + threadIdx.x) * V; c < inter; c += gridDim.y * 256 * V) {
    const float s = scale != nullptr ? scale[static_cast<size_t>(t) * scale_cols + c / block] : 1.f;
    if constexpr (V == 8) {
      float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (s != 0.f) load8(row + c, v);                 // (an expert that the token does not use is not read)
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = s != 0.f ? s * relu_squared(v[j]) : 0.f;
      store8(to + c, v);
    } else {
      to[c] = from_float<A>(s != 0.f ? s * relu_squared(sum_splits(row + c, nsplit, split_stride)) : 0.f);
    }
  }
}

// A choice without a router: the token's id names its experts.  scale[t, e] = weight for the `top` experts of row ids[t] of
// the table, 0 for the others, and 1 in the `always` columns after them (experts that every token uses).
__global__ void __launch_bounds__(256)
table_scale_kernel(const int* __restrict__ ids, const int* __restrict__ table, float* __restrict__ scale, int tokens, int vocab,
                   int experts, int always, int top, float weight) {
  const int cols = experts + always;
  const size_t total = static_cast<size_t>(tokens) * cols;
  for (size_t i = blockIdx.x * static_cast<size_t>(256) + threadIdx.x; i < total; i += static_cast<size_t>(gridDim.x) * 256) {
    const int t = static_cast<int>(i / cols), e = static_cast<int>(i % cols);
    float v = e < experts ? 0.f : 1.f;
    const int id = ids[t];
    if (e < experts && id >= 0 && id < vocab)
      for (int j = 0; j < top; ++j)
        if (table[static_cast<size_t>(id) * top + j] == e) v = weight;
    scale[i] = v;
  }
}

// weigh 0: the score weighs the expert's input (act(s g) * (s u)); 1: its result (s * act(g, u)).  scale_cols: columns of a
// row of the scale matrix; shared_scaled: the columns after the experts' take scale[t, experts], not 1.  kind, alpha:
// the gate (see gated_value); limit, shared_limit: its limit for the experts' and for the shared expert's columns.
struct GateOptions {
  int weigh;
  int scale_cols;
  int shared_scaled;
  int kind;
  float alpha;
  float limit;
  float shared_limit;
};

template <typename D, typename A>
__global__ void __launch_bounds__(256)
routed_gate_kernel(const D* __restrict__ gate_up, int nsplit, size_t split_stride, const float* __restrict__ scale,
                   int experts, int block, A* __restrict__ out, int inter, bool wide, GateOptions options) {
  const int t = blockIdx.x;
  const D* row = gate_up + static_cast<size_t>(t) * 2 * inter;
  if (wide) {
    // four columns a thread: eight values in one load, four out in one store (no partial sums, four columns in one
    // expert's block, rows that start at multiples of 32 bytes)
    for (int c = (blockIdx.y * 256 + threadIdx.x) * 4; c < inter; c += gridDim.y * 1024) {
      const int e = c / block;
      const bool own = e < experts;
      const float s = own ? scale[static_cast<size_t>(t) * options.scale_cols + e]
                          : (options.shared_scaled ? scale[static_cast<size_t>(t) * options.scale_cols + experts] : 1.f);
      float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (s != 0.f) load8(row + 2 * c, v);
      A* to = out + static_cast<size_t>(t) * inter + c;
      const float limit = own ? options.limit : options.shared_limit;
      if (s == 0.f) store4(to, 0.f, 0.f, 0.f, 0.f);
      else if (options.weigh == 1)
        store4(to, s * gated_value(v[0], v[1], options.kind, options.alpha, limit), s * gated_value(v[2], v[3], options.kind, options.alpha, limit),
               s * gated_value(v[4], v[5], options.kind, options.alpha, limit), s * gated_value(v[6], v[7], options.kind, options.alpha, limit));
      else store4(to, gated_value(s * v[0], s * v[1], kGateSilu, 1.f, 0.f), gated_value(s * v[2], s * v[3], kGateSilu, 1.f, 0.f),
                  gated_value(s * v[4], s * v[5], kGateSilu, 1.f, 0.f), gated_value(s * v[6], s * v[7], kGateSilu, 1.f, 0.f));
    }
    return;
  }
  for (int c = blockIdx.y * 256 + threadIdx.x; c < inter; c += gridDim.y * 256) {
    const int e = c / block;
    const bool own = e < experts;
    const float s = own ? scale[static_cast<size_t>(t) * options.scale_cols + e]
                        : (options.shared_scaled ? scale[static_cast<size_t>(t) * options.scale_cols + experts] : 1.f);
    float v = 0.f;
    if (s != 0.f) {                                    // an expert the token does not use: silu(0) * 0
      const float g = sum_splits(row + 2 * c, nsplit, split_stride);
      const float u = sum_splits(row + 2 * c + 1, nsplit, split_stride);
      if (options.weigh == 1) v = s * gated_value(g, u, options.kind, options.alpha, own ? options.limit : options.shared_limit);
      else v = gated_value(s * g, s * u, kGateSilu, 1.f, 0.f);
    }
    out[static_cast<size_t>(t) * inter + c] = from_float<A>(v);
  }
}

}  // namespace tlie

using namespace tlie;

// x: [tokens, inner] of x_dtype; w: [outputs, inner] and bias (or null) [outputs] of w_dtype; out: float [tokens, outputs].
// top 0: the sums; top > 0: the router's scale matrix (see above).
// mode 0: sigmoid scores, the picked ones keep theirs; mode 1: the largest sums are picked and keep their softmax over the
// picked ones.  extra: trailing outputs outside the choice, which become their sigmoids (top > 0 only).
extern "C" int tlie_few_outputs(const void* x, int x_dtype, const void* w, const void* bias, int w_dtype, float* out,
                                int tokens, int inner, int outputs, int top, int mode, int extra, void* stream) {
  if (tokens <= 0 || inner <= 0 || outputs <= 0 || outputs > 4096 || top < 0) return kBadArgument;
  if (mode < 0 || mode > 1 || extra < 0 || (top == 0 && (mode != 0 || extra != 0)) || (top > 0 && top > outputs - extra) || (mode == 1 && top > 64)) return kBadArgument;
  hipStream_t s = (hipStream_t)stream;
  const size_t lds = static_cast<size_t>(outputs) * sizeof(float);
#define TLIE_CASE(XC, X, WC, W)                                                                                       \
  if (x_dtype == XC && w_dtype == WC) {                                                                               \
    hipLaunchKernelGGL((few_outputs_kernel<X, W>), dim3(tokens), dim3(256), lds, s, (const X*)x, (const W*)w,          \
                       (const W*)bias, out, inner, outputs, top, mode, extra);                                                     \
    return launch_status();                                                                                           \
  }
  TLIE_CASE(kF32, float, kF32, float)
  TLIE_CASE(kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}

// gate_up: a product [nsplit][tokens][2 * inter], gate and up of a column side by side; scale: float [tokens, experts];
// the first experts * block columns are the experts', the rest a shared expert's; out: [tokens, inter] of out_dtype.
// weigh, scale_cols, shared_scaled, kind, alpha, limit, shared_limit: see GateOptions (weigh 0 takes the SiLU gate).
extern "C" int tlie_routed_gate(const void* gate_up, int in_dtype, int nsplit, long long split_stride, const float* scale,
                                int experts, int block, void* out, int out_dtype, int tokens, int inter, int weigh,
                                int scale_cols, int shared_scaled, int kind, float alpha, float limit, float shared_limit,
                                void* stream) {
  if (tokens <= 0 || inter <= 0 || experts < 0 || block <= 0 || nsplit < 1) return kBadArgument;
  if (weigh < 0 || weigh > 1 || scale_cols < experts + (shared_scaled ? 1 : 0) || (weigh == 0 && kind != kGateSilu)) return kBadArgument;
  if (kind != kGateSilu && kind != kGateClampedSwish) return kBadArgument;
  const GateOptions options{weigh, scale_cols, shared_scaled, kind, alpha, limit, shared_limit};
  if (static_cast<long long>(experts) * block > inter) return kBadArgument;
  const bool wide = nsplit == 1 && (inter & 3) == 0 && (block & 3) == 0 &&
                    ((reinterpret_cast<uintptr_t>(gate_up) | reinterpret_cast<uintptr_t>(out)) & 31) == 0;
  int across = (inter + (wide ? 1023 : 255)) / (wide ? 1024 : 256);
  if (across > 64) across = 64;
  const dim3 grid(tokens, across);
  hipStream_t s = (hipStream_t)stream;
#define TLIE_CASE(DC, D, AC, A)                                                                                       \
  if (in_dtype == DC && out_dtype == AC) {                                                                            \
    hipLaunchKernelGGL((routed_gate_kernel<D, A>), grid, dim3(256), 0, s, (const D*)gate_up, nsplit,                   \
                       (size_t)split_stride, scale, experts, block, (A*)out, inter, wide, options);                                  \
    return launch_status();                                                                                           \
  }
  TLIE_CASE(kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}

// x: [tokens, inner] of x_dtype; w: [outputs, inner] of w_dtype; correction (or null): float [outputs]; the last
// `identities` outputs stand for the identity.  scale: float [tokens, outputs - identities (+ 1 when there are identities)].
// groups divides outputs; of the groups `keep` stay (keep == groups: all), which must hold at least `top` outputs.
extern "C" int tlie_grouped_router(const void* x, int x_dtype, const void* w, int w_dtype, const float* correction,
                                   float* scale, int tokens, int inner, int outputs, int identities, int top, int groups,
                                   int keep, void* stream) {
  if (tokens <= 0 || inner <= 0 || outputs <= 0 || outputs > 4096 || identities < 0 || identities > outputs) return kBadArgument;
  if (groups <= 0 || outputs % groups != 0 || keep <= 0 || keep > groups) return kBadArgument;
  if (top <= 0 || top > keep * (outputs / groups)) return kBadArgument;
  hipStream_t s = (hipStream_t)stream;
  const size_t lds = (static_cast<size_t>(outputs) * 3 + groups) * sizeof(float);
#define TLIE_CASE(XC, X, WC, W)                                                                                       \
  if (x_dtype == XC && w_dtype == WC) {                                                                               \
    hipLaunchKernelGGL((grouped_router_kernel<X, W>), dim3(tokens), dim3(256), lds, s, (const X*)x, (const W*)w,       \
                       correction, scale, inner, outputs, identities, top, groups, keep);                             \
    return launch_status();                                                                                           \
  }
  TLIE_CASE(kF32, float, kF32, float)
  TLIE_CASE(kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}

// up: a product [nsplit][tokens][inter] of in_dtype; scale (or null): float [tokens, scale_cols], a number for every `block`
// columns; out: [tokens, inter] of out_dtype.
extern "C" int tlie_relu_squared(const void* up, int in_dtype, int nsplit, long long split_stride, const float* scale,
                                 int scale_cols, int block, void* out, int out_dtype, int tokens, int inter, void* stream) {
  if (tokens <= 0 || inter <= 0 || nsplit < 1) return kBadArgument;
  if (scale != nullptr && (block <= 0 || scale_cols < (inter + block - 1) / block)) return kBadArgument;
  const bool wide = nsplit == 1 && (inter & 7) == 0 && (scale == nullptr || (block & 7) == 0) &&
                    ((reinterpret_cast<uintptr_t>(up) | reinterpret_cast<uintptr_t>(out)) & 31) == 0;
  const int per_block = wide ? 2048 : 256;
  int across = (inter + per_block - 1) / per_block;
  if (across > 64) across = 64;
  const dim3 grid(tokens, across);
  hipStream_t s = (hipStream_t)stream;
#define TLIE_CASE(DC, D, AC, A)                                                                                       \
  if (in_dtype == DC && out_dtype == AC) {                                                                            \
    if (wide)                                                                                                         \
      hipLaunchKernelGGL((relu_squared_kernel<D, A, 8>), grid, dim3(256), 0, s, (const D*)up, nsplit,                  \
                         (size_t)split_stride, scale, scale_cols, block, (A*)out, inter);                             \
    else                                                                                                              \
      hipLaunchKernelGGL((relu_squared_kernel<D, A, 1>), grid, dim3(256), 0, s, (const D*)up, nsplit,                  \
                         (size_t)split_stride, scale, scale_cols, block, (A*)out, inter);                             \
    return launch_status();                                                                                           \
  }
  TLIE_CASE(kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}

// ids: int [tokens]; table: int [vocab, top]; scale: float [tokens, experts + always].
extern "C" int tlie_table_scale(const int* ids, const int* table, float* scale, int tokens, int vocab, int experts, int always, int top,
                                float weight, void* stream) {
  if (tokens <= 0 || vocab <= 0 || experts <= 0 || always < 0 || top <= 0 || ids == nullptr || table == nullptr || scale == nullptr) return kBadArgument;
  const long long total = static_cast<long long>(tokens) * (experts + always);
  const long long blocks = (total + 255) / 256;
  hipLaunchKernelGGL(table_scale_kernel, dim3(static_cast<unsigned>(blocks < 4096 ? blocks : 4096)), dim3(256), 0, (hipStream_t)stream, ids,
                     table, scale, tokens, vocab, experts, always, top, weight);
  return launch_status();
}
