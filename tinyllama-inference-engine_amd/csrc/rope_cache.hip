// Rotary positions on q and k, and the write of k and v into the paged cache, in one pass over
// the fused qkv projection's output.
//
// reference: RopeKernel (src/cuda/kernels.cu:86-115) rotates the pair (i, i + d/2) of every head
// by angle = float(position) * theta^(-2i/d), sine and cosine in float; KvUpdateKernel
// (kernels.cu:137-145) then copies the rotated key and the value to the cache row of the
// position.  Here all tokens of a step go in one launch, positions come from an array, the
// frequencies from a table made once per model, and the cache row is found through the slot map.
// A block serves a few heads of one token: it first forms the token's d/2 sines and cosines once
// (not once per head), then every thread sums its element's partial results, trades it with its
// rotation partner through LDS, and writes q or the cache.
#include "common.h"

namespace tlie {

// qkv: [nsplit][tokens][(nq + 2 nkv) * d], columns ordered q heads | k heads | v heads.
// q_out: [tokens][nq * d].  cache: [pages][2][nkv][page_size * d]: keys at index 0 as [row][dim],
// values at index 1 transposed, [dim][row] (the attention kernels read 4 consecutive rows of one dim).
// slot_map[t] = page * page_size + row of token t, or -1: nothing is written for that token.
// rot_dim <= d, even: dimensions from rot_dim on are copied unrotated.  inv_freq may be null
// (no rotation at all).  paired: within a q or k head the input's columns are stored with the two
// elements of a rotation pair side by side (element i at 2i, element i + rot_dim/2 at 2i + 1), as
// the product of few rows wants its weight's rows; outputs are in natural order either way.
// row_width: columns of a row of the product, of which q, k and v are the first.  head_scale (or null): float [nq], query head
// h is multiplied by head_scale[h].
// blockDim.x = heads_per_block * d; grid = (tokens, ceil(heads / heads_per_block)).
template <typename D, typename A>
__global__ void rope_cache_kernel(const D* __restrict__ qkv, int nsplit, size_t split_stride,
                                  const int* __restrict__ positions, const int* __restrict__ slot_map,
                                  const float* __restrict__ inv_freq, int rot_dim, A* __restrict__ q_out,
                                  A* __restrict__ cache, int nq, int nkv, int d, int page_size, int paired, int row_width,
                                  const float* __restrict__ head_scale) {
  extern __shared__ float lds[];
  float* cosines = lds;                  // rot_dim / 2
  float* sines = cosines + rot_dim / 2;  // rot_dim / 2
  float* values = sines + rot_dim / 2;   // blockDim.x
  const int t = blockIdx.x;
  const int heads = nq + 2 * nkv;
  const int half = rot_dim / 2;
  if (inv_freq != nullptr) {
    const float pos = static_cast<float>(positions[t]);
    for (int i = threadIdx.x; i < half; i += blockDim.x) sincosf(pos * inv_freq[i], &sines[i], &cosines[i]);
  }
  const int local_head = threadIdx.x / d, e = threadIdx.x % d;
  const int head = blockIdx.y * (blockDim.x / d) + local_head;
  const bool live = head < heads;
  float mine = 0.f;
  int column = e;
  if (paired && head < nq + nkv && e < rot_dim) column = e < half ? 2 * e : 2 * (e - half) + 1;
  if (live) mine = sum_splits(qkv + static_cast<size_t>(t) * row_width + head * d + column, nsplit, split_stride);
  if (head_scale != nullptr && head < nq) mine *= head_scale[head];
  values[threadIdx.x] = mine;
  __syncthreads();
  if (!live) return;
  float result = mine;
  if (inv_freq != nullptr && head < nq + nkv && e < rot_dim) {
    if (e < half) {
      result = mine * cosines[e] - values[threadIdx.x + half] * sines[e];
    } else {
      result = mine * cosines[e - half] + values[threadIdx.x - half] * sines[e - half];
    }
  }
  if (head < nq) {
    q_out[static_cast<size_t>(t) * nq * d + head * d + e] = from_float<A>(result);
    return;
  }
  const int slot = slot_map[t];
  if (slot < 0) return;
  const size_t head_stride = static_cast<size_t>(page_size) * d;
  A* page = cache + static_cast<size_t>(slot / page_size) * 2 * nkv * head_stride;
  const int row = slot % page_size;
  if (head < nq + nkv) {
    page[(head - nq) * head_stride + static_cast<size_t>(row) * d + e] = from_float<A>(result);
  } else {
    // value head (head - nq - nkv) lies after the nkv key heads: at head offset (head - nq), transposed
    page[(head - nq) * head_stride + static_cast<size_t>(e) * page_size + row] = from_float<A>(result);
  }
}

// The same for one summand with eight input columns a thread (16-byte loads): d % 8 == 0 and, where
// there is rotation, paired columns and rot_dim % 8 == 0, so that a thread holds four whole pairs.
// One block a token; blockDim.x covers (nq + 2 nkv) * d / 8 groups, or loops.
template <typename D, typename A>
__global__ void rope_cache_wide_kernel(const D* __restrict__ qkv, const int* __restrict__ positions,
                                       const int* __restrict__ slot_map, const float* __restrict__ inv_freq,
                                       int rot_dim, A* __restrict__ q_out, A* __restrict__ cache, int nq, int nkv,
                                       int d, int page_size, int row_width, const float* __restrict__ head_scale) {
  extern __shared__ float lds[];
  const int half = rot_dim / 2;
  float* cosines = lds;                  // half
  float* sines = cosines + half;         // half
  const int t = blockIdx.x;
  const int heads = nq + 2 * nkv, per_head = d / 8;
  const int slot = slot_map[t];
  // this thread's first eight columns are asked for before the angles are made: their way from memory
  // is then hidden behind the sines and cosines (and the barrier after them)
  float first_v[8];
  const bool first_live = static_cast<int>(threadIdx.x) < heads * per_head;
  if (first_live)
    load8(qkv + static_cast<size_t>(t) * row_width + threadIdx.x * 8, first_v);
  if (inv_freq != nullptr) {
    const float pos = static_cast<float>(positions[t]);
    for (int i = threadIdx.x; i < half; i += blockDim.x) sincosf(pos * inv_freq[i], &sines[i], &cosines[i]);
    __syncthreads();
  }
  const size_t head_stride = static_cast<size_t>(page_size) * d;
  A* page = cache + static_cast<size_t>(slot < 0 ? 0 : slot / page_size) * 2 * nkv * head_stride;
  const int row = slot < 0 ? 0 : slot % page_size;
  for (int g = threadIdx.x; g < heads * per_head; g += blockDim.x) {
    const int head = g / per_head, c = (g % per_head) * 8;
    if (head >= nq && slot < 0) continue;
    float v[8];
    if (g == static_cast<int>(threadIdx.x)) {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = first_v[j];
    } else {
      load8(qkv + static_cast<size_t>(t) * row_width + g * 8, v);
    }
    if (head_scale != nullptr && head < nq) {
      const float scale = head_scale[head];
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] *= scale;
    }
    if (head >= nq + nkv) {
      // a value head: after the nkv key heads of the page, transposed
      A* out = page + (head - nq) * head_stride + static_cast<size_t>(c) * page_size + row;
#pragma unroll
      for (int j = 0; j < 8; ++j) out[static_cast<size_t>(j) * page_size] = from_float<A>(v[j]);
      continue;
    }
    A* out = head < nq ? q_out + (static_cast<size_t>(t) * nq + head) * d
                       : page + (head - nq) * head_stride + static_cast<size_t>(row) * d;
    if (inv_freq != nullptr && c < rot_dim) {
      const int first = c / 2;           // v[2j], v[2j + 1] = elements first + j and first + j + half
      float lo[4], hi[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float cs = cosines[first + j], sn = sines[first + j];
        lo[j] = v[2 * j] * cs - v[2 * j + 1] * sn;
        hi[j] = v[2 * j + 1] * cs + v[2 * j] * sn;
      }
      store4(out + first, lo[0], lo[1], lo[2], lo[3]);
      store4(out + half + first, hi[0], hi[1], hi[2], hi[3]);
    } else {
      store8(out + c, v);
    }
  }
}

// The same for any sizes: value heads of a size dv of their own (a page then holds nkv planes of keys
// [row][d] and after them nkv planes of values [dv][row]), or no key and value heads at all (nkv = 0: the
// layer reads another layer's cache and only its queries are placed).  Columns in natural order; a
// rotated element reads its partner's summands itself.  One block a token.
// Options (each off when its pointer is null or its number zero):
//   q_norm, k_norm   float weights [nq * d], [nkv * d]: all of a token's query columns together (and all of its key
//                    columns together) are divided by their root mean square, eps inside the root, and multiplied by
//                    the weight, before the rotation
//   values_are_keys  the product has no value columns: a key head's columns as projected (before norm and rotation)
//                    are also its value head (nv = nkv, dv = d)
//   head_scale       float [nq]: query head h is multiplied by head_scale[h] (a factor of its scores)
//   temp_coef, temp_every   a query at position p is multiplied by 1 + temp_coef * ln(floor((p + 1) / temp_every) + 1)
struct PlaceOptions {
  const float* q_norm;
  const float* k_norm;
  float eps;
  int values_are_keys;
  float temp_coef;
  float temp_every;
  const float* head_scale;
  int stage;         // the launch gave LDS for the q and k columns (set by the entry point)
};

template <typename D, typename A>
__global__ void qkv_place_kernel(const D* __restrict__ qkv, int nsplit, size_t split_stride,
                                 const int* __restrict__ positions, const int* __restrict__ slot_map,
                                 const float* __restrict__ inv_freq, int rot_dim, A* __restrict__ q_out,
                                 A* __restrict__ cache, int nq, int nkv, int nv, int d, int dv, int page_size, int row_width,
                                 PlaceOptions options) {
  extern __shared__ float lds[];
  const int half = rot_dim / 2;
  float* cosines = lds;                  // half
  float* sines = cosines + half;         // half
  float* scratch = sines + half;         // 16
  float* staged = scratch + 16;          // the q and k columns as floats, when the launch gave the room (stage != 0)
  const int t = blockIdx.x;
  const int rotated = (nq + nkv) * d, width = rotated + (options.values_are_keys ? 0 : nv * dv);
  const D* in = qkv + static_cast<size_t>(t) * row_width;
  if (inv_freq != nullptr) {
    const float pos = static_cast<float>(positions[t]);
    for (int i = threadIdx.x; i < half; i += blockDim.x) sincosf(pos * inv_freq[i], &sines[i], &cosines[i]);
  }
  // With norms every q and k column is needed three times (its projection's sum of squares, itself, its rotation
  // partner): they are read once, into LDS, and the sums of squares are formed on the way.
  const bool stage = options.stage != 0;
  auto raw = [&](int c) { return stage ? staged[c] : sum_splits(in + c, nsplit, split_stride); };
  float q_scale = 1.f, k_scale = 1.f;
  if (options.q_norm != nullptr || options.k_norm != nullptr) {
    float q_square = 0.f, k_square = 0.f;
    for (int c = threadIdx.x; c < rotated; c += blockDim.x) {
      const float v = sum_splits(in + c, nsplit, split_stride);
      if (stage) staged[c] = v;
      if (c < nq * d) q_square += v * v;
      else k_square += v * v;
    }
    if (options.q_norm != nullptr) q_scale = rsqrtf(block_sum(q_square, scratch) / static_cast<float>(nq * d) + options.eps);
    if (options.k_norm != nullptr && nkv > 0) k_scale = rsqrtf(block_sum(k_square, scratch) / static_cast<float>(nkv * d) + options.eps);
  }
  __syncthreads();                       // the angles and the staged columns are written
  if (options.temp_every > 0.f)
    q_scale *= 1.f + options.temp_coef * logf(floorf(static_cast<float>(positions[t] + 1) / options.temp_every) + 1.f);
  // a column of q or k after its norm (and, for a query, its temperature), before the rotation
  auto normed = [&](int c) {
    const float v = raw(c);
    if (c < nq * d) {
      const float scaled = options.head_scale != nullptr ? v * q_scale * options.head_scale[c / d] : v * q_scale;
      return options.q_norm != nullptr ? scaled * options.q_norm[c] : scaled;
    }
    return options.k_norm != nullptr ? v * k_scale * options.k_norm[c - nq * d] : v;
  };
  const int slot = nkv > 0 ? slot_map[t] : -1;
  A* page = cache + static_cast<size_t>(slot < 0 ? 0 : slot / page_size) * page_size * (static_cast<size_t>(nkv) * d + static_cast<size_t>(nv) * dv);
  const int row = slot < 0 ? 0 : slot % page_size;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    if (c >= nq * d && slot < 0) break;  // (columns only grow: what is left is keys and values too)
    if (c >= rotated) {
      const int head = (c - rotated) / dv, e = (c - rotated) % dv;
      page[static_cast<size_t>(nkv) * page_size * d + (static_cast<size_t>(head) * dv + e) * page_size + row] =
          from_float<A>(sum_splits(in + c, nsplit, split_stride));
      continue;
    }
    const int head = c / d, e = c % d;
    float v = normed(c);
    if (inv_freq != nullptr && e < rot_dim) {
      if (e < half) v = v * cosines[e] - normed(c + half) * sines[e];
      else v = v * cosines[e - half] + normed(c - half) * sines[e - half];
    }
    if (head < nq) {
      q_out[static_cast<size_t>(t) * nq * d + c] = from_float<A>(v);
    } else {
      page[(static_cast<size_t>(head - nq) * page_size + row) * d + e] = from_float<A>(v);
      if (options.values_are_keys)
        page[static_cast<size_t>(nkv) * page_size * d + (static_cast<size_t>(head - nq) * d + e) * page_size + row] = from_float<A>(raw(c));
    }
  }
}

}  // namespace tlie

using namespace tlie;

// q heads of d | k heads of d | nv value heads of dv (nv = nkv, or fewer when several key heads share a value head:
// a page then holds the nkv planes of keys and after them nv planes of values); a row of the product is
// row_width columns long, of which these are the first.  See qkv_place_kernel and PlaceOptions (with values_are_keys
// the product holds no value columns).
extern "C" int tlie_qkv_place(const void* qkv, int in_dtype, int nsplit, long long split_stride, const int* positions,
                              const int* slot_map, const float* inv_freq, int rot_dim, void* q_out, void* cache,
                              int act_dtype, int tokens, int nq, int nkv, int nv, int d, int dv, int page_size, int row_width,
                              const float* q_norm, const float* k_norm, float norm_eps, int values_are_keys, float temp_coef,
                              float temp_every, const float* head_scale, void* stream) {
  if (tokens <= 0 || nq <= 0 || nkv < 0 || d <= 0 || dv <= 0 || page_size <= 0 || nsplit < 1) return kBadArgument;
  if (rot_dim < 0 || rot_dim > d || rot_dim % 2 != 0 || (nkv > 0 && (cache == nullptr || slot_map == nullptr))) return kBadArgument;
  if (nv < 0 || nv > nkv || (nkv > 0 && (nv == 0 || nkv % nv != 0))) return kBadArgument;
  if (values_are_keys && (nv != nkv || dv != d)) return kBadArgument;
  if ((q_norm != nullptr || k_norm != nullptr) && !(norm_eps > 0.f)) return kBadArgument;
  if (temp_every < 0.f) return kBadArgument;
  const int width = (nq + nkv) * d + (values_are_keys ? 0 : nv * dv);
  if (row_width < width) return kBadArgument;
  int threads = width >= 1024 ? 1024 : (width + 63) / 64 * 64;
  // with norms a workgroup waits several times for all its waves (two sums over the row); in a step of many tokens
  // smaller workgroups, more of which fit a compute unit, fill those waits with each other's work
  if ((q_norm != nullptr || k_norm != nullptr) && tokens > 64 && threads > 256) threads = 256;
  const bool normed = q_norm != nullptr || k_norm != nullptr;
  const size_t columns = static_cast<size_t>(nq + nkv) * d;
  const int stage = normed && columns <= 14000 ? 1 : 0;          // (beyond that a row does not fit beside the rest: every read goes to memory)
  const size_t lds = (static_cast<size_t>(rot_dim) + 16 + (stage ? columns : 0)) * sizeof(float);
  const PlaceOptions options{q_norm, k_norm, norm_eps, values_are_keys, temp_coef, temp_every, head_scale, stage};
  hipStream_t s = (hipStream_t)stream;
#define TLIE_CASE(DC, D, AC, A)                                                                                \
  if (in_dtype == DC && act_dtype == AC) {                                                                     \
    hipLaunchKernelGGL((qkv_place_kernel<D, A>), dim3(tokens), dim3(threads), lds, s, (const D*)qkv, nsplit,     \
                       (size_t)split_stride, positions, slot_map, inv_freq, rot_dim, (A*)q_out, (A*)cache, nq,  \
                       nkv, nv, d, dv, page_size, row_width, options);                                          \
    return launch_status();                                                                                    \
  }
  TLIE_CASE(kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}

extern "C" int tlie_rope_cache(const void* qkv, int in_dtype, int nsplit, long long split_stride,
                               const int* positions, const int* slot_map, const float* inv_freq, int rot_dim,
                               void* q_out, void* cache, int act_dtype, int tokens, int nq, int nkv, int d,
                               int page_size, int paired, int row_width, const float* head_scale, void* stream) {
  if (row_width < (nq + 2 * nkv) * d) return kBadArgument;
  if (tokens <= 0 || nq <= 0 || nkv <= 0 || d <= 0 || d > 1024 || page_size <= 0 || nsplit < 1) return kBadArgument;
  if (rot_dim < 0 || rot_dim > d || rot_dim % 2 != 0) return kBadArgument;
  const int heads = nq + 2 * nkv;
  hipStream_t s = (hipStream_t)stream;
  const bool aligned = ((reinterpret_cast<uintptr_t>(qkv) | reinterpret_cast<uintptr_t>(q_out) |
                         reinterpret_cast<uintptr_t>(cache)) & 31) == 0;
  if (nsplit == 1 && (d & 7) == 0 && (row_width & 7) == 0 && aligned && (inv_freq == nullptr || (paired && (rot_dim & 7) == 0))) {
    const int groups = heads * d / 8;
    const int wide = groups >= 1024 ? 1024 : (groups + 63) / 64 * 64;
    const size_t wide_lds = static_cast<size_t>(rot_dim) * sizeof(float);
#define TLIE_WIDE(DC, D, AC, A)                                                                              \
  if (in_dtype == DC && act_dtype == AC) {                                                                   \
    hipLaunchKernelGGL((rope_cache_wide_kernel<D, A>), dim3(tokens), dim3(wide), wide_lds, s, (const D*)qkv,   \
                       positions, slot_map, inv_freq, rot_dim, (A*)q_out, (A*)cache, nq, nkv, d, page_size,   \
                       row_width, head_scale);                                                               \
    return launch_status();                                                                                  \
  }
    TLIE_WIDE(kF32, float, kF32, float)
    TLIE_WIDE(kF32, float, kBF16, bf16)
    TLIE_WIDE(kBF16, bf16, kBF16, bf16)
#undef TLIE_WIDE
    return kBadArgument;
  }
  int heads_per_block = 256 / d;
  if (heads_per_block < 1) heads_per_block = 1;
  if (heads_per_block > heads) heads_per_block = heads;
  const int threads = heads_per_block * d;
  const dim3 grid(tokens, (heads + heads_per_block - 1) / heads_per_block);
  if (grid.y > 65535) return kBadArgument;
  const size_t lds = (static_cast<size_t>(rot_dim) + threads) * sizeof(float);
#define TLIE_CASE(DC, D, AC, A)                                                                              \
  if (in_dtype == DC && act_dtype == AC) {                                                                   \
    hipLaunchKernelGGL((rope_cache_kernel<D, A>), grid, dim3(threads), lds, s, (const D*)qkv, nsplit,         \
                       (size_t)split_stride, positions, slot_map, inv_freq, rot_dim, (A*)q_out, (A*)cache, nq, \
                       nkv, d, page_size, paired, row_width, head_scale);                                    \
    return launch_status();                                                                                  \
  }
  TLIE_CASE(kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}
