// A short causal convolution over time on columns of a product, and what becomes of its result head by head, in one pass:
//
//   y_t[c] = bias[c] + sum_j taps[c, n - 1 - j] * x_(t-j)[c]       zeros before the sequence's start
//   optionally silu;  per head optionally divided by its length, or by its root mean square times a weight the heads
//   share;  times a number;  optionally turned by the token's position;  then to an array, to the key rows or (transposed)
//   to the value rows of the paged cache.
//
// The columns are taken as up to three segments, each some heads of one size (or a plain stretch of channels, in pieces).
// A request's last n - 1 inputs x, oldest first, are its state: [n - 1][channels] floats at the start of its state row.
// Everything is float, whatever the product's type; what leaves is of the output's type.
//
// A wave takes a head (or several that fit its lanes) and walks tokens, a channel's last n inputs in registers.  The
// first workgroups (in x) take kConvTokens tokens each and skip a sequence's first n - 1 tokens of the step, whose window
// reaches into the state; the workgroups after them take a sequence each: those first tokens, from the state, and then
// the state's new rows, so that no workgroup reads state that another one writes.
//
// Tokens and sequences whose request slot is negative pad a recorded step: no state is read or written for them, and
// their rows of the array become zeros or stay unwritten.
#include "common.h"

namespace tlie {

constexpr int kConvTokens = 8, kConvMaxHead = 256;

struct ConvSegment {
  int first;               // its first channel
  int channels;
  int head;                // channels of a head (at most kConvMaxHead)
  int norm;                // 0: none; 1: divided by the length; 2: by the root mean square, times weight
  const float* weight;     // [head], or null: 1
  float eps;               // inside the root
  float scale;
  int rotated;             // turned by the position
  int target;              // 0: out, columns out_col ..; 1: key rows; 2: value rows
  int out_col;
};

struct ConvArgs {
  const void* in;          // [nsplit][tokens][row]
  int nsplit;
  size_t split_stride;
  int row, col;            // the channels are columns col .. of a row
  const void* taps;        // [channels, ntaps]
  const void* bias;        // [channels] or null
  float* state;
  size_t slot_stride;
  const int* token_seq;
  const int* token_slot;
  const int* seq_start;
  const int* seq_slot;
  int tokens, sequences, channels, ntaps, silu;
  int segments;
  ConvSegment segment[3];
  const int* positions;
  const float* inv_freq;   // [rot_dim / 2] or null
  int rot_dim;
  void* out;
  int out_row;
  void* cache;             // [pages][keys: nkv planes [row][d], values: nkv planes [dv][row]]
  const int* slot_map;
  int nkv, d, dv, page_size;
  int token_blocks;        // workgroups (in x) that take kConvTokens tokens each (set by the entry point)
};

__device__ __forceinline__ void wave_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// V: consecutive channels of a lane (4 where every segment's heads are a multiple of 4, then a head is one round of its
// lanes; else 1, in up to four rounds); NT: the most taps.
template <typename D, typename W, typename O, int V, int NT>
__global__ void __launch_bounds__(256)
short_conv_kernel(const ConvArgs a, int heads_per_block, int lane_bits) {
  constexpr int R = V == 4 ? 1 : kConvMaxHead / 64, N = R * V;
  extern __shared__ float lds[];
  const int half = a.rot_dim / 2;
  float* cosines = lds;                                // [kConvTokens][half]
  float* sines = cosines + kConvTokens * half;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* turn = sines + kConvTokens * half + wave * kConvMaxHead;       // this wave's head(s), for the rotation's partners
  const int back = a.ntaps - 1;
  const int token_blocks = a.token_blocks;
  const bool by_token = static_cast<int>(blockIdx.x) < token_blocks;
  int t0, t1, first = 0, count = 0, slot = -1;
  if (by_token) {
    t0 = blockIdx.x * kConvTokens;
    t1 = min(a.tokens, t0 + kConvTokens);
  } else {
    const int seq = blockIdx.x - token_blocks;
    slot = a.seq_slot[seq];
    first = a.seq_start[seq];
    count = a.seq_start[seq + 1] - first;
    if (slot < 0 || count <= 0) return;
    t0 = first;
    t1 = first + min(count, back);
  }
  float* held = by_token ? nullptr : a.state + static_cast<size_t>(slot) * a.slot_stride;
  if (a.inv_freq != nullptr) {
    for (int i = threadIdx.x; i < (t1 - t0) * half; i += 256) {
      const int b = i / half;
      sincosf(static_cast<float>(a.positions[t0 + b]) * a.inv_freq[i - b * half], &sines[i], &cosines[i]);
    }
    __syncthreads();
  }
  const D* in = static_cast<const D*>(a.in);
  const W* taps = static_cast<const W*>(a.taps);
  const int lanes = 1 << lane_bits, per_wave = 64 >> lane_bits;      // lanes a head, heads a wave
  const int sub = lane & (lanes - 1);
  turn += (lane >> lane_bits) * lanes * V;
  const int block_first = blockIdx.y * heads_per_block;
  for (int unit = block_first + wave * per_wave; unit < block_first + heads_per_block; unit += 4 * per_wave) {
    // this lane's segment and head
    int head = unit + (lane >> lane_bits), which = 0;
    ConvSegment seg = a.segment[0];
    for (; which < a.segments; ++which) {
      seg = a.segment[which];
      const int heads = (seg.channels + seg.head - 1) / seg.head;
      if (head < heads) break;
      head -= heads;
    }
    const bool live = which < a.segments && unit + (lane >> lane_bits) < block_first + heads_per_block;
    int inside[N];                                     // this lane's channels inside the head; -1: none
    float w[N][NT], x[N][NT], bias[N], norm_weight[N];
#pragma unroll
    for (int e = 0; e < N; ++e) {
      const int c = sub * V + (e / V) * lanes * V + e % V;
      inside[e] = live && c < seg.head && head * seg.head + c < seg.channels ? c : -1;
      const int channel = seg.first + head * seg.head + c;
      bias[e] = inside[e] >= 0 && a.bias != nullptr ? to_float(static_cast<const W*>(a.bias)[channel]) : 0.f;
      norm_weight[e] = inside[e] >= 0 && seg.weight != nullptr ? seg.weight[c] : 1.f;
#pragma unroll
      for (int j = 0; j < NT; ++j) {                   // w[e][j] weighs the input j tokens back
        w[e][j] = inside[e] >= 0 && j < a.ntaps ? to_float(taps[static_cast<size_t>(channel) * a.ntaps + back - j]) : 0.f;
        x[e][j] = 0.f;
      }
    }
    // the inputs of token t on this lane's channels (zeros for t < 0)
    auto fetch = [&](int t, float (&v)[N]) {
#pragma unroll
      for (int e = 0; e < N; ++e) v[e] = 0.f;
      if (t < 0) return;
      const D* from = in + static_cast<size_t>(t) * a.row + a.col + seg.first + head * seg.head;
      if (V == 4) {
        if (inside[0] < 0) return;
        for (int s = 0; s < a.nsplit; ++s) {
          const float4 part = load4(from + s * a.split_stride + inside[0]);
          v[0] += part.x, v[N > 1 ? 1 : 0] += part.y, v[N > 2 ? 2 : 0] += part.z, v[N > 3 ? 3 : 0] += part.w;
        }
      } else {
#pragma unroll
        for (int e = 0; e < N; ++e)
          if (inside[e] >= 0) v[e] = sum_splits(from + inside[e], a.nsplit, a.split_stride);
      }
    };
    auto shift = [&](const float (&v)[N]) {            // a token's inputs join the windows
#pragma unroll
      for (int e = 0; e < N; ++e) {
#pragma unroll
        for (int j = NT - 1; j > 0; --j) x[e][j] = x[e][j - 1];
        x[e][0] = v[e];
      }
    };
    // all of this workgroup's tokens are asked for before the first is worked on
    float ahead[kConvTokens][N];
#pragma unroll
    for (int b = 0; b < kConvTokens; ++b) fetch(t0 + b < t1 ? t0 + b : -1, ahead[b]);
    if (by_token) {
#pragma unroll
      for (int j = NT - 1; j > 0; --j) {
        float v[N];
        fetch(j <= back ? t0 - j : -1, v);
        shift(v);
      }
    } else {
#pragma unroll
      for (int e = 0; e < N; ++e)
#pragma unroll
        for (int j = 0; j < NT; ++j)
          if (j < back && inside[e] >= 0)
            x[e][j] = held[static_cast<size_t>(back - 1 - j) * a.channels + seg.first + head * seg.head + inside[e]];
    }
#pragma unroll
    for (int b = 0; b < kConvTokens; ++b) {
      const int t = t0 + b;
      if (t >= t1) break;
      shift(ahead[b]);
      bool pad = false;
      if (by_token) {
        pad = a.token_slot[t] < 0;
        if (!pad && t - a.seq_start[a.token_seq[t]] < back) continue;        // (its sequence's workgroup takes it)
      }
      float y[N];
      float squares = 0.f;
#pragma unroll
      for (int e = 0; e < N; ++e) {
        y[e] = bias[e];
#pragma unroll
        for (int j = 0; j < NT; ++j) y[e] += w[e][j] * x[e][j];
        if (a.silu) y[e] = y[e] / (1.f + expf(-y[e]));
        if (inside[e] < 0 || pad) y[e] = 0.f;
        squares += y[e] * y[e];
      }
      float scale = seg.scale;
      // (the lanes of a head are neighbours; the sum runs over them alone, for every head alike)
      for (int offset = lanes >> 1; offset > 0; offset >>= 1) squares += __shfl_xor(squares, offset, 64);
      if (seg.norm == 1) scale /= sqrtf(squares + seg.eps);
      else if (seg.norm == 2) scale /= sqrtf(squares / static_cast<float>(seg.head) + seg.eps);
#pragma unroll
      for (int e = 0; e < N; ++e) y[e] *= scale * norm_weight[e];
      if (a.inv_freq != nullptr) {                     // (the same for the whole launch)
        wave_fence();                                  // the token before has been read
#pragma unroll
        for (int e = 0; e < N; ++e)
          if (inside[e] >= 0) turn[inside[e]] = y[e];
        wave_fence();
        if (seg.rotated) {
          const float* cs = cosines + (t - t0) * half;
          const float* sn = sines + (t - t0) * half;
#pragma unroll
          for (int e = 0; e < N; ++e) {
            const int i = inside[e];
            if (i >= 0 && i < a.rot_dim)
              y[e] = i < half ? y[e] * cs[i] - turn[i + half] * sn[i] : y[e] * cs[i - half] + turn[i - half] * sn[i - half];
          }
        }
      }
      if (seg.target == 0) {
        O* to = static_cast<O*>(a.out) + static_cast<size_t>(t) * a.out_row + seg.out_col + head * seg.head;
        if (V == 4) {
          if (inside[0] >= 0) store4(to + inside[0], y[0], y[N > 1 ? 1 : 0], y[N > 2 ? 2 : 0], y[N > 3 ? 3 : 0]);
        } else {
#pragma unroll
          for (int e = 0; e < N; ++e)
            if (inside[e] >= 0) to[inside[e]] = from_float<O>(y[e]);
        }
        continue;
      }
      const int place = a.slot_map[t];
      if (place < 0 || pad) continue;
      O* page = static_cast<O*>(a.cache) + static_cast<size_t>(place / a.page_size) * a.page_size * a.nkv * (a.d + a.dv);
      const int r = place % a.page_size;
      if (seg.target == 1) {
        O* to = page + (static_cast<size_t>(head) * a.page_size + r) * a.d;
        if (V == 4) {
          if (inside[0] >= 0) store4(to + inside[0], y[0], y[N > 1 ? 1 : 0], y[N > 2 ? 2 : 0], y[N > 3 ? 3 : 0]);
        } else {
#pragma unroll
          for (int e = 0; e < N; ++e)
            if (inside[e] >= 0) to[inside[e]] = from_float<O>(y[e]);
        }
      } else {
        O* to = page + static_cast<size_t>(a.nkv) * a.page_size * a.d + static_cast<size_t>(head) * a.dv * a.page_size + r;
#pragma unroll
        for (int e = 0; e < N; ++e)
          if (inside[e] >= 0) to[static_cast<size_t>(inside[e]) * a.page_size] = from_float<O>(y[e]);
      }
    }
    if (by_token) continue;
    // the state's new rows: the last `back` inputs.  A sequence that brought fewer tokens has them in its windows.
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      if (j >= back) break;
      float v[N];
      if (count > back) {
        fetch(first + count - 1 - j, v);
      } else {
#pragma unroll
        for (int e = 0; e < N; ++e) v[e] = x[e][j];
      }
      float* to = held + static_cast<size_t>(back - 1 - j) * a.channels + seg.first + head * seg.head;
#pragma unroll
      for (int e = 0; e < N; ++e)
        if (inside[e] >= 0) to[inside[e]] = v[e];
    }
  }
}

}  // namespace tlie

using namespace tlie;

// segments: `count` rows of (first, channels, head, norm, rotated, target, out_col) with weights, eps and scales beside
// them; everything else as in ConvArgs.  in_dtype, w_dtype: of the product and of taps and bias; out_dtype: of out and
// cache.  The cache's pages are nkv planes of keys [row][d], then nkv planes of values [dv][row].
extern "C" int tlie_short_conv(const void* in, int in_dtype, int nsplit, long long split_stride, int row, int col,
                               const void* taps, const void* bias, int w_dtype, float* state, long long slot_stride,
                               const int* token_seq, const int* token_slot, const int* seq_start, const int* seq_slot,
                               int tokens, int sequences, int max_new, int channels, int ntaps, int silu, int count,
                               const int* table,
                               const void* const* weights, const float* eps, const float* scales, const int* positions,
                               const float* inv_freq, int rot_dim, void* out, int out_row, int out_dtype, void* cache,
                               const int* slot_map, int nkv, int d, int dv, int page_size, void* stream) {
  if (tokens <= 0 || sequences <= 0 || channels <= 0 || ntaps < 1 || ntaps > 8 || nsplit < 1 || count < 1 || count > 3) return kBadArgument;
  if (col < 0 || col + channels > row || (ntaps > 1 && (state == nullptr || slot_stride < static_cast<long long>(ntaps - 1) * channels))) return kBadArgument;
  if (rot_dim < 0 || rot_dim % 2 != 0 || rot_dim > kConvMaxHead || (inv_freq == nullptr && rot_dim != 0)) return kBadArgument;
  ConvArgs a{in, nsplit, (size_t)split_stride, row, col, taps, bias, state, (size_t)slot_stride, token_seq, token_slot, seq_start,
             seq_slot, tokens, sequences, channels, ntaps, silu, count, {}, positions, inv_freq, rot_dim, out, out_row, cache,
             slot_map, nkv, d, dv, page_size, 0};
  bool by_four = true;
  int widest = 0, heads = 0, at = 0;
  for (int s = 0; s < count; ++s) {
    const int* f = table + 7 * s;
    ConvSegment& seg = a.segment[s];
    seg = ConvSegment{f[0], f[1], f[2], f[3], static_cast<const float*>(weights[s]), eps[s], scales[s], f[4], f[5], f[6]};
    if (seg.first != at || seg.channels <= 0 || seg.head <= 0 || seg.head > kConvMaxHead || seg.norm < 0 || seg.norm > 2) return kBadArgument;
    if ((seg.norm != 0 || seg.rotated || seg.target != 0) && seg.channels % seg.head != 0) return kBadArgument;
    if (seg.norm != 0 && !(seg.eps > 0.f)) return kBadArgument;
    if (seg.rotated && (inv_freq == nullptr || rot_dim > seg.head || positions == nullptr)) return kBadArgument;
    if (seg.target == 0 && (out == nullptr || seg.out_col < 0 || seg.out_col + seg.channels > out_row)) return kBadArgument;
    if (seg.target < 0 || seg.target > 2 || (seg.target != 0 && (cache == nullptr || slot_map == nullptr || page_size <= 0 || nkv <= 0))) return kBadArgument;
    if (seg.target == 1 && (seg.head != d || seg.channels != nkv * d)) return kBadArgument;
    if (seg.target == 2 && (seg.head != dv || seg.channels != nkv * dv)) return kBadArgument;
    by_four = by_four && seg.head % 4 == 0 && seg.channels % 4 == 0 && (seg.target != 0 || (seg.out_col % 4 == 0 && out_row % 4 == 0));
    if (seg.head > widest) widest = seg.head;
    heads += (seg.channels + seg.head - 1) / seg.head;
    at += seg.channels;
  }
  if (at != channels) return kBadArgument;
  by_four = by_four && row % 4 == 0 && col % 4 == 0 && (nsplit == 1 || split_stride % 4 == 0) &&
            ((reinterpret_cast<uintptr_t>(in) |
              reinterpret_cast<uintptr_t>(out) | reinterpret_cast<uintptr_t>(cache)) & 15) == 0;
  int lane_bits = 0;
  while (lane_bits < 6 && ((by_four ? 4 : 1) << lane_bits) < widest) ++lane_bits;
  const int per_pass = 4 * (64 >> lane_bits);          // heads the four waves take at once
  const int passes = (heads + per_pass - 1) / per_pass;
  // (a step in which no sequence brings more tokens than its workgroup takes needs no others: what pads it stays unwritten)
  const int token_blocks = max_new <= ntaps - 1 ? 0 : (tokens + kConvTokens - 1) / kConvTokens;
  a.token_blocks = token_blocks;
  // few tokens: every pass a workgroup of its own; many: a workgroup takes several passes on one set of angles
  int per_block = 1;
  while (per_block < passes && static_cast<long long>(token_blocks + sequences) * (passes / (per_block * 2)) >= 2048) per_block *= 2;
  const int across = (passes + per_block - 1) / per_block;
  if (across > 65535) return kBadArgument;
  const dim3 grid(token_blocks + sequences, across);
  const size_t lds = (static_cast<size_t>(kConvTokens) * rot_dim + 4 * kConvMaxHead) * sizeof(float);
  hipStream_t s = (hipStream_t)stream;
#define TLIE_LAUNCH(D, W, O, V, NT) \
  hipLaunchKernelGGL((short_conv_kernel<D, W, O, V, NT>), grid, dim3(256), lds, s, a, per_block * per_pass, lane_bits)
#define TLIE_CASE(DC, D, WC, W, OC, O)                                                       \
  if (in_dtype == DC && w_dtype == WC && out_dtype == OC) {                                  \
    if (by_four) {                                                                           \
      if (ntaps <= 4) TLIE_LAUNCH(D, W, O, 4, 4);                                            \
      else TLIE_LAUNCH(D, W, O, 4, 8);                                                       \
    } else {                                                                                 \
      if (ntaps <= 4) TLIE_LAUNCH(D, W, O, 1, 4);                                            \
      else TLIE_LAUNCH(D, W, O, 1, 8);                                                       \
    }                                                                                        \
    return launch_status();                                                                  \
  }
  TLIE_CASE(kF32, float, kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kF32, float)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kBF16, bf16)
#undef TLIE_CASE
#undef TLIE_LAUNCH
  return kBadArgument;
}
