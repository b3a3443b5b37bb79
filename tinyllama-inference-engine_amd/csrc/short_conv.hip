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

constexpr int kConvTokens = 8, kConvMaxHead = 256, kConvMaxTaps = 8;       // tokens of a workgroup in a step that brings a sequence several

struct ConvSegment {
  int first;               // its first channel
  int channels;
  int head;                // channels of a head (at most kConvMaxHead)
  int norm;                // 0: none; 1: divided by the length; 2: by the root mean square, times weight
  const float* weight;     // [head], or null: 1
  float eps;               // inside the root
  float scale;
  int rotated;             // turned by the position
  int target;              // 0: out, columns out_col ..; 1: key rows; 2: value rows; 3: out, head by head (see ConvArgs)
  int out_col;
  int heads;               // how many (set by the entry point; 0: the segment is not there)
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
  ConvSegment segment[3];
  const int* positions;
  const float* inv_freq;   // [rot_dim / 2] or null
  int rot_dim;
  void* out;               // [tokens][out_row]; or (target 3) the channels' heads as planes [plane_rows][head] one after the other
  int out_row;
  int plane_rows;          // of the planes (target 3): at least the tokens
  void* cache;             // [pages][keys: nkv planes [row][d], values: nkv planes [dv][row]]
  const int* slot_map;
  int nkv, d, dv, page_size;
  int token_blocks;        // workgroups (in x) that take kConvTokens tokens each (set by the entry point)
  int normed;              // whether any segment has a norm (set by the entry point)
};

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;
typedef __attribute__((__vector_size__(2 * sizeof(uint32_t)))) uint32_t uintx2;
__device__ __forceinline__ floatx4 as_floatx4(const float4& v) { return floatx4{v.x, v.y, v.z, v.w}; }

// Four inputs as they come (bfloat16 stays packed until it is used), and as floats.
template <typename D> struct ConvFour;
template <> struct ConvFour<float> { typedef floatx4 type; };
template <> struct ConvFour<bf16> { typedef uintx2 type; };
__device__ __forceinline__ floatx4 four_floats(const floatx4& v) { return v; }
__device__ __forceinline__ floatx4 four_floats(const uintx2& v) { return floatx4{bf16_lo(v[0]), bf16_hi(v[0]), bf16_lo(v[1]), bf16_hi(v[1])}; }

// A lane's segment: the one that unit `head` (counted over all segments' heads) falls into; `head` becomes the head's
// number in it.
struct ConvPlace {
  bool live;
  int first, channels, head, norm, rotated, target, out_col;
  const float* weight;
  float eps, scale;
};
__device__ __forceinline__ ConvPlace place_of(const ConvArgs& a, int& head) {
  int which = 0;
  if (head >= a.segment[0].heads) {
    head -= a.segment[0].heads;
    which = 1;
    if (head >= a.segment[1].heads) {
      head -= a.segment[1].heads;
      which = 2;
    }
  }
  auto pick = [&](auto first, auto second, auto third) { return which == 0 ? first : (which == 1 ? second : third); };
  const ConvSegment &p = a.segment[0], &q = a.segment[1], &r = a.segment[2];
  ConvPlace seg;
  seg.live = head < pick(p.heads, q.heads, r.heads);
  seg.first = pick(p.first, q.first, r.first), seg.channels = pick(p.channels, q.channels, r.channels);
  seg.head = pick(p.head, q.head, r.head), seg.norm = pick(p.norm, q.norm, r.norm), seg.rotated = pick(p.rotated, q.rotated, r.rotated);
  seg.target = pick(p.target, q.target, r.target), seg.out_col = pick(p.out_col, q.out_col, r.out_col);
  seg.weight = pick(p.weight, q.weight, r.weight), seg.eps = pick(p.eps, q.eps, r.eps), seg.scale = pick(p.scale, q.scale, r.scale);
  return seg;
}

// Where the head's channel 0 of token t goes, and how far apart its channels lie there; null: nowhere.
template <typename O>
__device__ __forceinline__ O* destination(const ConvArgs& a, const ConvPlace& seg, int head, int t, bool pad, int& step) {
  step = 1;
  O* out = static_cast<O*>(a.out);
  if (seg.target == 0) return out + static_cast<size_t>(t) * a.out_row + seg.out_col + head * seg.head;
  if (seg.target == 3)
    return out + static_cast<size_t>(seg.out_col + head * seg.head) * a.plane_rows + static_cast<size_t>(t) * seg.head;
  const int place = a.slot_map[t];
  if (place < 0 || pad) return nullptr;
  O* page = static_cast<O*>(a.cache) + static_cast<size_t>(place / a.page_size) * a.page_size * a.nkv * (a.d + a.dv);
  const int r = place % a.page_size;
  if (seg.target == 1) return page + (static_cast<size_t>(head) * a.page_size + r) * a.d;
  step = a.page_size;
  return page + static_cast<size_t>(a.nkv) * a.page_size * a.d + static_cast<size_t>(head) * a.dv * a.page_size + r;
}

__device__ __forceinline__ void wave_fence() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// Any sizes.  A lane's channels lie a wave's lanes apart, up to four of them.
template <typename D, typename W, typename O>
__global__ void __launch_bounds__(256)
short_conv_kernel(const ConvArgs a, int lane_bits) {
  constexpr int N = kConvMaxHead / 64, NT = kConvMaxTaps;
  extern __shared__ float lds[];
  const int half = a.rot_dim / 2;
  float* cosines = lds;                                // [kConvTokens][half]
  float* sines = cosines + kConvTokens * half;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* turn = sines + kConvTokens * half + wave * kConvMaxHead;       // this wave's head(s), for the rotation's partners
  const int back = a.ntaps - 1;
  const bool by_token = static_cast<int>(blockIdx.x) < a.token_blocks;
  int t0, t1, first = 0, count = 0, slot = -1;
  if (by_token) {
    t0 = blockIdx.x * kConvTokens;
    t1 = min(a.tokens, t0 + kConvTokens);
  } else {
    const int seq = blockIdx.x - a.token_blocks;
    slot = a.seq_slot[seq];
    first = a.seq_start[seq];
    count = a.seq_start[seq + 1] - first;
    if (slot < 0 || count <= 0) return;
    t0 = first;
    t1 = first + min(count, back);                     // (fewer than kConvTokens)
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
  turn += (lane >> lane_bits) * lanes;
  int head = (blockIdx.y * 4 + wave) * per_wave + (lane >> lane_bits);
  const ConvPlace seg = place_of(a, head);
  int inside[N];                                       // this lane's channels inside the head; -1: none
  float w[N][NT], x[N][NT], bias[N], norm_weight[N];
#pragma unroll
  for (int e = 0; e < N; ++e) {
    const int c = sub + e * lanes;
    inside[e] = seg.live && c < seg.head && head * seg.head + c < seg.channels ? c : -1;
    const int channel = seg.first + head * seg.head + c;
    bias[e] = inside[e] >= 0 && a.bias != nullptr ? to_float(static_cast<const W*>(a.bias)[channel]) : 0.f;
    norm_weight[e] = inside[e] >= 0 && seg.weight != nullptr ? seg.weight[c] : 1.f;
#pragma unroll
    for (int j = 0; j < NT; ++j) {                     // w[e][j] weighs the input j tokens back
      w[e][j] = inside[e] >= 0 && j < a.ntaps ? to_float(taps[static_cast<size_t>(channel) * a.ntaps + back - j]) : 0.f;
      x[e][j] = 0.f;
    }
  }
  auto fetch = [&](int t, int e) {
    const int channel = seg.first + head * seg.head + inside[e];
    return sum_splits(in + static_cast<size_t>(t) * a.row + a.col + channel, a.nsplit, a.split_stride);
  };
  auto shift = [&](int t) {                            // the input of token t joins the windows
#pragma unroll
    for (int e = 0; e < N; ++e) {
#pragma unroll
      for (int j = NT - 1; j > 0; --j) x[e][j] = x[e][j - 1];
      x[e][0] = inside[e] >= 0 && t >= 0 ? fetch(t, e) : 0.f;
    }
  };
  if (by_token) {
    for (int j = back; j > 0; --j) shift(t0 - j);
  } else {
#pragma unroll
    for (int e = 0; e < N; ++e)
#pragma unroll
      for (int j = 0; j < NT; ++j)
        if (j < back && inside[e] >= 0)
          x[e][j] = held[static_cast<size_t>(back - 1 - j) * a.channels + seg.first + head * seg.head + inside[e]];
  }
  for (int t = t0; t < t1; ++t) {
    shift(t);
    bool pad = false;
    if (by_token) {
      pad = a.token_slot[t] < 0;
      if (!pad && t - a.seq_start[a.token_seq[t]] < back) continue;          // (its sequence's workgroup takes it)
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
    if (a.inv_freq != nullptr) {                       // (the same for the whole launch)
      wave_fence();                                    // the token before has been read
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
    int step;
    O* to = destination<O>(a, seg, head, t, pad, step);
    if (to == nullptr) continue;
#pragma unroll
    for (int e = 0; e < N; ++e)
      if (inside[e] >= 0) to[static_cast<size_t>(inside[e]) * step] = from_float<O>(y[e]);
  }
  if (by_token) return;
  // the state's new rows: the last `back` inputs.  A sequence that brought fewer tokens has them in its windows.
#pragma unroll
  for (int e = 0; e < N; ++e) {
    if (inside[e] < 0) continue;
    const int channel = seg.first + head * seg.head + inside[e];
#pragma unroll
    for (int j = 0; j < NT; ++j)
      if (j < back) held[static_cast<size_t>(back - 1 - j) * a.channels + channel] = count > back ? fetch(first + count - 1 - j, e) : x[e][j];
  }
}

// Four taps, and channels that a lane takes four by four: every segment's heads and channels, the product's columns and
// the arrays' rows are multiples of four, and a head's rotated halves too.  The loads are straight-line code without
// conditions (what is not there is read from a place that is, and not used), so that all of a wave's are on their way
// together.  TOKENS: the launch has workgroups that take kConvTokens tokens each; without, only sequences' workgroups.
template <typename D, typename W, typename O, bool TOKENS>
__global__ void __launch_bounds__(256, TOKENS && sizeof(O) == 2 ? 3 : 4)
short_conv_wide_kernel(const ConvArgs a, int lane_bits) {
  constexpr int BACK = 3;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int half = a.rot_dim / 2;
  float* cosines = lds;                                // [tokens][half]
  float* sines = cosines + kConvTokens * half;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const bool by_token = TOKENS && static_cast<int>(blockIdx.x) < a.token_blocks;
  int t0, t1, first = 0, count = 0, slot = 0;
  if (by_token) {
    t0 = blockIdx.x * kConvTokens;
    t1 = min(a.tokens, t0 + kConvTokens);
  } else {
    const int seq = blockIdx.x - a.token_blocks;
    slot = a.seq_slot[seq];
    first = a.seq_start[seq];
    count = a.seq_start[seq + 1] - first;
    if (slot < 0 || count <= 0) return;
    t0 = first;
    t1 = first + min(count, BACK);
  }
  const int lanes = 1 << lane_bits, per_wave = 64 >> lane_bits;
  int head = (blockIdx.y * 4 + wave) * per_wave + (lane >> lane_bits);
  const ConvPlace seg = place_of(a, head);
  const int c = (lane & (lanes - 1)) * 4;              // this lane's first channel inside the head
  const bool live = seg.live && c < seg.head;
  const int channel = live ? seg.first + head * seg.head + c : 0;
  const D* in = static_cast<const D*>(a.in) + a.col + channel;
  typedef typename ConvFour<D>::type Four;
  auto load = [&](int t) {                             // the inputs of token t
    const D* from = in + static_cast<size_t>(t) * a.row;
    Four v = *reinterpret_cast<const Four*>(from);
    if constexpr (sizeof(D) == 4)                      // (only floats come in parts)
      for (int p = 1; p < a.nsplit; ++p) v += *reinterpret_cast<const Four*>(from + p * a.split_stride);
    return v;
  };
  float weights[16];
  load8(static_cast<const W*>(a.taps) + static_cast<size_t>(channel) * 4, *reinterpret_cast<float(*)[8]>(weights));
  load8(static_cast<const W*>(a.taps) + static_cast<size_t>(channel) * 4 + 8, *reinterpret_cast<float(*)[8]>(weights + 8));
  floatx4 w[4];                                        // w[j] weighs the input j tokens back
#pragma unroll
  for (int j = 0; j < 4; ++j) w[j] = floatx4{weights[3 - j], weights[7 - j], weights[11 - j], weights[15 - j]};
  floatx4 bias = {0.f, 0.f, 0.f, 0.f}, norm_weight = {1.f, 1.f, 1.f, 1.f};
  if (a.bias != nullptr) bias = as_floatx4(load4(static_cast<const W*>(a.bias) + channel));
  if (a.normed && seg.weight != nullptr) norm_weight = *reinterpret_cast<const floatx4*>(seg.weight + (live ? c : 0));
  floatx4 window[BACK];                                // window[j]: the input j + 1 tokens back
  Four rows[TOKENS ? kConvTokens : 1];
  float* held = nullptr;
  if (by_token) {
#pragma unroll
    for (int j = 0; j < BACK; ++j) window[j] = four_floats(load(max(t0 - 1 - j, 0)));
#pragma unroll
    for (int b = 0; b < kConvTokens; ++b) rows[TOKENS ? b : 0] = load(min(t0 + b, t1 - 1));
  } else {
    held = a.state + static_cast<size_t>(slot) * a.slot_stride + channel;
#pragma unroll
    for (int j = 0; j < BACK; ++j) window[j] = *reinterpret_cast<const floatx4*>(held + static_cast<size_t>(BACK - 1 - j) * a.channels);
    rows[0] = load(t0);
  }
  // which of the tokens are this workgroup's, and which pad the step (a lane a token, then the same for the whole wave)
  unsigned mine = ~0u, padding = 0;
  if (by_token) {
    const int t = min(t0 + (lane & (kConvTokens - 1)), t1 - 1);
    const bool pad = a.token_slot[t] < 0;
    const bool later = t - a.seq_start[a.token_seq[t]] >= BACK;
    mine = static_cast<unsigned>(__ballot(pad || later)), padding = static_cast<unsigned>(__ballot(pad));
  }
  if (a.inv_freq != nullptr) {
    for (int i = threadIdx.x; i < (t1 - t0) * half; i += 256) {
      const int b = i / half;
      sincosf(static_cast<float>(a.positions[t0 + b]) * a.inv_freq[i - b * half], &sines[i], &cosines[i]);
    }
    __syncthreads();
  }
  const bool turned = a.inv_freq != nullptr && seg.rotated && c < a.rot_dim;
  const int angle = c < half ? c : c - half, partner = lane + (c < half ? half / 4 : -half / 4);
  // A page's value rows are written dim by dim: where the workgroup's tokens are the page's rows 8 n .. 8 n + 7, all at once.
  bool together = false;
  if (TOKENS && sizeof(O) == 2 && by_token && a.slot_map != nullptr && t1 - t0 == kConvTokens && (mine & 0xff) == 0xff && padding == 0) {
    const int place = a.slot_map[t0 + (lane & (kConvTokens - 1))], begin = __builtin_amdgcn_readfirstlane(place);
    together = begin >= 0 && begin % 8 == 0 && a.page_size % 8 == 0 && __all(place == begin + (lane & (kConvTokens - 1)));
  }
  float columns[TOKENS && sizeof(O) == 2 ? 4 : 1][kConvTokens];
  auto token = [&](int b, const floatx4& x) {          // token t0 + b, whose inputs are x
    const int t = t0 + b;
    const bool pad = (padding >> b) & 1;
    floatx4 y = bias + w[0] * x + w[1] * window[0] + w[2] * window[1] + w[3] * window[2];
    window[2] = window[1], window[1] = window[0], window[0] = x;
    if (!((mine >> b) & 1)) return;                    // (its sequence's workgroup takes it; the same for the whole workgroup)
    if (a.silu) {
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] = y[e] / (1.f + expf(-y[e]));
    }
    if (!live || pad) y = floatx4{0.f, 0.f, 0.f, 0.f};
    if (a.normed) {
      float scale = seg.scale, squares = y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3];
      for (int offset = lanes >> 1; offset > 0; offset >>= 1) squares += __shfl_xor(squares, offset, 64);
      if (seg.norm == 1) scale /= sqrtf(squares + seg.eps);
      else if (seg.norm == 2) scale /= sqrtf(squares / static_cast<float>(seg.head) + seg.eps);
      y *= scale * norm_weight;
    } else {
      y *= seg.scale;
    }
    if (a.inv_freq != nullptr) {
      floatx4 other;
#pragma unroll
      for (int e = 0; e < 4; ++e) other[e] = __shfl(y[e], partner, 64);
      if (turned) {
        const floatx4 cs = *reinterpret_cast<const floatx4*>(cosines + b * half + angle), sn = *reinterpret_cast<const floatx4*>(sines + b * half + angle);
        y = c < half ? y * cs - other * sn : y * cs + other * sn;
      }
    }
    if (together && seg.target == 2) {
#pragma unroll
      for (int e = 0; e < 4; ++e) columns[TOKENS && sizeof(O) == 2 ? e : 0][b] = y[e];
      return;
    }
    int step;
    O* to = destination<O>(a, seg, head, t, pad, step);
    if (to == nullptr || !live) return;
    if (step == 1) {
      store4(to + c, y[0], y[1], y[2], y[3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) to[static_cast<size_t>(c + e) * step] = from_float<O>(y[e]);
    }
  };
  if (by_token) {
#pragma unroll
    for (int b = 0; b < kConvTokens; ++b) {
      if (t0 + b >= t1) break;
      token(b, four_floats(rows[TOKENS ? b : 0]));
    }
    if (TOKENS && sizeof(O) == 2 && together && seg.target == 2 && live) {
      int step;
      O* to = destination<O>(a, seg, head, t0, false, step);
#pragma unroll
      for (int e = 0; e < 4; ++e) store8(to + static_cast<size_t>(c + e) * step, columns[TOKENS && sizeof(O) == 2 ? e : 0]);
    }
    return;
  }
  token(0, four_floats(rows[0]));
  for (int b = 1; b < t1 - t0; ++b) token(b, four_floats(load(t0 + b)));
  // the state's new rows: the last inputs.  A sequence that brought no more has them in its window.
  if (count > BACK) {
#pragma unroll
    for (int j = 0; j < BACK; ++j) window[j] = four_floats(load(first + count - 1 - j));
  }
  if (!live) return;
#pragma unroll
  for (int j = 0; j < BACK; ++j) *reinterpret_cast<floatx4*>(held + static_cast<size_t>(BACK - 1 - j) * a.channels) = window[j];
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
                               const float* inv_freq, int rot_dim, void* out, int out_row, int plane_rows, int out_dtype, void* cache,
                               const int* slot_map, int nkv, int d, int dv, int page_size, void* stream) {
  if (in_dtype == kBF16 && nsplit != 1) return kBadArgument;
  if (tokens <= 0 || sequences <= 0 || channels <= 0 || ntaps < 1 || ntaps > 8 || nsplit < 1 || count < 1 || count > 3) return kBadArgument;
  if (col < 0 || col + channels > row || (ntaps > 1 && (state == nullptr || slot_stride < static_cast<long long>(ntaps - 1) * channels))) return kBadArgument;
  if (rot_dim < 0 || rot_dim % 2 != 0 || rot_dim > kConvMaxHead || (inv_freq == nullptr && rot_dim != 0)) return kBadArgument;
  ConvArgs a{in, nsplit, (size_t)split_stride, row, col, taps, bias, state, (size_t)slot_stride, token_seq, token_slot, seq_start,
             seq_slot, tokens, sequences, channels, ntaps, silu, {}, positions, inv_freq, rot_dim, out, out_row, plane_rows, cache,
             slot_map, nkv, d, dv, page_size, 0, 0};
  const auto aligned = [](const void* p, unsigned bytes) { return (reinterpret_cast<uintptr_t>(p) & (bytes - 1)) == 0; };
  // (the wide form: what it needs besides is asked of the segments below)
  bool wide = ntaps == 4 && row % 4 == 0 && col % 4 == 0 && channels % 4 == 0 && slot_stride % 4 == 0 && rot_dim % 8 == 0 &&
              (nsplit == 1 || split_stride % 4 == 0) && aligned(in, 16) && aligned(out, 16) && aligned(cache, 16) && aligned(taps, 32) &&
              aligned(bias, 16) && aligned(state, 16);
  int widest = 0, heads = 0, at = 0;
  for (int s = 0; s < count; ++s) {
    const int* f = table + 7 * s;
    ConvSegment& seg = a.segment[s];
    seg = ConvSegment{f[0], f[1], f[2], f[3], static_cast<const float*>(weights[s]), eps[s], scales[s], f[4], f[5], f[6], 0};
    if (seg.first != at || seg.channels <= 0 || seg.head <= 0 || seg.head > kConvMaxHead || seg.norm < 0 || seg.norm > 2) return kBadArgument;
    if ((seg.norm != 0 || seg.rotated || seg.target != 0) && seg.channels % seg.head != 0) return kBadArgument;
    if (seg.norm != 0 && !(seg.eps > 0.f)) return kBadArgument;
    if (seg.rotated && (inv_freq == nullptr || rot_dim > seg.head || positions == nullptr)) return kBadArgument;
    if (seg.target < 0 || seg.target > 3) return kBadArgument;
    if (seg.target == 0 || seg.target == 3) {
      if (out == nullptr || seg.out_col < 0 || seg.out_col + seg.channels > out_row || (seg.target == 3 && plane_rows < tokens)) return kBadArgument;
    } else if (cache == nullptr || slot_map == nullptr || page_size <= 0 || nkv <= 0) {
      return kBadArgument;
    }
    if (seg.target == 1 && (seg.head != d || seg.channels != nkv * d)) return kBadArgument;
    if (seg.target == 2 && (seg.head != dv || seg.channels != nkv * dv)) return kBadArgument;
    wide = wide && seg.head % 4 == 0 && seg.channels % seg.head == 0 && aligned(seg.weight, 16) &&
           (seg.target == 1 || seg.target == 2 || (seg.out_col % 4 == 0 && (seg.target == 3 || out_row % 4 == 0))) &&
           (seg.target != 1 || (page_size * (d + dv) * nkv) % 4 == 0);
    if (seg.head > widest) widest = seg.head;
    if (seg.norm != 0) a.normed = 1;
    seg.heads = (seg.channels + seg.head - 1) / seg.head;
    heads += seg.heads;
    at += seg.channels;
  }
  if (at != channels) return kBadArgument;
  // (a step in which no sequence brings more tokens than its workgroup takes needs no others: what pads it stays unwritten)
  const bool tokens_too = max_new > ntaps - 1;
  if (tokens_too) a.token_blocks = (tokens + kConvTokens - 1) / kConvTokens;
  int lane_bits = 0;
  while (lane_bits < 6 && ((wide ? 4 : 1) << lane_bits) < widest) ++lane_bits;
  const int per_block = 4 * (64 >> lane_bits);         // heads the four waves take at once
  const int across = (heads + per_block - 1) / per_block;
  if (across > 65535) return kBadArgument;
  const dim3 grid(a.token_blocks + sequences, across);
  const size_t lds = (static_cast<size_t>(kConvTokens) * rot_dim + (wide ? 0 : 4 * kConvMaxHead)) * sizeof(float);
  hipStream_t s = (hipStream_t)stream;
#define TLIE_CASE(DC, D, WC, W, OC, O)                                                                                       \
  if (in_dtype == DC && w_dtype == WC && out_dtype == OC) {                                                                  \
    if (!wide) hipLaunchKernelGGL((short_conv_kernel<D, W, O>), grid, dim3(256), lds, s, a, lane_bits);                      \
    else if (tokens_too) hipLaunchKernelGGL((short_conv_wide_kernel<D, W, O, true>), grid, dim3(256), lds, s, a, lane_bits); \
    else hipLaunchKernelGGL((short_conv_wide_kernel<D, W, O, false>), grid, dim3(256), lds, s, a, lane_bits);                \
    return launch_status();                                                                                                  \
  }
  TLIE_CASE(kF32, float, kF32, float, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16, kF32, float)
  TLIE_CASE(kF32, float, kBF16, bf16, kBF16, bf16)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kF32, float)
  TLIE_CASE(kBF16, bf16, kBF16, bf16, kBF16, bf16)
#undef TLIE_CASE
  return kBadArgument;
}
