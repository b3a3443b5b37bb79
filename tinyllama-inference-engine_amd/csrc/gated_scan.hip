// Mixers with a matrix state per head that decays by one number a token and head, token by token.  Per head, with a query
// q and a key k (dim values each, shared by the heads of a group), a value v (vdim values), S (dim x vdim):
//   additive      S' = g S + w k v^T,                      o = S'^T q + D v
//   delta rule    S' = g S + k u^T, u = w (v - g S^T k),   o = S'^T q
// The gates come from columns of a product and three numbers a head (rate A, bias, skip D), float whatever the type:
//   additive      w = softplus(z_a + bias),  g = exp(-exp(A) w)
//   delta rule    w = sigmoid(z_b),          g = exp(-exp(A) softplus(z_a + bias))
// S is the request's state (zero when it is admitted) and is carried from step to step; everything is float.
//
// A sequence that brings few tokens of the step is walked token by token: a workgroup owns 64 columns of one head's S,
// each thread four columns of every 16th dim, and since S'^T q = g S^T q + (k . q) u, the sums a token needs run over the
// state as it was: they meet once a token.
//
// A sequence that brings many is taken in chunks of 32 tokens.  With c_i the running sum of log g inside a chunk and S the
// state before it:
//   O = diag(e^c) Q S + P U,   S <- e^(c_last) S + (diag(e^(c_last - c)) K)^T U,    P_ij = e^(c_i - c_j) q_i . k_j  (j <= i)
//   additive      U = diag(w) V
//   delta rule    (I + M) U = diag(w) (V - diag(e^c) K S),   M_ij = w_i e^(c_i - c_j) k_i . k_j  (j < i)
// A first kernel makes every chunk's P and, for the delta rule, T = (I + M)^-1 diag(w), which depend on no state (the
// chunks of a step side by side); a second one walks a sequence's chunks with the state in registers, a workgroup for 16
// or 32 columns of a head.  All products are the matrix cores' 32-bit ones (v_mfma_f32_16x16x4_f32: operands, products
// and sums float).
//
// Sequences whose request slot is negative pad a recorded step: nothing is read or written for them.
#include "common.h"

namespace tlie {

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float floatx4;

constexpr int kChunk = 32, kChunkedFrom = 24, kGatedBatch = 4, kGatedMaxDim = 256;
constexpr int kPartFloats = 2 * kChunk * kChunk + 2 * kChunk;        // of a chunk of a head: P, T, e^c, and what a key counts at the chunk's end

struct GatedArgs {
  const float* in;             // q, k and v, head by head: the head with the channels c .. c + w - 1 is the plane [plane_rows][w] at c * plane_rows
  int q_first, k_first, v_first;       // the first channels of q and k (heads of dim) and of v (planes of v_width)
  int v_width, plane_rows;
  const void* gates;           // [nsplit][tokens][gate_row] of the product's type
  int nsplit;
  size_t split_stride;
  int gate_row, a_col, b_col;
  const float* rate;           // [heads]
  const float* bias;           // [heads]
  const float* skip;           // [heads] or null (additive only)
  float* state;                // [slots][heads][tiles][dim][64], a slot's row slot_stride after the one before
  size_t slot_stride;
  float* parts;                // [sequences][chunks][heads][kPartFloats]
  const int* seq_start;
  const int* seq_slot;
  float* out;                  // [tokens][heads * vdim]
  int heads, groups, dim, vdim, tiles, chunks, chunked, sequences;
};

__device__ __forceinline__ float softplus32(float v) { return v > 20.f ? v : log1pf(expf(v)); }

// Group g's queries or keys ([plane_rows][dim]), and the column of head h's values ([plane_rows][v_width]).
__device__ __forceinline__ const float* head_plane(const GatedArgs& a, int first, int g) {
  return a.in + (static_cast<size_t>(first) + static_cast<size_t>(g) * a.dim) * a.plane_rows;
}
__device__ __forceinline__ const float* value_column(const GatedArgs& a, int h, int col) {
  const int c = h * a.vdim + col, plane = c / a.v_width;
  return a.in + (static_cast<size_t>(a.v_first) + static_cast<size_t>(plane) * a.v_width) * a.plane_rows + (c - plane * a.v_width);
}

// A token's and head's gates: log g, and w.
template <typename D, bool DELTA>
__device__ __forceinline__ void gates_of(const GatedArgs& a, size_t t, int h, float& log_g, float& w) {
  const D* row = static_cast<const D*>(a.gates) + t * a.gate_row;
  const float step = softplus32(sum_splits(row + a.a_col + h, a.nsplit, a.split_stride) + a.bias[h]);
  log_g = -expf(a.rate[h]) * step;
  w = DELTA ? 1.f / (1.f + expf(-sum_splits(row + a.b_col + h, a.nsplit, a.split_stride))) : step;
}

// Few tokens: DI dims a thread (dim <= 16 * DI).
template <typename D, bool DELTA, int DI>
__global__ void __launch_bounds__(256)
gated_walk_kernel(const GatedArgs a) {
  constexpr int DMAX = 16 * DI;
  __shared__ __attribute__((aligned(16))) float qs[kGatedBatch][DMAX];
  __shared__ __attribute__((aligned(16))) float ks[kGatedBatch][DMAX];
  __shared__ __attribute__((aligned(16))) float vs[kGatedBatch][64];
  __shared__ float gs[kGatedBatch], ws[kGatedBatch], kq[kGatedBatch];
  __shared__ __attribute__((aligned(16))) float met[2][4][2][64];      // (a buffer in turn) a wave's part of S^T k and S^T q
  const int seq = blockIdx.x, h = blockIdx.y, tile = blockIdx.z;
  const int slot = a.seq_slot[seq];
  if (slot < 0) return;
  const int first = a.seq_start[seq], count = a.seq_start[seq + 1] - first;
  if (count <= 0 || (a.chunked && count >= kChunkedFrom)) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = (threadIdx.x & 15) * 4, part = threadIdx.x >> 4;     // four columns of the tile; dims part, part + 16, ...
  const int group = h / (a.heads / a.groups), base = tile * 64;
  float* st = a.state + static_cast<size_t>(slot) * a.slot_stride + (static_cast<size_t>(h) * a.tiles + tile) * a.dim * 64;
  float4 S[DI];
#pragma unroll
  for (int i = 0; i < DI; ++i) {
    const int d = part + 16 * i;
    S[i] = d < a.dim ? *reinterpret_cast<const float4*>(st + d * 64 + col) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const float skip = !DELTA && a.skip != nullptr ? a.skip[h] : 0.f;
  const float* queries = head_plane(a, a.q_first, group);
  const float* keys = head_plane(a, a.k_first, group);
  const float* values = value_column(a, h, min(base + lane, a.vdim - 1));
  int turn = 0;
  for (int t0 = 0; t0 < count; t0 += kGatedBatch) {
    const int nb = min(kGatedBatch, count - t0);
    __syncthreads();                                   // the batch before has been read
    for (int i = threadIdx.x; i < nb * DMAX; i += 256) {
      const int b = i / DMAX, d = i - b * DMAX;
      const size_t at = static_cast<size_t>(first + t0 + b) * a.dim + d;
      qs[b][d] = d < a.dim ? queries[at] : 0.f;
      ks[b][d] = d < a.dim ? keys[at] : 0.f;
    }
    {
      const int b = threadIdx.x >> 6;
      if (b < nb) vs[b][lane] = base + lane < a.vdim ? values[static_cast<size_t>(first + t0 + b) * a.v_width] : 0.f;
      if (b < nb && lane == 0) {
        float log_g, w;
        gates_of<D, DELTA>(a, static_cast<size_t>(first + t0 + b), h, log_g, w);
        gs[b] = expf(log_g), ws[b] = w;
      }
    }
    __syncthreads();
    if (wave < nb) {                                   // k . q of token `wave` of the batch
      float sum = 0.f;
#pragma unroll
      for (int d = 0; d < DMAX; d += 64)
        if (d + lane < DMAX) sum += ks[wave][d + lane] * qs[wave][d + lane];
      sum = wave_sum(sum);
      if (lane == 0) kq[wave] = sum;
    }
    for (int b = 0; b < nb; ++b) {
      float4 pk = make_float4(0.f, 0.f, 0.f, 0.f), pq = pk;
#pragma unroll
      for (int i = 0; i < DI; ++i) {
        const float q = qs[b][part + 16 * i];
        pq.x += S[i].x * q, pq.y += S[i].y * q, pq.z += S[i].z * q, pq.w += S[i].w * q;
        if (DELTA) {
          const float k = ks[b][part + 16 * i];
          pk.x += S[i].x * k, pk.y += S[i].y * k, pk.z += S[i].z * k, pk.w += S[i].w * k;
        }
      }
#pragma unroll
      for (int offset = 16; offset < 64; offset <<= 1) {
        pq.x += __shfl_xor(pq.x, offset, 64), pq.y += __shfl_xor(pq.y, offset, 64);
        pq.z += __shfl_xor(pq.z, offset, 64), pq.w += __shfl_xor(pq.w, offset, 64);
        if (DELTA) {
          pk.x += __shfl_xor(pk.x, offset, 64), pk.y += __shfl_xor(pk.y, offset, 64);
          pk.z += __shfl_xor(pk.z, offset, 64), pk.w += __shfl_xor(pk.w, offset, 64);
        }
      }
      if (lane < 16) {
        *reinterpret_cast<float4*>(&met[turn][wave][1][col]) = pq;
        if (DELTA) *reinterpret_cast<float4*>(&met[turn][wave][0][col]) = pk;
      }
      __syncthreads();                                 // (the other buffer is written next: one barrier a token)
      float4 sq = *reinterpret_cast<const float4*>(&met[turn][0][1][col]), sk = make_float4(0.f, 0.f, 0.f, 0.f);
      if (DELTA) sk = *reinterpret_cast<const float4*>(&met[turn][0][0][col]);
#pragma unroll
      for (int w = 1; w < 4; ++w) {
        const float4 m = *reinterpret_cast<const float4*>(&met[turn][w][1][col]);
        sq.x += m.x, sq.y += m.y, sq.z += m.z, sq.w += m.w;
        if (DELTA) {
          const float4 n = *reinterpret_cast<const float4*>(&met[turn][w][0][col]);
          sk.x += n.x, sk.y += n.y, sk.z += n.z, sk.w += n.w;
        }
      }
      turn ^= 1;
      const float g = gs[b], w = ws[b], dot = kq[b];
      const float4 v = *reinterpret_cast<const float4*>(&vs[b][col]);
      float4 u;
      if (DELTA) u = make_float4(w * (v.x - g * sk.x), w * (v.y - g * sk.y), w * (v.z - g * sk.z), w * (v.w - g * sk.w));
      else u = make_float4(w * v.x, w * v.y, w * v.z, w * v.w);
#pragma unroll
      for (int i = 0; i < DI; ++i) {
        const float k = ks[b][part + 16 * i];
        S[i].x = g * S[i].x + k * u.x, S[i].y = g * S[i].y + k * u.y;
        S[i].z = g * S[i].z + k * u.z, S[i].w = g * S[i].w + k * u.w;
      }
      if (part == 0) {
        const float o[4] = {g * sq.x + dot * u.x + skip * v.x, g * sq.y + dot * u.y + skip * v.y,
                            g * sq.z + dot * u.z + skip * v.z, g * sq.w + dot * u.w + skip * v.w};
        float* to = a.out + (static_cast<size_t>(first + t0 + b) * a.heads + h) * a.vdim + base + col;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (base + col + j < a.vdim) to[j] = o[j];
      }
    }
  }
#pragma unroll
  for (int i = 0; i < DI; ++i) {
    const int d = part + 16 * i;
    if (d < a.dim) *reinterpret_cast<float4*>(st + d * 64 + col) = S[i];
  }
}

// acc += A B on floats, A 16 x 4 (a lane: row lane % 16, column lane / 16), B 4 x 16 (row lane / 16, column lane % 16);
// acc[r]: row 4 * (lane / 16) + r, column lane % 16.
__device__ __forceinline__ floatx4 mfma_f32(float a, float b, floatx4 acc) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, acc, 0, 0, 0);
}

// Four steps of that at once: a lane brings four consecutive inner indices of its row of A and of its column of B (16 bytes
// each from LDS), so that the sixteen inner indices of the lanes' four groups are met in another order, the same for both.
__device__ __forceinline__ floatx4 mfma_f32_by16(const float4& a, const float4& b, floatx4 acc) {
  acc = mfma_f32(a.x, b.x, acc);
  acc = mfma_f32(a.y, b.y, acc);
  acc = mfma_f32(a.z, b.z, acc);
  return mfma_f32(a.w, b.w, acc);
}
__device__ __forceinline__ float4 lds4(const float* p) { return *reinterpret_cast<const float4*>(p); }

// Four columns d .. d + 3 of a token's row (those from dim on are zeros).
__device__ __forceinline__ float4 row4(const float* from, int d, int dim, bool by_four) {
  if (by_four) return *reinterpret_cast<const float4*>(from + d);
  float4 v = make_float4(from[d], 0.f, 0.f, 0.f);
  if (d + 1 < dim) v.y = from[d + 1];
  if (d + 2 < dim) v.z = from[d + 2];
  if (d + 3 < dim) v.w = from[d + 3];
  return v;
}

// A workgroup of four waves a (chunk of a sequence, group of heads): the products K K^T and Q K^T of the chunk's 32 tokens
// are made once for the group, then wave by wave the heads' own P and T.  blockIdx.z: a share of the group's heads.
constexpr int kSquareRow = kChunk + 4;                 // a row of a 32 x 32 array in LDS

template <typename D, bool DELTA>
__global__ void __launch_bounds__(256)
gated_chunk_kernel(const GatedArgs a, int dim_padded) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int row = dim_padded + 4;                      // (dim_padded: a multiple of 16)
  float* K = lds;                                      // [32][row]
  float* Q = K + kChunk * row;
  float* QK = Q + kChunk * row;                        // [32][kSquareRow]
  float* KK = QK + kChunk * kSquareRow;
  float* work = KK + (DELTA ? kChunk * kSquareRow : 0);       // a wave's: c [32] (doubles), w [32], and (delta) M [32][kSquareRow]
  const int seq = blockIdx.x / a.chunks, chunk = blockIdx.x % a.chunks, group = blockIdx.y;
  const int slot = a.seq_slot[seq];
  if (slot < 0) return;
  const int first = a.seq_start[seq], count = a.seq_start[seq + 1] - first;
  const int begin = chunk * kChunk, n = min(kChunk, count - begin);
  if (count < kChunkedFrom || n <= 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  {
    // a thread: every eighth token's columns 4 * (thread % 32), and on by 128
    const bool by_four = (a.dim & 3) == 0 && (a.k_first & 3) == 0 && (a.q_first & 3) == 0;
    const float* keys = head_plane(a, a.k_first, group) + static_cast<size_t>(first + begin) * a.dim;
    const float* queries = head_plane(a, a.q_first, group) + static_cast<size_t>(first + begin) * a.dim;
    const int r0 = threadIdx.x >> 5;
    for (int d = (threadIdx.x & 31) * 4; d < dim_padded; d += 128) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = r0 + 8 * i;
        float4 k = make_float4(0.f, 0.f, 0.f, 0.f), q = k;
        if (r < n && d < a.dim) {
          k = row4(keys + r * a.dim, d, a.dim, by_four);
          q = row4(queries + r * a.dim, d, a.dim, by_four);
        }
        *reinterpret_cast<float4*>(K + r * row + d) = k;
        *reinterpret_cast<float4*>(Q + r * row + d) = q;
      }
    }
  }
  __syncthreads();
  {
    // wave w: rows (w / 2), columns (w % 2) of the 2 x 2 tiles; above the diagonal nobody reads
    const int ti = wave >> 1, tj = wave & 1;
    if (ti >= tj) {
      floatx4 qk = {0.f, 0.f, 0.f, 0.f}, kk = qk;
      const float* ai = Q + (ti * 16 + (lane & 15)) * row + (lane >> 4) * 4;
      const float* ki = K + (ti * 16 + (lane & 15)) * row + (lane >> 4) * 4;
      const float* bj = K + (tj * 16 + (lane & 15)) * row + (lane >> 4) * 4;
#pragma unroll 4
      for (int d = 0; d < dim_padded; d += 16) {
        const float4 b = lds4(bj + d);
        qk = mfma_f32_by16(lds4(ai + d), b, qk);
        if (DELTA) kk = mfma_f32_by16(lds4(ki + d), b, kk);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int at = (ti * 16 + (lane >> 4) * 4 + r) * kSquareRow + tj * 16 + (lane & 15);
        QK[at] = qk[r];
        if (DELTA) KK[at] = kk[r];
      }
    }
  }
  __syncthreads();
  const int ratio = a.heads / a.groups;
  double* c = reinterpret_cast<double*>(work + wave * (3 * kChunk + (DELTA ? kChunk * kSquareRow : 0)));
  float* w = reinterpret_cast<float*>(c + kChunk);
  float* M = w + kChunk;
  // (every wave makes as many rounds: the barriers below are met by all)
  for (int h0 = blockIdx.z * 4; h0 < ratio; h0 += gridDim.z * 4) {
    const bool live = h0 + wave < ratio;
    const int h = group * ratio + min(h0 + wave, ratio - 1);
    float* part = a.parts + ((static_cast<size_t>(seq) * a.chunks + chunk) * a.heads + h) * kPartFloats;
    float log_g = 0.f, strength = 0.f;
    if (lane < n) gates_of<D, DELTA>(a, static_cast<size_t>(first + begin + lane), h, log_g, strength);
    // the running sum over the chunk's tokens (lanes 0 .. 31): in double, since what is used of it are differences, and
    // a token that forgets nearly everything must not cost the tokens after it their digits
    double run = log_g;
#pragma unroll
    for (int offset = 1; offset < kChunk; offset <<= 1) {
      const double other = __shfl_up(run, offset, 64);
      if (lane >= offset) run += other;
    }
    const double whole = __shfl(run, kChunk - 1, 64);
    if (lane < kChunk) c[lane] = run, w[lane] = strength;
    __syncthreads();
    if (live) {
      if (lane < kChunk) {
        part[2 * kChunk * kChunk + lane] = expf(static_cast<float>(run));
        part[2 * kChunk * kChunk + kChunk + lane] = expf(static_cast<float>(whole - run)) * (DELTA ? 1.f : strength);
      }
#pragma unroll
      for (int turn = 0; turn < kChunk * kChunk / 256; ++turn) {
        const int i = lane * 4 + turn * 256, r = i >> 5, j0 = i & 31;
        float p[4], m[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int j = j0 + e;
          const float keeps = j <= r ? expf(static_cast<float>(c[r] - c[j])) : 0.f;
          p[e] = j <= r ? QK[r * kSquareRow + j] * keeps * (DELTA ? 1.f : w[j]) : 0.f;
          m[e] = DELTA && j < r ? w[r] * keeps * KK[r * kSquareRow + j] : 0.f;
        }
        *reinterpret_cast<float4*>(part + i) = make_float4(p[0], p[1], p[2], p[3]);
        if (DELTA) *reinterpret_cast<float4*>(M + r * kSquareRow + j0) = make_float4(m[0], m[1], m[2], m[3]);
      }
    }
    __syncthreads();                                   // M is written (additive: c and w have been read)
    if (!DELTA) continue;
    if (live && lane < kChunk) {
      // lane j: column j of (I + M)^-1, row by row, times the column's w
      float x[kChunk];
#pragma unroll
      for (int i = 0; i < kChunk; ++i) {
        float s0 = i == lane ? 1.f : 0.f, s1 = 0.f, s2 = 0.f, s3 = 0.f;
#pragma unroll
        for (int k = 0; k < i; k += 4) {               // (M is zero from the diagonal on; x beyond i is not read)
          const float4 m = lds4(M + i * kSquareRow + k);
          s0 -= m.x * x[k];
          if (k + 1 < i) s1 -= m.y * x[k + 1];
          if (k + 2 < i) s2 -= m.z * x[k + 2];
          if (k + 3 < i) s3 -= m.w * x[k + 3];
        }
        x[i] = (s0 + s1) + (s2 + s3);
      }
      const float mine = w[lane];
#pragma unroll
      for (int i = 0; i < kChunk; ++i) part[kChunk * kChunk + i * kChunk + lane] = x[i] * mine;
    }
    __syncthreads();                                   // c, w and M have been read
  }
}

// A sequence's chunks one after the other: a workgroup of eight waves for NC tiles of 16 columns of a head's S.  Wave w keeps
// the 16-dim tiles w, w + 8, ... of S (TPW of them) in registers; all of S, the values and what becomes of them lie in LDS
// column by column, so that the matrix cores' operands are 16-byte reads there.
// The products with S are shared out over the waves by 16 tokens and a stretch of dims (delta rule: waves 0 .. 3 those of K,
// 4 .. 7 those of Q, two stretches; additive: all those of Q, four stretches), and their parts meet in LDS.  Waves 0 and 1
// then make U of 16 tokens each (delta), waves 6 and 7 the results.
// BY4: the dims are a multiple of 4, and keys and queries lie at multiples of 16 bytes.
template <bool DELTA, int TPW, int NC, bool BY4>
__global__ void __launch_bounds__(512)
gated_chain_kernel(const GatedArgs a) {
  constexpr int DP = TPW * 128, ROW = DP + 4, COLS = NC * 16, TROW = kSquareRow, PARTS = DELTA ? 2 : 4, LENGTH = DP / PARTS;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* K = lds;                                      // [32][ROW]
  float* Q = K + kChunk * ROW;                         // [32][ROW]
  float* S = Q + kChunk * ROW;                         // [COLS][ROW]
  float* P = S + COLS * ROW;                           // [32][TROW]
  float* V = P + kChunk * TROW;                        // [COLS][TROW]
  float* UW = V + COLS * TROW;                         // [COLS][TROW]: what joins the state, as much as it counts at the chunk's end
  float* QS = UW + COLS * TROW;                        // [PARTS - 1][COLS][TROW]: the other parts of Q S
  float* E = QS + (PARTS - 1) * COLS * TROW;           // e^c [32], then what a key counts at the chunk's end [32]
  float* T = E + 2 * kChunk;                           // delta: [32][TROW]
  float* KS = T + kChunk * TROW;                       // delta: [2][COLS][TROW]: the parts of K S
  float* U = KS + 2 * COLS * TROW;                     // delta: [COLS][TROW]
  // Workgroups of one head read the same keys and queries chunk by chunk: they are dealt to the same die (every eighth
  // workgroup goes to one), whose L2 then brings them once.
  const int column_tiles = (a.vdim + COLS - 1) / COLS, place = blockIdx.x >> 3;
  const int unit = (place / column_tiles) * 8 + (blockIdx.x & 7), col0 = place % column_tiles * COLS;
  if (unit >= a.sequences * a.heads) return;
  const int seq = unit / a.heads, h = unit - seq * a.heads;
  const int slot = a.seq_slot[seq];
  if (slot < 0) return;
  const int first = a.seq_start[seq], count = a.seq_start[seq + 1] - first;
  if (count < kChunkedFrom) return;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), low = lane & 15, high = lane >> 4;
  const int group = h / (a.heads / a.groups);
  const int half = wave & 1;                           // which 16 of the chunk's tokens
  const int stretch = DELTA ? (wave >> 1) & 1 : wave >> 1;
  const bool of_keys = DELTA && wave < 4, joining = DELTA && wave < 2, results = wave >= 6;
  const float skip = !DELTA && a.skip != nullptr ? a.skip[h] : 0.f;
  float* state = a.state + static_cast<size_t>(slot) * a.slot_stride + static_cast<size_t>(h) * a.tiles * a.dim * 64;
  auto state_at = [&](int d, int col) { return state + (static_cast<size_t>(col >> 6) * a.dim + d) * 64 + (col & 63); };
  floatx4 s[TPW][NC];
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int n = 0; n < NC; ++n) {
      const int d0 = (wave + 8 * i) * 16 + high * 4, col = col0 + n * 16 + low;
#pragma unroll
      for (int r = 0; r < 4; ++r) s[i][n][r] = d0 + r < a.dim && col < a.vdim ? *state_at(d0 + r, col) : 0.f;
      *reinterpret_cast<floatx4*>(S + (n * 16 + low) * ROW + d0) = s[i][n];
    }
  // The next chunk's keys, queries, values, P, T and numbers are asked for while this one is worked on: a thread brings four
  // dims of PER tokens' keys and queries, NC values, and four elements of P (waves 0 .. 3) or T.  The loads are straight-line
  // code, none of them under a condition: what lies beyond the dims, the columns or (in a sequence's last chunk) the tokens
  // is read from the nearest place that is there, and meets zeros: of S beyond the dims, of P, T and the tokens' w beyond
  // the tokens; columns beyond the head's are no one's.
  constexpr int PER = kChunk * DP / 4 / 512, K_ROWS = 512 / (DP / 4), V_ROWS = 512 / COLS;
  const int k_token = threadIdx.x / (DP / 4), k_dim = (threadIdx.x % (DP / 4)) * 4, v_token = threadIdx.x / COLS, v_col = threadIdx.x % COLS;
  const float* k_at = head_plane(a, a.k_first, group) + static_cast<size_t>(first) * a.dim;        // (the same for the whole workgroup)
  const float* q_at = head_plane(a, a.q_first, group) + static_cast<size_t>(first) * a.dim;
  const float* v_at = value_column(a, h, min(col0 + v_col, a.vdim - 1)) + static_cast<size_t>(first) * a.v_width;
  const float* part_at = a.parts + (static_cast<size_t>(seq) * a.chunks * a.heads + h) * kPartFloats;
  unsigned dim_at[BY4 ? 1 : 4];
#pragma unroll
  for (int e = 0; e < (BY4 ? 1 : 4); ++e) dim_at[e] = k_dim + e < a.dim ? k_dim + e : 0;
  const unsigned square_at = (DELTA ? threadIdx.x : threadIdx.x & 255) * 4;
  struct Ahead {
    floatx4 k[PER], q[PER], square;          // (the compiler keeps these in registers, and float4's class type not)
    float v[NC], w[NC], e;
  };
  auto fetch = [&](Ahead& to, int n) __attribute__((always_inline)) {                 // n: tokens from the chunk's first on
    const unsigned last = min(n, kChunk) - 1;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const unsigned from = min(static_cast<unsigned>(k_token + K_ROWS * i), last) * a.dim;
      if constexpr (BY4) {
        to.k[i] = *reinterpret_cast<const floatx4*>(k_at + (from + dim_at[0]));
        to.q[i] = *reinterpret_cast<const floatx4*>(q_at + (from + dim_at[0]));
      } else {
        const float* k = k_at + from;
        const float* q = q_at + from;
        to.k[i] = floatx4{k[dim_at[0]], k[dim_at[1]], k[dim_at[2]], k[dim_at[3]]};
        to.q[i] = floatx4{q[dim_at[0]], q[dim_at[1]], q[dim_at[2]], q[dim_at[3]]};
      }
    }
    to.square = *reinterpret_cast<const floatx4*>(part_at + square_at);
    to.e = part_at[2 * kChunk * kChunk + (threadIdx.x & 63)];
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      to.v[i] = v_at[min(static_cast<unsigned>(v_token + V_ROWS * i), last) * a.v_width];
      to.w[i] = DELTA ? 1.f : part_at[2 * kChunk * kChunk + kChunk + v_token + V_ROWS * i];
    }
  };
  // A chunk's results leave while the next chunk is worked on: a wait for what was asked for ahead is then no wait for
  // these stores (they count alike, and in order).
  floatx4 o[NC];
  float* out_at = a.out + (static_cast<size_t>(first + half * 16 + high * 4) * a.heads + h) * a.vdim + col0 + low;
  const size_t out_row = static_cast<size_t>(a.heads) * a.vdim;
  auto leave = [&](int n) {                            // n: tokens of the chunk and after it
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (half * 16 + high * 4 + r < n && col0 + c * 16 + low < a.vdim) out_at[r * out_row + c * 16] = o[c][r];
    out_at += kChunk * out_row;
  };
  auto work = [&](const Ahead& now, Ahead& next, int left) __attribute__((always_inline)) {       // left: tokens of this chunk and after it
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      *reinterpret_cast<floatx4*>(K + (k_token + K_ROWS * i) * ROW + k_dim) = now.k[i];
      *reinterpret_cast<floatx4*>(Q + (k_token + K_ROWS * i) * ROW + k_dim) = now.q[i];
    }
    {
      const int t = threadIdx.x & 255;
      float* to = (DELTA && threadIdx.x >= 256 ? T : P) + (t >> 3) * TROW + (t & 7) * 4;
      *reinterpret_cast<floatx4*>(to) = now.square;         // (additive: both halves of the workgroup write the same)
    }
    E[threadIdx.x & 63] = now.e;                          // (so does every wave)
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int at = v_col * TROW + v_token + V_ROWS * i;
      V[at] = now.v[i];
      if (!DELTA) UW[at] = now.v[i] * now.w[i];
    }
    lds_barrier();
    if (results && left < count) leave(left + kChunk);
    // (the last chunk asks for itself again, which nobody uses)
    const int more = left > kChunk ? 1 : 0;
    k_at += more * kChunk * a.dim, q_at += more * kChunk * a.dim, v_at += more * kChunk * a.v_width;
    part_at += static_cast<size_t>(more * a.heads) * kPartFloats;
    fetch(next, left - more * kChunk);
#pragma unroll
    for (int n = 0; n < NC; ++n) o[n] = floatx4{0.f, 0.f, 0.f, 0.f};
    {
      const float* from = (of_keys ? K : Q) + (half * 16 + low) * ROW + stretch * LENGTH + high * 4;
      const float* with = S + low * ROW + stretch * LENGTH + high * 4;
#pragma unroll
      for (int d = 0; d < LENGTH; d += 16) {
        const float4 x = lds4(from + d);
#pragma unroll
        for (int n = 0; n < NC; ++n) o[n] = mfma_f32_by16(x, lds4(with + n * 16 * ROW + d), o[n]);
      }
    }
    if (!results) {
      // (the parts of Q S that meet the result waves' own: delta rule, stretch 0 of waves 4 and 5; additive, stretches 0 .. 2)
      float* to = (of_keys ? KS + stretch * COLS * TROW : QS + (DELTA ? 0 : stretch) * COLS * TROW) + half * 16 + high * 4;
#pragma unroll
      for (int n = 0; n < NC; ++n) *reinterpret_cast<floatx4*>(to + (n * 16 + low) * TROW) = o[n];
    }
    lds_barrier();                                     // the parts are written, S has been read
    if (DELTA) {
      if (joining) {
        floatx4 u[NC];
#pragma unroll
        for (int n = 0; n < NC; ++n) u[n] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          if (j > half) break;                         // (T is zero above its diagonal: the first 16 tokens need no more)
          const float4 x = lds4(T + (half * 16 + low) * TROW + j * 16 + high * 4), e = lds4(E + j * 16 + high * 4);
#pragma unroll
          for (int n = 0; n < NC; ++n) {
            const int at = (n * 16 + low) * TROW + j * 16 + high * 4;
            const float4 v = lds4(V + at), k0 = lds4(KS + at), k1 = lds4(KS + COLS * TROW + at);
            const float4 rest = make_float4(v.x - e.x * (k0.x + k1.x), v.y - e.y * (k0.y + k1.y), v.z - e.z * (k0.z + k1.z), v.w - e.w * (k0.w + k1.w));
            u[n] = mfma_f32_by16(x, rest, u[n]);
          }
        }
        const float4 counts = lds4(E + kChunk + half * 16 + high * 4);
#pragma unroll
        for (int n = 0; n < NC; ++n) {
          const int at = (n * 16 + low) * TROW + half * 16 + high * 4;
          *reinterpret_cast<floatx4*>(U + at) = u[n];
          *reinterpret_cast<float4*>(UW + at) = make_float4(u[n][0] * counts.x, u[n][1] * counts.y, u[n][2] * counts.z, u[n][3] * counts.w);
        }
      }
      lds_barrier();
    }
    if (results) {
      const float* joins = DELTA ? U : V;              // (additive: P holds the tokens' w)
      const float4 e = lds4(E + half * 16 + high * 4);
#pragma unroll
      for (int n = 0; n < NC; ++n) {
        const int at = (n * 16 + low) * TROW + half * 16 + high * 4;
#pragma unroll
        for (int p = 0; p < PARTS - 1; ++p) o[n] += *reinterpret_cast<const floatx4*>(QS + p * COLS * TROW + at);
        o[n][0] *= e.x, o[n][1] *= e.y, o[n][2] *= e.z, o[n][3] *= e.w;
      }
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        if (j > half) break;
        const float4 x = lds4(P + (half * 16 + low) * TROW + j * 16 + high * 4);
#pragma unroll
        for (int n = 0; n < NC; ++n) o[n] = mfma_f32_by16(x, lds4(joins + (n * 16 + low) * TROW + j * 16 + high * 4), o[n]);
      }
      if (!DELTA) {
#pragma unroll
        for (int n = 0; n < NC; ++n) {
          const float4 v = lds4(V + (n * 16 + low) * TROW + half * 16 + high * 4);
          o[n][0] += skip * v.x, o[n][1] += skip * v.y, o[n][2] += skip * v.z, o[n][3] += skip * v.w;
        }
      }
    }
    const float keeps = E[kChunk - 1];
#pragma unroll
    for (int i = 0; i < TPW; ++i) {
      const int d0 = (wave + 8 * i) * 16;
      if (d0 >= a.dim) break;                          // (the same for the whole wave; beyond dim S stays zero)
#pragma unroll
      for (int n = 0; n < NC; ++n) s[i][n] *= keeps;
#pragma unroll
      for (int j = 0; j < kChunk; j += 16) {
        const float* key = K + (j + high * 4) * ROW + d0 + low;
        float4 x = make_float4(key[0], key[ROW], key[2 * ROW], key[3 * ROW]);
        if (d0 + 16 > a.dim && d0 + low >= a.dim) x = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int n = 0; n < NC; ++n) s[i][n] = mfma_f32_by16(x, lds4(UW + (n * 16 + low) * TROW + j + high * 4), s[i][n]);
      }
#pragma unroll
      for (int n = 0; n < NC; ++n) *reinterpret_cast<floatx4*>(S + (n * 16 + low) * ROW + d0 + high * 4) = s[i][n];
    }
    lds_barrier();                                     // S is whole, what this chunk left in LDS has been read
  };
  // (two places in turn for what is asked for ahead: with one, the compiler would wait for it to move it there)
  Ahead even, odd;
  fetch(even, count);
  for (int left = count; left > 0; left -= 2 * kChunk) {
    work(even, odd, left);
    if (left > kChunk) work(odd, even, left - kChunk);
  }
  if (results) leave((count - 1) % kChunk + 1);
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int n = 0; n < NC; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (wave + 8 * i) * 16 + high * 4 + r, col = col0 + n * 16 + low;
        if (d < a.dim && col < a.vdim) *state_at(d, col) = s[i][n][r];
      }
}

template <bool DELTA, int TPW, int NC>
constexpr size_t chain_lds() {
  constexpr int ROW = TPW * 128 + 4, COLS = NC * 16;
  return sizeof(float) * ((2 * kChunk + COLS) * ROW + (kChunk + 2 * COLS + (DELTA ? 1 : 3) * COLS) * kSquareRow + 2 * kChunk +
                          (DELTA ? (kChunk + 3 * COLS) * kSquareRow : 0));
}

}  // namespace tlie

using namespace tlie;

extern "C" int tlie_gated_scan_part_floats() { return kPartFloats; }

// in: float, the heads of q and k (groups of them, dim each) and of v (heads * vdim channels, in planes of v_width) from the
// channels q_first, k_first, v_first on, each a plane [plane_rows][width] (see GatedArgs; `channels` of them in all); gates: a product [nsplit][tokens][gate_row] of gate_dtype with a column a head at a_col (and, delta, at b_col); rate, bias, skip
// (or null): float [heads]; state: float [slots, heads, tiles, dim * 64], tiles = ceil(vdim / 64), a slot's row
// slot_stride floats after the one before it; out: float [tokens, heads * vdim].  chunks 0: every sequence is walked token
// by token; chunks > 0 (at least ceil(most tokens of a sequence / 32)): those that bring 24 tokens or more in chunks,
// with parts: float [sequences, chunks, heads, tlie_gated_scan_part_floats()] as scratch.
extern "C" int tlie_gated_scan(const float* in, int plane_rows, int channels, int q_first, int k_first, int v_first, int v_width,
                               const void* gates, int gate_dtype,
                               int nsplit, long long split_stride, int gate_row, int a_col, int b_col, const float* rate,
                               const float* bias, const float* skip, int delta, float* state, long long slot_stride,
                               const int* seq_start, const int* seq_slot, float* out, int sequences, int heads, int groups,
                               int dim, int vdim, int chunks, float* parts, void* stream) {
  if (sequences <= 0 || heads <= 0 || groups <= 0 || heads % groups != 0 || dim <= 0 || dim > kGatedMaxDim || vdim <= 0 || nsplit < 1) return kBadArgument;
  if (q_first < 0 || k_first < 0 || v_first < 0 || q_first + groups * dim > channels || k_first + groups * dim > channels ||
      v_first + heads * vdim > channels || v_width <= 0 || (heads * vdim) % v_width != 0 || plane_rows <= 0)
    return kBadArgument;
  if (32ll * dim > 2147483647ll || 32ll * v_width > 2147483647ll) return kBadArgument;
  if (a_col < 0 || a_col + heads > gate_row || (delta && (b_col < 0 || b_col + heads > gate_row || skip != nullptr))) return kBadArgument;
  const int tiles = (vdim + 63) / 64;
  if (heads > 65535 || tiles > 65535 || sequences > 65535 || groups > 65535 || chunks < 0 || (chunks > 0 && parts == nullptr)) return kBadArgument;
  if (slot_stride < static_cast<long long>(heads) * tiles * dim * 64 || slot_stride % 4 != 0) return kBadArgument;
  if ((reinterpret_cast<uintptr_t>(in) | reinterpret_cast<uintptr_t>(state) | reinterpret_cast<uintptr_t>(parts)) & 15) return kBadArgument;
  if (gate_dtype != kF32 && gate_dtype != kBF16) return kBadArgument;
  hipStream_t s = (hipStream_t)stream;
  const GatedArgs a{in, q_first, k_first, v_first, v_width, plane_rows, gates, nsplit, (size_t)split_stride, gate_row, a_col, b_col, rate, bias, skip,
                    state, (size_t)slot_stride, parts, seq_start, seq_slot, out, heads, groups, dim, vdim, tiles, chunks, chunks > 0, sequences};
#define TLIE_WALK(D, DELTA, DI) hipLaunchKernelGGL((gated_walk_kernel<D, DELTA, DI>), dim3(sequences, heads, tiles), dim3(256), 0, s, a)
#define TLIE_WALKS(D, DELTA)                 \
  if (dim <= 64) TLIE_WALK(D, DELTA, 4);     \
  else if (dim <= 128) TLIE_WALK(D, DELTA, 8); \
  else TLIE_WALK(D, DELTA, 16)
  if (gate_dtype == kF32) {
    if (delta) { TLIE_WALKS(float, true); } else { TLIE_WALKS(float, false); }
  } else {
    if (delta) { TLIE_WALKS(bf16, true); } else { TLIE_WALKS(bf16, false); }
  }
#undef TLIE_WALKS
#undef TLIE_WALK
  if (launch_status() != kOk) return kLaunchFailed;
  if (chunks == 0) return kOk;
  if (static_cast<long long>(sequences) * chunks > 2147483647LL) return kBadArgument;
  const int padded = (dim + 15) / 16 * 16;
  const size_t lds = sizeof(float) * (2 * kChunk * (padded + 4) + (delta ? 2 : 1) * kChunk * kSquareRow + 4 * (3 * kChunk + (delta ? kChunk * kSquareRow : 0)));
  // the heads of a group are shared out over workgroups until there are some thousand of them
  int shares = 1;
  const int rounds = (heads / groups + 3) / 4;
  while (shares < rounds && static_cast<long long>(sequences) * chunks * groups * shares < 1024) ++shares;
  const dim3 grid(sequences * chunks, groups, shares);
#define TLIE_CHUNK(D, DELTA) hipLaunchKernelGGL((gated_chunk_kernel<D, DELTA>), grid, dim3(256), lds, s, a, padded)
#define TLIE_BIG(KERNEL, BYTES)                                                                                      \
  if (BYTES > 65536) {                                                                                               \
    static const hipError_t raised = hipFuncSetAttribute(reinterpret_cast<const void*>(&KERNEL), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); \
    if (raised != hipSuccess) return kLaunchFailed;                                                                  \
  }
  if (gate_dtype == kF32) {
    if (delta) {
      TLIE_BIG((gated_chunk_kernel<float, true>), lds)
      TLIE_CHUNK(float, true);
    } else {
      TLIE_BIG((gated_chunk_kernel<float, false>), lds)
      TLIE_CHUNK(float, false);
    }
  } else {
    if (delta) {
      TLIE_BIG((gated_chunk_kernel<bf16, true>), lds)
      TLIE_CHUNK(bf16, true);
    } else {
      TLIE_BIG((gated_chunk_kernel<bf16, false>), lds)
      TLIE_CHUNK(bf16, false);
    }
  }
#undef TLIE_CHUNK
  if (launch_status() != kOk) return kLaunchFailed;
  const int column_tiles = (vdim + 15) / 16;
  const bool by_four = (dim & 3) == 0 && (k_first & 3) == 0 && (q_first & 3) == 0;
  const bool two = static_cast<long long>(column_tiles) * heads * sequences > 512;
#define TLIE_CHAIN(DELTA, TPW, NC)                                                                                \
  do {                                                                                                            \
    constexpr size_t bytes = chain_lds<DELTA, TPW, NC>();                                                          \
    const dim3 chain((sequences * heads + 7) / 8 * 8 * ((column_tiles + NC - 1) / NC));                            \
    if (by_four) {                                                                                                \
      TLIE_BIG((gated_chain_kernel<DELTA, TPW, NC, true>), bytes)                                                  \
      hipLaunchKernelGGL((gated_chain_kernel<DELTA, TPW, NC, true>), chain, dim3(512), bytes, s, a);               \
    } else {                                                                                                      \
      TLIE_BIG((gated_chain_kernel<DELTA, TPW, NC, false>), bytes)                                                 \
      hipLaunchKernelGGL((gated_chain_kernel<DELTA, TPW, NC, false>), chain, dim3(512), bytes, s, a);              \
    }                                                                                                             \
  } while (0)
#define TLIE_CHAINS(DELTA, NC)                 \
  if (dim <= 128) TLIE_CHAIN(DELTA, 1, NC);    \
  else TLIE_CHAIN(DELTA, 2, NC)
  if (delta) {
    if (two) { TLIE_CHAINS(true, 2); } else { TLIE_CHAINS(true, 1); }
  } else {
    if (two) { TLIE_CHAINS(false, 2); } else { TLIE_CHAINS(false, 1); }
  }
#undef TLIE_CHAINS
#undef TLIE_CHAIN
#undef TLIE_BIG
  return launch_status();
}
