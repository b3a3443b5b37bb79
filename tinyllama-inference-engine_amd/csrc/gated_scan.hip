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
  const float* in;             // [tokens][row]: q, k and v
  int row, q_col, k_col, v_col;
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
  int heads, groups, dim, vdim, tiles, chunks, chunked;
};

__device__ __forceinline__ float softplus32(float v) { return v > 20.f ? v : log1pf(expf(v)); }

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
  int turn = 0;
  for (int t0 = 0; t0 < count; t0 += kGatedBatch) {
    const int nb = min(kGatedBatch, count - t0);
    __syncthreads();                                   // the batch before has been read
    for (int i = threadIdx.x; i < nb * DMAX; i += 256) {
      const int b = i / DMAX, d = i - b * DMAX;
      const float* row = a.in + static_cast<size_t>(first + t0 + b) * a.row;
      qs[b][d] = d < a.dim ? row[a.q_col + group * a.dim + d] : 0.f;
      ks[b][d] = d < a.dim ? row[a.k_col + group * a.dim + d] : 0.f;
    }
    {
      const int b = threadIdx.x >> 6;
      if (b < nb) vs[b][lane] = base + lane < a.vdim ? a.in[static_cast<size_t>(first + t0 + b) * a.row + a.v_col + h * a.vdim + base + lane] : 0.f;
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

// A workgroup of four waves a (chunk of a sequence, group of heads): the products K K^T and Q K^T of the chunk's 32 tokens
// are made once for the group, then wave by wave the heads' own P and T.  blockIdx.z: a share of the group's heads.
template <typename D, bool DELTA>
__global__ void __launch_bounds__(256)
gated_chunk_kernel(const GatedArgs a, int dim_padded) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int row = dim_padded + 4;
  float* K = lds;                                      // [32][row]
  float* Q = K + kChunk * row;
  float* QK = Q + kChunk * row;                        // [32][33]
  float* KK = QK + kChunk * 33;
  float* work = KK + kChunk * 33;                      // a wave's: c [32] (doubles), w [32], and (delta) M [32][33]
  const int seq = blockIdx.x / a.chunks, chunk = blockIdx.x % a.chunks, group = blockIdx.y;
  const int slot = a.seq_slot[seq];
  if (slot < 0) return;
  const int first = a.seq_start[seq], count = a.seq_start[seq + 1] - first;
  const int begin = chunk * kChunk, n = min(kChunk, count - begin);
  if (count < kChunkedFrom || n <= 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int i = threadIdx.x; i < kChunk * dim_padded; i += 256) {
    const int r = i / dim_padded, d = i - r * dim_padded;
    const bool there = r < n && d < a.dim;
    const float* from = a.in + static_cast<size_t>(first + begin + (there ? r : 0)) * a.row + group * a.dim + (there ? d : 0);
    K[r * row + d] = there ? from[a.k_col] : 0.f;
    Q[r * row + d] = there ? from[a.q_col] : 0.f;
  }
  __syncthreads();
  {
    // wave w: rows (w / 2), columns (w % 2) of the 2 x 2 tiles; above the diagonal nobody reads
    const int ti = wave >> 1, tj = wave & 1;
    if (ti >= tj) {
      floatx4 qk = {0.f, 0.f, 0.f, 0.f}, kk = qk;
      const float* ai = Q + (ti * 16 + (lane & 15)) * row + (lane >> 4);
      const float* ki = K + (ti * 16 + (lane & 15)) * row + (lane >> 4);
      const float* bj = K + (tj * 16 + (lane & 15)) * row + (lane >> 4);
      for (int d = 0; d < dim_padded; d += 4) {
        const float b = bj[d];
        qk = mfma_f32(ai[d], b, qk);
        if (DELTA) kk = mfma_f32(ki[d], b, kk);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int at = (ti * 16 + (lane >> 4) * 4 + r) * 33 + tj * 16 + (lane & 15);
        QK[at] = qk[r];
        if (DELTA) KK[at] = kk[r];
      }
    }
  }
  __syncthreads();
  const int ratio = a.heads / a.groups;
  double* c = reinterpret_cast<double*>(work + wave * (3 * kChunk + (DELTA ? kChunk * 33 : 0)));
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
      for (int i = lane; i < kChunk * kChunk; i += 64) {
        const int r = i >> 5, j = i & 31;
        const float keeps = j <= r ? expf(static_cast<float>(c[r] - c[j])) : 0.f;
        part[i] = j <= r ? QK[r * 33 + j] * keeps * (DELTA ? 1.f : w[j]) : 0.f;
        if (DELTA) M[r * 33 + j] = j < r ? w[r] * keeps * KK[r * 33 + j] : 0.f;
      }
    }
    if (!DELTA) {
      __syncthreads();                                 // c and w have been read
      continue;
    }
    __syncthreads();
    if (live && lane < kChunk) {
      // lane j: column j of (I + M)^-1, row by row, times the column's w
      float x[kChunk];
#pragma unroll
      for (int i = 0; i < kChunk; ++i) {
        float sum = i == lane ? 1.f : 0.f;
#pragma unroll
        for (int k = 0; k < i; ++k) sum -= M[i * 33 + k] * x[k];
        x[i] = sum;
      }
      const float mine = w[lane];
#pragma unroll
      for (int i = 0; i < kChunk; ++i) part[kChunk * kChunk + i * kChunk + lane] = x[i] * mine;
    }
    __syncthreads();                                   // c, w and M have been read
  }
}

// A sequence's chunks one after the other: a workgroup of four waves for NC tiles of 16 columns of a head's S; wave w keeps
// the 16-dim tiles w, w + 4, ... of S (TPW of them) in registers, and all of S lies in LDS as an operand.
// DELTA: waves 0 and 1 make V - e^c K S of 16 tokens each, waves 2 and 3 the state's part of the results.  Additive: there
// is only the latter, and the waves share its dims in two halves.
template <bool DELTA, int TPW, int NC>
__global__ void __launch_bounds__(256)
gated_chain_kernel(const GatedArgs a) {
  constexpr int DP = TPW * 64, ROW = DP + 4, SROW = NC * 16 + 4, TROW = kChunk + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* K = lds;                                      // [32][ROW]
  float* Q = K + kChunk * ROW;                         // [32][ROW]
  float* S = Q + kChunk * ROW;                         // [DP][SROW]
  float* P = S + DP * SROW;                            // [32][TROW]
  float* U = P + kChunk * TROW;                        // [32][SROW]
  float* E = U + kChunk * SROW;                        // e^c [32], then what a key counts at the chunk's end [32]
  float* X = E + 2 * kChunk;                           // [32][SROW]: delta: what T is multiplied with; additive: half of the results' sums
  float* T = X + kChunk * SROW;                        // [32][TROW] (delta)
  const int seq = blockIdx.z, h = blockIdx.y, col0 = blockIdx.x * NC * 16;
  const int slot = a.seq_slot[seq];
  if (slot < 0) return;
  const int first = a.seq_start[seq], count = a.seq_start[seq + 1] - first;
  if (count < kChunkedFrom) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, low = lane & 15, high = lane >> 4;
  const int group = h / (a.heads / a.groups);
  const int half = wave & 1;                           // which 16 of the chunk's tokens this wave's results are
  const float skip = !DELTA && a.skip != nullptr ? a.skip[h] : 0.f;
  float* state = a.state + static_cast<size_t>(slot) * a.slot_stride + static_cast<size_t>(h) * a.tiles * a.dim * 64;
  auto state_at = [&](int d, int col) { return state + (static_cast<size_t>(col >> 6) * a.dim + d) * 64 + (col & 63); };
  floatx4 s[TPW][NC];
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int n = 0; n < NC; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (wave + 4 * i) * 16 + high * 4 + r, col = col0 + n * 16 + low;
        const float v = d < a.dim && col < a.vdim ? *state_at(d, col) : 0.f;
        s[i][n][r] = v;
        S[d * SROW + n * 16 + low] = v;
      }
  // the next chunk's keys, queries, P, T and numbers are asked for while this one is worked on
  constexpr int PER = kChunk * DP / 4 / 256;           // float4 of K (and of Q) a thread
  const bool by_four = (a.dim & 3) == 0 && (a.row & 3) == 0 && (a.k_col & 3) == 0 && (a.q_col & 3) == 0;
  float4 nk[PER], nq[PER], np, nt;
  float ne = 0.f;
  auto fetch = [&](int begin) {
    const int n = min(kChunk, count - begin);
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int at = threadIdx.x + 256 * i, r = at / (DP / 4), d = (at % (DP / 4)) * 4;
      nk[i] = nq[i] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (r < n && d < a.dim) {
        const float* from = a.in + static_cast<size_t>(first + begin + r) * a.row + group * a.dim + d;
        if (by_four) {
          nk[i] = *reinterpret_cast<const float4*>(from + a.k_col);
          nq[i] = *reinterpret_cast<const float4*>(from + a.q_col);
        } else {
          nk[i].x = from[a.k_col], nq[i].x = from[a.q_col];
          if (d + 1 < a.dim) nk[i].y = from[a.k_col + 1], nq[i].y = from[a.q_col + 1];
          if (d + 2 < a.dim) nk[i].z = from[a.k_col + 2], nq[i].z = from[a.q_col + 2];
          if (d + 3 < a.dim) nk[i].w = from[a.k_col + 3], nq[i].w = from[a.q_col + 3];
        }
      }
    }
    const float* part = a.parts + ((static_cast<size_t>(seq) * a.chunks + begin / kChunk) * a.heads + h) * kPartFloats;
    np = *reinterpret_cast<const float4*>(part + threadIdx.x * 4);
    if (DELTA) nt = *reinterpret_cast<const float4*>(part + kChunk * kChunk + threadIdx.x * 4);
    if (threadIdx.x < 2 * kChunk) ne = part[2 * kChunk * kChunk + threadIdx.x];
  };
  fetch(0);
  for (int begin = 0; begin < count; begin += kChunk) {
    const int left = count - begin;
    __syncthreads();                                   // the chunk before has been read, and S is whole
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int at = threadIdx.x + 256 * i, r = at / (DP / 4), d = (at % (DP / 4)) * 4;
      *reinterpret_cast<float4*>(K + r * ROW + d) = nk[i];
      *reinterpret_cast<float4*>(Q + r * ROW + d) = nq[i];
    }
    *reinterpret_cast<float4*>(P + (threadIdx.x >> 3) * TROW + (threadIdx.x & 7) * 4) = np;
    if (DELTA) *reinterpret_cast<float4*>(T + (threadIdx.x >> 3) * TROW + (threadIdx.x & 7) * 4) = nt;
    if (threadIdx.x < 2 * kChunk) E[threadIdx.x] = ne;
    // this wave's 16 tokens' values, where it needs them
    float v[NC][4];
#pragma unroll
    for (int n = 0; n < NC; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int token = half * 16 + high * 4 + r, col = col0 + n * 16 + low;
        v[n][r] = token < left && col < a.vdim ? a.in[static_cast<size_t>(first + begin + token) * a.row + a.v_col + h * a.vdim + col] : 0.f;
      }
    __syncthreads();
    if (begin + kChunk < count) fetch(begin + kChunk);
    floatx4 o[NC];
#pragma unroll
    for (int n = 0; n < NC; ++n) o[n] = floatx4{0.f, 0.f, 0.f, 0.f};
    {
      const float* from = (DELTA && wave < 2 ? K : Q) + (half * 16 + low) * ROW + high;
      const int d0 = DELTA ? 0 : (wave >> 1) * (DP / 2), d1 = DELTA ? DP : d0 + DP / 2;
#pragma unroll 8
      for (int d = d0; d < d1; d += 4) {
        const float x = from[d];
#pragma unroll
        for (int n = 0; n < NC; ++n) o[n] = mfma_f32(x, S[(d + high) * SROW + n * 16 + low], o[n]);
      }
    }
    if (wave < 2) {
#pragma unroll
      for (int n = 0; n < NC; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int token = half * 16 + high * 4 + r, at = token * SROW + n * 16 + low;
          if (DELTA) {
            X[at] = v[n][r] - E[token] * o[n][r];
          } else {
            X[at] = o[n][r];
            U[at] = v[n][r];
          }
        }
    }
    __syncthreads();                                   // X (and, additive, U) are written, S has been read
    if (DELTA) {
      if (wave < 2) {
        floatx4 u[NC];
#pragma unroll
        for (int n = 0; n < NC; ++n) u[n] = floatx4{0.f, 0.f, 0.f, 0.f};
        for (int j = 0; j < half * 16 + 16; j += 4) {
          const float x = T[(half * 16 + low) * TROW + j + high];
#pragma unroll
          for (int n = 0; n < NC; ++n) u[n] = mfma_f32(x, X[(j + high) * SROW + n * 16 + low], u[n]);
        }
#pragma unroll
        for (int n = 0; n < NC; ++n)
#pragma unroll
          for (int r = 0; r < 4; ++r) U[(half * 16 + high * 4 + r) * SROW + n * 16 + low] = u[n][r];
      }
      __syncthreads();
    }
    if (wave >= 2) {
#pragma unroll
      for (int n = 0; n < NC; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int token = half * 16 + high * 4 + r;
          if (!DELTA) o[n][r] += X[token * SROW + n * 16 + low];
          o[n][r] *= E[token];
        }
      for (int j = 0; j < half * 16 + 16; j += 4) {
        const float x = P[(half * 16 + low) * TROW + j + high];
#pragma unroll
        for (int n = 0; n < NC; ++n) o[n] = mfma_f32(x, U[(j + high) * SROW + n * 16 + low], o[n]);
      }
#pragma unroll
      for (int n = 0; n < NC; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int token = half * 16 + high * 4 + r, col = col0 + n * 16 + low;
          if (token < left && col < a.vdim)
            a.out[(static_cast<size_t>(first + begin + token) * a.heads + h) * a.vdim + col] = DELTA ? o[n][r] : o[n][r] + skip * v[n][r];
        }
    }
    const float keeps = E[kChunk - 1];
#pragma unroll
    for (int i = 0; i < TPW; ++i) {
      const int d0 = (wave + 4 * i) * 16;
      if (d0 >= a.dim) break;                          // (the same for the whole wave; beyond dim S stays zero)
#pragma unroll
      for (int n = 0; n < NC; ++n) s[i][n] *= keeps;
#pragma unroll
      for (int j = 0; j < kChunk; j += 4) {
        const float x = K[(j + high) * ROW + d0 + low] * E[kChunk + j + high];
#pragma unroll
        for (int n = 0; n < NC; ++n) s[i][n] = mfma_f32(x, U[(j + high) * SROW + n * 16 + low], s[i][n]);
      }
#pragma unroll
      for (int n = 0; n < NC; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[(d0 + high * 4 + r) * SROW + n * 16 + low] = s[i][n][r];
    }
  }
#pragma unroll
  for (int i = 0; i < TPW; ++i)
#pragma unroll
    for (int n = 0; n < NC; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (wave + 4 * i) * 16 + high * 4 + r, col = col0 + n * 16 + low;
        if (d < a.dim && col < a.vdim) *state_at(d, col) = s[i][n][r];
      }
}

template <bool DELTA, int TPW, int NC>
constexpr size_t chain_lds() {
  constexpr int DP = TPW * 64, ROW = DP + 4, SROW = NC * 16 + 4, TROW = kChunk + 4;
  return sizeof(float) * (2 * kChunk * ROW + DP * SROW + kChunk * TROW + 2 * kChunk * SROW + 2 * kChunk + (DELTA ? kChunk * TROW : 0));
}

}  // namespace tlie

using namespace tlie;

extern "C" int tlie_gated_scan_part_floats() { return kPartFloats; }

// in: float [tokens, row] with q (groups * dim), k (groups * dim) and v (heads * vdim) at q_col, k_col, v_col; gates: a
// product [nsplit][tokens][gate_row] of gate_dtype with a column a head at a_col (and, delta, at b_col); rate, bias, skip
// (or null): float [heads]; state: float [slots, heads, tiles, dim * 64], tiles = ceil(vdim / 64), a slot's row
// slot_stride floats after the one before it; out: float [tokens, heads * vdim].  chunks 0: every sequence is walked token
// by token; chunks > 0 (at least ceil(most tokens of a sequence / 32)): those that bring 24 tokens or more in chunks,
// with parts: float [sequences, chunks, heads, tlie_gated_scan_part_floats()] as scratch.
extern "C" int tlie_gated_scan(const float* in, int row, int q_col, int k_col, int v_col, const void* gates, int gate_dtype,
                               int nsplit, long long split_stride, int gate_row, int a_col, int b_col, const float* rate,
                               const float* bias, const float* skip, int delta, float* state, long long slot_stride,
                               const int* seq_start, const int* seq_slot, float* out, int sequences, int heads, int groups,
                               int dim, int vdim, int chunks, float* parts, void* stream) {
  if (sequences <= 0 || heads <= 0 || groups <= 0 || heads % groups != 0 || dim <= 0 || dim > kGatedMaxDim || vdim <= 0 || nsplit < 1) return kBadArgument;
  if (q_col < 0 || k_col < 0 || v_col < 0 || q_col + groups * dim > row || k_col + groups * dim > row || v_col + heads * vdim > row) return kBadArgument;
  if (a_col < 0 || a_col + heads > gate_row || (delta && (b_col < 0 || b_col + heads > gate_row || skip != nullptr))) return kBadArgument;
  const int tiles = (vdim + 63) / 64;
  if (heads > 65535 || tiles > 65535 || sequences > 65535 || groups > 65535 || chunks < 0 || (chunks > 0 && parts == nullptr)) return kBadArgument;
  if (slot_stride < static_cast<long long>(heads) * tiles * dim * 64 || slot_stride % 4 != 0) return kBadArgument;
  if ((reinterpret_cast<uintptr_t>(in) | reinterpret_cast<uintptr_t>(state) | reinterpret_cast<uintptr_t>(parts)) & 15) return kBadArgument;
  if (gate_dtype != kF32 && gate_dtype != kBF16) return kBadArgument;
  hipStream_t s = (hipStream_t)stream;
  const GatedArgs a{in, row, q_col, k_col, v_col, gates, nsplit, (size_t)split_stride, gate_row, a_col, b_col, rate, bias, skip,
                    state, (size_t)slot_stride, parts, seq_start, seq_slot, out, heads, groups, dim, vdim, tiles, chunks, chunks > 0};
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
  const int padded = (dim + 3) / 4 * 4;
  const size_t lds = sizeof(float) * (2 * kChunk * (padded + 4) + 2 * kChunk * 33 + 4 * (3 * kChunk + (delta ? kChunk * 33 : 0)));
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
  const bool two = static_cast<long long>(column_tiles) * heads * sequences > 512;
#define TLIE_CHAIN(DELTA, TPW, NC)                                                                                        \
  do {                                                                                                                    \
    constexpr size_t bytes = chain_lds<DELTA, TPW, NC>();                                                                  \
    TLIE_BIG((gated_chain_kernel<DELTA, TPW, NC>), bytes)                                                                  \
    hipLaunchKernelGGL((gated_chain_kernel<DELTA, TPW, NC>), dim3((column_tiles + NC - 1) / NC, heads, sequences), dim3(256), \
                       bytes, s, a);                                                                                      \
  } while (0)
#define TLIE_CHAINS(DELTA, NC)                 \
  if (dim <= 64) TLIE_CHAIN(DELTA, 1, NC);     \
  else if (dim <= 128) TLIE_CHAIN(DELTA, 2, NC); \
  else TLIE_CHAIN(DELTA, 4, NC)
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
