// y = x . W^T for many rows of x (prompt steps), bfloat16 on the matrix cores: this library's own
// product of many rows, which runs where the vendor's library cannot be called (its file is not beside
// torch, or it has no algorithm for a shape within its workspace).
//
// reference: every product of the reference's device path is a library call (cublasGemmEx,
// src/cuda/kernels.cu:342-368); so are this engine's products of more than 64 rows.  Measured against
// that library on the MI355X (2048 tokens, TinyLlama's four matrices): this kernel reaches 0.5 to 0.7
// PFLOP/s where the library reaches 0.7 to 1.05, so the library stays the first choice; the plain
// 32-bit kernel, the only stand-in before, reaches 0.06.
//
// A workgroup of four waves owns a tile of 128 rows of W by 128 tokens and all of K.  K is walked
// in steps of 64: the step's 128 x 64 pieces of W and of x go from global memory straight into LDS
// (global_load_lds_dwordx4: no registers in between), two buffers in turn, so that a step's loads fly
// while the step before it is multiplied; two workgroups fit a compute unit and fill each other's
// waits.  LDS rows are 128 bytes; the 16-byte piece c of row r lies at piece c ^ (r % 8), so that the
// 8 lanes that read one piece of 8 neighbouring rows hit all banks once.  Each wave multiplies 64 rows
// of W by 64 tokens with v_mfma_f32_32x32x16_bf16, W as the first operand: a lane then holds, for one
// token, groups of four neighbouring outputs, which it stores as 8 or 16 bytes.
//
// The same tiles serve a routed feed-forward whose tokens use a few of many experts (the vendor's library takes no row
// lists).  A plan, made on the device from the router's scale matrix, holds per expert how many tokens use it and which, in
// the order of the tokens; a tile belongs to one expert, and its lanes ask for their own rows:
//   first product    hidden[pair] = s * max(W_up[e] x[token], 0)^2 for every (expert, token) pair, an expert's pairs side by
//                    side, the experts in order (s: the token's number for the expert)
//   second product   y[pair] = W_down[e] hidden[pair], W_down[e] a range of columns of one wide matrix
//   sum              out[token] = the sum of its pairs' y, in the order of the experts
// The grid covers the most tiles a plan can have; workgroups beyond the plan's tiles leave at once.  What a pair's row
// becomes depends on that row alone, wherever it stands.
#include "common.h"

namespace tlie {

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 bf16x8;
typedef __attribute__((__vector_size__(16 * sizeof(float)))) float floatx16;
typedef __attribute__((address_space(3))) uint32_t lds_word;

constexpr int kTileRows = 128;              // rows of W, and tokens, a workgroup
constexpr int kTileK = 64;                  // k values a step
constexpr int kTilePieces = kTileRows * kTileK / 8;   // 16-byte pieces of one operand's part of a step

// One 16-byte piece per lane from global memory into LDS at `base` + lane * 16 (base: the same for the wave).
__device__ __forceinline__ void load_piece(const uint16_t* from, uint4* base) {
  // (C-style casts: the address spaces are what the builtin's signature asks for)
  __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)from,
                                   (lds_word*)static_cast<uintptr_t>(static_cast<uint32_t>(reinterpret_cast<uintptr_t>(base))), 16, 0, 0);
}

struct TileBuffers {
  // two buffers, each W's part [128 rows][8 pieces] and then x's part; two arrays, named apart in the code
  // below, so that the compiler knows that a step's reads do not touch what the next step's loads write
  uint4 (&first)[2][kTilePieces];
  uint4 (&second)[2][kTilePieces];
};

// The product of a tile: from_w, from_x are the lane's 4 pieces of W and of x of step 0 (see `tile_piece`); acc as below.
__device__ __forceinline__ void tile_product(const uint16_t* (&from_w)[4], const uint16_t* (&from_x)[4], int steps, TileBuffers buffers,
                                             floatx16 (&acc)[2][2]) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  auto issue = [&](int step, uint4 (&buffer)[2][kTilePieces]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      load_piece(from_w[i] + step * kTileK, &buffer[0][wave * 256 + i * 64]);
      load_piece(from_x[i] + step * kTileK, &buffer[1][wave * 256 + i * 64]);
    }
  };
#pragma unroll
  for (int fn = 0; fn < 2; ++fn)
#pragma unroll
    for (int fm = 0; fm < 2; ++fm)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[fn][fm][r] = 0.f;

  // where this lane's operands lie in a buffer: row (lane % 32) of a group of 32, piece 2 kk + lane / 32
  const int wave_n = (wave & 1) * 64, wave_m = (wave >> 1) * 64;
  const int swizzle = lane & 7, high = lane >> 5;
  auto multiply = [&](const uint4 (&buffer)[2][kTilePieces]) {
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
      const int piece = (kk * 2 + high) ^ swizzle;
      uint4 wv[2], xv[2];
#pragma unroll
      for (int f = 0; f < 2; ++f) {
        wv[f] = buffer[0][(wave_n + f * 32 + (lane & 31)) * 8 + piece];
        xv[f] = buffer[1][(wave_m + f * 32 + (lane & 31)) * 8 + piece];
      }
#pragma unroll
      for (int fn = 0; fn < 2; ++fn)
#pragma unroll
        for (int fm = 0; fm < 2; ++fm)
          acc[fn][fm] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*reinterpret_cast<const bf16x8*>(&wv[fn]),
                                                                *reinterpret_cast<const bf16x8*>(&xv[fm]), acc[fn][fm], 0, 0, 0);
    }
  };
  issue(0, buffers.first);
  for (int step = 0; step < steps; step += 2) {
    __builtin_amdgcn_s_waitcnt(0x0f70);            // vmcnt(0): this wave's pieces of the step have landed
    __syncthreads();                               // everyone's have; and the other buffer has been read by all
    if (step + 1 < steps) issue(step + 1, buffers.second);
    multiply(buffers.first);
    if (step + 1 >= steps) break;
    __builtin_amdgcn_s_waitcnt(0x0f70);
    __syncthreads();
    if (step + 2 < steps) issue(step + 2, buffers.first);
    multiply(buffers.second);
  }
}

// What lies at piece i of this lane's 4 pieces of an operand in LDS: piece c (8 values of k) of row `row` of the tile.
__device__ __forceinline__ void tile_piece(int i, int& row, int& c) {
  const int piece = (threadIdx.x >> 6) * 256 + i * 64 + (threadIdx.x & 63);
  row = piece >> 3;
  c = (piece & 7) ^ (row & 7);
}

// x [M, K], w [N, K] bfloat16; out bfloat16 [M, N] or out_f32 float [M, N].  K % 64 == 0, N % 4 == 0.
__global__ void __launch_bounds__(256, 2)
gemm_tiles_kernel(const uint16_t* __restrict__ x, const uint16_t* __restrict__ w, uint16_t* __restrict__ out,
                  float* __restrict__ out_f32, int M, int N, int K, int tiles_n, int tiles_m) {
  __shared__ __attribute__((aligned(16))) uint4 buffer0[2][kTilePieces];
  __shared__ __attribute__((aligned(16))) uint4 buffer1[2][kTilePieces];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  // Workgroups are dealt to the chip's eight dies in turn; a die's workgroups take neighbouring
  // tiles (the same rows of W, all tokens), so that a die's L2 reads those rows of W once.
  const int total = tiles_n * tiles_m;
  const int per_die = (total + 7) / 8;
  const int id = (blockIdx.x & 7) * per_die + (blockIdx.x >> 3);
  if (id >= total) return;                                           // (the same for the whole workgroup)
  const int n0 = (id / tiles_m) * kTileRows, m0 = (id % tiles_m) * kTileRows;

  // ---- what this lane brings into LDS each step: 4 pieces of W and 4 of x ----
  const uint16_t* from_w[4];
  const uint16_t* from_x[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    int row, c;
    tile_piece(i, row, c);
    from_w[i] = w + static_cast<size_t>(min(n0 + row, N - 1)) * K + c * 8;      // (rows beyond the matrix: its last row, never stored)
    from_x[i] = x + static_cast<size_t>(min(m0 + row, M - 1)) * K + c * 8;
  }
  floatx16 acc[2][2];
  tile_product(from_w, from_x, K / kTileK, TileBuffers{buffer0, buffer1}, acc);

  // acc[fn][fm][4 g + j] = y[token m0 + wave_m + 32 fm + lane % 32][output n0 + wave_n + 32 fn + 8 g + 4 (lane / 32) + j]
  const int wave_n = (wave & 1) * 64, wave_m = (wave >> 1) * 64, high = lane >> 5;
#pragma unroll
  for (int fm = 0; fm < 2; ++fm) {
    const int m = m0 + wave_m + fm * 32 + (lane & 31);
    if (m >= M) continue;
#pragma unroll
    for (int fn = 0; fn < 2; ++fn)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int n = n0 + wave_n + fn * 32 + g * 8 + high * 4;       // the first of four neighbouring outputs
        if (n >= N) continue;                                         // (N is a multiple of 4)
        const float v0 = acc[fn][fm][g * 4], v1 = acc[fn][fm][g * 4 + 1], v2 = acc[fn][fm][g * 4 + 2], v3 = acc[fn][fm][g * 4 + 3];
        if (out_f32 != nullptr)
          *reinterpret_cast<float4*>(out_f32 + static_cast<size_t>(m) * N + n) = make_float4(v0, v1, v2, v3);
        else
          *reinterpret_cast<uint2*>(out + static_cast<size_t>(m) * N + n) = make_uint2(pack_bf16(v0, v1), pack_bf16(v2, v3));
      }
  }
}

// ---- a routed feed-forward's products over the pairs of experts and tokens -------------------------------------------

// A workgroup an expert: the tokens whose number for it is not zero, in order.  scale: float [tokens, scale_cols]; lists:
// int [experts, tokens], of which the first counts[e] of row e are written; ranks: int [tokens, experts], a token's place in
// the expert's list (written for the tokens that use it).
__global__ void __launch_bounds__(1024)
route_plan_kernel(const float* __restrict__ scale, int scale_cols, int tokens, int experts, int* __restrict__ counts,
                  int* __restrict__ lists, int* __restrict__ ranks) {
  __shared__ int wave_counts[16];
  const int e = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  int* list = lists + static_cast<size_t>(e) * tokens;
  int before = 0;                                      // of the tokens of the rounds so far (the same in every thread)
  for (int t0 = 0; t0 < tokens; t0 += 1024) {
    const int t = t0 + threadIdx.x;
    const bool uses = t < tokens && scale[static_cast<size_t>(t) * scale_cols + e] != 0.f;
    const unsigned long long mask = __ballot(uses);
    if (lane == 0) wave_counts[wave] = __popcll(mask);
    __syncthreads();
    int at = before, round = 0;
    for (int w = 0; w < 16; ++w) {
      if (w < wave) at += wave_counts[w];
      round += wave_counts[w];
    }
    if (uses) {
      at += __popcll(mask & ((1ull << lane) - 1));
      list[at] = t;
      ranks[static_cast<size_t>(t) * experts + e] = at;
    }
    before += round;
    __syncthreads();                                   // wave_counts has been read
  }
  if (threadIdx.x == 0) counts[e] = before;
}

// A running sum over the lanes of a wave, this lane's own value included.
__device__ __forceinline__ int wave_running_sum(int v, int lane) {
#pragma unroll
  for (int offset = 1; offset < 64; offset <<= 1) {
    const int other = __shfl_up(v, offset, 64);
    if (lane >= offset) v += other;
  }
  return v;
}

struct RoutedTile {
  int expert, rows;        // the tile's expert, and how many tokens use it
  int first_pair;          // the expert's first pair among all pairs
  int n_tile, m_tile;
};

// This workgroup's tile of a plan: the experts' tiles lie one expert after the other; inside an expert's, the tiles that
// share rows of W side by side; and the plan's tiles, however many it has, are dealt to the eight dies in equal stretches.
// Every wave finds it by itself; false: there is none for this workgroup.
__device__ __forceinline__ bool routed_tile(const int* __restrict__ counts, int experts, int tiles_n, RoutedTile& tile) {
  const int lane = threadIdx.x & 63;
  int total = 0;
  for (int e = lane; e < experts; e += 64) total += (counts[e] + kTileRows - 1) / kTileRows;
#pragma unroll
  for (int offset = 32; offset > 0; offset >>= 1) total += __shfl_xor(total, offset, 64);
  total *= tiles_n;
  const int per_die = (total + 7) / 8, place = blockIdx.x >> 3;
  const int id = (blockIdx.x & 7) * per_die + place;
  if (place >= per_die || id >= total) return false;
  int tiles_before = 0, pairs_before = 0;
  for (int e0 = 0; e0 < experts; e0 += 64) {
    const int rows = e0 + lane < experts ? counts[e0 + lane] : 0;
    const int tiles = (rows + kTileRows - 1) / kTileRows * tiles_n;
    const int tiles_to = tiles_before + wave_running_sum(tiles, lane), pairs_to = pairs_before + wave_running_sum(rows, lane);
    const unsigned long long beyond = __ballot(tiles_to > id);
    if (beyond != 0) {
      const int owner = __ffsll(beyond) - 1;
      tile.expert = e0 + owner;
      tile.rows = __builtin_amdgcn_readlane(rows, owner);
      tile.first_pair = __builtin_amdgcn_readlane(pairs_to, owner) - tile.rows;
      const int mine = __builtin_amdgcn_readlane(tiles, owner), inside = id - (__builtin_amdgcn_readlane(tiles_to, owner) - mine);
      const int m_tiles = mine / tiles_n;
      tile.n_tile = inside / m_tiles;
      tile.m_tile = inside - tile.n_tile * m_tiles;
      return true;
    }
    tiles_before = __builtin_amdgcn_readlane(tiles_to, 63);
    pairs_before = __builtin_amdgcn_readlane(pairs_to, 63);
  }
  return false;
}

// FIRST: the rows of x are the tokens of the expert's list, W_up[e] the rows e * N .. of w (K = w's row), and what is
// stored is the weighed activation, s * max(y, 0)^2 or (gated: the rows of w alternate gate and up) s * silu(gate) * up,
// half as many columns; else the rows of x are the pairs' own, and W_down[e] the columns e * K .. of w, whose
// rows are w_row long.  out: bfloat16 [pairs, N], room for `pairs` of them.  K % 64 == 0, N % 4 == 0.
template <bool FIRST>
__global__ void __launch_bounds__(256, 2)
routed_tiles_kernel(const uint16_t* __restrict__ x, const uint16_t* __restrict__ w, const int* __restrict__ counts,
                    const int* __restrict__ lists, const float* __restrict__ scale, int scale_cols, uint16_t* __restrict__ out,
                    int tokens, int experts, int pairs, int N, int K, int tiles_n, int gated, int w_row) {
  __shared__ __attribute__((aligned(16))) uint4 buffer0[2][kTilePieces];
  __shared__ __attribute__((aligned(16))) uint4 buffer1[2][kTilePieces];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  RoutedTile tile;
  if (!routed_tile(counts, experts, tiles_n, tile)) return;          // (the same for the whole workgroup)
  const int n0 = tile.n_tile * kTileRows, m0 = tile.m_tile * kTileRows;
  const int* list = lists + static_cast<size_t>(tile.expert) * tokens;
  const uint16_t* from_w[4];
  const uint16_t* from_x[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    int row, c;
    tile_piece(i, row, c);
    const int n = min(n0 + row, N - 1), m = min(m0 + row, tile.rows - 1);       // (rows beyond: the last one's, never stored)
    if (FIRST) {
      from_w[i] = w + (static_cast<size_t>(tile.expert) * N + n) * K + c * 8;
      from_x[i] = x + static_cast<size_t>(list[m]) * K + c * 8;
    } else {
      from_w[i] = w + static_cast<size_t>(n) * w_row + static_cast<size_t>(tile.expert) * K + c * 8;
      from_x[i] = x + static_cast<size_t>(min(tile.first_pair + m, pairs - 1)) * K + c * 8;
    }
  }
  floatx16 acc[2][2];
  tile_product(from_w, from_x, K / kTileK, TileBuffers{buffer0, buffer1}, acc);

  const int wave_n = (wave & 1) * 64, wave_m = (wave >> 1) * 64, high = lane >> 5;
#pragma unroll
  for (int fm = 0; fm < 2; ++fm) {
    const int m = m0 + wave_m + fm * 32 + (lane & 31);
    if (m >= tile.rows || tile.first_pair + m >= pairs) continue;    // (a token with more experts than were made room for)
    const float s = FIRST ? scale[static_cast<size_t>(list[m]) * scale_cols + tile.expert] : 1.f;
    uint16_t* to = out + static_cast<size_t>(tile.first_pair + m) * (gated ? N / 2 : N);
#pragma unroll
    for (int fn = 0; fn < 2; ++fn)
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        const int n = n0 + wave_n + fn * 32 + g * 8 + high * 4;
        if (n >= N) continue;
        if (FIRST && gated) {                                        // two gates with their ups
          const float first = s * gated_value(acc[fn][fm][g * 4], acc[fn][fm][g * 4 + 1], 0, 1.f, 0.f);
          const float second = s * gated_value(acc[fn][fm][g * 4 + 2], acc[fn][fm][g * 4 + 3], 0, 1.f, 0.f);
          *reinterpret_cast<uint32_t*>(to + n / 2) = pack_bf16(first, second);
          continue;
        }
        float v[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          v[j] = acc[fn][fm][g * 4 + j];
          if (FIRST) v[j] = fmaxf(v[j], 0.f), v[j] = s * v[j] * v[j];
        }
        *reinterpret_cast<uint2*>(to + n) = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
      }
  }
}

// out[t, :] = the sum of the rows of y of token t's pairs, in the order of the experts, in float, stored as bfloat16.  A
// workgroup a token; width % 8 == 0.
__global__ void __launch_bounds__(256)
routed_sum_kernel(const bf16* __restrict__ y, const float* __restrict__ scale, int scale_cols, const int* __restrict__ counts,
                  const int* __restrict__ ranks, bf16* __restrict__ out, int experts, int width, int most) {
  extern __shared__ int pair_rows[];                   // the token's pairs' rows of y, at most `most`
  __shared__ int found;
  const int t = blockIdx.x, lane = threadIdx.x & 63;
  if (threadIdx.x < 64) {
    int pairs_before = 0, have = 0;
    for (int e0 = 0; e0 < experts; e0 += 64) {
      const int e = e0 + lane;
      const int rows = e < experts ? counts[e] : 0;
      const int to = pairs_before + wave_running_sum(rows, lane);
      const bool uses = e < experts && scale[static_cast<size_t>(t) * scale_cols + e] != 0.f;
      const unsigned long long mask = __ballot(uses);
      if (uses) {
        const int at = have + __popcll(mask & ((1ull << lane) - 1));
        if (at < most) pair_rows[at] = to - rows + ranks[static_cast<size_t>(t) * experts + e];
      }
      have += __popcll(mask);
      pairs_before = __builtin_amdgcn_readlane(to, 63);
    }
    if (lane == 0) found = have < most ? have : most;
  }
  __syncthreads();
  const int count = found;
  for (int c = (blockIdx.y * 256 + threadIdx.x) * 8; c < width; c += gridDim.y * 2048) {
    float sum[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int i = 0; i < count; ++i) {
      float v[8];
      load8(y + static_cast<size_t>(pair_rows[i]) * width + c, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) sum[j] += v[j];
    }
    store8(out + static_cast<size_t>(t) * width + c, sum);
  }
}

}  // namespace tlie

using namespace tlie;

// x [M, K], w [N, K]: bfloat16; K a multiple of 64, N a multiple of 4.  out: bfloat16 [M, N], or float [M, N] when
// out_is_f32 is not 0.
extern "C" int tlie_gemm_tiles(const void* x, const void* w, void* out, int out_is_f32, int M, int N, int K, void* stream) {
  if (M <= 0 || N <= 0 || K <= 0 || (K % kTileK) != 0 || (N & 3) != 0 || out == nullptr) return kBadArgument;
  const int tiles_n = (N + kTileRows - 1) / kTileRows, tiles_m = (M + kTileRows - 1) / kTileRows;
  const long long total = static_cast<long long>(tiles_n) * tiles_m;
  if (total > (1 << 28)) return kBadArgument;
  const dim3 grid(static_cast<unsigned>((total + 7) / 8 * 8));
  hipLaunchKernelGGL(gemm_tiles_kernel, grid, dim3(256), 0, (hipStream_t)stream, (const uint16_t*)x, (const uint16_t*)w,
                     out_is_f32 ? nullptr : (uint16_t*)out, out_is_f32 ? (float*)out : nullptr, M, N, K, tiles_n, tiles_m);
  return launch_status();
}

// scale: float [tokens, scale_cols], column e the tokens' numbers for expert e (0: not used); counts: int [experts]; lists:
// int [experts, tokens]; ranks: int [tokens, experts].
extern "C" int tlie_route_plan(const float* scale, int scale_cols, int tokens, int experts, int* counts, int* lists, int* ranks,
                               void* stream) {
  if (tokens <= 0 || experts <= 0 || scale_cols < experts || scale == nullptr || counts == nullptr || lists == nullptr || ranks == nullptr)
    return kBadArgument;
  hipLaunchKernelGGL(route_plan_kernel, dim3(experts), dim3(1024), 0, (hipStream_t)stream, scale, scale_cols, tokens, experts, counts, lists, ranks);
  return launch_status();
}

// counts, lists: a plan of `tokens` tokens and `experts` experts, of which a token uses at most `most`.
// first 1: x [tokens, K], w [experts * N (or more), K], scale [tokens, scale_cols]; out [tokens * most, N] gets s * max(y, 0)^2 of
// every pair; first 2: w's rows alternate gate and up, out [tokens * most, N / 2] gets s * silu(gate) * up.
// first 0: x [tokens * most, K] the pairs' rows, w [N, w_row], w_row at least experts * K; out [tokens * most, N].  K % 64 == 0, N % 4 == 0.
extern "C" int tlie_routed_tiles(const void* x, const void* w, const int* counts, const int* lists, const float* scale, int scale_cols,
                                 void* out, int tokens, int experts, int most, int N, int K, int first, int w_row, void* stream) {
  if (first < 0 || first > 2 || (first == 0 && (w_row < experts * K || (w_row & 7) != 0))) return kBadArgument;
  if (tokens <= 0 || experts <= 0 || most <= 0 || most > experts || N <= 0 || K <= 0 || (K % kTileK) != 0 || (N & 3) != 0) return kBadArgument;
  if (x == nullptr || w == nullptr || out == nullptr || counts == nullptr || lists == nullptr || (first && (scale == nullptr || scale_cols < experts)))
    return kBadArgument;
  const int tiles_n = (N + kTileRows - 1) / kTileRows;
  // the most tiles of 128 rows that tokens * most pairs in `experts` lists (of at most `tokens`) can take
  const long long pairs = static_cast<long long>(tokens) * most;
  const long long m_tiles = pairs / kTileRows + experts;
  const long long total = m_tiles * tiles_n;
  if (total > (1 << 28) || pairs > 2147483647LL) return kBadArgument;
  const dim3 grid(static_cast<unsigned>((total + 7) / 8 * 8));
  hipStream_t s = (hipStream_t)stream;
  if (first)
    hipLaunchKernelGGL(routed_tiles_kernel<true>, grid, dim3(256), 0, s, (const uint16_t*)x, (const uint16_t*)w, counts, lists, scale,
                       scale_cols, (uint16_t*)out, tokens, experts, (int)pairs, N, K, tiles_n, first == 2 ? 1 : 0, w_row);
  else
    hipLaunchKernelGGL(routed_tiles_kernel<false>, grid, dim3(256), 0, s, (const uint16_t*)x, (const uint16_t*)w, counts, lists, scale,
                       scale_cols, (uint16_t*)out, tokens, experts, (int)pairs, N, K, tiles_n, first == 2 ? 1 : 0, w_row);
  return launch_status();
}

// y: bfloat16 [pairs, width]; out: bfloat16 [tokens, width]; width % 8 == 0; the plan as above.
extern "C" int tlie_routed_sum(const void* y, const float* scale, int scale_cols, const int* counts, const int* ranks, void* out,
                               int tokens, int experts, int most, int width, void* stream) {
  if (tokens <= 0 || experts <= 0 || most <= 0 || most > 4096 || width <= 0 || (width & 7) != 0 || scale_cols < experts) return kBadArgument;
  if (y == nullptr || scale == nullptr || counts == nullptr || ranks == nullptr || out == nullptr) return kBadArgument;
  int across = (width + 2047) / 2048;
  if (across > 64) across = 64;
  hipLaunchKernelGGL(routed_sum_kernel, dim3(tokens, across), dim3(256), static_cast<size_t>(most) * sizeof(int), (hipStream_t)stream,
                     (const bf16*)y, scale, scale_cols, counts, ranks, (bf16*)out, experts, width, most);
  return launch_status();
}
