// Recurrences over a matrix state S [dim, columns] per head, walked token after token.  A column of S is spread over R
// neighbouring lanes (RP rows each), so sums over the rows are sums over RP registers and a butterfly over R lanes inside the
// vector unit, and columns need nothing of each other - a block takes 256 / R columns of one head.  The recurrence is a chain
// through the tokens whose length nothing shortens, so what counts is a wave's instructions per token: with four rows a lane,
// one request's heads of 128 x 128 are 1,024 waves - one on every vector unit of the device.  A tile of tokens' vectors passes
// through LDS for all columns of the block; the next tile's values are asked for before this tile's tokens are walked; a
// whole tile is walked without a loop (constant LDS addresses, a token's reads issued one token ahead) and its outputs are
// stored after the next tile's barriers, which would otherwise wait for them.  A request's state lies in its slot transposed,
// [heads, columns, dim]: a lane's rows of a column are consecutive floats.
//
// The rules (q, k the head's vectors, v a column's value, g the decay - one per key channel, or one per head):
//   kDelta     S <- g S;  u = beta (v - S^T k);  S <- S + k u;  o = S^T q
//   kAdd       S <- g S + k (beta v);            o = S^T q
//   kAddAfter  o = S^T q + bonus v;              S <- g S + k v
// Since (g S + k u)^T q = (g S)^T q + u (k . q), the sums of the first two are taken over the decayed state in one pass.
//
// (A workspace holds kRowsBehind rows more than the step has tokens: a walk may read, and ignores, rows behind the last.)
// What a walk reads per token is a row of float32 (`prepared_width` floats): [q (groups x dim) | k (groups x dim) | g (heads x
// dim, where decays are per channel) | beta (heads) | dot (heads) | g (heads, where decays are per head)], dot being k . q
// (kAddAfter: the bonus); head h reads q and k of group h / (heads / groups).
#pragma once

#include "common.h"

namespace akv {

enum StateRule : int { kDelta = 0, kAdd = 1, kAddAfter = 2 };

__device__ __forceinline__ float softplus_of(float z) { return z > 20.f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float sigmoid_of(float z) { return 1.f / (1.f + expf(-z)); }

constexpr int kRowsBehind = 32;
__host__ __device__ inline int prepared_scalars(bool head_decay) { return head_decay ? 3 : 2; }
// (rounded up to whole 16-byte pieces: rows can then be read four floats at a time)
__host__ __device__ inline long prepared_width(int heads, int groups, int dim, bool head_decay) {
  const long floats = 2L * groups * dim + (head_decay ? 0L : static_cast<long>(heads) * dim) +
                      static_cast<long>(prepared_scalars(head_decay)) * heads;
  return (floats + 3) / 4 * 4;
}
__host__ __device__ inline long prepared_scalars_at(int heads, int groups, int dim, bool head_decay) {
  return 2L * groups * dim + (head_decay ? 0L : static_cast<long>(heads) * dim);
}

// The state's loads end here.  Registers that a loop carries and whose loads may still be on their way when it is entered make
// the compiler wait for ALL loads at their first use inside the loop, on every turn - the next tile's among them.
template <int N> __device__ __forceinline__ void settle(float (&v)[N]) {
#pragma unroll
  for (int i = 0; i < N; ++i) asm volatile("" : "+v"(v[i]));
}

// Sums over the R neighbouring lanes of a column, in all of them, without a trip through LDS: exchanges inside quads, the
// two mirrors of a row of 16 lanes, then swaps of rows and of the wave's halves.
template <int CTRL> __device__ __forceinline__ float lane_exchange(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xF, 0xF, true));
}
template <int R> __device__ __forceinline__ float column_sum(float v) {
  if (R >= 2) v += lane_exchange<0xB1>(v);       // quad_perm [1, 0, 3, 2]
  if (R >= 4) v += lane_exchange<0x4E>(v);       // quad_perm [2, 3, 0, 1]
  if (R >= 8) v += lane_exchange<0x141>(v);      // row_half_mirror
  if (R >= 16) v += lane_exchange<0x140>(v);     // row_mirror
  if (R >= 32) {
    const uint32_t bits = __float_as_uint(v);
    const auto swapped = __builtin_amdgcn_permlane16_swap(bits, bits, false, false);
    v = __uint_as_float(swapped[0]) + __uint_as_float(swapped[1]);
  }
  if (R >= 64) {
    const uint32_t bits = __float_as_uint(v);
    const auto swapped = __builtin_amdgcn_permlane32_swap(bits, bits, false, false);
    v = __uint_as_float(swapped[0]) + __uint_as_float(swapped[1]);
  }
  return v;
}

// Tokens of a tile: what 48 KB of LDS hold of their q, k and g, CAP at most.  Every tile costs two barriers, its loads'
// addresses and its stores: 32 tokens instead of 16 took an eighth off a long walk's time.  Steps of single tokens take
// tiles of 4: many blocks of little LDS fit a compute unit and hide each other's loads of the state.
template <int RP, int R, int CAP, bool HEAD_DECAY> struct StateTile {
  static constexpr int kSegment = RP == 4 ? 4 : RP + 4;     // (padding keeps the longer segments of neighbouring lanes in different banks)
  static constexpr int kArray = R * kSegment;
  static constexpr int kColumns = 256 / R;
  static constexpr int kArrays = HEAD_DECAY ? 2 : 3;        // q, k and, per channel, g
  static constexpr int kScalars = HEAD_DECAY ? 3 : 2;       // beta, dot and, per head, g
  static constexpr int kRoom = 12288 / (kArrays * kArray);
  static constexpr int kTokens = kRoom >= CAP ? CAP : kRoom >= 16 ? 16 : kRoom >= 1 ? kRoom : 1;
  static constexpr int kFloats = kTokens * (kArrays * kArray + kColumns + kScalars);
};

// What a lane needs of one token: its RP rows of q, k and g, its column's value, the head's scalars.
template <int RP, bool HEAD_DECAY> struct TokenOperands {
  float q[RP], k[RP], g[HEAD_DECAY ? 1 : RP], value, beta, dot;
  __device__ __forceinline__ void read(const float* qs, int array, const float* value_at, const float* scalar_at) {
#pragma unroll
    for (int i = 0; i < RP; i += 4) {
      const float4 q4 = *reinterpret_cast<const float4*>(qs + i);
      const float4 k4 = *reinterpret_cast<const float4*>(qs + array + i);
      q[i] = q4.x, q[i + 1] = q4.y, q[i + 2] = q4.z, q[i + 3] = q4.w;
      k[i] = k4.x, k[i + 1] = k4.y, k[i + 2] = k4.z, k[i + 3] = k4.w;
      if constexpr (!HEAD_DECAY) {
        const float4 g4 = *reinterpret_cast<const float4*>(qs + 2 * array + i);
        g[i] = g4.x, g[i + 1] = g4.y, g[i + 2] = g4.z, g[i + 3] = g4.w;
      }
    }
    value = *value_at, beta = scalar_at[0], dot = scalar_at[1];
    if constexpr (HEAD_DECAY) g[0] = scalar_at[2];
  }
  __device__ __forceinline__ float decay(int i) const { return HEAD_DECAY ? g[0] : g[i]; }
};

// A block: one request, one head, 256 / R columns of S.  Thread (column, part): rows part * RP .. part * RP + RP - 1.
// LDS: per token of a tile its arrays (q, k, g) of R segments, then the tile's values [tile][columns] and its scalars.
// values: a token's row at `value_stride`, head h's `vdim` values from column h * vdim on.  With `ones` a head has one column
// more than it has values, whose value is 1 for every token.  raw_out [tokens, heads, vdim + ones].
template <typename T, int RP, int R, int CAP, int RULE, bool HEAD_DECAY>
__global__ __launch_bounds__(256) void state_walk_kernel(const float* __restrict__ prepared, const T* __restrict__ token_values,
                                                         long value_stride, float* __restrict__ state,
                                                         long state_stride, const int* __restrict__ q_start,
                                                         const int* __restrict__ seq_slots, float* __restrict__ raw_out,
                                                         int heads, int groups, int dim, int vdim, int ones) {
  using Tile = StateTile<RP, R, CAP, HEAD_DECAY>;
  constexpr int SP = Tile::kSegment, kArray = Tile::kArray, kColumns = Tile::kColumns, kTile = Tile::kTokens;
  constexpr int kArrays = Tile::kArrays, kScalars = Tile::kScalars;
  constexpr int kPadded = R * RP;
  constexpr int kVectorLoads = (kTile * kPadded + 255) / 256, kValueLoads = (kTile * kColumns + 255) / 256;
  __shared__ __attribute__((aligned(16))) float lds[Tile::kFloats];
  float* values = lds + kTile * kArrays * kArray;  // [tile][columns]
  float* scalars = values + kTile * kColumns;      // [tile][scalars]
  const int columns = vdim + ones;
  const int column_blocks = (columns + kColumns - 1) / kColumns;
  const int r = blockIdx.x / (heads * column_blocks);
  const int h = blockIdx.x / column_blocks % heads;
  const int part = threadIdx.x % R;
  const int col0 = blockIdx.x % column_blocks * kColumns;
  const int col = col0 + threadIdx.x / R;
  const bool works = col < columns;
  const int first = q_start[r], last = q_start[r + 1];
  const long width = prepared_width(heads, groups, dim, HEAD_DECAY);
  const int share = heads / groups;
  const long q_off = static_cast<long>(h / share) * dim, k_off = static_cast<long>(groups + h / share) * dim;
  const long g_off = 2L * groups * dim + static_cast<long>(h) * dim, b_off = prepared_scalars_at(heads, groups, dim, HEAD_DECAY) + h;

  float S[RP];
  float* kept = state + static_cast<long>(seq_slots[r]) * state_stride + (static_cast<long>(h) * columns + (works ? col : 0)) * dim;
  const bool whole_fours = dim % 4 == 0 && state_stride % 4 == 0;      // (16-byte accesses need their alignment)
#pragma unroll
  for (int i = 0; i < RP; i += 4) {
    const int d = part * RP + i;
    if (works && whole_fours && d < dim) {
      const float4 four = *reinterpret_cast<const float4*>(kept + d);
      S[i] = four.x, S[i + 1] = four.y, S[i + 2] = four.z, S[i + 3] = four.w;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) S[i + e] = works && d + e < dim ? kept[d + e] : 0.f;
    }
  }

  settle(S);

  // a tile's operands on their way from memory: asked for one tile ahead, laid into LDS when the tile before is done
  // (with four rows a lane the segments lie in LDS without padding: where rows of the workspace allow 16-byte loads, four
  // neighbouring floats travel together)
  constexpr int kFourLoads = (kTile * kPadded / 4 + 255) / 256;
  constexpr int kFetched = RP == 4 && 4 * kFourLoads > kVectorLoads ? 4 * kFourLoads : kVectorLoads;
  const bool fours = RP == 4 && dim % 4 == 0 && (reinterpret_cast<uintptr_t>(prepared) & 15) == 0;
  float fetched_q[kFetched], fetched_k[kFetched], fetched_g[HEAD_DECAY ? 1 : kFetched], fetched_s = 0.f;
  T fetched_v[kValueLoads];      // (as they are stored: a conversion in `fetch` would wait for its loads)
  // (loads are never skipped: a token or row that the tile does not have reads a neighbour's address, and what it read
  // is replaced by a value without effect when the tile is laid down - no branch stands between a load and the walk)
  int fetched_count = 0;
  auto fetch = [&](int t0) {
    const int count = min(kTile, last - t0);
    fetched_count = count;
    if (fours) {
#pragma unroll
      for (int j = 0; j < kFourLoads; ++j) {
        const int index = threadIdx.x + j * 256;
        const int tt = min(index / (kPadded / 4), count - 1), d = index % (kPadded / 4) * 4;
        const float* row = prepared + static_cast<long>(t0 + tt) * width + (d < dim ? d : 0);
        const float4 q4 = *reinterpret_cast<const float4*>(row + q_off);
        const float4 k4 = *reinterpret_cast<const float4*>(row + k_off);
        fetched_q[4 * j] = q4.x, fetched_q[4 * j + 1] = q4.y, fetched_q[4 * j + 2] = q4.z, fetched_q[4 * j + 3] = q4.w;
        fetched_k[4 * j] = k4.x, fetched_k[4 * j + 1] = k4.y, fetched_k[4 * j + 2] = k4.z, fetched_k[4 * j + 3] = k4.w;
        if constexpr (!HEAD_DECAY) {
          const float4 g4 = *reinterpret_cast<const float4*>(row + g_off);
          fetched_g[4 * j] = g4.x, fetched_g[4 * j + 1] = g4.y, fetched_g[4 * j + 2] = g4.z, fetched_g[4 * j + 3] = g4.w;
        }
      }
    } else {
#pragma unroll
    for (int j = 0; j < kVectorLoads; ++j) {
      const int index = threadIdx.x + j * 256;
      const int tt = index / kPadded, d = index % kPadded;
      const bool real = tt < count && d < dim;
      const float* row = prepared + static_cast<long>(t0 + tt) * width;
      fetched_q[j] = real ? row[q_off + d] : 0.f;
      fetched_k[j] = real ? row[k_off + d] : 0.f;
      if constexpr (!HEAD_DECAY) fetched_g[j] = real ? row[g_off + d] : 1.f;
    }
    }
#pragma unroll
    for (int j = 0; j < kValueLoads; ++j) {
      const int index = threadIdx.x + j * 256;
      const int tt = index / kColumns, c = col0 + index % kColumns;
      fetched_v[j] = token_values[static_cast<long>(t0 + min(tt, count - 1)) * value_stride + static_cast<long>(h) * vdim +
                                  (c < vdim ? c : 0)];
    }
    const int which = min(static_cast<int>(threadIdx.x), kScalars * count - 1);
    fetched_s = prepared[static_cast<long>(t0 + which / kScalars) * width + b_off + static_cast<long>(which % kScalars) * heads];
  };
  auto lay_down = [&]() {
    if (fours) {
#pragma unroll
      for (int j = 0; j < kFourLoads; ++j) {
        const int index = threadIdx.x + j * 256;
        if (index >= kTile * kPadded / 4) continue;
        float* at = lds + index / (kPadded / 4) * kArrays * kArray + index % (kPadded / 4) * 4;
        const bool real = index / (kPadded / 4) < fetched_count && index % (kPadded / 4) * 4 < dim;
        const float4 zeros = make_float4(0.f, 0.f, 0.f, 0.f), ones = make_float4(1.f, 1.f, 1.f, 1.f);
        *reinterpret_cast<float4*>(at) = real ? make_float4(fetched_q[4 * j], fetched_q[4 * j + 1], fetched_q[4 * j + 2], fetched_q[4 * j + 3]) : zeros;
        *reinterpret_cast<float4*>(at + kArray) = real ? make_float4(fetched_k[4 * j], fetched_k[4 * j + 1], fetched_k[4 * j + 2], fetched_k[4 * j + 3]) : zeros;
        if constexpr (!HEAD_DECAY)
          *reinterpret_cast<float4*>(at + 2 * kArray) = real ? make_float4(fetched_g[4 * j], fetched_g[4 * j + 1], fetched_g[4 * j + 2], fetched_g[4 * j + 3]) : ones;
      }
    } else {
#pragma unroll
      for (int j = 0; j < kVectorLoads; ++j) {
        const int index = threadIdx.x + j * 256;
        if (index >= kTile * kPadded) continue;
        const int tt = index / kPadded, d = index % kPadded;
        float* at = lds + tt * kArrays * kArray + (d / RP) * SP + d % RP;
        at[0] = fetched_q[j], at[kArray] = fetched_k[j];
        if constexpr (!HEAD_DECAY) at[2 * kArray] = fetched_g[j];
      }
    }
#pragma unroll
    for (int j = 0; j < kValueLoads; ++j) {
      const int index = threadIdx.x + j * 256;
      if (index < kTile * kColumns) {
        const int c = col0 + index % kColumns;
        values[index] = index / kColumns < fetched_count && c < columns ? (c < vdim ? to_float(fetched_v[j]) : 1.f) : 0.f;
      }
    }
    if (threadIdx.x < kScalars * kTile)
      scalars[threadIdx.x] = static_cast<int>(threadIdx.x) < kScalars * fetched_count ? fetched_s : 0.f;
  };

  // one token: the state decays, takes the token's write and is read out; returns the column's output
  auto walk = [&](const TokenOperands<RP, HEAD_DECAY>& now) {
    float sum_k[4] = {0.f, 0.f, 0.f, 0.f}, sum_q[4] = {0.f, 0.f, 0.f, 0.f};
    if constexpr (RULE == kAddAfter) {
#pragma unroll
      for (int i = 0; i < RP; i += 4) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          sum_q[e] = fmaf(S[i + e], now.q[i + e], sum_q[e]);
          S[i + e] = fmaf(now.k[i + e], now.value, S[i + e] * now.decay(i + e));
        }
      }
      return fmaf(now.dot, now.value, column_sum<R>((sum_q[0] + sum_q[1]) + (sum_q[2] + sum_q[3])));
    }
#pragma unroll
    for (int i = 0; i < RP; i += 4) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i + e] *= now.decay(i + e);
        if constexpr (RULE == kDelta) sum_k[e] = fmaf(S[i + e], now.k[i + e], sum_k[e]);
        sum_q[e] = fmaf(S[i + e], now.q[i + e], sum_q[e]);
      }
    }
    float u = now.beta * now.value;
    if constexpr (RULE == kDelta) u = now.beta * (now.value - column_sum<R>((sum_k[0] + sum_k[1]) + (sum_k[2] + sum_k[3])));
    const float from_q = column_sum<R>((sum_q[0] + sum_q[1]) + (sum_q[2] + sum_q[3]));
#pragma unroll
    for (int i = 0; i < RP; ++i) S[i] = fmaf(now.k[i], u, S[i]);
    return fmaf(u, now.dot, from_q);
  };

  // A whole tile's outputs wait in registers and are stored after the next tile's barriers: a barrier waits for every
  // store before it, and stores issued right before one would have the wave wait out their whole way to memory.
  float outs[kTile];
  int stored_from = -1;
  auto store_tile = [&]() {
    if (stored_from >= 0 && part == 0 && works) {
      float* out_at = raw_out + (static_cast<long>(stored_from) * heads + h) * columns + col;
#pragma unroll
      for (int tt = 0; tt < kTile; ++tt) out_at[static_cast<long>(tt) * heads * columns] = outs[tt];
    }
    stored_from = -1;
  };

  if (first < last) fetch(first);
  for (int t0 = first; t0 < last; t0 += kTile) {
    const int count = min(kTile, last - t0);
    __syncthreads();          // the tile before has been used by everybody
    lay_down();
    __syncthreads();
    if (t0 + kTile < last) fetch(t0 + kTile);
    store_tile();
    if (count == kTile) {
      // a whole tile: its tokens one after the other without a loop around them - every LDS address is a constant and
      // the tile's outputs leave in one go
      TokenOperands<RP, HEAD_DECAY> ahead[2];
      ahead[0].read(lds + part * SP, kArray, values + threadIdx.x / R, scalars);
#pragma unroll
      for (int tt = 0; tt < kTile; ++tt) {
        // the next token's reads are issued before this token's sums and stay there: a wave alone on its vector unit has
        // nobody to hide their way behind
        if (tt + 1 < kTile)
          ahead[(tt + 1) & 1].read(lds + (tt + 1) * kArrays * kArray + part * SP, kArray,
                                   values + (tt + 1) * kColumns + threadIdx.x / R, scalars + kScalars * (tt + 1));
        __builtin_amdgcn_sched_barrier(0);
        outs[tt] = walk(ahead[tt & 1]);
        __builtin_amdgcn_sched_barrier(0);
      }
      stored_from = t0;
    } else {
      for (int tt = 0; tt < count; ++tt) {
        TokenOperands<RP, HEAD_DECAY> now;
        now.read(lds + tt * kArrays * kArray + part * SP, kArray, values + tt * kColumns + threadIdx.x / R, scalars + kScalars * tt);
        const float out = walk(now);
        if (part == 0 && works) raw_out[(static_cast<long>(t0 + tt) * heads + h) * columns + col] = out;
      }
    }
  }
  store_tile();
  if (works) {
#pragma unroll
    for (int i = 0; i < RP; i += 4) {
      const int d = part * RP + i;
      if (whole_fours && d < dim) {
        *reinterpret_cast<float4*>(kept + d) = make_float4(S[i], S[i + 1], S[i + 2], S[i + 3]);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < dim) kept[d + e] = S[i + e];
      }
    }
  }
}

// ---- portions: tiles of 32 tokens ------------------------------------------------------------------------------------------
// No rule puts a token's read-out back into the state: the sums over the R lanes of a column can wait.  A lane keeps its share of
// every token's read-out until the tile has been walked; then the shares of a whole tile meet at once - at every exchange
// between lanes a lane gives away half of the tokens it holds and takes its partner's shares of the other half, so a tile
// costs one exchange a token instead of log2(R), and none of them is waited for.  (The delta rule's S^T k is needed at once.)
// A lane may take CP columns with one read of a token's vectors.  Tokens that a tile does not have are laid down as tokens
// without effect.  The tile's sums go through LDS to memory: neighbouring threads then store neighbouring columns.
template <int N, int R> struct TileSums {
  // v[0 .. N): a lane's shares of N tokens.  Leaves v[0 .. N / min(R, N)): whole sums; v[j] is token first_token(part) + j.
  static __device__ __forceinline__ void reduce(float (&v)[N], int part) {
    int held = N;
    if constexpr (R >= 64) {
#pragma unroll
      for (int j = 0; j < N; ++j) {
        const uint32_t bits = __float_as_uint(v[j]);
        const auto swapped = __builtin_amdgcn_permlane32_swap(bits, bits, false, false);
        v[j] = __uint_as_float(swapped[0]) + __uint_as_float(swapped[1]);
      }
    }
    if constexpr (R >= 32) {
#pragma unroll
      for (int j = 0; j < N / 2; ++j) {
        const auto swapped = __builtin_amdgcn_permlane16_swap(__float_as_uint(v[j]), __float_as_uint(v[j + N / 2]), false, false);
        v[j] = __uint_as_float(swapped[0]) + __uint_as_float(swapped[1]);
      }
      held = N / 2;
    }
    if constexpr (R >= 16) halve<0x140>(v, held, (part & 8) != 0), held /= 2;      // row_mirror
    if constexpr (R >= 8) halve<0x141>(v, held, (part & 4) != 0), held /= 2;       // row_half_mirror
    if constexpr (R >= 4) halve<0x4E>(v, held, (part & 2) != 0), held /= 2;        // quad_perm [2, 3, 0, 1]
    if constexpr (R >= 2) halve<0xB1>(v, held, (part & 1) != 0), held /= 2;        // quad_perm [1, 0, 3, 2]
  }
  static constexpr int kLeft = N / (R < 32 ? R : 32);
  static __device__ __forceinline__ int first_token(int part) {
    int token = 0, half = N / 2;
    if constexpr (R >= 32) token += (part & 16) ? half : 0, half /= 2;
    if constexpr (R >= 16) token += (part & 8) ? half : 0, half /= 2;
    if constexpr (R >= 8) token += (part & 4) ? half : 0, half /= 2;
    if constexpr (R >= 4) token += (part & 2) ? half : 0, half /= 2;
    if constexpr (R >= 2) token += (part & 1) ? half : 0;
    return token;
  }

 private:
  template <int CTRL> static __device__ __forceinline__ void halve(float (&v)[N], int held, bool upper) {
#pragma unroll
    for (int j = 0; j < N / 2; ++j) {
      if (j >= held / 2) break;
      const float mine = upper ? v[j + held / 2] : v[j], given = upper ? v[j] : v[j + held / 2];
      v[j] = mine + lane_exchange<CTRL>(given);
    }
  }
};

template <int R, int CP, int THREADS, bool HEAD_DECAY> struct SumTile {
  static constexpr int kTokens = 32;
  static constexpr int kArrays = HEAD_DECAY ? 2 : 3, kScalars = HEAD_DECAY ? 3 : 2;
  static constexpr int kArray = R * 4, kColumns = CP * (THREADS / R);
  static constexpr size_t kBytes = sizeof(float) * kTokens * (kArrays * kArray + 2 * kColumns + kScalars);
};

// A block: one request, one head, CP * THREADS / R columns.  Thread (lane group, part): rows part * 4 .. part * 4 + 3 of columns
// group, group + THREADS / R, ...  Blocks of neighbouring columns of a head, which read the same rows of the workspace, are
// given to one XCD.  (dim: a multiple of 4, at most 4 R)
template <typename T, int R, int CP, int THREADS, int RULE, bool HEAD_DECAY>
__global__ __launch_bounds__(THREADS) void tile_walk_kernel(const float* __restrict__ prepared, const T* __restrict__ token_values,
                                                                long value_stride, float* __restrict__ state,
                                                                long state_stride, const int* __restrict__ q_start,
                                                                const int* __restrict__ seq_slots, float* __restrict__ raw_out,
                                                                int units, int heads, int groups, int dim, int vdim, int ones) {
  using Tile = SumTile<R, CP, THREADS, HEAD_DECAY>;
  constexpr int kTile = Tile::kTokens, kArrays = Tile::kArrays, kArray = Tile::kArray, kColumns = Tile::kColumns;
  constexpr int kScalars = Tile::kScalars, kGroups = THREADS / R, kAhead = 2;
  constexpr bool kAfter = RULE == kAddAfter;
  extern __shared__ __attribute__((aligned(16))) float walk_lds[];
  float* vectors = walk_lds;                           // [tile][q, k (, g)][R * 4]
  float* values = vectors + kTile * kArrays * kArray;  // [tile][columns]
  float* sums = values + kTile * kColumns;             // [tile][columns]
  float* scalars = sums + kTile * kColumns;            // [tile][scalars]
  const int unit = static_cast<int>(blockIdx.x % kXcds * (gridDim.x / kXcds) + blockIdx.x / kXcds);
  if (unit >= units) return;
  const int columns = vdim + ones, column_blocks = (columns + kColumns - 1) / kColumns;
  const int r = unit / (heads * column_blocks), h = unit / column_blocks % heads, col0 = unit % column_blocks * kColumns;
  const int part = threadIdx.x % R, group = threadIdx.x / R;
  const int first = q_start[r], last = q_start[r + 1];
  const long width = prepared_width(heads, groups, dim, HEAD_DECAY);
  const int share = heads / groups;
  const long q_off = static_cast<long>(h / share) * dim, k_off = static_cast<long>(groups + h / share) * dim;
  const long g_off = 2L * groups * dim + static_cast<long>(h) * dim, b_off = prepared_scalars_at(heads, groups, dim, HEAD_DECAY) + h;
  const bool state_fours = state_stride % 4 == 0;

  float S[CP][4];
  float* kept[CP];
#pragma unroll
  for (int c = 0; c < CP; ++c) {
    const int col = col0 + group + c * kGroups;
    kept[c] = state + static_cast<long>(seq_slots[r]) * state_stride + (static_cast<long>(h) * columns + min(col, columns - 1)) * dim;
#pragma unroll
    for (int e = 0; e < 4; ++e) S[c][e] = 0.f;
    if (col < columns) {
      if (state_fours && part * 4 < dim) {
        const float4 four = *reinterpret_cast<const float4*>(kept[c] + part * 4);
        S[c][0] = four.x, S[c][1] = four.y, S[c][2] = four.z, S[c][3] = four.w;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (part * 4 + e < dim) S[c][e] = kept[c][part * 4 + e];
      }
    }
  }

#pragma unroll
  for (int c = 0; c < CP; ++c) settle(S[c]);

  // A tile on its way from memory: asked for while the tile before is walked.  (The workspace has room for a tile behind its
  // last row: rows that a tile does not have are read and replaced when the tile is laid down.)
  static_assert(kTile * R % THREADS == 0 && THREADS % R == 0, "a tile's pieces of 16 bytes are dealt evenly to the threads");
  constexpr int kFours = kTile * R / THREADS, kRowStep = THREADS / R;
  constexpr int kValueLoads = (kTile * kColumns + THREADS - 1) / THREADS, kScalarLoads = (kTile * kScalars + THREADS - 1) / THREADS;
  float4 next[kArrays][kFours];
  T next_values[kValueLoads];      // (as they are stored: a conversion here would wait for the loads)
  float next_scalars[kScalarLoads];
  int count = 0;
  const bool filled = dim == 4 * R;
  const int my_d = part * 4;
  const float* my_row = prepared + static_cast<long>(first + group) * width;      // (of the tile that is asked for next)
  const long offsets[3] = {q_off, k_off, g_off};
  auto fetch = [&](int t0) {
    count = min(kTile, last - t0);
    const int d = filled || my_d < dim ? my_d : 0;
#pragma unroll
    for (int a = 0; a < kArrays; ++a) {
      const float* from = my_row + offsets[a] + d;
#pragma unroll
      for (int j = 0; j < kFours; ++j) next[a][j] = *reinterpret_cast<const float4*>(from + static_cast<long>(j * kRowStep) * width);
    }
    my_row += static_cast<long>(kTile) * width;
#pragma unroll
    for (int j = 0; j < kValueLoads; ++j) {
      const int index = threadIdx.x + j * THREADS, c = col0 + index % kColumns;
      next_values[j] = token_values[static_cast<long>(t0 + min(index / kColumns, count - 1)) * value_stride +
                                    static_cast<long>(h) * vdim + (c < vdim ? c : 0)];
    }
#pragma unroll
    for (int j = 0; j < kScalarLoads; ++j) {
      const int index = min(static_cast<int>(threadIdx.x) + j * THREADS, kScalars * count - 1);
      next_scalars[j] = prepared[static_cast<long>(t0 + index / kScalars) * width + b_off + static_cast<long>(index % kScalars) * heads];
    }
  };
  auto lay_down = [&]() {
    float* at = vectors + group * kArrays * kArray + my_d;
    const bool whole = filled && count == kTile;      // (the same for the whole block)
#pragma unroll
    for (int j = 0; j < kFours; ++j) {
      const bool there = whole || (group + j * kRowStep < count && my_d < dim);
#pragma unroll
      for (int a = 0; a < kArrays; ++a) {
        const float other = a == 2 ? 1.f : 0.f;
        const float4 v = next[a][j];
        *reinterpret_cast<float4*>(at + j * kRowStep * kArrays * kArray + a * kArray) =
            make_float4(there ? v.x : other, there ? v.y : other, there ? v.z : other, there ? v.w : other);
      }
    }
#pragma unroll
    for (int j = 0; j < kValueLoads; ++j) {
      const int index = threadIdx.x + j * THREADS, c = col0 + index % kColumns;
      if (index < kTile * kColumns)
        values[index] = index / kColumns < count && c < columns ? (c < vdim ? to_float(next_values[j]) : 1.f) : 0.f;
    }
#pragma unroll
    for (int j = 0; j < kScalarLoads; ++j) {
      const int index = threadIdx.x + j * THREADS;
      if (index < kScalars * kTile)
        scalars[index] = index < kScalars * count ? next_scalars[j] : (index % kScalars == 2 ? 1.f : 0.f);
    }
  };
  // a tile's sums are taken out of LDS between the next tile's barriers and stored behind them: a barrier waits for every store
  // before it, and these stores then have a tile's walk to arrive
  constexpr int kStores = (kTile * kColumns + THREADS - 1) / THREADS;
  float leaving[kStores];
  auto take_sums = [&]() {
#pragma unroll
    for (int j = 0; j < kStores; ++j) leaving[j] = sums[min(static_cast<int>(threadIdx.x) + j * THREADS, kTile * kColumns - 1)];
  };
  auto store_sums = [&](int t0) {
#pragma unroll
    for (int j = 0; j < kStores; ++j) {
      const int index = threadIdx.x + j * THREADS, t = t0 + index / kColumns, c = col0 + index % kColumns;
      if (index < kTile * kColumns && t < last && c < columns) raw_out[(static_cast<long>(t) * heads + h) * columns + c] = leaving[j];
    }
  };

  const float with_bonus = part == 0 ? 1.f : 0.f;
  if (first < last) fetch(first);
  int walked = -1;
  for (int t0 = first; t0 < last; t0 += kTile) {
    __syncthreads();          // the tile before has been used by everybody, and its sums are in place
    lay_down();
    if (walked >= 0) take_sums();
    __syncthreads();
    if (t0 + kTile < last) fetch(t0 + kTile);
    if (walked >= 0) store_sums(walked);
    // the vectors of the tokens after the next are asked for before these tokens' sums and stay there: a wave alone on its
    // vector unit has nobody to hide their way behind
    float shares[CP][kTile];
    struct Operands {
      float4 q, k, g;
      float value[CP], head;
    } ahead[2][kAhead];
    auto read = [&](Operands (&into)[kAhead], int first_token) {
#pragma unroll
      for (int i = 0; i < kAhead; ++i) {
        const int tt = first_token + i;
        const float* at = vectors + tt * kArrays * kArray + part * 4;
        into[i].q = *reinterpret_cast<const float4*>(at), into[i].k = *reinterpret_cast<const float4*>(at + kArray);
        if constexpr (HEAD_DECAY) into[i].g.x = scalars[tt * kScalars + 2];
        else into[i].g = *reinterpret_cast<const float4*>(at + 2 * kArray);
        into[i].head = scalars[tt * kScalars + (kAfter ? 1 : 0)];
#pragma unroll
        for (int c = 0; c < CP; ++c) into[i].value[c] = values[tt * kColumns + group + c * kGroups];
      }
    };
    read(ahead[0], 0);
#pragma unroll
    for (int t2 = 0; t2 < kTile; t2 += kAhead) {
      if (t2 + kAhead < kTile) read(ahead[(t2 / kAhead + 1) & 1], t2 + kAhead);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int i = 0; i < kAhead; ++i) {
        const Operands& now = ahead[(t2 / kAhead) & 1][i];
        const float4 q = now.q, k = now.k;
        const float4 g = HEAD_DECAY ? make_float4(now.g.x, now.g.x, now.g.x, now.g.x) : now.g;
#pragma unroll
        for (int c = 0; c < CP; ++c) {
          float even, odd;
          if constexpr (kAfter) {
            even = fmaf(S[c][2], q.z, S[c][0] * q.x), odd = fmaf(S[c][3], q.w, S[c][1] * q.y);
            even = fmaf(now.head * with_bonus, now.value[c], even);
          }
          float u = kAfter ? now.value[c] : now.head * now.value[c];
          if constexpr (RULE == kDelta) {
            // u = beta (v - (g S)^T k), the decay taken out of the chain from one state to the next
            if constexpr (HEAD_DECAY) {
              const float sum = fmaf(S[c][2], k.z, S[c][0] * k.x) + fmaf(S[c][3], k.w, S[c][1] * k.y);
              u = fmaf(-now.head * g.x, column_sum<R>(sum), u);
            } else {
              const float sum = fmaf(S[c][2], k.z * g.z, S[c][0] * (k.x * g.x)) + fmaf(S[c][3], k.w * g.w, S[c][1] * (k.y * g.y));
              u = fmaf(-now.head, column_sum<R>(sum), u);
            }
          }
          S[c][0] = fmaf(k.x, u, S[c][0] * g.x), S[c][1] = fmaf(k.y, u, S[c][1] * g.y);
          S[c][2] = fmaf(k.z, u, S[c][2] * g.z), S[c][3] = fmaf(k.w, u, S[c][3] * g.w);
          if constexpr (!kAfter) even = fmaf(S[c][2], q.z, S[c][0] * q.x), odd = fmaf(S[c][3], q.w, S[c][1] * q.y);
          shares[c][t2 + i] = even + odd;
        }
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    using Sums = TileSums<kTile, R>;
#pragma unroll
    for (int c = 0; c < CP; ++c) {
      Sums::reduce(shares[c], part);
      if (R < 64 || part < 32) {
#pragma unroll
        for (int j = 0; j < Sums::kLeft; ++j)
          sums[(Sums::first_token(part) + j) * kColumns + group + c * kGroups] = shares[c][j];
      }
    }
    walked = t0;
  }
  if (walked >= 0) {
    __syncthreads();
    take_sums();
    store_sums(walked);
  }
#pragma unroll
  for (int c = 0; c < CP; ++c) {
    if (col0 + group + c * kGroups >= columns) continue;
    if (state_fours && part * 4 < dim) {
      *reinterpret_cast<float4*>(kept[c] + part * 4) = make_float4(S[c][0], S[c][1], S[c][2], S[c][3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (part * 4 + e < dim) kept[c][part * 4 + e] = S[c][e];
    }
  }
}

// Launches the walk for heads of `dim` x (vdim + ones); dims beyond 2,048 are refused.  `longest`: the most tokens a request
// of the step brings (short steps take small tiles; the sums are the same either way).
template <typename T, int RULE, bool HEAD_DECAY>
int launch_state_walk(const float* prepared, const T* values, long value_stride, float* state, long state_stride,
                      const int* q_start, const int* seq_slots, float* raw, int seqs, int heads, int groups, int dim, int vdim,
                      int ones, int longest, hipStream_t stream) {
  if (dim <= 0 || dim > 2048) return -2;
  const int rp = dim <= 256 ? 4 : dim <= 512 ? 8 : dim <= 1024 ? 16 : 32;
  int R = 1;
  while (R * rp < dim) R *= 2;
  if (longest >= 16 && dim % 4 == 0 && rp == 4 && R >= 8) {
#define AKV_TILES(R_, CP, THREADS)                                                                                              \
  do {                                                                                                                          \
    using Tile = SumTile<R_, CP, THREADS, HEAD_DECAY>;                                                                          \
    const auto kernel = &tile_walk_kernel<T, R_, CP, THREADS, RULE, HEAD_DECAY>;                                                \
    const int units = seqs * heads * ((vdim + ones + Tile::kColumns - 1) / Tile::kColumns);                                     \
    static bool allowed = false;                                                                                                \
    if (Tile::kBytes > 64 * 1024 && !allowed) {                                                                                 \
      if (hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize,                \
                              static_cast<int>(Tile::kBytes)) != hipSuccess)                                                    \
        return -2;                                                                                                              \
      allowed = true;                                                                                                           \
    }                                                                                                                           \
    kernel<<<(units + kXcds - 1) / kXcds * kXcds, THREADS, Tile::kBytes, stream>>>(                                             \
        prepared, values, value_stride, state, state_stride, q_start, seq_slots, raw, units, heads, groups, dim, vdim, ones);   \
  } while (0)
    if (R == 64) AKV_TILES(64, 1, 256);
    else if (R == 32) AKV_TILES(32, 1, 256);
    else if (R == 16) AKV_TILES(16, 1, 128);
    else AKV_TILES(8, 1, 128);
#undef AKV_TILES
    return 0;
  }
  const int columns = 256 / R, column_blocks = (vdim + ones + columns - 1) / columns;
  const unsigned grid = static_cast<unsigned>(static_cast<long>(seqs) * heads * column_blocks);
#define AKV_WALK(RP, R_)                                                                                                        \
  do {                                                                                                                          \
    if (longest < 16)                                                                                                           \
      state_walk_kernel<T, RP, R_, 4, RULE, HEAD_DECAY><<<grid, 256, 0, stream>>>(                                              \
          prepared, values, value_stride, state, state_stride, q_start, seq_slots, raw, heads, groups, dim, vdim, ones);        \
    else                                                                                                                        \
      state_walk_kernel<T, RP, R_, 8, RULE, HEAD_DECAY><<<grid, 256, 0, stream>>>(                                           \
          prepared, values, value_stride, state, state_stride, q_start, seq_slots, raw, heads, groups, dim, vdim, ones);        \
  } while (0)
  if (rp == 32) AKV_WALK(32, 64);
  else if (rp == 16) AKV_WALK(16, 64);
  else if (rp == 8) AKV_WALK(8, 64);
  else if (R == 64) AKV_WALK(4, 64);
  else if (R == 32) AKV_WALK(4, 32);
  else if (R == 16) AKV_WALK(4, 16);
  else if (R == 8) AKV_WALK(4, 8);
  else if (R == 4) AKV_WALK(4, 4);
  else if (R == 2) AKV_WALK(4, 2);
  else AKV_WALK(4, 1);
#undef AKV_WALK
  return 0;
}

// One wave per (token, head): o = raw / rms(raw over the head's values) * weight * act(gate).  raw [tokens, heads, vdim + ones].
// With `ones` (the matrix memory) raw is divided first by max(|the column of ones|, exp(-top)) + read_eps, `tops` [tokens,
// heads].  The weight is one per value channel, shared by the heads, or (`weight_per_head`) one per head and channel; gates at
// `gate_stride` per token; act 1: sigmoid, 2: silu.
template <typename T, typename TG>
__global__ __launch_bounds__(256) void state_finish_kernel(const float* __restrict__ raw, const float* __restrict__ tops,
                                                           float read_eps, const float* __restrict__ weight,
                                                           int weight_per_head, const TG* __restrict__ gates, long gate_stride,
                                                           int gate_act, float eps, T* __restrict__ out, long items, int heads,
                                                           int vdim, int ones) {
  const long item = static_cast<long>(blockIdx.x) * (blockDim.x / kWave) + threadIdx.x / kWave;
  const int lane = threadIdx.x & (kWave - 1);
  if (item >= items) return;
  const long n = item / heads;
  const int h = static_cast<int>(item % heads);
  const float* x = raw + item * (vdim + ones);
  float inverse = 1.f;
  if (ones) inverse = 1.f / (fmaxf(fabsf(x[vdim]), expf(-tops[item])) + read_eps);
  float squares = 0.f;
  for (int i = lane; i < vdim; i += kWave) {
    const float v = x[i] * inverse;
    squares = fmaf(v, v, squares);
  }
  const float scale = inverse * rsqrtf(wave_sum(squares) / static_cast<float>(vdim) + eps);
  const float* w = weight + (weight_per_head ? static_cast<long>(h) * vdim : 0);
  const TG* gate_row = gates + n * gate_stride + static_cast<long>(h) * vdim;
  for (int i = lane; i < vdim; i += kWave) {
    const float gate = to_float(gate_row[i]);
    out[item * vdim + i] = from_float<T>(x[i] * scale * w[i] * (gate_act == 1 ? sigmoid_of(gate) : gate * sigmoid_of(gate)));
  }
}

}  // namespace akv
