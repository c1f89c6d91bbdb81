// Two more mixers with a matrix state per head, walked by state_walk.h:
//   time mixing - a decay per key channel and token, w = exp(-exp(.)); the current token enters the read-out through a bonus
//   u per key channel: o = S^T r + (r . (u k)) v, then S <- diag(w) S + k v^T; its inputs are mixes of a token's row and the
//   row before it (`token_shift`);
//   a matrix memory - exponential input and forget gates per head under a running maximum m: with i and f the logs of the
//   gates, m' = max(f + m, i), S <- exp(f + m - m') S + exp(i - m') k v^T, n <- the same with k alone (the state's column of
//   ones), o = S^T q / (max(|n . q|, exp(-m')) + eps).
// Everything after the projections is float32.

#include "api_parts.h"
#include "state_walk.h"

using namespace akv;

namespace {

// ---- rows mixed with the row before them --------------------------------------------------------------------------------
// out [count][tokens][width]: row + (row before - row) * mu[s].  The row before a portion's first token is kept in the
// request's slot (zeros before its first token).  A thread takes VEC neighbouring channels of a token for all mixes.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void token_shift_kernel(const T* __restrict__ x, const float* __restrict__ mu, int count,
                                                          const float* __restrict__ state, long state_stride, long kept_at,
                                                          const int* __restrict__ seq_of_token,
                                                          const int* __restrict__ q_start, const int* __restrict__ seq_slots,
                                                          T* __restrict__ out, long tokens, int width) {
  const long n = blockIdx.x;
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * VEC;
  if (c >= width) return;
  const int r = seq_of_token[n];
  float now[VEC], gap[VEC];
  struct alignas(sizeof(T) * VEC) Pack { T v[VEC]; };
  const Pack mine = *reinterpret_cast<const Pack*>(x + n * width + c);
#pragma unroll
  for (int i = 0; i < VEC; ++i) now[i] = to_float(mine.v[i]);
  if (n > q_start[r]) {
    const Pack before = *reinterpret_cast<const Pack*>(x + (n - 1) * width + c);
#pragma unroll
    for (int i = 0; i < VEC; ++i) gap[i] = to_float(before.v[i]) - now[i];
  } else {
    const float* kept = state + static_cast<long>(seq_slots[r]) * state_stride + kept_at + c;
#pragma unroll
    for (int i = 0; i < VEC; ++i) gap[i] = kept[i] - now[i];
  }
  for (int s = 0; s < count; ++s) {
    Pack mixed;
#pragma unroll
    for (int i = 0; i < VEC; ++i) mixed.v[i] = from_float<T>(fmaf(gap[i], mu[static_cast<long>(s) * width + c + i], now[i]));
    *reinterpret_cast<Pack*>(out + (static_cast<long>(s) * tokens + n) * width + c) = mixed;
  }
}

// out = tanh(x), float32 -> T
template <typename T>
__global__ void tanh_rows_kernel(const float* __restrict__ x, T* __restrict__ out, long count) {
  const long i = static_cast<long>(blockIdx.x) * blockDim.x + threadIdx.x;
  if (i < count) out[i] = from_float<T>(tanhf(x[i]));
}

// ---- time mixing: what the walk reads of a token ----------------------------------------------------------------------------
// Blocks 0 .. tokens - 1 are tokens, a wave a head: r, k and the decays into the workspace, the bonus r . (u k).  Every
// further block is a request: its slot keeps the portion's last row for the next step's first mix.
template <typename T>
__global__ __launch_bounds__(256) void time_mixing_prepare_kernel(const T* __restrict__ r_rows, const T* __restrict__ k_rows,
                                                                  long row_stride, const float* __restrict__ decay_logits,
                                                                  const float* __restrict__ decay_bias,
                                                                  const float* __restrict__ bonus, float* __restrict__ prepared,
                                                                  int tokens, int heads, int dim, const T* __restrict__ x,
                                                                  int width, float* __restrict__ state, long state_stride,
                                                                  long kept_at, const int* __restrict__ q_start,
                                                                  const int* __restrict__ seq_slots) {
  if (static_cast<int>(blockIdx.x) >= tokens) {
    const int seq = blockIdx.x - tokens;
    const T* last = x + static_cast<long>(q_start[seq + 1] - 1) * width;
    float* kept = state + static_cast<long>(seq_slots[seq]) * state_stride + kept_at;
    for (int i = blockIdx.y * blockDim.x + threadIdx.x; i < width; i += gridDim.y * blockDim.x) kept[i] = to_float(last[i]);
    return;
  }
  const long n = blockIdx.x;
  const int lane = threadIdx.x & (kWave - 1);
  const int h = blockIdx.y * (blockDim.x / kWave) + threadIdx.x / kWave;
  if (h >= heads) return;
  float* row = prepared + n * prepared_width(heads, heads, dim, false);
  const long at = static_cast<long>(h) * dim, all = static_cast<long>(heads) * dim;
  float sum = 0.f;
  for (int i = lane; i < dim; i += kWave) {
    const float rv = to_float(r_rows[n * row_stride + at + i]), kv = to_float(k_rows[n * row_stride + at + i]);
    row[at + i] = rv;
    row[all + at + i] = kv;
    row[2 * all + at + i] = expf(-expf(decay_logits[n * all + at + i] + decay_bias[at + i]));
    sum = fmaf(rv * bonus[at + i], kv, sum);
  }
  sum = wave_sum(sum);
  if (lane == 0) {
    float* scalars = row + prepared_scalars_at(heads, heads, dim, false);
    scalars[h] = 1.f;
    scalars[heads + h] = sum;
  }
}

// ---- the matrix memory: gates under the running maximum --------------------------------------------------------------------
// A block is a (request, head); its threads take blockDim.x neighbouring tokens at a time.  m_t = max(f_t + m_(t-1), i_t) is a
// scan over pairs (sum of f, maximum): (f1, m1) then (f2, m2) is (f1 + f2, max(m1 + f2, m2)).
__device__ __forceinline__ void then_pair(float& f, float& m, float f_before, float m_before) {
  m = fmaxf(m_before + f, m);
  f += f_before;
}

template <typename T>
__global__ __launch_bounds__(1024) void matrix_memory_gates_kernel(const T* __restrict__ i_logits, const T* __restrict__ f_logits,
                                                                   long logit_stride, const float* __restrict__ i_bias,
                                                                   const float* __restrict__ f_bias, float cap,
                                                                   float* __restrict__ prepared, float* __restrict__ tops,
                                                                   float* __restrict__ state, long state_stride, long top_at,
                                                                   const int* __restrict__ q_start,
                                                                   const int* __restrict__ seq_slots, int heads, int dim) {
  __shared__ float wave_f[16], wave_m[16];
  const int seq = blockIdx.x, h = blockIdx.y;
  const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
  const int first = q_start[seq], last = q_start[seq + 1];
  float* kept = state + static_cast<long>(seq_slots[seq]) * state_stride + top_at + h;
  const long width = prepared_width(heads, heads, dim, true), at = prepared_scalars_at(heads, heads, dim, true);
  const float bias_i = i_bias[h], bias_f = f_bias[h];
  float m0 = *kept;
  for (int base = first; base < last; base += blockDim.x) {
    const int n = base + threadIdx.x;
    const bool real = n < last;
    float in = -INFINITY, f = 0.f;
    if (real) {
      in = cap * tanhf((to_float(i_logits[n * logit_stride + h]) + bias_i) / cap);
      const float z = cap * tanhf((to_float(f_logits[n * logit_stride + h]) + bias_f) / cap);
      f = -softplus_of(-z);
    }
    float sum_f = f, m = in;              // (a token beyond the portion: the identity of the scan)
#pragma unroll
    for (int offset = 1; offset < kWave; offset <<= 1) {
      const float before_f = __shfl_up(sum_f, offset, kWave), before_m = __shfl_up(m, offset, kWave);
      if (lane >= offset) then_pair(sum_f, m, before_f, before_m);
    }
    __syncthreads();                      // (the waves' pairs of the tokens before have been read)
    if (lane == kWave - 1) wave_f[wave] = sum_f, wave_m[wave] = m;
    __syncthreads();
    float start = m0;                     // m before this wave's first token
    for (int w = 0; w < wave; ++w) start = fmaxf(start + wave_f[w], wave_m[w]);
    const float m_here = fmaxf(start + sum_f, m);
    float m_before = __shfl_up(m_here, 1, kWave);
    if (lane == 0) m_before = start;
    if (real) {
      float* scalars = prepared + n * width + at;
      scalars[h] = expf(in - m_here);
      scalars[2 * heads + h] = expf(f + m_before - m_here);
      tops[static_cast<long>(n) * heads + h] = m_here;
    }
    float next = m0;
    for (int w = 0; w < static_cast<int>(blockDim.x) / kWave; ++w) next = fmaxf(next + wave_f[w], wave_m[w]);
    m0 = next;
  }
  if (threadIdx.x == 0) *kept = m0;
}

// q (times q_scale), k and k . q of every token, a wave a head
template <typename T>
__global__ __launch_bounds__(256) void matrix_memory_prepare_kernel(const T* __restrict__ q_rows, const T* __restrict__ k_rows,
                                                                    long row_stride, float q_scale, float* __restrict__ prepared,
                                                                    int heads, int dim) {
  const long n = blockIdx.x;
  const int lane = threadIdx.x & (kWave - 1);
  const int h = blockIdx.y * (blockDim.x / kWave) + threadIdx.x / kWave;
  if (h >= heads) return;
  float* row = prepared + n * prepared_width(heads, heads, dim, true);
  const long at = static_cast<long>(h) * dim, all = static_cast<long>(heads) * dim;
  float sum = 0.f;
  for (int i = lane; i < dim; i += kWave) {
    const float qv = to_float(q_rows[n * row_stride + at + i]) * q_scale, kv = to_float(k_rows[n * row_stride + at + i]);
    row[at + i] = qv;
    row[all + at + i] = kv;
    sum = fmaf(qv, kv, sum);
  }
  sum = wave_sum(sum);
  if (lane == 0) row[prepared_scalars_at(heads, heads, dim, true) + heads + h] = sum;
}

template <typename T>
int time_mixing(const T* r, const T* k, const T* v, const T* gates, long row_stride, const float* decay_logits,
                const float* decay_bias, const float* bonus, const float* norm_weight, float eps, const T* x, int width,
                float* state, long state_stride, long kept_at, const int* q_start, const int* seq_slots, float* workspace, T* out,
                int tokens, int seqs, int heads, int dim, int longest, hipStream_t stream) {
  float* prepared = workspace;
  float* raw = workspace + (static_cast<long>(tokens) + kRowsBehind) * prepared_width(heads, heads, dim, false);
  time_mixing_prepare_kernel<T><<<dim3(tokens + seqs, (heads + 3) / 4), 256, 0, stream>>>(
      r, k, row_stride, decay_logits, decay_bias, bonus, prepared, tokens, heads, dim, x, width, state, state_stride, kept_at,
      q_start, seq_slots);
  const int status = launch_state_walk<T, kAddAfter, false>(prepared, v, row_stride, state, state_stride, q_start, seq_slots, raw,
                                                            seqs, heads, heads, dim, dim, 0, longest, stream);
  if (status != 0) return status;
  const long items = static_cast<long>(tokens) * heads;
  state_finish_kernel<T, T><<<static_cast<unsigned>((items + 3) / 4), 256, 0, stream>>>(
      raw, nullptr, 0.f, norm_weight, 1, gates, row_stride, 2, eps, out, items, heads, dim, 0);
  return 0;
}

template <typename T>
int matrix_memory(const T* q, const T* k, const T* v, const T* gates, const T* i_logits, const T* f_logits, long row_stride,
                  const float* i_bias, const float* f_bias, float cap, float q_scale, float read_eps, const float* norm_weight,
                  float eps, float* state, long state_stride, long top_at, const int* q_start, const int* seq_slots,
                  float* workspace, T* out, int tokens, int seqs, int heads, int dim, int vdim, int longest,
                  hipStream_t stream) {
  float* prepared = workspace;
  float* raw = prepared + (static_cast<long>(tokens) + kRowsBehind) * prepared_width(heads, heads, dim, true);
  float* tops = raw + static_cast<long>(tokens) * heads * (vdim + 1);
  const int threads = min(1024, (longest + kWave - 1) / kWave * kWave);
  matrix_memory_gates_kernel<T><<<dim3(seqs, heads), threads, 0, stream>>>(i_logits, f_logits, row_stride, i_bias, f_bias, cap,
                                                                           prepared, tops, state, state_stride, top_at, q_start,
                                                                           seq_slots, heads, dim);
  matrix_memory_prepare_kernel<T><<<dim3(tokens, (heads + 3) / 4), 256, 0, stream>>>(q, k, row_stride, q_scale, prepared, heads,
                                                                                     dim);
  const int status = launch_state_walk<T, kAdd, true>(prepared, v, row_stride, state, state_stride, q_start, seq_slots, raw, seqs,
                                                      heads, heads, dim, vdim, 1, longest, stream);
  if (status != 0) return status;
  const long items = static_cast<long>(tokens) * heads;
  state_finish_kernel<T, T><<<static_cast<unsigned>((items + 3) / 4), 256, 0, stream>>>(
      raw, tops, read_eps, norm_weight, 1, gates, row_stride, 1, eps, out, items, heads, vdim, 1);
  return 0;
}

}  // namespace

extern "C" {

int akv_token_shift(const void* x, int dtype, const float* mu, int count, const float* state, long state_stride, long kept_at,
                    const int* seq_of_token, const int* q_start, const int* seq_slots, void* out, int tokens, int width,
                    hipStream_t stream) {
  if (tokens <= 0) return 0;
  if (width <= 0 || count <= 0) return -2;
#define AKV_SHIFT(VEC)                                                                                                          \
  AKV_DISPATCH(dtype, T, token_shift_kernel<T, VEC><<<dim3(tokens, (width / VEC + 255) / 256), 256, 0, stream>>>(                \
                             static_cast<const T*>(x), mu, count, state, state_stride, kept_at, seq_of_token, q_start, seq_slots, \
                             static_cast<T*>(out), tokens, width))
  if (width % 4 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 && reinterpret_cast<uintptr_t>(out) % 16 == 0) AKV_SHIFT(4);
  else AKV_SHIFT(1);
#undef AKV_SHIFT
  return AKV_LAUNCH_STATUS();
}

int akv_tanh_rows(const float* x, void* out, int dtype, long count, hipStream_t stream) {
  if (count <= 0) return 0;
  AKV_DISPATCH(dtype, T, tanh_rows_kernel<T><<<static_cast<unsigned>((count + 255) / 256), 256, 0, stream>>>(x, static_cast<T*>(out), count));
  return AKV_LAUNCH_STATUS();
}

long akv_time_mixing_workspace(int tokens, int heads, int dim) {
  return (static_cast<long>(tokens) + kRowsBehind) * (prepared_width(heads, heads, dim, false) + static_cast<long>(heads) * dim);
}

int akv_time_mixing(const void* r, const void* k, const void* v, const void* gates, int dtype, long row_stride,
                    const float* decay_logits, const float* decay_bias, const float* bonus, const float* norm_weight, float eps,
                    const void* x, int width, float* state, long state_stride, long kept_at, const int* q_start,
                    const int* seq_slots, float* workspace, void* out, int tokens, int seqs, int heads, int dim, int longest,
                    hipStream_t stream) {
  if (tokens <= 0 || seqs <= 0) return 0;
  if (heads <= 0 || dim <= 0 || dim > 2048 || width <= 0) return -2;
  int status = 0;
  AKV_DISPATCH(dtype, T, status = time_mixing<T>(static_cast<const T*>(r), static_cast<const T*>(k), static_cast<const T*>(v),
                                                 static_cast<const T*>(gates), row_stride, decay_logits, decay_bias, bonus,
                                                 norm_weight, eps, static_cast<const T*>(x), width, state, state_stride, kept_at,
                                                 q_start, seq_slots, workspace, static_cast<T*>(out), tokens, seqs, heads, dim,
                                                 longest, stream));
  if (status != 0) return status;
  return AKV_LAUNCH_STATUS();
}

long akv_matrix_memory_workspace(int tokens, int heads, int dim, int vdim) {
  return (static_cast<long>(tokens) + kRowsBehind) * (prepared_width(heads, heads, dim, true) + static_cast<long>(heads) * (vdim + 2));
}

int akv_matrix_memory(const void* q, const void* k, const void* v, const void* gates, const void* i_logits, const void* f_logits,
                      int dtype, long row_stride, const float* i_bias, const float* f_bias, float cap, float q_scale,
                      float read_eps, const float* norm_weight, float eps, float* state, long state_stride, long top_at,
                      const int* q_start, const int* seq_slots, float* workspace, void* out, int tokens, int seqs, int heads,
                      int dim, int vdim, int longest, hipStream_t stream) {
  if (tokens <= 0 || seqs <= 0) return 0;
  if (heads <= 0 || dim <= 0 || dim > 2048 || vdim <= 0 || longest <= 0 || !(cap > 0.f)) return -2;
  int status = 0;
  AKV_DISPATCH(dtype, T, status = matrix_memory<T>(static_cast<const T*>(q), static_cast<const T*>(k), static_cast<const T*>(v),
                                                   static_cast<const T*>(gates), static_cast<const T*>(i_logits),
                                                   static_cast<const T*>(f_logits), row_stride, i_bias, f_bias, cap, q_scale,
                                                   read_eps, norm_weight, eps, state, state_stride, top_at, q_start, seq_slots,
                                                   workspace, static_cast<T*>(out), tokens, seqs, heads, dim, vdim, longest,
                                                   stream));
  if (status != 0) return status;
  return AKV_LAUNCH_STATUS();
}
}
