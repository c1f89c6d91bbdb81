// The gated delta rule, its decay per key channel or per head.  Per request and head, token after token, with S [dim, vdim]:
//     S <- g * S (row d times g_d, or all of it times g_h);  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
// where q and k are unit vectors per head (q also times dim^(-1/2)), beta = sigmoid(.), g = exp(-rate_h softplus(. + bias)).
// Everything after the projections and the short convolutions is float32: the unit norms, sigmoid, softplus, the
// exponentials, the state and its sums, the norm of the outputs.
//
// Three kernels.  `delta_prepare` is token-wise: the unit vectors, decays, betas and k . q of every token, float32, into a
// workspace.  The walk over a request's tokens is state_walk.h's with the rule kDelta.
// `state_finish_kernel` is token-wise again: o / rms(o) times a weight per value channel and a gate.

#include "api_parts.h"
#include "state_walk.h"

using namespace akv;

namespace {

// A wave is a token's unit of work: units 0 .. groups - 1 are a q / k pair (sums of squares and the product from one pass
// over the raw vectors: k . q of the unit vectors follows without reading them back; the scalars of the pair's heads go
// along), every further unit 256 decays of channels.  conv rows: [q (groups x dim) | k (groups x dim) | v ...] after
// convolution and activation; beta_logits at `beta_stride` per token; decay logits (TD) at `decay_stride` per token.
template <typename T, typename TD, bool HEAD_DECAY>
__global__ __launch_bounds__(256) void delta_prepare_kernel(const T* __restrict__ conv, long conv_stride,
                                                            const T* __restrict__ beta_logits, long beta_stride,
                                                            const TD* __restrict__ decay_logits, long decay_stride,
                                                            const float* __restrict__ decay_bias,
                                                            const float* __restrict__ rate, float unit_eps, float q_scale,
                                                            float* __restrict__ prepared, int heads, int groups, int dim) {
  const long n = blockIdx.x;
  const int lane = threadIdx.x & (kWave - 1);
  const int unit = blockIdx.y * (blockDim.x / kWave) + threadIdx.x / kWave;
  const long width = prepared_width(heads, groups, dim, HEAD_DECAY);
  float* row = prepared + n * width;
  float* g = row + 2L * groups * dim;
  float* beta = row + prepared_scalars_at(heads, groups, dim, HEAD_DECAY);
  const TD* logits = decay_logits + n * decay_stride;
  const int share = heads / groups;
  if (unit < groups) {
    const T* qs = conv + n * conv_stride + static_cast<long>(unit) * dim;
    const T* ks = qs + static_cast<long>(groups) * dim;
    float qq = 0.f, kk = 0.f, qk = 0.f;
    for (int i = lane; i < dim; i += kWave) {
      const float a = to_float(qs[i]), b = to_float(ks[i]);
      qq = fmaf(a, a, qq), kk = fmaf(b, b, kk), qk = fmaf(a, b, qk);
    }
    const float q_unit = q_scale / sqrtf(wave_sum(qq) + unit_eps), k_unit = 1.f / sqrtf(wave_sum(kk) + unit_eps);
    const float dot = wave_sum(qk) * q_unit * k_unit;
    for (int i = lane; i < dim; i += kWave) {
      row[static_cast<long>(unit) * dim + i] = to_float(qs[i]) * q_unit;
      row[static_cast<long>(groups + unit) * dim + i] = to_float(ks[i]) * k_unit;
    }
    for (int j = lane; j < share; j += kWave) {
      const int h = unit * share + j;
      beta[h] = sigmoid_of(to_float(beta_logits[n * beta_stride + h]));
      beta[heads + h] = dot;
      if constexpr (HEAD_DECAY) beta[2 * heads + h] = expf(-rate[h] * softplus_of(to_float(logits[h]) + decay_bias[h]));
    }
    return;
  }
  if constexpr (!HEAD_DECAY) {
    const int first = (unit - groups) * 256;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = first + e * kWave + lane;
      if (i < heads * dim) g[i] = expf(-rate[i / dim] * softplus_of(to_float(logits[i]) + decay_bias[i]));
    }
  }
}

template <typename T, typename TD, typename TG, bool HEAD_DECAY>
int delta_rule(const T* conv, long conv_stride, const T* beta_logits, long beta_stride, const TD* decay_logits,
               long decay_stride, const float* decay_bias, const float* rate, const TG* gates, long gate_stride, int gate_act,
               const float* norm_weight, float unit_eps, float norm_eps, float q_scale, float* state, long state_stride,
               const int* q_start, const int* seq_slots, float* workspace, T* out, int tokens, int seqs, int heads, int groups,
               int dim, int vdim, int longest, hipStream_t stream) {
  float* prepared = workspace;
  float* raw = workspace + (static_cast<long>(tokens) + kRowsBehind) * prepared_width(heads, groups, dim, HEAD_DECAY);
  const int units = groups + (HEAD_DECAY ? 0 : (heads * dim + 255) / 256);
  const dim3 prepare_grid(static_cast<unsigned>(tokens), static_cast<unsigned>((units + 3) / 4));
  delta_prepare_kernel<T, TD, HEAD_DECAY><<<prepare_grid, 256, 0, stream>>>(conv, conv_stride, beta_logits, beta_stride,
                                                                            decay_logits, decay_stride, decay_bias, rate,
                                                                            unit_eps, q_scale, prepared, heads, groups, dim);
  const int status = launch_state_walk<T, kDelta, HEAD_DECAY>(prepared, conv + 2L * groups * dim, conv_stride, state,
                                                              state_stride, q_start, seq_slots, raw, seqs, heads, groups, dim,
                                                              vdim, 0, longest, stream);
  if (status != 0) return status;
  const long items = static_cast<long>(tokens) * heads;
  state_finish_kernel<T, TG><<<static_cast<unsigned>((items + 3) / 4), 256, 0, stream>>>(
      raw, nullptr, 0.f, norm_weight, 0, gates, gate_stride, gate_act, norm_eps, out, items, heads, vdim, 0);
  return 0;
}

}  // namespace

extern "C" {

long akv_delta_rule_workspace(int tokens, int heads, int groups, int dim, int vdim, int decay_per_head) {
  return (static_cast<long>(tokens) + kRowsBehind) * (prepared_width(heads, groups, dim, decay_per_head != 0) + static_cast<long>(heads) * vdim);
}

int akv_delta_rule(const void* conv, long conv_stride, int dtype, const void* beta_logits, long beta_stride,
                   const void* decay_logits, int decay_dtype, long decay_stride, const float* decay_bias, const float* rate,
                   int decay_per_head, const void* gates, int gate_dtype, long gate_stride, int gate_act,
                   const float* norm_weight, float unit_eps, float norm_eps, float q_scale, float* state, long state_stride,
                   const int* q_start, const int* seq_slots, float* workspace, void* out, int tokens, int seqs, int heads,
                   int groups, int dim, int vdim, int longest, hipStream_t stream) {
  if (tokens <= 0 || seqs <= 0) return 0;
  if (heads <= 0 || groups <= 0 || heads % groups != 0 || dim <= 0 || vdim <= 0 || dim > 2048) return -2;
  if (gate_act != 1 && gate_act != 2) return -2;
  // decays per channel come from a product of their own with float32 sums, as do their gates; decays per head and their
  // gates are columns of the layer's first product
  const int own = decay_per_head ? dtype : static_cast<int>(kF32);
  if (decay_dtype != own || gate_dtype != own) return -1;
  int status = 0;
#define AKV_DELTA(TD, HEAD)                                                                                                    \
  status = delta_rule<T, TD, TD, HEAD>(static_cast<const T*>(conv), conv_stride, static_cast<const T*>(beta_logits), beta_stride, \
                                       static_cast<const TD*>(decay_logits), decay_stride, decay_bias, rate,                    \
                                       static_cast<const TD*>(gates), gate_stride, gate_act, norm_weight, unit_eps, norm_eps,   \
                                       q_scale, state, state_stride, q_start, seq_slots, workspace, static_cast<T*>(out), tokens, \
                                       seqs, heads, groups, dim, vdim, longest, stream)
  AKV_DISPATCH(dtype, T, {
    if (decay_per_head) AKV_DELTA(T, true);
    else AKV_DELTA(float, false);
  });
#undef AKV_DELTA
  if (status != 0) return status;
  return AKV_LAUNCH_STATUS();
}
}
