// delta_device.h — device pieces shared by the delta-rule operators (pnorm_ops.hip) and the operators with a decay per key channel
// (chan_ops.hip): gate functions, the 8-lane sum, the preparation of a row (filters, silu, unit norms, write strengths).
#pragma once
#include "common.h"

namespace {

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_x(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

__device__ __forceinline__ float sum8(float v) {                    // over the 8 lanes of an aligned group; every lane gets the sum
  v += dpp_f<0xB1>(v);
  v += dpp_f<0x4E>(v);
  v += dpp_f<0x141>(v);
  return v;
}

// Gated delta rule, preparation of a row: channels [q: G dim ; k: G dim ; v: H vdim] of the raw projections go through their causal
// filter (earlier inputs from the rows before it in this call, then from the sequence's state) and silu; q and k heads become unit
// vectors (q also times q_scale); beta = sigmoid(b), decay = exp(-exp(a_log) softplus(a + dt_bias)) (a_log NULL: no decay per head).
struct DeltaPrepArgs {
  const float* proj; int64_t ld;             // raw [q ; k ; v] at column 0, b at off_b, a at off_a
  int H, G, dim, vdim, taps, off_b, off_a;
  const bf16_t* w_conv;                      // [2 G dim + H vdim, taps], the last tap multiplies the current row
  float* state;                              // [n_seq, taps - 1, channels]
  int advance;                               // 1: every row is alone in its sequence and moves the state on by itself
  const float *a_log, *dt_bias;              // device fp32 [H]
  float unit_eps, q_scale;
  const int32_t *row_seq, *row_slot, *row_back;
  float* qkv; int64_t ldo;                   // [M, channels]
  float* bd; int64_t ldbd;                   // [M, 2 H]: beta, decay ([M, H]: beta)
};

__device__ __forceinline__ float conv_silu(const DeltaPrepArgs& a, int m, int c, int n, int seq, int slot, int back) {
  float acc = 0.f;
  for (int k = 0; k < a.taps; ++k) {
    float v = 0.f;
    if (k <= back) v = a.proj[(int64_t)(m - k) * a.ld + c];
    else if (slot - k >= 0) v = a.state[((int64_t)seq * (a.taps - 1) + (k - back - 1)) * n + c];
    acc = fmaf(bf16_to_f32(a.w_conv[(int64_t)c * a.taps + (a.taps - 1 - k)]), v, acc);
  }
  if (a.advance && a.taps > 1) {                // a one-row sequence: entry i becomes entry i - 1, entry 0 this row's input
    float* st = a.state + (int64_t)seq * (a.taps - 1) * n + c;
    for (int i = a.taps - 2; i >= 1; --i) st[(int64_t)i * n] = st[(int64_t)(i - 1) * n];
    st[0] = a.proj[(int64_t)m * a.ld + c];
  }
  return silu_x(acc);
}

// one wave (back: rows of the same sequence directly before row m in this call): unit < 2 G = a q or k head of row m (its unit norm is a wave's reduction), then 256 value channels per unit
__device__ __forceinline__ void delta_prep_unit(const DeltaPrepArgs& a, int m, int unit, int lane, int back) {
  const int nqk = 2 * a.G * a.dim, nv = a.H * a.vdim, n = nqk + nv;
  const int seq = a.row_seq[m], slot = a.row_slot[m];
  float* out = a.qkv + (int64_t)m * a.ldo;
  if (unit < 2 * a.G) {
    const int c0 = unit * a.dim;
    float ss = 0.f;
    for (int d = lane; d < a.dim; d += 64) {
      const float v = conv_silu(a, m, c0 + d, n, seq, slot, back);
      out[c0 + d] = v;
      ss = fmaf(v, v, ss);
    }
    ss = wave_sum(ss);
    const float r = (unit < a.G ? a.q_scale : 1.0f) / sqrtf(ss + a.unit_eps);
    for (int d = lane; d < a.dim; d += 64) out[c0 + d] *= r;      // the lane rereads what it wrote itself
  } else {
    const int e0 = (unit - 2 * a.G) * 256;
    for (int e = e0 + lane; e < min(nv, e0 + 256); e += 64) out[nqk + e] = conv_silu(a, m, nqk + e, n, seq, slot, back);
  }
}

// 256 threads: the write strengths (and decays) of row m
__device__ __forceinline__ void delta_prep_strengths(const DeltaPrepArgs& a, int m, int tid) {
  const float* row = a.proj + (int64_t)m * a.ld;
  for (int h = tid; h < a.H; h += 256) {
    a.bd[(int64_t)m * a.ldbd + h] = sigmoid_f(row[a.off_b + h]);
    if (a.a_log) a.bd[(int64_t)m * a.ldbd + a.H + h] = expf(-expf(a.a_log[h]) * softplus_f(row[a.off_a + h] + a.dt_bias[h]));
  }
}

inline int64_t delta_prep_units(int H, int G, int vdim) { return 2 * (int64_t)G + mn_cdiv((int64_t)H * vdim, 256); }

}  // namespace
