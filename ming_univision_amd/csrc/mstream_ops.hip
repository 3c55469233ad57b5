// mstream_ops.hip — operators of sequence models whose residual is several parallel streams (mingnative.h section 14).  Rows are fp32,
// weights bf16, the streams' mixing numbers fp32 in device memory; everything here is fp32 arithmetic.
//   mn_streams_update_norm   streams <- mix of the streams + out * sublayer result (expert results summed in the launch); the next
//                            sublayer's input read from the new streams and RMS-normed
#include <math.h>

#include "common.h"

namespace {

constexpr int PLAIN_MAX_STREAMS = 32;

template <int GW>
__device__ __forceinline__ void ld_vals(const float* p, float (&v)[GW]) {
  if constexpr (GW == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
  } else {
    v[0] = *p;
  }
}

template <int GW>
__device__ __forceinline__ void st_vals(float* p, const float (&v)[GW]) {
  if constexpr (GW == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else *p = v[0];
}

// the normed value of column c
__device__ __forceinline__ float normed(float u, float r, const bf16_t* w, int c, int one_plus) {
  const float wt = bf16_to_f32(w[c]);
  return u * r * (one_plus ? 1.0f + wt : wt);
}

// One workgroup per row; a thread owns NV groups of GW columns in every stream, so the streams may be updated in place.  The
// sublayer input stays in registers between its read and its norm.
template <int S, int GW, int NV>
__global__ __launch_bounds__(256) void streams_kernel(mn_streams_args a) {
  __shared__ float red[4];
  const int m = blockIdx.x, tid = threadIdx.x, ng = a.n / GW;
  float mix[S][S], wo[S], wi[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    wi[s] = a.in ? a.in[s] : 1.0f;
    wo[s] = a.mix ? a.out[s] : 0.f;
#pragma unroll
    for (int t = 0; t < S; ++t) mix[s][t] = a.mix ? a.mix[s * S + t] : (s == t ? 1.f : 0.f);
  }
  const float* src = a.src + (int64_t)m * a.src_row;
  float* dst = a.dst ? a.dst + (int64_t)m * S * a.n : nullptr;
  float u[NV][GW];
  float xs[NV][S][GW], y[NV][GW];
  // every load of the row is requested before the first value is used
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int gi = tid + 256 * i, c = GW * (gi < ng ? gi : 0);
#pragma unroll
    for (int s = 0; s < S; ++s) ld_vals<GW>(src + s * a.src_stream + c, xs[i][s]);
    if (a.y) {
      ld_vals<GW>(a.y + (int64_t)m * a.ldy + c, y[i]);
    } else {
#pragma unroll
      for (int e = 0; e < GW; ++e) y[i][e] = 0.f;
    }
  }
  for (int j = 0; j < a.top; ++j) {
    const int z = m * a.top + j;
    const int64_t r = a.slot_of ? a.slot_of[z] : z;
    const float wt = a.ew ? a.ew[z] : 1.0f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int gi = tid + 256 * i, c = GW * (gi < ng ? gi : 0);
      float t[GW];
      ld_vals<GW>(a.ye + r * a.ldye + c, t);
#pragma unroll
      for (int e = 0; e < GW; ++e) y[i][e] = fmaf(wt, t[e], y[i][e]);
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int gi = tid + 256 * i;
    const bool on = gi < ng;
    float acc[GW];
#pragma unroll
    for (int e = 0; e < GW; ++e) acc[e] = 0.f;
#pragma unroll
    for (int t = 0; t < S; ++t) {
      float v[GW];
#pragma unroll
      for (int e = 0; e < GW; ++e) {
        float x = xs[i][t][e];
        if (a.mix) {
          x = wo[t] * y[i][e];
#pragma unroll
          for (int s = 0; s < S; ++s) x = fmaf(mix[s][t], xs[i][s][e], x);
        }
        v[e] = x;
        acc[e] = fmaf(wi[t], x, acc[e]);
      }
      if (dst && on) st_vals<GW>(dst + (int64_t)t * a.n + GW * gi, v);
    }
#pragma unroll
    for (int e = 0; e < GW; ++e) {
      u[i][e] = on ? acc[e] : 0.f;
      ss = fmaf(u[i][e], u[i][e], ss);
    }
  }
  if (!a.h && !a.h16) return;
  float r = 1.0f;
  if (a.w) r = 1.0f / sqrtf(block_sum(ss, red) / (float)a.n + a.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int gi = tid + 256 * i, c = GW * gi;
    if (gi >= ng) continue;
    float o[GW];
#pragma unroll
    for (int e = 0; e < GW; ++e) o[e] = a.w ? normed(u[i][e], r, a.w, c + e, a.one_plus) : u[i][e];
    if (a.h) st_vals<GW>(a.h + (int64_t)m * a.ldh + c, o);
    if (a.h16) {
      if constexpr (GW == 4) {
        *reinterpret_cast<uint2*>(a.h16 + (int64_t)m * a.ldh16 + c) = make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
      } else {
        a.h16[(int64_t)m * a.ldh16 + c] = f32_to_bf16(o[0]);
      }
    }
  }
}

// Any number of streams (up to PLAIN_MAX_STREAMS) and any row length: a thread's column of all streams lies in LDS, the sublayer input is
// read again from the stored streams for the norm.
__global__ __launch_bounds__(256) void streams_plain_kernel(mn_streams_args a) {
  extern __shared__ float col[];                      // [S][256]
  __shared__ float red[4];
  const int m = blockIdx.x, tid = threadIdx.x, S = a.S;
  const float* src = a.src + (int64_t)m * a.src_row;
  float* dst = a.dst ? a.dst + (int64_t)m * S * a.n : nullptr;
  auto read = [&](int c) {                            // the sublayer input of column c, the streams being updated on the way
    for (int s = 0; s < S; ++s) col[s * 256 + tid] = src[s * a.src_stream + c];
    float y = a.y ? a.y[(int64_t)m * a.ldy + c] : 0.f;
    for (int j = 0; j < a.top; ++j) {
      const int z = m * a.top + j;
      const int64_t r = a.slot_of ? a.slot_of[z] : z;
      y = fmaf(a.ew ? a.ew[z] : 1.0f, a.ye[r * a.ldye + c], y);
    }
    float u = 0.f;
    for (int t = 0; t < S; ++t) {
      float x = col[t * 256 + tid];
      if (a.mix) {
        x = a.out[t] * y;
        for (int s = 0; s < S; ++s) x = fmaf(a.mix[s * S + t], col[s * 256 + tid], x);
      }
      if (dst) dst[(int64_t)t * a.n + c] = x;
      u = fmaf(a.in ? a.in[t] : 1.0f, x, u);
    }
    return u;
  };
  float ss = 0.f;
  for (int c = tid; c < a.n; c += 256) {
    const float u = read(c);
    ss = fmaf(u, u, ss);
    if (!a.w) {
      if (a.h) a.h[(int64_t)m * a.ldh + c] = u;
      if (a.h16) a.h16[(int64_t)m * a.ldh16 + c] = f32_to_bf16(u);
    }
  }
  if (!a.w || (!a.h && !a.h16)) return;
  const float r = 1.0f / sqrtf(block_sum(ss, red) / (float)a.n + a.eps);
  const float* now = dst ? dst : src;                 // a thread rereads only columns it wrote itself (without a store there is no update)
  const int64_t stride = dst ? a.n : a.src_stream;
  for (int c = tid; c < a.n; c += 256) {
    float u = 0.f;
    for (int t = 0; t < S; ++t) u = fmaf(a.in ? a.in[t] : 1.0f, now[t * stride + c], u);
    const float o = normed(u, r, a.w, c, a.one_plus);
    if (a.h) a.h[(int64_t)m * a.ldh + c] = o;
    if (a.h16) a.h16[(int64_t)m * a.ldh16 + c] = f32_to_bf16(o);
  }
}

template <int S, int GW>
bool launch_streams(const mn_streams_args& a, int M, hipStream_t st) {
  const int per = (int)mn_cdiv(a.n / GW, 256);
  if (per > 8) return false;
#define MN_ST(NV_) hipLaunchKernelGGL((streams_kernel<S, GW, NV_>), dim3((unsigned)M), dim3(256), 0, st, a)
  if (per <= 1) MN_ST(1);
  else if (per <= 2) MN_ST(2);
  else if (per <= 4) MN_ST(4);
  else MN_ST(8);
#undef MN_ST
  return true;
}

}  // namespace

extern "C" size_t mn_sizeof_streams_args(void) { return sizeof(mn_streams_args); }

extern "C" int mn_streams_update_norm(const mn_streams_args* p, int M, void* stream) {
  MN_CHECK_ARG(p && p->src && M >= 1 && p->n >= 1 && p->S >= 1 && p->S <= PLAIN_MAX_STREAMS && p->top >= 0 && p->src_row >= 0 && p->src_stream >= 0,
               "mn_streams_update_norm: bad args (1 .. %d streams)", PLAIN_MAX_STREAMS);
  const mn_streams_args a = *p;
  MN_CHECK_ARG((!a.mix || a.out) && (a.top == 0 || a.ye) && (a.mix || (!a.y && a.top == 0)) && (a.dst || a.h || a.h16),
               "mn_streams_update_norm: a result needs the mixing numbers; something must be written");
  MN_CHECK_ARG((!a.h || a.ldh >= a.n) && (!a.h16 || a.ldh16 >= a.n) && (!a.y || a.ldy >= a.n) && (a.top == 0 || a.ldye >= a.n),
               "mn_streams_update_norm: row strides below a row");
  const uintptr_t al = (uintptr_t)a.src | (uintptr_t)a.dst | (uintptr_t)a.y | (uintptr_t)a.ye | (uintptr_t)a.h;
  const bool vec = (a.n % 4) == 0 && (al & 15) == 0 && (((uintptr_t)a.h16) & 7) == 0 && (a.src_row % 4) == 0 && (a.src_stream % 4) == 0 &&
                   (!a.y || (a.ldy % 4) == 0) && (a.top == 0 || (a.ldye % 4) == 0) && (!a.h || (a.ldh % 4) == 0) && (!a.h16 || (a.ldh16 % 4) == 0);
  hipStream_t st = mn_stream(stream);
  bool done = false;
#define MN_S(S_) done = vec ? launch_streams<S_, 4>(a, M, st) : launch_streams<S_, 1>(a, M, st)
  switch (a.S) {
    case 1: MN_S(1); break;
    case 2: MN_S(2); break;
    case 3: MN_S(3); break;
    case 4: MN_S(4); break;
    default: break;
  }
#undef MN_S
  if (!done) {
    MN_CHECK_ARG(!a.mix || a.dst || !a.w, "mn_streams_update_norm: rows of this size need the updated streams stored");
    hipLaunchKernelGGL(streams_plain_kernel, dim3((unsigned)M), dim3(256), (size_t)a.S * 256 * sizeof(float), st, a);
  }
  MN_CHECK_LAUNCH("mn_streams_update_norm");
  return MN_OK;
}
