// mstream_ops.hip — operators of sequence models whose residual is several parallel streams (mingnative.h section 14).  Rows are fp32,
// weights bf16, the streams' mixing numbers fp32 in device memory; everything here is fp32 arithmetic.
//   mn_streams_update_norm   streams <- mix of the streams + out * sublayer result (expert results summed in the launch); the next
//                            sublayer's input read from the new streams and RMS-normed; for few rows also its router: logits, picks, scores
//   mn_silu_split_rows_scaled   slab sums of the experts' gate and up products -> silu(s gate) * (s up) as bf16 hi / lo rows
#include <math.h>

#include "common.h"
#include "router_device.h"

namespace {

constexpr int PLAIN_MAX_STREAMS = 32;
constexpr int FEW_ROWS = 64;                            // up to here a row gets 16 waves, hi / lo rows and slabs
constexpr int ROUTE_MAX_N = 8192, ROUTE_MAX_EXPERTS = 512, ROUTE_MAX_EXPERTS_MANY_ROWS = 16;   // every row reads the whole router

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

// the results a row takes, summed over the slabs they lie in
template <int GW>
__device__ __forceinline__ void ld_slabs(const mn_streams_args& a, int64_t r, int c, float (&t)[GW]) {
  const float* p = a.ye + r * a.ldye + c;
  ld_vals<GW>(p, t);
  for (int z = 1; z < a.ye_slabs; ++z) {
    float u[GW];
    ld_vals<GW>(p + z * a.ye_slab, u);
#pragma unroll
    for (int e = 0; e < GW; ++e) t[e] += u[e];
  }
}

// h16's low parts: what the bf16 value leaves of v
__device__ __forceinline__ float low_part(float v) { return v - bf16_to_f32(f32_to_bf16(v)); }

// One workgroup per row; a thread owns NV groups of GW columns in every stream, so the streams may be updated in place.  The
// sublayer input stays in registers between its read and its norm.  ROUTE: the row's router logits too (a wave per expert, the normed row
// in LDS, the first weights requested before anything else), then the picks and their scores by one wave.  NT = 1024: low parts and slabs too.
template <int S, int GW, int NV, int NT, bool ROUTE>
__global__ __launch_bounds__(NT) void streams_kernel(mn_streams_args a) {
  __shared__ float red[NT / 64];
  extern __shared__ __align__(16) float hs[];           // ROUTE: [n] normed row, [experts] logits
  typedef uint32_t u4 __attribute__((ext_vector_type(4)));
  const int m = blockIdx.x, tid = threadIdx.x, ng = a.n / GW;
  const int lane = tid & 63, wave = tid >> 6;
  constexpr bool FEW = NT == 1024;
  constexpr int PF = 4;                                 // weight pieces (8 values per lane) of the wave's first expert in flight
  u4 gw[ROUTE ? PF : 1];
  if constexpr (ROUTE) {
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int k = 8 * lane + 512 * i;
      gw[i] = u4{0u, 0u, 0u, 0u};
      if (wave < a.experts && k < a.n) gw[i] = *reinterpret_cast<const u4*>(a.router + (int64_t)wave * a.n + k);
    }
  }
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
    const int gi = tid + NT * i, c = GW * (gi < ng ? gi : 0);
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
      const int gi = tid + NT * i, c = GW * (gi < ng ? gi : 0);
      float t[GW];
      if constexpr (FEW) ld_slabs<GW>(a, r, c, t);
      else ld_vals<GW>(a.ye + r * a.ldye + c, t);
#pragma unroll
      for (int e = 0; e < GW; ++e) y[i][e] = fmaf(wt, t[e], y[i][e]);
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int gi = tid + NT * i;
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
    const int gi = tid + NT * i, c = GW * gi;
    if (gi >= ng) continue;
    float o[GW];
#pragma unroll
    for (int e = 0; e < GW; ++e) o[e] = a.w ? normed(u[i][e], r, a.w, c + e, a.one_plus) : u[i][e];
    if (a.h) st_vals<GW>(a.h + (int64_t)m * a.ldh + c, o);
    if (a.h16) {
      if constexpr (GW == 4) {
        *reinterpret_cast<uint2*>(a.h16 + (int64_t)m * a.ldh16 + c) = make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
        if (FEW && a.h16_lo)
          *reinterpret_cast<uint2*>(a.h16_lo + (int64_t)m * a.ldh16 + c) =
              make_uint2(pack_bf16x2(low_part(o[0]), low_part(o[1])), pack_bf16x2(low_part(o[2]), low_part(o[3])));
      } else {
        a.h16[(int64_t)m * a.ldh16 + c] = f32_to_bf16(o[0]);
        if (FEW && a.h16_lo) a.h16_lo[(int64_t)m * a.ldh16 + c] = f32_to_bf16(low_part(o[0]));
      }
    }
    if constexpr (ROUTE) st_vals<GW>(hs + c, o);
  }
  if constexpr (ROUTE) {
    float* lg = hs + a.n;
    __syncthreads();
    for (int e = wave; e < a.experts; e += NT / 64) {
      const bf16_t* wr = a.router + (int64_t)e * a.n;
      float s = 0.f;
      auto piece = [&](u4 q, int k) {
        const float4 x = *reinterpret_cast<const float4*>(hs + k), y4 = *reinterpret_cast<const float4*>(hs + k + 4);
        s = fmaf(bf16lo_to_f32(q.x), x.x, s); s = fmaf(bf16hi_to_f32(q.x), x.y, s);
        s = fmaf(bf16lo_to_f32(q.y), x.z, s); s = fmaf(bf16hi_to_f32(q.y), x.w, s);
        s = fmaf(bf16lo_to_f32(q.z), y4.x, s); s = fmaf(bf16hi_to_f32(q.z), y4.y, s);
        s = fmaf(bf16lo_to_f32(q.w), y4.z, s); s = fmaf(bf16hi_to_f32(q.w), y4.w, s);
      };
      if (e != wave) {                                  // the next experts' first pieces
#pragma unroll
        for (int i = 0; i < PF; ++i) {
          const int k = 8 * lane + 512 * i;
          if (k < a.n) gw[i] = *reinterpret_cast<const u4*>(wr + k);
        }
      }
#pragma unroll
      for (int i = 0; i < PF; ++i) {
        const int k = 8 * lane + 512 * i;
        if (k < a.n) piece(gw[i], k);
      }
      for (int k = 8 * lane + 512 * PF; k < a.n; k += 512) piece(*reinterpret_cast<const u4*>(wr + k), k);
      s = wave_sum(s);
      if (lane == 0) lg[e] = s;
    }
    __syncthreads();
    if (wave == 0) wave_topk<true>(lg, a.experts, a.picks, lane, a.idx + (int64_t)m * a.picks, a.pw + (int64_t)m * a.picks);
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
      float t[1];
      ld_slabs<1>(a, r, c, t);
      y = fmaf(a.ew ? a.ew[z] : 1.0f, t[0], y);
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
      if (a.h16_lo) a.h16_lo[(int64_t)m * a.ldh16 + c] = f32_to_bf16(low_part(u));
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
    if (a.h16_lo) a.h16_lo[(int64_t)m * a.ldh16 + c] = f32_to_bf16(low_part(o));
  }
}

template <int S, int GW, bool ROUTE>
bool launch_streams(const mn_streams_args& a, int M, hipStream_t st) {
#define MN_ST(NV_, NT_) hipLaunchKernelGGL((streams_kernel<S, GW, NV_, NT_, ROUTE>), dim3((unsigned)M), dim3(NT_), lds, st, a)
  const size_t lds = ROUTE ? ((size_t)a.n + a.experts) * sizeof(float) : 0;
  if (M <= FEW_ROWS) {                                  // few rows: the row's latency is the launch
    const int per = (int)mn_cdiv(a.n / GW, 1024);
    if (per > 2) return false;
    if (per <= 1) MN_ST(1, 1024);
    else MN_ST(2, 1024);
    return true;
  }
  const int per = (int)mn_cdiv(a.n / GW, 256);
  if (per > 8 || a.h16_lo || a.ye_slabs > 1) return false;
  if (per <= 1) MN_ST(1, 256);
  else if (per <= 2) MN_ST(2, 256);
  else if (per <= 4) MN_ST(4, 256);
  else MN_ST(8, 256);
#undef MN_ST
  return true;
}

// P fp32 [nz][M][2 n] -> y bf16 [2][M][n] (high rows, then low rows) = silu(s gate) * (s up), s = x_scale[m]; four columns per thread
__global__ __launch_bounds__(256) void silu_split_kernel(const float* __restrict__ P, int nz, int M, int n, const float* __restrict__ x_scale,
                                                         bf16_t* __restrict__ y) {
  typedef float f4 __attribute__((ext_vector_type(4)));
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i >= (int64_t)M * n) return;
  const int m = (int)(i / n), c = (int)(i % n);
  const int64_t slab = (int64_t)M * 2 * n;
  const float* p = P + (int64_t)m * 2 * n + c;
  f4 g = *reinterpret_cast<const f4*>(p), u = *reinterpret_cast<const f4*>(p + n);
  for (int z = 1; z < nz; ++z) {
    g += *reinterpret_cast<const f4*>(p + z * slab);
    u += *reinterpret_cast<const f4*>(p + n + z * slab);
  }
  const float s = x_scale ? x_scale[m] : 1.0f;
  float o[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float gv = s * g[e];
    o[e] = gv / (1.0f + expf(-gv)) * (s * u[e]);
  }
  *reinterpret_cast<uint2*>(y + i) = make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
  *reinterpret_cast<uint2*>(y + (int64_t)M * n + i) =
      make_uint2(pack_bf16x2(low_part(o[0]), low_part(o[1])), pack_bf16x2(low_part(o[2]), low_part(o[3])));
}

}  // namespace

extern "C" size_t mn_sizeof_streams_args(void) { return sizeof(mn_streams_args); }

// whether the update can take the router of `experts` outputs along
extern "C" int mn_streams_router_ok(int M, int S, int n, int experts, const uint16_t* router) {
  return M >= 1 && S >= 1 && S <= 4 && n >= 8 && n <= ROUTE_MAX_N && (n % 8) == 0 && experts >= 1 &&
         experts <= (M <= FEW_ROWS ? ROUTE_MAX_EXPERTS : ROUTE_MAX_EXPERTS_MANY_ROWS) && router && (((uintptr_t)router) & 15) == 0;
}

extern "C" int mn_streams_update_norm(const mn_streams_args* p, int M, void* stream) {
  MN_CHECK_ARG(p && p->src && M >= 1 && p->n >= 1 && p->S >= 1 && p->S <= PLAIN_MAX_STREAMS && p->top >= 0 && p->src_row >= 0 && p->src_stream >= 0,
               "mn_streams_update_norm: bad args (1 .. %d streams)", PLAIN_MAX_STREAMS);
  const mn_streams_args a = *p;
  MN_CHECK_ARG((!a.mix || a.out) && (a.top == 0 || a.ye) && (a.mix || (!a.y && a.top == 0)) && (a.dst || a.h || a.h16),
               "mn_streams_update_norm: a result needs the mixing numbers; something must be written");
  MN_CHECK_ARG((!a.h || a.ldh >= a.n) && (!a.h16 || a.ldh16 >= a.n) && (!a.y || a.ldy >= a.n) && (a.top == 0 || a.ldye >= a.n) &&
                   (!a.h16_lo || a.h16) && a.ye_slabs >= 0,
               "mn_streams_update_norm: row strides below a row, or low parts without high ones");
  const uintptr_t al = (uintptr_t)a.src | (uintptr_t)a.dst | (uintptr_t)a.y | (uintptr_t)a.ye | (uintptr_t)a.h;
  const bool vec = (a.n % 4) == 0 && (al & 15) == 0 && ((((uintptr_t)a.h16) | ((uintptr_t)a.h16_lo)) & 7) == 0 && (a.src_row % 4) == 0 &&
                   (a.src_stream % 4) == 0 && (!a.y || (a.ldy % 4) == 0) && (a.top == 0 || ((a.ldye % 4) == 0 && (a.ye_slab % 4) == 0)) &&
                   (!a.h || (a.ldh % 4) == 0) && (!a.h16 || (a.ldh16 % 4) == 0);
  hipStream_t st = mn_stream(stream);
  if (a.router) {
    MN_CHECK_ARG(mn_streams_router_ok(M, a.S, a.n, a.experts, a.router) && vec && a.w && a.idx && a.pw && a.picks >= 1 && a.picks <= a.experts &&
                     (a.h || a.h16) && (M <= FEW_ROWS || (!a.h16_lo && a.ye_slabs <= 1)),
                 "mn_streams_update_norm: no router on rows like these (M=%d, n=%d, %d experts), or nothing to route", M, a.n, a.experts);
#define MN_R(S_) launch_streams<S_, 4, true>(a, M, st)
    switch (a.S) {
      case 1: MN_R(1); break;
      case 2: MN_R(2); break;
      case 3: MN_R(3); break;
      default: MN_R(4); break;
    }
#undef MN_R
    MN_CHECK_LAUNCH("mn_streams_update_norm(router)");
    return MN_OK;
  }
  bool done = false;
#define MN_S(S_) done = vec ? launch_streams<S_, 4, false>(a, M, st) : launch_streams<S_, 1, false>(a, M, st)
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

extern "C" int mn_silu_split_rows_scaled(const float* P, int nz, int M, int n, const float* x_scale, uint16_t* y, void* stream) {
  MN_CHECK_ARG(P && y && nz >= 1 && M >= 1 && n >= 4 && (n % 4) == 0 && (((uintptr_t)P) & 15) == 0 && (((uintptr_t)y) & 7) == 0,
               "mn_silu_split_rows_scaled: bad args (n=%d: a multiple of 4)", n);
  hipLaunchKernelGGL(silu_split_kernel, dim3((unsigned)mn_cdiv((int64_t)M * n, 1024)), dim3(256), 0, mn_stream(stream), P, nz, M, n, x_scale, y);
  MN_CHECK_LAUNCH("mn_silu_split_rows_scaled");
  return MN_OK;
}
