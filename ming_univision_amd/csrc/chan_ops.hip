// chan_ops.hip — operators of sequence-model layers whose recurrences decay per key channel (mingnative.h section 13).  Rows are fp32,
// weights bf16; everything here is fp32 arithmetic.
//   mn_add_layernorm_rows     x += y + sum_j w_j expert_j;  n = LayerNorm(x) w   (residual sum, expert combine and norm in one launch)
//   mn_xielu_rows             the two-sided quadratic / exponential activation
//   mn_token_table_rows       table rows chosen by token id (the experts of a table-routed mixture)
//   mn_low_rank_gate_rows     second stage of low-rank projections with the gate functions behind them
//   mn_rows_prep_launch       decode rows: the delta rule's preparation, the low-rank gates, the activation and the table rows in one launch
//   mn_channel_state_rows     S <- diag(g) S, then a delta-rule write or a plain k v^T, o = S^T q: prompt rows and decode rows
//   mn_gemv_glu_indexed       silu(gate) * up of the expert an index names
#include <math.h>

#include "common.h"
#include "delta_device.h"
#include "mfma_f32_tiles.h"

namespace {

// ---------------------------------------------------------------------------------------------------------------------------
// One workgroup per row with the row in registers: NV groups of GW consecutive values per thread.
struct AddLnArgs {
  float* x; int64_t ldx;
  const float* y; int64_t ldy;                 // optional sublayer result
  const float* ye; int64_t ldye;               // optional expert results, combined with ew (or the constant ew_all)
  const int32_t* slot_of; const float* ew; float ew_all; int top;
  const bf16_t* w; float eps;                  // w NULL: only the sum
  float* h; int64_t ldh; bf16_t* h16; int64_t ldh16;
  int n;
};

template <int GW>
__device__ __forceinline__ void ld_group(const float* p, float (&v)[GW]) {
  if constexpr (GW == 4) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
  } else {
    v[0] = *p;
  }
}

template <int GW, int NV>
__global__ __launch_bounds__(256) void add_ln_kernel(AddLnArgs a) {
  __shared__ float red[4];
  const int m = blockIdx.x, tid = threadIdx.x, ng = a.n / GW;
  float xv[NV][GW];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int gi = tid + 256 * i, c = GW * (gi < ng ? gi : 0);
    ld_group<GW>(a.x + (int64_t)m * a.ldx + c, xv[i]);
    if (a.y) {
      float t[GW];
      ld_group<GW>(a.y + (int64_t)m * a.ldy + c, t);
#pragma unroll
      for (int e = 0; e < GW; ++e) xv[i][e] += t[e];
    }
  }
  for (int j = 0; j < a.top; ++j) {
    const int z = m * a.top + j;
    const int64_t r = a.slot_of ? a.slot_of[z] : z;
    const float wt = a.ew ? a.ew[z] : a.ew_all;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int gi = tid + 256 * i, c = GW * (gi < ng ? gi : 0);
      float t[GW];
      ld_group<GW>(a.ye + r * a.ldye + c, t);
#pragma unroll
      for (int e = 0; e < GW; ++e) xv[i][e] = fmaf(wt, t[e], xv[i][e]);
    }
  }
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int gi = tid + 256 * i;
    if (gi >= ng) {
#pragma unroll
      for (int e = 0; e < GW; ++e) xv[i][e] = 0.f;
    }
#pragma unroll
    for (int e = 0; e < GW; ++e) s += xv[i][e];
    if (gi < ng && (a.y || a.top > 0)) {
#pragma unroll
      for (int e = 0; e < GW; ++e) a.x[(int64_t)m * a.ldx + GW * gi + e] = xv[i][e];
    }
  }
  if (!a.w) return;
  const float mean = block_sum(s, red) / (float)a.n;
  float q = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if (tid + 256 * i < ng) {
#pragma unroll
      for (int e = 0; e < GW; ++e) { const float d = xv[i][e] - mean; q = fmaf(d, d, q); }
    }
  const float r = 1.0f / sqrtf(block_sum(q, red) / (float)a.n + a.eps);
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int gi = tid + 256 * i;
    if (gi >= ng) continue;
    float o[GW];
#pragma unroll
    for (int e = 0; e < GW; ++e) o[e] = (xv[i][e] - mean) * r * bf16_to_f32(a.w[GW * gi + e]);
    if (a.h) {
#pragma unroll
      for (int e = 0; e < GW; ++e) a.h[(int64_t)m * a.ldh + GW * gi + e] = o[e];
    }
    if (a.h16) {
#pragma unroll
      for (int e = 0; e < GW; ++e) a.h16[(int64_t)m * a.ldh16 + GW * gi + e] = f32_to_bf16(o[e]);
    }
  }
}

// rows of any length: the summed row lies in x between the passes
__global__ __launch_bounds__(256) void add_ln_long_kernel(AddLnArgs a) {
  __shared__ float red[4];
  const int m = blockIdx.x, tid = threadIdx.x;
  float* xr = a.x + (int64_t)m * a.ldx;
  float s = 0.f;
  for (int c = tid; c < a.n; c += 256) {
    float v = xr[c];
    if (a.y) v += a.y[(int64_t)m * a.ldy + c];
    for (int j = 0; j < a.top; ++j) {
      const int z = m * a.top + j;
      const int64_t r = a.slot_of ? a.slot_of[z] : z;
      v = fmaf(a.ew ? a.ew[z] : a.ew_all, a.ye[r * a.ldye + c], v);
    }
    if (a.y || a.top > 0) xr[c] = v;              // every thread rereads only what it wrote itself
    s += v;
  }
  if (!a.w) return;
  const float mean = block_sum(s, red) / (float)a.n;
  float q = 0.f;
  for (int c = tid; c < a.n; c += 256) { const float d = xr[c] - mean; q = fmaf(d, d, q); }
  const float r = 1.0f / sqrtf(block_sum(q, red) / (float)a.n + a.eps);
  for (int c = tid; c < a.n; c += 256) {
    const float o = (xr[c] - mean) * r * bf16_to_f32(a.w[c]);
    if (a.h) a.h[(int64_t)m * a.ldh + c] = o;
    if (a.h16) a.h16[(int64_t)m * a.ldh16 + c] = f32_to_bf16(o);
  }
}

// ---------------------------------------------------------------------------------------------------------------------------
// z > 0: ap z^2 + z / 2;  z <= 0: an (exp(z) - 1 - z) + z / 2
struct XieluArgs {
  const float* x; int64_t ldx;
  float ap, an;
  float* y; int64_t ldy; bf16_t* y16; int64_t ldy16;
  int M, n;
};

__device__ __forceinline__ float xielu(float z, float ap, float an) {
  return (z > 0.f ? ap * z * z : an * (expm1f(z) - z)) + 0.5f * z;
}

// four consecutive columns per thread: block b of the row's ceil(n / 1024)
__device__ __forceinline__ void xielu_block(const XieluArgs& a, int m, int b, int tid) {
  const int c0 = (b * 256 + tid) * 4;
  if (c0 >= a.n) return;
  const float* xr = a.x + (int64_t)m * a.ldx + c0;
  const bool full = c0 + 4 <= a.n;
  float v[4];
  if (full && (((uintptr_t)xr) & 15) == 0) {
    ld_group<4>(xr, v);
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = c0 + e < a.n ? xr[e] : 0.f;
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = xielu(v[e], a.ap, a.an);
  if (a.y) {
    float* yr = a.y + (int64_t)m * a.ldy + c0;
    if (full && (((uintptr_t)yr) & 15) == 0) {
      *reinterpret_cast<float4*>(yr) = make_float4(v[0], v[1], v[2], v[3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) if (c0 + e < a.n) yr[e] = v[e];
    }
  }
  if (a.y16) {
    bf16_t* yr = a.y16 + (int64_t)m * a.ldy16 + c0;
    if (full && (((uintptr_t)yr) & 7) == 0) {
      *reinterpret_cast<uint2*>(yr) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) if (c0 + e < a.n) yr[e] = f32_to_bf16(v[e]);
    }
  }
}

__global__ __launch_bounds__(256) void xielu_kernel(XieluArgs a) { xielu_block(a, blockIdx.y, blockIdx.x, threadIdx.x); }

// idx[m, j] = table[tok[m], j], w[m, j] = 1 / top; a token outside the table reads its nearest row
__global__ __launch_bounds__(256) void token_table_kernel(const int32_t* __restrict__ table, int vocab, int top, const int32_t* __restrict__ tok,
                                                          int M, int32_t* __restrict__ idx, float* __restrict__ w) {
  const int e = blockIdx.x * 256 + threadIdx.x;
  if (e >= M * top) return;
  const int m = e / top, t = min(max(tok[m], 0), vocab - 1);
  idx[e] = table[(int64_t)t * top + (e - m * top)];
  if (w) w[e] = 1.0f / (float)top;
}

// ---------------------------------------------------------------------------------------------------------------------------
// Low-rank gates: out[m, n] = f(sum_k w[n, k] a[m, k] + bias[n]) with f by job (MN_LOW_RANK_*).  Up to two jobs share a launch.
struct LowRankArgs {
  mn_low_rank_job job[2];
  int M, nb0;                                  // workgroups (along x) of job 0
};

__device__ __forceinline__ float gate_value(const mn_low_rank_job& j, int n, float z) {
  if (j.bias) z += bf16_to_f32(j.bias[n]);
  if (j.kind == MN_LOW_RANK_DECAY) return expf(-expf(j.a_log[n / j.head_n]) * softplus_f(z));
  if (j.kind == MN_LOW_RANK_ROOT) return expf(-softplus_f(-z) * j.root);           // sigmoid(z)^root
  if (j.kind == MN_LOW_RANK_SIGMOID) return sigmoid_f(z);
  return z;
}

// Few rows: 8 lanes per output (32 outputs a workgroup), up to 8 rows of a together; lane s finishes row s.
constexpr int LR_ROWS = 8;
__device__ __forceinline__ void low_rank_few(const LowRankArgs& a, int bx, int by, int tid) {
  const bool second = bx >= a.nb0;
  const mn_low_rank_job& j = a.job[second ? 1 : 0];
  const int n = (bx - (second ? a.nb0 : 0)) * 32 + (tid >> 3), s = tid & 7, m0 = by * LR_ROWS, rows = min(LR_ROWS, a.M - m0);
  const int nn = min(n, j.n - 1);
  const bf16_t* wr = j.w + (int64_t)nn * j.k;
  const bool vec = (j.k & 7) == 0 && (j.lda & 3) == 0 && (((uintptr_t)j.w | (uintptr_t)j.a) & 15) == 0;
  float acc[LR_ROWS];
#pragma unroll
  for (int r = 0; r < LR_ROWS; ++r) acc[r] = 0.f;
  for (int k0 = 8 * s; k0 < j.k; k0 += 64) {
    float wv[8];
    if (vec) {
      const uint4 q = *reinterpret_cast<const uint4*>(wr + k0);
      wv[0] = bf16lo_to_f32(q.x); wv[1] = bf16hi_to_f32(q.x); wv[2] = bf16lo_to_f32(q.y); wv[3] = bf16hi_to_f32(q.y);
      wv[4] = bf16lo_to_f32(q.z); wv[5] = bf16hi_to_f32(q.z); wv[6] = bf16lo_to_f32(q.w); wv[7] = bf16hi_to_f32(q.w);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) wv[e] = k0 + e < j.k ? bf16_to_f32(wr[k0 + e]) : 0.f;
    }
#pragma unroll
    for (int r = 0; r < LR_ROWS; ++r) {
      if (r >= rows) break;
      const float* ar = j.a + (int64_t)(m0 + r) * j.lda + k0;
      if (vec) {
        float t[4], u[4];
        ld_group<4>(ar, t);
        ld_group<4>(ar + 4, u);
#pragma unroll
        for (int e = 0; e < 4; ++e) { acc[r] = fmaf(wv[e], t[e], acc[r]); acc[r] = fmaf(wv[4 + e], u[e], acc[r]); }
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[r] = fmaf(wv[e], k0 + e < j.k ? ar[e] : 0.f, acc[r]);
      }
    }
  }
  float mine = 0.f;
#pragma unroll
  for (int r = 0; r < LR_ROWS; ++r) {
    const float t = sum8(acc[r]);
    if (r == s) mine = t;
  }
  if (n < j.n && s < rows) j.out[(int64_t)(m0 + s) * j.ldo + n] = gate_value(j, n, mine);
}

__global__ __launch_bounds__(256) void low_rank_few_kernel(LowRankArgs a) { low_rank_few(a, blockIdx.x, blockIdx.y, threadIdx.x); }

// Decode rows: everything between the stacked product and the recurrence.  blockIdx.x runs over the parts (delta units | low-rank outputs |
// activation | table), blockIdx.y over the rows (low-rank: over groups of LR_ROWS rows).
struct RowsPrepArgs {
  DeltaPrepArgs delta;
  LowRankArgs lr;
  XieluArgs act;
  const int32_t *table, *tok; int vocab, top; int32_t* idx;
  int M, n_delta, n_lr, n_act;                 // workgroups of the first three parts
};
__global__ __launch_bounds__(256) void rows_prep_kernel(RowsPrepArgs a) {
  const int m = blockIdx.y, tid = threadIdx.x;
  int b = blockIdx.x;
  if (b < a.n_delta) {
    delta_prep_unit(a.delta, m, b * 4 + (tid >> 6), tid & 63, 0);
    if (b == 0) delta_prep_strengths(a.delta, m, tid);
    return;
  }
  b -= a.n_delta;
  if (b < a.n_lr) {
    if (m * LR_ROWS < a.M) low_rank_few(a.lr, b, m, tid);
    return;
  }
  b -= a.n_lr;
  if (b < a.n_act) {
    xielu_block(a.act, m, b, tid);
    return;
  }
  for (int j = tid; j < a.top; j += 256) a.idx[m * a.top + j] = a.table[(int64_t)min(max(a.tok[m], 0), a.vocab - 1) * a.top + j];
}

// Many rows: 64 x 64 output tiles on the fp32 matrix cores (v_mfma_f32_16x16x4_f32; operand layouts in mfma_f32_tiles.h), k in pieces
// of 32 staged as fp32; wave w owns 16 rows x 64 columns.
__global__ __launch_bounds__(256) void low_rank_mfma_kernel(LowRankArgs a) {
  constexpr int KC = 32, LD = KC + 4;
  __shared__ float As[64 * LD], Ws[64 * LD];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const bool second = (int)blockIdx.x >= a.nb0;
  const mn_low_rank_job& j = a.job[second ? 1 : 0];
  const int n0 = ((int)blockIdx.x - (second ? a.nb0 : 0)) * 64, m0 = blockIdx.y * 64;
  f32x4 acc[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) acc[c] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < j.k; k0 += KC) {
    __syncthreads();
#pragma unroll
    for (int t = 0; t < 64 * KC / 256; ++t) {
      const int e = tid + 256 * t, r = e / KC, k = k0 + e % KC, m = min(m0 + r, a.M - 1), n = min(n0 + r, j.n - 1);
      As[r * LD + e % KC] = k < j.k ? j.a[(int64_t)m * j.lda + k] : 0.f;
      Ws[r * LD + e % KC] = k < j.k ? bf16_to_f32(j.w[(int64_t)n * j.k + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int it = 0; it < KC / 4; ++it) {
      const float av = As[(16 * wave + c16) * LD + 4 * it + g4];
#pragma unroll
      for (int c = 0; c < 4; ++c) acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, Ws[(16 * c + c16) * LD + 4 * it + g4], acc[c], 0, 0, 0);
    }
  }
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const int n = n0 + 16 * c + c16;
    if (n >= j.n) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int m = m0 + 16 * wave + 4 * g4 + i;
      if (m < a.M) j.out[(int64_t)m * j.ldo + n] = gate_value(j, n, acc[c][i]);
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------------
// Recurrence with a decay per key channel.  Every value column of a head's state is a recurrence of its own: with s = S[:, c]
//   s_i <- g_i s_i;   u = DELTA ? beta (v_c - s . k) : v_c;   s <- s + k u;   o_c = s . q = (g s_old) . q + u (k . q)
struct ChanArgs {
  const float* qkv; int64_t ld;              // per row [q: G dim ; k: G dim ; v: H vdim]
  const float* g; int64_t ldg;               // per row [H dim]
  const float* beta; int64_t ldb;            // per row [H] (DELTA)
  int H, G, dim, vdim;
  float o_scale;
  float* state;                              // [n_seq, H, dim, vdim]
  const int32_t *row_seq, *row_slot, *row_back;
  const int32_t* blk_tab;                    // optional: runs of rows; a sequence's first row in the call starts a run
  float* out; int64_t ldo;                   // [M, H vdim]
  int M;
  const int32_t* chunk_tab; float* ws; float* wsp;      // scan: chunks of rows; [n_chunks, H, dim, vdim] states; [n_chunks, H, dim] decay products
};

template <int LPC>
__device__ __forceinline__ float lanes_sum(float v) { return LPC == 16 ? row16_sum(v) : sum8(v); }

// Prompt rows, heads of at most NS LPC state rows: the workgroup of a sequence's FIRST row in the call walks that sequence's rows.  LPC
// lanes share C neighbouring value columns (NT / LPC * C columns a workgroup); a lane holds the state rows 4 (s + LPC jj) + t, t < 4,
// jj < NS / 4, in registers.  Rows come in batches of DBT: a batch's q, k, g, v and write strengths go global -> registers (while the
// previous batch is computed) -> LDS; the steps then run from LDS and registers alone, the operands of step r + 1 requested ahead of
// step r, without a barrier or a memory access between steps.  Only the sum that the write needs (s . k) is reduced within a step; the
// read-outs' partial sums s . q go to LDS lane by lane and are added up once per batch.  LDS rows are padded with zeros to DP values,
// under which padded state rows stay 0.
//   MODE WALK       from the sequence's state to its state
//   MODE CHUNK_END  a workgroup per CHUNK of rows: from zero, no outputs; the chunk's end state and its decay product per key channel
//   MODE CHUNK_OUT  a workgroup per chunk: from the chunk's start state in the workspace, outputs only
enum { WALK = 0, CHUNK_END = 1, CHUNK_OUT = 2 };
template <int NS, int LPC, int C, int NT, int DBT, bool DELTA, bool VEC, int MODE>
__global__ __launch_bounds__(NT) void chan_walk_kernel(ChanArgs a) {
  constexpr int CPB = NT / LPC * C, DP = NS * LPC, Q4 = DBT * DP / 4 / NT, NV = (DBT * CPB + NT - 1) / NT, PS = LPC + 4, NP = (DP + NT - 1) / NT;
  constexpr bool OUT = MODE != CHUNK_END;
  static_assert(Q4 * 4 * NT == DBT * DP && DBT <= NT && DBT % 2 == 0, "a batch is staged by whole 16-byte pieces per thread");
  static_assert(!DELTA || MODE == WALK, "the delta rule's write needs the state before it");
  __shared__ __align__(16) float opl[3][DBT][DP];             // q, k, g
  __shared__ __align__(16) float vs[DBT][CPB];
  __shared__ __align__(16) float part[OUT ? DBT * CPB * PS : 4];   // s . q by lanes
  __shared__ float us[DELTA ? DBT : 1][CPB];                  // what each step wrote
  __shared__ float bs[2][DBT];                                // beta, k . q
  const int m0 = MODE != WALK ? a.chunk_tab[2 * blockIdx.y] : (a.blk_tab ? a.blk_tab[2 * blockIdx.y] : blockIdx.y);
  if (MODE == WALK && a.row_back[m0] != 0) return;
  const int ncb = (a.vdim + CPB - 1) / CPB, h = blockIdx.x / ncb, cb = blockIdx.x - h * ncb;
  const int tid = threadIdx.x, s = tid % LPC, cl = tid / LPC, c = cb * CPB + C * cl;
  const int d = a.dim, kvh = h / (a.H / a.G);
  int n = 1;
  if (MODE == WALK) {
    for (;;) {
      const int m = m0 + n + tid;
      const int cnt = __syncthreads_count(m < a.M && a.row_back[m] == m - m0);
      n += cnt;
      if (cnt < NT) break;
    }
  } else {
    n = a.chunk_tab[2 * blockIdx.y + 1];
  }
  const int64_t hde = (int64_t)d * a.vdim;
  float* sp = MODE == WALK ? a.state + ((int64_t)a.row_seq[m0] * a.H + h) * hde : a.ws + ((int64_t)blockIdx.y * a.H + h) * hde;
  const bool fresh = MODE == CHUNK_END || (MODE == WALK && a.row_slot[m0] == 0);
  float S[C][NS];
#pragma unroll
  for (int cc = 0; cc < C; ++cc)
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      const int i = 4 * (s + LPC * (j >> 2)) + (j & 3);
      S[cc][j] = (c + cc < a.vdim && !fresh && i < d) ? sp[(int64_t)i * a.vdim + c + cc] : 0.f;
    }
  __syncthreads();                             // the state has arrived: from here on only a batch's loads are in flight
  float gp[NP];
#pragma unroll
  for (int t = 0; t < NP; ++t) gp[t] = 1.f;
  f32x4 rq[3][Q4];
  float rv[NV], rb = 0.f;
  const float* const src0[3] = {a.qkv + (int64_t)kvh * d, a.qkv + (int64_t)(a.G + kvh) * d, a.g + (int64_t)h * d};
  const int64_t lds_[3] = {a.ld, a.ld, a.ldg};
  const float* const srcv = a.qkv + (int64_t)2 * a.G * d + (int64_t)h * a.vdim;
  // raw loads at clamped addresses; what does not count is replaced when the batch goes to LDS
  auto fetch = [&](int b0) {
#pragma unroll
    for (int t = 0; t < Q4; ++t) {
      const int e = tid + NT * t, r = e / (DP / 4), i = 4 * (e % (DP / 4));
      const int64_t m = m0 + min(b0 + r, n - 1);
#pragma unroll
      for (int w = OUT ? 0 : 1; w < 3; ++w) {
        const float* src = src0[w] + m * lds_[w];
        if constexpr (VEC) {
          rq[w][t] = *reinterpret_cast<const f32x4*>(src + min(i, d - 4));
        } else {
#pragma unroll
          for (int u = 0; u < 4; ++u) rq[w][t][u] = src[min(i + u, d - 1)];
        }
      }
    }
#pragma unroll
    for (int t = 0; t < NV; ++t) {
      const int e = tid + NT * t, r = e / CPB, cc = cb * CPB + e % CPB;
      rv[t] = srcv[(m0 + min(b0 + r, n - 1)) * a.ld + min(cc, a.vdim - 1)];
    }
    if (DELTA) rb = a.beta[(int64_t)(m0 + min(b0 + tid % DBT, n - 1)) * a.ldb + h];
  };
  fetch(0);
  for (int b0 = 0; b0 < n; b0 += DBT) {
    const int rows = min(DBT, n - b0);
    lds_barrier();                             // the previous batch's sums have been taken
    // rows past the sequence: no decay, no key — the state passes them unchanged
#pragma unroll
    for (int t = 0; t < Q4; ++t) {
      const int e = tid + NT * t, r = e / (DP / 4), i = 4 * (e % (DP / 4));
      const float pad[3] = {0.f, 0.f, r < rows ? 0.f : 1.f};
#pragma unroll
      for (int w = OUT ? 0 : 1; w < 3; ++w) {
        f32x4 x = rq[w][t];
#pragma unroll
        for (int u = 0; u < 4; ++u) x[u] = (r < rows && i + u < d) ? x[u] : pad[w];
        *reinterpret_cast<f32x4*>(&opl[w][r][i]) = x;
      }
    }
#pragma unroll
    for (int t = 0; t < NV; ++t) { const int e = tid + NT * t; if (e < DBT * CPB) (&vs[0][0])[e] = rv[t]; }
    if (DELTA && tid < DBT) bs[0][tid] = rb;
    lds_barrier();
    if (b0 + DBT < n) fetch(b0 + DBT);         // in flight while this batch is computed
    if (DELTA) {                               // k . q of every row: 16 threads a row
      for (int r = tid >> 4; r < DBT; r += NT / 16) {
        float t = 0.f;
#pragma unroll
        for (int i = tid & 15; i < DP; i += 16) t = fmaf(opl[0][r][i], opl[1][r][i], t);
        t = row16_sum(t);
        if ((tid & 15) == 0) bs[1][r] = t;
      }
    }
    if (MODE == CHUNK_END && cb == 0) {        // the channels' decay over the chunk
#pragma unroll
      for (int t = 0; t < NP; ++t)
        if (tid + NT * t < DP)
          for (int r = 0; r < DBT; ++r) gp[t] *= opl[2][r][tid + NT * t];
    }
    struct Row { float q[NS], k[NS], g[NS], v[C], beta; } A, B;
    auto load_row = [&](int r, Row& x) {
#pragma unroll
      for (int jj = 0; jj < NS / 4; ++jj) {
        const int i = 4 * (s + LPC * jj);
        const f32x4 k4 = *reinterpret_cast<const f32x4*>(&opl[1][r][i]), g4 = *reinterpret_cast<const f32x4*>(&opl[2][r][i]);
#pragma unroll
        for (int u = 0; u < 4; ++u) { x.k[4 * jj + u] = k4[u]; x.g[4 * jj + u] = g4[u]; }
        if (OUT) {
          const f32x4 q4 = *reinterpret_cast<const f32x4*>(&opl[0][r][i]);
#pragma unroll
          for (int u = 0; u < 4; ++u) x.q[4 * jj + u] = q4[u];
        }
      }
#pragma unroll
      for (int cc = 0; cc < C; ++cc) x.v[cc] = vs[r][C * cl + cc];
      if (DELTA) x.beta = bs[0][r];
    };
    auto step = [&](int r, const Row& x) {
#pragma unroll
      for (int cc = 0; cc < C; ++cc) {
        float q0 = 0.f, q1 = 0.f;
        if (DELTA) {
#pragma unroll
          for (int j = 0; j < NS; ++j) S[cc][j] *= x.g[j];
          float k0 = S[cc][0] * x.k[0], k1 = S[cc][1] * x.k[1];
#pragma unroll
          for (int j = 2; j < NS; j += 2) { k0 = fmaf(S[cc][j], x.k[j], k0); k1 = fmaf(S[cc][j + 1], x.k[j + 1], k1); }
          const float pk = lanes_sum<LPC>(k0 + k1);
          q0 = S[cc][0] * x.q[0]; q1 = S[cc][1] * x.q[1];
#pragma unroll
          for (int j = 2; j < NS; j += 2) { q0 = fmaf(S[cc][j], x.q[j], q0); q1 = fmaf(S[cc][j + 1], x.q[j + 1], q1); }
          const float u = x.beta * (x.v[cc] - pk);
#pragma unroll
          for (int j = 0; j < NS; ++j) S[cc][j] = fmaf(x.k[j], u, S[cc][j]);
          if (s == 0) us[r][C * cl + cc] = u;
        } else {
#pragma unroll
          for (int j = 0; j < NS; ++j) S[cc][j] = fmaf(x.g[j], S[cc][j], x.k[j] * x.v[cc]);
          if (OUT) {
            q0 = S[cc][0] * x.q[0]; q1 = S[cc][1] * x.q[1];
#pragma unroll
            for (int j = 2; j < NS; j += 2) { q0 = fmaf(S[cc][j], x.q[j], q0); q1 = fmaf(S[cc][j + 1], x.q[j + 1], q1); }
          }
        }
        if (OUT) part[(r * CPB + C * cl + cc) * PS + s] = q0 + q1;
      }
    };
    // two rows per turn, each row's operands requested one step ahead
    load_row(0, A);
    for (int r = 0; r < rows; r += 2) {
      load_row(r + 1, B);
      step(r, A);
      load_row(min(r + 2, DBT - 2), A);
      step(r + 1, B);
    }
    if (!OUT) continue;
    lds_barrier();
#pragma unroll
    for (int t = 0; t < NV; ++t) {             // the batch's outputs, a row's columns side by side
      const int e = tid + NT * t, r = e / CPB, cc = cb * CPB + e % CPB;
      if (r < rows && cc < a.vdim) {
        f32x4 o = *reinterpret_cast<const f32x4*>(&part[e * PS]);
#pragma unroll
        for (int w = 1; w < LPC / 4; ++w) o += *reinterpret_cast<const f32x4*>(&part[e * PS + 4 * w]);
        float v = (o[0] + o[1]) + (o[2] + o[3]);
        if (DELTA) v = fmaf(us[r][e % CPB], bs[1][r], v);
        a.out[(int64_t)(m0 + b0 + r) * a.ldo + (int64_t)h * a.vdim + cc] = v * a.o_scale;
      }
    }
  }
  if (MODE == CHUNK_OUT) return;
  if (MODE == CHUNK_END && cb == 0) {
#pragma unroll
    for (int t = 0; t < NP; ++t)
      if (tid + NT * t < d) a.wsp[((int64_t)blockIdx.y * a.H + h) * d + tid + NT * t] = gp[t];
  }
#pragma unroll
  for (int cc = 0; cc < C; ++cc) {
    if (c + cc >= a.vdim) continue;
#pragma unroll
    for (int j = 0; j < NS; ++j) {
      const int i = 4 * (s + LPC * (j >> 2)) + (j & 3);
      if (i < d) sp[(int64_t)i * a.vdim + c + cc] = S[cc][j];
    }
  }
}

// The carry between the chunk passes: grid (ceil(dim vdim / 256), H, n_chunks); the workgroup of a sequence's first chunk in the call turns
// that sequence's end states into start states, S <- P S + E, and leaves the last state in the arena.
__global__ __launch_bounds__(256) void chan_carry_kernel(ChanArgs a, int n_chunks) {
  const int x = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, c0 = blockIdx.z, de = a.dim * a.vdim, i = x / a.vdim;
  const int r0 = a.chunk_tab[2 * c0];
  if (a.row_back[r0] != 0 || x >= de) return;
  float* sp = a.state + ((int64_t)a.row_seq[r0] * a.H + h) * de + x;
  float S = a.row_slot[r0] == 0 ? 0.f : *sp;
  float* w = a.ws + ((int64_t)c0 * a.H + h) * de + x;
  const float* p = a.wsp + ((int64_t)c0 * a.H + h) * a.dim + i;
  const int64_t sw = (int64_t)a.H * de, spd = (int64_t)a.H * a.dim;
  constexpr int PRE = 4;                       // chunks whose states are requested together
  for (int ch = c0; ch < n_chunks;) {
    float E[PRE], P[PRE];
    int cnt = 0;
#pragma unroll
    for (int t = 0; t < PRE; ++t) {
      const int cc = min(ch + t, n_chunks - 1);
      if (cnt == t && ch + t < n_chunks && (ch + t == c0 || a.row_back[a.chunk_tab[2 * cc]] != 0)) cnt = t + 1;    // the next sequence ends the run
      E[t] = w[(int64_t)min(t, n_chunks - 1 - ch) * sw];
      P[t] = p[(int64_t)min(t, n_chunks - 1 - ch) * spd];
    }
#pragma unroll
    for (int t = 0; t < PRE; ++t)
      if (t < cnt) {
        w[(int64_t)t * sw] = S;
        S = fmaf(P[t], S, E[t]);
      }
    if (cnt < PRE) break;
    ch += PRE; w += PRE * sw; p += PRE * spd;
  }
  *sp = S;
}

// The same walk for any head size, the state staying in the arena: grid (ceil(vdim / 32), H, rows or runs), 8 lanes per column.
template <bool DELTA>
__global__ __launch_bounds__(256) void chan_walk_any_kernel(ChanArgs a) {
  extern __shared__ float lds[];             // q, k, g of the row
  const int m0 = a.blk_tab ? a.blk_tab[2 * blockIdx.z] : blockIdx.z;
  if (a.row_back && a.row_back[m0] != 0) return;
  const int h = blockIdx.y, tid = threadIdx.x, s = tid & 7, c = blockIdx.x * 32 + (tid >> 3), d = a.dim, kvh = h / (a.H / a.G);
  const bool on = c < a.vdim;
  float* sp = a.state + (((int64_t)a.row_seq[m0] * a.H + h) * d) * a.vdim + (on ? c : 0);
  if (a.row_slot[m0] == 0 && on)
    for (int i = s; i < d; i += 8) sp[(int64_t)i * a.vdim] = 0.f;
  for (int m = m0; m < a.M && (m == m0 || (a.row_back && a.row_back[m] == m - m0)); ++m) {
    const float* row = a.qkv + (int64_t)m * a.ld;
    __syncthreads();
    for (int i = tid; i < d; i += 256) {
      lds[i] = row[(int64_t)kvh * d + i];
      lds[d + i] = row[(int64_t)(a.G + kvh) * d + i];
      lds[2 * d + i] = a.g[(int64_t)m * a.ldg + (int64_t)h * d + i];
    }
    const float v = on ? row[(int64_t)2 * a.G * d + (int64_t)h * a.vdim + c] : 0.f;
    __syncthreads();
    float pk = 0.f, pq = 0.f, kq = 0.f;
    for (int i = s; i < d; i += 8) {
      const float sv = on ? lds[2 * d + i] * sp[(int64_t)i * a.vdim] : 0.f;
      pk = fmaf(sv, lds[d + i], pk);
      pq = fmaf(sv, lds[i], pq);
      kq = fmaf(lds[d + i], lds[i], kq);
    }
    pk = sum8(pk); pq = sum8(pq); kq = sum8(kq);
    const float u = DELTA ? a.beta[(int64_t)m * a.ldb + h] * (v - pk) : v;
    if (on) {
      for (int i = s; i < d; i += 8) sp[(int64_t)i * a.vdim] = fmaf(lds[d + i], u, lds[2 * d + i] * sp[(int64_t)i * a.vdim]);
      if (s == 0) a.out[(int64_t)m * a.ldo + (int64_t)h * a.vdim + c] = fmaf(u, kq, pq) * a.o_scale;
    }
  }
}

// Decode rows (every row alone in its sequence): grid (M, H, ceil(vdim / 32)); a workgroup owns 32 value columns of one head's state, its
// 8 groups of 32 threads hold the state's rows sub, sub + 8, .. in registers (NR of them), partial dot products meet in LDS.
template <int NR, bool DELTA>
__global__ __launch_bounds__(256) void chan_step_kernel(ChanArgs a) {
  extern __shared__ float lds[];             // q, k, g [3][dim]; partial sums [3][8][32]
  const int m = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, cl = tid & 31, sub = tid >> 5, c = blockIdx.z * 32 + cl;
  const int d = a.dim, kvh = h / (a.H / a.G);
  const float* row = a.qkv + (int64_t)m * a.ld;
  const bool on = c < a.vdim;
  const bool fresh = a.row_slot[m] == 0;
  float* sp = a.state + (((int64_t)a.row_seq[m] * a.H + h) * d) * a.vdim + (on ? c : 0);
  float S[NR];
#pragma unroll
  for (int t = 0; t < NR; ++t) {
    const int i = sub + 8 * t;
    const float v = sp[(int64_t)(i < d ? i : 0) * a.vdim];       // a readable address; what does not count is zeroed
    S[t] = (on && !fresh && i < d) ? v : 0.f;
  }
  for (int i = tid; i < d; i += 256) {
    lds[i] = row[(int64_t)kvh * d + i];
    lds[d + i] = row[(int64_t)(a.G + kvh) * d + i];
    lds[2 * d + i] = a.g[(int64_t)m * a.ldg + (int64_t)h * d + i];
  }
  const float v = on ? row[(int64_t)2 * a.G * d + (int64_t)h * a.vdim + c] : 0.f;
  const float beta = DELTA ? a.beta[(int64_t)m * a.ldb + h] : 0.f;
  float* part = lds + 3 * d;
  __syncthreads();
  float pk = 0.f, pq = 0.f, kq = 0.f;
#pragma unroll
  for (int t = 0; t < NR; ++t) {
    const int i = sub + 8 * t;
    if (i < d) {
      const float q = lds[i], k = lds[d + i];
      S[t] *= lds[2 * d + i];
      pq = fmaf(S[t], q, pq);
      if (DELTA) pk = fmaf(S[t], k, pk);
      kq = fmaf(k, q, kq);
    }
  }
  part[sub * 32 + cl] = pq; part[256 + sub * 32 + cl] = kq;
  if (DELTA) part[512 + sub * 32 + cl] = pk;
  __syncthreads();
  pk = pq = kq = 0.f;
#pragma unroll
  for (int t = 0; t < 8; ++t) {
    pq += part[t * 32 + cl]; kq += part[256 + t * 32 + cl];
    if (DELTA) pk += part[512 + t * 32 + cl];
  }
  const float u = DELTA ? beta * (v - pk) : v;
  if (!on) return;
#pragma unroll
  for (int t = 0; t < NR; ++t) {
    const int i = sub + 8 * t;
    if (i < d) sp[(int64_t)i * a.vdim] = fmaf(lds[d + i], u, S[t]);
  }
  if (sub == 0) a.out[(int64_t)m * a.ldo + (int64_t)h * a.vdim + c] = fmaf(u, kq, pq) * a.o_scale;
}

bool chan_vec(const ChanArgs& a) {
  return (a.dim & 3) == 0 && (a.ld & 3) == 0 && (a.ldg & 3) == 0 && (((uintptr_t)a.qkv | (uintptr_t)a.g) & 15) == 0;
}

template <bool DELTA>
int chan_rows(const ChanArgs& a, bool distinct, int n_runs, hipStream_t st) {
  const int d = a.dim;
  if (distinct && d <= 512) {
    const dim3 grid((unsigned)a.M, (unsigned)a.H, (unsigned)mn_cdiv(a.vdim, 32));
    const size_t lds = ((size_t)3 * d + 768) * sizeof(float);
    if (d <= 32) hipLaunchKernelGGL((chan_step_kernel<4, DELTA>), grid, dim3(256), lds, st, a);
    else if (d <= 64) hipLaunchKernelGGL((chan_step_kernel<8, DELTA>), grid, dim3(256), lds, st, a);
    else if (d <= 128) hipLaunchKernelGGL((chan_step_kernel<16, DELTA>), grid, dim3(256), lds, st, a);
    else if (d <= 256) hipLaunchKernelGGL((chan_step_kernel<32, DELTA>), grid, dim3(256), lds, st, a);
    else hipLaunchKernelGGL((chan_step_kernel<64, DELTA>), grid, dim3(256), lds, st, a);
    MN_CHECK_LAUNCH("mn_channel_state_rows(step)");
    return MN_OK;
  }
  if (!distinct && d <= 256) {
    const bool vec = chan_vec(a);
#define MN_CW(NS_, LPC_, NT_, DB_)                                                                                                         \
  do {                                                                                                                                     \
    const dim3 grid((unsigned)(a.H * mn_cdiv(a.vdim, NT_ / LPC_)), (unsigned)n_runs);                                                     \
    if (vec) hipLaunchKernelGGL((chan_walk_kernel<NS_, LPC_, 1, NT_, DB_, DELTA, true, WALK>), grid, dim3(NT_), 0, st, a);                \
    else hipLaunchKernelGGL((chan_walk_kernel<NS_, LPC_, 1, NT_, DB_, DELTA, false, WALK>), grid, dim3(NT_), 0, st, a);                   \
  } while (0)
    if (d <= 32) MN_CW(4, 8, 128, 16); else if (d <= 64) MN_CW(4, 16, 128, 16); else if (d <= 128) MN_CW(8, 16, 128, 16); else MN_CW(16, 16, 128, 8);
#undef MN_CW
    MN_CHECK_LAUNCH("mn_channel_state_rows(walk)");
    return MN_OK;
  }
  hipLaunchKernelGGL((chan_walk_any_kernel<DELTA>), dim3((unsigned)mn_cdiv(a.vdim, 32), (unsigned)a.H, (unsigned)n_runs), dim3(256),
                     (size_t)3 * d * sizeof(float), st, a);
  MN_CHECK_LAUNCH("mn_channel_state_rows(any)");
  return MN_OK;
}

// ---------------------------------------------------------------------------------------------------------------------------
// one wave per output: act[z, n] = silu(W_i[n] . a) * (W_i[N + n] . a), i = w_idx[z].  VEC as in mn_gemv_f32_indexed.
template <bool VEC>
__global__ __launch_bounds__(256) void gemv_glu_indexed_kernel(const float* __restrict__ A, int64_t lda, int a_div, const bf16_t* __restrict__ W,
                                                               int64_t ldw, int64_t w_bs, const int32_t* __restrict__ w_idx, int n_idx,
                                                               float* __restrict__ C, int64_t ldc, int N, int K,
                                                               const float* __restrict__ x_scale) {
  const int z = blockIdx.y, n = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (n >= N || (unsigned)w_idx[z] >= (unsigned)n_idx) return;
  const float* ar = A + (int64_t)(z / a_div) * lda;
  const bf16_t* wg = W + (int64_t)w_idx[z] * w_bs + (int64_t)n * ldw;
  const bf16_t* wu = wg + (int64_t)N * ldw;
  float sg = 0.f, su = 0.f;
  if (VEC) {
    for (int k = lane * 8; k < K; k += 512) {
      const uint4 gv = *reinterpret_cast<const uint4*>(wg + k), uv = *reinterpret_cast<const uint4*>(wu + k);
      float av[8];
      ld_group<4>(ar + k, *reinterpret_cast<float(*)[4]>(av));
      ld_group<4>(ar + k + 4, *reinterpret_cast<float(*)[4]>(av + 4));
      const uint32_t g4[4] = {gv.x, gv.y, gv.z, gv.w}, u4[4] = {uv.x, uv.y, uv.z, uv.w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        sg = fmaf(av[2 * e], bf16lo_to_f32(g4[e]), sg); sg = fmaf(av[2 * e + 1], bf16hi_to_f32(g4[e]), sg);
        su = fmaf(av[2 * e], bf16lo_to_f32(u4[e]), su); su = fmaf(av[2 * e + 1], bf16hi_to_f32(u4[e]), su);
      }
    }
  } else {
    for (int k = lane; k < K; k += 64) { sg = fmaf(ar[k], bf16_to_f32(wg[k]), sg); su = fmaf(ar[k], bf16_to_f32(wu[k]), su); }
  }
  sg = wave_sum(sg);
  su = wave_sum(su);
  if (x_scale) { sg *= x_scale[z]; su *= x_scale[z]; }
  if (lane == 0) C[(int64_t)z * ldc + n] = silu_x(sg) * su;
}

}  // namespace

extern "C" int mn_add_layernorm_rows(float* x, int64_t ldx, const float* y, int64_t ldy, const float* ye, int64_t ldye, const int32_t* slot_of,
                                     const float* ew, float ew_all, int top, const uint16_t* w, float eps, float* h, int64_t ldh, uint16_t* h16,
                                     int64_t ldh16, int M, int n, void* stream) {
  MN_CHECK_ARG(x && M >= 1 && n >= 1 && top >= 0 && (top == 0 || ye) && (!w || h || h16), "mn_add_layernorm_rows: bad args");
  if (!ye) top = 0;
  AddLnArgs a{x, ldx, y, ldy, ye, ldye, slot_of, ew, ew_all, top, w, eps, h, ldh, h16, ldh16, n};
  hipStream_t st = mn_stream(stream);
  const bool vec = (n % 4) == 0 && (ldx % 4) == 0 && (!y || (ldy % 4) == 0) && (top == 0 || (ldye % 4) == 0) &&
                   ((((uintptr_t)x) | ((uintptr_t)y) | ((uintptr_t)ye)) & 15) == 0;
#define MN_LN(G_, V_) hipLaunchKernelGGL((add_ln_kernel<G_, V_>), dim3((unsigned)M), dim3(256), 0, st, a)
  if (vec && n <= 1024) MN_LN(4, 1);
  else if (vec && n <= 2048) MN_LN(4, 2);
  else if (vec && n <= 4096) MN_LN(4, 4);
  else if (vec && n <= 8192) MN_LN(4, 8);
  else if (n <= 256) MN_LN(1, 1);
  else if (n <= 1024) MN_LN(1, 4);
  else if (n <= 4096) MN_LN(1, 16);
  else hipLaunchKernelGGL(add_ln_long_kernel, dim3((unsigned)M), dim3(256), 0, st, a);
#undef MN_LN
  MN_CHECK_LAUNCH("mn_add_layernorm_rows");
  return MN_OK;
}

extern "C" int mn_xielu_rows(const float* x, int64_t ldx, float alpha_pos, float alpha_neg, float* y, int64_t ldy, uint16_t* y16, int64_t ldy16,
                             int M, int n, void* stream) {
  MN_CHECK_ARG(x && (y || y16) && M >= 1 && M <= 65535 && n >= 1, "mn_xielu_rows: bad args");
  XieluArgs a{x, ldx, alpha_pos, alpha_neg, y, ldy, y16, ldy16, M, n};
  hipLaunchKernelGGL(xielu_kernel, dim3((unsigned)mn_cdiv(n, 1024), (unsigned)M), dim3(256), 0, mn_stream(stream), a);
  MN_CHECK_LAUNCH("mn_xielu_rows");
  return MN_OK;
}

extern "C" int mn_token_table_rows(const int32_t* table, int vocab, int top, const int32_t* tok, int M, int32_t* idx, float* w, void* stream) {
  MN_CHECK_ARG(table && tok && idx && vocab >= 1 && top >= 1 && M >= 1 && (int64_t)M * top < ((int64_t)1 << 31), "mn_token_table_rows: bad args");
  hipLaunchKernelGGL(token_table_kernel, dim3((unsigned)mn_cdiv((int64_t)M * top, 256)), dim3(256), 0, mn_stream(stream), table, vocab, top, tok, M, idx, w);
  MN_CHECK_LAUNCH("mn_token_table_rows");
  return MN_OK;
}

extern "C" size_t mn_sizeof_low_rank_job(void) { return sizeof(mn_low_rank_job); }
extern "C" size_t mn_sizeof_rows_prep(void) { return sizeof(mn_rows_prep); }

namespace {
bool low_rank_ok(const mn_low_rank_job& j) {
  return j.a && j.w && j.out && j.k >= 1 && j.n >= 1 && j.kind >= MN_LOW_RANK_LINEAR && j.kind <= MN_LOW_RANK_SIGMOID &&
         (j.kind != MN_LOW_RANK_DECAY || (j.a_log && j.head_n >= 1));
}
}  // namespace

extern "C" int mn_low_rank_gate_rows(const mn_low_rank_job* jobs, int n_jobs, int M, void* stream) {
  MN_CHECK_ARG(jobs && (n_jobs == 1 || n_jobs == 2) && M >= 1, "mn_low_rank_gate_rows: one or two jobs");
  for (int i = 0; i < n_jobs; ++i) MN_CHECK_ARG(low_rank_ok(jobs[i]), "mn_low_rank_gate_rows: job %d: bad sizes or null operands", i);
  LowRankArgs a;
  a.job[0] = jobs[0];
  a.job[1] = jobs[n_jobs - 1];
  a.M = M;
  const bool few = M <= 64;
  const int tile = few ? 32 : 64, rows = few ? LR_ROWS : 64;
  a.nb0 = (int)mn_cdiv(jobs[0].n, tile);
  const dim3 grid((unsigned)(a.nb0 + (n_jobs == 2 ? mn_cdiv(jobs[1].n, tile) : 0)), (unsigned)mn_cdiv(M, rows));
  MN_CHECK_ARG(grid.y <= 65535, "mn_low_rank_gate_rows: too many rows");
  if (few) hipLaunchKernelGGL(low_rank_few_kernel, grid, dim3(256), 0, mn_stream(stream), a);
  else hipLaunchKernelGGL(low_rank_mfma_kernel, grid, dim3(256), 0, mn_stream(stream), a);
  MN_CHECK_LAUNCH("mn_low_rank_gate_rows");
  return MN_OK;
}

extern "C" int mn_rows_prep_launch(const mn_rows_prep* p, const int32_t* row_seq, const int32_t* row_slot, int M, void* stream) {
  MN_CHECK_ARG(p && M >= 1 && M <= 64 && p->n_jobs >= 0 && p->n_jobs <= 2 && p->act_n >= 0 && p->top >= 0, "mn_rows_prep_launch: bad args (M=%d: at most 64)", M);
  MN_CHECK_ARG(!p->delta || (p->proj && p->w_conv && row_seq && row_slot && p->qkv && p->beta && p->H >= 1 && p->G >= 1 && (p->H % p->G) == 0 &&
                             p->dim >= 1 && p->vdim >= 1 && p->taps >= 1 && (p->taps == 1 || p->conv_state) && p->ldbeta >= p->H),
               "mn_rows_prep_launch: bad delta-rule args");
  for (int i = 0; i < p->n_jobs; ++i) MN_CHECK_ARG(low_rank_ok(p->job[i]), "mn_rows_prep_launch: job %d: bad sizes or null operands", i);
  MN_CHECK_ARG(p->act_n == 0 || (p->act_x && p->act_y), "mn_rows_prep_launch: the activation needs its rows");
  MN_CHECK_ARG(p->top == 0 || (p->table && p->tok && p->idx && p->vocab >= 1), "mn_rows_prep_launch: the table needs its rows");
  RowsPrepArgs a{};
  a.M = M;
  if (p->delta) {
    a.delta = DeltaPrepArgs{p->proj, p->ld, p->H, p->G, p->dim, p->vdim, p->taps, p->off_b, 0, p->w_conv, p->conv_state, 1, nullptr, nullptr, p->unit_eps,
                            p->q_scale, row_seq, row_slot, nullptr, p->qkv, p->ldqkv, p->beta, p->ldbeta};
    a.n_delta = (int)mn_cdiv(delta_prep_units(p->H, p->G, p->vdim), 4);
  }
  if (p->n_jobs > 0) {
    a.lr.job[0] = p->job[0];
    a.lr.job[1] = p->job[p->n_jobs - 1];
    a.lr.M = M;
    a.lr.nb0 = (int)mn_cdiv(p->job[0].n, 32);
    a.n_lr = a.lr.nb0 + (p->n_jobs == 2 ? (int)mn_cdiv(p->job[1].n, 32) : 0);
  }
  if (p->act_n > 0) {
    a.act = XieluArgs{p->act_x, p->ld_act_x, p->act_pos, p->act_neg, p->act_y, p->ld_act_y, nullptr, 0, M, p->act_n};
    a.n_act = (int)mn_cdiv(p->act_n, 1024);
  }
  a.table = p->table; a.tok = p->tok; a.vocab = p->vocab; a.top = p->top; a.idx = p->idx;
  const int64_t blocks = (int64_t)a.n_delta + a.n_lr + a.n_act + (p->top > 0 ? 1 : 0);
  if (blocks == 0) return MN_OK;
  hipLaunchKernelGGL(rows_prep_kernel, dim3((unsigned)blocks, (unsigned)M), dim3(256), 0, mn_stream(stream), a);
  MN_CHECK_LAUNCH("mn_rows_prep_launch");
  return MN_OK;
}

extern "C" int mn_channel_state_rows(const float* qkv, int64_t ld, const float* g, int64_t ldg, const float* beta, int64_t ldb, int M, int H, int G,
                                     int dim, int vdim, float o_scale, float* state, const int32_t* row_seq, const int32_t* row_slot,
                                     const int32_t* row_back, const int32_t* blk_tab, int n_blk, int flags, float* out, int64_t ldo, void* stream) {
  const bool distinct = (flags & MN_SEQ_ROWS_DISTINCT) != 0;
  MN_CHECK_ARG(qkv && g && state && row_seq && row_slot && (row_back || distinct) && out && M >= 1 && M <= 65535 && H >= 1 && H <= 65535 && G >= 1 &&
                   (H % G) == 0 && dim >= 1 && dim <= 4096 && vdim >= 1 && mn_cdiv(vdim, 32) <= 65535,
               "mn_channel_state_rows: bad args (dim=%d: at most 4096)", dim);
  MN_CHECK_ARG(!blk_tab || (n_blk >= 1 && n_blk <= M), "mn_channel_state_rows: bad table of runs");
  ChanArgs a{qkv, ld, g, ldg, beta, ldb, H, G, dim, vdim, o_scale, state, row_seq, row_slot, distinct ? nullptr : row_back, distinct ? nullptr : blk_tab,
             out, ldo, M, nullptr, nullptr, nullptr};
  const int n_runs = a.blk_tab ? n_blk : M;
  return beta ? chan_rows<true>(a, distinct, n_runs, mn_stream(stream)) : chan_rows<false>(a, distinct, n_runs, mn_stream(stream));
}

extern "C" int mn_channel_chunk_rows(void) { return 128; }

extern "C" size_t mn_channel_scan_workspace_bytes(int n_chunks, int H, int dim, int vdim) {
  if (n_chunks < 1 || H < 1 || dim < 1 || vdim < 1) return 0;
  return (size_t)n_chunks * H * dim * ((size_t)vdim + 1) * sizeof(float);
}

extern "C" int mn_channel_state_rows_scan(const float* qkv, int64_t ld, const float* g, int64_t ldg, int M, int H, int G, int dim, int vdim,
                                          float o_scale, float* state, const int32_t* row_seq, const int32_t* row_slot, const int32_t* row_back,
                                          const int32_t* chunk_tab, int n_chunks, float* out, int64_t ldo, void* workspace,
                                          size_t workspace_bytes, void* stream) {
  MN_CHECK_ARG(qkv && g && state && row_seq && row_slot && row_back && chunk_tab && out && workspace && M >= 1 && H >= 1 && H <= 65535 && G >= 1 &&
                   (H % G) == 0 && dim >= 1 && dim <= 256 && vdim >= 1 && n_chunks >= 1 && n_chunks <= 65535,
               "mn_channel_state_rows_scan: bad args (dim=%d: at most 256)", dim);
  MN_CHECK_ARG(workspace_bytes >= mn_channel_scan_workspace_bytes(n_chunks, H, dim, vdim), "mn_channel_state_rows_scan: workspace too small");
  float* ws = (float*)workspace;
  ChanArgs a{qkv, ld, g, ldg, nullptr, 0, H, G, dim, vdim, o_scale, state, row_seq, row_slot, row_back, nullptr, out, ldo, M, chunk_tab, ws,
             ws + (size_t)n_chunks * H * dim * vdim};
  hipStream_t st = mn_stream(stream);
  const bool vec = chan_vec(a);
  const dim3 carry((unsigned)mn_cdiv((int64_t)dim * vdim, 256), (unsigned)H, (unsigned)n_chunks);
#define MN_CS(NS_, LPC_, DB_)                                                                                                              \
  do {                                                                                                                                     \
    const dim3 grid((unsigned)(H * mn_cdiv(vdim, 128 / LPC_ * 2)), (unsigned)n_chunks);                                                   \
    if (vec) hipLaunchKernelGGL((chan_walk_kernel<NS_, LPC_, 2, 128, DB_, false, true, CHUNK_END>), grid, dim3(128), 0, st, a);           \
    else hipLaunchKernelGGL((chan_walk_kernel<NS_, LPC_, 2, 128, DB_, false, false, CHUNK_END>), grid, dim3(128), 0, st, a);              \
    hipLaunchKernelGGL(chan_carry_kernel, carry, dim3(256), 0, st, a, n_chunks);                                                          \
    if (vec) hipLaunchKernelGGL((chan_walk_kernel<NS_, LPC_, 2, 128, DB_, false, true, CHUNK_OUT>), grid, dim3(128), 0, st, a);           \
    else hipLaunchKernelGGL((chan_walk_kernel<NS_, LPC_, 2, 128, DB_, false, false, CHUNK_OUT>), grid, dim3(128), 0, st, a);              \
  } while (0)
  if (dim <= 32) MN_CS(4, 8, 16); else if (dim <= 64) MN_CS(4, 16, 16); else if (dim <= 128) MN_CS(8, 16, 16); else MN_CS(16, 16, 8);
#undef MN_CS
  MN_CHECK_LAUNCH("mn_channel_state_rows_scan");
  return MN_OK;
}

extern "C" int mn_gemv_glu_indexed(const float* A, int64_t lda, int a_div, const uint16_t* W, int64_t ldw, int64_t w_bs, const int32_t* w_idx,
                                   int n_idx, float* C, int64_t ldc, int Z, int N, int K, void* stream) {
  return mn_gemv_glu_indexed_scaled(A, lda, a_div, W, ldw, w_bs, w_idx, n_idx, nullptr, C, ldc, Z, N, K, stream);
}

extern "C" int mn_gemv_glu_indexed_scaled(const float* A, int64_t lda, int a_div, const uint16_t* W, int64_t ldw, int64_t w_bs, const int32_t* w_idx,
                                          int n_idx, const float* x_scale, float* C, int64_t ldc, int Z, int N, int K, void* stream) {
  MN_CHECK_ARG(A && W && w_idx && C && a_div >= 1 && Z >= 1 && Z <= 65535 && N >= 1 && K >= 1 && n_idx >= 1, "mn_gemv_glu_indexed: bad args (Z=%d)", Z);
  const bool vec = (K % 8) == 0 && (ldw % 8) == 0 && (w_bs % 8) == 0 && (lda % 4) == 0 && (((uintptr_t)W | (uintptr_t)A) & 15) == 0;
  const dim3 grid((unsigned)mn_cdiv(N, 4), (unsigned)Z);
  if (vec) hipLaunchKernelGGL((gemv_glu_indexed_kernel<true>), grid, dim3(256), 0, mn_stream(stream), A, lda, a_div, W, ldw, w_bs, w_idx, n_idx, C, ldc, N, K, x_scale);
  else hipLaunchKernelGGL((gemv_glu_indexed_kernel<false>), grid, dim3(256), 0, mn_stream(stream), A, lda, a_div, W, ldw, w_bs, w_idx, n_idx, C, ldc, N, K, x_scale);
  MN_CHECK_LAUNCH("mn_gemv_glu_indexed");
  return MN_OK;
}
