// talk_attn.hip — softmax attention whose heads' scores are mixed by a matrix before the softmax (mingnative.h section 13).
//   score_h(i, j) = sum_g talk[h, g] (q_g(i) . k_(g / rep)(j)),  out_h(i) = sum_j softmax_h(i, j) v_(h / rep)(j),  rep = H / G,
// over the keys of the row's window and / or chunk (chunks of `chunk` positions counted from position 0), with an optional sink per head
// in the softmax's denominator.  A workgroup holds ALL heads of its rows: the mixing needs every head's score of a (row, key) pair.
#include <math.h>

#include "common.h"
#include "mfma_f32_tiles.h"

namespace {

struct TalkArgs {
  const float* q; int64_t ldq;                 // [M, H dim], scaled
  const float *k, *v; int64_t ldk, ldv;        // arenas [n_seq, t_max, ld]
  const float *talk, *sink;                    // [H, H]; [H] or NULL
  const int32_t *row_seq, *row_slot, *blk_tab;
  int H, G, dim, t_max, window, chunk, rows, nsplit, ovec;
  float* out; int64_t ldo; bf16_t* out16; int64_t ldo16;
  float* part;
};

// the oldest position row `pos` sees; it never falls as pos grows
__device__ __forceinline__ int first_key(int pos, int window, int chunk) {
  int t = window > 0 ? max(0, pos - window + 1) : 0;
  if (chunk > 0) t = max(t, pos - pos % chunk);
  return t;
}

// 1 / (the softmax's normaliser), numerator and denominator relative to max(m, sink)
__device__ __forceinline__ float talk_inv(float m, float l, const float* sink, int h) {
  if (!sink) return 1.0f / l;
  const float sk = sink[h], mm = fmaxf(m, sk), f = expf(m - mm);
  return f / (l * f + expf(sk - mm));
}

// 16 bytes of a row of `dim` (a multiple of 4) values; past its end the row's last ones.  Keys need no mask there (the queries are zero
// padded) and neither do values (their columns are not written), so every load stands alone in the instruction stream.
__device__ __forceinline__ f32x4 ld4(const float* row, int d, int dim) { return *reinterpret_cast<const f32x4*>(row + min(d, dim - 4)); }

// Matrix-core form (v_mfma_f32_16x16x4_f32: scores, mixing and values stay fp32).  A workgroup of 4 waves owns a run of up to `rows` rows
// of one sequence with all heads; the query vectors (row, head) of a key/value head form TV tiles of 16 (vector r rep + head % rep).  A
// wave owns KW work units of (key/value head, TW of its tiles) through both products; keys are walked in tiles of 16:
//   scores  every lane takes 16-byte pieces of ITS key (lane c16 = key, g4 = piece): the k order of the products is the order of those
//           pieces, so keys go straight from the arena to the B operand; results to LDS
//   mixing  one 16 x 16 tile of (mixed head, key) per (row, 16 heads): talk x the row's scores of all heads, then visibility and the
//           running maximum / sum; the weights go to LDS
//   values  lane c16 takes the columns 4 c16 .. of a 64-column block of ITS key rows (16-byte loads), so result tile (b, i) holds the
//           columns 64 b + 4 c16 + i
// The next tile's keys and values are requested as soon as the present ones have been multiplied.
template <int NBD, int KW, int TW, int HB>
__global__ __launch_bounds__(256, (KW * TW * NBD <= 2 && HB == 1 ? 2 : 1)) void talk_attn_mfma_kernel(TalkArgs a) {
  constexpr int U = KW * TW, LS = 17, LP = 20, HP = 16 * HB, LT = HP + 1, RU = HB == 4 ? 4 : 2 * HB, ND = 4 * NBD;
  extern __shared__ float lds[];
  const int tid = threadIdx.x, b = blockIdx.x, sp = blockIdx.y;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, c16 = lane & 15, g4 = lane >> 4;
  const int rep = a.H / a.G, TV = (a.rows * rep + 15) / 16, TVB = (TV + TW - 1) / TW, NV = a.G * TV * 16;
  const int r0 = a.blk_tab ? a.blk_tab[2 * b] : b;
  const int nr = a.blk_tab ? min(a.blk_tab[2 * b + 1], a.rows) : 1;
  const int seq = a.row_seq[r0], pos0 = a.row_slot[r0], posL = pos0 + nr - 1;
  const int tF = first_key(pos0, a.window, a.chunk), nk = posL - tF + 1;
  const int ntile = (nk + 15) / 16, tps = (ntile + a.nsplit - 1) / a.nsplit;
  const int t0 = sp * tps, t1 = min(ntile, t0 + tps);
  float* Sl = lds;                             // [NV][LS] raw scores
  float* Pl = Sl + (NV * LS + 3) / 4 * 4;      // [NV][LP] weights
  float* Cl = Pl + NV * LP;                    // [NV] rescale of the tile; at the end the normalisers
  float* Tl = Cl + NV;                         // [HP][LT]
  for (int e = tid; e < HP * HP; e += 256) {
    const int h = e / HP, g = e - h * HP;
    Tl[h * LT + g] = (h < a.H && g < a.H) ? a.talk[h * a.H + g] : 0.f;
  }
  // this wave's units
  int kap[KW], tile0[KW];
#pragma unroll
  for (int x = 0; x < KW; ++x) {
    const int wu = wave * KW + x;
    kap[x] = wu < a.G * TVB ? wu / TVB : -1;
    tile0[x] = (wu % TVB) * TW;
  }
  f32x4 qreg[U][ND], acc[U][ND], kreg[KW][ND], vreg[KW][4][NBD];
#pragma unroll
  for (int x = 0; x < KW; ++x)
#pragma unroll
    for (int w = 0; w < TW; ++w) {
      const int vv = 16 * (tile0[x] + w) + c16, r = vv / rep;
      const bool on = kap[x] >= 0 && tile0[x] + w < TV && r < nr;
      const float* src = a.q + (int64_t)(r0 + (on ? r : 0)) * a.ldq + (int64_t)(on ? kap[x] * rep + vv % rep : 0) * a.dim;
#pragma unroll
      for (int j = 0; j < ND; ++j) {
        const f32x4 t = ld4(src, 16 * j + 4 * g4, a.dim);
        qreg[x * TW + w][j] = (on && 16 * j + 4 * g4 < a.dim) ? t : f32x4{0.f, 0.f, 0.f, 0.f};
        acc[x * TW + w][j] = f32x4{0.f, 0.f, 0.f, 0.f};
      }
    }
  const float* kb = a.k + ((int64_t)seq * a.t_max + tF) * a.ldk;
  const float* vb = a.v + ((int64_t)seq * a.t_max + tF) * a.ldv;
  auto fetch_k = [&](int tile) {
    const float* row = kb + (int64_t)min(16 * tile + c16, nk - 1) * a.ldk;
#pragma unroll
    for (int x = 0; x < KW; ++x)
      if (kap[x] >= 0) {
#pragma unroll
        for (int j = 0; j < ND; ++j) kreg[x][j] = ld4(row + (int64_t)kap[x] * a.dim, 16 * j + 4 * g4, a.dim);
      }
  };
  auto fetch_v = [&](int tile) {
#pragma unroll
    for (int x = 0; x < KW; ++x)
      if (kap[x] >= 0) {
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          const float* row = vb + (int64_t)min(16 * tile + t + 4 * g4, nk - 1) * a.ldv + (int64_t)kap[x] * a.dim;
#pragma unroll
          for (int j = 0; j < NBD; ++j) vreg[x][t][j] = ld4(row, 64 * j + 4 * c16, a.dim);
        }
      }
  };
  // mixing: where head g = 4 t + g4 of row 0 lies among the vectors (as an operand), and head 16 hb + 4 g4 + i (as a result)
  int goff[4 * HB], poff[HB][4];
#pragma unroll
  for (int t = 0; t < 4 * HB; ++t) { const int g = 4 * t + g4; goff[t] = g < a.H ? (g / rep) * TV * 16 + g % rep : 0; }
#pragma unroll
  for (int hb = 0; hb < HB; ++hb)
#pragma unroll
    for (int i = 0; i < 4; ++i) { const int h = 16 * hb + 4 * g4 + i; poff[hb][i] = h < a.H ? (h / rep) * TV * 16 + h % rep : -1; }
  float mrun[RU][4], lrun[RU][4];
#pragma unroll
  for (int x = 0; x < RU; ++x)
#pragma unroll
    for (int i = 0; i < 4; ++i) { mrun[x][i] = -INFINITY; lrun[x][i] = 0.f; }
  if (t0 < t1) { fetch_k(t0); fetch_v(t0); }
  for (int tile = t0; tile < t1; ++tile) {
#pragma unroll
    for (int x = 0; x < KW; ++x) {
      if (kap[x] < 0) continue;
#pragma unroll
      for (int w = 0; w < TW; ++w) {
        if (tile0[x] + w >= TV) continue;
        f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f}, s2 = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < ND; ++j) {
          s = __builtin_amdgcn_mfma_f32_16x16x4f32(qreg[x * TW + w][j][0], kreg[x][j][0], s, 0, 0, 0);
          s2 = __builtin_amdgcn_mfma_f32_16x16x4f32(qreg[x * TW + w][j][1], kreg[x][j][1], s2, 0, 0, 0);
          s = __builtin_amdgcn_mfma_f32_16x16x4f32(qreg[x * TW + w][j][2], kreg[x][j][2], s, 0, 0, 0);
          s2 = __builtin_amdgcn_mfma_f32_16x16x4f32(qreg[x * TW + w][j][3], kreg[x][j][3], s2, 0, 0, 0);
        }
        s += s2;
        float* dst = Sl + (16 * (kap[x] * TV + tile0[x] + w) + 4 * g4) * LS + c16;
#pragma unroll
        for (int i = 0; i < 4; ++i) dst[i * LS] = s[i];
      }
    }
    if (tile + 1 < t1) fetch_k(tile + 1);
    lds_barrier();
    const int jk = 16 * tile + c16, tok = tF + jk;
#pragma unroll
    for (int x = 0; x < RU; ++x) {
      const int su = wave + 4 * x, r = su / HB, hb = su % HB;
      if (r >= nr) continue;
      f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int t = 0; t < 4 * HB; ++t)
        s = __builtin_amdgcn_mfma_f32_16x16x4f32(Tl[(16 * hb + c16) * LT + 4 * t + g4], Sl[(goff[t] + r * rep) * LS + c16], s, 0, 0, 0);
      const int pos = pos0 + r;
      const bool see = jk < nk && tok <= pos && tok >= first_key(pos, a.window, a.chunk);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float sc = see ? s[i] : -INFINITY;
        const float mnew = fmaxf(mrun[x][i], row16_max(sc));
        const float p = see ? fast_exp(sc - mnew) : 0.f;
        const float corr = mrun[x][i] == -INFINITY ? 0.f : fast_exp(mrun[x][i] - mnew);
        lrun[x][i] = lrun[x][i] * corr + row16_sum(p);
        mrun[x][i] = mnew;
        int po = poff[0][i];
#pragma unroll
        for (int y = 1; y < HB; ++y) if (hb == y) po = poff[y][i];
        if (po >= 0) {
          Pl[(po + r * rep) * LP + c16] = p;
          if (c16 == 0) Cl[po + r * rep] = corr;
        }
      }
    }
    lds_barrier();
#pragma unroll
    for (int x = 0; x < KW; ++x) {
      if (kap[x] < 0) continue;
#pragma unroll
      for (int w = 0; w < TW; ++w) {
        if (tile0[x] + w >= TV) continue;
        const int vt = 16 * (kap[x] * TV + tile0[x] + w);
        const f32x4 corr = *reinterpret_cast<const f32x4*>(Cl + vt + 4 * g4);
#pragma unroll
        for (int j = 0; j < ND; ++j) acc[x * TW + w][j] *= corr;
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          const float pa = Pl[(vt + c16) * LP + t + 4 * g4];
#pragma unroll
          for (int j = 0; j < NBD; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i)
              acc[x * TW + w][4 * j + i] = __builtin_amdgcn_mfma_f32_16x16x4f32(pa, vreg[x][t][j][i], acc[x * TW + w][4 * j + i], 0, 0, 0);
        }
      }
    }
    if (tile + 1 < t1) fetch_v(tile + 1);
  }
  // normalisers (or this split's statistics), then the result
  float* part = a.nsplit > 1 ? a.part + ((int64_t)b * a.nsplit + sp) * ((int64_t)NV * (2 + a.dim)) : nullptr;
  lds_barrier();
#pragma unroll
  for (int x = 0; x < RU; ++x) {
    const int su = wave + 4 * x, r = su / HB, hb = su % HB;
    if (r >= nr || c16 != 0) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      int po = poff[0][i];
#pragma unroll
      for (int y = 1; y < HB; ++y) if (hb == y) po = poff[y][i];
      if (po < 0) continue;
      if (part) { part[po + r * rep] = mrun[x][i]; part[NV + po + r * rep] = lrun[x][i]; }
      else Cl[po + r * rep] = talk_inv(mrun[x][i], lrun[x][i], a.sink, 16 * hb + 4 * g4 + i);
    }
  }
  lds_barrier();
#pragma unroll
  for (int x = 0; x < KW; ++x) {
    if (kap[x] < 0) continue;
#pragma unroll
    for (int w = 0; w < TW; ++w) {
      if (tile0[x] + w >= TV) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int vv = 16 * (tile0[x] + w) + 4 * g4 + i, r = vv / rep;
        if (r >= nr) continue;
        const int vid = kap[x] * TV * 16 + vv;
        const float inv = part ? 1.0f : Cl[vid];
        const int64_t col0 = (int64_t)(kap[x] * rep + vv % rep) * a.dim;
#pragma unroll
        for (int j = 0; j < NBD; ++j) {
          const int d = 64 * j + 4 * c16;
          if (d >= a.dim) continue;
          f32x4 val;
#pragma unroll
          for (int e = 0; e < 4; ++e) val[e] = acc[x * TW + w][4 * j + e][i] * inv;
          if (part) {
            *reinterpret_cast<f32x4*>(part + 2 * NV + (int64_t)vid * a.dim + d) = val;
            continue;
          }
          const int64_t row = r0 + r;
          if (a.ovec) {
            if (a.out) *reinterpret_cast<f32x4*>(a.out + row * a.ldo + col0 + d) = val;
            if (a.out16)
              *reinterpret_cast<uint2*>(a.out16 + row * a.ldo16 + col0 + d) = make_uint2(pack_bf16x2(val[0], val[1]), pack_bf16x2(val[2], val[3]));
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              if (a.out) a.out[row * a.ldo + col0 + d + e] = val[e];
              if (a.out16) a.out16[row * a.ldo16 + col0 + d + e] = f32_to_bf16(val[e]);
            }
          }
        }
      }
    }
  }
}

// grid (n_blk, G TV, ceil(dim / 64)): the splits' statistics and sums of a tile of 16 vectors become its rows' results
__global__ __launch_bounds__(256) void talk_attn_merge_kernel(TalkArgs a) {
  const int tid = threadIdx.x, b = blockIdx.x, rep = a.H / a.G, TV = (a.rows * rep + 15) / 16, NV = a.G * TV * 16;
  const int kap = blockIdx.y / TV, vt = blockIdx.y % TV;
  const int r0 = a.blk_tab ? a.blk_tab[2 * b] : b;
  const int nr = a.blk_tab ? min(a.blk_tab[2 * b + 1], a.rows) : 1;
  const int nv = min(16, nr * rep - 16 * vt);                 // vectors of this tile that exist
  if (nv <= 0) return;
  const int64_t stride = (int64_t)NV * (2 + a.dim);
  const float* base = a.part + (int64_t)b * a.nsplit * stride;
  __shared__ float wgt[16][64], inv[16];
  for (int i = tid >> 6; i < nv; i += 4) {                    // one wave per vector, one lane per split
    const int lane = tid & 63, vid = 16 * (kap * TV + vt) + i;
    const float ms = lane < a.nsplit ? base[lane * stride + vid] : -INFINITY;
    const float ls = lane < a.nsplit ? base[lane * stride + NV + vid] : 0.f;
    const float mx = wave_max(ms);
    const float w = ms == -INFINITY ? 0.f : expf(ms - mx);
    wgt[i][lane] = w;
    const float L = wave_sum(ls * w);
    if (lane == 0) inv[i] = talk_inv(mx, L, a.sink, kap * rep + (16 * vt + i) % rep);
  }
  __syncthreads();
  const int c0 = blockIdx.z * 64, cw = min(64, a.dim - c0);
  for (int e = tid; e < nv * cw; e += 256) {
    const int i = e / cw, d = c0 + e - i * cw, vv = 16 * vt + i;
    const float* src = base + 2 * NV + (int64_t)(kap * TV * 16 + vv) * a.dim + d;
    float t = 0.f;
#pragma unroll 8
    for (int s = 0; s < a.nsplit; ++s) t = fmaf(src[s * stride], wgt[i][s], t);      // a split without keys left zeros
    const float val = t * inv[i];
    const int64_t col = (int64_t)(kap * rep + vv % rep) * a.dim + d;
    if (a.out) a.out[(int64_t)(r0 + vv / rep) * a.ldo + col] = val;
    if (a.out16) a.out16[(int64_t)(r0 + vv / rep) * a.ldo16 + col] = f32_to_bf16(val);
  }
}

// Plain form for every shape (H <= 128, H dim <= 16384): one workgroup per row, keys in tiles of 64.
constexpr int PLAIN_OUT = 16, PLAIN_NT = 1024;
__global__ __launch_bounds__(PLAIN_NT) void talk_attn_plain_kernel(TalkArgs a) {
  extern __shared__ float lds[];               // raw scores [H][64], mixed scores / weights [H][64], per head: running max, sum, rescale
  const int m = blockIdx.x, tid = threadIdx.x, lane = tid & 63, rep = a.H / a.G;
  float* raw = lds;
  float* mix = raw + 64 * a.H;
  float* st = mix + 64 * a.H;
  const int seq = a.row_seq[m], pos = a.row_slot[m], tF = first_key(pos, a.window, a.chunk), nk = pos - tF + 1;
  const float* kb = a.k + ((int64_t)seq * a.t_max + tF) * a.ldk;
  const float* vb = a.v + ((int64_t)seq * a.t_max + tF) * a.ldv;
  const float* q = a.q + (int64_t)m * a.ldq;
  for (int h = tid; h < a.H; h += PLAIN_NT) { st[h] = -INFINITY; st[a.H + h] = 0.f; }
  float acc[PLAIN_OUT];
#pragma unroll
  for (int o = 0; o < PLAIN_OUT; ++o) acc[o] = 0.f;
  for (int j0 = 0; j0 < nk; j0 += 64) {
    const int nt = min(64, nk - j0);
    __syncthreads();
    for (int h = tid >> 6; h < a.H; h += PLAIN_NT / 64) {
      float s = 0.f;
      if (lane < nt) {
        const float* kp = kb + (int64_t)(j0 + lane) * a.ldk + (int64_t)(h / rep) * a.dim;
        for (int d = 0; d < a.dim; ++d) s = fmaf(q[h * a.dim + d], kp[d], s);
      }
      raw[h * 64 + lane] = s;
    }
    __syncthreads();
    for (int h = tid >> 6; h < a.H; h += PLAIN_NT / 64) {
      float s = 0.f;
      for (int g = 0; g < a.H; ++g) s = fmaf(a.talk[h * a.H + g], raw[g * 64 + lane], s);
      if (lane >= nt) s = -INFINITY;
      const float m_old = st[h], m_new = fmaxf(m_old, wave_max(s));
      const float p = lane < nt ? expf(s - m_new) : 0.f;
      const float alpha = m_old == -INFINITY ? 0.f : expf(m_old - m_new), sum = wave_sum(p);
      mix[h * 64 + lane] = p;
      if (lane == 0) { st[h] = m_new; st[a.H + h] = st[a.H + h] * alpha + sum; st[2 * a.H + h] = alpha; }
    }
    __syncthreads();
#pragma unroll
    for (int o = 0; o < PLAIN_OUT; ++o) {
      const int e = tid + PLAIN_NT * o;
      if (e >= a.H * a.dim) break;
      const int h = e / a.dim, d = e - h * a.dim;
      const float* vp = vb + (int64_t)j0 * a.ldv + (int64_t)(h / rep) * a.dim + d;
      float t = acc[o] * st[2 * a.H + h];
      for (int j = 0; j < nt; ++j) t = fmaf(mix[h * 64 + j], vp[(int64_t)j * a.ldv], t);
      acc[o] = t;
    }
  }
  __syncthreads();
#pragma unroll
  for (int o = 0; o < PLAIN_OUT; ++o) {
    const int e = tid + PLAIN_NT * o;
    if (e >= a.H * a.dim) break;
    const int h = e / a.dim;
    const float val = acc[o] * talk_inv(st[h], st[a.H + h], a.sink, h);
    if (a.out) a.out[(int64_t)m * a.ldo + e] = val;
    if (a.out16) a.out16[(int64_t)m * a.ldo16 + e] = f32_to_bf16(val);
  }
}

struct TalkShape { int nbd, kw, tw, hb; };      // nbd 0: no matrix-core instance
TalkShape talk_shape(int H, int G, int dim, int rows) {
  TalkShape s{0, 0, 0, 0};
  if (H < 1 || G < 1 || (H % G) != 0 || dim < 4 || (dim % 4) != 0 || rows < 1) return s;
  const int rep = H / G, TV = (rows * rep + 15) / 16;
  const int nbd = dim <= 64 ? 1 : (dim <= 128 ? 2 : (dim <= 256 ? 4 : 0)), hb = H <= 16 ? 1 : (H <= 32 ? 2 : (H <= 64 ? 4 : 0));
  if (!nbd || !hb || rows > 8 || (hb == 4 && rows > 4)) return s;
  static const int cand[6][2] = {{1, 1}, {1, 2}, {2, 1}, {1, 4}, {2, 2}, {4, 1}};
  for (const auto& c : cand) {
    if (c[0] * c[1] * nbd > 4) continue;
    if (G * mn_cdiv(TV, c[1]) <= 4 * c[0]) { s = TalkShape{nbd, c[0], c[1], hb}; break; }
  }
  return s;
}
size_t talk_lds(int H, int G, int rows, int hb) {
  const size_t NV = (size_t)G * ((rows * (H / G) + 15) / 16) * 16, HP = 16 * hb;
  return ((NV * 17 + 3) / 4 * 4 + NV * 20 + NV + HP * (HP + 1)) * sizeof(float);
}

}  // namespace

extern "C" int mn_talk_attn_block_rows(int H, int G, int dim) {
  for (int r = 8; r >= 1; r /= 2)
    if (talk_shape(H, G, dim, r).nbd) return r;
  return 0;
}

extern "C" int mn_talk_attn_splits(int n_blk, int max_keys) {
  if (n_blk < 1 || max_keys < 1) return 1;
  int64_t ns = mn_cdiv(2 * (int64_t)mn_num_cus(), n_blk);
  const int64_t tiles = mn_cdiv(max_keys, 16);
  if (ns > tiles) ns = tiles;
  return ns > 64 ? 64 : (ns < 1 ? 1 : (int)ns);
}

extern "C" size_t mn_talk_attn_workspace_bytes(int n_blk, int H, int G, int dim, int rows, int nsplit) {
  if (nsplit <= 1 || n_blk < 1 || H < 1 || G < 1 || (H % G) != 0 || dim < 1 || rows < 1) return 0;
  return (size_t)n_blk * nsplit * G * ((rows * (H / G) + 15) / 16) * 16 * (2 + (size_t)dim) * sizeof(float);
}

extern "C" int mn_talk_attn(const float* q, int64_t ldq, const float* k_arena, int64_t ldk, const float* v_arena, int64_t ldv, const float* talk,
                            const float* sink, const int32_t* row_seq, const int32_t* row_slot, int M, const int32_t* blk_tab, int n_blk, int rows,
                            int H, int G, int dim, int t_max, int window, int chunk, float* out, int64_t ldo, uint16_t* out16, int64_t ldo16,
                            int nsplit, void* workspace, size_t workspace_bytes, int variant, void* stream) {
  MN_CHECK_ARG(q && k_arena && v_arena && talk && row_seq && row_slot && (out || out16) && M >= 1 && H >= 1 && G >= 1 && (H % G) == 0 && dim >= 1 &&
                   t_max >= 1 && window >= 0 && chunk >= 0 && ldk >= (int64_t)G * dim && ldv >= (int64_t)G * dim,
               "mn_talk_attn: bad args");
  MN_CHECK_ARG(rows >= 1 && rows <= 8 && n_blk >= 1 && n_blk <= M && (blk_tab || (rows == 1 && n_blk == M)),
               "mn_talk_attn: runs of 1 .. 8 rows; without a table every row is a run");
  MN_CHECK_ARG(variant >= -1 && variant <= MN_TALK_ATTN_PLAIN, "mn_talk_attn: unknown variant %d", variant);
  const TalkShape s = talk_shape(H, G, dim, rows);
  const size_t lds = s.nbd ? talk_lds(H, G, rows, s.hb) : 0;
  const bool fits = s.nbd && lds <= 64 * 1024 && (ldq % 4) == 0 && (ldk % 4) == 0 && (ldv % 4) == 0 &&
                    (((uintptr_t)q | (uintptr_t)k_arena | (uintptr_t)v_arena | (uintptr_t)workspace) & 15) == 0;
  if (variant < 0) variant = fits ? MN_TALK_ATTN_MFMA : MN_TALK_ATTN_PLAIN;
  MN_CHECK_ARG(variant == MN_TALK_ATTN_PLAIN || fits, "mn_talk_attn: no matrix-core instance for H=%d G=%d dim=%d rows=%d", H, G, dim, rows);
  if (variant == MN_TALK_ATTN_PLAIN) nsplit = 1;
  MN_CHECK_ARG(nsplit >= 1 && nsplit <= 64 && (nsplit == 1 || (workspace && workspace_bytes >= mn_talk_attn_workspace_bytes(n_blk, H, G, dim, rows, nsplit))),
               "mn_talk_attn: 1 .. 64 key splits with their workspace");
  const int ovec = (!out || ((ldo % 4) == 0 && (((uintptr_t)out) & 15) == 0)) && (!out16 || ((ldo16 % 4) == 0 && (((uintptr_t)out16) & 7) == 0));
  TalkArgs a{q, ldq, k_arena, v_arena, ldk, ldv, talk, sink, row_seq, row_slot, blk_tab, H, G, dim, t_max, window, chunk, rows, nsplit, ovec,
             out, ldo, out16, ldo16, (float*)workspace};
  hipStream_t st = mn_stream(stream);
  if (variant == MN_TALK_ATTN_PLAIN) {
    MN_CHECK_ARG(H <= 112 && (int64_t)H * dim <= PLAIN_NT * PLAIN_OUT, "mn_talk_attn: H=%d heads of %d values: at most 112 heads, %d values", H, dim, PLAIN_NT * PLAIN_OUT);
    hipLaunchKernelGGL(talk_attn_plain_kernel, dim3((unsigned)M), dim3(PLAIN_NT), ((size_t)128 * H + 3 * H) * sizeof(float), st, a);
    MN_CHECK_LAUNCH("mn_talk_attn(plain)");
    return MN_OK;
  }
  const dim3 grid((unsigned)n_blk, (unsigned)nsplit);
#define MN_TA(N_, K_, T_)                                                                                              \
  do {                                                                                                                 \
    if (s.hb == 1) hipLaunchKernelGGL((talk_attn_mfma_kernel<N_, K_, T_, 1>), grid, dim3(256), lds, st, a);            \
    else if (s.hb == 2) hipLaunchKernelGGL((talk_attn_mfma_kernel<N_, K_, T_, 2>), grid, dim3(256), lds, st, a);       \
    else hipLaunchKernelGGL((talk_attn_mfma_kernel<N_, K_, T_, 4>), grid, dim3(256), lds, st, a);                      \
  } while (0)
  const int key = 100 * s.nbd + 10 * s.kw + s.tw;
  switch (key) {
    case 111: MN_TA(1, 1, 1); break;
    case 112: MN_TA(1, 1, 2); break;
    case 121: MN_TA(1, 2, 1); break;
    case 114: MN_TA(1, 1, 4); break;
    case 122: MN_TA(1, 2, 2); break;
    case 141: MN_TA(1, 4, 1); break;
    case 211: MN_TA(2, 1, 1); break;
    case 212: MN_TA(2, 1, 2); break;
    case 221: MN_TA(2, 2, 1); break;
    default: MN_TA(4, 1, 1); break;
  }
#undef MN_TA
  MN_CHECK_LAUNCH("mn_talk_attn");
  if (nsplit > 1) {
    const int TV = (rows * (H / G) + 15) / 16;
    hipLaunchKernelGGL(talk_attn_merge_kernel, dim3((unsigned)n_blk, (unsigned)(G * TV), (unsigned)mn_cdiv(dim, 64)), dim3(256), 0, st, a);
    MN_CHECK_LAUNCH("mn_talk_attn(merge)");
  }
  return MN_OK;
}
