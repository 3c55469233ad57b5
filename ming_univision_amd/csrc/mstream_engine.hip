// mstream_engine.hip — the step function of sequence models whose residual is several parallel streams (mingnative.h section 14): one pass
// of the layers over the rows of a step as a chain of launches on the caller's stream.  A layer is
//   h = norm(sum_s in1[s] x_s)                      mn_streams_update_norm: the previous sublayer's result is written into the streams (the
//                                                   experts' results summed) by the same launch
//   [q ; k ; v ; gate] = W_in h + b                 ONE product
//   whole-projection norms, rotation, value mixing, append; the block attention over the row's chunk / window, the heads' sinks in
//   the denominator, the output gate in its epilogue; W_o
//   h = norm(sum_s in2[s] x_s)
//   router -> picks and weights (few rows or few experts: in the launch that norms); experts fed with weight * h: the weight scales the gate and up products
// Matrix products go through the routing of seq_linear.h; the experts run
//   MN_SEQ_ARITH_BF16, M > 64      sorted by expert on a grouped bf16 MFMA GEMM: the 256 x 256-tile kernel over the list of live row tiles when
//                                  width and expert width are multiples of 64, else the 128-tile kernel when they are multiples of 8
//   MN_SEQ_ARITH_BF16, 9 .. 64     sorted by expert on the grouped weight-streaming MFMA product (bf16 hi / lo rows): every chosen expert's
//                                  weights once; its slabs are summed by the activation's launch and by the next read of the streams
//   otherwise                   one (row, pick) pair at a time against the weights its index names (fp32 FMA)
#include "seq_linear.h"

extern "C" size_t mn_sizeof_ms_layer(void) { return sizeof(mn_ms_layer); }
extern "C" size_t mn_sizeof_ms_model(void) { return sizeof(mn_ms_model); }
extern "C" size_t mn_sizeof_ms_state(void) { return sizeof(mn_ms_state); }

namespace {

constexpr int STREAM_SLABS = 2;      // most K-range slabs of a grouped weight-streaming product (mn_stream_mfma_grouped_slices)

inline int pad8(int n) { return (n + 7) / 8 * 8; }

struct MDims {
  int cq, ck, cv, hv, off_g, n_in, n_router;
};

MDims mdims(const mn_ms_layer& l) {
  MDims d{};
  d.cq = l.heads * l.dim; d.ck = l.kv_heads * l.dim; d.cv = l.kv_heads * l.vdim; d.hv = l.heads * l.vdim;
  d.off_g = d.cq + d.ck + d.cv;
  d.n_in = pad8(d.off_g + (l.has_gate ? d.hv : 0));
  d.n_router = pad8(l.experts);
  return d;
}

struct MPlan {
  int n_in = 8, cq = 1, cv = 1, hv = 1, n_router = 8, top = 1, ff = 1, experts = 1;
  size_t gemm_ws = 0, attn_ws = 0;
};

enum { EXPERTS_INDEXED = 0, EXPERTS_GROUPED = 1, EXPERTS_TILES = 2, EXPERTS_STREAM = 3 };
int expert_route(const mn_ms_model* m, const mn_ms_layer& l, int M) {
  if (m->arith != MN_SEQ_ARITH_BF16 || M <= 8 || l.experts > 128 || (int64_t)M * l.top > 65536 ||
      ((((uintptr_t)l.w_gate_up) | ((uintptr_t)l.w_down)) & 15) != 0)
    return EXPERTS_INDEXED;
  const int64_t W = m->width, ff = l.expert_ff;
  if (M <= 64 && (W % 8) == 0 && (ff % 8) == 0) return EXPERTS_STREAM;
  if ((W % 64) == 0 && (ff % 64) == 0 && 2 * ff * W * 2 < ((int64_t)1 << 32) && (int64_t)M * l.top * (W > ff ? W : ff) * 2 < ((int64_t)1 << 32))
    return EXPERTS_TILES;
  if ((W % 8) == 0 && (ff % 8) == 0) return EXPERTS_GROUPED;
  return EXPERTS_INDEXED;
}

MPlan make_plan(const mn_ms_model* m, int M) {
  MPlan p;
  auto up = [](int& a, int b) { if (b > a) a = b; };
  for (int i = 0; i < m->n_layers; ++i) {
    const mn_ms_layer& l = m->layers[i];
    const MDims d = mdims(l);
    up(p.n_in, d.n_in); up(p.cq, d.cq); up(p.cv, d.cv); up(p.hv, d.hv); up(p.n_router, d.n_router);
    if (l.experts > 0) { up(p.top, l.top); up(p.ff, l.expert_ff); up(p.experts, l.experts); }
    // key splits are chosen so that a launch has about two workgroups per compute unit: (runs x heads x splits) stays below four
    const size_t aw = (size_t)4 * mn_num_cus() * 16 * (2 + (size_t)l.vdim) * sizeof(float);
    if (aw > p.attn_ws) p.attn_ws = aw;
    if (m->arith == MN_SEQ_ARITH_BF16 && M > 8 && M <= 64) {       // scratch of the weight-streaming MFMA route: the largest product of the stack
      const int W = m->width;
      const int shapes[3][2] = {{d.n_in, W}, {W, d.hv}, {d.n_router, W}};
      for (const auto& nk : shapes) {
        if (nk[0] < 1 || nk[1] < 8 || (nk[1] % 8) != 0) continue;
        const size_t g = mn_skinny_workspace_bytes(M, nk[0], nk[1], MN_EPI_NONE);
        if (g > p.gemm_ws) p.gemm_ws = g;
      }
    }
  }
  return p;
}

}  // namespace

extern "C" size_t mn_ms_workspace_bytes(const mn_ms_model* m, int M) {
  if (!m || !m->layers || M < 1) return 0;
  const MPlan p = make_plan(m, M);
  const size_t W = m->width, R = (size_t)M, Z = R * p.top, few = M <= 64 ? STREAM_SLABS : 1;       // few rows: hi / lo rows, slabs
  size_t n = 0;
  n += al(R * m->streams * W * 4);                     // the streams
  n += al(R * W * 4) + al(few * R * W * 2);            // normed rows + bf16
  n += al(R * p.n_in * 4);                             // stacked input projections
  n += al(R * p.cq * 4);                               // queries
  n += al(R * p.cv * 4);                               // the values later layers mix in
  n += al(R * p.hv * 4) + al(R * p.hv * 2);            // gated heads + bf16
  n += al(R * W * 4);                                  // sublayer result
  n += al(R * p.n_router * 4);                         // router logits
  n += al(Z * 4) + 2 * al(Z * 4);                      // chosen experts; weights, weights in the sorted order
  n += al(few * Z * 2 * p.ff * 4);                     // [gate ; up] of the pairs
  n += al(Z * p.ff * 4) + al(few * Z * p.ff * 2);      // their activation + bf16
  n += al(few * Z * W * 4);                            // their results
  n += al(Z * W * 2);                                  // gathered bf16 rows
  n += 2 * al(((size_t)p.experts + 1) * 4) + 2 * al(Z * 4);   // counts, offsets, perm, slot_of
  n += 2 * al((Z / 256 + p.experts + 1) * 4) + al(4);         // live row tiles of the grouped products, their count
  n += al(p.gemm_ws) + al(p.attn_ws);
  return n;
}

extern "C" int mn_ms_step(const mn_ms_model* m, const mn_ms_state* st, const float* x, int64_t ldx, int M, const int32_t* row_seq,
                          const int32_t* row_slot, const int32_t* blk_tab, int n_blk, int max_len, int flags, float* out, float* trace,
                          void* workspace, size_t workspace_bytes, void* stream) {
  MN_CHECK_ARG(m && st && m->layers && m->final_w && x && row_seq && row_slot && out && workspace, "mn_ms_step: null pointer");
  MN_CHECK_ARG(st->k && st->v, "mn_ms_step: null state table");
  MN_CHECK_ARG(M >= 1 && M <= 65535 && m->width >= 1 && m->n_layers >= 1 && m->streams >= 1, "mn_ms_step: bad sizes (M=%d)", M);
  MN_CHECK_ARG(workspace_bytes >= mn_ms_workspace_bytes(m, M), "mn_ms_step: workspace too small");
  const bool one_row = (flags & MN_SEQ_ROWS_DISTINCT) != 0;
  MN_CHECK_ARG(one_row || (blk_tab && n_blk >= 1 && n_blk <= M), "mn_ms_step: rows that share sequences need the table of their runs");
  MN_CHECK_ARG(max_len >= 1 && max_len <= st->t_max, "mn_ms_step: max_len=%d outside the cache (t_max=%d)", max_len, st->t_max);
  if (one_row) n_blk = M;
  const MPlan p = make_plan(m, M);
  const int W = m->width, S = m->streams, arith = m->arith;
  const size_t R = (size_t)M, Zmax = R * p.top, few = M <= 64 ? STREAM_SLABS : 1;
  MN_CHECK_ARG(Zmax <= 65535, "mn_ms_step: %d rows x %d picks exceed 65535 (row, expert) pairs per step", M, p.top);
  const bool want16 = arith == MN_SEQ_ARITH_BF16 && M > 64;       // bf16 copies feed the tiled MFMA GEMMs only
  char* wp = reinterpret_cast<char*>(workspace);
  auto take = [&](size_t bytes) { char* q = wp; wp += al(bytes); return q; };
  float* xs = (float*)take(R * S * W * 4);
  float* hf = (float*)take(R * W * 4);
  uint16_t* hh = (uint16_t*)take(few * R * W * 2);
  float* pin = (float*)take(R * p.n_in * 4);
  float* qf = (float*)take(R * p.cq * 4);
  float* vfirst = (float*)take(R * p.cv * 4);
  float* cat = (float*)take(R * p.hv * 4);
  uint16_t* cath = (uint16_t*)take(R * p.hv * 2);
  float* yf = (float*)take(R * W * 4);
  float* rl = (float*)take(R * p.n_router * 4);
  int32_t* tidx = (int32_t*)take(Zmax * 4);
  float* tw = (float*)take(Zmax * 4);
  float* tws = (float*)take(Zmax * 4);
  float* gu = (float*)take(few * Zmax * 2 * p.ff * 4);
  float* ea = (float*)take(Zmax * p.ff * 4);
  uint16_t* eah = (uint16_t*)take(few * Zmax * p.ff * 2);
  float* ye = (float*)take(few * Zmax * W * 4);
  uint16_t* xg = (uint16_t*)take(Zmax * W * 2);
  int32_t* counts = (int32_t*)take(((size_t)p.experts + 1) * 4);
  int32_t* offsets = (int32_t*)take(((size_t)p.experts + 1) * 4);
  int32_t* perm = (int32_t*)take(Zmax * 4);
  int32_t* slot_of = (int32_t*)take(Zmax * 4);
  int32_t* tile_g = (int32_t*)take((Zmax / 256 + p.experts + 1) * 4);
  int32_t* tile_m0 = (int32_t*)take((Zmax / 256 + p.experts + 1) * 4);
  int32_t* n_tiles = (int32_t*)take(4);
  uint16_t* const hh_buf = hh;
  void* gws = p.gemm_ws ? take(p.gemm_ws) : nullptr;
  const size_t gwb = p.gemm_ws;
  void* aws = take(p.attn_ws);
  if (!want16) hh = cath = nullptr;
  int rc;
#define MN_TRY(call) do { rc = (call); if (rc != MN_OK) return rc; } while (0)
  // where the streams lie (at the start: the input row, for every stream) and the sublayer result they have not taken yet
  mn_streams_args sa;
  memset(&sa, 0, sizeof(sa));
  sa.src = x; sa.src_row = ldx; sa.src_stream = 0;
  sa.S = S; sa.n = W; sa.eps = m->eps; sa.one_plus = m->norm_one_plus;
  // the streams take what is pending; sum_s in[s] x_s, normed with w (NULL: as it is), goes to h / h16
  // and, with a router, its picks and scores to tidx / tw; hi_lo: h16 holds the low parts behind its M rows
  struct Route { const uint16_t* w; int experts, picks; };
  auto streams_stage = [&](const float* in, const uint16_t* w, float* h, uint16_t* h16, const Route* r = nullptr, bool hi_lo = false) -> int {
    mn_streams_args a = sa;
    a.dst = a.mix ? xs : nullptr;
    a.in = in; a.w = w; a.h = h; a.ldh = W; a.h16 = h16; a.ldh16 = W;
    if (hi_lo) a.h16_lo = h16 + R * W;
    if (r) { a.router = r->w; a.experts = r->experts; a.picks = r->picks; a.idx = tidx; a.pw = tw; }
    const int rc2 = mn_streams_update_norm(&a, M, stream);
    if (a.dst) { sa.src = xs; sa.src_row = (int64_t)S * W; sa.src_stream = W; }
    sa.mix = sa.out = nullptr; sa.y = sa.ye = nullptr; sa.slot_of = nullptr; sa.ew = nullptr; sa.top = 0; sa.ye_slabs = 0;
    return rc2;
  };
  bool have_first = false;
  int first_cv = 0;
  for (int li = 0; li < m->n_layers; ++li) {
    const mn_ms_layer& l = m->layers[li];
    const MDims d = mdims(l);
    const int H = l.heads, G = l.kv_heads, E = l.experts, top = l.top, ff = l.expert_ff, Z = M * top;
    MN_CHECK_ARG(H >= 1 && G >= 1 && (H % G) == 0 && l.dim >= 1 && l.vdim >= 1 && l.window >= 0 && l.chunk >= 0 && l.norm1 && l.w_in && l.w_o &&
                     l.hc1_in && l.hc1_out && l.hc1_mix && (l.rot_dims == 0 || l.rot_freq) && st->k[li] && st->v[li],
                 "mn_ms_step: layer %d: attention: bad sizes, null weights or arenas", li);
    MN_CHECK_ARG(E == 0 || (E >= 1 && top >= 1 && top <= E && ff >= 1 && l.norm2 && l.w_router && l.w_gate_up && l.w_down && l.hc2_in && l.hc2_out &&
                            l.hc2_mix),
                 "mn_ms_step: layer %d: experts: bad sizes or null weights", li);
    MN_CHECK_ARG(!l.v_mix || !have_first || d.cv == first_cv, "mn_ms_step: layer %d: %d values do not mix with the first mixing layer's %d", li, d.cv,
                 first_cv);
    // ---- attention ----
    MN_TRY(streams_stage(l.hc1_in, l.norm1, (hh && mfma_ok(l.w_in, W)) ? nullptr : hf, hh));
    MN_TRY(linear(arith, M, hf, W, hh, W, l.w_in, d.n_in, W, l.b_in, pin, d.n_in, gws, gwb, stream));
    const bool keep = l.v_mix && !have_first, mixes = l.v_mix && have_first;
    MN_TRY(mn_proj_norm_rope_mix_append(pin, d.n_in, M, H, G, l.dim, l.vdim, l.q_norm, l.k_norm, m->eps, l.rot_dims, l.rot_interleaved, l.rot_freq,
                                        l.rot_mag, l.scale, keep ? vfirst : nullptr, d.cv, mixes ? vfirst : nullptr, d.cv, l.v_lambda, row_seq,
                                        row_slot, qf, d.cq, st->k[li], d.ck, st->v[li], d.cv, st->t_max, stream));
    if (keep) { have_first = true; first_cv = d.cv; }
    int keys = max_len;
    if (l.window > 0 && l.window + 3 < keys) keys = l.window + 3;
    if (l.chunk > 0 && l.chunk + 3 < keys) keys = l.chunk + 3;
    int ns = mn_window_attn_splits(n_blk, H, G, one_row, keys);
    while (ns > 1 && mn_window_attn_workspace_bytes(n_blk, H, G, l.vdim, one_row, ns) > p.attn_ws) --ns;
    const bool cat16_only = cath && mfma_ok(l.w_o, d.hv);
    MN_TRY(mn_window_pool_attn_blocks_gate(qf, d.cq, st->k[li], 0, st->v[li], 0, nullptr, nullptr, l.sink, 0.0f, l.chunk,
                                           l.has_gate ? pin + d.off_g : nullptr, d.n_in, row_seq, row_slot, blk_tab, n_blk, one_row, H, G, l.dim,
                                           l.vdim, st->t_max, 1, l.window, 0, 1.0f, cat16_only ? nullptr : cat, d.hv, cath, d.hv, ns, aws,
                                           p.attn_ws, -1, stream));
    MN_TRY(linear(arith, M, cat, d.hv, cath, d.hv, l.w_o, W, d.hv, nullptr, yf, W, gws, gwb, stream));
    sa.mix = l.hc1_mix; sa.out = l.hc1_out; sa.y = yf; sa.ldy = W;
    // ---- experts ----
    if (E > 0) {
      const int route = expert_route(m, l, M);
      const bool stream_rows = route == EXPERTS_STREAM;
      const bool ride = mn_streams_router_ok(M, S, W, E, l.w_router) && (((uintptr_t)sa.src) & 15) == 0 && (sa.src_row % 4) == 0;
      if (ride) {
        const Route r{l.w_router, E, top};
        MN_TRY(streams_stage(l.hc2_in, l.norm2, route == EXPERTS_INDEXED ? hf : nullptr, route == EXPERTS_INDEXED ? nullptr : hh_buf, &r, stream_rows));
      } else {
        const bool h16_only = hh && mfma_ok(l.w_router, W) && route != EXPERTS_INDEXED;
        uint16_t* const h16 = route == EXPERTS_INDEXED ? hh : hh_buf;
        MN_TRY(streams_stage(l.hc2_in, l.norm2, h16_only ? nullptr : hf, h16, nullptr, stream_rows));
        MN_TRY(linear(arith, M, hf, W, hh, W, l.w_router, d.n_router, W, nullptr, rl, d.n_router, gws, gwb, stream));
        MN_TRY(mn_router_sigmoid_topk_rows(rl, d.n_router, M, E, top, tidx, tw, stream));
      }
      const uint16_t* h16 = hh_buf;
      const int32_t* so = nullptr;
      if (route == EXPERTS_TILES) {
        const int max_mtiles = Z / 256 + E;
        MN_TRY(mn_moe_sort_weights(tidx, tw, M, top, E, counts, offsets, perm, slot_of, tws, 256, tile_g, tile_m0, n_tiles, stream));
        MN_TRY(mn_gemm256_grouped_tiles_scaled(h16, W, 0, M, perm, l.w_gate_up, W, (int64_t)2 * ff * W, offsets, counts, E, tile_g, tile_m0, n_tiles,
                                               max_mtiles, tws, eah, ff, 0, ff, W, 6, stream));
        MN_TRY(mn_gemm256_grouped_tiles(eah, ff, 0, Z, nullptr, l.w_down, ff, (int64_t)W * ff, offsets, counts, E, tile_g, tile_m0, n_tiles,
                                        max_mtiles, ye, W, 0, W, ff, 0, stream));
        so = slot_of;
      } else if (route == EXPERTS_STREAM) {
        MN_TRY(mn_moe_sort_weights(tidx, tw, M, top, E, counts, offsets, perm, slot_of, tws, 0, nullptr, nullptr, nullptr, stream));
        const int nz = mn_stream_mfma_grouped(h16, M, l.w_gate_up, (int64_t)2 * ff * W, gu, Z, offsets, perm, E, M, 2 * ff, W, stream);
        if (nz < 0) return nz;
        MN_TRY(mn_silu_split_rows_scaled(gu, nz, Z, ff, tws, eah, stream));
        const int nz2 = mn_stream_mfma_grouped(eah, Z, l.w_down, (int64_t)W * ff, ye, Z, offsets, nullptr, E, M, W, ff, stream);
        if (nz2 < 0) return nz2;
        sa.ye_slab = (int64_t)Z * W; sa.ye_slabs = nz2;
        so = slot_of;
      } else if (route == EXPERTS_GROUPED) {
        MN_TRY(mn_moe_sort_weights(tidx, tw, M, top, E, counts, offsets, perm, slot_of, tws, 0, nullptr, nullptr, nullptr, stream));
        MN_TRY(mn_gather_rows_bf16(h16, W, perm, xg, W, Z, W, stream));
        MN_TRY(mn_gemm_bf16_grouped(xg, W, l.w_gate_up, W, (int64_t)2 * ff * W, offsets, counts, E, gu, 2 * ff, M, 2 * ff, W, MN_GEMM_F32, stream));
        MN_TRY(mn_silu_mul_rows_scaled(gu, 2 * ff, tws, nullptr, 0, eah, ff, Z, ff, stream));
        MN_TRY(mn_gemm_bf16_grouped(eah, ff, l.w_down, ff, (int64_t)W * ff, offsets, counts, E, ye, W, M, W, ff, MN_GEMM_F32, stream));
        so = slot_of;
      } else {
        MN_TRY(mn_gemv_glu_indexed_scaled(hf, W, top, l.w_gate_up, W, (int64_t)2 * ff * W, tidx, E, tw, ea, ff, Z, ff, W, stream));
        MN_TRY(mn_gemv_f32_indexed_upto(ea, ff, 1, l.w_down, ff, (int64_t)W * ff, tidx, E, ye, W, Z, W, ff, stream));
      }
      sa.mix = l.hc2_mix; sa.out = l.hc2_out; sa.ye = ye; sa.ldye = W; sa.slot_of = so; sa.top = top;     // the next read of the streams sums them
    }
    if (trace) MN_TRY(streams_stage(nullptr, nullptr, trace + (size_t)li * R * W, nullptr));
  }
  MN_TRY(streams_stage(nullptr, m->final_w, out, nullptr));
#undef MN_TRY
  return MN_OK;
}
