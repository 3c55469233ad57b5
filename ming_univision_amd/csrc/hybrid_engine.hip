// hybrid_engine.hip — the step function of hybrid-mixer sequence models (mingnative.h sections 11 and 13): one pass of the layer runs over
// the rows of a step as a chain of launches on the caller's stream.  A run is
//   h = norm(x) w                                  (RMS or LayerNorm, fused with the previous run's residual add and expert combine)
//   [mixer's inputs ; up ; router] = W_in h        ONE product for the mixer's and the feed-forward's input projections
//   mixer    attention:      head norms + temperature + append, then the block attention with the heads' sinks
//            lightning:      the recurrence (row by row, one decode row cut over many workgroups, or the chunked scan), RMS x sigmoid gate
//            talk attention: rotation + unit norms + append (values = the projected keys), the attention with mixed heads
//            channel delta:  filters + silu + unit norms + write strengths; the low-rank decays and gates in one launch (decode rows: all
//                            of this and the feed-forward's activation in one launch); the recurrence; per-head RMS x gate
//            gla:            the low-rank decays, the recurrence straight from the stacked product, per-head RMS x silu gate
//   x += [mixer | act(up)] [W_o | W_down]^T        ONE product for the mixer's output and the dense / shared expert's down projection
//   experts of a mixture: as in pmix_engine.hip (sorted by expert on the grouped MFMA GEMMs, or pair by pair on fp32 FMA); picks that
//            stand for the input itself get no product: they sort behind the last expert and the combine adds w * h for them.
// Matrix products go through the routing of seq_linear.h.
#include "seq_linear.h"

extern "C" size_t mn_sizeof_hyb_layer(void) { return sizeof(mn_hyb_layer); }
extern "C" size_t mn_sizeof_hyb_model(void) { return sizeof(mn_hyb_model); }
extern "C" size_t mn_sizeof_hyb_state(void) { return sizeof(mn_hyb_state); }

namespace {

struct HDims {
  int cq;                                                        // floats of a row's prepared queries (channel delta: its q, k and v channels)
  int n_mix;                                                     // rows of the mixer in the stacked product
  int off_g, off_a1, off_g1, off_b;                              // columns: the gate, the low-rank projections, the write strengths
  int n_up, n_router, off_up, off_router, n_in, hv, n_cat;
  int n_dec, n_gate, n_beta;                                     // decays, low-rank gates, write strengths of a row
};

bool attention_kind(int kind) { return kind == MN_HYB_ATTENTION || kind == MN_HYB_TALK_ATTENTION; }

HDims hdims(const mn_hyb_layer& l) {
  HDims d{};
  const int G = (l.kind == MN_HYB_LIGHTNING || l.kind == MN_HYB_GLA) ? l.heads : l.kv_heads;
  const int q = l.heads * l.dim, k = G * l.dim, v = G * l.vdim;
  d.hv = l.heads * l.vdim;
  d.cq = q;
  switch (l.kind) {
    case MN_HYB_LIGHTNING: d.off_g = q + k + v; d.n_mix = d.off_g + d.hv; break;
    case MN_HYB_TALK_ATTENTION: d.n_mix = q + k; break;
    case MN_HYB_CHANNEL_DELTA:
      d.cq = 2 * k + d.hv;
      d.off_a1 = d.cq; d.off_g1 = d.off_a1 + l.rank_a; d.off_b = d.off_g1 + l.rank_g;
      d.n_mix = d.off_b + l.heads;
      d.n_dec = q; d.n_gate = d.hv; d.n_beta = l.heads;
      break;
    case MN_HYB_GLA: d.off_g = q + k + v; d.off_a1 = d.off_g + d.hv; d.n_mix = d.off_a1 + l.rank_a; d.n_dec = q; break;
    default: d.n_mix = q + k + v;
  }
  d.n_up = l.ff_kind == MN_HYB_FF_NONE ? 0 : l.ff;
  d.n_router = l.ff_kind == MN_HYB_FF_MOE && !l.table ? l.experts + l.pass : 0;
  d.off_up = d.n_mix;
  d.off_router = d.off_up + d.n_up;
  d.n_in = (d.off_router + d.n_router + 7) / 8 * 8;             // zero rows pad the stack to a multiple of 8
  d.n_cat = d.hv + d.n_up;
  return d;
}

struct HPlan {
  int n_in = 1, cq = 1, hv = 1, n_cat = 1, top = 1, eff = 1, eup = 1, experts = 1, dec = 1, gate = 1, beta = 1;
  size_t gemm_ws = 0, attn_ws = 0;
  int64_t lin = 0;                                               // largest heads x dim x vdim of a lightning recurrence
  size_t gla = 0;                                                // largest bytes of a gla layer's chunk state
};

enum { EXPERTS_INDEXED = 0, EXPERTS_GROUPED = 1, EXPERTS_TILES = 2 };
int expert_route(const mn_hyb_model* m, const mn_hyb_layer& l, int M) {
  if (m->arith != MN_SEQ_ARITH_BF16 || M <= 8 || l.experts + 1 > 128 || (int64_t)M * l.top > 65536 ||
      ((((uintptr_t)l.w_up) | ((uintptr_t)l.w_down)) & 15) != 0)
    return EXPERTS_INDEXED;
  const int64_t W = m->width, ff = l.expert_ff;
  if ((W % 64) == 0 && (ff % 64) == 0 && (l.expert_glu ? 2 : 1) * ff * W * 2 < ((int64_t)1 << 32) && (int64_t)M * l.top * (W > ff ? W : ff) * 2 < ((int64_t)1 << 32))
    return EXPERTS_TILES;
  if ((W % 8) == 0 && (ff % 8) == 0) return EXPERTS_GROUPED;
  return EXPERTS_INDEXED;
}

HPlan make_plan(const mn_hyb_model* m, int M) {
  HPlan p;
  for (int i = 0; i < m->n_layers; ++i) {
    const mn_hyb_layer& l = m->layers[i];
    const HDims d = hdims(l);
    if (d.n_in > p.n_in) p.n_in = d.n_in;
    if (d.cq > p.cq) p.cq = d.cq;
    if (d.hv > p.hv) p.hv = d.hv;
    if (d.n_cat > p.n_cat) p.n_cat = d.n_cat;
    if (l.ff_kind == MN_HYB_FF_MOE) {
      if (l.top > p.top) p.top = l.top;
      if (l.expert_ff > p.eff) p.eff = l.expert_ff;
      const int up = (l.expert_glu ? 2 : 1) * l.expert_ff;       // values of a pair's input product
      if (up > p.eup) p.eup = up;
      if (l.experts > p.experts) p.experts = l.experts;
    }
    if (d.n_dec > p.dec) p.dec = d.n_dec;
    if (d.n_gate > p.gate) p.gate = d.n_gate;
    if (d.n_beta > p.beta) p.beta = d.n_beta;
    if (l.kind == MN_HYB_ATTENTION) {
      const size_t aw = (size_t)4 * mn_num_cus() * 16 * (2 + (size_t)l.vdim) * sizeof(float);
      if (aw > p.attn_ws) p.attn_ws = aw;
    } else if (l.kind == MN_HYB_TALK_ATTENTION) {                // (runs x splits) of a launch stay near two workgroups per compute unit
      const size_t aw = mn_talk_attn_workspace_bytes(mn_num_cus(), l.heads, l.kv_heads, l.dim, M > 1 && m->block_rows > 0 ? m->block_rows : 1, 2);
      if (aw > p.attn_ws) p.attn_ws = aw;
    } else if (l.kind == MN_HYB_LIGHTNING) {
      const int64_t s = (int64_t)l.heads * l.dim * l.vdim;
      if (s > p.lin) p.lin = s;
    } else if (l.kind == MN_HYB_GLA) {
      const size_t s = mn_channel_scan_workspace_bytes(1, l.heads, l.dim, l.vdim);
      if (s > p.gla) p.gla = s;
    }
    if (m->arith == MN_SEQ_ARITH_BF16 && M > 8 && M <= 64) {       // scratch of the weight-streaming MFMA route: the largest product of the stack
      const int W = m->width;
      const int shapes[2][2] = {{d.n_in, W}, {W, d.n_cat}};
      for (const auto& nk : shapes) {
        if (nk[0] < 1 || nk[1] < 8 || (nk[1] % 8) != 0) continue;
        const size_t g = mn_skinny_workspace_bytes(M, nk[0], nk[1], MN_EPI_NONE);
        if (g > p.gemm_ws) p.gemm_ws = g;
      }
    }
  }
  return p;
}

// chunk states the scans of a step may hold: full chunks plus one ragged chunk for each of up to 64 sequences; steps too short for a
// scan hold none
inline size_t scan_bytes(const HPlan& p, int M) {
  const int c = mn_lightning_chunk_rows(), g = mn_channel_chunk_rows();
  const size_t light = M >= 2 * c ? (size_t)(mn_cdiv(M, c) + 64) * (size_t)p.lin * sizeof(float) : 0;
  const size_t chan = M >= 2 * g ? (size_t)(mn_cdiv(M, g) + 64) * p.gla : 0;
  return light > chan ? light : chan;
}

}  // namespace

extern "C" size_t mn_hyb_workspace_bytes(const mn_hyb_model* m, int M) {
  if (!m || !m->layers || M < 1) return 0;
  const HPlan p = make_plan(m, M);
  const size_t W = m->width, R = (size_t)M, Z = R * p.top;
  size_t n = 0;
  n += al(R * W * 4);                                  // residual
  n += al(R * W * 4) + al(R * W * 2);                  // normed rows + bf16
  n += al(R * p.n_in * 4);                             // stacked input projections
  n += al(R * p.cq * 4);                               // queries
  n += al(R * p.hv * 4);                               // the recurrence's heads before their norm
  n += al(R * p.n_cat * 4) + al(R * p.n_cat * 2);      // [mixer | activation] + bf16
  n += al(R * W * 4);                                  // their joined output product
  n += 2 * al(Z * 4);                                  // chosen experts, weights
  n += al(Z * p.eup * 4);                              // [gate ; up] or up of the pairs
  n += al(Z * p.eff * 4) + al(Z * p.eff * 2);          // their activation + bf16
  n += al(Z * W * 4);                                  // their results
  n += al(Z * W * 2);                                  // gathered bf16 rows
  n += 2 * al(((size_t)p.experts + 2) * 4) + 2 * al(Z * 4);   // counts, offsets, perm, slot_of
  n += 2 * al((Z / 256 + p.experts + 2) * 4) + al(4);         // live row tiles of the grouped products, their count
  n += al(p.gemm_ws) + al(p.attn_ws);
  n += al(scan_bytes(p, M));                           // chunk states of the recurrence's scan
  n += al(R * p.dec * 4) + al(R * p.gate * 4) + al(R * p.beta * 4);   // decays per key channel, low-rank gates, write strengths
  return n;
}

extern "C" int mn_hyb_step(const mn_hyb_model* m, const mn_hyb_state* st, const float* x, int64_t ldx, int M, const int32_t* row_tok,
                           const int32_t* row_seq, const int32_t* row_slot, const int32_t* row_back, const int32_t* blk_tab, int n_blk,
                           const int32_t* chunk_tab, int n_chunks, int max_len, int flags, float* out, float* trace, void* workspace, size_t workspace_bytes, void* stream) {
  MN_CHECK_ARG(m && st && m->layers && m->run_layer && m->final_w && x && row_seq && row_slot && row_back && out && workspace,
               "mn_hyb_step: null pointer");
  MN_CHECK_ARG(st->k && st->v && st->lin && st->conv, "mn_hyb_step: null state table");
  MN_CHECK_ARG(M >= 1 && M <= 65535 && m->width >= 1 && m->n_layers >= 1 && m->n_runs >= 1, "mn_hyb_step: bad sizes (M=%d)", M);
  MN_CHECK_ARG(workspace_bytes >= mn_hyb_workspace_bytes(m, M), "mn_hyb_step: workspace too small");
  const bool one_row = (flags & MN_SEQ_ROWS_DISTINCT) != 0;
  MN_CHECK_ARG(one_row || (blk_tab && n_blk >= 1 && n_blk <= M), "mn_hyb_step: rows that share sequences need the table of their runs");
  MN_CHECK_ARG(max_len >= 1 && max_len <= st->t_max, "mn_hyb_step: max_len=%d outside the cache (t_max=%d)", max_len, st->t_max);
  if (one_row) n_blk = M;
  const HPlan p = make_plan(m, M);
  const int W = m->width, arith = m->arith;
  const size_t R = (size_t)M, Zmax = R * p.top;
  MN_CHECK_ARG(Zmax <= 65535, "mn_hyb_step: %d rows x %d picks exceed 65535 (row, expert) pairs per step", M, p.top);
  const bool want16 = arith == MN_SEQ_ARITH_BF16 && M > 64;       // bf16 copies feed the tiled MFMA GEMMs only
  char* wp = reinterpret_cast<char*>(workspace);
  auto take = [&](size_t bytes) { char* q = wp; wp += al(bytes); return q; };
  float* xr = (float*)take(R * W * 4);
  float* hf = (float*)take(R * W * 4);
  uint16_t* hh = (uint16_t*)take(R * W * 2);
  float* pin = (float*)take(R * p.n_in * 4);
  float* qf = (float*)take(R * p.cq * 4);
  float* lo = (float*)take(R * p.hv * 4);
  float* cat = (float*)take(R * p.n_cat * 4);
  uint16_t* cath = (uint16_t*)take(R * p.n_cat * 2);
  float* yf = (float*)take(R * W * 4);
  int32_t* tidx = (int32_t*)take(Zmax * 4);
  float* tw = (float*)take(Zmax * 4);
  float* gu = (float*)take(Zmax * p.eup * 4);
  float* ea = (float*)take(Zmax * p.eff * 4);
  uint16_t* eah = (uint16_t*)take(Zmax * p.eff * 2);
  float* ye = (float*)take(Zmax * W * 4);
  uint16_t* xg = (uint16_t*)take(Zmax * W * 2);
  int32_t* counts = (int32_t*)take(((size_t)p.experts + 2) * 4);
  int32_t* offsets = (int32_t*)take(((size_t)p.experts + 2) * 4);
  int32_t* perm = (int32_t*)take(Zmax * 4);
  int32_t* slot_of = (int32_t*)take(Zmax * 4);
  int32_t* tile_g = (int32_t*)take((Zmax / 256 + p.experts + 2) * 4);
  int32_t* tile_m0 = (int32_t*)take((Zmax / 256 + p.experts + 2) * 4);
  int32_t* n_tiles = (int32_t*)take(4);
  uint16_t* const hh_buf = hh;
  void* gws = p.gemm_ws ? take(p.gemm_ws) : nullptr;
  const size_t gwb = p.gemm_ws;
  void* aws = take(p.attn_ws);
  const size_t scan_cap = scan_bytes(p, M);
  void* scanws = take(scan_cap);
  float* dec = (float*)take(R * p.dec * 4);
  float* gat = (float*)take(R * p.gate * 4);
  float* bet = (float*)take(R * p.beta * 4);
  if (!want16) hh = cath = nullptr;
  hipStream_t hs = mn_stream(stream);
  int rc;
#define MN_TRY(call) do { rc = (call); if (rc != MN_OK) return rc; } while (0)
  hipLaunchKernelGGL(copy_rows_kernel, dim3((unsigned)mn_cdiv(W, 256), (unsigned)M), dim3(256), 0, hs, x, ldx, xr, W);
  MN_CHECK_LAUNCH("mn_hyb_step(copy)");
  // what has not been added to x yet: a sublayer result, and the results of the experts with their weights
  struct { const float* y; const float* ye; const int32_t* so; const float* w; float w_all; int top; } pend = {nullptr, nullptr, nullptr, nullptr, 0.f, 0};
  const bool layer_norm = m->norm == MN_HYB_NORM_LAYER;
  // decode rows without bf16 copies: residual add + norm as one workgroup per row with the row in registers (the launch the
  // parallel-mixer step uses for its decode rows, here without a filter)
  const bool fuse = one_row && !want16 && W <= 8192;
  // x += what is pending; then the norm with weight w (NULL: the sum only) into h / h16
  auto norm_stage = [&](const uint16_t* w, float* h, uint16_t* h16) -> int {
    int rc2;
    if (layer_norm)
      rc2 = mn_add_layernorm_rows(xr, W, pend.y, W, pend.ye, W, pend.so, pend.w, pend.w_all, pend.top, w, m->eps, h, W, h16, W, M, W, stream);
    else if (fuse && w && h && !h16)
      rc2 = mn_axpy_rms_filter_rows(xr, W, pend.y, W, 1.0f, w, m->eps, nullptr, 0, nullptr, row_seq, row_slot, h, W, M, W, stream);
    else
      rc2 = mn_axpy_rms_rows(xr, W, pend.y, W, 1.0f, w, m->eps, h, W, h16, W, M, W, stream);
    pend = {nullptr, nullptr, nullptr, nullptr, 0.f, 0};
    return rc2;
  };
  for (int ri = 0; ri < m->n_runs; ++ri) {
    const int li = m->run_layer[ri];
    MN_CHECK_ARG(li >= 0 && li < m->n_layers, "mn_hyb_step: run %d names layer %d", ri, li);
    const mn_hyb_layer& l = m->layers[li];
    const HDims d = hdims(l);
    const bool attn = l.kind == MN_HYB_ATTENTION, talk = l.kind == MN_HYB_TALK_ATTENTION, delta = l.kind == MN_HYB_CHANNEL_DELTA,
               gla = l.kind == MN_HYB_GLA, moe = l.ff_kind == MN_HYB_FF_MOE;
    MN_CHECK_ARG(l.kind >= MN_HYB_ATTENTION && l.kind <= MN_HYB_GLA && l.heads >= 1 && l.dim >= 1 && l.vdim >= 1 &&
                     (!(attn || talk || delta) || (l.kv_heads >= 1 && (l.heads % l.kv_heads) == 0)) && l.ff_kind >= MN_HYB_FF_NONE &&
                     l.ff_kind <= MN_HYB_FF_MOE && (l.ff_kind != MN_HYB_FF_DENSE || l.ff >= 1) &&
                     (!moe || (l.experts >= 1 && l.pass >= 0 && l.top >= 1 && l.top <= l.experts + l.pass && l.expert_ff >= 1 && l.ff >= 0 &&
                               l.w_up && l.w_down && (!l.table || (row_tok && m->vocab >= 1 && l.pass == 0)))) && l.norm1 && l.w_in && l.w_out,
                 "mn_hyb_step: layer %d: bad sizes or null weights", li);
    MN_CHECK_ARG((l.kind != MN_HYB_LIGHTNING || (l.decay && l.mix_norm)) &&
                     (!talk || (l.talk && l.vdim == l.dim && l.window >= 0 && l.chunk >= 0 && (l.rot_dims == 0 || l.rot_freq))) &&
                     (!delta || (l.conv >= 1 && l.rank_a >= 1 && l.rank_g >= 1 && l.w_conv && l.a_log && l.w_a2 && l.b_a2 && l.w_g2 && l.mix_norm)) &&
                     (!gla || (l.rank_a >= 1 && l.w_a2 && l.mix_norm)),
                 "mn_hyb_step: layer %d: bad sizes or null weights of its mixer", li);
    MN_CHECK_ARG(attention_kind(l.kind) ? (st->k[ri] && st->v[ri]) : (st->lin[ri] && (!delta || l.conv == 1 || st->conv[ri])),
                 "mn_hyb_step: run %d: null state", ri);
    // ---- the input both sublayers read, and their stacked projections ----
    // rows wide enough for the bf16 copy need the fp32 rows only where something still reads them
    const int route = moe ? expert_route(m, l, M) : EXPERTS_TILES;
    const bool h16_only = layer_norm && hh && mfma_ok(l.w_in, W) && route != EXPERTS_INDEXED && (!moe || l.pass == 0);
    const bool cat16_only = cath && mfma_ok(l.w_out, d.n_cat);
    MN_TRY(norm_stage(l.norm1, h16_only ? nullptr : hf, hh));
    MN_TRY(linear(arith, M, hf, W, hh, W, l.w_in, d.n_in, W, nullptr, pin, d.n_in, gws, gwb, stream));
    // ---- decode rows of the channel-decay mixers: what depends on the stacked product alone, in one launch ----
    const int E = l.experts, top = l.top, eff = l.expert_ff, Z = M * top;
    const bool prepped = one_row && M <= 64 && !cath && (delta || gla) && (d.n_up == 0 || l.ff_act == MN_HYB_ACT_XIELU) && (!moe || (l.table && layer_norm));
    const mn_low_rank_job jobs[2] = {
        {pin + d.off_a1, d.n_in, l.w_a2, l.b_a2, l.a_log, dec, d.n_dec, l.rank_a, d.n_dec, delta ? MN_LOW_RANK_DECAY : MN_LOW_RANK_ROOT, l.dim, l.root},
        {pin + d.off_g1, d.n_in, l.w_g2, nullptr, nullptr, gat, d.hv, l.rank_g, d.hv, MN_LOW_RANK_SIGMOID, 1, 1.0f}};
    const float unit_scale = 1.0f / sqrtf((float)l.dim);
    if (prepped) {
      mn_rows_prep r;
      memset(&r, 0, sizeof(r));
      if (delta) {
        r.delta = 1; r.proj = pin; r.ld = d.n_in; r.H = l.heads; r.G = l.kv_heads; r.dim = l.dim; r.vdim = l.vdim; r.taps = l.conv; r.off_b = d.off_b;
        r.w_conv = l.w_conv; r.conv_state = st->conv[ri]; r.unit_eps = l.unit_eps; r.q_scale = unit_scale;
        r.qkv = qf; r.ldqkv = d.cq; r.beta = bet; r.ldbeta = l.heads;
      }
      r.n_jobs = delta ? 2 : 1; r.job[0] = jobs[0]; r.job[1] = jobs[1];
      if (d.n_up > 0) {
        r.act_x = pin + d.off_up; r.ld_act_x = d.n_in; r.act_pos = l.act_pos; r.act_neg = l.act_neg;
        r.act_y = cat + d.hv; r.ld_act_y = d.n_cat; r.act_n = d.n_up;
      }
      if (moe) { r.table = l.table; r.tok = row_tok; r.vocab = m->vocab; r.top = top; r.idx = tidx; }
      MN_TRY(mn_rows_prep_launch(&r, row_seq, row_slot, M, stream));
    }
    // ---- mixer ----
    if (attn) {
      MN_TRY(mn_head_norm_temp_append(pin, d.n_in, M, l.heads, l.kv_heads, l.dim, l.vdim, l.q_norm, l.k_norm, m->eps, l.scale, l.temp_coef,
                                      l.temp_every, row_seq, row_slot, qf, d.cq, st->k[ri], st->v[ri], st->t_max, stream));
      int ns = mn_window_attn_splits(n_blk, l.heads, l.kv_heads, one_row, max_len);
      while (ns > 1 && mn_window_attn_workspace_bytes(n_blk, l.heads, l.kv_heads, l.vdim, one_row, ns) > p.attn_ws) --ns;
      MN_TRY(mn_window_pool_attn_blocks_sink(qf, d.cq, st->k[ri], st->v[ri], nullptr, nullptr, l.sink, row_seq, row_slot, blk_tab, n_blk, one_row,
                                             l.heads, l.kv_heads, l.dim, l.vdim, st->t_max, 1, 0, 0, 1.0f, cat, d.n_cat, cath, d.n_cat, ns, aws,
                                             p.attn_ws, -1, stream));
    } else if (talk) {
      const int ck = l.kv_heads * l.dim, rows = one_row ? 1 : m->block_rows;
      MN_TRY(mn_rope_unit_append_from(pin, d.n_in, M, l.heads, l.kv_heads, l.dim, l.dim, l.heads * l.dim, l.rot_dims, l.rot_freq, 1.0f, 1, m->eps,
                                      l.scale, row_seq, row_slot, qf, d.cq, st->k[ri], st->v[ri], st->t_max, stream));
      int keys = max_len;
      if (l.window > 0 && l.window + rows - 1 < keys) keys = l.window + rows - 1;
      if (l.chunk > 0 && l.chunk + rows - 1 < keys) keys = l.chunk + rows - 1;
      int ns = mn_talk_attn_splits(n_blk, keys);
      while (ns > 1 && mn_talk_attn_workspace_bytes(n_blk, l.heads, l.kv_heads, l.dim, rows, ns) > p.attn_ws) --ns;
      MN_TRY(mn_talk_attn(qf, d.cq, st->k[ri], ck, st->v[ri], ck, l.talk, l.sink, row_seq, row_slot, M, one_row ? nullptr : blk_tab, n_blk, rows,
                          l.heads, l.kv_heads, l.dim, st->t_max, l.window, l.chunk, cat16_only ? nullptr : cat, d.n_cat, cath, d.n_cat, ns, aws,
                          p.attn_ws, -1, stream));
    } else if (delta) {
      if (!prepped) {
        MN_TRY(mn_delta_prep_rows(pin, d.n_in, M, l.heads, l.kv_heads, l.dim, l.vdim, d.off_b, 0, l.w_conv, l.conv, st->conv[ri], one_row ? 1 : 0,
                                  nullptr, nullptr, l.unit_eps, unit_scale, row_seq, row_slot, row_back, qf, d.cq, bet, l.heads, stream));
        if (l.conv > 1 && !one_row) MN_TRY(mn_tap_state_update(pin, d.n_in, l.conv, st->conv[ri], row_seq, row_back, M, d.cq, stream));
        MN_TRY(mn_low_rank_gate_rows(jobs, 2, M, stream));
      }
      MN_TRY(mn_channel_state_rows(qf, d.cq, dec, d.n_dec, bet, l.heads, M, l.heads, l.kv_heads, l.dim, l.vdim, 1.0f, st->lin[ri], row_seq, row_slot,
                                   row_back, blk_tab, n_blk, one_row ? MN_SEQ_ROWS_DISTINCT : 0, lo, d.hv, stream));
      MN_TRY(mn_head_rms_gate_rows(lo, d.hv, l.mix_norm, m->eps, gat, d.hv, MN_GATE_ACT_NONE, cat16_only ? nullptr : cat, d.n_cat, cath, d.n_cat, M,
                                   l.heads, l.vdim, stream));
    } else if (gla) {
      if (!prepped) MN_TRY(mn_low_rank_gate_rows(jobs, 1, M, stream));
      if (!one_row && chunk_tab && n_chunks >= 1 && M >= 2 * mn_channel_chunk_rows() && l.dim <= 256 &&
          mn_channel_scan_workspace_bytes(n_chunks, l.heads, l.dim, l.vdim) <= scan_cap)
        MN_TRY(mn_channel_state_rows_scan(pin, d.n_in, dec, d.n_dec, M, l.heads, l.heads, l.dim, l.vdim, unit_scale, st->lin[ri], row_seq, row_slot,
                                          row_back, chunk_tab, n_chunks, lo, d.hv, scanws, scan_cap, stream));
      else
        MN_TRY(mn_channel_state_rows(pin, d.n_in, dec, d.n_dec, nullptr, 0, M, l.heads, l.heads, l.dim, l.vdim, unit_scale, st->lin[ri], row_seq,
                                     row_slot, row_back, blk_tab, n_blk, one_row ? MN_SEQ_ROWS_DISTINCT : 0, lo, d.hv, stream));
      MN_TRY(mn_head_rms_gate_rows(lo, d.hv, l.mix_norm, m->eps, pin + d.off_g, d.n_in, MN_GATE_ACT_SILU, cat16_only ? nullptr : cat, d.n_cat, cath,
                                   d.n_cat, M, l.heads, l.vdim, stream));
    } else {
      const size_t lds3 = mn_lightning_scan_lds_bytes(l.dim, l.vdim);
      const bool scan = !one_row && chunk_tab && n_chunks >= 1 && M >= 2 * mn_lightning_chunk_rows() && lds3 <= 64 * 1024 &&
                        mn_lightning_scan_workspace_bytes(n_chunks, l.heads, l.dim, l.vdim) <= scan_cap;
      if (scan)
        MN_TRY(mn_lightning_rows_scan(pin, d.n_in, M, l.heads, l.dim, l.vdim, l.decay, st->lin[ri], row_seq, row_slot, row_back, chunk_tab,
                                      n_chunks, lo, d.hv, scanws, scan_cap, stream));
      else
        MN_TRY(mn_lightning_rows(pin, d.n_in, M, l.heads, l.dim, l.vdim, l.decay, st->lin[ri], row_seq, row_slot, row_back,
                                 one_row ? MN_SEQ_ROWS_DISTINCT : 0, lo, d.hv, stream));
      MN_TRY(mn_rms_sigmoid_gate_rows(lo, d.hv, l.mix_norm, m->eps, pin + d.off_g, d.n_in, cat, d.n_cat, cath, d.n_cat, M, d.hv, stream));
    }
    // ---- the feed-forward's activation and router; the joined output product ----
    if (moe && l.table && !prepped) MN_TRY(mn_token_table_rows(l.table, m->vocab, top, row_tok, M, tidx, layer_norm ? nullptr : tw, stream));
    const bool ride = moe && !l.table && d.n_up > 0 && !cath && l.ff_act == MN_HYB_ACT_RELU2;   // few rows: the shared activation rides the router's launch
    if (moe && !l.table)
      MN_TRY(mn_router_softmax_topk_rows(pin + d.off_router, d.n_in, M, d.n_router, E, top, l.correction, tidx, tw, ride ? pin + d.off_up : nullptr,
                                         d.n_in, ride ? cat + d.hv : nullptr, d.n_cat, ride ? d.n_up : 0, stream));
    if (d.n_up > 0 && !ride && !prepped) {
      float* ay = cat16_only ? nullptr : cat + d.hv;
      uint16_t* ah = cath ? cath + d.hv : nullptr;
      if (l.ff_act == MN_HYB_ACT_XIELU)
        MN_TRY(mn_xielu_rows(pin + d.off_up, d.n_in, l.act_pos, l.act_neg, ay, d.n_cat, ah, d.n_cat, M, d.n_up, stream));
      else
        MN_TRY(mn_relu2_rows(pin + d.off_up, d.n_in, ay, d.n_cat, ah, d.n_cat, M, d.n_up, stream));
    }
    MN_TRY(linear(arith, M, cat, d.n_cat, cath, d.n_cat, l.w_out, W, d.n_cat, nullptr, yf, W, gws, gwb, stream));
    pend.y = yf;
    if (moe) {
      const uint16_t* h16 = hh;
      const int32_t* so = nullptr;
      const int glu = l.expert_glu, eup = glu ? 2 * eff : eff;
      if (route != EXPERTS_INDEXED && !h16) {          // few rows: the input was written in fp32 only
        MN_TRY(mn_f32_to_bf16(hf, hh_buf, (int64_t)M * W, stream));
        h16 = hh_buf;
      }
      if (route == EXPERTS_TILES) {                    // group E (the picks that pass the input through) gets no tiles
        const int max_mtiles = Z / 256 + E;
        MN_TRY(mn_ep_dispatch(tidx, M, top, E + 1, 0, E, counts, offsets, perm, slot_of, 256, tile_g, tile_m0, n_tiles, stream));
        MN_TRY(mn_gemm256_grouped_tiles(h16, W, 0, M, perm, l.w_up, W, (int64_t)eup * W, offsets, counts, E, tile_g, tile_m0, n_tiles, max_mtiles,
                                        eah, eff, 0, eff, W, glu ? 6 : 7, stream));   // silu(gate) * up or the squared relu in the epilogue
        MN_TRY(mn_gemm256_grouped_tiles(eah, eff, 0, Z, nullptr, l.w_down, eff, (int64_t)W * eff, offsets, counts, E, tile_g, tile_m0, n_tiles,
                                        max_mtiles, ye, W, 0, W, eff, 0, stream));
        so = slot_of;
      } else if (route == EXPERTS_GROUPED) {
        MN_TRY(mn_moe_sort(tidx, M, top, E + 1, counts, offsets, perm, slot_of, stream));
        MN_TRY(mn_gather_rows_bf16(h16, W, perm, xg, W, Z, W, stream));
        MN_TRY(mn_gemm_bf16_grouped(xg, W, l.w_up, W, (int64_t)eup * W, offsets, counts, E, gu, eup, M, eup, W, MN_GEMM_F32, stream));
        if (glu) MN_TRY(mn_silu_mul_rows(gu, eup, nullptr, 0, eah, eff, Z, eff, stream));
        else MN_TRY(mn_relu2_rows(gu, eff, nullptr, 0, eah, eff, Z, eff, stream));
        MN_TRY(mn_gemm_bf16_grouped(eah, eff, l.w_down, eff, (int64_t)W * eff, offsets, counts, E, ye, W, M, W, eff, MN_GEMM_F32, stream));
        so = slot_of;
      } else {
        if (glu) {
          MN_TRY(mn_gemv_glu_indexed(hf, W, top, l.w_up, W, (int64_t)eup * W, tidx, E, ea, eff, Z, eff, W, stream));
        } else {
          MN_TRY(mn_gemv_f32_indexed_upto(hf, W, top, l.w_up, W, (int64_t)eff * W, tidx, E, gu, eff, Z, eff, W, stream));
          MN_TRY(mn_relu2_rows(gu, eff, ea, eff, nullptr, 0, Z, eff, stream));
        }
        MN_TRY(mn_gemv_f32_indexed_upto(ea, eff, 1, l.w_down, eff, (int64_t)W * eff, tidx, E, ye, W, Z, W, eff, stream));
      }
      if (layer_norm && l.pass == 0) {                 // the next norm's launch combines them
        pend.ye = ye; pend.so = so; pend.w = l.table ? nullptr : tw; pend.w_all = 1.0f / (float)top; pend.top = top;
      } else {
        MN_TRY(mn_moe_combine_pass_residual(xr, W, ye, W, so, tidx, tw, top, E, hf, W, yf, W, M, W, stream));
        pend.y = nullptr;
      }
    }
    if (trace) {
      if (pend.y || pend.ye) MN_TRY(norm_stage(nullptr, nullptr, nullptr));
      hipLaunchKernelGGL(copy_rows_kernel, dim3((unsigned)mn_cdiv(W, 256), (unsigned)M), dim3(256), 0, hs, xr, (int64_t)W,
                         trace + (size_t)ri * R * W, W);
      MN_CHECK_LAUNCH("mn_hyb_step(trace)");
    }
  }
  MN_TRY(norm_stage(m->final_w, out, nullptr));
#undef MN_TRY
  return MN_OK;
}
