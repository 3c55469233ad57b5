"""Sabezen on the HIP path against tests/sabezen_oracle.py (plain float64 restatement, one function per mechanism).

Small random models of several shapes (all three mixers in different orders, dense and table-routed feed-forwards and none, sizes that are
no multiples of 4 or 8, one head, everything equal or 1, chunks of 1, of a few tokens and longer than any request, no chunk, no rotation,
partial and full rotation, one filter tap, many heads on one key head, as many key heads as heads, states beyond the register walk).
fp32 arithmetic is held to 1e-4 of the logits' scale, the bf16-MFMA arithmetic to 3e-2.  Covers: every operator alone (attention with
scores scaled up until one key decides — the chunk's first slot, the last slot of the chunk before it, the row's own slot, window edges,
key-tile and key-split edges — in runs of rows across chunk borders and in decode rows, on the matrix-core and the plain kernel; the
recurrences row by row, as decode rows and as a chunked scan on stale, stored and fresh states, with decays near 0 and writes kept for
hundreds of tokens); whole prompts with the residual stream after every layer; token-by-token decoding; portions down to two tokens;
several unequal requests in one pass against each alone; inputs longer than a pass; cache sequences that are released and reused; the
first positions of a sequence; long decoding; the bf16 arithmetic; greedy generation through the generation entry point; the captured
decode step; the trace runner."""
import copy
import ctypes as C
import json
import os
import subprocess

import numpy as np
import pytest
import torch

from tests import sabezen_oracle as O

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64


def config(name):
    A, Dl, Gl, dense, moe = O.attention_layer, O.delta_layer, O.gla_layer, O.dense, O.moe
    if name == "mixed":     # all mixers, both feed-forwards, a layer without one, small chunks
        return O.small_config([Dl(mlp=dense(96)), Gl(mlp=moe(7, 3, 16)), A(mlp=dense(40)), Dl(heads=2, kv_heads=1, dim=32, vdim=24, conv=4, rank_a=16, rank_g=8),
                               A(heads=6, kv_heads=2, dim=20, rot=(700.0, 20), chunk=23, mlp=moe(4, 1, 24)), Gl(heads=2, dim=24, vdim=8, tau=3.0, mlp=dense(32))])
    if name == "odd":       # no size a multiple of 4 or 8 (products on the fp32 FMA kernels, attention on the plain kernel), other constants
        return O.small_config([A(heads=3, kv_heads=1, dim=10, scale=0.4, rot=(500.0, 6), chunk=13, mlp=dense(30)),
                               Dl(heads=3, kv_heads=3, dim=10, vdim=6, conv=5, rank_a=5, rank_g=3, mlp=moe(3, 2, 14)),
                               Gl(heads=5, dim=6, vdim=7, tau=1.0, rank=9, mlp=dense(22))], width=44, vocab=61, scale=0.7, eps=1e-3)
    if name == "ones":      # values a model may happen to make equal or 1; no chunk, no rotation, one tap, a chunk of one position
        return O.small_config([A(heads=1, kv_heads=1, dim=32, scale=1.0, rot=None, chunk=None, mlp=dense(32)),
                               Dl(heads=1, kv_heads=1, dim=32, vdim=32, conv=1, rank_a=32, rank_g=32, mlp=moe(1, 1, 32)),
                               A(heads=32, kv_heads=32, dim=4, scale=1.0, rot=(32.0, 4), chunk=1, mlp=moe(2, 2, 32)),
                               Gl(heads=1, dim=32, vdim=32, tau=1.0, rank=1, mlp=dense(32))], width=32, vocab=32, scale=1.0)
    if name == "wide":      # twelve heads on one key head, forty heads on five, states of 136 and 264 rows
        return O.small_config([A(heads=12, kv_heads=1, dim=8, rot=(10000.0, 8), chunk=70, mlp=dense(16)),
                               Dl(heads=2, kv_heads=1, dim=136, vdim=40, conv=2, mlp=dense(16)),
                               A(heads=40, kv_heads=5, dim=8, rot=(100.0, 2), chunk=33, mlp=moe(9, 4, 8)), Gl(heads=2, dim=264, vdim=12, tau=20.0)],
                              width=32, vocab=40, scale=3.0)
    if name == "tail":      # heads of 72 and 132 values (the attention's larger instances), chunks longer than any request
        return O.small_config([Gl(heads=4, dim=8, vdim=72, tau=5.0), A(heads=4, kv_heads=4, dim=72, scale=0.1, rot=(1e6, 72), chunk=1000, mlp=dense(64)),
                               A(heads=3, kv_heads=3, dim=132, scale=0.1, rot=(1e4, 64), chunk=300, mlp=moe(16, 2, 64)),
                               Dl(heads=4, kv_heads=2, dim=24, vdim=8, conv=4, mlp=dense(64))], width=64, vocab=50)
    raise KeyError(name)


MODELS = ("mixed", "odd", "ones", "wide", "tail")


def build(cfg, sd, arith="f32", t_max=512, n_seq=1):
    from ming_univision_amd.configuration import SabezenConfig
    from ming_univision_amd.sabezen import SabezenDecoder
    return SabezenDecoder(SabezenConfig.from_dict(O.config_json(cfg)), {k: v.cuda() for k, v in sd.items()}, t_max=t_max, n_seq=n_seq, arith=arith)


def make(name, arith="f32", seed=0, t_max=512, n_seq=1, peaky=1.0):
    cfg = config(name)
    if peaky != 1.0:
        cfg = copy.deepcopy(cfg)
        for ly in cfg["layers"]:
            if ly["type"] == "attention":
                ly["mixer"]["scale"] *= peaky
    sd = O.random_weights(cfg, seed)
    return cfg, sd, build(cfg, sd, arith, t_max, n_seq)


def toks(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def err(got, want):
    want = want.double()
    return float((got.double().cpu() - want).abs().max() / want.abs().max().clamp_min(1e-9))


def ref_logits(cfg, sd, t):
    return O.forward(cfg, sd, t)[0]


def run_spans(dec, ids, spans, trace=False):
    ids = torch.tensor(ids, device="cuda")
    return dec.forward_spans(dec.embed(ids), spans, trace=trace, tokens=ids)


def run_portions(dec, seq, tokens, cuts):
    """Feed `tokens` to cache sequence `seq` in portions of the given sizes; returns the logits of every position."""
    out, at = [], 0
    for n in cuts:
        out.append(dec.logits(run_spans(dec, tokens[at:at + n], [(seq, n, at)])))
        at += n
    assert at == len(tokens)
    return torch.cat(out, 0)


def _api():
    from ming_univision_amd._lib import check, current_stream, lib, ptr
    return check, current_stream, lib(), ptr


def _rows(spans, block_rows=1 << 30, chunk_rows=0):
    from ming_univision_amd.sequences import rows_of_spans
    t = rows_of_spans(spans, block_rows, chunk_rows)
    return {k: torch.from_numpy(v).cuda() for k, v in t.items() if k != "max_len"}


def _bf(t):
    return t.to(torch.bfloat16)


_KEEP = []


def D(t):
    """A device copy that outlives the launch it is passed to (the pointer alone would not keep the memory)."""
    _KEEP.append(t.cuda())
    return _KEEP[-1]


@pytest.fixture(autouse=True)
def _drop_device_copies():
    yield
    torch.cuda.synchronize()
    _KEEP.clear()


# ---- operators alone -------------------------------------------------------------------------------------------------------
def test_residual_sum_expert_combine_and_layer_norm():
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(0)
    for M, n, top in ((5, 44, 2), (3, 1, 0), (70, 1000, 3), (2, 2100, 1), (3, 4096, 2), (2, 8200, 2), (3, 8192, 0), (2, 5001, 1)):
        for aligned in (True, False):
            ld = n + (4 if aligned else 3)
            x, y, w = torch.randn(M, ld, generator=g) * 2 + 3, torch.randn(M, ld, generator=g), _bf(1 + 0.2 * torch.randn(n, generator=g))
            ye = torch.randn(max(1, M * top), ld, generator=g)
            slot, ew = torch.randperm(max(1, M * top), generator=g).to(torch.int32), torch.rand(max(1, M * top), generator=g)
            for weights in (True, False):
                xd, h, h16 = x.cuda(), torch.zeros(M, n, device="cuda"), torch.zeros(M, n, dtype=torch.bfloat16, device="cuda")
                check(L.mn_add_layernorm_rows(ptr(xd), ld, ptr(D(y)), ld, ptr(D(ye)) if top else None, ld, ptr(D(slot)), ptr(D(ew)) if weights else None,
                                              0.25, top, ptr(D(w)), 1e-3, ptr(h), n, ptr(h16), n, M, n, stream()))
                ref = x[:, :n].double() + y[:, :n].double()
                for j in range(top):
                    z = torch.arange(M) * top + j
                    ref = ref + (ew[z].double() if weights else torch.full((M,), 0.25, dtype=F64))[:, None] * ye[slot[z].long()][:, :n].double()
                nref = O.layer_norm(ref, w, 1e-3)
                assert err(xd[:, :n], ref) < 1e-6 and bool((xd[:, n:].cpu() == x[:, n:]).all())
                assert err(h, nref) < 5e-6 and err(h16.float(), nref) < 1e-2, (M, n, top)
        xd = x.cuda()                                                # the sum alone
        check(L.mn_add_layernorm_rows(ptr(xd), ld, ptr(D(y)), ld, None, 0, None, None, 0.0, 0, None, 1e-3, None, 0, None, 0, M, n, stream()))
        assert err(xd[:, :n], x[:, :n].double() + y[:, :n].double()) < 1e-6


def test_xielu_and_table_rows():
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(1)
    for M, n in ((5, 44), (3, 1), (70, 1023), (2, 4100)):
        x = torch.randn(M, n + 1, generator=g) * 4
        x[0, 0], x[-1, n - 1] = -1e-4, 60.0
        p, q = torch.tensor(0.7, dtype=F64), torch.tensor(-1.3, dtype=F64)
        y, y16 = torch.zeros(M, n + 3, device="cuda"), torch.zeros(M, n, dtype=torch.bfloat16, device="cuda")
        check(L.mn_xielu_rows(ptr(D(x)), n + 1, float(O.softplus(p)), 0.5 + float(O.softplus(q)), ptr(y), n + 3, ptr(y16), n, M, n, stream()))
        ref = O.xielu(x[:, :n].double(), p, q)
        off = ((y[:, :n].double().cpu() - ref) / (ref.abs() + x[:, :n].double().abs())).abs().max()     # the two terms may cancel: relative to both
        assert float(off) < 2e-6 and err(y16.float(), ref) < 1e-2
        assert bool((y[:, n:] == 0).all())
    table, tok = torch.randint(0, 9, (13, 3), generator=g).to(torch.int32), torch.tensor([0, 12, 5, 5, 7], dtype=torch.int32)
    idx, w = torch.zeros(5, 3, dtype=torch.int32, device="cuda"), torch.zeros(5, 3, device="cuda")
    check(L.mn_token_table_rows(ptr(D(table)), 13, 3, ptr(D(tok)), 5, ptr(idx), ptr(w), stream()))
    assert bool((idx.cpu() == table[tok.long()]).all()) and bool((w == 1 / 3).all())


def low_rank_refs(a, cases):
    out = []
    for k0, k, w, b, kind, a_log, hn, root in cases:
        z = a[:, k0:k0 + k].double() @ w.double().T + (0 if b is None else b.double())
        if kind == 1:
            z = torch.exp(-torch.exp(a_log.double()).repeat_interleave(hn) * O.softplus(z))
        elif kind == 2:
            z = torch.sigmoid(z) ** root
        elif kind == 3:
            z = torch.sigmoid(z)
        out.append(z)
    return out


def test_low_rank_gates():
    from ming_univision_amd._lib import LowRankJob
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(2)
    for M in (1, 7, 20, 64, 65, 200):
        for k1, n1, k2, n2 in ((8, 32, 24, 40), (5, 30, 3, 18), (128, 200, 64, 70), (1, 4, 33, 129)):
            ld = k1 + k2 + (0 if (k1 + k2) % 4 == 0 else 1)
            a = torch.randn(M, ld, generator=g) * 3
            hn = 2
            cases = [(0, k1, _bf(torch.randn(n1, k1, generator=g) * k1 ** -0.5), _bf(torch.randn(n1, generator=g)), 1, torch.randn(n1 // hn, generator=g), hn, 1.0),
                     (k1, k2, _bf(torch.randn(n2, k2, generator=g) * k2 ** -0.5), None, 3, None, 1, 1.0)]
            if M % 2:
                cases[1] = (k1, k2, cases[1][2], _bf(2 * torch.randn(n2, generator=g)), 2, None, 1, 1 / 7.0)
            ad = D(a)
            outs = [torch.zeros(M, n1 + 1, device="cuda"), torch.zeros(M, n2, device="cuda")]
            jobs = (LowRankJob * 2)(*[LowRankJob(ad.data_ptr() + 4 * k0, ld, D(w).data_ptr(), D(b).data_ptr() if b is not None else None,
                                                 D(al).data_ptr() if al is not None else None, o.data_ptr(), o.shape[1], k, w.shape[0], kind, h, root)
                                      for (k0, k, w, b, kind, al, h, root), o in zip(cases, outs)])
            check(L.mn_low_rank_gate_rows(jobs, 2, M, stream()))
            for o, r in zip(outs, low_rank_refs(a, cases)):
                assert float((o[:, :r.shape[1]].double().cpu() - r).abs().max()) < 1e-5, (M, k1, k2)
            single = torch.zeros(M, n2, device="cuda")
            job = LowRankJob.from_buffer_copy(jobs[1])
            job.out = single.data_ptr()
            check(L.mn_low_rank_gate_rows(C.byref(job), 1, M, stream()))
            assert bool((single == outs[1]).all())


def test_rotated_unit_keys_and_values_from_the_projected_keys():
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(3)
    from ming_univision_amd.daberax import rotary_frequencies
    for H, G, d, rot in ((4, 2, 16, {"base": 1e4, "dims": 8}), (3, 1, 10, {"base": 500.0, "dims": 10}), (2, 2, 130, None)):
        spans = [(1, 7, 0), (0, 1, 999), (2, 5, 94)]
        M, t_max, eps, scale, ld = 13, 1004, 1e-5, 0.37, H * d + G * d + 3
        r = _rows(spans)
        qk = torch.randn(M, ld, generator=g) * 3
        q, ka, va = torch.zeros(M, H * d, device="cuda"), torch.full((3, t_max, G * d), 7.0, device="cuda"), torch.full((3, t_max, G * d), 7.0, device="cuda")
        fr = rotary_frequencies(rot, "cuda") if rot else None
        check(L.mn_rope_unit_append_from(ptr(D(qk)), ld, M, H, G, d, d, H * d, rot["dims"] if rot else 0, ptr(fr), 1.0, 1, eps, scale,
                                         ptr(r["row_seq"]), ptr(r["row_slot"]), ptr(q), H * d, ptr(ka), ptr(va), t_max, stream()))
        pos, seqs = r["row_slot"].tolist(), r["row_seq"].tolist()
        for m in range(M):
            qq, kk = qk[m:m + 1, :H * d].double().reshape(1, H, d), qk[m:m + 1, H * d:H * d + G * d].double().reshape(1, G, d)
            v = kk.clone()
            if rot:
                f = O.rotary_frequencies(rot)
                qq, kk = O.rotate_halves(qq, f, pos[m]), O.rotate_halves(kk, f, pos[m])
            tol = 2e-5 if pos[m] < 100 else 2e-4
            assert err(q[m], O.unit_rms(qq, eps).reshape(-1) * scale) < tol and err(ka[seqs[m], pos[m]], O.unit_rms(kk, eps).reshape(-1)) < tol
            assert err(va[seqs[m], pos[m]], v.reshape(-1)) < 1e-7
        ka[r["row_seq"].long(), r["row_slot"].long()] = 7.0
        assert bool((ka == 7.0).all())


def talk_case(H, G, d, T, chunk, window, rows, needle, scale, variant, nsplit=0, one_row=False, seed=0, sink=True, block=0, spread=0.4):
    """A sequence of T cached tokens; `rows` = consecutive positions of the query rows.  needle = (row index, key slot): that key is made to
    dominate that row's raw scores.  Returns (got, reference) [rows, H, d]."""
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(seed)
    k, v, q = torch.randn(T, G, d, generator=g), torch.randn(T, G, d, generator=g), torch.randn(len(rows), H, d, generator=g)
    if needle is not None:
        ri, slot = needle
        q[ri] = 6.0 * k[slot].repeat_interleave(H // G, 0) / scale / d ** 0.5
    talk = torch.eye(H) + spread * torch.randn(H, H, generator=g) * H ** -0.5
    sk = torch.randn(H, generator=g) if sink else None
    t_max, M = T + 5, len(rows)
    ka, va = torch.full((2, t_max, G * d), 1e4), torch.full((2, t_max, G * d), 1e4)      # slots past the sequence hold junk that must not be read
    ka[1, :T], va[1, :T] = k.reshape(T, -1), v.reshape(T, -1)
    row_seq, row_slot = torch.ones(M, dtype=torch.int32), torch.tensor(rows, dtype=torch.int32)
    br = 1 if one_row else (block or L.mn_talk_attn_block_rows(H, G, d) or 8)
    blk = torch.tensor([[i, min(br, M - i)] for i in range(0, M, br)], dtype=torch.int32)
    n_blk = blk.shape[0]
    ns = (nsplit or L.mn_talk_attn_splits(n_blk, T)) if variant == 0 else 1
    ws = torch.zeros(max(L.mn_talk_attn_workspace_bytes(n_blk, H, G, d, br, ns), 16), dtype=torch.uint8, device="cuda")
    out, out16 = torch.zeros(M, H * d, device="cuda"), torch.zeros(M, H * d, dtype=torch.bfloat16, device="cuda")
    check(L.mn_talk_attn(ptr(D(q.reshape(M, -1) * scale)), H * d, ptr(D(ka)), G * d, ptr(D(va)), G * d, ptr(D(talk)), ptr(D(sk)) if sink else None,
                         ptr(D(row_seq)), ptr(D(row_slot)), M, None if one_row else ptr(D(blk)), n_blk, br, H, G, d, t_max, window, chunk, ptr(out), H * d,
                         ptr(out16), H * d, ns, ptr(ws), ws.numel(), variant, stream()))
    ref = torch.zeros(M, H, d, dtype=F64)
    for i, p in enumerate(rows):
        lo = max(p - p % chunk if chunk else 0, p - window + 1 if window else 0, 0)
        kk, vv = k[lo:p + 1].double(), v[lo:p + 1].double()
        raw = torch.stack([(kk[:, h // (H // G)] @ q[i, h].double()) * scale for h in range(H)])
        s = talk.double() @ raw
        s = torch.cat([s, (sk.double() if sink else torch.full((H,), -torch.inf, dtype=F64))[:, None]], 1)
        w = torch.softmax(s, 1)[:, :-1]
        for h in range(H):
            ref[i, h] = w[h] @ vv[:, h // (H // G)]
    assert err(out16.float().reshape(M, H, d), ref) < 1e-2
    return out.reshape(M, H, d), ref


SHAPES = ((4, 2, 16), (6, 3, 20), (12, 1, 8), (8, 8, 40), (20, 4, 72), (40, 5, 8), (3, 3, 132), (2, 1, 256))


@pytest.mark.parametrize("variant", [0, 1])
def test_attention_needles_at_chunk_tile_and_split_edges(variant):
    """One key decides a row: its chunk's first slot, the last slot of the chunk before (which attracts the query and must not be seen), the
    row's own slot, slots around 16-key tile edges, in runs that cross a chunk border, with forced key splits; windows likewise."""
    for H, G, d in SHAPES:
        T = 300
        for chunk, window in ((0, 0), (51, 0), (1, 0), (100, 0), (0, 24), (64, 17), (1000, 0)):
            rows = list(range(196, 208))                             # 204 = 4 * 51 and 200 = 2 * 100 lie inside a run
            cases = [(0, 0), (4, 200), (3, 199), (8, 203), (8, 204), (11, 207), (5, 201 - 15), (11, 192)]
            for ri, slot in cases:
                for ns in ((1, 3) if variant == 0 else (1,)):
                    got, ref = talk_case(H, G, d, T, chunk, window, rows, (ri, slot), 0.3, variant, nsplit=ns)
                    assert err(got, ref) < 3e-5, (H, G, d, chunk, window, ri, slot, ns)


def test_attention_needles_in_decode_rows():
    for H, G, d in SHAPES:
        T, p = 700, 650
        for chunk, window in ((0, 0), (65, 0), (130, 0), (651, 0), (0, 100)):
            lo = max(p - p % chunk if chunk else 0, p - window + 1 if window else 0)
            for slot in {lo, max(lo - 1, 0), p, min(lo + 63, p), min(lo + 16, p), 0}:
                for ns in (0, 1, 5, 64):
                    got, ref = talk_case(H, G, d, T, chunk, window, [p], (0, slot), 0.3, 0, nsplit=ns, one_row=True)
                    assert err(got, ref) < 3e-5, (H, G, d, chunk, slot, ns)


def test_attention_runs_of_every_length_and_no_sink():
    """Runs shorter than the kernel's, rows from position 0 on, no sink, a strong mixing of the heads."""
    for H, G, d in SHAPES:
        for block in (1, 2, 3):
            got, ref = talk_case(H, G, d, 40, 7, 0, list(range(0, 11)), None, 0.3, 0, block=block, sink=False, spread=2.0)
            assert err(got, ref) < 3e-5, (H, G, d, block)


def state_inputs(g, T, H, G, d, e, low=0.3):
    q, k = torch.randn(T, G, d, generator=g), torch.randn(T, G, d, generator=g)
    q, k = q / q.norm(dim=-1, keepdim=True), k / k.norm(dim=-1, keepdim=True)
    return q, k, torch.randn(T, H, e, generator=g), torch.rand(T, H, d, generator=g) ** low, torch.rand(T, H, generator=g)


def run_state(L, check, stream, ptr, q, k, v, dec, beta, state, seq, past, cuts, mode="rows", o_scale=1.0, block=3):
    """Rows of one sequence through the recurrence in calls of the given sizes; mode rows | decode | scan; beta None: plain writes."""
    T, G, d = q.shape
    H, e = v.shape[1], v.shape[2]
    out = torch.zeros(T, H * e, device="cuda")
    at = 0
    for n in cuts:
        sl = slice(at, at + n)
        qkv = torch.cat([q[sl].reshape(n, -1), k[sl].reshape(n, -1), v[sl].reshape(n, -1)], 1).contiguous()
        r = _rows([(seq, n, past + at)], block, L.mn_channel_chunk_rows())
        o = C.c_void_p(out.data_ptr() + 4 * at * H * e)
        if mode == "scan":
            n_ch = r["chunk_tab"].shape[0]
            ws = torch.full((L.mn_channel_scan_workspace_bytes(n_ch, H, d, e) // 4,), 9.0, device="cuda")
            _KEEP.append(ws)
            check(L.mn_channel_state_rows_scan(ptr(D(qkv)), qkv.shape[1], ptr(D(dec[sl].reshape(n, -1))), H * d, n, H, G, d, e, o_scale, ptr(state),
                                               ptr(r["row_seq"]), ptr(r["row_slot"]), ptr(r["row_back"]), ptr(r["chunk_tab"]), n_ch, o, H * e,
                                               ptr(ws), 4 * ws.numel(), stream()))
        else:
            table = mode == "rows" and n > 5
            check(L.mn_channel_state_rows(ptr(D(qkv)), qkv.shape[1], ptr(D(dec[sl].reshape(n, -1))), H * d, ptr(D(beta[sl])) if beta is not None else None,
                                          H, n, H, G, d, e, o_scale, ptr(state), ptr(r["row_seq"]), ptr(r["row_slot"]), ptr(r["row_back"]),
                                          ptr(r["blk_tab"]) if table else None, r["blk_tab"].shape[0] if table else 0, 1 if mode == "decode" else 0, o,
                                          H * e, stream()))
        _KEEP.append(r)
        at += n
    return out.reshape(T, H, e)


def state_ref(q, k, v, dec, beta, rep):
    q, k = q.double().repeat_interleave(rep, 1), k.double().repeat_interleave(rep, 1)
    if beta is None:
        return O.gated_linear_attention(q, k, v.double(), dec.double())
    return O.channel_delta_rule(q, k, v.double(), beta.double(), dec.double())


def test_recurrences_rows_decode_rows_and_states():
    """Row walk and decode rows against the recurrence: a sequence that starts on a stale state (slot 0 reads nothing), continues from
    the stored state across calls cut anywhere, and a second sequence whose state stays untouched; states of 10 .. 520 rows."""
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(5)
    for H, G, d, e in ((4, 2, 16, 16), (3, 3, 10, 6), (2, 1, 136, 40), (1, 1, 256, 33), (2, 2, 260, 8), (2, 1, 520, 5), (4, 1, 64, 300), (2, 2, 100, 17)):
        T = 45
        q, k, v, dec, beta = state_inputs(g, T, H, G, d, e)
        for b in (beta, None):
            ref, S = state_ref(q, k, v, dec, b, H // G)
            for cuts, mode in (([45], "rows"), ([7, 2, 1, 30, 5], "rows"), ([1] * 45, "decode"), ([20] + [1] * 25, "both")):
                state = torch.full((2, H, d, e), 3.0, device="cuda")
                if mode == "both":
                    a1 = run_state(L, check, stream, ptr, q[:20], k[:20], v[:20], dec[:20], None if b is None else b[:20], state, 1, 0, [20], o_scale=0.5)
                    a2 = run_state(L, check, stream, ptr, q[20:], k[20:], v[20:], dec[20:], None if b is None else b[20:], state, 1, 20, [1] * 25,
                                   "decode", o_scale=0.5)
                    got = torch.cat([a1, a2])
                else:
                    got = run_state(L, check, stream, ptr, q, k, v, dec, b, state, 1, 0, cuts, mode, o_scale=0.5)
                assert err(got, ref * 0.5) < 2e-5, (H, d, e, b is None, mode, cuts[:3])
                assert err(state[1], S) < 2e-5 and bool((state[0] == 3.0).all())


def test_chunked_scan_of_the_plain_recurrence():
    """Prompts of several chunks with ragged ends, two sequences in a call, continued from a stored state, with decays so small that a
    chunk's product underflows beside decays of exactly 1."""
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(6)
    c = L.mn_channel_chunk_rows()
    for H, G, d, e in ((2, 2, 16, 16), (3, 1, 10, 7), (2, 2, 128, 40), (1, 1, 200, 9)):
        T = 2 * c + 37
        q, k, v, dec, _ = state_inputs(g, T, H, G, d, e, low=0.05)
        dec[:, :, 0], dec[:, :, 1], dec[::3, :, 2] = 1.0, 1e-3, 1e-30
        ref, S = state_ref(q, k, v, dec, None, H // G)
        for cuts in ([T], [c, T - c], [5, c + 1, T - c - 6]):
            state = torch.full((2, H, d, e), 3.0, device="cuda")
            got = run_state(L, check, stream, ptr, q, k, v, dec, None, state, 1, 0, cuts, "scan", o_scale=2.0)
            assert err(got, ref * 2) < 2e-5 and err(state[1], S) < 2e-5 and bool((state[0] == 3.0).all()), (H, d, cuts)
        # two sequences in one call: one fresh, one continued
        n0, n1 = c + 9, 40
        state = torch.full((2, H, d, e), 3.0, device="cuda")
        run_state(L, check, stream, ptr, q[:60], k[:60], v[:60], dec[:60], None, state, 0, 0, [60])
        sel = torch.cat([torch.arange(n0), torch.arange(60, 60 + n1)])
        qkv = torch.cat([q[sel].reshape(len(sel), -1), k[sel].reshape(len(sel), -1), v[sel].reshape(len(sel), -1)], 1).contiguous()
        r = _rows([(1, n0, 0), (0, n1, 60)], 4, c)
        n_ch = r["chunk_tab"].shape[0]
        ws = torch.zeros(L.mn_channel_scan_workspace_bytes(n_ch, H, d, e) // 4, device="cuda")
        out = torch.zeros(len(sel), H * e, device="cuda")
        check(L.mn_channel_state_rows_scan(ptr(D(qkv)), qkv.shape[1], ptr(D(dec[sel].reshape(len(sel), -1))), H * d, len(sel), H, G, d, e, 1.0,
                                           ptr(state), ptr(r["row_seq"]), ptr(r["row_slot"]), ptr(r["row_back"]), ptr(r["chunk_tab"]), n_ch, ptr(out),
                                           H * e, ptr(ws), 4 * ws.numel(), stream()))
        ref1, S1 = state_ref(q[:n0], k[:n0], v[:n0], dec[:n0], None, H // G)
        ref0, S0 = state_ref(q[:60 + n1], k[:60 + n1], v[:60 + n1], dec[:60 + n1], None, H // G)
        out = out.reshape(-1, H, e)
        assert err(out[:n0], ref1) < 2e-5 and err(out[n0:], ref0[60:]) < 2e-5 and err(state[1], S1) < 2e-5 and err(state[0], S0) < 2e-5


def test_a_write_is_kept_for_hundreds_of_tokens():
    """Orthonormal keys: what token 0 wrote under its key is read back 400 tokens later, faded by exactly the product of THAT channel's
    decays while the other channels decay fast — in one piece, in portions, decoded, and in the scan."""
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(7)
    H, G, d, e, T = 2, 1, 64, 16, 401
    k = torch.zeros(T, G, d)
    k[0, 0, 0] = 1.0
    for t in range(1, T):
        k[t, 0, 1 + (t % (d - 1))] = 1.0
    q = torch.zeros(T, G, d)
    q[:, 0, 0] = 1.0
    v = torch.randn(T, H, e, generator=g)
    for keep in (1.0, 0.995):
        dec = torch.full((T, H, d), 0.3)
        dec[:, :, 0] = keep
        want = v[0].double() * float(torch.tensor(keep)) ** 400
        for b in (torch.ones(T, H), None):
            for cuts, mode in (([T], "rows"), ([100, 2, 299], "rows"), ([1] * T, "decode"), ([T], "scan")):
                if mode == "scan" and b is not None:
                    continue
                state = torch.full((1, H, d, e), -2.0, device="cuda")
                got = run_state(L, check, stream, ptr, q, k, v, dec, b, state, 0, 0, cuts, mode)
                assert err(got[400], want) < 3e-5, (keep, b is None, mode)


def test_decode_rows_preparation_in_one_launch():
    """The launch that prepares decode rows against the operators one by one: filters and their states moved on, unit norms, strengths,
    both low-rank jobs, the activation and the table rows."""
    from ming_univision_amd._lib import LowRankJob, RowsPrep
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(8)
    for M, H, G, d, e, taps, n_act, top in ((3, 4, 2, 16, 12, 3, 44, 2), (20, 3, 3, 10, 6, 5, 0, 0), (64, 2, 1, 40, 300, 1, 2100, 3), (1, 1, 1, 8, 8, 2, 7, 0)):
        n = 2 * G * d + H * e
        ra, rg = 8, 5
        ld = n + ra + rg + H + n_act + 1
        x = torch.randn(M, ld, generator=g) * 2
        wc, w1, b1, w2 = (_bf(torch.randn(*s, generator=g) * 0.6) for s in ((n, taps), (H * d, ra), (H * d,), (H * e, rg)))
        a_log, st0 = torch.randn(H, generator=g), torch.randn(M + 1, max(taps - 1, 1), n, generator=g)
        seq, slot = torch.randperm(M + 1, generator=g)[:M].to(torch.int32), torch.randint(0, 6, (M,), generator=g).to(torch.int32)
        table, tok = torch.randint(0, 5, (9, max(top, 1)), generator=g).to(torch.int32), torch.randint(0, 9, (M,), generator=g).to(torch.int32)
        xd, sd_, ld_ = D(x), D(seq), D(slot)
        res = []
        for fused in (True, False):
            st = st0.clone().cuda()
            qkv, beta, dec, gat = (torch.zeros(M, c, device="cuda") for c in (n, H, H * d, H * e))
            act, idx = torch.zeros(M, max(n_act, 1), device="cuda"), torch.zeros(M, max(top, 1), dtype=torch.int32, device="cuda")
            jobs = (LowRankJob * 2)(LowRankJob(xd.data_ptr() + 4 * n, ld, D(w1).data_ptr(), D(b1).data_ptr(), D(a_log).data_ptr(), dec.data_ptr(), H * d, ra,
                                               H * d, 1, d, 1.0),
                                    LowRankJob(xd.data_ptr() + 4 * (n + ra), ld, D(w2).data_ptr(), None, None, gat.data_ptr(), H * e, rg, H * e, 3, 1, 1.0))
            act_x = C.c_void_p(xd.data_ptr() + 4 * (n + ra + rg + H))
            if fused:
                r = RowsPrep(proj=xd.data_ptr(), ld=ld, delta=1, H=H, G=G, dim=d, vdim=e, taps=taps, off_b=n + ra + rg, w_conv=D(wc).data_ptr(),
                             conv_state=st.data_ptr(), unit_eps=1e-6, q_scale=d ** -0.5, qkv=qkv.data_ptr(), ldqkv=n, beta=beta.data_ptr(), ldbeta=H,
                             n_jobs=2, job=jobs, act_x=act_x.value, ld_act_x=ld, act_pos=0.8, act_neg=1.1, act_y=act.data_ptr(), ld_act_y=max(n_act, 1),
                             act_n=n_act, table=D(table).data_ptr(), tok=D(tok).data_ptr(), vocab=9, top=top, idx=idx.data_ptr())
                check(L.mn_rows_prep_launch(C.byref(r), ptr(sd_), ptr(ld_), M, stream()))
            else:
                back = torch.zeros(M, dtype=torch.int32, device="cuda")
                check(L.mn_delta_prep_rows(ptr(xd), ld, M, H, G, d, e, n + ra + rg, 0, ptr(D(wc)), taps, ptr(st), 1, None, None, 1e-6, d ** -0.5,
                                           ptr(sd_), ptr(ld_), ptr(back), ptr(qkv), n, ptr(beta), H, stream()))
                check(L.mn_low_rank_gate_rows(jobs, 2, M, stream()))
                if n_act:
                    check(L.mn_xielu_rows(act_x, ld, 0.8, 1.1, ptr(act), n_act, None, 0, M, n_act, stream()))
                if top:
                    check(L.mn_token_table_rows(ptr(D(table)), 9, top, ptr(D(tok)), M, ptr(idx), None, stream()))
            torch.cuda.synchronize()
            res.append((qkv, beta, dec, gat, act, idx, st))
        for a, b in zip(*res):
            assert bool((a == b).all()), (M, H, d)
        # the unfused preparation itself: write strengths alone, filters from the stored state
        qkv, beta = res[0][0].double().cpu(), res[0][1].double().cpu()
        assert err(beta, torch.sigmoid(x[:, n + ra + rg:n + ra + rg + H].double())) < 1e-6
        for m in range(M):
            hist = [x[m, :n].double()] + [st0[seq[m], i].double() if slot[m] - i - 1 >= 0 else torch.zeros(n, dtype=F64) for i in range(taps - 1)]
            y = O.silu(sum(wc[:, taps - 1 - i].double() * hist[i] for i in range(taps)))
            qq, kk = y[:G * d].reshape(G, d), y[G * d:2 * G * d].reshape(G, d)
            qq, kk = (t / torch.sqrt((t * t).sum(-1, keepdim=True) + 1e-6) for t in (qq, kk))
            assert err(qkv[m], torch.cat([qq.reshape(-1) * d ** -0.5, kk.reshape(-1), y[2 * G * d:]])) < 1e-5


def test_head_norm_gates_and_gated_expert_products():
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(9)
    for M, H, e in ((5, 4, 16), (3, 3, 6), (2, 1, 300), (70, 6, 64)):
        x, gate, w = torch.randn(M, H * e + 2, generator=g) * 3, torch.randn(M, H * e + 1, generator=g), _bf(1 + 0.2 * torch.randn(e, generator=g))
        for act, f in ((0, lambda z: z), (1, O.silu), (2, torch.sigmoid)):
            y, y16 = torch.zeros(M, H * e, device="cuda"), torch.zeros(M, H * e, dtype=torch.bfloat16, device="cuda")
            check(L.mn_head_rms_gate_rows(ptr(D(x)), H * e + 2, ptr(D(w)), 1e-4, ptr(D(gate)), H * e + 1, act, ptr(y), H * e, ptr(y16), H * e, M, H, e,
                                          stream()))
            ref = (O.unit_rms(x[:, :H * e].double().reshape(M, H, e), 1e-4) * w.double()).reshape(M, -1) * f(gate[:, :H * e].double())
            assert err(y, ref) < 1e-6 and err(y16.float(), ref) < 1e-2
    for M, top, E, N, K in ((3, 2, 5, 24, 64), (4, 3, 4, 14, 44), (1, 1, 1, 8, 2048), (8, 2, 8, 100, 520)):
        x, w = torch.randn(M, K, generator=g), _bf(torch.randn(E, 2 * N, K, generator=g) * K ** -0.5)
        idx = torch.randint(0, E, (M * top,), generator=g).to(torch.int32)
        out = torch.full((M * top, N), 7.0, device="cuda")
        check(L.mn_gemv_glu_indexed(ptr(D(x)), K, top, ptr(D(w)), K, 2 * N * K, ptr(D(idx)), E, ptr(out), N, M * top, N, K, stream()))
        y = torch.stack([w[idx[z].item()].double() @ x[z // top].double() for z in range(M * top)])
        assert err(out, O.silu(y[:, :N]) * y[:, N:]) < 1e-5
        check(L.mn_gemv_glu_indexed(ptr(D(x)), K, top, ptr(D(w)), K, 2 * N * K, ptr(D(torch.full_like(idx, E))), E, ptr(out.fill_(7.0)), N, M * top, N, K,
                                    stream()))
        assert bool((out == 7.0).all())                              # an index that names no expert leaves its row


# ---- whole models ------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", MODELS)
def test_prompt_layers_and_logits(name):
    cfg, sd, dec = make(name)
    t = toks(cfg, 81)
    ref, streams = O.forward(cfg, sd, t)
    hid, tr = run_spans(dec, t, [(0, len(t), 0)], trace=True)
    assert tr.shape[0] == len(cfg["layers"])
    for r in range(tr.shape[0]):
        assert err(tr[r], streams[r]) < 1e-4, r
    assert err(dec.logits(hid), ref) < 1e-4


@pytest.mark.parametrize("name", ["mixed", "odd", "ones"])
def test_first_tokens(name):
    """The first positions: recurrences and filters from nothing on a reused sequence, a softmax over one key and the sink."""
    cfg, sd, dec = make(name)
    run_portions(dec, 0, toks(cfg, 9, 8), [9])            # leaves keys and states behind
    t = toks(cfg, 6, 5)
    ref = ref_logits(cfg, sd, t)
    assert err(run_portions(dec, 0, t, [1] * 6), ref) < 1e-4
    assert err(run_portions(dec, 0, t, [2, 2, 2]), ref) < 1e-4
    assert err(run_portions(dec, 0, t[:1], [1]), ref[:1]) < 1e-4


@pytest.mark.parametrize("name", MODELS)
def test_portions_and_decoding(name):
    cfg, sd, dec = make(name)
    t = toks(cfg, 150, 2)
    ref = ref_logits(cfg, sd, t)
    assert err(run_portions(dec, 0, t, [110] + [1] * 40), ref) < 1e-4                       # prefill against token-by-token decoding
    assert err(run_portions(dec, 0, t, [7, 2, 13, 2, 2, 1, 19, 3, 2, 24, 70, 5]), ref) < 1e-4    # portions cut inside chunks and key tiles
    assert err(run_portions(dec, 0, t[:75], [1] * 75), ref[:75]) < 1e-4


def test_long_prompts_take_the_scan_and_portions_agree():
    """A prompt of several scan chunks in one piece (the scan), in portions below the scan's size, and cut in the middle of scan chunks."""
    cfg, sd, dec = make("mixed", t_max=400)
    t = toks(cfg, 333, 4)
    ref = ref_logits(cfg, sd, t)
    for cuts in ([333], [100, 100, 100, 33], [290, 1, 2, 40]):
        assert err(run_portions(dec, 0, t, cuts), ref) < 1e-4, cuts


def test_single_far_keys_decide_in_prompts_and_decoding():
    """Peaky attention, so that single keys — at a chunk's start, or just inside it — carry the result, in one piece, in portions and decoded."""
    for name in ("mixed", "tail"):
        cfg, sd, dec = make(name, peaky=8.0, seed=7)
        t = toks(cfg, 140, 9)
        ref = ref_logits(cfg, sd, t)
        assert err(run_portions(dec, 0, t, [140]), ref) < 3e-4
        assert err(run_portions(dec, 0, t, [80] + [1] * 60), ref) < 3e-4
        assert err(run_portions(dec, 0, t, [9, 3, 4, 5, 11, 2, 30, 66, 10]), ref) < 3e-4


def test_unequal_requests_share_a_pass():
    """Three requests of different lengths in one pass, then a pass that mixes a prompt portion of one with single decode rows of
    the others: every request's logits equal the oracle on that request alone."""
    for arith, tol in (("f32", 1e-4), ("bf16", 3e-2)):
        cfg, sd, dec = make("mixed", n_seq=4, arith=arith)
        reqs = {3: toks(cfg, 120, 1), 0: toks(cfg, 9, 2), 2: toks(cfg, 43, 3)}
        refs = {s: ref_logits(cfg, sd, t) for s, t in reqs.items()}
        first = {3: 70, 0: 8, 2: 42}
        lg = dec.logits(run_spans(dec, [x for s, t in reqs.items() for x in t[:first[s]]], [(s, first[s], 0) for s in reqs]))
        r0 = 0
        for s in reqs:
            assert err(lg[r0:r0 + first[s]], refs[s][:first[s]]) < tol
            r0 += first[s]
        lg = dec.logits(run_spans(dec, [reqs[0][8]] + reqs[3][70:120] + [reqs[2][42]], [(0, 1, 8), (3, 50, 70), (2, 1, 42)]))
        assert err(lg[0:1], refs[0][8:9]) < tol and err(lg[1:51], refs[3][70:120]) < tol and err(lg[51:52], refs[2][42:43]) < tol


def test_inputs_longer_than_a_pass(monkeypatch):
    """More rows than one pass through the stack takes: the passes cut a sequence inside a chunk and a key tile, and a later sequence
    starts inside a pass; the trace is stitched across passes."""
    from ming_univision_amd import seq_lm
    monkeypatch.setattr(seq_lm, "MAX_ROWS", 70)
    cfg, sd, dec = make("mixed", n_seq=2)
    a, b = toks(cfg, 160, 1), toks(cfg, 31, 2)
    (ra, sa), rb = O.forward(cfg, sd, a), ref_logits(cfg, sd, b)
    hid, tr = run_spans(dec, a + b, [(1, 160, 0), (0, 31, 0)], trace=True)
    lg = dec.logits(hid)
    assert err(lg[:160], ra) < 1e-4 and err(lg[160:], rb) < 1e-4 and err(tr[-1][:160], sa[-1]) < 1e-4


def test_released_sequences_are_reused():
    """A cache sequence that held a longer request is given back and reused: its old keys, filter and recurrent states stay in memory and
    must not leak into the next request (nothing is cleared)."""
    from ming_univision_amd.sequences import SequenceSlots
    cfg, sd, dec = make("mixed")
    slots = SequenceSlots(dec)
    a, b = slots.alloc(), slots.alloc()
    assert (a, b) == (0, 1) and dec.n_seq >= 2
    other = toks(cfg, 20, 2)
    run_portions(dec, a, toks(cfg, 70, 1), [70])
    run_portions(dec, b, other, [20])
    slots.release(a)
    assert slots.alloc() == a
    t = toks(cfg, 30, 4)
    assert err(run_portions(dec, a, t, [3, 1, 1, 25]), ref_logits(cfg, sd, t)) < 1e-4
    c = slots.alloc()                                     # growing the caches keeps live sequences
    assert c == 2 and dec.n_seq >= 3
    more = toks(cfg, 6, 6)
    assert err(dec.logits(run_spans(dec, more, [(a, 6, 30)])), ref_logits(cfg, sd, t + more)[30:]) < 1e-4
    assert err(dec.logits(run_spans(dec, other[:5], [(b, 5, 0)])), ref_logits(cfg, sd, other[:5])) < 1e-4       # b starts again on its old slots
    dec.release_sequences(2)
    assert err(dec.logits(run_spans(dec, more, [(a, 6, 36)])), ref_logits(cfg, sd, t + more + more)[36:]) < 1e-4  # a lives on after the shrink


def test_long_decoding():
    """300 decoded tokens: chunks fill and end, the recurrent states and the filters are carried by decode rows alone."""
    for name in ("odd", "mixed"):
        cfg, sd, dec = make(name)
        t = toks(cfg, 300, 11)
        assert err(run_portions(dec, 0, t, [5] + [1] * 295), ref_logits(cfg, sd, t)) < 1e-4


def test_bf16_arithmetic():
    """Serving arithmetic: portions above 64 rows take the bf16 MFMA products (the experts the grouped ones), portions of 9 .. 64 rows the
    weight-streaming MFMA route on hi/lo rows, rows fed a few at a time fp32 FMA."""
    for name in ("mixed", "odd", "wide", "tail"):         # "odd": no K is a multiple of 8
        cfg, sd, dec = make(name, arith="bf16")
        t = toks(cfg, 150)
        ref = ref_logits(cfg, sd, t)
        for cuts in ([150], [70, 40, 31, 9]):
            e = (run_portions(dec, 0, t, cuts).double().cpu() - ref).abs().amax(-1) / ref.abs().max()
            assert float(e.max()) < 6e-2 and float(e.median()) < 1.5e-2, (name, cuts, float(e.max()), float(e.median()))
        assert err(run_portions(dec, 0, t[:30], [1] * 30), ref[:30]) < 1e-4


def test_bf16_expert_routes():
    """Widths that are multiples of 64 put the gated experts on the 256-tile grouped GEMM with its epilogue, others of 8 on the grouped
    GEMM with the activation behind it, the rest on pair-by-pair products: all against the oracle, prompts and shared decode batches."""
    for W, ff in ((64, 64), (128, 64), (64, 40), (44, 30)):
        cfg = O.small_config([O.gla_layer(mlp=O.moe(6, 2, ff)), O.attention_layer(mlp=O.moe(5, 3, ff))], width=W, vocab=70)
        sd = O.random_weights(cfg, 3)
        dec = build(cfg, sd, "bf16", n_seq=16)
        t = toks(cfg, 90, 1)
        ref = ref_logits(cfg, sd, t)
        assert err(run_portions(dec, 0, t, [90]), ref) < 5e-2 and err(run_portions(dec, 0, t, [50, 20, 20]), ref) < 5e-2
        prompts = {s: toks(cfg, 3 + s, 20 + s) for s in range(16)}   # sixteen sequences decode one row each
        for s, p in prompts.items():
            run_portions(dec, s, p[:-1], [len(p) - 1])
        lg = dec.logits(run_spans(dec, [p[-1] for p in prompts.values()], [(s, 1, len(p) - 1) for s, p in prompts.items()]))
        for i, p in enumerate(prompts.values()):
            assert err(lg[i:i + 1], ref_logits(cfg, sd, p)[-1:]) < 5e-2, (W, ff, i)


def test_greedy_generation_entry_point():
    """SabezenForCausalLM.generate: unequal prompts in one lock-step batch; every new token is the oracle's arg-max given the tokens before
    it (or the oracle's two best are within 1e-4), alone or batched, with and without the captured decode step; sampled generation
    returns tokens and gives its cache sequences back."""
    from ming_univision_amd.sabezen import SabezenForCausalLM
    cfg, sd, dec = make("mixed")
    lm = SabezenForCausalLM(dec)
    prompts = [toks(cfg, 17, 1), toks(cfg, 3, 2), toks(cfg, 40, 3)]
    new = lm.generate(prompts, max_new_tokens=12)
    alone = [lm.generate([p], max_new_tokens=12, use_graph=False)[0] for p in prompts]
    for p, out, solo in zip(prompts, new, alone):
        assert len(out) == 12
        ref = ref_logits(cfg, sd, p + out)
        for i, tok in enumerate(out):
            row = ref[len(p) - 1 + i]
            assert int(row.argmax()) == tok or float(row.max() - row[tok]) < 1e-4
        assert solo == out
    assert not lm.slots.length and lm.slots.next == 3
    out = lm.generate(prompts, max_new_tokens=5, do_sample=True, top_k=8, generator=torch.Generator(device="cuda").manual_seed(0))
    assert all(len(o) == 5 and all(0 <= x < cfg["vocab"] for x in o) for o in out) and not lm.slots.length


def test_decode_graph_replays():
    """The captured decode step against the oracle: every replay is checked (not only the first), with eager work and host
    synchronisations between replays, across a re-capture; in fp32 and, with ten sequences, on the grouped expert route."""
    for arith, B, tol in (("f32", 3, 1e-4), ("bf16", 10, 3e-2)):
        cfg, sd, dec = make("mixed", n_seq=B, arith=arith)
        prompts = {s: toks(cfg, 5 + 7 * (s % 4), 1 + s) for s in range(B)}
        follow = {s: toks(cfg, 24, 30 + s) for s in prompts}
        refs = {s: ref_logits(cfg, sd, prompts[s] + follow[s]) for s in prompts}
        for s, p in prompts.items():
            run_portions(dec, s, p, [len(p)])
        row_seq = torch.tensor(list(prompts), dtype=torch.int32, device="cuda")
        slot = torch.tensor([len(p) for p in prompts.values()], dtype=torch.int32, device="cuda")
        ln = slot + 1
        g = dec.decode_graph(row_seq, slot, ln)
        g.span = 16                                               # re-capture every 16 tokens
        other = torch.tensor(toks(cfg, 7, 99), device="cuda")
        for i in range(24):
            ids = torch.tensor([follow[s][i] for s in prompts], device="cuda")
            hid = g.run(dec.embed(ids), max(len(p) for p in prompts.values()) + i + 1, tokens=ids)
            lg = dec.logits(hid.clone())
            torch.cuda.synchronize()
            for k, s in enumerate(prompts):
                assert err(lg[k:k + 1], refs[s][len(prompts[s]) + i][None]) < tol, (arith, i, s)
            dec.logits(dec.embed(other))                          # eager work between replays
        assert slot.tolist() == [len(p) + 24 for p in prompts.values()]


def test_a_table_that_names_no_expert_is_refused():
    cfg = config("mixed")
    sd = O.random_weights(cfg, 3)
    sd["l1.mlp.table"][5, 1] = 7
    with pytest.raises(ValueError, match="table"):
        build(cfg, sd)


def test_trace_runner(tmp_path):
    """bin/trace_run on a saved model: a request in portions interleaved with a second one, logits against the oracle; the first
    request's cache sequence is reused by a third."""
    from safetensors.torch import save_file
    cfg = config("mixed")
    sd = O.random_weights(cfg, 3)
    mdir, odir = tmp_path / "model", tmp_path / "out"
    mdir.mkdir()
    (mdir / "config.json").write_text(json.dumps(O.config_json(cfg)))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(mdir / "model.safetensors"))
    a, b, c = toks(cfg, 25, 1), toks(cfg, 6, 2), toks(cfg, 11, 3)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:10], "want": [0, 9]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:5], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[10:12], "want": [1]}, {"id": "b", "tokens": b[5:], "want": [0]}], "end": ["b"]},
        {"step": 3, "entries": [{"id": "a", "tokens": a[12:], "want": [12]}], "end": ["a"]},
        {"step": 4, "entries": [{"id": "c", "tokens": c, "want": [0, 10]}], "end": ["c"]},
    ]
    for dtype, tol in (("float32", 1e-4), ("bfloat16", 5e-2)):
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(mdir), "--dtype", dtype, "--out", str(odir), "--max-tokens", "64"],
                           input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(5)]
        ra, rb, rc = (ref_logits(cfg, sd, x) for x in (a, b, c))
        want = {0: ra[[0, 9]], 2: torch.stack([ra[11], rb[5]]), 3: ra[[24]], 4: rc[[0, 10]]}
        assert not (odir / "1.f32").exists()
        for n, ref in want.items():
            got = torch.from_numpy(np.fromfile(odir / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))
            assert err(got, ref) < tol, (dtype, n)
            os.unlink(odir / f"{n}.f32")
