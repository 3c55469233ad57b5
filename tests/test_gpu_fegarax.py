"""Fegarax on the HIP path against tests/fegarax_oracle.py (plain float64 restatement, one function per mechanism).

Small random models of several shapes (layers that mix values and layers that do not, with and without experts, sizes that are no
multiples of 4 or 8, one head, everything equal or 1, one stream to six, chunks of 1, of a few tokens and longer than any request, no
chunk, no rotation, scaled and plain frequencies, values narrower and wider than keys, many heads on one key head, as many key heads as
heads).  fp32 arithmetic is held to 1e-4 of the logits' scale, the bf16-MFMA arithmetic to a few 1e-2.  Covers: every operator alone
(streams updated in place and from one shared row, with dense and expert results, with and without norm; attention whose scores are scaled
up until one key decides — the chunk's first slot, the last slot of the chunk before it, the row's own slot, window edges, key-tile and
key-split edges — in runs of rows across chunk borders and in decode rows, on the matrix-core and the plain kernel; append with
rotation, kept and mixed values; sigmoid router; experts fed with weight times input on all their routes); whole prompts with the streams'
sum after every layer; token-by-token decoding; portions down to two tokens; several unequal requests in one pass against each alone;
inputs longer than a pass; cache sequences that are released and reused; the first positions of a sequence; long decoding; the bf16
arithmetic; greedy generation through the generation entry point; the captured decode step; the trace runner."""
import copy
import ctypes as C
import json
import os
import subprocess

import numpy as np
import pytest
import torch

from tests import fegarax_oracle as O

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F64 = torch.float64
GEMM_F32 = 2              # MN_GEMM_F32


def config(name):
    A, moe = O.attention_layer, O.moe
    if name == "mixed":     # layers with and without mixed values, experts and chunks; values narrower and wider than keys
        return O.small_config([A(v_mix=False, mlp=moe(7, 3, 16)), A(mlp=moe(4, 1, 24)), A(heads=8, kv_heads=4, dim=24, vdim=6, chunk=23, rot=(700.0, 24)),
                               A(heads=6, kv_heads=1, dim=12, vdim=24, chunk=None, rot=(1e4, 4), scaling=None, mlp=moe(5, 2, 40)),
                               A(heads=2, kv_heads=2, dim=20, vdim=40, v_mix=False, rot=None, mlp=moe(9, 1, 32))])
    if name == "odd":       # no size a multiple of 4 or 8 (products on the fp32 FMA kernels, attention on the plain kernel), other constants
        return O.small_config([A(heads=3, kv_heads=1, dim=10, vdim=18, scale=0.4, rot=(500.0, 6), scaling=(2.0, 40, 64.0, 0.01), chunk=13, mlp=moe(3, 2, 14)),
                               A(heads=6, kv_heads=3, dim=14, vdim=6, scale=0.5, rot=(30.0, 14), scaling=(9.0, 100, 3.0, 1.0), chunk=7, mlp=moe(5, 1, 22))],
                              width=42, vocab=61, streams=5, scale=0.7, eps=1e-3)
    if name == "ones":      # values a model may happen to make equal or 1
        return O.small_config([A(heads=1, kv_heads=1, dim=32, vdim=32, scale=1.0, rot=None, chunk=None, mlp=moe(1, 1, 32)),
                               A(heads=32, kv_heads=32, dim=4, vdim=1, scale=1.0, rot=(32.0, 4), scaling=(1.0, 32, 1.0, 1.0), chunk=1, mlp=moe(2, 2, 32)),
                               A(heads=1, kv_heads=1, dim=1, vdim=32, scale=1.0, rot=None, chunk=32)], width=32, vocab=32, streams=1, scale=1.0)
    if name == "wide":      # twelve heads on one key head, forty heads on five, six streams, a wide router
        return O.small_config([A(heads=12, kv_heads=1, dim=8, vdim=40, rot=(10000.0, 8), chunk=70, mlp=moe(70, 5, 8)),
                               A(heads=40, kv_heads=5, dim=8, vdim=8, rot=(100.0, 2), scaling=None, chunk=33, mlp=moe(9, 4, 8))],
                              width=32, vocab=40, streams=6, scale=3.0)
    if name == "tail":      # heads of 72, 132 and 260 values (the attention's larger instances and the plain kernel), chunks longer than any request
        return O.small_config([A(heads=4, kv_heads=4, dim=72, vdim=33, scale=0.1, rot=(1e6, 72), scaling=(16.0, 64, 4.0, 1.0), chunk=1000, mlp=moe(16, 2, 64)),
                               A(heads=3, kv_heads=3, dim=132, vdim=44, scale=0.1, rot=(1e4, 64), chunk=300, mlp=moe(3, 1, 64)),
                               A(heads=2, kv_heads=1, dim=20, vdim=132), A(heads=2, kv_heads=2, dim=260, vdim=66, scale=0.05, rot=(1e4, 260), chunk=90)],
                              width=64, vocab=50, streams=2)
    raise KeyError(name)


MODELS = ("mixed", "odd", "ones", "wide", "tail")


def build(cfg, sd, arith="f32", t_max=512, n_seq=1):
    from ming_univision_amd.configuration import FegaraxConfig
    from ming_univision_amd.fegarax import FegaraxDecoder
    return FegaraxDecoder(FegaraxConfig.from_dict(cfg), {k: v.cuda() for k, v in sd.items()}, t_max=t_max, n_seq=n_seq, arith=arith)


def make(name, arith="f32", seed=0, t_max=512, n_seq=1, peaky=1.0):
    cfg = config(name)
    if peaky != 1.0:
        cfg = copy.deepcopy(cfg)
        for ly in cfg["layers"]:
            ly["mixer"]["scale"] *= peaky
    sd = O.random_weights(cfg, seed)
    return cfg, sd, build(cfg, sd, arith, t_max, n_seq)


def toks(cfg, n, seed=1):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def clear(cfg, sd, n, seed=1):
    """Tokens without close calls between experts: the bf16 products' rounding moves the router's logits by a few 1e-2."""
    return O.clear_tokens(cfg, sd, n, seed, gap=0.08)


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


def _rows(spans, block_rows=1 << 30):
    from ming_univision_amd.sequences import rows_of_spans
    t = rows_of_spans(spans, block_rows)
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
def streams_call(a, M):
    check, stream, L, ptr = _api()
    check(L.mn_streams_update_norm(C.byref(a), M, stream()))


def test_streams_update_combine_and_norm():
    """Streams of 1 .. 7 copies and rows of 1 .. 9000 values: updated in place from their own rows, from one shared row (the first sublayer),
    with a dense result, expert results through a slot table or in order, weights or none, either norm form or none, both outputs."""
    from ming_univision_amd._lib import StreamsArgs
    g = torch.Generator().manual_seed(0)
    for M, n, S, top in ((5, 44, 3, 2), (3, 1, 2, 0), (70, 1000, 4, 3), (2, 2100, 1, 1), (3, 4096, 2, 2), (2, 8200, 3, 2), (3, 8192, 4, 0), (2, 5001, 3, 1),
                         (3, 64, 6, 2), (2, 300, 7, 0), (2, 9000, 5, 1)):
        for aligned in (True, False):
            ld = n + (4 if aligned else 3)
            X, x0, y = torch.randn(M, S, n, generator=g), torch.randn(M, ld, generator=g), torch.randn(M, ld, generator=g)
            ye, ew = torch.randn(max(1, M * top), ld, generator=g), torch.rand(max(1, M * top), generator=g)
            slot = torch.randperm(max(1, M * top), generator=g).to(torch.int32)
            mix, wi, wo = torch.randn(S, S, generator=g), torch.randn(S, generator=g), torch.randn(S, generator=g)
            w = _bf(0.2 * torch.randn(n, generator=g))
            for first in (False, True):
                for slots, weights, dense in ((True, False, True), (False, True, top == 0)):
                    old = torch.stack([x0[:, :n]] * S, 1) if first else X
                    r = torch.zeros(M, n, dtype=F64) + (y[:, :n].double() if dense else 0)
                    for j in range(top):
                        z = torch.arange(M) * top + j
                        r = r + (ew[z].double()[:, None] if weights else 1.0) * ye[slot[z].long() if slots else z][:, :n].double()
                    new = O.streams_write(old.double().transpose(0, 1), r, mix, wo)
                    u = O.streams_read(new, wi)
                    dst, h, h16 = X.clone().cuda(), torch.zeros(M, n, device="cuda"), torch.zeros(M, n, dtype=torch.bfloat16, device="cuda")
                    src = D(x0) if first else dst
                    a = StreamsArgs(src=src.data_ptr(), src_row=ld if first else S * n, src_stream=0 if first else n, dst=dst.data_ptr(), S=S, n=n,
                                    mix=D(mix).data_ptr(), out=D(wo).data_ptr(), in_=D(wi).data_ptr(), y=D(y).data_ptr() if dense else None, ldy=ld,
                                    ye=D(ye).data_ptr() if top else None, ldye=ld, slot_of=D(slot).data_ptr() if slots else None,
                                    ew=D(ew).data_ptr() if weights else None, top=top, one_plus=int(slots), w=D(w).data_ptr(), eps=1e-3,
                                    h=h.data_ptr(), ldh=n, h16=h16.data_ptr(), ldh16=n)
                    streams_call(a, M)
                    ref = O.rms(u, 1e-3) * (w.double() + (1.0 if slots else 0.0))
                    assert err(dst.transpose(0, 1), new) < 1e-6 and err(h, ref) < 5e-6 and err(h16.float(), ref) < 1e-2, (M, n, S, top, first)
                    # reading alone: the streams' sum without a norm, and a normed read that changes nothing
                    keep = dst.clone()
                    a = StreamsArgs(src=dst.data_ptr(), src_row=S * n, src_stream=n, S=S, n=n, h=h.data_ptr(), ldh=n)
                    streams_call(a, M)
                    assert float((h.double().cpu() - new.sum(0)).abs().max()) < 1e-6 * S * float(new.abs().max())
                    a = StreamsArgs(src=dst.data_ptr(), src_row=S * n, src_stream=n, S=S, n=n, in_=D(wi).data_ptr(), w=D(w).data_ptr(), one_plus=1,
                                    eps=1e-3, h=h.data_ptr(), ldh=n)
                    streams_call(a, M)
                    assert err(h, O.norm_zero(u, w, 1e-3)) < 5e-6 and bool((keep == dst).all())


def test_streams_update_takes_the_router_along():
    """The update also computes the router on the normed rows (fp32), picks and scores; few rows: expert results that lie in slabs, bf16 rows
    with their low parts; every number of streams the form has, routers of 1 .. 300 outputs, rows of 8 .. 8192 values."""
    from ming_univision_amd._lib import StreamsArgs
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(4)
    for M, n, S, E, picks, top in ((1, 8, 1, 1, 1, 0), (5, 64, 3, 7, 3, 2), (64, 200, 2, 16, 2, 1), (3, 2048, 4, 8, 2, 2), (2, 8192, 4, 20, 5, 0), (7, 4104, 3, 65, 9, 3),
                                   (20, 520, 1, 300, 4, 2), (2, 6000, 2, 33, 33, 1), (65, 64, 3, 16, 2, 2),
                                   (100, 2056, 4, 8, 8, 1), (70, 8192, 2, 1, 1, 0), (90, 1000, 1, 5, 2, 3)):
        few = M <= 64
        X, y, slabs = torch.randn(M, S, n, generator=g), torch.randn(M, n, generator=g), 1 + (M % 3 if few else 0)
        Z = max(1, M * top)
        ye, slot, ew = torch.randn(slabs, Z, n, generator=g), torch.randperm(Z, generator=g).to(torch.int32), torch.rand(Z, generator=g)
        mix, wi, wo = torch.randn(S, S, generator=g) * 0.5, torch.randn(S, generator=g), torch.randn(S, generator=g)
        w, rt = _bf(0.2 * torch.randn(n, generator=g)), _bf(torch.randn(E, n, generator=g) * 3 * n ** -0.5)
        assert L.mn_streams_router_ok(M, S, n, E, ptr(D(rt))) == 1
        r = y.double()
        for j in range(top):
            z = torch.arange(M) * top + j
            r = r + ew[z].double()[:, None] * ye.double().sum(0)[slot[z].long()]
        new = O.streams_write(X.double().transpose(0, 1), r, mix, wo)
        href = O.norm_zero(O.streams_read(new, wi), w, 1e-3)
        zref = href @ rt.double().T
        for both in (True, False):
            dst, h, hl = X.clone().cuda(), torch.zeros(M, n, device="cuda"), torch.zeros(2, M, n, dtype=torch.bfloat16, device="cuda")
            idx, pw = torch.full((M, picks), -1, dtype=torch.int32, device="cuda"), torch.zeros(M, picks, device="cuda")
            a = StreamsArgs(src=dst.data_ptr(), src_row=S * n, src_stream=n, dst=dst.data_ptr(), S=S, n=n, mix=D(mix).data_ptr(), out=D(wo).data_ptr(),
                            in_=D(wi).data_ptr(), y=D(y).data_ptr(), ldy=n, ye=D(ye).data_ptr(), ldye=n, slot_of=D(slot).data_ptr(), ew=D(ew).data_ptr(),
                            top=top, one_plus=1, w=D(w).data_ptr(), eps=1e-3, h=h.data_ptr() if both else None, ldh=n, h16=hl.data_ptr(), ldh16=n,
                            h16_lo=hl[1].data_ptr() if few else None, ye_slab=Z * n, ye_slabs=slabs, experts=E, router=D(rt).data_ptr(), idx=idx.data_ptr(), pw=pw.data_ptr(),
                            picks=picks)
            streams_call(a, M)
            assert err(dst.transpose(0, 1), new) < 2e-6 and err(hl.double().sum(0), href) < (2e-5 if few else 1e-2), (M, n, S)
            if both:
                assert err(h, href) < 5e-6
            got = torch.gather(zref, 1, idx.cpu().long())            # the picks: distinct, in falling order, the largest up to rounding
            assert all(len(set(row)) == picks for row in idx.tolist())
            assert float((got - torch.topk(zref, picks, dim=1).values).abs().max()) < 2e-5 * float(zref.abs().max())
            assert float((pw.double().cpu() - torch.sigmoid(got)).abs().max()) < 2e-5
    t = D(torch.zeros(4, 64, dtype=torch.bfloat16))
    assert L.mn_streams_router_ok(65, 3, 64, 17, ptr(t)) == 0 and L.mn_streams_router_ok(64, 3, 64, 513, ptr(t)) == 0 and L.mn_streams_router_ok(5, 5, 64, 4, ptr(t)) == 0
    assert L.mn_streams_router_ok(5, 3, 60, 4, ptr(t)) == 0 and L.mn_streams_router_ok(5, 3, 8200, 4, ptr(t)) == 0


def test_streams_refuse_what_they_do_not_take():
    from ming_univision_amd._lib import StreamsArgs
    t = torch.zeros(2, 33, 8, device="cuda")
    for bad in (dict(S=33), dict(S=0), dict(n=0), dict(h=None, ldh=0), dict(ldh=4), dict(y=t.data_ptr(), ldy=8)):
        a = dict(src=t.data_ptr(), src_row=33 * 8, src_stream=8, S=3, n=8, h=t.data_ptr(), ldh=8)
        a.update(bad)
        with pytest.raises(RuntimeError):
            streams_call(StreamsArgs(**a), 2)


def test_norms_rotation_mixed_values_and_append():
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(1)
    yarn = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}
    from ming_univision_amd.sakinex import rotary_table
    for H, G, d, e, rot in ((4, 2, 16, 16, {"base": 1e4, "dims": 16, "scaling": yarn}), (3, 1, 10, 18, {"base": 500.0, "dims": 6}), (1, 1, 130, 5, None),
                            (5, 5, 64, 72, {"base": 2e5, "dims": 40, "scaling": yarn}), (8, 2, 24, 12, {"base": 1e4, "dims": 20, "scaling": yarn})):
        for many in (False, True):
            spans = [(1, 7, 0), (0, 1, 2999), (2, 5 + 80 * many, 94)]
            M, t_max, n_seq, eps, scale, lam = 13 + 80 * many, 3004, 3, 1e-5, 0.37, 0.3
            r = _rows(spans)
            nq, nk, nv = H * d, G * d, G * e
            for ld, normed in ((nq + nk + nv + 3, True), (-(-(nq + nk + nv) // 4) * 4, False)):
                qkv, vf = torch.randn(M, ld, generator=g) * 3, torch.randn(M, nv + 1, generator=g)
                qw, kw = _bf(1 + 0.2 * torch.randn(nq, generator=g)), _bf(1 + 0.2 * torch.randn(nk, generator=g))
                q, keep = torch.zeros(M, nq, device="cuda"), torch.zeros(M, nv + 1, device="cuda")
                ka, va = torch.full((n_seq, t_max, nk), 7.0, device="cuda"), torch.full((n_seq, t_max, nv), 7.0, device="cuda")
                fr, mag = rotary_table(rot, "cuda") if rot else (None, 1.0)
                check(L.mn_proj_norm_rope_mix_append(ptr(D(qkv)), ld, M, H, G, d, e, ptr(D(qw)) if normed else None, ptr(D(kw)) if normed else None, eps,
                                                     rot["dims"] if rot else 0, 0, ptr(fr), mag, scale, ptr(keep), nv + 1, ptr(D(vf)), nv + 1, lam,
                                                     ptr(r["row_seq"]), ptr(r["row_slot"]), ptr(q), nq, ptr(ka), nk, ptr(va), nv, t_max, stream()))
                x, v = qkv.double(), qkv[:, nq + nk:nq + nk + nv].double()
                qr = (O.rms(x[:, :nq], eps) * qw.double() if normed else x[:, :nq]).reshape(M, H, d)
                kr = (O.rms(x[:, nq:nq + nk], eps) * kw.double() if normed else x[:, nq:nq + nk]).reshape(M, G, d)
                pos, seqs = r["row_slot"].cpu().tolist(), r["row_seq"].cpu().tolist()
                if rot:
                    f, m = O.rotary_frequencies(rot)
                    qr = torch.cat([O.rotate_halves(qr[i:i + 1], f, m, pos[i]) for i in range(M)])
                    kr = torch.cat([O.rotate_halves(kr[i:i + 1], f, m, pos[i]) for i in range(M)])
                q, kc, vc, kept = q.cpu(), ka.cpu(), va.cpu(), keep.cpu()
                vm = (1 - lam) * v + lam * vf[:, :nv].double()
                for i in range(M):
                    tol = 2e-5 if pos[i] < 200 else 3e-4             # an fp32 angle near 3000 radians is rounded to 1.2e-4
                    assert err(q[i], qr[i].reshape(-1) * scale) < tol, (H, d, i)
                    assert err(kc[seqs[i], pos[i]], kr[i].reshape(-1)) < tol and err(vc[seqs[i], pos[i]], vm[i]) < 1e-6
                assert err(kept[:, :nv], v) < 1e-7 and bool((kept[:, nv] == 0).all())
                ka[r["row_seq"].long(), r["row_slot"].long()] = 7.0
                assert bool((ka == 7.0).all())                       # nothing else was written


def attention_case(H, G, d, e, T, chunk, window, rows, needle, scale, variant, nsplit=0, one_row=False, seed=0, sink=True, gate=True):
    """A sequence of T cached tokens; `rows` = consecutive positions of the query rows.  needle = (row index, key slot): that key is made to
    dominate that row's scores.  Returns (got, reference) [rows, H, e]."""
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(seed)
    k, v, q = torch.randn(T, G, d, generator=g), torch.randn(T, G, e, generator=g), torch.randn(len(rows), H, d, generator=g)
    if needle is not None:
        ri, slot = needle
        q[ri] = 6.0 * k[slot].repeat_interleave(H // G, 0) / scale / d ** 0.5
    gt = torch.randn(len(rows), H * e + 3, generator=g) * 2
    sk = torch.zeros(H) if sink is True else (torch.randn(H, generator=g) if sink else None)
    t_max, M = T + 5, len(rows)
    ka, va = torch.full((2, t_max, G * d), 1e4), torch.full((2, t_max, G * e), 1e4)      # slots past the sequence hold junk that must not be read
    ka[1, :T], va[1, :T] = k.reshape(T, -1), v.reshape(T, -1)
    row_seq, row_slot = torch.ones(M, dtype=torch.int32), torch.tensor(rows, dtype=torch.int32)
    br = 1 if one_row else L.mn_window_attn_block_rows()
    blk = torch.tensor([[i, min(br, M - i)] for i in range(0, M, br)], dtype=torch.int32)
    n_blk = blk.shape[0]
    ns = nsplit or L.mn_window_attn_splits(n_blk, H, G, int(one_row), T)
    ws = torch.zeros(max(L.mn_window_attn_workspace_bytes(n_blk, H, G, e, int(one_row), ns), 16), dtype=torch.uint8, device="cuda")
    out, out16 = torch.zeros(M, H * e, device="cuda"), torch.zeros(M, H * e, dtype=torch.bfloat16, device="cuda")
    check(L.mn_window_pool_attn_blocks_gate(ptr(D(q.reshape(M, -1) * scale)), H * d, ptr(D(ka)), 0, ptr(D(va)), 0, None, None,
                                            ptr(D(sk)) if sk is not None else None, 0.0, chunk, ptr(D(gt)) if gate else None, H * e + 3, ptr(D(row_seq)),
                                            ptr(D(row_slot)), None if one_row else ptr(D(blk)), n_blk, int(one_row), H, G, d, e, t_max, 1, window, 0,
                                            1.0, ptr(out), H * e, ptr(out16), H * e, ns, ptr(ws), ws.numel(), variant, stream()))
    ref = torch.zeros(M, H, e, dtype=F64)
    for i, p in enumerate(rows):
        lo = max(p - p % chunk if chunk else 0, p - window + 1 if window else 0, 0)
        kk, vv = k[lo:p + 1].double(), v[lo:p + 1].double()
        for h in range(H):
            s = (kk[:, h // (H // G)] @ q[i, h].double()) * scale
            if sk is not None:
                s = torch.cat([s, sk[h:h + 1].double()])
            ref[i, h] = torch.softmax(s, 0)[:p + 1 - lo] @ vv[:, h // (H // G)]
    if gate:
        ref = ref * torch.sigmoid(gt[:, :H * e].double()).reshape(M, H, e)
    assert err(out16.float().reshape(M, H, e), ref) < 1e-2
    return out.reshape(M, H, e), ref


SHAPES = ((4, 2, 16, 16), (6, 3, 20, 12), (12, 1, 8, 40), (3, 1, 10, 18), (2, 2, 72, 136), (40, 5, 8, 8), (4, 2, 132, 36))


@pytest.mark.parametrize("variant", [0, 1])
def test_attention_needles_at_chunk_tile_and_split_edges(variant):
    """One key decides a row: its chunk's first slot, the last slot of the chunk before (which attracts the query and must not be seen), the
    row's own slot, slots around 16-key tile edges, in runs that cross a chunk border, with forced key splits; windows and both likewise."""
    for H, G, d, e in SHAPES:
        T = 300
        for chunk, window in ((0, 0), (51, 0), (1, 0), (100, 0), (0, 24), (64, 17), (1000, 0)):
            rows = list(range(196, 208))                             # 204 = 4 * 51 and 200 = 2 * 100 lie inside a run
            for ri, slot in ((0, 0), (4, 200), (3, 199), (8, 203), (8, 204), (11, 207), (5, 201 - 15), (11, 192)):
                for ns in (1, 3):
                    got, ref = attention_case(H, G, d, e, T, chunk, window, rows, (ri, slot), 0.3, variant, nsplit=ns)
                    assert err(got, ref) < 3e-5, (H, G, d, chunk, window, ri, slot, ns)


def test_attention_needles_in_decode_rows():
    for H, G, d, e in SHAPES + ((2, 1, 260, 300),):
        T, p = 700, 650
        for chunk, window in ((0, 0), (65, 0), (130, 0), (651, 0), (0, 100), (130, 40)):
            lo = max(p - p % chunk if chunk else 0, p - window + 1 if window else 0)
            for slot in {lo, max(lo - 1, 0), p, min(lo + 63, p), min(lo + 16, p), 0}:
                for ns in (0, 1, 5, 64):
                    got, ref = attention_case(H, G, d, e, T, chunk, window, [p], (0, slot), 0.3, 1, nsplit=ns, one_row=True)
                    assert err(got, ref) < 3e-5, (H, G, d, chunk, slot, ns)


def test_attention_first_rows_sinks_and_gates():
    """Rows from position 0 on, with the denominator's extra one, other sinks and none, gated and not; scores so low that the extra one takes
    all the weight, and so high that it takes none."""
    for H, G, d, e in SHAPES:
        for sink in (True, "random", False):
            for gate in (True, False):
                for variant in (0, 1):
                    got, ref = attention_case(H, G, d, e, 40, 7, 0, list(range(0, 11)), None, 0.3, variant, sink=sink, gate=gate)
                    assert err(got, ref) < 3e-5, (H, G, d, sink, gate)
        for scale in (8.0, 40.0):
            got, ref = attention_case(H, G, d, e, 40, 7, 0, list(range(0, 11)), None, scale, 0)
            assert err(got, ref) < 2e-4, (H, d, scale)


def test_sigmoid_router():
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(2)
    for M, E, top in ((5, 7, 3), (1, 1, 1), (70, 64, 6), (9, 65, 65), (3, 300, 8), (2, 4096, 4)):
        z = torch.randn(M, E + 3, generator=g) * 3
        idx, w = torch.zeros(M, top, dtype=torch.int32, device="cuda"), torch.zeros(M, top, device="cuda")
        check(L.mn_router_sigmoid_topk_rows(ptr(D(z)), E + 3, M, E, top, ptr(idx), ptr(w), stream()))
        order = torch.argsort(z[:, :E], dim=1, descending=True, stable=True)[:, :top]
        assert bool((idx.cpu() == order).all())
        assert float((w.double().cpu() - torch.sigmoid(torch.gather(z[:, :E].double(), 1, order))).abs().max()) < 1e-6


def glu(x, w, s):
    y = (s * x.double()) @ w.double().T
    n = w.shape[0] // 2
    return O.silu(y[:n]) * y[n:]


def test_experts_are_fed_with_weight_times_input():
    """The routes: pair by pair, the grouped product followed by the activation, the 256-tile product with its scaled epilogue, the grouped
    weight-streaming product (few rows, high and low bf16 parts: fp32-class results)."""
    check, stream, L, ptr = _api()
    g = torch.Generator().manual_seed(3)
    for M, top, E, N, K in ((3, 2, 5, 24, 64), (4, 3, 4, 14, 44), (1, 1, 1, 8, 2048), (8, 2, 8, 100, 520), (90, 2, 6, 64, 128), (300, 3, 4, 192, 64), (40, 1, 3, 40, 72)):
        x, w = torch.randn(M, K, generator=g), _bf(torch.randn(E, 2 * N, K, generator=g) * K ** -0.5)
        idx, s = torch.randint(0, E, (M * top,), generator=g).to(torch.int32), 0.05 + torch.rand(M * top, generator=g)
        Z = M * top
        ref = torch.stack([glu(x[z // top], w[idx[z].item()], float(s[z])) for z in range(Z)])
        out = torch.full((Z, N), 7.0, device="cuda")
        check(L.mn_gemv_glu_indexed_scaled(ptr(D(x)), K, top, ptr(D(w)), K, 2 * N * K, ptr(D(idx)), E, ptr(D(s)), ptr(out), N, Z, N, K, stream()))
        assert err(out, ref) < 1e-5
        if K % 8 or N % 8:
            continue
        counts, offsets = torch.zeros(E + 1, dtype=torch.int32, device="cuda"), torch.zeros(E + 1, dtype=torch.int32, device="cuda")
        perm, slot = torch.zeros(Z, dtype=torch.int32, device="cuda"), torch.zeros(Z, dtype=torch.int32, device="cuda")
        ws = torch.zeros(Z, device="cuda")
        tile_g, tile_m0 = (torch.zeros(Z // 256 + E + 1, dtype=torch.int32, device="cuda") for _ in range(2))
        n_tiles = torch.zeros(1, dtype=torch.int32, device="cuda")
        x16, wd = D(_bf(x)), D(w)
        for tiles in (False, True):
            ws.zero_()
            check(L.mn_moe_sort_weights(ptr(D(idx)), ptr(D(s)), M, top, E, ptr(counts), ptr(offsets), ptr(perm), ptr(slot), ptr(ws), 256 if tiles else 0,
                                        ptr(tile_g) if tiles else None, ptr(tile_m0) if tiles else None, ptr(n_tiles) if tiles else None, stream()))
            sl = slot.long().cpu()
            assert bool((ws.cpu()[sl] == s).all()) and bool((perm.cpu()[sl] == torch.arange(Z) // top).all())
            y16 = torch.zeros(Z, N, dtype=torch.bfloat16, device="cuda")
            if tiles:
                if K % 64 or N % 64:
                    continue
                check(L.mn_gemm256_grouped_tiles_scaled(ptr(x16), K, 0, M, ptr(perm), ptr(wd), K, 2 * N * K, ptr(offsets), ptr(counts), E, ptr(tile_g),
                                                        ptr(tile_m0), ptr(n_tiles), Z // 256 + E, ptr(ws), ptr(y16), N, 0, N, K, 6, stream()))
            else:
                xg, gu = torch.zeros(Z, K, dtype=torch.bfloat16, device="cuda"), torch.zeros(Z, 2 * N, device="cuda")
                check(L.mn_gather_rows_bf16(ptr(x16), K, ptr(perm), ptr(xg), K, Z, K, stream()))
                check(L.mn_gemm_bf16_grouped(ptr(xg), K, ptr(wd), K, 2 * N * K, ptr(offsets), ptr(counts), E, ptr(gu), 2 * N, Z, 2 * N, K, GEMM_F32, stream()))
                check(L.mn_silu_mul_rows_scaled(ptr(gu), 2 * N, ptr(ws), None, 0, ptr(y16), N, Z, N, stream()))
                y32 = torch.zeros(Z, N, device="cuda")
                check(L.mn_silu_mul_rows_scaled(ptr(gu), 2 * N, None, ptr(y32), N, None, 0, Z, N, stream()))     # no factors: the plain form
                assert err(y32, O.silu(gu[:, :N].double().cpu()) * gu[:, N:].double().cpu()) < 1e-6
                _KEEP.append((xg, gu))
            assert err(y16.float()[slot.long()], ref) < 2e-2, (M, N, K, tiles)
        if M <= 64 and int(counts.max()) <= 64:
            hi = _bf(x)
            Y = D(torch.stack([hi, _bf(x - hi.float())]).contiguous())
            P, y2 = torch.zeros(2, Z, 2 * N, device="cuda"), torch.zeros(2, Z, N, dtype=torch.bfloat16, device="cuda")
            nz = L.mn_stream_mfma_grouped(ptr(Y), M, ptr(wd), 2 * N * K, ptr(P), Z, ptr(offsets), ptr(perm), E, min(64, Z), 2 * N, K, stream())
            assert 1 <= nz <= 2
            check(L.mn_silu_split_rows_scaled(ptr(P), nz, Z, N, ptr(ws), ptr(y2), stream()))
            assert err(y2.double().sum(0)[slot.long()], ref) < 1e-4, (M, N, K)


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
    """The first positions on a reused sequence: a softmax over one key and the extra one."""
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
        reqs = {3: clear(cfg, sd, 120, 1), 0: clear(cfg, sd, 9, 2), 2: clear(cfg, sd, 43, 3)}
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
    """A cache sequence that held a longer request is given back and reused: its old keys and values stay in memory and must not leak into
    the next request (nothing is cleared)."""
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
    """300 decoded tokens: chunks fill and end many times."""
    for name in ("odd", "mixed"):
        cfg, sd, dec = make(name)
        t = toks(cfg, 300, 11)
        assert err(run_portions(dec, 0, t, [5] + [1] * 295), ref_logits(cfg, sd, t)) < 1e-4


def test_bf16_arithmetic():
    """Serving arithmetic: portions above 64 rows take the bf16 MFMA products (the experts the grouped ones), portions of 9 .. 64 rows the
    weight-streaming MFMA route on hi/lo rows, rows fed a few at a time fp32 FMA."""
    for name in ("mixed", "odd", "wide", "tail"):         # "odd": no K is a multiple of 8
        cfg, sd, dec = make(name, arith="bf16")
        t = clear(cfg, sd, 150)
        ref = ref_logits(cfg, sd, t)
        for cuts in ([150], [70, 40, 31, 9]):
            e = (run_portions(dec, 0, t, cuts).double().cpu() - ref).abs().amax(-1) / ref.abs().max()
            assert float(e.max()) < 6e-2 and float(e.median()) < 1.5e-2, (name, cuts, float(e.max()), float(e.median()))
        assert err(run_portions(dec, 0, t[:30], [1] * 30), ref[:30]) < 1e-4


def test_bf16_expert_routes():
    """Widths that are multiples of 64 put the experts on the 256-tile grouped GEMM with its scaled epilogue, others of 8 on the grouped
    GEMM with the activation behind it, the rest on pair-by-pair products: all against the oracle, prompts and shared decode batches."""
    for W, ff in ((64, 64), (128, 64), (64, 40), (44, 30)):
        cfg = O.small_config([O.attention_layer(mlp=O.moe(6, 2, ff)), O.attention_layer(mlp=O.moe(5, 3, ff))], width=W, vocab=70)
        sd = O.random_weights(cfg, 3)
        dec = build(cfg, sd, "bf16", n_seq=16)
        t = clear(cfg, sd, 90, 1)
        ref = ref_logits(cfg, sd, t)
        assert err(run_portions(dec, 0, t, [90]), ref) < 5e-2 and err(run_portions(dec, 0, t, [50, 20, 20]), ref) < 5e-2
        prompts = {s: clear(cfg, sd, 3 + s, 20 + s) for s in range(16)}   # sixteen sequences decode one row each
        for s, p in prompts.items():
            run_portions(dec, s, p[:-1], [len(p) - 1])
        lg = dec.logits(run_spans(dec, [p[-1] for p in prompts.values()], [(s, 1, len(p) - 1) for s, p in prompts.items()]))
        for i, p in enumerate(prompts.values()):
            assert err(lg[i:i + 1], ref_logits(cfg, sd, p)[-1:]) < 5e-2, (W, ff, i)


def test_greedy_generation_entry_point():
    """FegaraxForCausalLM.generate: unequal prompts in one lock-step batch; every new token is the oracle's arg-max given the tokens before
    it (or the oracle's two best are within 1e-4), alone or batched, with and without the captured decode step; sampled generation
    returns tokens and gives its cache sequences back."""
    from ming_univision_amd.fegarax import FegaraxForCausalLM
    cfg, sd, dec = make("mixed")
    lm = FegaraxForCausalLM(dec)
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
        whole = {s: clear(cfg, sd, 5 + 7 * (s % 4) + 24, 1 + s) for s in range(B)}
        prompts, follow = {s: t[:-24] for s, t in whole.items()}, {s: t[-24:] for s, t in whole.items()}
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


def test_trace_runner(tmp_path):
    """bin/trace_run on a saved model: a request in portions interleaved with a second one, logits against the oracle; the first
    request's cache sequence is reused by a third."""
    from safetensors.torch import save_file
    cfg = config("mixed")
    sd = O.random_weights(cfg, 3)
    mdir, odir = tmp_path / "model", tmp_path / "out"
    mdir.mkdir()
    (mdir / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(mdir / "model.safetensors"))
    a, b, c = clear(cfg, sd, 25, 1), clear(cfg, sd, 6, 2), clear(cfg, sd, 11, 3)
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
