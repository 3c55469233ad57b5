"""Sabezen: a decoder-only language model of parallel layers with channel-wise decaying recurrences and mixed attention heads, served by
libmingnative's hybrid-mixer step function (mingnative.h sections 11 and 13: mn_hyb_step).

Per layer, with x the fp32 residual stream of a token:
    h = LayerNorm(x) w                              one norm (no bias); the mixer and the feed-forward both read it
    x += mixer(h) + ff(h)
    mixer "attention":     q, k = W h, values = the projected keys; rotary half pairs on the first rot.dims values of a head, then q and k
                           divided by their root mean square; scores q . k * scale, mixed over the heads by a matrix; a position sees
                           its own chunk of mask.size positions up to itself; softmax with one added to the denominator; W_o
    mixer "channel_delta": q, k (kv_heads) and v (heads) through a short causal filter and silu; q, k unit vectors; per head
                           S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q with beta = sigmoid(W_b h) and
                           g = exp(-exp(A_log) softplus(W_a2 (W_a1 h) + dt_bias)) per key channel; per-head RMS norm times
                           sigmoid(W_g2 (W_g1 h)); W_o
    mixer "gla":           S <- diag(a) S + k v^T, o = S^T q, a = sigmoid(W_a2 (W_a1 h) + bias)^(1 / tau); per-head RMS norm times
                           silu(W_g h); W_o
    ff dense:              W_down xielu(W_up h)
    ff moe:                the mean of W_down (silu(W_gate h) * W_up h) over the experts that a table names for the token's id
The input embeddings are scaled by embedding.scale; then LayerNorm and the vocabulary projection.

This module owns HBM residency, like the other decoders' modules:
  * weights bf16; everything that reads h is stacked at load into ONE matrix (attention [q ; k], channel delta [q ; k ; v ; a1 ; g1 ; b],
    gla [q ; k ; v ; g ; a1], then the dense feed-forward's up) and the mixer's output projection is joined with the dense feed-forward's
    down projection along their inputs; experts lie in [experts, 2 ff, width] / [experts, width, ff] blocks, tables as int32; mixing
    matrices and A_log as fp32 device vectors, rotary frequencies computed once in double on the host, the activation's two factors
    once in fp32;
  * per layer: fp32 key / value arenas [n_seq, t_max, .] (attention), the fp32 recurrent state [n_seq, heads, dim, vdim] and, for channel
    delta, the filters' last inputs [n_seq, conv - 1, channels]; cache sequences are numbered as in the other decoders
    (`sequences.SequenceSlots`); a number that is given back is reused as it is: a row at position 0 reads no state;
  * per-row int32 bookkeeping on the device, so a lock-step decode loop never syncs with the host.
`arith`: "bf16" = matrix products of steps above 8 rows on the bf16 MFMA kernels (fp32 accumulate), everything else fp32;
"f32" = fp32 FMA everywhere.
"""
import ctypes as C
import glob
import math
import os

import torch

from ._lib import HybLayer, HybModel, lib
from .configuration import SabezenConfig, sabezen_param_shapes
from .daberax import UNIT_EPS, rotary_frequencies
from .seq_lm import ARITH, HybridSteps, SeqCausalLM, SeqDecoder

KIND = {"attention": 2, "channel_delta": 3, "gla": 4}
FF_NONE, FF_DENSE, FF_MOE = 0, 1, 2
ACT_XIELU, NORM_LAYER = 1, 1


def _softplus(z):
    return max(z, 0.0) + math.log1p(math.exp(-abs(z)))


class SabezenDecoder(HybridSteps, SeqDecoder):
    """Weights + per-layer caches and states + the C-ABI tables of the stack."""

    def __init__(self, cfg: SabezenConfig, sd, t_max=2048, n_seq=1, arith="bf16"):
        """sd: {checkpoint tensor name: CUDA tensor, bf16 (tables: integer)}."""
        assert arith in ARITH, f"arith={arith!r}: 'bf16' or 'f32'"
        self.cfg, self.arith = cfg, arith
        shapes = sabezen_param_shapes(cfg, lambda k: sd[k].shape[0] if k in sd else 0)
        missing = [k for k, shp in shapes.items() if k not in sd or tuple(sd[k].shape) != tuple(shp)]
        if missing:
            raise ValueError(f"checkpoint does not fit the configuration: missing or mis-shaped tensors {missing[:8]}")
        dev = sd["embed"].device
        self.device = dev
        self.embed_w, self.head_w = sd["embed"].contiguous(), sd["head"].contiguous()
        self.t_max, self.n_seq = int(t_max), int(n_seq)
        W = cfg.width
        self._keep = []                                  # packed tensors the C tables point to
        bf = dict(dtype=torch.bfloat16, device=dev)
        layers = (HybLayer * len(cfg.layers))()
        self.dims = []                                   # per layer: {state key: shape behind the sequence axis (per token for k, v)}
        self.needs_tokens = False
        for i, ly in enumerate(cfg.layers):
            m, mlp, p, L, t = ly["mixer"], ly.get("mlp"), f"l{i}.", layers[i], ly["type"]
            H, d = int(m["heads"]), int(m["dim"])
            e = int(m.get("vdim", d))
            L.kind, L.heads, L.kv_heads, L.dim, L.vdim = KIND[t], H, int(m.get("kv_heads", H)), d, e
            G = L.kv_heads
            L.norm1 = self._p(sd[p + "norm1"])
            if t == "attention":
                stack = [sd[p + "mix.q"], sd[p + "mix.k"]]
                L.scale = float(m["scale"])
                L.talk = self._f(sd[p + "mix.talk"].float())
                L.sink = self._f(torch.zeros(H, dtype=torch.float32, device=dev))      # exp(0) joins every head's denominator
                L.chunk = int((m.get("mask") or {}).get("size") or 0)
                rot = m.get("rot")
                if rot and int(rot["dims"]) > 0:
                    L.rot_dims, L.rot_freq = int(rot["dims"]), self._f(rotary_frequencies(rot, dev))
                self.dims.append(dict(k=(G * d,), v=(G * d,)))
            elif t == "channel_delta":
                stack = [sd[p + "mix." + n] for n in ("q", "k", "v", "a1", "g1", "b")]
                L.conv, L.unit_eps = int(m["conv"]), UNIT_EPS
                L.w_conv = self._p(torch.cat([sd[p + "mix.q.conv"], sd[p + "mix.k.conv"], sd[p + "mix.v.conv"]], 0))
                L.rank_a, L.rank_g = sd[p + "mix.a1"].shape[0], sd[p + "mix.g1"].shape[0]
                L.a_log = self._f(sd[p + "mix.A_log"].float())
                L.w_a2, L.b_a2, L.w_g2 = self._p(sd[p + "mix.a2"]), self._p(sd[p + "mix.dt_bias"]), self._p(sd[p + "mix.g2"])
                L.mix_norm = self._p(sd[p + "mix.norm"])
                self.dims.append(dict(lin=(H, d, e), conv=(L.conv - 1, 2 * G * d + H * e) if L.conv > 1 else None))
            else:
                stack = [sd[p + "mix." + n] for n in ("q", "k", "v", "g", "a1")]
                L.rank_a, L.root = sd[p + "mix.a1"].shape[0], 1.0 / float(m["tau"])
                L.w_a2, L.b_a2 = self._p(sd[p + "mix.a2"]), self._p(sd[p + "mix.a2.b"])
                L.mix_norm = self._p(sd[p + "mix.norm"])
                self.dims.append(dict(lin=(H, d, e)))
            out = [sd[p + "mix.o"]]
            L.ff_kind = FF_NONE
            if mlp is not None and mlp["kind"] == "dense":
                L.ff_kind, L.ff, L.ff_act = FF_DENSE, int(mlp["ff"]), ACT_XIELU
                act = sd[p + "mlp.act"].double().tolist()
                L.act_pos, L.act_neg = _softplus(act[0]), 0.5 + _softplus(act[1])
                stack.append(sd[p + "mlp.up"])
                out.append(sd[p + "mlp.down"])
            elif mlp is not None:
                E, q = int(mlp["router"]["experts"]), p + "mlp."
                L.ff_kind, L.experts, L.top, L.expert_ff, L.expert_glu = FF_MOE, E, int(mlp["router"]["top"]), int(mlp["expert"]["ff"]), 1
                table = sd[q + "table"].to(torch.int32).contiguous()
                if int(table.min()) < 0 or int(table.max()) >= E:
                    raise ValueError(f"layer {i}: the expert table names experts outside 0 .. {E - 1}")
                self._keep.append(table)
                L.table = table.data_ptr()
                L.w_up = self._p(torch.stack([torch.cat([sd[f"{q}e{j}.gate"], sd[f"{q}e{j}.up"]], 0) for j in range(E)]))
                L.w_down = self._p(torch.stack([sd[f"{q}e{j}.down"] for j in range(E)]))
                self.needs_tokens = True
            rows = sum(x.shape[0] for x in stack)
            stack.append(torch.zeros(-rows % 8, W, **bf))                # zero rows: the stack's row count a multiple of 8
            L.w_in = self._p(torch.cat(stack, 0))
            L.w_out = self._p(torch.cat(out, 1))
        self._layers = layers
        n = len(cfg.layers)
        self.runs, self.n_trace = list(range(n)), n
        self._run_layer = (C.c_int32 * n)(*self.runs)
        # rows per run of the attention: what every attention layer's matrix-core kernel takes (a layer without an instance takes any)
        takes = [lib().mn_talk_attn_block_rows(L.heads, L.kv_heads, L.dim) for L in layers if L.kind == KIND["attention"]]
        self.block_rows = min([int(r) for r in takes if r > 0] or [8])
        if any(L.kind == KIND["gla"] for L in layers):
            self.chunk_rows = int(lib().mn_channel_chunk_rows())
        s = HybModel()
        s.width, s.n_layers, s.n_runs, s.arith, s.eps = W, n, n, ARITH[arith], cfg.eps
        s.norm, s.vocab, s.block_rows = NORM_LAYER, cfg.vocab, self.block_rows
        s.layers = C.cast(layers, C.POINTER(HybLayer))
        s.run_layer = self._run_layer
        s.final_w = self._p(sd["final.norm"])
        self.struct = s
        self._ws, self._decode_tabs = {}, {}
        self._init_state()

    # ---- construction ---------------------------------------------------------------------------------------------------------
    @classmethod
    def from_pretrained(cls, path, device="cuda", **kw):
        """A directory with config.json and *.safetensors (bf16 tensors under the checkpoint's names, integer tables)."""
        from .infer import load_safetensors_dir
        cfg = SabezenConfig.from_pretrained(path)
        if not glob.glob(os.path.join(path, "*.safetensors")):
            raise FileNotFoundError(f"{path}: no *.safetensors")
        sd = {k: v.to(device, torch.bfloat16 if v.is_floating_point() else torch.int32) for k, v in load_safetensors_dir(path).items()}
        return cls(cfg, sd, **kw)

    @classmethod
    def synthetic(cls, cfg, device="cuda", seed=0, rank=128, **kw):
        """Random weights of the architecture (synth.py's rule by tensor name); rank: of the low-rank projections."""
        from .synth import synth_tensor
        sd = {}
        for k, shp in sabezen_param_shapes(cfg, lambda name: rank).items():
            if k.endswith("mlp.table"):
                g = torch.Generator().manual_seed(seed + len(sd))
                E = int(cfg.layers[int(k[1:k.index(".")])]["mlp"]["router"]["experts"])
                sd[k] = torch.rand(shp[0], E, generator=g).argsort(1)[:, :shp[1]].to(device, torch.int32)
                continue
            mean, std = 0.0, shp[-1] ** -0.5
            if k == "embed" or k.endswith("dt_bias"):
                std = 1.0
            elif k.endswith("A_log"):
                mean, std = -1.0, 0.5
            elif k.endswith("a2.b"):
                mean, std = 2.0, 1.0
            elif k.endswith(".conv") or k.endswith(".act"):
                std = 0.5
            elif "norm" in k:
                mean, std = 1.0, 0.05
            sd[k] = synth_tensor(k, shp, seed, device, torch.bfloat16, mean=mean, std=std)
            if k.endswith(".talk"):
                sd[k] = (sd[k] + torch.eye(shp[0], dtype=torch.bfloat16, device=device)).contiguous()
        return cls(cfg, sd, **kw)

    # ---- vocabulary -----------------------------------------------------------------------------------------------------------
    def embed(self, ids):
        x = super().embed(ids)
        return x.mul_(self.cfg.embed_scale) if self.cfg.embed_scale != 1.0 else x


class SabezenForCausalLM(SeqCausalLM):
    """`SeqCausalLM` over a `SabezenDecoder`."""

    @classmethod
    def from_pretrained(cls, path, device="cuda", t_max=2048, arith="bf16", eos_token_id=None):
        return cls(SabezenDecoder.from_pretrained(path, device=device, t_max=t_max, arith=arith), eos_token_id)
