"""Fegarax: a decoder-only language model whose residual is several parallel streams, served by libmingnative's multi-stream step function
(mingnative.h section 14: mn_ms_step).

Per token, with x_1 .. x_S its fp32 residual streams (all equal to the scaled embedding at the start), N a layer's norm
N(u) = u / sqrt(mean(u^2) + eps) (1 + w), and for each of a layer's two sublayers f the numbers in, out, mix:
    u = sum_s in[s] x_s;   y = f(N(u));   x_t <- sum_s mix[s, t] x_s + out[t] y
    attention  q, k, v = W h + b; q and k RMS-normed over their whole rows, then rotary half pairs (YaRN frequencies) on the first rot.dims
               values of a head; v <- (1 - lambda) v + lambda v_first in every v_mix layer after the first one; a position sees its own
               chunk of mask.size positions up to itself; softmax with one added to the denominator; heads times sigmoid(W_g h); W_o
    experts    the top experts by s = sigmoid(W_router h): sum of W_down (silu(W_gate s h) * W_up s h)
Then N of the streams' sum, and the embedding table (unscaled) as vocabulary projection.

This module owns HBM residency, like the other decoders' modules:
  * weights bf16; [q ; k ; v ; g] stacked at load into ONE matrix with one bias row (zero for g), experts in [experts, 2 ff, width] /
    [experts, width, ff] blocks, the router padded to a multiple of 8 rows; the streams' numbers as fp32 device vectors, rotary frequencies
    computed once in double on the host, lambda as a host number;
  * per layer: fp32 key / value arenas [n_seq, t_max, .], the values as mixed; cache sequences are numbered as in the other decoders
    (`sequences.SequenceSlots`); a number that is given back is reused as it is: a row reads no slot after its own and none before its chunk;
  * per-row int32 bookkeeping on the device, so a lock-step decode loop never syncs with the host.
`arith`: "bf16" = matrix products of steps above 8 rows on the bf16 MFMA kernels (fp32 accumulate), everything else fp32;
"f32" = fp32 FMA everywhere.
"""
import ctypes as C
import glob
import os

import torch

from ._lib import MsLayer, MsModel, lib
from .configuration import FegaraxConfig, fegarax_param_shapes
from .sakinex import rotary_table
from .seq_lm import ARITH, MultiStreamSteps, SeqCausalLM, SeqDecoder


class FegaraxDecoder(MultiStreamSteps, SeqDecoder):
    """Weights + per-layer caches + the C-ABI tables of the stack."""

    def __init__(self, cfg: FegaraxConfig, sd, t_max=2048, n_seq=1, arith="bf16"):
        """sd: {checkpoint tensor name: bf16 CUDA tensor}."""
        assert arith in ARITH, f"arith={arith!r}: 'bf16' or 'f32'"
        self.cfg, self.arith = cfg, arith
        missing = [k for k, shp in fegarax_param_shapes(cfg).items() if k not in sd or tuple(sd[k].shape) != tuple(shp)]
        if missing:
            raise ValueError(f"checkpoint does not fit the configuration: missing or mis-shaped tensors {missing[:8]}")
        dev = sd["embed"].device
        self.device = dev
        self.embed_w = self.head_w = sd["embed"].contiguous()
        self.t_max, self.n_seq = int(t_max), int(n_seq)
        W, S = cfg.width, cfg.streams or 1
        self._keep = []                                  # packed tensors the C tables point to
        bf = dict(dtype=torch.bfloat16, device=dev)
        one = {n: torch.ones(shp, dtype=torch.float32, device=dev) for n, shp in (("in", (1,)), ("out", (1,)), ("mix", (1, 1)))}
        layers = (MsLayer * len(cfg.layers))()
        self.dims = []                                   # per layer: {state key: shape per cached token}
        for i, ly in enumerate(cfg.layers):
            m, mlp, p, L = ly["mixer"], ly.get("mlp"), f"l{i}.", layers[i]
            H, G, d, e = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
            L.heads, L.kv_heads, L.dim, L.vdim, L.scale, L.has_gate = H, G, d, e, float(m["scale"]), 1
            L.norm1 = self._p(sd[p + "norm1"])
            stack = [sd[p + "mix." + n] for n in ("q", "k", "v", "g")]
            bias = [sd[p + "mix." + n + ".b"] for n in ("q", "k", "v")]
            rows, biased = sum(x.shape[0] for x in stack), sum(b.shape[0] for b in bias)
            pad = -rows % 8                              # zero rows: the stack's row count a multiple of 8
            L.w_in = self._p(torch.cat(stack + [torch.zeros(pad, W, **bf)], 0))
            L.b_in = self._p(torch.cat(bias + [torch.zeros(rows + pad - biased, **bf)]))
            L.q_norm, L.k_norm, L.w_o = self._p(sd[p + "mix.q.norm"]), self._p(sd[p + "mix.k.norm"]), self._p(sd[p + "mix.o"])
            L.sink = self._f(torch.zeros(H, dtype=torch.float32, device=dev))      # exp(0) joins every head's denominator
            L.chunk = int((m.get("mask") or {}).get("size") or 0)
            rot, L.rot_mag = m.get("rot"), 1.0
            if rot and int(rot["dims"]) > 0:
                freq, L.rot_mag = rotary_table(rot, dev)
                L.rot_dims, L.rot_freq = int(rot["dims"]), self._f(freq)
            if m.get("v_mix"):
                L.v_mix, L.v_lambda = 1, float(sd[p + "mix.vmix"].float())
            if mlp is not None:
                E, q = int(mlp["router"]["experts"]), p + "mlp."
                L.experts, L.top, L.expert_ff = E, int(mlp["router"]["top"]), int(mlp["expert"]["ff"])
                L.norm2 = self._p(sd[p + "norm2"])
                L.w_router = self._p(torch.cat([sd[q + "router"], torch.zeros(-E % 8, W, **bf)], 0))
                L.w_gate_up = self._p(torch.stack([torch.cat([sd[f"{q}e{j}.gate"], sd[f"{q}e{j}.up"]], 0) for j in range(E)]))
                L.w_down = self._p(torch.stack([sd[f"{q}e{j}.down"] for j in range(E)]))
            for sub in (1, 2) if mlp is not None else (1,):
                for n in ("in", "out", "mix"):
                    setattr(L, f"hc{sub}_{n}", self._f(one[n] if cfg.streams is None else sd[f"{p}hc{sub}.{n}"].float()))
            self.dims.append(dict(k=(G * d,), v=(G * e,)))
        self._layers = layers
        self.n_trace = len(cfg.layers)
        self.block_rows = int(lib().mn_window_attn_block_rows())
        s = MsModel()
        s.width, s.n_layers, s.streams, s.arith, s.norm_one_plus, s.eps = W, len(cfg.layers), S, ARITH[arith], 1, cfg.eps
        s.layers = C.cast(layers, C.POINTER(MsLayer))
        s.final_w = self._p(sd["final.norm"])
        self.struct = s
        self._ws, self._decode_tabs = {}, {}
        self._init_state()

    # ---- construction ---------------------------------------------------------------------------------------------------------
    @classmethod
    def from_pretrained(cls, path, device="cuda", **kw):
        """A directory with config.json and *.safetensors (bf16 tensors under the checkpoint's names)."""
        from .infer import load_safetensors_dir
        cfg = FegaraxConfig.from_pretrained(path)
        if not glob.glob(os.path.join(path, "*.safetensors")):
            raise FileNotFoundError(f"{path}: no *.safetensors")
        return cls(cfg, {k: v.to(device, torch.bfloat16) for k, v in load_safetensors_dir(path).items()}, **kw)

    @classmethod
    def synthetic(cls, cfg, device="cuda", seed=0, **kw):
        """Random weights of the architecture (synth.py's rule by tensor name); the streams mix with weight on and off the diagonal."""
        from .synth import synth_tensor
        sd = {}
        for k, shp in fegarax_param_shapes(cfg).items():
            mean, std = 0.0, (shp[-1] if shp else 1) ** -0.5
            if k == "embed":
                std = 1.0
            elif k.endswith(".norm1") or k.endswith(".norm2") or k == "final.norm":
                std = 0.05
            elif k.endswith(".q.norm") or k.endswith(".k.norm"):
                mean, std = 1.0, 0.05
            elif k.endswith(".b"):
                std = 0.1
            elif k.endswith(".vmix"):
                mean, std = 0.4, 0.1
            elif ".hc" in k:
                mean, std = (1.0 if k.endswith(".out") else 1.0 / shp[-1]) if not k.endswith(".mix") else 0.0, 0.1
            sd[k] = synth_tensor(k, shp or (1,), seed, device, torch.bfloat16, mean=mean, std=std).reshape(shp)
            if k.endswith(".mix") and ".hc" in k:
                sd[k] = (sd[k] + torch.eye(shp[0], dtype=torch.bfloat16, device=device)).contiguous()
        return cls(cfg, sd, **kw)

    # ---- vocabulary -----------------------------------------------------------------------------------------------------------
    def embed(self, ids):
        x = super().embed(ids)
        return x.mul_(self.cfg.embed_scale) if self.cfg.embed_scale != 1.0 else x


class FegaraxForCausalLM(SeqCausalLM):
    """`SeqCausalLM` over a `FegaraxDecoder`."""

    @classmethod
    def from_pretrained(cls, path, device="cuda", t_max=2048, arith="bf16", eos_token_id=None):
        return cls(FegaraxDecoder.from_pretrained(path, device=device, t_max=t_max, arith=arith), eos_token_id)
