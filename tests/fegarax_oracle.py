"""Fegarax in plain float64 on the CPU: one function per mechanism, whole sequences at a time, no cache and no code shared with the
package.  The tests hold the served path (native step function, arenas, kernels) against it.

A model is (cfg, sd): cfg the dict of a config.json, sd {tensor name: torch tensor}.  Notation: X [streams, T, width] are the residual
streams of one sequence whose first row is position 0.

    start          every stream is the scaled embedding
    sublayer q     u = sum_s in_q[s] X_s;  y = f(norm_q(u));  X_t <- sum_s mix_q[s, t] X_s + out_q[t] y
    norm           u / sqrt(mean(u^2) + eps) * (1 + w)
    attention      biased projections, q and k normed over their whole rows, YaRN half-pair rotation, chunks of positions that see only
                   themselves, softmax with one added to its denominator, values mixed with those of the first mixing layer, output gate
    experts        sum over the chosen experts e of E_e(s_e h), s = sigmoid(router h), the largest scores chosen
    end            the streams' sum, norm, the embedding table as vocabulary projection
"""
import math

import torch

F64 = torch.float64


def f64(t):
    return t.detach().to("cpu", F64)


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_zero(x, w, eps):
    """RMS norm whose stored weight is zero where it does nothing."""
    return rms(x, eps) * (1.0 + f64(w))


def silu(z):
    return z * torch.sigmoid(z)


# ---- streams -------------------------------------------------------------------------------------------------------------------
def streams_read(X, w_in):
    u = torch.zeros_like(X[0])
    for s in range(X.shape[0]):
        u = u + float(w_in[s]) * X[s]
    return u


def streams_write(X, y, mix, w_out):
    """All streams at once from the old ones; mix is indexed [from, to]."""
    S = X.shape[0]
    new = []
    for t in range(S):
        row = float(w_out[t]) * y
        for s in range(S):
            row = row + float(mix[s, t]) * X[s]
        new.append(row)
    return torch.stack(new)


# ---- attention -----------------------------------------------------------------------------------------------------------------
def rotary_frequencies(rot):
    """-> (frequencies [dims / 2], factor of cos and sin)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def turns_to_index(t):
        return dims * math.log(original / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turns_to_index(float(sc["fast"]))), 0)
    hi = min(math.ceil(turns_to_index(float(sc["slow"]))), dims - 1)
    width = max(hi - lo, 0.001)
    out = []
    for i in range(dims // 2):
        r = min(max((i - lo) / width, 0.0), 1.0)
        out.append(float(f[i]) / factor * r + float(f[i]) * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(factor) + 1.0


def rotate_halves(x, freq, mag, pos0=0):
    """x [T, heads, n]: values (i, i + len(freq)), i < len(freq), of a head turn by position * freq_i and grow by mag; the rest pass."""
    T, half = x.shape[0], freq.numel()
    ang = torch.arange(pos0, pos0 + T, dtype=F64)[:, None] * freq[None, :]
    c, s = (torch.cos(ang) * mag)[:, None, :], (torch.sin(ang) * mag)[:, None, :]
    a, b = x[..., :half], x[..., half:2 * half]
    out = x.clone()
    out[..., :half] = a * c - b * s
    out[..., half:2 * half] = b * c + a * s
    return out


def visible(T, chunk=None):
    """[T, T] mask: row i sees column j <= i of its own chunk of `chunk` positions."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    m = j <= i
    if chunk:
        m &= (i // int(chunk)) == (j // int(chunk))
    return m


def sink_softmax_attention(q, k, v, scale, mask, sink=True):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; sink: the softmax's denominator has one added."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        s = ((q[:, h] @ k[:, h // rep].T) * scale).masked_fill(~mask, -math.inf)
        top = torch.clamp(s.amax(-1, keepdim=True), min=0.0) if sink else s.amax(-1, keepdim=True)
        p = torch.exp(s - top)
        out[:, h] = p @ v[:, h // rep] / (p.sum(-1, keepdim=True) + (torch.exp(-top) if sink else 0.0))
    return out


def attention_mixer(h, sd, p, m, eps, v_first):
    """-> (result, values of this layer as later layers mix them in)."""
    H, G, d, e = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q, k, v = (h @ f64(sd[p + n]).T + f64(sd[p + n + ".b"]) for n in ("q", "k", "v"))
    q = (rms(q, eps) * f64(sd[p + "q.norm"])).reshape(T, H, d)
    k = (rms(k, eps) * f64(sd[p + "k.norm"])).reshape(T, G, d)
    if m.get("rot"):
        fr, mag = rotary_frequencies(m["rot"])
        q, k = rotate_halves(q, fr, mag), rotate_halves(k, fr, mag)
    own = v
    if m.get("v_mix") and v_first is not None:
        lam = float(sd[p + "vmix"])
        v = (1.0 - lam) * v + lam * v_first
    o = sink_softmax_attention(q, k, v.reshape(T, G, e), float(m["scale"]), visible(T, (m.get("mask") or {}).get("size")))
    o = o.reshape(T, H * e) * torch.sigmoid(h @ f64(sd[p + "g"]).T)
    return o @ f64(sd[p + "o"]).T, own


# ---- experts -------------------------------------------------------------------------------------------------------------------
def pick_experts(h, w_router, top, gaps=None):
    """-> (experts [T, top], their scores [T, top]); gaps: a list that receives the distance [T] of the chosen logits from the next one."""
    z = h @ f64(w_router).T
    idx = torch.argsort(z, dim=-1, descending=True, stable=True)[:, :top]
    if gaps is not None and top < z.shape[1]:
        best = torch.topk(z, top + 1, dim=-1).values
        gaps.append(best[:, top - 1] - best[:, top])
    return idx, torch.sigmoid(torch.gather(z, 1, idx))


def expert_mixture(h, sd, p, mlp, gaps=None):
    idx, w = pick_experts(h, sd[p + "router"], int(mlp["router"]["top"]), gaps)
    y = torch.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        gate, up, down = (f64(sd[f"{p}e{e}.{n}"]) for n in ("gate", "up", "down"))
        for j in range(idx.shape[1]):
            rows = (idx[:, j] == e).nonzero()[:, 0]
            if rows.numel():
                x = w[rows, j][:, None] * h[rows]
                y[rows] += (silu(x @ gate.T) * (x @ up.T)) @ down.T
    return y


# ---- the model -----------------------------------------------------------------------------------------------------------------
def forward(cfg, sd, tokens, gaps=None):
    """-> (logits [T, vocab], the streams' sum after every layer [layers, T, width]); gaps as in pick_experts, one entry per routed layer."""
    eps = float(cfg["norm"]["eps"])
    x = f64(sd["embed"])[torch.as_tensor(tokens, dtype=torch.long)] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    X = torch.stack([x] * int(cfg["streams"]))
    v_first, trace = None, []
    for i, ly in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = norm_zero(streams_read(X, sd[p + "hc1.in"]), sd[p + "norm1"], eps)
        y, own = attention_mixer(h, sd, p + "mix.", ly["mixer"], eps, v_first)
        if v_first is None and ly["mixer"].get("v_mix"):
            v_first = own
        X = streams_write(X, y, sd[p + "hc1.mix"], sd[p + "hc1.out"])
        if ly.get("mlp") is not None:
            h = norm_zero(streams_read(X, sd[p + "hc2.in"]), sd[p + "norm2"], eps)
            X = streams_write(X, expert_mixture(h, sd, p + "mlp.", ly["mlp"], gaps), sd[p + "hc2.mix"], sd[p + "hc2.out"])
        trace.append(X.sum(0))
    return norm_zero(X.sum(0), sd["final.norm"], eps) @ f64(sd["embed"]).T, torch.stack(trace)


# ---- small models for the tests ----------------------------------------------------------------------------------------------------
def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def attention_layer(heads=4, kv_heads=2, dim=16, vdim=12, scale=0.3, rot=(10000.0, 8), scaling=(4.0, 64, 8.0, 1.0), chunk=11, v_mix=True, mlp=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if chunk:
        m["mask"] = {"size": chunk}
    if v_mix:
        m["v_mix"] = True
    return {"type": "attention", "mixer": m, "mlp": mlp}


def small_config(layers, width=64, vocab=80, streams=3, scale=2.5, eps=1e-5):
    return {"architecture": "Fegarax", "width": width, "vocab": vocab, "streams": streams, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


def param_shapes(cfg):
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    s = {"embed": (V, W), "final.norm": (W,)}
    for i, ly in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", ly["mixer"], ly.get("mlp")
        nq, nk, nv, no = (m[a] * m[b] for a, b in (("heads", "dim"), ("kv_heads", "dim"), ("kv_heads", "vdim"), ("heads", "vdim")))
        for n, rows in (("q", nq), ("k", nk), ("v", nv)):
            s.update({f"{p}mix.{n}": (rows, W), f"{p}mix.{n}.b": (rows,)})
        s.update({p + "norm1": (W,), p + "mix.q.norm": (nq,), p + "mix.k.norm": (nk,), p + "mix.g": (no, W), p + "mix.o": (W, no)})
        if m.get("v_mix"):
            s[p + "mix.vmix"] = ()
        if mlp is not None:
            ff = mlp["expert"]["ff"]
            for j in range(mlp["router"]["experts"]):
                s.update({f"{p}mlp.e{j}.gate": (ff, W), f"{p}mlp.e{j}.up": (ff, W), f"{p}mlp.e{j}.down": (W, ff)})
            s.update({p + "norm2": (W,), p + "mlp.router": (mlp["router"]["experts"], W)})
        for q in (1, 2) if mlp is not None else (1,):
            s.update({f"{p}hc{q}.in": (S,), f"{p}hc{q}.out": (S,), f"{p}hc{q}.mix": (S, S)})
    return s


def random_weights(cfg, seed=0):
    """bf16 tensors under the checkpoint's names.  The streams read, mix and take results unequally; experts' scores lie well apart."""
    g = torch.Generator().manual_seed(seed)
    sd = {}
    for k, shp in param_shapes(cfg).items():
        r = torch.randn(shp, generator=g)
        if k == "embed":
            t = r
        elif k.endswith((".q.norm", ".k.norm")):
            t = 1.0 + 0.2 * r
        elif k.endswith((".norm1", ".norm2", "final.norm")):
            t = 0.2 * r
        elif k.endswith(".b"):
            t = 0.3 * r
        elif k.endswith(".vmix"):
            t = 0.4 + 0.2 * r
        elif ".hc" in k and k.endswith(".mix"):
            t = 0.7 * torch.eye(shp[0]) + 0.3 * r
        elif ".hc" in k:
            t = 0.5 + 0.4 * r
        elif k.endswith(".router"):
            t = 2.5 * r * shp[-1] ** -0.5
        else:
            t = 1.3 * r * shp[-1] ** -0.5
        sd[k] = t.to(torch.bfloat16)
    return sd


def clear_tokens(cfg, sd, n, seed=1, gap=0.06):
    """n random tokens none of which has a close call between experts (a chosen logit and the next one less than `gap` apart): rounding in
    the products before a router must not change what it picks.  A token that has one is drawn again; the tokens before it do not depend on it."""
    g = torch.Generator().manual_seed(seed)
    t = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    for _ in range(20 * n):
        gaps = []
        forward(cfg, sd, t, gaps)
        close = (torch.stack(gaps).amin(0) < gap).nonzero() if gaps else []
        if len(close) == 0:
            return t
        t[int(close[0])] = int(torch.randint(0, cfg["vocab"], (1,), generator=g))
    raise RuntimeError("no tokens without close calls")
