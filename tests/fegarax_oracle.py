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
def pick_experts(h, w_router, top):
    """-> (experts [T, top], their scores [T, top])."""
    s = torch.sigmoid(h @ f64(w_router).T)
    idx = torch.argsort(s, dim=-1, descending=True, stable=True)[:, :top]
    return idx, torch.gather(s, 1, idx)


def expert_mixture(h, sd, p, mlp):
    idx, w = pick_experts(h, sd[p + "router"], int(mlp["router"]["top"]))
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
def forward(cfg, sd, tokens):
    """-> (logits [T, vocab], the streams' sum after every layer [layers, T, width])."""
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
            X = streams_write(X, expert_mixture(h, sd, p + "mlp.", ly["mlp"]), sd[p + "hc2.mix"], sd[p + "hc2.out"])
        trace.append(X.sum(0))
    return norm_zero(X.sum(0), sd["final.norm"], eps) @ f64(sd["embed"]).T, torch.stack(trace)
