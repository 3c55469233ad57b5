"""Sabezen in plain float64 on the CPU: one function per mechanism, whole sequences at a time, no cache and no code shared with the
package.  The tests hold the served path (native step function, arenas, recurrent states, kernels) against it.

A model is (cfg, sd): cfg the dict of a config.json, sd {tensor name: torch tensor}.  Notation: x [T, width] is the residual stream of
one sequence whose first row is position 0.

    layer          h = layer_norm(x) (a weight, no bias);  x <- x + mixer(h) + ff(h)
    channel_delta  delta rule with a decay per key channel on filtered, silu'd, unit-length q / k:
                   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
    gla            S <- diag(a) S + k v^T,  o = S^T q,  a = sigmoid(z)^(1 / tau)
    attention      grouped heads whose values are the projected keys, rotary half pairs then a unit RMS per head, the heads' scores mixed
                   by a matrix, chunks of positions that see only themselves, softmax with one added to the denominator
    ff             dense W_down xielu(W_up h), or a mixture of silu-gated experts that a table picks by token id
"""
import math

import torch

F64 = torch.float64


def f64(t):
    return t.detach().to("cpu", F64)


def layer_norm(x, w, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * f64(w)


def unit_rms(y, eps):
    return y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def xielu(z, p, q):
    """p, q: 0-dim tensors; both branches meet at 0 with slope 1/2."""
    neg = torch.clamp(z, max=0.0)
    return torch.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (torch.expm1(neg) - neg)) + 0.5 * z


# ---- attention -----------------------------------------------------------------------------------------------------------------
def rotary_frequencies(rot):
    dims, base = int(rot["dims"]), float(rot["base"])
    return torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)


def rotate_halves(x, freq, pos0=0):
    """x [T, ..., n]: values (i, i + len(freq)), i < len(freq), of the last axis turn by the angle position * freq_i; the rest pass."""
    T, half = x.shape[0], freq.numel()
    ang = torch.arange(pos0, pos0 + T, dtype=F64)[:, None] * freq[None, :]
    shape = [T] + [1] * (x.dim() - 2) + [half]
    c, s = torch.cos(ang).reshape(shape), torch.sin(ang).reshape(shape)
    a, b = x[..., :half], x[..., half:2 * half]
    out = x.clone()
    out[..., :half] = a * c - b * s
    out[..., half:2 * half] = b * c + a * s
    return out


def visible(T, chunk=None, window=None):
    """[T, T] mask: row i sees column j <= i of its own chunk (counted from position 0) and, with a window, i - j < window."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    m = j <= i
    if chunk:
        m &= (i // int(chunk)) == (j // int(chunk))
    if window:
        m &= (i - j) < int(window)
    return m


def talking_attention(q, k, v, talk, scale, mask, sink=True):
    """q [T, H, d], k [T, G, d], v [T, G, e], talk [H, H] -> [T, H, e]; raw scores of head g read key head g // (H / G), the score of head
    h is sum_g talk[h, g] raw_g; sink: the softmax's denominator has one added."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    raw = torch.stack([(q[:, h] @ k[:, h // rep].T) * scale for h in range(H)])          # [H, T, T]
    s = (talk @ raw.reshape(H, -1)).reshape(H, T, T).masked_fill(~mask, -math.inf)
    top = s.amax(-1, keepdim=True)
    top = torch.clamp(top, min=0.0) if sink else top
    p = torch.exp(s - top)
    p = p / (p.sum(-1, keepdim=True) + (torch.exp(-top) if sink else 0.0))
    return torch.stack([p[h] @ v[:, h // rep] for h in range(H)], 1)


def attention_mixer(h, sd, p, m, eps):
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    T = h.shape[0]
    q = (h @ f64(sd[p + "q"]).T).reshape(T, H, d)
    k = (h @ f64(sd[p + "k"]).T).reshape(T, G, d)
    v = k
    if m.get("rot"):
        fr = rotary_frequencies(m["rot"])
        q, k = rotate_halves(q, fr), rotate_halves(k, fr)
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    o = talking_attention(q, k, v, f64(sd[p + "talk"]), float(m["scale"]), visible(T, (m.get("mask") or {}).get("size")))
    return o.reshape(T, H * d) @ f64(sd[p + "o"]).T


# ---- recurrences ---------------------------------------------------------------------------------------------------------------
def causal_conv(x, w):
    """x [T, C], w [C, taps] (last column multiplies the current row, zeros before the start) -> [T, C]."""
    T, C = x.shape
    taps = w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, C, dtype=F64), x], 0)
    out = torch.zeros(T, C, dtype=F64)
    for j in range(taps):
        out += pad[j:j + T] * w[:, j]
    return out


def channel_delta_rule(q, k, v, beta, g, S0=None):
    """q, k, g [T, H, d], v [T, H, e], beta [T, H] -> ([T, H, e], final state [H, d, e])."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64) if S0 is None else S0.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = S * g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - torch.einsum("hde,hd->he", S, k[t]))
        S = S + torch.einsum("hd,he->hde", k[t], u)
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out, S


def gated_linear_attention(q, k, v, a, S0=None):
    """q, k, a [T, H, d], v [T, H, e] -> ([T, H, e], final state [H, d, e])."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64) if S0 is None else S0.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = S * a[t][:, :, None] + torch.einsum("hd,he->hde", k[t], v[t])
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out, S


def channel_decays(z, a_log, dt_bias):
    """z [T, H * d], a_log [H], dt_bias [H * d] -> exp(-exp(a_log) softplus(z + dt_bias)) [T, H, d]."""
    H = a_log.numel()
    return torch.exp(-torch.exp(a_log)[None, :, None] * softplus(z + dt_bias).reshape(z.shape[0], H, -1))


def channel_delta_mixer(h, sd, p, m, eps):
    H, G, d, e = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = silu(causal_conv(h @ f64(sd[p + "q"]).T, f64(sd[p + "q.conv"]))).reshape(T, G, d)
    k = silu(causal_conv(h @ f64(sd[p + "k"]).T, f64(sd[p + "k.conv"]))).reshape(T, G, d)
    v = silu(causal_conv(h @ f64(sd[p + "v"]).T, f64(sd[p + "v.conv"]))).reshape(T, H, e)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * d ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    q, k = q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1)
    beta = torch.sigmoid(h @ f64(sd[p + "b"]).T)
    g = channel_decays(h @ f64(sd[p + "a1"]).T @ f64(sd[p + "a2"]).T, f64(sd[p + "A_log"]), f64(sd[p + "dt_bias"]))
    o, _ = channel_delta_rule(q, k, v, beta, g)
    o = unit_rms(o, eps) * f64(sd[p + "norm"]) * torch.sigmoid(h @ f64(sd[p + "g1"]).T @ f64(sd[p + "g2"]).T).reshape(T, H, e)
    return o.reshape(T, H * e) @ f64(sd[p + "o"]).T


def gla_mixer(h, sd, p, m, eps):
    H, d, e = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = (h @ f64(sd[p + "q"]).T).reshape(T, H, d) * d ** -0.5
    k = (h @ f64(sd[p + "k"]).T).reshape(T, H, d)
    v = (h @ f64(sd[p + "v"]).T).reshape(T, H, e)
    z = h @ f64(sd[p + "a1"]).T @ f64(sd[p + "a2"]).T + f64(sd[p + "a2.b"])
    a = torch.sigmoid(z) ** (1.0 / float(m["tau"]))
    o, _ = gated_linear_attention(q, k, v, a.reshape(T, H, d))
    o = (unit_rms(o, eps) * f64(sd[p + "norm"])).reshape(T, H * e) * silu(h @ f64(sd[p + "g"]).T)
    return o @ f64(sd[p + "o"]).T


MIXERS = {"attention": attention_mixer, "channel_delta": channel_delta_mixer, "gla": gla_mixer}


# ---- feed-forwards and the stack -------------------------------------------------------------------------------------------------
def dense_ff(h, sd, p, mlp, tokens):
    act = f64(sd[p + "act"])
    return xielu(h @ f64(sd[p + "up"]).T, act[0], act[1]) @ f64(sd[p + "down"]).T


def table_moe_ff(h, sd, p, mlp, tokens):
    top = int(mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens.tolist()):
        for e in sd[p + "table"][tok].tolist():
            up = silu(f64(sd[f"{p}e{e}.gate"]) @ h[t]) * (f64(sd[f"{p}e{e}.up"]) @ h[t])
            out[t] += f64(sd[f"{p}e{e}.down"]) @ up / top
    return out


FF = {"dense": dense_ff, "moe": table_moe_ff}


def forward(cfg, sd, tokens):
    """tokens: list of ids of one sequence -> (logits [T, vocab], residual streams after every layer [layers, T, width])."""
    eps = float(cfg["norm"]["eps"])
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    x = f64(sd["embed"])[tokens] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    streams = []
    for i, ly in enumerate(cfg["layers"]):
        p, mlp = f"l{i}.", ly.get("mlp")
        h = layer_norm(x, sd[p + "norm1"], eps)
        y = MIXERS[ly["type"]](h, sd, p + "mix.", ly["mixer"], eps)
        if mlp is not None:
            y = y + FF[mlp["kind"]](h, sd, p + "mlp.", mlp, tokens)
        x = x + y
        streams.append(x)
    return layer_norm(x, sd["final.norm"], eps) @ f64(sd["head"]).T, torch.stack(streams)


# ---- small models for the tests ----------------------------------------------------------------------------------------------------
def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def delta_layer(heads=4, kv_heads=2, dim=16, vdim=12, conv=3, rank_a=8, rank_g=16, mlp=None):
    """rank_a, rank_g are no configuration keys: the tensors' shapes give them."""
    return {"type": "channel_delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), "mlp": mlp,
            "_ranks": (rank_a, rank_g)}


def gla_layer(heads=3, dim=16, vdim=20, tau=8.0, rank=8, mlp=None):
    return {"type": "gla", "mixer": dict(heads=heads, dim=dim, vdim=vdim, tau=tau), "mlp": mlp, "_ranks": (rank, 0)}


def attention_layer(heads=4, kv_heads=2, dim=16, scale=0.3, rot=(10000.0, 8), chunk=11, mlp=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale)
    if rot:
        m["rot"] = {"base": rot[0], "dims": rot[1]}
    if chunk:
        m["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def small_config(layers, width=64, vocab=80, scale=2.5, eps=1e-5):
    return {"architecture": "Sabezen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}


def config_json(cfg):
    """The configuration as a checkpoint's config.json holds it."""
    return {**cfg, "layers": [{k: v for k, v in ly.items() if not k.startswith("_")} for ly in cfg["layers"]]}


def param_shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for i, ly in enumerate(cfg["layers"]):
        p, m, t, mlp = f"l{i}.", ly["mixer"], ly["type"], ly.get("mlp")
        H, d, e = m["heads"], m["dim"], m["vdim"]
        s.update({p + "norm1": (W,), p + "mix.o": (W, H * e)})
        if t == "attention":
            s.update({p + "mix.q": (H * d, W), p + "mix.k": (m["kv_heads"] * d, W), p + "mix.talk": (H, H)})
        elif t == "channel_delta":
            G, taps, (ra, rg) = m["kv_heads"], m["conv"], ly["_ranks"]
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
                s.update({f"{p}mix.{n}": (rows, W), f"{p}mix.{n}.conv": (rows, taps)})
            s.update({p + "mix.b": (H, W), p + "mix.A_log": (H,), p + "mix.norm": (e,), p + "mix.a1": (ra, W), p + "mix.a2": (H * d, ra),
                      p + "mix.dt_bias": (H * d,), p + "mix.g1": (rg, W), p + "mix.g2": (H * e, rg)})
        else:
            ra = ly["_ranks"][0]
            s.update({p + "mix.q": (H * d, W), p + "mix.k": (H * d, W), p + "mix.v": (H * e, W), p + "mix.g": (H * e, W), p + "mix.norm": (e,),
                      p + "mix.a1": (ra, W), p + "mix.a2": (H * d, ra), p + "mix.a2.b": (H * d,)})
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            s.update({p + "mlp.up": (mlp["ff"], W), p + "mlp.down": (W, mlp["ff"]), p + "mlp.act": (2,)})
        else:
            ff = mlp["expert"]["ff"]
            for j in range(mlp["router"]["experts"]):
                s.update({f"{p}mlp.e{j}.gate": (ff, W), f"{p}mlp.e{j}.up": (ff, W), f"{p}mlp.e{j}.down": (W, ff)})
            s[p + "mlp.table"] = (V, mlp["router"]["top"])
    return s


def random_weights(cfg, seed=0):
    """bf16 tensors under the checkpoint's names (tables int32): norm weights around 1, decays spread between slow and fast, a mixing
    matrix with weight on and off its diagonal."""
    g = torch.Generator().manual_seed(seed)
    sd = {}
    for k, shp in param_shapes(cfg).items():
        if k.endswith("mlp.table"):
            n = cfg["layers"][int(k[1:k.index(".")])]["mlp"]["router"]["experts"]
            sd[k] = torch.stack([torch.randperm(n, generator=g)[:shp[1]] for _ in range(shp[0])]).to(torch.int32)
            continue
        r = torch.randn(shp, generator=g)
        if k == "embed":
            t = r
        elif "norm" in k:
            t = 1.0 + 0.1 * r
        elif k.endswith("A_log"):
            t = -1.0 + r
        elif k.endswith("dt_bias"):
            t = r
        elif k.endswith("a2.b"):
            t = 1.0 + r
        elif k.endswith(".act"):
            t = 0.5 * r
        elif k.endswith(".conv"):
            t = 0.6 * r
        elif k.endswith(".talk"):
            t = torch.eye(shp[0]) + 0.5 * r
        else:
            t = 1.3 * r * shp[-1] ** -0.5
        sd[k] = t.to(torch.bfloat16)
    return sd
