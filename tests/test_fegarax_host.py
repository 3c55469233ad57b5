"""Fegarax without a GPU: configuration, registry and tensor shapes of the package, and the float64 restatement held against independent
closed forms (what a position sees, the softmax's extra one, the scaled rotation, the streams as one matrix, mixed values, the experts)."""
import json
import math

import pytest
import torch

from ming_univision_amd.configuration import FegaraxConfig, config_from_pretrained, fegarax_param_shapes
from tests import fegarax_oracle as O

F64 = torch.float64


def small():
    return O.small_config([O.attention_layer(mlp=O.moe(5, 2, 16)), O.attention_layer(rot=None, chunk=None, v_mix=False),
                           O.attention_layer(heads=6, kv_heads=3, vdim=8, scaling=None, mlp=O.moe(3, 1, 24))])


def test_config_registry_and_shapes(tmp_path):
    cfg = small()
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    name, c = config_from_pretrained(str(tmp_path))
    assert name == "fegarax" and isinstance(c, FegaraxConfig) and c.embed_scale == 2.5 and c.eps == 1e-5 and c.streams == 3
    want = {k: tuple(v) for k, v in O.param_shapes(cfg).items()}
    assert {k: tuple(v) for k, v in fegarax_param_shapes(c).items()} == want
    assert "l1.norm2" not in want and "l1.hc2.in" not in want and "l1.mix.vmix" not in want and want["l2.hc2.mix"] == (3, 3)
    assert FegaraxConfig.from_dict({**cfg, "embedding": None}).embed_scale == 1.0
    assert FegaraxConfig.from_dict(c.to_dict()).to_dict() == c.to_dict()
    assert not any(".hc" in k for k in fegarax_param_shapes(FegaraxConfig.from_dict({k: v for k, v in cfg.items() if k != "streams"})))


@pytest.mark.parametrize("edit, text", [
    (lambda c: c["layers"][0].update(type="conv"), "unknown mixer"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "do not divide"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "at most"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "positive"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"].pop("vdim"), "lacks"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=9), "do not mix"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "top <= experts"),
    (lambda c: c["layers"][0].update(mlp={"kind": "other"}), "feed-forward"),
    (lambda c: c.update(streams=0), "streams"),
])
def test_config_validation(edit, text):
    cfg = small()
    edit(cfg)
    with pytest.raises(ValueError, match=text):
        FegaraxConfig.from_dict(cfg)


def test_what_a_position_sees():
    m = O.visible(11, chunk=4)
    for i in range(11):
        assert [j for j in range(11) if m[i, j]] == [j for j in range(11) if j <= i and j // 4 == i // 4]
    assert bool((O.visible(5) == torch.ones(5, 5, dtype=torch.bool).tril()).all())
    assert bool((O.visible(5, chunk=1) == torch.eye(5, dtype=torch.bool)).all())


def test_the_softmax_denominator_has_one_added():
    g = torch.Generator().manual_seed(0)
    T, d, e = 6, 4, 3
    q, k, v = torch.randn(T, 2, d, generator=g, dtype=F64), torch.randn(T, 1, d, generator=g, dtype=F64), torch.randn(T, 1, e, generator=g, dtype=F64)
    out = O.sink_softmax_attention(q, k, v, 0.7, O.visible(T))
    for i in range(T):
        for h in range(2):
            w = torch.exp((k[:i + 1, 0] @ q[i, h]) * 0.7)
            assert torch.allclose(out[i, h], (w / (1 + w.sum())) @ v[:i + 1, 0])
    one = torch.ones(1, 1, d, dtype=F64)
    low = O.sink_softmax_attention(-one, one, v[:1], 5.0, O.visible(1))          # a very negative score: almost nothing is returned
    assert torch.allclose(low[0, 0], v[0, 0] * math.exp(-20) / (1 + math.exp(-20)))
    assert torch.allclose(O.sink_softmax_attention(-one, one, v[:1], 5.0, O.visible(1), sink=False)[0, 0], v[0, 0])
    high = O.sink_softmax_attention(200 * one, one, v[:1], 5.0, O.visible(1))    # a very large one does not overflow
    assert torch.allclose(high[0, 0], v[0, 0])


def test_rotation_turns_half_pairs_with_scaled_frequencies():
    f, mag = O.rotary_frequencies({"base": 10000.0, "dims": 16, "scaling": {"factor": 8.0, "original": 512, "fast": 16.0, "slow": 1.0}})
    plain, one = O.rotary_frequencies({"base": 10000.0, "dims": 16})
    assert one == 1.0 and abs(mag - (0.1 * math.log(8.0) + 1)) < 1e-12
    at = [16 * math.log(512 / (2 * math.pi * t)) / (2 * math.log(10000.0)) for t in (16.0, 1.0)]
    lo, hi = math.floor(at[0]), math.ceil(at[1])
    assert 0 <= lo < hi < 8
    for i in range(8):
        r = min(max((i - lo) / (hi - lo), 0), 1)
        assert abs(float(f[i]) - float(plain[i]) * (r / 8 + 1 - r)) < 1e-15
    assert torch.allclose(f[:lo + 1], plain[:lo + 1]) and torch.allclose(f[hi:], plain[hi:] / 8)
    g = torch.Generator().manual_seed(1)
    x, fr = torch.randn(5, 2, 10, generator=g, dtype=F64), torch.tensor([1.0, 0.3, 0.01], dtype=F64)
    y = O.rotate_halves(x, fr, 1.3, pos0=7)
    assert bool((y[..., 6:] == x[..., 6:]).all())
    for t in range(5):
        for i in range(3):
            c, s = 1.3 * math.cos((7 + t) * float(fr[i])), 1.3 * math.sin((7 + t) * float(fr[i]))
            assert torch.allclose(y[t, :, i], x[t, :, i] * c - x[t, :, i + 3] * s) and torch.allclose(y[t, :, i + 3], x[t, :, i + 3] * c + x[t, :, i] * s)


def test_package_rotary_table_agrees():
    """The table the decoder uploads against the oracle's, the ramp inside, clamped at both ends and degenerate."""
    from ming_univision_amd.sakinex import rotary_table
    for base, dims, scaling in ((1e4, 16, (8.0, 512, 16.0, 1.0)), (5e4, 32, (4.0, 4096, 32.0, 1.0)), (500.0, 6, (2.0, 40, 64.0, 0.01)), (100.0, 2, (3.0, 1000, 1.0, 1.0)),
                                (1e6, 64, None)):
        rot = {"base": base, "dims": dims}
        if scaling:
            rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
        f, mag = O.rotary_frequencies(rot)
        got, m = rotary_table(rot, "cpu")
        assert torch.allclose(got.double(), f, rtol=1e-6, atol=0) and abs(m - mag) < 1e-6


def test_streams_are_one_matrix():
    g = torch.Generator().manual_seed(2)
    X, y = torch.randn(3, 5, 7, generator=g, dtype=F64), torch.randn(5, 7, generator=g, dtype=F64)
    mix, w_in, w_out = torch.randn(3, 3, generator=g, dtype=F64), torch.randn(3, generator=g, dtype=F64), torch.randn(3, generator=g, dtype=F64)
    assert torch.allclose(O.streams_read(X, w_in), torch.einsum("s,stc->tc", w_in, X))
    assert torch.allclose(O.streams_write(X, y, mix, w_out), torch.einsum("st,snc->tnc", mix, X) + w_out[:, None, None] * y)


def test_experts_are_fed_with_score_times_input():
    """One expert of two chosen by hand: the score multiplies the expert's input (a silu-gated product is no homogeneous function of it),
    and the scores are not renormalised."""
    g = torch.Generator().manual_seed(3)
    W, ff = 6, 4
    h = torch.randn(1, W, generator=g, dtype=F64)
    sd = {f"e{j}.{n}": torch.randn((ff, W) if n != "down" else (W, ff), generator=g) for j in range(3) for n in ("gate", "up", "down")}
    sd["router"] = torch.randn(3, W, generator=g)
    y = O.expert_mixture(h, sd, "", O.moe(3, 2, ff))
    s = torch.sigmoid(h @ sd["router"].double().T)[0]
    want = torch.zeros(1, W, dtype=F64)
    for j in s.argsort(descending=True)[:2].tolist():
        x = s[j] * h
        want += (O.silu(x @ sd[f"e{j}.gate"].double().T) * (x @ sd[f"e{j}.up"].double().T)) @ sd[f"e{j}.down"].double().T
    assert torch.allclose(y, want)


def test_values_are_mixed_with_the_first_mixing_layer():
    """Layer 0 does not mix, layer 1 is the first that does (its own factor is unused), layer 3 reads layer 1's values."""
    mk = O.attention_layer
    cfg = O.small_config([mk(v_mix=False), mk(), mk(v_mix=False), mk()], width=24, vocab=20)
    sd = O.random_weights(cfg, 1)
    t = [3, 1, 4, 1, 5, 9]
    base = O.forward(cfg, sd, t)[0]
    for layer, same in ((1, True), (3, False)):
        sd2 = {**sd, f"l{layer}.mix.vmix": torch.tensor(0.9)}
        assert torch.allclose(O.forward(cfg, sd2, t)[0], base) == same
    h, own = torch.randn(4, 24, dtype=F64), None
    m = cfg["layers"][3]["mixer"]
    full = {**sd, "l3.mix.vmix": torch.tensor(1.0)}                    # lambda = 1: the layer's own values do not count
    vf = torch.randn(4, 24, dtype=F64)
    a, own = O.attention_mixer(h, full, "l3.mix.", m, 1e-5, vf)
    b, _ = O.attention_mixer(h, {**full, "l3.mix.v": -full["l3.mix.v"]}, "l3.mix.", m, 1e-5, vf)
    assert torch.allclose(a, b) and own.shape == (4, 24)


def test_chunks_cut_the_past():
    cfg = O.small_config([O.attention_layer(chunk=4, mlp=O.moe(4, 2, 8)), O.attention_layer(chunk=4)], width=32, vocab=20)
    sd = O.random_weights(cfg, 1)
    a = [3, 1, 4, 1, 5, 9, 2, 6]
    la, _ = O.forward(cfg, sd, a)
    lb, _ = O.forward(cfg, sd, [7, 7, 7, 7] + a[4:])
    assert torch.allclose(la[4:], lb[4:]) and not torch.allclose(la[3], lb[3])
    lc, _ = O.forward(cfg, sd, a[:5] + [0, 0, 0])
    assert torch.allclose(la[:5], lc[:5])
