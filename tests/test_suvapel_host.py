"""Host-side pieces of Suvapel that need no GPU: configuration reader and registry, what the layers ask of the cache manager, the joint
matrices, and the restatement's own consistency (its mechanisms against direct definitions and closed forms)."""
import math

import pytest
import torch

import suvapel_oracle as O

EPS = 1e-5
F64 = torch.float64


def delta(heads=4, kv_heads=2, dim=12, vdim=10, conv=4, low=6):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "low": low}


def parallel(heads=4, kv_heads=2, dim=16, vdim=8, conv=3, size=9, keep=2, dims=8):
    return {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": 0.3, "mask": {"size": size, "keep_first": keep},
                     "rot": {"base": 500.0, "dims": dims, "scaling": {"factor": 3.0, "original": 64, "fast": 8.0, "slow": 1.0}}},
            "right": delta(heads=2, kv_heads=1, dim=6, vdim=14), "left_scale": 0.7, "right_scale": 0.5}


def small_config():
    return {"architecture": "Suvapel", "vocab": 50, "width": 32, "norm": {"eps": EPS}, "residual_mult": 0.4, "token_side": {"dim": 7},
            "layers": [{"type": "delta", "mixer": delta(), "mlp": {"kind": "dense", "ff": 40}},
                       {"type": "parallel", "mixer": parallel(), "mlp": {"kind": "dense", "ff": 24}},
                       {"type": "delta", "mixer": delta(heads=3, kv_heads=3, conv=1), "mlp": None}]}


def test_registry_and_configuration():
    from zhilight_amd import registry
    from zhilight_amd._lib import ZLError
    from zhilight_amd.suvapel import SuvapelConfig, SuvapelModel
    cfg = small_config()
    assert registry.model_class(cfg) is SuvapelModel and "suvapel" in registry.registered()
    c = SuvapelConfig.from_dict(cfg)
    assert (c.vocab, c.width, c.eps, c.residual_mult, c.side_dim) == (50, 32, EPS, 0.4, 7) and c.layers[2].mlp is None
    for breakage in (lambda d: d["layers"][0].update(type="something else"),
                     lambda d: d["layers"][1]["mlp"].update(kind="sparse"),
                     lambda d: d.pop("norm"),
                     lambda d: d["token_side"].pop("dim"),
                     lambda d: d.pop("vocab")):
        bad = small_config()
        breakage(bad)
        with pytest.raises(ZLError):
            SuvapelConfig.from_dict(bad)
    with pytest.raises(ZLError):
        SuvapelModel.from_config(cfg, dtype="float16", device="cpu")


def test_model_layout_and_cache():
    from zhilight_amd.cache import CacheManager
    from zhilight_amd.mixers import GatedDeltaRule, GatedFF, WindowAttention
    from zhilight_amd.suvapel import SuvapelModel
    model = SuvapelModel.from_config(small_config(), dtype="float32", device="cpu")
    assert [[type(p) for p in l.sub.parts] for l in model.layers] == [[GatedDeltaRule, GatedFF], [WindowAttention, GatedDeltaRule, GatedFF], [GatedDeltaRule]]
    assert [l.sub.scales for l in model.layers] == [[1.0, 1.0], [0.7, 0.5, 1.0], [1.0]]
    left, right, ff = model.layers[1].sub.parts
    assert left.head_gate and left.has_gate and left.window == 9 and left.keep_first == 2 and left.taps == 3 and left.rot_dims == 8 and not left.qk_norm
    assert right.per_channel and right.lowrank_gate and right.gate_act == "sigmoid" and ff.act == "silu" and ff.has_bias
    d = model.layers[0].sub.parts[0]
    assert not d.per_channel and not d.lowrank_gate and d.gate_act == "silu" and [l.side.column for l in model.layers] == [0, 7, 14]
    cache = model.bind_cache(CacheManager(256, 3, "cpu"))
    assert sorted(cache.planes) == ["l1.mix.left.k", "l1.mix.left.v"]
    assert sorted(cache.states) == ["l0.mix.S", "l0.mix.conv", "l1.mix.left.conv", "l1.mix.right.S", "l1.mix.right.conv", "l2.mix.S"]     # (one tap: no tail)
    assert cache.states["l0.mix.S"].shape == (3, 4, 10, 12) and cache.states["l1.mix.right.conv"].shape == (3, 3, 2 * 6 + 2 * 14)
    assert cache.states["l1.mix.left.conv"].shape == (3, 2, 4 * 16 + 2 * 16 + 2 * 8)


def test_joint_matrices(monkeypatch):
    """everything that reads h is one matrix: low-rank rows first (padded to whole 16-byte pieces), then the parts in order, biases beside
    zeros; everything that joins the residual is one matrix of output projections side by side; low-rank second steps are block-diagonal"""
    from zhilight_amd import seqops
    from zhilight_amd.suvapel import SuvapelModel
    monkeypatch.setattr(seqops, "_cuda", lambda *ts: None)                       # (nothing is launched: the weights' layout on the CPU)
    cfg = small_config()
    sd = O.random_weights(cfg, 3)
    model = SuvapelModel.from_config(cfg, dtype="float32", device="cpu").load_weights(sd)
    j, p = model.layers[1].sub, "l1.mix."
    n_left, n_right = 4 * 16 + 2 * 16 + 2 * 8 + 4, 2 * 6 + 2 * 14 + 2
    assert j.n_lead == 16 and j.col0 == [16, 16 + n_left, 16 + n_left + n_right] and j.w_in.shape == (16 + n_left + n_right + 48, 32)
    assert torch.equal(j.w_in[:6], sd[p + "right.a1"].float()) and torch.equal(j.w_in[6:12], sd[p + "right.g1"].float()) and not j.w_in[12:16].any()
    assert torch.equal(j.w_in[16 + n_left - 4:16 + n_left], sd[p + "left.g"].float()) and torch.equal(j.w_in[j.col0[1] + 6:j.col0[1] + 12], sd[p + "right.k"].float())
    assert torch.equal(j.in_bias[j.col0[2]:], torch.cat([sd["l1.mlp.gate.b"], sd["l1.mlp.up.b"]]).float()) and not j.in_bias[:j.col0[2]].any()
    assert j.out_at == [(0, 32), (32, 60), (60, 84)] and torch.equal(j.out_bias, sd["l1.mlp.down.b"].float())
    assert torch.equal(j.w_out, torch.cat([sd[p + "left.o"], sd[p + "right.o"], sd["l1.mlp.down"]], 1).float())
    low = j.parts[1].w_low
    assert low.shape == (2 * 6 + 2 * 14, 16) and torch.equal(low[:12, :6], sd[p + "right.a2"].float()) and torch.equal(low[12:, 6:12], sd[p + "right.g2"].float())
    assert not low[:12, 6:].any() and not low[12:, :6].any() and not low[:, 12:].any()
    j = model.layers[0].sub
    assert j.n_lead == 0 and j.col0[0] == 0 and j.w_in.shape[0] == 4 * 12 + 4 * 10 + 4 + 4 + 4 * 10 + 80
    assert torch.allclose(j.parts[0].rate, torch.exp(sd["l0.mix.A_log"].float())) and j.parts[0].norm_w.shape == (40,)
    assert model.layers[2].sub.in_bias is None and model.layers[2].sub.out_bias is None
    # a part with an output scale passes it on to its bias
    from zhilight_amd.mixers import GatedFF, JoinedSublayers
    s = JoinedSublayers(32, [("mlp.", GatedFF(32, 24, act="silu", bias=True), 1.0)]).load(lambda n: sd["l1." + n], "", torch.float32, "cpu")
    assert torch.equal(s.out_bias, sd["l1.mlp.down.b"].float())


def test_scaled_frequencies_and_gain():
    from zhilight_amd.mixers import scaled_frequencies
    from zhilight_amd.suvapel import SuvapelModel
    rot = small_config()["layers"][1]["mixer"]["left"]["rot"]
    f, gain = O.frequencies(rot)
    got, g2 = scaled_frequencies(8, 500.0, rot["scaling"])
    assert torch.allclose(got.double(), f, rtol=1e-6) and abs(gain - g2) < 1e-15 and abs(gain - (0.1 * math.log(3.0) + 1.0)) < 1e-15
    assert not torch.allclose(f, O.frequencies({"dims": 8, "base": 500.0})[0])
    left = SuvapelModel.from_config(small_config(), device="cpu").layers[1].sub.parts[0]
    left._tables("cpu")
    assert left.rot_gain == g2 and torch.equal(left.qk_freq, got) and left.prep.rot_gain == pytest.approx(gain)


def test_visibility_of_window_and_kept_first_keys():
    m = O.visible(12, 4, 2)
    assert m[11].nonzero().flatten().tolist() == [0, 1, 8, 9, 10, 11] and m[3].nonzero().flatten().tolist() == [0, 1, 2, 3]
    assert m[4].nonzero().flatten().tolist() == [0, 1, 2, 3, 4] and m[0].nonzero().flatten().tolist() == [0]
    assert O.visible(5, 0, 0).sum() == 15


def test_delta_rule_stores_one_value_per_key():
    """orthonormal keys, beta 1, no decay: reading a key gives its latest value back, whatever was written under the others"""
    T, d, e = 9, 3, 4
    g = torch.Generator().manual_seed(1)
    keys = torch.eye(d, dtype=F64)[torch.tensor([0, 1, 2, 1, 0, 2, 2, 0, 1])]
    v = torch.randn(T, 1, e, generator=g, dtype=F64)
    one = torch.ones(T, 1, dtype=F64)
    o = O.delta_recurrence(keys[:, None], keys[:, None], v, one, torch.ones(T, 1, d, dtype=F64))
    assert torch.allclose(o, v, atol=1e-12)                                      # (the read-out sees the token's own write)
    o = O.delta_recurrence(torch.eye(d, dtype=F64)[torch.zeros(T, dtype=torch.long)][:, None], keys[:, None], v, one, torch.ones(T, 1, d, dtype=F64))
    assert torch.allclose(o[3], v[0], atol=1e-12) and torch.allclose(o[6], v[4], atol=1e-12) and torch.allclose(o[8], v[7], atol=1e-12)
    # a decay per key channel acts on that key's row only
    dec = torch.ones(T, 1, d, dtype=F64)
    dec[:, :, 0] = 0.5
    o = O.delta_recurrence(torch.eye(d, dtype=F64)[torch.zeros(T, dtype=torch.long)][:, None], keys[:, None], v, one, dec)
    assert torch.allclose(o[3], v[0] * 0.125, atol=1e-12)


def test_delta_rule_against_its_transition_matrices():
    """S_t = (I - beta k k^T) diag(g) S_{t-1} + beta k v^T"""
    g = torch.Generator().manual_seed(2)
    T, H, d, e = 7, 2, 4, 3
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=F64) for n in (d, d, e))
    beta, dec = torch.rand(T, H, generator=g, dtype=F64), torch.rand(T, H, d, generator=g, dtype=F64)
    o = O.delta_recurrence(q, k, v, beta, dec)
    for h in range(H):
        S = torch.zeros(d, e, dtype=F64)
        for t in range(T):
            S = (torch.eye(d, dtype=F64) - beta[t, h] * torch.outer(k[t, h], k[t, h])) @ torch.diag(dec[t, h]) @ S + beta[t, h] * torch.outer(k[t, h], v[t, h])
            assert torch.allclose(o[t, h], S.T @ q[t, h], atol=1e-12)


def test_convolution_softplus_and_norms():
    u = torch.arange(5, dtype=F64)[:, None] + 1.0
    assert O.causal_conv(u, torch.tensor([[100.0, 10.0, 1.0]], dtype=F64))[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0, 345.0]
    z = torch.tensor([-40.0, -1.0, 0.0, 5.0, 29.0, 31.0, 500.0], dtype=F64)
    assert torch.allclose(O.softplus(z), torch.nn.functional.softplus(z, threshold=1000.0).nan_to_num(posinf=500.0), rtol=1e-12)
    x = torch.tensor([[3.0, -4.0]], dtype=F64)
    assert torch.allclose(O.unit_vector(x), x / 5.0, atol=1e-7) and float(O.unit_vector(torch.zeros(1, 2, dtype=F64)).abs().max()) == 0.0
    assert torch.allclose(O.tanh_norm(x, 0.5, torch.tensor([2.0, 1.0], dtype=F64), torch.tensor([0.1, 0.2], dtype=F64)),
                          torch.tensor([[2.0 * math.tanh(1.5) + 0.1, math.tanh(-2.0) + 0.2]], dtype=F64))


def test_model_restatement_is_causal_and_reads_the_side_embedding():
    cfg = small_config()
    sd = O.random_weights(cfg, 7)
    toks = torch.randint(0, 50, (40,), generator=torch.Generator().manual_seed(8)).tolist()
    layers = []
    full = O.forward(toks, sd, cfg, layers)
    assert torch.allclose(full[:25], O.forward(toks[:25], sd, cfg), atol=1e-9) and len(layers) == 3 and layers[0].shape == (40, 32)
    other = dict(sd)
    other["side.embed"] = sd["side.embed"].clone()
    other["side.embed"][toks[30], 7:14] += 1.0                                   # (the second layer's columns of one token)
    again = []
    O.forward(toks, other, cfg, again)
    first = min(i for i, t in enumerate(toks) if t == toks[30])
    assert torch.equal(layers[0], again[0]) and torch.equal(layers[1][:first], again[1][:first]) and not torch.allclose(layers[1][first], again[1][first])
