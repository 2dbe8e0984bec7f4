"""Host-side pieces of Zasazen that need no GPU: configuration reader and registry, the order of layer runs, what every pass asks of the cache
manager, slopes, padding of the small state-space projections, and the restatement's own consistency (its mechanisms against direct
per-token definitions and closed forms)."""
import math

import pytest
import torch

import zasazen_oracle as O

EPS = 1e-5
F64 = torch.float64


def mamba(inner=24, state=6, rank=3, conv=4):
    return {"inner": inner, "state": state, "dt_rank": rank, "conv": conv}


def parallel(heads=4, kv_heads=2, dim=16, vdim=8, rh=2, rd=12, rv=10, rot=8, every=9):
    return {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 0.3, "q_temp": {"coef": 0.4, "every": every}},
            "right": {"heads": rh, "dim": rd, "vdim": rv, "decay": [1.0 - 2.0 ** -(3 + h) for h in range(rh)], "rot": {"base": 500.0, "dims": rot}}}


def small_config():
    moe = {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 6, "top": 2}, "shared": {"ff": 24}}
    return {"architecture": "Zasazen", "vocab": 50, "width": 32, "embedding": {"scale": 3.0}, "norm": {"eps": EPS},
            "loop": {"start": 1, "stop": 3, "times": 3},
            "layers": [{"type": "mamba1", "mixer": mamba(), "mlp": {"kind": "dense", "ff": 40}},
                       {"type": "parallel", "mixer": parallel(), "mlp": moe},
                       {"type": "mamba1", "mixer": mamba(conv=1), "mlp": None},
                       {"type": "parallel", "mixer": parallel(kv_heads=4), "mlp": {"kind": "dense", "ff": 20}}]}


def test_registry_and_configuration():
    from zhilight_amd import registry
    from zhilight_amd._lib import ZLError
    from zhilight_amd.zasazen import ZasazenConfig, ZasazenModel
    cfg = small_config()
    assert registry.model_class(cfg) is ZasazenModel and "zasazen" in registry.registered()
    c = ZasazenConfig.from_dict(cfg)
    assert (c.vocab, c.width, c.embedding_scale, c.eps, c.loop) == (50, 32, 3.0, EPS, (1, 3, 3)) and c.layers[2].mlp is None
    for breakage in (lambda d: d["layers"][0].update(type="something else"),
                     lambda d: d["layers"][1]["mlp"].update(kind="sparse"),
                     lambda d: d.pop("norm"),
                     lambda d: d.pop("embedding"),
                     lambda d: d["loop"].update(stop=9),
                     lambda d: d["loop"].update(start=3),
                     lambda d: d["loop"].update(times=0),
                     lambda d: d.pop("vocab")):
        bad = small_config()
        breakage(bad)
        with pytest.raises(ZLError):
            ZasazenConfig.from_dict(bad)


def test_order_of_layer_runs():
    from zhilight_amd.zasazen import ZasazenConfig
    cfg = small_config()
    c = ZasazenConfig.from_dict(cfg)
    assert c.runs() == [(0, 0), (1, 0), (2, 0), (1, 1), (2, 1), (1, 2), (2, 2), (3, 0)]
    assert [c.passes(i) for i in range(4)] == [1, 3, 3, 1]
    assert [i for i, _ in c.runs()] == [i for i, _ in O.runs(cfg)]
    cfg["loop"] = {"start": 0, "stop": 4, "times": 1}
    assert ZasazenConfig.from_dict(cfg).runs() == [(i, 0) for i in range(4)]
    del cfg["loop"]
    c = ZasazenConfig.from_dict(cfg)
    assert c.runs() == [(i, 0) for i in range(4)] and c.loop is None and c.passes(1) == 1


def test_model_layout_and_a_cache_per_pass():
    """built on the CPU: which mixers and feed-forwards exist, with which constants; weights are shared by the passes, caches are not"""
    from zhilight_amd.cache import CacheManager
    from zhilight_amd.mixers import Mamba1Mixer, ParallelMixers, PlainFF, RoutedExpertsFF
    from zhilight_amd.zasazen import ZasazenModel
    cfg = small_config()
    model = ZasazenModel.from_config(cfg, dtype="float32", device="cpu")
    assert [type(l.mixer) for l in model.layers] == [Mamba1Mixer, ParallelMixers, Mamba1Mixer, ParallelMixers]
    assert [type(l.ff) for l in model.layers] == [PlainFF, RoutedExpertsFF, type(None), PlainFF]
    left, right, ff = model.layers[1].mixer.left, model.layers[1].mixer.right, model.layers[1].ff
    assert left.whole_norm and not left.qk_norm and left.has_bias and left.slope_bias and left.q_temp == (0.4, 9) and left.rot_dims == 0 and left.window == 0
    assert right.act is None and right.gate_act == "silu" and right.norm_groups == 2 and not right.has_norm_weight and right.rot_dims == 8
    assert abs(right.key_scale - 12 ** -0.5) < 1e-15
    assert (ff.score, ff.has_router_bias, ff.has_correction, ff.shared_ff, ff.shared_gate, ff.top) == ("chosen", True, False, 24, True, 2)
    layer = model.layers[1]
    layer.mixer.w_in = torch.zeros(3)
    for l in model.layers:
        l._replicate()
    assert len(layer.passes) == 3 and all(p.w_in is layer.mixer.w_in for p in layer.passes) and layer.passes[1].left is not layer.mixer.left
    cache = model.bind_cache(CacheManager(256, 3, "cpu"))
    assert sorted(cache.planes) == sorted([f"l1.mix{t}.left.{n}" for t in ("", ".pass1", ".pass2") for n in "kv"] + ["l3.mix.left.k", "l3.mix.left.v"])
    assert sorted(cache.states) == sorted(["l0.mix.conv", "l0.mix.ssm", "l3.mix.right.S"] + [f"l1.mix{t}.right.S" for t in ("", ".pass1", ".pass2")] +
                                          [f"l2.mix{t}.ssm" for t in ("", ".pass1", ".pass2")])       # (one tap: no convolution tail)
    assert cache.states["l0.mix.ssm"].shape == (3, 6, 24) and cache.states["l0.mix.conv"].shape == (3, 3, 24)
    assert cache.states["l1.mix.right.S"].shape == (3, 2, 12, 10) and cache.planes["l3.mix.left.v"].shape == (4, 64, 4 * 8)
    a, b = layer.passes[0], layer.passes[2]
    assert a.left.k_cache is not b.left.k_cache and a.right.state is not b.right.state


def test_joint_input_projections(monkeypatch):
    """left and right rows of the parallel mixers are one matrix with the left one's biases; the shared expert's rows follow the router's; the
    small state-space projection is padded to rows of eight"""
    from zhilight_amd import mixers, seqops
    from zhilight_amd.zasazen import FF_BUILDERS, MIXER_BUILDERS
    monkeypatch.setattr(seqops, "_cuda", lambda *ts: None)                       # (nothing is launched: the weights' layout on the CPU)
    cfg = small_config()
    sd = O.random_weights(cfg, 3)
    get = lambda n: sd[n]
    p = MIXER_BUILDERS["parallel"]("m", 32, cfg["layers"][1]["mixer"], EPS).load(get, "l1.mix.", torch.float32, "cpu")
    rows = 4 * 16 + 2 * 16 + 2 * 8
    assert p.col == rows and p.w_in.shape == (rows + 2 * (2 * 12 + 2 * 10), 32)
    assert torch.equal(p.w_in[64:96], sd["l1.mix.left.k"].float()) and torch.equal(p.w_in[rows + 24:rows + 48], sd["l1.mix.right.k"].float())
    assert torch.equal(p.in_bias[64:96], sd["l1.mix.left.k.b"].float()) and not p.in_bias[rows:].any()
    assert p.left.prep.x_heads == 4 and p.left.prep.x_col0 == rows and p.left.prep.x_rot == 8 and p.left.prep.temp_every == 9
    f = FF_BUILDERS["moe"](32, cfg["layers"][1]["mlp"]).load(get, "l1.mlp.", torch.float32, "cpu")
    assert f.shared_col == 6 and f.w_router.shape == (6 + 48 + 1, 32) and torch.equal(f.w_router[54:], sd["l1.mlp.shared.sg"].float())
    m = MIXER_BUILDERS["mamba1"]("m", 32, cfg["layers"][0]["mixer"], EPS).load(get, "l0.mix.", torch.float32, "cpu")
    assert m.low == 8 and m.w_x.shape == (8 + 12, 24) and not m.w_x[3:8].any() and torch.equal(m.w_x[8:], sd["l0.mix.x"].float()[3:])
    assert m.w_dt.shape == (24, 8) and not m.w_dt[:, 3:].any() and m.a2.shape == (6, 24)
    assert torch.allclose(torch.exp2(m.a2.double() * 0.7), torch.exp(-torch.exp(sd["l0.mix.A_log"].double()) * 0.7).t(), rtol=1e-6)
    s = mixers.linear_slopes(6, "cpu")
    assert s.tolist() == [torch.tensor(2.0 ** (-8.0 * (h + 1) / 6), dtype=torch.float32).item() for h in range(6)] == \
        [torch.tensor(v, dtype=torch.float32).item() for v in O.slopes(6)]


def test_selective_scan_against_its_closed_form():
    """one channel, one state: y_t = sum_j exp(A sum_{i=j+1..t} dt_i) dt_j x_j B_j C_t + D x_t"""
    g = torch.Generator().manual_seed(1)
    T = 12
    x, dt = torch.randn(T, 1, generator=g, dtype=F64), torch.rand(T, 1, generator=g, dtype=F64)
    B, C = torch.randn(T, 1, generator=g, dtype=F64), torch.randn(T, 1, generator=g, dtype=F64)
    A, D = torch.tensor([[-0.8]], dtype=F64), torch.tensor([0.3], dtype=F64)
    y = O.selective_scan(x, dt, A, B, C, D)
    for t in range(T):
        ref = 0.3 * float(x[t]) + sum(math.exp(-0.8 * float(dt[j + 1:t + 1].sum())) * float(dt[j] * x[j] * B[j]) for j in range(t + 1)) * float(C[t])
        assert abs(float(y[t]) - ref) < 1e-12


def test_convolution_and_softplus():
    u = torch.arange(5, dtype=F64)[:, None] + 1.0
    out = O.causal_conv(u, torch.tensor([[100.0, 10.0, 1.0]], dtype=F64), torch.tensor([0.5], dtype=F64))
    assert out[:, 0].tolist() == [1.5, 12.5, 123.5, 234.5, 345.5]
    z = torch.tensor([-40.0, -1.0, 0.0, 5.0, 29.0, 31.0, 500.0], dtype=F64)
    assert torch.allclose(O.softplus(z), torch.nn.functional.softplus(z, threshold=1000.0)[:7].nan_to_num(posinf=500.0), rtol=1e-12)


def test_retention_against_its_quadratic_form():
    """o_t = sum_j decay^(t - j) (q_t . k_j) v_j"""
    g = torch.Generator().manual_seed(2)
    T, H, d, e = 9, 2, 4, 3
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=F64) for n in (d, d, e))
    dec = [0.5, 0.97]
    o = O.retention(q, k, v, dec)
    for h in range(H):
        w = torch.tril(torch.tensor([[dec[h] ** max(t - j, 0) for j in range(T)] for t in range(T)], dtype=F64))
        assert torch.allclose(o[:, h], ((q[:, h] @ k[:, h].T) * w) @ v[:, h], atol=1e-12)


def test_query_temperature_steps_and_slopes():
    t = O.query_temperature(30, 0.5, 10)
    assert [float(t[p]) for p in (0, 8)] == [1.0, 1.0] and abs(float(t[9]) - (1.0 + 0.5 * math.log(2.0))) < 1e-15
    assert float(t[9]) == float(t[18]) and abs(float(t[29]) - (1.0 + 0.5 * math.log(4.0))) < 1e-15
    assert O.slopes(8) == [2.0 ** -(h + 1) for h in range(8)] and O.slopes(2) == [2.0 ** -4, 2.0 ** -8]
    # equal scores: weights fall by e^-slope per step back
    z = torch.zeros(3, 1, 2, dtype=F64)
    v = torch.eye(3, dtype=F64).reshape(3, 1, 3)
    w = O.sloped_attention(z, z, v, 1.0)[2, 0]
    assert abs(float(w[1] / w[2]) - math.exp(-O.slopes(1)[0])) < 1e-15 and abs(float(w.sum()) - 1.0) < 1e-15


def test_router_weights_are_a_softmax_over_the_chosen():
    g = torch.Generator().manual_seed(6)
    sd = {"router": torch.randn(6, 8, generator=g, dtype=F64), "router.b": torch.randn(6, generator=g, dtype=F64)}
    h = torch.randn(30, 8, generator=g, dtype=F64)
    margins = []
    ids, wts = O.route(h, sd, "", 3, margins)
    for t in range(30):
        z = sd["router"] @ h[t] + sd["router.b"]
        best = sorted(range(6), key=lambda i: -z[i])[:3]
        assert ids[t].tolist() == best
        assert torch.allclose(wts[t], torch.exp(z[best]) / torch.exp(z[best]).sum())
    assert margins[0] > 0


def test_loop_entry():
    """W_in = [I | 0] without step vectors is a plain stack of the unrolled layers; W_in = [0 | I] starts every pass from the embedding"""
    cfg = small_config()
    sd = O.random_weights(cfg, 4)
    W = cfg["width"]
    eye, zero = torch.eye(W), torch.zeros(W, W)
    toks = [3, 9, 1, 40, 7, 11]
    sd["loop.step"] = torch.zeros_like(sd["loop.step"])
    sd["loop.in"] = torch.cat([eye, zero], 1)
    layers = []
    O.model(toks, sd, cfg, layers)
    x = sd["embed"].double()[toks] * 3.0
    for i, _ in O.runs(cfg):
        x = O.layer(x, sd, i, cfg["layers"][i], EPS)
    assert len(layers) == 8 and torch.allclose(layers[-1], x, atol=1e-10)
    sd["loop.in"] = torch.cat([zero, eye], 1)
    layers = []
    O.model(toks, sd, cfg, layers)
    assert torch.allclose(layers[1], layers[3], atol=1e-12) and torch.allclose(layers[2], layers[6], atol=1e-12)
    assert not torch.allclose(layers[0], layers[2])


def test_model_restatement_is_causal():
    cfg = small_config()
    sd = O.random_weights(cfg, 7)
    toks = torch.randint(0, 50, (40,), generator=torch.Generator().manual_seed(8)).tolist()
    layers = []
    full = O.model(toks, sd, cfg, layers)
    assert torch.allclose(full[:25], O.model(toks[:25], sd, cfg), atol=1e-9) and len(layers) == 8 and layers[0].shape == (40, 32)
    fixed = O.random_weights(cfg, 7, fixed_choice=True)
    margins = []
    O.model(toks, fixed, cfg, None, margins)
    assert min(margins) > 0.1
