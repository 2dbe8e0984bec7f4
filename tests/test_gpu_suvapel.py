"""Suvapel on the GPU against the plain float64 restatement in tests/suvapel_oracle.py: every mechanism alone, then the model through the
engine's step function -- whole prompts, token-by-token decoding, portions down to two tokens, mixed batches, reused pages and slots, keys
at window edges, page borders and among the kept first ones, long decoding, odd sizes, greedy generation through the scheduler.  Small random
configurations made here; nothing is read from disk.

fp32 serving is held to rounding of fp32 sums everywhere, bf16 serving to bf16 rounding of the matrix-product inputs."""
import math

import numpy as np
import pytest
import torch

import suvapel_oracle as O

pytestmark = pytest.mark.gpu

F32_TOL, BF16_TOL = 3e-5, 4e-2
EPS = 1e-5
F64 = torch.float64
DTYPES = [torch.float32, torch.bfloat16]


def rel(got, ref):
    got, ref = got.double().cpu(), ref.double().cpu()
    return float((got - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


def rel_rows(got, ref):
    got, ref = got.double().cpu(), ref.double().cpu()
    return (got - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-30)


def tol(dtype):
    return F32_TOL if dtype == torch.float32 else BF16_TOL


def assert_close(got, ref, dtype, what=""):
    """all positions together within the tolerance, and no single position more than four times off"""
    e = rel_rows(got, ref)
    assert rel(got, ref) < tol(dtype) and float(e.max()) < 4 * tol(dtype), (what, rel(got, ref), float(e.max()), int(e.argmax()))


def bf(t):
    return t.to(torch.bfloat16).to(F64)


# ------------------------------------------------------------------------------------------------------------------------------------
# configurations
# ------------------------------------------------------------------------------------------------------------------------------------
def delta_m(heads=4, kv_heads=2, dim=24, vdim=20, conv=4, low=10):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "low": low}


def attn_m(heads=4, kv_heads=2, dim=40, vdim=32, conv=3, scale=0.2, size=37, keep=5, dims=16, base=2000.0, factor=5.0, original=128, fast=12.0, slow=1.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale, "mask": {"size": size, "keep_first": keep},
            "rot": {"base": base, "dims": dims, "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}}}


def delta_l(ff=72, **kw):
    return {"type": "delta", "mixer": delta_m(**kw), "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def parallel_l(left, right, ls=0.8, rs=0.6, ff=56):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": ls, "right_scale": rs}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def model_cfg(layers, width=96, vocab=160, mult=0.45, side=16):
    return {"architecture": "Suvapel", "vocab": vocab, "width": width, "norm": {"eps": EPS}, "residual_mult": mult, "token_side": {"dim": side}, "layers": layers}


def cfg_a():
    """both mixers, with a feed-forward and without; windows within a page and across pages"""
    return model_cfg([parallel_l(attn_m(), delta_m(heads=2, kv_heads=2, dim=16, vdim=24)), delta_l(),
                      parallel_l(attn_m(heads=8, kv_heads=2, dim=32, vdim=48, size=80, keep=3, conv=4, dims=32), delta_m(heads=4, kv_heads=1, dim=36, vdim=12, conv=2, low=5), ff=None),
                      delta_l(heads=3, kv_heads=3, dim=40, vdim=36, conv=3, ff=None)])


def cfg_odd(one=1):
    """sizes no matrix-core kernel and no 16-byte access takes, and values that a particular model may make equal or 1: one head, heads = kv
    heads, one tap, a window of one key, no kept keys, all of a head rotated, key and value sizes that differ by one, ranks of 1 and 3,
    scales and multipliers of 1, one column of side input; keys and values of `one` number (a unit vector or norm of one number is
    its sign, which rounding may flip near 0: 1 is for fp32)"""
    return model_cfg([parallel_l(attn_m(heads=3, kv_heads=3, dim=10, vdim=7, conv=1, size=1, keep=0, dims=10, factor=1.0), delta_m(heads=1, kv_heads=1, dim=5, vdim=3 * one, conv=1, low=1), 1.0, 1.0, ff=33),
                      delta_l(heads=5, kv_heads=1, dim=9, vdim=10, conv=6, ff=17), delta_l(heads=2, kv_heads=2, dim=33, vdim=one, conv=2, ff=None),
                      parallel_l(attn_m(heads=5, kv_heads=1, dim=14, vdim=9, conv=2, size=65, keep=70, dims=2, fast=3.0), delta_m(heads=6, kv_heads=3, dim=one, vdim=18, conv=5, low=3), -0.5, 2.0, ff=None)],
                     width=70, vocab=90, mult=1.0, side=1)


def make(cfg, sd, dtype, dev, max_tokens=2048, max_seqs=4, max_step_tokens=512):
    from zhilight_amd.engine import Engine
    from zhilight_amd.registry import model_class
    model = model_class(cfg).from_config(cfg, dtype=dtype, device=dev).load_weights(sd)
    return Engine(model, max_tokens=max_tokens, max_seqs=max_seqs, max_step_tokens=max_step_tokens)


def run_portions(eng, rid, tokens, portions, release=True):
    from zhilight_amd.engine import Entry
    out, at = [], 0
    for n in portions:
        out.append(eng.run_step([Entry(rid, tokens[at:at + n], list(range(n)))]))
        at += n
    assert at == len(tokens)
    if release:
        eng.release(rid)
    return torch.cat(out, dim=0)


def tokens_of(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


def new_cache(dev, max_tokens=1024, slots=3):
    from zhilight_amd.cache import CacheManager
    return CacheManager(max_tokens, slots, dev)


def batch_of(cache, portions, dev):
    """a RaggedBatch of [(sequence, tokens)] on the cache manager"""
    from zhilight_amd import seqops
    seqs = []
    for sid, n in portions:
        if sid not in cache.seqs:
            cache.admit(sid)
        pos0, slot, pages = cache.extend(sid, n)
        seqs.append((n, pos0, slot, list(pages)))
    return seqops.RaggedBatch(seqs, cache.page_size, dev)


def feed(part, cache, h, portions, dev, sid="s"):
    out, at = [], 0
    for n in portions:
        out.append(part.forward(h[at:at + n].to(dev).contiguous(), batch_of(cache, [(sid, n)], dev)))
        at += n
    assert at == h.shape[0]
    return torch.cat(out)


def delta_weights(m, W, seed, per_channel):
    layer = {"type": "delta", "mixer": m, "mlp": None}
    if per_channel:
        layer = parallel_l(attn_m(), m, ff=None)
    sd = O.random_weights(model_cfg([layer], width=W), seed)
    cut = "l0.mix.right." if per_channel else "l0.mix."
    return {k[len(cut):]: v for k, v in sd.items() if k.startswith(cut)}


def delta_mixer(m, W, sd, dtype, dev, cache, per_channel):
    from zhilight_amd.mixers import GatedDeltaRule
    how = dict(decay="channel", gate="lowrank", gate_act="sigmoid") if per_channel else {}
    mix = GatedDeltaRule("m", W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], EPS, **how).load(lambda n: sd[n], "", dtype, dev)
    mix.bind(cache, dtype)
    return mix


# ------------------------------------------------------------------------------------------------------------------------------------
# mechanisms alone
# ------------------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m,n,k", [(1, 37, 64), (2, 24, 50), (7, 40, 96), (16, 33, 72), (70, 130, 40), (300, 50, 600), (2048, 2048, 32)])
def test_product_with_a_looked_up_factor(dev, dtype, m, n, k):
    """gelu(x . w^T) times the row of a table that the token picks, columns from the middle of the table, on every product kernel"""
    from zhilight_amd import seqops
    g = torch.Generator().manual_seed(m + n)
    x, w, table = torch.randn(m, k, generator=g).to(dtype), (torch.randn(n, k, generator=g) * k ** -0.5).to(dtype), torch.randn(11, n + 9, generator=g).to(dtype)
    rows = torch.randint(0, 11, (m,), generator=g, dtype=torch.int32)
    got = seqops.gemm_nt(x.to(dev), w.to(dev), act="gelu_tanh", factor=(table.to(dev), 5, rows.to(dev)))
    ref = O.gelu_tanh(x.double() @ w.double().T) * table.double()[rows.long(), 5:5 + n]
    assert rel(got, ref) < 1e-5
    if dtype == torch.bfloat16:
        assert rel(seqops.gemm_nt(x.to(dev), w.to(dev), act="gelu_tanh", out_dtype=dtype, factor=(table.to(dev), 5, rows.to(dev))), ref) < 5e-3
    b = torch.randn(n, generator=g)                                              # the epilogue without an activation: bias, leading columns again
    y, lead = seqops.gemm_nt(x.to(dev), w.to(dev), bias=b.to(dev), lead=8)
    assert rel(y, x.double() @ w.double().T + b.double()) < 1e-5 and torch.equal(lead, y[:, :8].to(dtype))


@pytest.mark.parametrize("W", [64, 70, 300, 4096])
def test_tanh_norm_alone_and_behind_the_residual(dev, W):
    from zhilight_amd import seqops
    g = torch.Generator().manual_seed(W)
    x, y, s = (torch.randn(6, W, generator=g) for _ in range(3))
    w, b, nw = (torch.randn(W, generator=g) for _ in range(3))
    ref = x.double() + 0.3 * y.double() + 0.7 * O.unit_rms(s.double(), EPS) * nw.double()
    xd = x.to(dev)
    h, none = seqops.add_branches(xd, [(y.to(dev), None, 0.3), (s.to(dev), nw.to(dev), 0.7)], EPS, torch.float32, w.to(dev), tanh=(0.6, b.to(dev)))
    assert none is None and rel(xd, ref) < 1e-6 and rel(h, O.tanh_norm(ref, 0.6, w.double(), b.double())) < 1e-6
    rows = torch.tensor([4, 0, 4], dtype=torch.int32)
    assert rel(seqops.tanh_norm(xd, w.to(dev), b.to(dev), 0.6, torch.float32, rows=rows.to(dev)), O.tanh_norm(ref, 0.6, w.double(), b.double())[rows.long()]) < 1e-6
    h16, _ = seqops.add_branches(xd, [], EPS, torch.bfloat16, w.to(dev), tanh=(0.6, b.to(dev)))
    assert rel(xd, ref) < 1e-6 and torch.equal(h16, h.to(torch.bfloat16)) and torch.equal(seqops.tanh_norm(xd, w.to(dev), b.to(dev), 0.6, torch.bfloat16), h16)


@pytest.mark.parametrize("dim,dims", [(40, 16), (64, 64), (18, 2), (88, 40)])
def test_rotation_with_rescaled_frequencies_and_gain(dev, dim, dims):
    """queries and cached keys at positions far apart; the coordinates behind the rotated part unchanged, values untouched"""
    from zhilight_amd import seqops
    from zhilight_amd.mixers import scaled_frequencies
    H, G, e, T = 3, 1, 8, 70
    rot = {"base": 5000.0, "dims": dims, "scaling": {"factor": 6.0, "original": 200, "fast": 16.0, "slow": 2.0}}
    g = torch.Generator().manual_seed(dim)
    q, k, v = torch.randn(T, H, dim, generator=g), torch.randn(T, G, dim, generator=g), torch.randn(T, G, e, generator=g)
    f, gain = O.frequencies(rot)
    fd, gd = scaled_frequencies(dims, 5000.0, rot["scaling"], dev)
    cache = new_cache(dev)
    kc, vc = cache.add_plane("k", (G * dim,), torch.float32), cache.add_plane("v", (G * e,), torch.float32)
    batch_of(cache, [("s", 640)], dev)
    b = batch_of(cache, [("s", T)], dev)
    proj = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1).to(dev)
    seqops.rope_norm_store(proj, 0, H * dim, (H + G) * dim, H, G, dim, e, fd, dims, None, EPS, False, b, kc, vc, prep=seqops.head_prep(rot_gain=gd))
    pos = torch.arange(640, 640 + T)
    assert rel(proj[:, :H * dim].reshape(T, H, dim), O.rotate_half(q.double(), pos, f, gain)) < 2e-5
    rows = torch.tensor([cache.seqs["s"]["pages"][int(p) // 64] * 64 + int(p) % 64 for p in pos])
    assert rel(kc.reshape(-1, G, dim).cpu()[rows], O.rotate_half(k.double(), pos, f, gain)) < 2e-5
    assert torch.equal(proj[:, -G * e:].cpu(), v.reshape(T, -1))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,keep", [(90, 7), (64, 0), (65, 1), (1, 3), (130, 64), (37, 70)])
def test_one_far_key_at_every_edge(dev, dtype, size, keep):
    """ONE key stands out (a coordinate of its own); its value is seen exactly by the queries whose window or kept first keys hold it: keys
    just inside and outside the window, at page borders, the last kept and the first not kept, in portions and for single tokens"""
    from zhilight_amd import seqops
    H, G, d, e, T = 2, 1, 32, 16, 300
    g = torch.Generator().manual_seed(size + keep)
    places = sorted({0, max(keep - 1, 0), keep, 63, 64, 127, 128, 200 - size if size < 200 else 1, 250 - size if size < 250 else 2})
    q = torch.zeros(T, H, d)
    q[..., 0] = 4.0
    q[..., 1:] = 0.3 * torch.randn(T, H, d - 1, generator=g)
    v = torch.randn(T, G, e, generator=g)
    for j in places:
        k = 0.3 * torch.randn(T, G, d, generator=g)
        k[..., 0] = 0.0
        k[j, :, 0] = 3.0
        if dtype == torch.bfloat16:
            k, v = bf(k).float(), bf(v).float()
        ref = O.softmax_attention(q.double(), k.double(), v.double(), 1.0, O.visible(T, size, keep))
        for portions in ([T], [100] + [1] * 12 + [T - 112], [j + 2] + [1] * min(60, T - j - 2) + ([T - j - 2 - min(60, T - j - 2)] if T - j - 2 > 60 else [])):
            cache = new_cache(dev)
            kc, vc = cache.add_plane("k", (G * d,), dtype), cache.add_plane("v", (G * e,), dtype)
            batch_of(cache, [("other", 3)], dev)                                 # (pages that do not start at 0)
            got, at = [], 0
            for n in portions:
                b = batch_of(cache, [("s", n)], dev)
                proj = torch.cat([q[at:at + n].reshape(n, -1), k[at:at + n].reshape(n, -1), v[at:at + n].reshape(n, -1)], 1).to(dev)
                seqops.rope_norm_store(proj, 0, H * d, (H + G) * d, H, G, d, e, None, 0, None, EPS, False, b, kc, vc)
                acc, ml, ns = seqops.window_attention(proj, 0, kc, vc, b, 1.0, size, H, G, d, e, all_kv=False, keep_first=keep)
                got.append(seqops.head_mix_gate(acc, ml, ns, None, None, None, 0, b, H, G, e, torch.float32))
                at += n
            err = rel_rows(torch.cat(got), ref.reshape(T, -1))
            assert float(err.max()) < (2e-5 if dtype == torch.float32 else 3e-2), (size, keep, j, portions[:3], float(err.max()), int(err.argmax()))
    # the sight of that key is not a small thing: hiding it changes the output
    blind = O.softmax_attention(q.double(), k.double(), v.double(), 1.0, O.visible(T, size, keep) & (torch.arange(T) != j)[None, :] | torch.eye(T, dtype=torch.bool))
    seen = O.visible(T, size, keep)[:, j] & (torch.arange(T) != j)
    if seen.any():
        assert float(rel_rows(blind.reshape(T, -1), ref.reshape(T, -1))[seen].median()) > 0.3


@pytest.mark.parametrize("vdim", [16, 33, 128])
def test_gate_per_head_into_columns_of_a_wider_row(dev, vdim):
    from zhilight_amd import seqops
    H, G, S, T = 6, 2, 3, 9
    g = torch.Generator().manual_seed(vdim)
    cache = new_cache(dev)
    b = batch_of(cache, [("s", T)], dev)
    acc, m, l = torch.randn(T, H, S, vdim, generator=g), torch.randn(T, H, S, generator=g), torch.rand(T, H, S, generator=g) + 0.5
    gate = torch.randn(T, H + 5, generator=g)
    wide = torch.full((T, H * vdim + 20), 7.0, device=dev)
    w = torch.exp(m.double() - m.double().max(-1, keepdim=True).values)
    ref = (w[..., None] * acc.double()).sum(2) / (w * l.double()).sum(-1, keepdim=True)
    ref = 0.6 * (ref * O.sigmoid(gate.double()[:, 3:3 + H])[:, :, None]).reshape(T, -1)
    out = seqops.head_mix_gate(acc.to(dev), torch.stack([m, l], -1).to(dev), S, None, None, gate.to(dev), 3, b, H, G, vdim, torch.float32, gate_per_head=True,
                               out=wide[:, 8:8 + H * vdim], out_scale=0.6)
    assert rel(out, ref) < 1e-6 and bool((wide[:, :8] == 7.0).all()) and bool((wide[:, 8 + H * vdim:] == 7.0).all())
    # the other two steps that write into a shared row
    y, wn, gt = torch.randn(T, H * vdim, generator=g), torch.randn(H * vdim, generator=g), torch.randn(T, H * vdim, generator=g)
    ref = 0.6 * (O.unit_rms(y.double().reshape(T, H, vdim), EPS).reshape(T, -1) * wn.double() * O.sigmoid(gt.double()))
    seqops.linear_attn_finish(y.to(dev), False, 1.0, None, 0.0, H, vdim, H, wn.to(dev), EPS, gt.to(dev), 0, torch.float32, out=wide[:, 20:], out_scale=0.6)
    assert rel(wide[:, 20:], ref) < 1e-6
    gu = torch.randn(T, 2 * vdim + 3, generator=g)
    seqops.act_mul(gu.to(dev), torch.float32, kind="silu", col0=3, ff=vdim, out=wide[:, 1:1 + vdim])
    assert rel(wide[:, 1:1 + vdim], O.silu(gu.double()[:, 3:3 + vdim]) * gu.double()[:, 3 + vdim:]) < 1e-6 and bool((wide[:, 0] == 7.0).all())
    assert rel(wide[:, 20 + vdim:], ref[:, vdim:]) < 1e-6


def scan_inputs(g, T, H, G, d, e, per_channel, strong=False):
    q, k = (O.unit_vector(torch.randn(T, G, d, generator=g, dtype=F64)) for _ in range(2))
    q = q * d ** -0.5
    v, beta = torch.randn(T, H, e, generator=g, dtype=F64), torch.rand(T, H, generator=g, dtype=F64)
    dec = torch.exp(-O.softplus(torch.randn(T, H, d if per_channel else 1, generator=g, dtype=F64) * (8.0 if strong else 1.0) - (0.0 if strong else 3.0)))
    qkv = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1).float()
    q, k, v = qkv[:, :G * d].double().reshape(T, G, d), qkv[:, G * d:2 * G * d].double().reshape(T, G, d), qkv[:, 2 * G * d:].double().reshape(T, H, e)
    gates = torch.zeros(T, H, 4)
    gates[..., 0] = beta
    gates[..., 1] = 1.0 if per_channel else dec[..., 0]
    spread = torch.arange(H) // (H // G)
    gates[..., 2] = (q * k).sum(-1)[:, spread]
    decay = dec.reshape(T, -1).float() if per_channel else None
    ref = O.delta_recurrence(q[:, spread], k[:, spread], v, gates[..., 0].double(), dec.float().double().expand(T, H, d))
    return qkv, gates, decay, ref.reshape(T, -1)


@pytest.mark.parametrize("per_channel", [False, True])
@pytest.mark.parametrize("d,e,H,G", [(1, 3, 2, 1), (7, 5, 3, 1), (16, 16, 4, 2), (20, 33, 2, 2), (32, 8, 2, 1), (33, 9, 1, 1), (64, 64, 4, 4), (100, 40, 2, 1),
                                     (128, 128, 2, 2), (130, 17, 2, 1), (256, 20, 1, 1), (300, 6, 1, 1), (512, 12, 2, 1)])
def test_delta_scan_sizes_and_portions(dev, d, e, H, G, per_channel):
    """every instantiation, with and without 16-byte pieces, chunks full and partial, the state carried over portions; other slots untouched"""
    from zhilight_amd import seqops
    g = torch.Generator().manual_seed(d + e)
    T = 53
    qkv, gates, decay, ref = scan_inputs(g, T, H, G, d, e, per_channel)
    for portions in ([T], [16, 1, 2, 4, 30], [1] * 5 + [48], [3, 32, 18]):
        cache = new_cache(dev)
        st = cache.add_state("S", (H, e, d))
        batch_of(cache, [("x", 1), ("s", 1)], dev)
        cache.seqs["s"]["len"] = 0
        st[2] = 5.0
        out, at = [], 0
        for n in portions:
            b = batch_of(cache, [("s", n)], dev)
            cut = [None if t is None else t[at:at + n].to(dev).contiguous() for t in (qkv, gates, decay)]
            out.append(seqops.delta_scan(*cut, st, H, G, d, e, b))
            at += n
        assert rel(torch.cat(out), ref) < 5e-6 and float(rel_rows(torch.cat(out), ref).max()) < 5e-5, portions
        assert bool((st[2] == 5.0).all()) and not bool(st[0].any())


@pytest.mark.parametrize("per_channel", [False, True])
def test_delta_scan_many_sequences_and_strong_decays(dev, per_channel):
    """enough columns that every group of lanes takes two; unequal portions in one launch; decays from e^-20 to 1"""
    from zhilight_amd import seqops
    H, G, d, e = 16, 8, 64, 64
    counts = [1, 37, 2, 16, 1, 50, 17, 33]
    g = torch.Generator().manual_seed(3)
    cache = new_cache(dev, 2048, len(counts))
    st = cache.add_state("S", (H, e, d))
    parts = [scan_inputs(g, n, H, G, d, e, per_channel, strong=True) for n in counts]
    b = batch_of(cache, [(i, n) for i, n in enumerate(counts)], dev)
    cut = [None if parts[0][j] is None else torch.cat([p[j] for p in parts]).to(dev) for j in range(3)]
    y = seqops.delta_scan(*cut, st, H, G, d, e, b)
    assert rel(y, torch.cat([p[3] for p in parts])) < 5e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("per_channel", [False, True])
@pytest.mark.parametrize("m", [delta_m(), delta_m(heads=1, kv_heads=1, dim=7, vdim=11, conv=1, low=1), delta_m(heads=6, kv_heads=2, dim=70, vdim=45, conv=2, low=8),
                               delta_m(heads=4, kv_heads=4, dim=130, vdim=64, conv=3, low=17), delta_m(heads=2, kv_heads=1, dim=300, vdim=9, conv=6)])
def test_delta_mixer_in_portions(dev, dtype, per_channel, m):
    """the whole mixer -- convolution with portions shorter than its reach, unit vectors, gates, low-rank pairs, norm -- in several cuts"""
    W, T = 64, 61
    sd = delta_weights(m, W, 11, per_channel)
    g = torch.Generator().manual_seed(5)
    h = bf(torch.randn(T, W, generator=g))
    ref = O.delta_mixer(h, sd, "", m, EPS, per_channel)
    for portions in ([T], [1] * 7 + [54], [2, 1, 3, 2, 20, 1, 32]):
        cache = new_cache(dev)
        mix = delta_mixer(m, W, sd, dtype, dev, cache, per_channel)
        batch_of(cache, [("x", 1)], dev)
        assert_close(feed(mix, cache, h.to(dtype), portions, dev), ref, dtype, portions)


def test_delta_mixer_many_tokens_in_blocks(dev):
    """steps long enough that a workgroup convolves a block of tokens: several sequences whose starts fall inside blocks, portions shorter than
    the convolution's reach among them"""
    m, W = delta_m(heads=8, kv_heads=8, dim=64, vdim=64, conv=4, low=16), 64
    sd = delta_weights(m, W, 12, True)
    counts = [300, 1, 2, 401, 3, 5, 360, 1, 1, 90]
    g = torch.Generator().manual_seed(6)
    cache = new_cache(dev, 64 * 40, len(counts))
    mix = delta_mixer(m, W, sd, torch.float32, dev, cache, True)
    hs = [bf(torch.randn(n + 7, W, generator=g)) for n in counts]
    refs = [O.delta_mixer(h, sd, "", m, EPS, True) for h in hs]
    for lo, hi in ((lambda n: 0, lambda n: n), (lambda n: n, lambda n: n + 7)):
        cut = [(lo(n), hi(n)) for n in counts]
        b = batch_of(cache, [(i, z - a) for i, (a, z) in enumerate(cut)], dev)
        got = mix.forward(torch.cat([h[a:z] for h, (a, z) in zip(hs, cut)]).float().to(dev), b)
        assert_close(got, torch.cat([r[a:z] for r, (a, z) in zip(refs, cut)]), torch.float32)


@pytest.mark.parametrize("per_channel", [False, True])
def test_a_token_still_shows_two_hundred_tokens_later(dev, per_channel):
    """a mixer whose decay is close to 1 and that writes once: the value under that key comes back, through prompts and decoding"""
    m, W, T = delta_m(heads=2, kv_heads=2, dim=16, vdim=8, conv=2, low=4), 32, 240
    sd = dict(delta_weights(m, W, 13, per_channel))
    sd["A_log"], sd["dt_bias"] = torch.full_like(sd["A_log"], -4.0), torch.full_like(sd["dt_bias"], -6.0)
    sd["b"] = torch.zeros_like(sd["b"])
    sd["b"][:, 0] = 20.0                                                         # (beta: open where the input's first coordinate is positive, shut elsewhere)
    g = torch.Generator().manual_seed(14)
    h = bf(torch.randn(T, W, generator=g))
    h[:, 0] = -1.0
    h[5, 0] = 1.0
    h2 = h.clone()
    h2[5, 1:] = -h[5, 1:]
    ref, ref2 = (O.delta_mixer(x, sd, "", m, EPS, per_channel) for x in (h, h2))
    assert rel(ref2[210:], ref[210:]) > 0.3                                      # (it is that one token's doing)
    for portions in ([T], [64, 1, 2, 133] + [1] * 40):
        cache = new_cache(dev)
        assert_close(feed(delta_mixer(m, W, sd, torch.float32, dev, cache, per_channel), cache, h.float(), portions, dev), ref, torch.float32, portions[:3])


@pytest.mark.parametrize("dtype", DTYPES)
def test_joined_sublayers_against_their_sum(dev, dtype):
    """two products for everything that runs side by side, output scales and biases included, against the parts' own sum"""
    from zhilight_amd.mixers import GatedFF, JoinedSublayers
    from zhilight_amd.suvapel import MIXER_BUILDERS
    W, T = 64, 50
    layer = parallel_l(attn_m(), delta_m(low=11), -0.7, 1.3, ff=40)
    sd = O.random_weights(model_cfg([layer], width=W), 15)
    h = bf(torch.randn(T, W, generator=torch.Generator().manual_seed(16)))
    ref = O.mixer(h, sd, "l0.mix.", layer, EPS) + O.dense_ff(h, sd, "l0.mlp.")
    for portions in ([T], [1] * 12 + [38], [2, 30, 18]):
        cache = new_cache(dev)
        j = JoinedSublayers(W, MIXER_BUILDERS["parallel"]("l0.mix", W, layer["mixer"], EPS) + [("mlp.", GatedFF(W, 40, act="silu", bias=True), 1.0)])
        j.load(lambda n: sd[n], "l0.", dtype, dev).bind(cache, dtype)
        assert_close(feed(j, cache, h.to(dtype), portions, dev), ref, dtype, portions)


@pytest.mark.parametrize("dtype", DTYPES)
def test_feed_forward_with_biases_alone(dev, dtype):
    from zhilight_amd.mixers import GatedFF
    W, ff = 64, 90
    sd = O.random_weights(model_cfg([delta_l(ff=ff)], width=W), 17)
    ffn = GatedFF(W, ff, act="silu", bias=True).load(lambda n: sd[n], "l0.mlp.", dtype, dev)
    for T in (1, 5, 100):
        h = bf(torch.randn(T, W, generator=torch.Generator().manual_seed(T)))
        assert_close(ffn.forward(h.to(dtype).to(dev)), O.dense_ff(h, sd, "l0.mlp."), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dim", [1, 9, 24, 256])
def test_token_side_input(dev, dtype, dim):
    from zhilight_amd import seqops
    from zhilight_amd.mixers import TokenSideInput
    W = 70
    cfg = model_cfg([delta_l(), delta_l(), delta_l()], width=W, side=dim)
    sd = O.random_weights(cfg, 18)
    for T in (1, 6, 80):
        g = torch.Generator().manual_seed(T)
        x, toks = bf(torch.randn(T, W, generator=g)), torch.randint(0, 160, (T,), generator=g, dtype=torch.int32)
        e = sd["side.embed"].double()[toks.long()][:, 2 * dim:3 * dim]
        ref = O.token_side(x, e, sd, "l2.side.", 0.45, EPS)
        side = TokenSideInput(W, dim, 2 * dim).load(lambda n: sd[n], "l2.side.", dtype, dev)
        xd = x.float().to(dev)
        seqops.add_branches(xd, [side.branch(x.to(dtype).to(dev), sd["side.embed"].to(dtype).to(dev), toks.to(dev), 0.45)], EPS, dtype)
        assert_close(xd - x.float().to(dev), ref - x, dtype, T)


# ------------------------------------------------------------------------------------------------------------------------------------
# the model through the engine
# ------------------------------------------------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_a():
    cfg = cfg_a()
    sd = O.random_weights(cfg, 21)
    toks = tokens_of(cfg, 230, 22)
    layers = []
    return cfg, sd, toks, O.forward(toks, sd, cfg, layers), layers


@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_prompt_and_every_layer(dev, dtype, model_a):
    cfg, sd, toks, logits, layers = model_a
    eng = make(cfg, sd, dtype, dev)
    assert_close(run_portions(eng, "w", toks, [len(toks)]), logits, dtype)
    b = batch_of(eng.cache, [("L", len(toks))], dev)
    got = eng.model.forward_layers(torch.tensor(toks, dtype=torch.int32, device=dev), b)
    assert len(got) == len(layers) == 4
    for i, (x, ref) in enumerate(zip(got, layers)):
        assert_close(x, ref, dtype, f"layer {i}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_token_by_token_from_the_first_token_and_after_a_prompt(dev, dtype, model_a):
    cfg, sd, toks, logits, _ = model_a
    eng = make(cfg, sd, dtype, dev)
    assert_close(run_portions(eng, "d0", toks[:100], [1] * 100), logits[:100], dtype, "from the first token")
    assert_close(run_portions(eng, "d1", toks, [50] + [1] * 180), logits, dtype, "long decoding across page borders and windows")


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_many_sizes(dev, dtype, model_a):
    cfg, sd, toks, logits, _ = model_a
    eng = make(cfg, sd, dtype, dev)
    for portions in ([2] * 20 + [3, 5, 1, 60, 64, 1, 2, 54], [63, 1, 64, 65, 37], [128, 2, 100], [36, 2, 35, 2, 155]):
        assert_close(run_portions(eng, "p", toks, portions), logits, dtype, portions[:3])


@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_with_reused_pages_and_slots(dev, dtype):
    """five unequal requests in mixed steps (portions beside single tokens) in a pool that only holds them because pages and slots come
    back; each request's logits equal its logits alone"""
    from zhilight_amd.engine import Entry
    cfg = cfg_a()
    sd = O.random_weights(cfg, 23)
    lens = [150, 97, 201, 64, 33]
    reqs = {f"r{i}": tokens_of(cfg, n, 30 + i) for i, n in enumerate(lens)}
    refs = {k: O.forward(v, sd, cfg) for k, v in reqs.items()}
    eng = make(cfg, sd, dtype, dev, max_tokens=64 * 8, max_seqs=3)
    got, at = {k: [] for k in reqs}, {k: 0 for k in reqs}
    waiting, live = list(reqs), []
    rng = np.random.default_rng(5)

    def pages(k):
        return (len(reqs[k]) + 63) // 64
    while waiting or live:
        while waiting and len(live) < 3 and sum(pages(k) for k in live) + pages(waiting[0]) <= 8:
            live.append(waiting.pop(0))
        entries = []
        for k in live:
            left = len(reqs[k]) - at[k]
            n = min(left, int(rng.choice([1, 1, 2, 7, 40, 64])))
            if rng.random() < 0.2 and len(live) > 1 and entries:
                continue                                                        # (left out of a step, goes on later)
            entries.append(Entry(k, reqs[k][at[k]:at[k] + n], list(range(n))))
        out = eng.run_step(entries)
        row = 0
        for e in entries:
            got[e.rid].append(out[row:row + len(e.tokens)])
            row += len(e.tokens)
            at[e.rid] += len(e.tokens)
            if at[e.rid] == len(reqs[e.rid]):
                eng.release(e.rid)
                live.remove(e.rid)
    for k in reqs:
        assert_close(torch.cat(got[k]), refs[k], dtype, k)
    assert len(eng.cache.free_pages) == 8 and len(eng.cache.free_slots) == 3


def test_same_bits_after_pages_and_slots_were_used_by_others(dev):
    cfg = cfg_a()
    sd = O.random_weights(cfg, 24)
    eng = make(cfg, sd, torch.bfloat16, dev, max_tokens=64 * 4, max_seqs=2)
    a, b = tokens_of(cfg, 130, 1), tokens_of(cfg, 120, 2)
    first = run_portions(eng, "a", a, [100, 1, 29])
    run_portions(eng, "b", b, [120], release=False)
    eng.release("b")
    assert torch.equal(first, run_portions(eng, "a2", a, [100, 1, 29]))


@pytest.mark.parametrize("dtype", DTYPES)
def test_odd_sizes_whole_in_portions_and_decoded(dev, dtype):
    cfg = cfg_odd(1 if dtype == torch.float32 else 6)
    sd = O.random_weights(cfg, 27)
    toks = tokens_of(cfg, 140, 26)
    logits = O.forward(toks, sd, cfg)
    eng = make(cfg, sd, dtype, dev)
    assert_close(run_portions(eng, "w", toks, [140]), logits, dtype, "whole")
    assert_close(run_portions(eng, "p", toks, [2, 2, 1, 60, 5, 1, 1, 68]), logits, dtype, "portions")
    assert_close(run_portions(eng, "d", toks[:70], [1] * 70), logits[:70], dtype, "decoded")


def test_medium_configuration_other_kernel_instantiations(dev):
    """head sizes up to 128, 16 heads on 4 kv heads, a delta rule of 128 x 64 states, long portions"""
    cfg = model_cfg([parallel_l(attn_m(heads=16, kv_heads=4, dim=128, vdim=64, scale=0.09, size=150, keep=4, dims=64, conv=4), delta_m(heads=4, kv_heads=4, dim=128, vdim=64, low=32), ff=256),
                     delta_l(heads=8, kv_heads=4, dim=128, vdim=64, ff=512)], width=256, vocab=300, side=64)
    sd = O.random_weights(cfg, 29)
    toks = tokens_of(cfg, 420, 30)
    logits = O.forward(toks, sd, cfg)
    for dtype in DTYPES:
        eng = make(cfg, sd, dtype, dev)
        assert_close(run_portions(eng, "w", toks, [300, 1, 1, 118]), logits, dtype, "medium")


@pytest.mark.parametrize("drop", ["token_side", "mask", "rot", "scaling"])
def test_parts_that_a_configuration_may_leave_out(dev, drop):
    cfg = model_cfg([parallel_l(attn_m(), delta_m()), delta_l()])
    sd = O.random_weights(cfg, 34)
    toks = tokens_of(cfg, 90, 35)
    left = cfg["layers"][0]["mixer"]["left"]
    ref = {**cfg, "layers": cfg["layers"]}
    if drop == "token_side":
        cfg = {k: v for k, v in cfg.items() if k != "token_side"}
        sd = {k: torch.zeros_like(v) if k.endswith("side.norm") else v for k, v in sd.items()}       # (the restatement always has one)
    elif drop == "mask":
        left.pop("mask")
        ref = {**cfg, "layers": [{**cfg["layers"][0], "mixer": {**cfg["layers"][0]["mixer"], "left": {**left, "mask": {"size": 0}}}}, cfg["layers"][1]]}
    elif drop == "rot":
        left.pop("rot")
        ref = {**cfg, "layers": [{**cfg["layers"][0], "mixer": {**cfg["layers"][0]["mixer"], "left": {**left, "rot": {"dims": 0, "base": 2.0}}}}, cfg["layers"][1]]}
    else:
        left["rot"].pop("scaling")
    if drop == "rot":                                                            # (no frequencies: nothing is rotated)
        logits = None
        keep, O_rotate = O.frequencies, O.rotate_half
        try:
            O.frequencies, O.rotate_half = lambda rot: (torch.zeros(0, dtype=F64), 1.0), lambda x, pos, f, gain: x
            logits = O.forward(toks, sd, ref)
        finally:
            O.frequencies, O.rotate_half = keep, O_rotate
    else:
        logits = O.forward(toks, sd, ref)
    eng = make(cfg, sd, torch.float32, dev)
    assert_close(run_portions(eng, "w", toks, [50, 1, 2, 37]), logits, torch.float32, drop)


def test_greedy_generation_through_the_scheduler(dev):
    """Engine.generate under a small step budget (prompts cut into portions, decode tokens beside them) gives what feeding the restatement
    its own arg-max gives"""
    from zhilight_amd.engine import SamplingParams
    cfg = cfg_a()
    sd = O.random_weights(cfg, 31)
    prompts = [tokens_of(cfg, n, 40 + n) for n in (40, 9, 75)]
    eng = make(cfg, sd, torch.float32, dev, max_tokens=64 * 10, max_seqs=2, max_step_tokens=48)
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=4))
    for p, out in zip(prompts, outs):
        assert len(out) == 4
        logits = O.forward(list(p) + out, sd, cfg)[len(p) - 1:-1]
        for row, tok in zip(logits, out):
            top2 = torch.topk(row, 2).values
            assert int(torch.argmax(row)) == tok or float(top2[0] - top2[1]) < 1e-3           # (a tie within rounding may go either way)


def test_trace_replayer_on_a_model_folder(dev, tmp_path, capsys):
    """a folder with config.json and model.safetensors through the registry's loader and the trace replayer: two requests in mixed steps
    (a portion beside single tokens), one leaves and its pages and slot are taken again; the written logits are the restatement's"""
    import io
    import json
    from safetensors.torch import save_file
    from zhilight_amd import trace
    cfg = cfg_a()
    sd = O.random_weights(cfg, 33)
    folder, out = tmp_path / "model", tmp_path / "out"
    folder.mkdir()
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(folder / "model.safetensors"))
    a, b, c = tokens_of(cfg, 90, 1), tokens_of(cfg, 70, 2), tokens_of(cfg, 100, 3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:60], "want": [0, 59]}, {"id": "b", "tokens": b[:2], "want": [1]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:70], "want": [67]}, {"id": "a", "tokens": a[60:61], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[61:90], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "c", "tokens": c, "want": [99]}, {"id": "a", "tokens": [a[0]], "want": [0]}], "end": ["a", "c"]}]
    stream = io.StringIO("".join(json.dumps(s) + "\n" for s in steps))
    assert trace.replay(str(folder), "float32", str(out), max_tokens=256, max_seqs=2, stream=stream, device=str(dev)) == 0
    assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    la, lb, lc = O.forward(a + [a[0]], sd, cfg), O.forward(b, sd, cfg), O.forward(c, sd, cfg)
    want = {0: torch.stack([la[0], la[59], lb[1]]), 1: torch.stack([lb[69], la[60]]), 3: torch.stack([lc[99], la[90]])}
    assert not (out / "2.f32").exists()
    for n, ref in want.items():
        got = torch.from_numpy(np.fromfile(str(out / f"{n}.f32"), dtype="<f4").reshape(ref.shape[0], cfg["vocab"]))
        assert_close(got, ref, torch.float32, f"step {n}")
