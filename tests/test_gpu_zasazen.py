"""Zasazen on the GPU against the plain float64 restatement in tests/zasazen_oracle.py: every mechanism alone, then the model through the
engine's step function -- whole prompts, token-by-token decoding, portions down to two tokens, mixed batches, reused pages and slots, keys
far back and at page borders, steps of the query temperature, long decoding, odd sizes, greedy generation through the scheduler.  Small
random configurations made here; nothing is read from disk.

fp32 serving is held to rounding of fp32 sums everywhere, bf16 serving to bf16 rounding of the matrix-product inputs.  The bf16 MODEL tests
use weights without close calls (zasazen_oracle.random_weights, fixed_choice); ordinary routers are tested in fp32 through the same models
and on the router alone."""
import math

import numpy as np
import pytest
import torch

import zasazen_oracle as O

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
def mamba_cfg(inner=112, state=16, rank=6, conv=4):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": rank, "conv": conv}, "mlp": None}


def parallel_cfg(heads=4, kv_heads=2, dim=40, vdim=32, scale=0.2, coef=0.3, every=37, rh=3, rd=24, rv=20, rot=16, base=4000.0, decay=None):
    decay = decay or [1.0 - 2.0 ** -(3 + 2 * h) for h in range(rh)]
    return {"type": "parallel", "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                                                   "q_temp": {"coef": coef, "every": every}},
                                          "right": {"heads": rh, "dim": rd, "vdim": rv, "decay": decay, "rot": {"base": base, "dims": rot}}}, "mlp": None}


def dense(ff=144):
    return {"kind": "dense", "ff": ff}


def moe(ff=48, experts=10, top=3, shared=80):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared}}


def with_mlp(layer, mlp):
    layer = dict(layer)
    layer["mlp"] = mlp
    return layer


def model_cfg(layers, width=96, vocab=160, scale=5.0, loop=(0, 1, 1)):
    cfg = {"architecture": "Zasazen", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": EPS}, "layers": layers}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def cfg_a():
    """both mixers, both feed-forwards and a layer without one; the two middle layers run twice"""
    return model_cfg([with_mlp(parallel_cfg(), dense()), with_mlp(mamba_cfg(), moe()),
                      with_mlp(parallel_cfg(heads=8, kv_heads=4, dim=32, vdim=16, every=50, rh=2, rd=32, rv=48, rot=32), moe(ff=40, experts=8, top=2, shared=32)),
                      mamba_cfg(inner=70, state=5, rank=9, conv=2)], loop=(1, 3, 2))


def cfg_odd():
    """sizes no matrix-core kernel takes, and values that a particular model may make equal or 1: heads = kv heads, one kv head, one
    retention head, no rotated coordinates, one tap, one state, a rank of 1, all experts chosen, one chosen, no shared expert, every layer
    in a loop of three passes, a temperature step at every position"""
    odd = with_mlp(parallel_cfg(heads=3, kv_heads=3, dim=20, vdim=12, every=1, coef=0.05, rh=1, rd=10, rv=7, rot=6, decay=[0.9375]), moe(ff=20, experts=4, top=4, shared=24))
    single = moe(ff=32, experts=5, top=1)
    del single["shared"]
    return model_cfg([with_mlp(mamba_cfg(inner=33, state=1, rank=1, conv=1), dense(50)), odd,
                      with_mlp(parallel_cfg(heads=4, kv_heads=1, dim=16, vdim=16, rh=2, rd=9, rv=33, rot=0, decay=[1.0, 0.5]), single),
                      mamba_cfg(inner=130, state=40, rank=8, conv=6)], width=72, vocab=90, scale=1.0, loop=(0, 4, 3))


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


def oracle_model(cfg, sd, toks, fixed=True):
    """(logits, the residual after every layer run); with fixed-choice weights no router choice may be a close call"""
    layers, margins = [], []
    logits = O.model(toks, sd, cfg, layers, margins)
    assert not fixed or not margins or min(margins) > 0.1, margins
    return logits, layers


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


def mixed_sum(mixer, h, batch):
    """what a mixer's branches add to a residual of zeros"""
    from zhilight_amd import seqops
    x = torch.zeros(h.shape, dtype=torch.float32, device=h.device)
    seqops.add_branches(x, mixer.branches(h, batch), EPS, h.dtype)
    return x


def feed(mixer, cache, h, portions, dev, sid="s"):
    out, at = [], 0
    for n in portions:
        out.append(mixed_sum(mixer, h[at:at + n].to(dev).contiguous(), batch_of(cache, [(sid, n)], dev)))
        at += n
    assert at == h.shape[0]
    return torch.cat(out)


def build_mixer(layer, sd, prefix, width, dtype, dev, cache):
    from zhilight_amd import zasazen
    mix = zasazen.MIXER_BUILDERS[layer["type"]]("m" + prefix, width, layer["mixer"], EPS)
    mix.load(lambda n: sd[n], prefix, dtype, dev)
    mix.bind(cache, dtype)
    return mix


# ------------------------------------------------------------------------------------------------------------------------------------
# mechanisms alone
# ------------------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [1, 2, 3, 8, 13, 70, 300])
def test_product_epilogues(dev, dtype, m):
    """bias, activation and the leading columns in the serving format, on every product kernel (few rows, up to 16, tiles)"""
    from zhilight_amd import seqops
    acts = {None: lambda z: z, "relu2": lambda z: torch.relu(z) ** 2, "gelu_tanh": O.gelu_tanh, "silu": O.silu, "softplus": O.softplus}
    for n, k in ((70, 48), (200, 33), (40, 1000)):                              # (the last: k divided over workgroups above 16 rows)
        g = torch.Generator().manual_seed(n + m)
        x, w, b = bf(torch.randn(m, k, generator=g)), bf(torch.randn(n, k, generator=g) * 2 * k ** -0.5), torch.randn(n, generator=g)
        xd, wd, bd = x.to(dev).to(dtype), w.to(dev).to(dtype), b.to(dev)
        for name, fn in acts.items():
            ref = fn(x @ w.T + b.double())
            assert rel(seqops.gemm_nt(xd, wd, bias=bd, act=name), ref) < 3e-6, name
            assert rel(seqops.gemm_nt(xd, wd, act=name), fn(x @ w.T)) < 3e-6, name
            y, lead = seqops.gemm_nt(xd, wd, bias=bd, act=name, lead=24)
            assert rel(y, ref) < 3e-6 and lead.dtype == dtype and torch.equal(lead, y[:, :24].to(dtype))
        assert torch.equal(seqops.gemm_nt(xd, wd, bias=bd, act="gelu_tanh", out_dtype=dtype), seqops.gemm_nt(xd, wd, bias=bd, act="gelu_tanh").to(dtype))


@pytest.mark.parametrize("W", [77, 96, 2048])
def test_branches_join_the_residual_with_two_norms(dev, W):
    from zhilight_amd import seqops
    T = 5
    g = torch.Generator().manual_seed(W)
    x = torch.randn(T, W, generator=g) * 2
    ys = [torch.randn(T, W, generator=g) * (3.0 if i != 1 else 1e-3) for i in range(4)]            # (one tiny: eps inside the root decides)
    w = [1.0 + 0.3 * torch.randn(W, generator=g) for _ in range(6)]
    coefs = [0.5, 0.5, 1.0, -2.0]
    for n, normed in ((0, ()), (1, ()), (1, (0,)), (2, (0, 1)), (3, (0, 1)), (4, (1, 3))):
        new = x.double()
        for i in range(n):
            new = new + coefs[i] * (O.rms_norm(ys[i].double(), w[i].double(), EPS) if i in normed else ys[i].double())
        xd = x.to(dev)
        br = [(ys[i].to(dev), w[i].to(dev) if i in normed else None, coefs[i]) for i in range(n)]
        wide = torch.full((T, 2 * W + 3), 7.0, device=dev, dtype=torch.bfloat16)
        h1, h2 = seqops.add_branches(xd, br, EPS, torch.bfloat16, w[4].to(dev), w[5].to(dev), xt=wide[:, W:2 * W])
        assert rel(xd, new) < 1e-6 and rel(h1, O.rms_norm(new, w[4].double(), EPS)) < 4e-3 and rel(h2, O.rms_norm(new, w[5].double(), EPS)) < 4e-3
        assert torch.equal(wide[:, W:2 * W], xd.to(torch.bfloat16)) and bool((wide[:, :W] == 7).all()) and bool((wide[:, 2 * W:] == 7).all())
        xd = x.to(dev)
        h1, h2 = seqops.add_branches(xd, br, EPS, torch.float32, None, w[5].to(dev))
        assert h1 is None and rel(h2, O.rms_norm(new, w[5].double(), EPS)) < 1e-6
        xd = x.to(dev)
        assert seqops.add_branches(xd, br, EPS, torch.float32) == (None, None) and rel(xd, new) < 1e-6


def scan_inputs(T, inner, N, seed):
    g = torch.Generator().manual_seed(seed)
    x, z = torch.randn(T, inner, generator=g), torch.randn(T, inner, generator=g)
    dt = torch.nn.functional.softplus(torch.randn(T, inner, generator=g) * 1.5 - 2.0)
    bc = torch.randn(T, 2 * N + 3, generator=g)
    A = -torch.exp(torch.rand(inner, N, generator=g) * 5.0 - 3.0)
    A[0, 0] = -1e-4                                                            # (a state that hardly forgets)
    return x, z, dt, bc, A, torch.randn(inner, generator=g)


@pytest.mark.parametrize("N,inner", [(1, 20), (5, 64), (8, 65), (16, 200), (33, 70), (64, 130), (70, 64), (130, 33), (256, 64)])
def test_selective_scan_state_sizes_segments_and_portions(dev, N, inner):
    """every instantiation (states per wave, waves), channels past a workgroup's edge; whole portions, segments, portions of many sizes
    with the state carried between them"""
    from zhilight_amd import seqops
    T = 150
    x, z, dt, bc, A, D = scan_inputs(T, inner, N, N)
    ref = O.selective_scan(x.double(), dt.double(), A.double(), bc[:, 1:1 + N].double(), bc[:, 3 + N:].double(), D.double()) * O.silu(z.double())
    zrow = torch.cat([torch.zeros(T, 2), z], 1)
    a2 = (A.double() * math.log2(math.e)).float().t().contiguous().to(dev)
    for portions, seg in (([T], 0), ([T], 32), ([T], 40), ([T], 149), ([1, 2, 7, 8, 9, 1, 1, 60, 61], 16), ([1] * 30 + [120], None)):
        cache = new_cache(dev)
        state = cache.add_state("S", (N, inner))
        cache.admit("a")
        cache.admit("s")
        state.fill_(3.0)                                                        # (other slots hold something else)
        state[cache.seqs["s"]["slot"]].zero_()
        out, at = [], 0
        for n in portions:
            b = batch_of(cache, [("s", n)], dev)
            sl = slice(at, at + n)
            out.append(seqops.selective_scan(x[sl].contiguous().to(dev), dt[sl].contiguous().to(dev), bc[sl].contiguous().to(dev), 1, 3 + N,
                                             zrow[sl].contiguous().to(dev), 2, a2, D.to(dev), state, b, torch.float32, seg_len=seg))
            at += n
        assert_close(torch.cat(out), ref, torch.float32, (portions[:3], seg))
        assert bool((state[cache.seqs["a"]["slot"]] == 3.0).all())


def test_selective_scan_several_sequences_in_one_launch(dev):
    from zhilight_amd import seqops
    N, inner, lens = 16, 96, [1, 90, 2, 41]
    ins = [scan_inputs(2 * n, inner, N, n) for n in lens]
    A, D = ins[0][4], ins[0][5]
    a2 = (A.double() * math.log2(math.e)).float().t().contiguous().to(dev)
    cache = new_cache(dev, slots=4)
    state = cache.add_state("S", (N, inner))
    got = [[] for _ in lens]
    for half in (0, 1):
        b = batch_of(cache, [(str(i), n) for i, n in enumerate(lens)], dev)
        x, z, dt, bc = (torch.cat([ins[i][j][half * n:(half + 1) * n] for i, n in enumerate(lens)]).to(dev).contiguous() for j in range(4))
        y = seqops.selective_scan(x, dt, bc, 0, N, z, 0, a2, D.to(dev), state, b, torch.float32, seg_len=20)
        for i, part in enumerate(torch.split(y, lens)):
            got[i].append(part)
    for i in range(len(lens)):
        x, z, dt, bc = (t.double() for t in ins[i][:4])
        ref = O.selective_scan(x, dt, A.double(), bc[:, :N], bc[:, N:2 * N], D.double()) * O.silu(z)
        assert_close(torch.cat(got[i]), ref, torch.float32, i)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("inner,state,rank,conv", [(112, 16, 6, 4), (70, 5, 9, 2), (33, 1, 1, 1), (64, 40, 8, 7)])
def test_state_space_mixer_in_portions(dev, dtype, inner, state, rank, conv):
    """portions shorter than the convolution's reach, decoding, segments"""
    W, T = 96, 170
    layer = mamba_cfg(inner, state, rank, conv)
    sd = O.random_weights(model_cfg([layer], loop=None), 5)
    h = bf(torch.randn(T, W, generator=torch.Generator().manual_seed(6)))
    ref = O.mamba1_mixer(h, sd, "l0.mix.", layer["mixer"], EPS)
    for portions, seg in (([T], None), ([1] * 9 + [2, 2, 3, 60, 1, 93], None), ([2] * 10 + [150], 32), ([5, 165], 64)):
        cache = new_cache(dev)
        mix = build_mixer(layer, sd, "l0.mix.", W, dtype, dev, cache)
        mix.scan_segment = seg
        cache.admit("s")
        assert_close(feed(mix, cache, h.to(dtype), portions, dev), ref, dtype, (portions[:3], seg))


def sloped_kernels(q, k, v, scale, dtype, dev, portions, mfma=True, n_splits=None, shuffle_pages=False):
    """[q | k | v] rows through the cache-writing kernel (no norm, no rotation) and the attention kernels with linear slopes"""
    from zhilight_amd import mixers, seqops
    T, H, d = q.shape
    G, e = k.shape[1], v.shape[2]
    cache = new_cache(dev, max_tokens=64 * ((T + 63) // 64 + 3))
    if shuffle_pages:
        cache.free_pages = cache.free_pages[::-1]
    kp, vp = cache.add_plane("k", (G * d,), dtype), cache.add_plane("v", (G * e,), dtype)
    rows = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], dim=1).float()
    form = seqops.score_form(H, slope=mixers.linear_slopes(H, dev))
    out, at = [], 0
    for n in portions:
        b = batch_of(cache, [("s", n)], dev)
        proj = rows[at:at + n].to(dev).contiguous()
        seqops.rope_norm_store(proj, 0, H * d, H * d + G * d, H, G, d, e, None, 0, None, EPS, False, b, kp, vp)
        acc, ml, ns = seqops.window_attention(proj, 0, kp, vp, b, scale, 0, H, G, d, e, all_kv=False, mfma=mfma, n_splits=n_splits, form=form)
        out.append(seqops.head_mix_gate(acc, ml, ns, None, None, None, 0, b, H, G, e, torch.float32))
        at += n
    assert at == T
    return torch.cat(out).reshape(T, H, e)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("j", [0, 1, 63, 64, 65, 127, 128, 200])
def test_sloped_attention_one_far_key(dev, dtype, j):
    """one key far back, at page borders and at the very start, found by every head -- the steep ones too -- from inside a portion and from
    single tokens; both kernel families; the slope decides how much of it is left"""
    T, H, G, d, e, scale = 300, 8, 4, 24, 16, 1.0
    g = torch.Generator().manual_seed(j)
    q, k, v = bf(torch.randn(T, H, d, generator=g) * 0.3), bf(torch.randn(T, G, d, generator=g) * 0.3), bf(torch.randn(T, G, e, generator=g))
    s = O.slopes(H)
    k[:, :, 0] = 0.0                                                            # (one coordinate is the far key's own)
    k[j] = 0.0
    k[j, :, 0] = 1.0
    for i in (290, 297, 299):
        for a in range(H):                                                      # its score: what the slope takes off at this distance, plus 3
            q[i, a, 0] = bf(torch.tensor(s[a] * (i - j) + 3.0))
    v[j] = bf(8.0 * torch.randn(G, e, generator=g))
    ref = O.sloped_attention(q, k, v, scale)
    hidden = v.clone()
    hidden[j] = v[j + 1]
    for a in range(H):
        assert rel(O.sloped_attention(q, k, hidden, scale)[[290, 297, 299], a], ref[[290, 297, 299], a]) > 0.05           # it shows in every head
    for mfma, splits in ((True, None), (False, None), (False, 3)):
        got = sloped_kernels(q, k, v, scale, dtype, dev, [296, 1, 1, 1, 1], mfma=mfma, n_splits=splits, shuffle_pages=splits == 3)
        assert_close(got.reshape(T, -1), ref.reshape(T, -1), dtype, (j, mfma, splits))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e", [(4, 2, 8, 16), (3, 3, 72, 48), (2, 1, 160, 16), (8, 1, 256, 128), (6, 2, 20, 12), (1, 1, 64, 80)])
def test_sloped_attention_head_sizes_and_groups(dev, dtype, H, G, d, e):
    T = 200
    g = torch.Generator().manual_seed(d)
    q, k, v = bf(torch.randn(T, H, d, generator=g)), bf(torch.randn(T, G, d, generator=g)), bf(torch.randn(T, G, e, generator=g))
    ref = O.sloped_attention(q, k, v, 2.0 * d ** -0.5)
    steeper = O.slopes
    try:                                                                        # (slopes one head further along are visible)
        O.slopes = lambda n: [2.0 ** (-8.0 * (a + 2) / n) for a in range(n)]
        assert H == 1 or rel(O.sloped_attention(q, k, v, 2.0 * d ** -0.5), ref) > 0.05
    finally:
        O.slopes = steeper
    got = sloped_kernels(q, k, v, 2.0 * d ** -0.5, dtype, dev, [130, 1, 1, 2, 66])
    assert_close(got.reshape(T, -1), ref.reshape(T, -1), dtype, (d, e))


@pytest.mark.parametrize("dtype", DTYPES)
def test_slopes_beside_the_other_score_forms(dev, dtype):
    """a factor per head, a cap and chunks together with slopes: the slope's loss comes after the cap"""
    from zhilight_amd import seqops
    T, H, G, d, e, cap, chunk = 150, 4, 2, 24, 16, 2.0, 70
    g = torch.Generator().manual_seed(4)
    q, k, v = bf(torch.randn(T, H, d, generator=g)), bf(torch.randn(T, G, d, generator=g)), bf(torch.randn(T, G, e, generator=g))
    temp, slope = torch.tensor([0.5, 2.0, 1.0, 3.0]), torch.tensor([0.5, 0.1, 0.02, 0.3])
    i = torch.arange(T)
    dist = (i[:, None] - i[None, :]).double()
    vis = (dist >= 0) & (i[:, None] // chunk == i[None, :] // chunk)
    ref = torch.zeros(T, H, e, dtype=F64)
    for a in range(H):
        s = cap * torch.tanh((q[:, a] @ k[:, a // 2].T) * 0.3 * float(temp[a]) / cap) - float(slope[a]) * dist
        ref[:, a] = torch.softmax(s.masked_fill(~vis, -math.inf), -1) @ v[:, a // 2]
    form = seqops.score_form(H, head_scale=temp.to(dev), softcap=cap, chunk=chunk, slope=slope.to(dev))
    for mfma in (True, False):
        cache = new_cache(dev)
        kp, vp = cache.add_plane("k", (G * d,), dtype), cache.add_plane("v", (G * e,), dtype)
        out, at = [], 0
        for n in (100, 1, 49):
            b = batch_of(cache, [("s", n)], dev)
            proj = torch.cat([t.reshape(T, -1)[at:at + n] for t in (q, k, v)], 1).float().to(dev)
            seqops.rope_norm_store(proj, 0, H * d, H * d + G * d, H, G, d, e, None, 0, None, EPS, False, b, kp, vp)
            acc, ml, ns = seqops.window_attention(proj, 0, kp, vp, b, 0.3, 0, H, G, d, e, all_kv=False, mfma=mfma, form=form)
            out.append(seqops.head_mix_gate(acc, ml, ns, None, None, None, 0, b, H, G, e, torch.float32))
            at += n
        assert_close(torch.cat(out).reshape(T, -1), ref.reshape(T, -1), dtype, mfma)


def test_whole_row_norm_temperature_and_further_heads(dev):
    """one launch: a norm over all query heads and one over all key heads, weights per number, the temperature's steps (position p counts
    p + 1), other heads of the same rows rotated in place -- the columns between untouched; and the whole-row norm before a rotation"""
    from zhilight_amd import mixers, seqops
    T, H, G, d, e, every, coef = 90, 3, 2, 20, 12, 29, 0.7
    XH, xd, xrot = 4, 14, 8
    g = torch.Generator().manual_seed(12)
    nq, nk, nv, nx = H * d, G * d, G * e, XH * xd
    rows = torch.randn(T, nq + nk + nv + nx + 5, generator=g)
    rows[:, nq:nq + nk] *= 2.5
    qw, kw = 1.0 + 0.3 * torch.randn(nq, generator=g), 1.0 + 0.3 * torch.randn(nk, generator=g)
    freq = mixers.rotary_frequencies(xrot, 300.0, 1.0, dev)
    for rot in (0, 12):
        qk_freq = mixers.rotary_frequencies(rot, 70.0, 1.0, dev) if rot else None
        prep = seqops.head_prep(True, qw.to(dev), kw.to(dev), (coef, every), (nq + nk + nv, XH, xd, xrot, freq))
        cache = new_cache(dev)
        kp, vp = cache.add_plane("k", (nk,), torch.float32), cache.add_plane("v", (nv,), torch.float32)
        b = batch_of(cache, [("s", T)], dev)
        proj = rows.to(dev)
        seqops.rope_norm_store(proj, 0, nq, nq + nk, H, G, d, e, qk_freq, rot, None, EPS, False, b, kp, vp, prep=prep)
        q = O.rms_norm(rows[:, :nq].double(), qw.double(), EPS).reshape(T, H, d)
        k = O.rms_norm(rows[:, nq:nq + nk].double(), kw.double(), EPS).reshape(T, G, d)
        q, k = O.rotate_half(q, rot, 70.0), O.rotate_half(k, rot, 70.0)
        q = q * O.query_temperature(T, coef, every)[:, None, None]
        x = O.rotate_half(rows[:, nq + nk + nv:-5].double().reshape(T, XH, xd), xrot, 300.0)
        assert rel(proj[:, :nq], q.reshape(T, -1)) < 2e-6 and rel(proj[:, nq + nk + nv:-5], x.reshape(T, -1)) < 2e-6
        assert torch.equal(proj[:, nq:nq + nk + nv].cpu(), rows[:, nq:nq + nk + nv]) and torch.equal(proj[:, -5:].cpu(), rows[:, -5:])
        assert rel(kp[:2].reshape(128, -1)[:T], k.reshape(T, -1)) < 2e-6
        for p in (every - 2, every - 1, every, 2 * every - 2, 2 * every - 1):          # around the steps, position by position
            assert rel(proj[p, :nq], q[p].reshape(-1)) < 2e-6, p
        assert torch.equal(vp[0].reshape(nv, 64).t().cpu(), rows[:64, nq + nk:nq + nk + nv])
    t = O.query_temperature(T, coef, every)
    assert float(t[every - 2]) == 1.0 and float(t[every - 1]) > 1.4                    # (the step shows)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rh,rd,rv,rot", [(3, 24, 20, 16), (1, 10, 7, 6), (2, 64, 48, 64), (4, 33, 130, 0)])
def test_retention_alone_in_portions_and_segments(dev, dtype, rh, rd, rv, rot):
    """rotated queries and keys, a fixed decay per head (one close to 1 with a far token that stands out), the norm per head"""
    from zhilight_amd.mixers import DecayLinearAttention
    W, T = 96, 230
    layer = parallel_cfg(rh=rh, rd=rd, rv=rv, rot=rot, decay=[0.998046875, 0.875, 0.984375, 1.0][:rh])
    m = layer["mixer"]["right"]
    sd = O.random_weights(model_cfg([layer], loop=None), 15, fixed_choice=True)
    h = bf(torch.randn(T, W, generator=torch.Generator().manual_seed(16)))
    h[3] *= 6.0
    ref = O.right_branch(h, sd, "l0.mix.right.", m, EPS)
    h0 = h.clone()
    h0[3] = h[4]
    assert rel(O.right_branch(h0, sd, "l0.mix.right.", m, EPS)[200:], ref[200:]) > 0.02           # token 3 still shows two hundred tokens later
    for portions, seg in (([T], None), ([T], 32), ([1] * 7 + [2, 3, 60, 1, 1, 156], 64), ([100] + [1] * 130, None)):
        cache = new_cache(dev)
        mix = DecayLinearAttention("r", W, rh, rd, rv, m["decay"], EPS, act=None, norm_groups=rh, norm_weight=False, gate_act="silu", rot_dims=rot,
                                   rot_base=m["rot"]["base"], key_scale=rd ** -0.5).load(lambda n: sd[n], "l0.mix.right.", dtype, dev)
        mix.scan_segment = seg
        mix.bind(cache, dtype)
        out, at = [], 0
        for n in portions:
            out.append(mix.forward(h[at:at + n].to(dtype).to(dev).contiguous(), batch_of(cache, [("s", n)], dev)))
            at += n
        assert_close(torch.cat(out), ref, dtype, (portions[:3], seg))


@pytest.mark.parametrize("dtype", DTYPES)
def test_parallel_mixers_in_portions(dev, dtype):
    W, T = 96, 200
    for layer in (parallel_cfg(), parallel_cfg(heads=6, kv_heads=6, dim=16, vdim=48, every=64, rh=1, rd=40, rv=16, rot=40)):
        sd = O.random_weights(model_cfg([layer], loop=None), 5, fixed_choice=True)
        h = bf(torch.randn(T, W, generator=torch.Generator().manual_seed(6)))
        ref = O.parallel_mixer(h, sd, "l0.mix.", layer["mixer"], EPS)
        plain = dict(layer["mixer"], left=dict(layer["mixer"]["left"], q_temp=None))
        assert rel(O.parallel_mixer(h, sd, "l0.mix.", plain, EPS), ref) > 0.01                      # the temperature shows
        unbiased = dict(sd, **{f"l0.mix.left.{n}.b": torch.zeros_like(sd[f"l0.mix.left.{n}.b"]) for n in "qkv"})
        assert rel(O.parallel_mixer(h, unbiased, "l0.mix.", layer["mixer"], EPS), ref) > 0.05
        for portions in ([T], [1] * 6 + [2, 3, 61, 64, 1, 1, 62], [36, 1, 1, 162]):
            cache = new_cache(dev)
            mix = build_mixer(layer, sd, "l0.mix.", W, dtype, dev, cache)
            cache.admit("s")
            assert_close(feed(mix, cache, h.to(dtype), portions, dev), ref, dtype, portions[:2])


@pytest.mark.parametrize("experts,top", [(12, 3), (5, 1), (6, 6), (64, 8), (100, 2)])
def test_router_choice_among_the_logits(dev, experts, top):
    from zhilight_amd import seqops
    W, T = 64, 200
    g = torch.Generator().manual_seed(experts)
    h = bf(torch.randn(T, W, generator=g))
    sd = {"router": bf(torch.randn(experts, W, generator=g)), "router.b": bf(torch.randn(experts, generator=g) * 2.0)}
    sd["router"][0] *= 40.0                                                     # (logits hundreds apart: a softmax over all of them would underflow)
    ids_ref, w_ref = O.route(h, sd, "", top)
    logits = torch.cat([h @ sd["router"].T, torch.full((T, 7), 1e6, dtype=F64)], 1).float().to(dev)      # (other columns of wider rows)
    ids, wts = seqops.moe_route(logits, None, 1, 1, top, False, score="chosen", n_out=experts, logit_bias=sd["router.b"].float().to(dev))
    assert (ids.cpu().long() == ids_ref).all()
    assert rel(wts, w_ref) < 1e-5 and float((wts.sum(-1) - 1.0).abs().max()) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff,shared,T", [(48, 80, 1), (48, 80, 7), (48, 20, 300), (20, 33, 5), (20, 33, 130), (48, 0, 40)])
def test_experts_with_a_gated_shared_expert(dev, dtype, ff, shared, T):
    from zhilight_amd import zasazen
    f = moe(ff=ff, experts=6, top=2, shared=shared)
    if not shared:
        del f["shared"]
    W = 64
    sd = O.random_weights(model_cfg([with_mlp(mamba_cfg(), f)], width=W, loop=None), 13)
    h = bf(torch.randn(T, W, generator=torch.Generator().manual_seed(14)))
    margins = []
    O.route(h, sd, "l0.mlp.", 2, margins)
    assert margins[0] > 1e-4                                                    # (exact inputs: only a tie within fp32 sums could differ)
    ref = O.experts_ff(h, sd, "l0.mlp.", f)
    ff_ = zasazen.FF_BUILDERS["moe"](W, f).load(lambda n: sd[n], "l0.mlp.", dtype, dev)
    assert_close(ff_.forward(h.to(dev).to(dtype).contiguous()), ref, dtype, (ff, shared, T))


@pytest.mark.parametrize("dtype", DTYPES)
def test_dense_feed_forward(dev, dtype):
    from zhilight_amd import zasazen
    W, f = 72, dense(100)
    sd = O.random_weights(model_cfg([with_mlp(mamba_cfg(), f)], width=W, loop=None), 15)
    for T in (1, 5, 33, 200):
        h = bf(torch.randn(T, W, generator=torch.Generator().manual_seed(16)))
        ff_ = zasazen.FF_BUILDERS["dense"](W, f).load(lambda n: sd[n], "l0.mlp.", dtype, dev)
        assert_close(ff_.forward(h.to(dev).to(dtype).contiguous()), O.dense_ff(h, sd, "l0.mlp."), dtype, T)


# ------------------------------------------------------------------------------------------------------------------------------------
# the model through the engine
# ------------------------------------------------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def model_a():
    cfg = cfg_a()
    sd = O.random_weights(cfg, 21, fixed_choice=True)
    toks = tokens_of(cfg, 230, 22)
    logits, layers = oracle_model(cfg, sd, toks)
    return cfg, sd, toks, logits, layers


@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_prompt_and_every_layer_run(dev, dtype, model_a):
    cfg, sd, toks, logits, layers = model_a
    eng = make(cfg, sd, dtype, dev)
    assert_close(run_portions(eng, "w", toks, [len(toks)]), logits, dtype)
    b = batch_of(eng.cache, [("L", len(toks))], dev)
    got = eng.model.forward_layers(torch.tensor(toks, dtype=torch.int32, device=dev), b)
    assert len(got) == len(layers) == 6
    for i, (x, ref) in enumerate(zip(got, layers)):
        assert_close(x, ref, dtype, f"layer run {i}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_token_by_token_from_the_first_token_and_after_a_prompt(dev, dtype, model_a):
    cfg, sd, toks, logits, _ = model_a
    eng = make(cfg, sd, dtype, dev)
    assert_close(run_portions(eng, "d0", toks[:100], [1] * 100), logits[:100], dtype, "from the first token")
    assert_close(run_portions(eng, "d1", toks, [50] + [1] * 180), logits, dtype, "long decoding across page borders and temperature steps")


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
    sd = O.random_weights(cfg, 23, fixed_choice=True)
    lens = [150, 97, 201, 64, 33]
    reqs = {f"r{i}": tokens_of(cfg, n, 30 + i) for i, n in enumerate(lens)}
    refs = {k: oracle_model(cfg, sd, v)[0] for k, v in reqs.items()}
    eng = make(cfg, sd, dtype, dev, max_tokens=64 * 8, max_seqs=3)
    got = {k: [] for k in reqs}
    at = {k: 0 for k in reqs}
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
    sd = O.random_weights(cfg, 24, fixed_choice=True)
    eng = make(cfg, sd, torch.bfloat16, dev, max_tokens=64 * 4, max_seqs=2)
    a, b = tokens_of(cfg, 130, 1), tokens_of(cfg, 120, 2)
    first = run_portions(eng, "a", a, [100, 1, 29])
    run_portions(eng, "b", b, [120], release=False)
    eng.release("b")
    again = run_portions(eng, "a2", a, [100, 1, 29])
    assert torch.equal(first, again)


@pytest.mark.parametrize("dtype", DTYPES)
def test_odd_sizes_whole_in_portions_and_decoded(dev, dtype):
    cfg = cfg_odd()
    sd = O.random_weights(cfg, 25, fixed_choice=True)
    toks = tokens_of(cfg, 140, 26)
    logits, _ = oracle_model(cfg, sd, toks)
    eng = make(cfg, sd, dtype, dev)
    assert_close(run_portions(eng, "w", toks, [140]), logits, dtype, "whole")
    assert_close(run_portions(eng, "p", toks, [2, 2, 1, 60, 5, 1, 1, 68]), logits, dtype, "portions")
    assert_close(run_portions(eng, "d", toks[:70], [1] * 70), logits[:70], dtype, "decoded")


@pytest.mark.parametrize("loop", [None, (0, 1, 1), (2, 3, 1), (1, 2, 4), (0, 3, 2)])
def test_loops_at_every_place(dev, loop):
    cfg = model_cfg([with_mlp(mamba_cfg(inner=48), dense(40)), with_mlp(parallel_cfg(), dense(40)), mamba_cfg(inner=40, state=3)], loop=loop)
    sd = O.random_weights(cfg, 35)
    toks = tokens_of(cfg, 70, 36)
    logits, layers = oracle_model(cfg, sd, toks)
    eng = make(cfg, sd, torch.float32, dev)
    assert_close(run_portions(eng, "p", toks, [30, 1, 2, 37]), logits, torch.float32, loop)
    got = eng.model.forward_layers(torch.tensor(toks, dtype=torch.int32, device=dev), batch_of(eng.cache, [("L", 70)], dev))
    assert len(got) == len(layers)
    for x, ref in zip(got, layers):
        assert_close(x, ref, torch.float32, loop)


def test_router_choices_through_the_model_in_fp32(dev):
    """ordinary routers and retention matrices (close calls allowed): fp32 serving follows the restatement's choices"""
    cfg = cfg_a()
    sd = O.random_weights(cfg, 27)
    toks = tokens_of(cfg, 120, 28)
    logits, _ = oracle_model(cfg, sd, toks, fixed=False)
    eng = make(cfg, sd, torch.float32, dev)
    assert rel(run_portions(eng, "w", toks, [50, 1, 1, 68]), logits) < 1e-4


def test_medium_configuration_other_kernel_instantiations(dev):
    """head sizes up to 128, 16 heads on 4 kv heads, 600 channels of 64 states, 32 experts; long portions in segments by the default length"""
    cfg = model_cfg([with_mlp(parallel_cfg(heads=16, kv_heads=4, dim=128, vdim=64, scale=0.09, every=100, rh=4, rd=64, rv=128, rot=64), moe(ff=64, experts=32, top=4, shared=128)),
                     with_mlp(mamba_cfg(inner=600, state=64, rank=20, conv=4), dense(512))], width=256, vocab=300, loop=(0, 2, 2))
    sd = O.random_weights(cfg, 29, fixed_choice=True)
    toks = tokens_of(cfg, 420, 30)
    logits, _ = oracle_model(cfg, sd, toks)
    for dtype in DTYPES:
        eng = make(cfg, sd, dtype, dev)
        assert_close(run_portions(eng, "w", toks, [300, 1, 1, 118]), logits, dtype, "medium")


def test_greedy_generation_through_the_scheduler(dev):
    """Engine.generate under a small step budget (prompts cut into portions, decode tokens beside them) gives what feeding the restatement
    its own arg-max gives"""
    from zhilight_amd.engine import SamplingParams
    cfg = cfg_a()
    sd = O.random_weights(cfg, 31, fixed_choice=True)
    prompts = [tokens_of(cfg, n, 40 + n) for n in (40, 9, 75)]
    eng = make(cfg, sd, torch.float32, dev, max_tokens=64 * 10, max_seqs=2, max_step_tokens=48)
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=4))
    for p, out in zip(prompts, outs):
        assert len(out) == 4
        logits = O.model(list(p) + out, sd, cfg)[len(p) - 1:-1]
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
    sd = O.random_weights(cfg, 33, fixed_choice=True)
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
    la, lb, lc = O.model(a + [a[0]], sd, cfg), O.model(b, sd, cfg), O.model(c, sd, cfg)
    want = {0: torch.stack([la[0], la[59], lb[1]]), 1: torch.stack([lb[69], la[60]]), 3: torch.stack([lc[99], la[90]])}
    assert not (out / "2.f32").exists()
    for n, ref in want.items():
        got = torch.from_numpy(np.fromfile(str(out / f"{n}.f32"), dtype="<f4").reshape(ref.shape[0], cfg["vocab"]))
        assert_close(got, ref, torch.float32, f"step {n}")
