"""Zasazen: a decoder-only model whose mixer and feed-forward run side by side on two norms of the same residual, whose layers each pick one
sequence mixer -- a selective state space with a decay per channel and state, or attention with a linear distance bias beside a retention
layer -- and a dense or mixture-of-experts feed-forward, and some of whose layers run several times in a row with the same weights.

Shape of a layer (x is the fp32 residual; N = RMS norm with a plain weight, u / sqrt(mean(u^2) + eps) * w):
    x = x + (mixer(N1(x)) + ff(N2(x)))          both read the same x; no N2 without a feed-forward
Embedding: x0 = table[token] * embedding.scale.  Layers loop.start .. loop.stop - 1 run loop.times times; right before the first of them, in
pass t, x = W_in [x; x0] + step[t].  Every pass has a cache and states of its own.  Output: N, then the vocabulary projection.

Configuration keys: vocab, width, embedding.scale, norm.eps, loop.{start, stop, times} (or none), layers[i] = {type, mixer, mlp}:
    type "mamba1"      mixer: inner, state, dt_rank, conv (taps)
    type "parallel"    mixer: left.{heads, kv_heads, dim, vdim, scale, q_temp.{coef, every}}, right.{heads, dim, vdim, decay, rot.{dims, base}}
    mlp (or null)      kind "dense": ff;  kind "moe": expert.ff, router.{experts, top}, shared.ff (or no shared expert)
Tensors: embed, head, final.norm, loop.in (width, 2 width), loop.step (times, width), l<i>.norm1 / norm2, l<i>.mix.*, l<i>.mlp.* (see the
mixer classes in mixers.py).

The model runs RAGGED steps like the other models of the engine: every launch covers all tokens of a step; cached rows live in paged planes
of the engine's CacheManager, recurrent states and convolution tails in its slot states.  One launch (seqops.add_branches) sums the results
that ran side by side into the residual and writes what is read next: both norms of the new row, or its copy for the product at the loop's
entry.
"""
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from . import seqops
from ._lib import ZLError
from .mixers import DecayLinearAttention, Mamba1Mixer, ParallelMixers, PlainFF, RoutedExpertsFF, WindowAttention, _mat, _rand, _vec, replica
from .registry import register_model

_DTYPES = {"bfloat16": torch.bfloat16, "bf16": torch.bfloat16, "float32": torch.float32, "fp32": torch.float32,
           torch.bfloat16: torch.bfloat16, torch.float32: torch.float32}


@dataclass
class ZasazenLayerConfig:
    type: str
    mixer: dict
    mlp: Optional[dict]


@dataclass
class ZasazenConfig:
    vocab: int
    width: int
    embedding_scale: float
    eps: float
    loop: Optional[tuple]                 # (start, stop, times)
    max_positions: int
    layers: List[ZasazenLayerConfig] = field(default_factory=list)

    @classmethod
    def from_dict(cls, cfg):
        try:
            layers = [ZasazenLayerConfig(l["type"], dict(l["mixer"]), None if l.get("mlp") is None else dict(l["mlp"])) for l in cfg["layers"]]
            loop = cfg.get("loop")
            if loop is not None:
                loop = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
            c = cls(int(cfg["vocab"]), int(cfg["width"]), float(cfg["embedding"]["scale"]), float(cfg["norm"]["eps"]), loop,
                    int(cfg.get("max_positions", 1 << 24)), layers)                       # (positions are fp32: exact to 2^24)
        except KeyError as e:
            raise ZLError(f"Zasazen config: missing key {e}")
        if loop is not None and not (0 <= loop[0] < loop[1] <= len(layers) and loop[2] >= 1):
            raise ZLError("Zasazen config: the loop must cover at least one of the layers, at least once")
        for i, l in enumerate(c.layers):
            if l.type not in MIXER_BUILDERS:
                raise ZLError(f"Zasazen config: layer {i}: unknown mixer type {l.type!r}")
            if l.mlp is not None and l.mlp.get("kind") not in FF_BUILDERS:
                raise ZLError(f"Zasazen config: layer {i}: unknown feed-forward kind {l.mlp.get('kind')!r}")
        return c

    def runs(self):
        """[(layer, pass)] in the order of execution; layers outside the loop have the one pass 0"""
        n = len(self.layers)
        a, b, times = self.loop if self.loop is not None else (0, 0, 0)
        return [(i, 0) for i in range(a)] + [(i, t) for t in range(times) for i in range(a, b)] + [(i, 0) for i in range(b, n)]

    def passes(self, i):
        return self.loop[2] if self.loop is not None and self.loop[0] <= i < self.loop[1] else 1


def _mamba1(name, width, m, eps):
    return Mamba1Mixer(name, width, int(m["inner"]), int(m["state"]), int(m["dt_rank"]), int(m["conv"]))


def _parallel(name, width, m, eps):
    a, r = m["left"], m["right"]
    temp, rot = a.get("q_temp"), r.get("rot") or {}
    left = WindowAttention(name + ".left", width, int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"]), float(a["scale"]), 0, 0, 10000.0,
                           1.0, eps, qk_norm=False, rotate_values=False, talk=False, gate=False, bias=True, whole_norm=True,
                           q_temp=None if temp is None else (float(temp["coef"]), int(temp["every"])), slope_bias=True)
    H = int(r["heads"])
    right = DecayLinearAttention(name + ".right", width, H, int(r["dim"]), int(r["vdim"]), list(r["decay"]), eps, act=None, norm_groups=H,
                                 norm_weight=False, gate_act="silu", rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 10000.0)),
                                 key_scale=int(r["dim"]) ** -0.5)
    return ParallelMixers(name, left, right, coef=0.5)


MIXER_BUILDERS = {"mamba1": _mamba1, "parallel": _parallel}


def _dense(width, f):
    return PlainFF(width, int(f["ff"]), act="gelu_tanh")


def _experts(width, f):
    r, shared = f["router"], f.get("shared")
    return RoutedExpertsFF(width, int(f["expert"]["ff"]), int(r["experts"]), int(r["top"]), correction=False, score="chosen", act="silu",
                           router_bias=True, shared_ff=0 if shared is None else int(shared["ff"]), shared_gate=shared is not None)


FF_BUILDERS = {"dense": _dense, "moe": _experts}


class ZasazenLayer:
    def __init__(self, idx, cfg: ZasazenConfig, lc: ZasazenLayerConfig):
        self.idx, self.name, self.width, self.n_passes = idx, f"l{idx}", cfg.width, cfg.passes(idx)
        self.mixer = MIXER_BUILDERS[lc.type](self.name + ".mix", cfg.width, lc.mixer, cfg.eps)
        self.ff = FF_BUILDERS[lc.mlp["kind"]](cfg.width, lc.mlp) if lc.mlp is not None else None
        self.norm1 = self.norm2 = None
        self.passes = []                  # the mixer once per pass: the same weights, caches and states of their own

    def load(self, get, dtype, device):
        self.norm1 = _vec(get, self.name + ".norm1", self.width, device)
        self.mixer.load(get, self.name + ".mix.", dtype, device)
        if self.ff is not None:
            self.norm2 = _vec(get, self.name + ".norm2", self.width, device)
            self.ff.load(get, self.name + ".mlp.", dtype, device)
        self._replicate()

    def init_random(self, gen, dtype, device):
        self.norm1 = 1.0 + 0.1 * torch.randn(self.width, generator=gen, device=device)
        self.mixer.init_random(gen, dtype, device)
        if self.ff is not None:
            self.norm2 = 1.0 + 0.1 * torch.randn(self.width, generator=gen, device=device)
            self.ff.init_random(gen, dtype, device)
        self._replicate()

    def _replicate(self):
        self.passes = [self.mixer] + [replica(self.mixer, f"{self.name}.mix.pass{t}") for t in range(1, self.n_passes)]

    def forward(self, h1, h2, batch, t):
        """the layer's results in pass t, as the branches that join the residual together"""
        out = self.passes[t].branches(h1, batch)
        if self.ff is not None:
            out.append((self.ff.forward(h2), None, 1.0))
        return out

    def weight_bytes(self):
        return self.mixer.weight_bytes() + (self.ff.weight_bytes() if self.ff is not None else 0)


@register_model("Zasazen")
class ZasazenModel:
    ragged = True                    # the engine drives it with RaggedBatch steps and a CacheManager

    def __init__(self, cfg: ZasazenConfig, dtype="bfloat16", device="cuda:0"):
        if dtype not in _DTYPES:
            raise ZLError(f"Zasazen serves in bfloat16 or float32, not {dtype}")
        self.cfg, self.dtype, self.device = cfg, _DTYPES[dtype], torch.device(device)
        self.layers = [ZasazenLayer(i, cfg, lc) for i, lc in enumerate(cfg.layers)]
        self.final_norm = self.embed = self.head = self.loop_in = self.loop_step = None
        self.page_size = 64

    @classmethod
    def from_config(cls, cfg: dict, dtype="bfloat16", device="cuda:0"):
        return cls(ZasazenConfig.from_dict(cfg), dtype, device)

    @property
    def vocab_size(self):
        return self.cfg.vocab

    @property
    def max_positions(self):
        return self.cfg.max_positions

    def load_weights(self, ckpt):
        c, dev, dt = self.cfg, self.device, self.dtype

        def get(name):
            return ckpt[name]
        self.embed, self.head = (_mat(get, name, (c.vocab, c.width), dt, dev) for name in ("embed", "head"))
        self.final_norm = _vec(get, "final.norm", c.width, dev)
        if c.loop is not None:
            self.loop_in = _mat(get, "loop.in", (c.width, 2 * c.width), dt, dev)
            self.loop_step = _mat(get, "loop.step", (c.loop[2], c.width), torch.float32, dev)
        for layer in self.layers:
            layer.load(get, dt, dev)
        return self

    def init_random(self, seed=0):
        c, dev, dt = self.cfg, self.device, self.dtype
        gen = torch.Generator(device=dev).manual_seed(seed)
        self.embed = _rand(gen, (c.vocab, c.width), 1.0 / max(c.embedding_scale, 1e-6), dt, dev)
        self.head = _rand(gen, (c.vocab, c.width), c.width ** -0.5, dt, dev)
        self.final_norm = 1.0 + 0.1 * torch.randn(c.width, generator=gen, device=dev)
        if c.loop is not None:
            self.loop_in = _rand(gen, (c.width, 2 * c.width), (2 * c.width) ** -0.5, dt, dev)
            self.loop_step = _rand(gen, (c.loop[2], c.width), 0.1, torch.float32, dev)
        for layer in self.layers:
            layer.init_random(gen, dt, dev)
        return self

    def bind_cache(self, cache):
        """register every pass's per-token planes and per-sequence states with the engine's cache manager"""
        if cache.page_size != self.page_size:
            raise ZLError("cache page size mismatch")
        for layer in self.layers:
            for mixer in layer.passes:
                mixer.bind(cache, self.dtype)
        return cache

    def _run(self, tokens, batch, keep=None):
        c = self.cfg
        W = c.width
        x = seqops.embed(tokens, self.embed, None, c.embedding_scale, batch)
        runs = c.runs()
        if c.loop is not None:                                 # [x | x0] in the serving format: what the product at the loop's entry reads
            entry = torch.empty((batch.n_tok, 2 * W), dtype=self.dtype, device=x.device)
            seqops.add_branches(x, [], c.eps, self.dtype, xt=entry[:, W:])
        branches = []
        for i, t in runs:
            layer = self.layers[i]
            if c.loop is not None and i == c.loop[0]:
                seqops.add_branches(x, branches, c.eps, self.dtype, xt=entry[:, :W])
                self._keep(keep, x, branches)
                x, branches = seqops.gemm_nt(entry, self.loop_in, bias=self.loop_step[t]), []
            h1, h2 = seqops.add_branches(x, branches, c.eps, self.dtype, layer.norm1, layer.norm2)
            self._keep(keep, x, branches)
            branches = layer.forward(h1, h2, batch, t)
        if branches:
            seqops.add_branches(x, branches, c.eps, self.dtype)
            self._keep(keep, x, branches)
        return x

    @staticmethod
    def _keep(keep, x, branches):
        if keep is not None and branches:
            keep.append(x.clone())

    def forward(self, tokens, batch, want_rows):
        """tokens: int32 device (n_tok) in the batch's flat order; want_rows: int32 device, flat token indices whose logits are wanted
        (None or empty: the step only advances caches and states).  Returns fp32 logits (len(want_rows), vocab) or None."""
        x = self._run(tokens, batch)
        if want_rows is None or want_rows.numel() == 0:
            return None
        return seqops.gemm_nt(seqops.rms_norm(x, self.final_norm, self.cfg.eps, self.dtype, rows=want_rows), self.head)

    def forward_layers(self, tokens, batch):
        """the residual after every layer run (a looped layer counts in every pass; debugging and tests): list of fp32 (n_tok, width) copies"""
        out = []
        self._run(tokens, batch, keep=out)
        return out

    def weight_bytes(self):
        """bytes a step reads once; the looped layers are read once per pass"""
        extra = [self.loop_in] * (self.cfg.loop[2] if self.cfg.loop is not None else 0)
        return sum(l.weight_bytes() * l.n_passes for l in self.layers) + sum(t.numel() * t.element_size() for t in [self.embed, self.head] + extra)
