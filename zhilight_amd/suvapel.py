"""Suvapel: a decoder-only model whose mixer and feed-forward run side by side on ONE norm of the residual -- a norm that takes no statistics --
whose layers each pick one sequence mixer: a gated delta rule, or windowed attention beside a gated delta rule with a decay per key channel;
and whose layers end with a second, per-layer embedding of the token.

Shape of a layer (x is the fp32 residual; m = residual_mult):
    h = N1(x),  N(u) = tanh(alpha u) * w + b
    x = x + m * (mixer(h) + ff(h))                                   no ff term without a feed-forward
    x = x + m * R(W_proj (gelu_tanh(W_gate x) * e))                  e = the layer's dim columns of side.embed[token]; R an RMS norm with a weight
Embedding: table[token].  Output: N, then the vocabulary projection.

Configuration keys: vocab, width, norm.eps, residual_mult, token_side.dim, layers[i] = {type, mixer, mlp}:
    type "delta"       mixer: heads, kv_heads, dim, vdim, conv (taps); a decay per head, a silu gate
    type "parallel"    mixer: left_scale, right_scale, left.{heads, kv_heads, dim, vdim, conv, scale, rot.{dims, base, scaling}, mask.{size,
                       keep_first}} (attention with a sigmoid gate per head), right.{heads, kv_heads, dim, vdim, conv} (delta rule, a decay per key
                       channel and a sigmoid gate, both from low-rank pairs)
    mlp (or null)      kind "dense": ff
Tensors: embed, side.embed (vocab, layers * dim), head, final.norm, l<i>.norm1 (each with .b and .alpha), l<i>.mix.*, l<i>.mlp.*, l<i>.side.* (see
the classes in mixers.py).

The model runs RAGGED steps like the other models of the engine: every launch covers all tokens of a step; cached rows live in paged planes
of the engine's CacheManager, recurrent states and convolution tails in its slot states.  A layer is two large products (JoinedSublayers:
everything that reads h in one, everything that joins the residual in the other) with the mixers' kernels between, one launch that adds the
result and writes x in the serving format, two small products of the side input, and one launch that adds it and writes the next norm.
"""
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from . import seqops
from ._lib import ZLError
from .mixers import GatedDeltaRule, GatedFF, JoinedSublayers, TokenSideInput, WindowAttention, _mat, _rand, _vec
from .registry import register_model

_DTYPES = {"bfloat16": torch.bfloat16, "bf16": torch.bfloat16, "float32": torch.float32, "fp32": torch.float32,
           torch.bfloat16: torch.bfloat16, torch.float32: torch.float32}


@dataclass
class SuvapelLayerConfig:
    type: str
    mixer: dict
    mlp: Optional[dict]


@dataclass
class SuvapelConfig:
    vocab: int
    width: int
    eps: float
    residual_mult: float
    side_dim: int                         # 0: no per-layer token input
    max_positions: int
    layers: List[SuvapelLayerConfig] = field(default_factory=list)

    @classmethod
    def from_dict(cls, cfg):
        try:
            layers = [SuvapelLayerConfig(l["type"], dict(l["mixer"]), None if l.get("mlp") is None else dict(l["mlp"])) for l in cfg["layers"]]
            side = cfg.get("token_side")
            c = cls(int(cfg["vocab"]), int(cfg["width"]), float(cfg["norm"]["eps"]), float(cfg.get("residual_mult", 1.0)),
                    0 if side is None else int(side["dim"]), int(cfg.get("max_positions", 1 << 24)), layers)      # (positions are fp32: exact to 2^24)
        except KeyError as e:
            raise ZLError(f"Suvapel config: missing key {e}")
        for i, l in enumerate(c.layers):
            if l.type not in MIXER_BUILDERS:
                raise ZLError(f"Suvapel config: layer {i}: unknown mixer type {l.type!r}")
            if l.mlp is not None and l.mlp.get("kind") != "dense":
                raise ZLError(f"Suvapel config: layer {i}: unknown feed-forward kind {l.mlp.get('kind')!r}")
        return c


def _delta(name, width, m, eps):
    """[(tensor prefix, part, scale)]"""
    return [("mix.", GatedDeltaRule(name, width, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), int(m["conv"]), eps), 1.0)]


def _parallel(name, width, m, eps):
    a, r = m["left"], m["right"]
    rot, mask = a.get("rot") or {}, a.get("mask") or {}
    left = WindowAttention(name + ".left", width, int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"]), float(a["scale"]),
                           int(mask.get("size", 0)), int(rot.get("dims", 0)), float(rot.get("base", 10000.0)), rot.get("scaling") or 1.0, eps,
                           qk_norm=False, rotate_values=False, talk=False, gate=False, head_gate=True, conv_taps=int(a.get("conv", 0)),
                           keep_first=int(mask.get("keep_first", 0)))
    right = GatedDeltaRule(name + ".right", width, int(r["heads"]), int(r["kv_heads"]), int(r["dim"]), int(r["vdim"]), int(r["conv"]), eps,
                           decay="channel", gate="lowrank", gate_act="sigmoid")
    return [("mix.left.", left, float(m["left_scale"])), ("mix.right.", right, float(m["right_scale"]))]


MIXER_BUILDERS = {"delta": _delta, "parallel": _parallel}


class TanhNorm:
    """tanh(alpha x) * w + b; tensors <name>, <name>.b (width), <name>.alpha (a number)"""

    def __init__(self, width):
        self.width = width

    def load(self, get, name, device):
        self.w, self.b = _vec(get, name, self.width, device), _vec(get, name + ".b", self.width, device)
        self.alpha = float(get(name + ".alpha").to(torch.float32).reshape(()))
        return self

    def init_random(self, gen, device):
        self.w, self.b = 1.0 + 0.1 * torch.randn(self.width, generator=gen, device=device), 0.1 * torch.randn(self.width, generator=gen, device=device)
        self.alpha = 0.7
        return self


class SuvapelLayer:
    def __init__(self, idx, cfg: SuvapelConfig, lc: SuvapelLayerConfig):
        self.idx, self.name = idx, f"l{idx}"
        parts = MIXER_BUILDERS[lc.type](self.name + ".mix", cfg.width, lc.mixer, cfg.eps)
        if lc.mlp is not None:
            parts.append(("mlp.", GatedFF(cfg.width, int(lc.mlp["ff"]), act="silu", bias=True), 1.0))
        self.norm1, self.sub = TanhNorm(cfg.width), JoinedSublayers(cfg.width, parts)
        self.side = TokenSideInput(cfg.width, cfg.side_dim, idx * cfg.side_dim) if cfg.side_dim else None

    def load(self, get, dtype, device):
        self.norm1.load(get, self.name + ".norm1", device)
        self.sub.load(get, self.name + ".", dtype, device)
        if self.side is not None:
            self.side.load(get, self.name + ".side.", dtype, device)

    def init_random(self, gen, dtype, device):
        self.norm1.init_random(gen, device)
        self.sub.init_random(gen, dtype, device)
        if self.side is not None:
            self.side.init_random(gen, dtype, device)

    def weight_bytes(self):
        return self.sub.weight_bytes() + (self.side.weight_bytes() if self.side is not None else 0)


@register_model("Suvapel")
class SuvapelModel:
    ragged = True                    # the engine drives it with RaggedBatch steps and a CacheManager

    def __init__(self, cfg: SuvapelConfig, dtype="bfloat16", device="cuda:0"):
        if dtype not in _DTYPES:
            raise ZLError(f"Suvapel serves in bfloat16 or float32, not {dtype}")
        self.cfg, self.dtype, self.device = cfg, _DTYPES[dtype], torch.device(device)
        self.layers = [SuvapelLayer(i, cfg, lc) for i, lc in enumerate(cfg.layers)]
        self.final_norm = TanhNorm(cfg.width)
        self.embed = self.side_embed = self.head = None
        self.page_size = 64

    @classmethod
    def from_config(cls, cfg: dict, dtype="bfloat16", device="cuda:0"):
        return cls(SuvapelConfig.from_dict(cfg), dtype, device)

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
        if c.side_dim:
            self.side_embed = _mat(get, "side.embed", (c.vocab, len(c.layers) * c.side_dim), dt, dev)
        self.final_norm.load(get, "final.norm", dev)
        for layer in self.layers:
            layer.load(get, dt, dev)
        return self

    def init_random(self, seed=0):
        c, dev, dt = self.cfg, self.device, self.dtype
        gen = torch.Generator(device=dev).manual_seed(seed)
        self.embed = _rand(gen, (c.vocab, c.width), 1.0, dt, dev)
        self.head = _rand(gen, (c.vocab, c.width), c.width ** -0.5, dt, dev)
        if c.side_dim:
            self.side_embed = _rand(gen, (c.vocab, len(c.layers) * c.side_dim), 1.0, dt, dev)
        self.final_norm.init_random(gen, dev)
        for layer in self.layers:
            layer.init_random(gen, dt, dev)
        return self

    def bind_cache(self, cache):
        """register every layer's per-token planes and per-sequence states with the engine's cache manager"""
        if cache.page_size != self.page_size:
            raise ZLError("cache page size mismatch")
        for layer in self.layers:
            layer.sub.bind(cache, self.dtype)
        return cache

    def _run(self, tokens, batch, keep=None):
        c, dt, m = self.cfg, self.dtype, self.cfg.residual_mult
        x = seqops.embed(tokens, self.embed, None, 1.0, batch)

        def join(branch, norm):
            """x += the branch; N(x) of the next norm"""
            h = seqops.add_branches(x, branch, c.eps, dt, None if norm is None else norm.w, tanh=None if norm is None else (norm.alpha, norm.b))[0]
            if keep is not None and branch:
                keep.append(x.clone())
            return h
        h = join([], self.layers[0].norm1) if self.layers else None
        for i, layer in enumerate(self.layers):
            branch = (layer.sub.forward(h, batch), None, m)
            if layer.side is not None:
                xt = x if dt == torch.float32 else torch.empty(x.shape, dtype=dt, device=x.device)
                seqops.add_branches(x, [branch], c.eps, dt, xt=None if xt is x else xt)
                branch = layer.side.branch(xt, self.side_embed, tokens, m)
            h = join([branch], self.layers[i + 1].norm1 if i + 1 < len(self.layers) else None)
        return x

    def forward(self, tokens, batch, want_rows):
        """tokens: int32 device (n_tok) in the batch's flat order; want_rows: int32 device, flat token indices whose logits are wanted
        (None or empty: the step only advances caches and states).  Returns fp32 logits (len(want_rows), vocab) or None."""
        x = self._run(tokens, batch)
        if want_rows is None or want_rows.numel() == 0:
            return None
        n = self.final_norm
        return seqops.gemm_nt(seqops.tanh_norm(x, n.w, n.b, n.alpha, self.dtype, rows=want_rows), self.head)

    def forward_layers(self, tokens, batch):
        """the residual after every layer (debugging and tests): list of fp32 (n_tok, width) copies"""
        out = []
        self._run(tokens, batch, keep=out)
        return out

    def weight_bytes(self):
        tables = [t for t in (self.embed, self.head, self.side_embed) if t is not None]
        return sum(l.weight_bytes() for l in self.layers) + sum(t.numel() * t.element_size() for t in tables)
