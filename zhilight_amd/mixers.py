"""Sequence mixers and feed-forwards for ragged steps: each is a weight container + the kernel sequence of its forward, with every
constant a constructor argument, so that a model description picks and sizes them (tupitar.py and retotar.py do; another design can).

A mixer's forward takes h (n_tok, width) in the serving format and the step's RaggedBatch and returns fp32 (n_tok, width).  What it keeps
between steps it registers with the CacheManager in `bind`: per-token rows as a paged plane, per-sequence state as a slot state.
All per-sequence arithmetic that must not lose bits (norms, softmax, the recurrence, its state) is fp32 inside the kernels in both serving
formats; matrices are in the serving format, small vectors fp32.
"""
import copy
import math

import torch

from . import seqops
from ._lib import ZLError


def _mat(get, name, shape, dtype, device):
    t = get(name)
    if tuple(t.shape) != tuple(shape):
        raise ZLError(f"tensor {name}: shape {tuple(t.shape)}, expected {tuple(shape)}")
    return t.to(device=device, dtype=dtype).contiguous()


def _vec(get, name, n, device):
    t = get(name)
    if t.numel() != n:
        raise ZLError(f"tensor {name}: {t.numel()} values, expected {n}")
    return t.to(device=device, dtype=torch.float32).reshape(n).contiguous()


def _rand(gen, shape, std, dtype, device):
    return (torch.randn(shape, generator=gen, device=device, dtype=torch.float32) * std).to(dtype)


def replica(mixer, name):
    """The same mixer -- the same weight tensors -- under another name: once bound it keeps a cache or state of its own.  For layers that run
    several times over a sequence with shared weights."""
    m = copy.copy(mixer)
    m.name = name
    for part in getattr(mixer, "parts", ()):
        setattr(m, part, replica(getattr(mixer, part), name + "." + part))
    return m


class SideRows:
    """Mixers and feed-forwards whose first step is ONE product over their input can carry more rows in it for their caller: a layer that
    needs another projection of the same input (a gate of the sub-layer's result, say) attaches its matrix after load / init_random and
    finds the fp32 outputs in `side` = (tensor, first column) after forward -- one launch and one pass over the input less."""
    side = None
    side_col0 = None
    _side_matrix = "w_in"

    def attach_side(self, w):
        m = getattr(self, self._side_matrix)
        if w.shape[1] != m.shape[1] or w.dtype != m.dtype:
            raise ZLError("side rows must have the input projection's width and format")
        self.side_col0 = m.shape[0]
        setattr(self, self._side_matrix, torch.cat([m, w], dim=0).contiguous())


class LatentAttention(SideRows):
    """Causal attention whose keys and values are up-projections of a cached, RMS-normed low-rank latent; optional learned per-head sink in
    the softmax denominator, per-head sigmoid output gate, sliding window (`window` > 0: position p sees p - window < j <= p), and a
    ROTATED part: with rot_dim > 0 every query head has rot_dim more coordinates behind its `dim` unrotated ones, the down-projection
    rot_dim more rows behind the latent -- one key part shared by all heads -- and both are turned by the position (neighbouring pairs
    (2i, 2i + 1), angle p * rot_base^(-2i / rot_dim)); score = (q_plain . k_plain + q_rot . k_rot) * scale.  The cached row is [latent |
    rotated key part]; the up-projections are widened on the host (identity columns in uk, zeros in uv), so the kernels see one latent of
    rank + rot_dim numbers and heads of dim + rot_dim.  rot_layout "half" pairs coordinate i with i + rot_dim / 2 instead of its
    neighbour; rot_scaling {factor, original, fast, slow} rescales the frequencies for contexts longer than `original` (scaled_frequencies).
    Tensors under `prefix`: q (heads*(dim+rot_dim), width), dkv (rank+rot_dim, width), dkv.norm (rank), uk (heads*dim, rank), uv (heads*vdim,
    rank), sink (heads), g (heads, width), o (width, heads*vdim).  q | dkv | g are fused into one product."""

    def __init__(self, name, width, heads, dim, vdim, rank, scale, eps, sink=True, gate=True, rot_dim=0, rot_base=10000.0, window=0,
                 rot_layout="pairs", rot_scaling=None):
        if rot_dim % 2 or rot_dim < 0 or window < 0 or rot_layout not in ("pairs", "half"):
            raise ZLError("latent attention: the rotated part is even, the window not negative, the layout pairs or half")
        self.rot_layout, self.rot_scaling, self.rot_gain = rot_layout, (dict(rot_scaling) if rot_scaling else None), 1.0
        self.name, self.width, self.heads, self.dim, self.vdim, self.rank = name, width, heads, dim, vdim, rank
        self.scale, self.eps, self.has_sink, self.has_gate = float(scale), float(eps), sink, gate
        self.rot, self.rot_base, self.window = int(rot_dim), float(rot_base), int(window)
        self.qdim, self.row = dim + self.rot, rank + self.rot      # a query head's size; a cached row's size
        self.cache = None
        self.prompt_kernel = True         # bf16 portions on the matrix-core kernel (False: everything on the latent-space kernel)
        self.decode_mfma = True           # bf16 single tokens: the split pass on the matrix cores (False: the fp32 VALU kernel)

    def _widen(self, uk, uv):
        """the up-projections over the cached row [latent | rotated key part]: a head's keys are [W_uk,h c | k_rot] (identity columns pass
        the shared part through, exactly: 1.0 times a number, summed with zeros), its values ignore the part (zero columns)"""
        H, d, v, r, t = self.heads, self.dim, self.vdim, self.rank, self.rot
        if t == 0:
            return uk.contiguous(), uv.contiguous()
        k2 = torch.zeros((H, d + t, r + t), dtype=uk.dtype, device=uk.device)
        k2[:, :d, :r] = uk.reshape(H, d, r)
        k2[:, d:, r:] = torch.eye(t, dtype=uk.dtype, device=uk.device)
        v2 = torch.zeros((H * v, r + t), dtype=uv.dtype, device=uv.device)
        v2[:, :r] = uv
        return k2.reshape(H * (d + t), r + t).contiguous(), v2.contiguous()

    def load(self, get, prefix, dtype, device):
        H, d, v, r, W = self.heads, self.dim, self.vdim, self.rank, self.width
        parts = [_mat(get, prefix + "q", (H * self.qdim, W), dtype, device), _mat(get, prefix + "dkv", (self.row, W), dtype, device)]
        if self.has_gate:
            parts.append(_mat(get, prefix + "g", (H, W), dtype, device))
        self.w_in = torch.cat(parts, dim=0).contiguous()
        self.dkv_norm = _vec(get, prefix + "dkv.norm", r, device)
        self.w_uk, self.w_uv = self._widen(_mat(get, prefix + "uk", (H * d, r), dtype, device), _mat(get, prefix + "uv", (H * v, r), dtype, device))
        self.sink = _vec(get, prefix + "sink", H, device) if self.has_sink else None
        self.w_o = _mat(get, prefix + "o", (W, H * v), dtype, device)
        self._tables(device)
        return self

    def _tables(self, device):
        self.freq = None
        if self.rot:
            self.freq, self.rot_gain = scaled_frequencies(self.rot, self.rot_base, self.rot_scaling, device)

    def init_random(self, gen, dtype, device):
        H, d, v, r, W = self.heads, self.dim, self.vdim, self.rank, self.width
        self.w_in = _rand(gen, (H * self.qdim + self.row + (H if self.has_gate else 0), W), W ** -0.5, dtype, device)
        self.dkv_norm = torch.ones(r, device=device)
        self.w_uk, self.w_uv = self._widen(_rand(gen, (H * d, r), r ** -0.5, dtype, device), _rand(gen, (H * v, r), r ** -0.5, dtype, device))
        self.sink = torch.zeros(H, device=device) if self.has_sink else None
        self.w_o = _rand(gen, (W, H * v), (H * v) ** -0.5, dtype, device)
        self._tables(device)
        return self

    def bind(self, cache, dtype):
        self.cache = cache.add_plane(self.name + ".latent", (self.row,), dtype)

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.w_uk, self.w_uv, self.w_o))

    def forward(self, h, batch):
        H, d, r = self.heads, self.qdim, self.row                                # (sizes as the kernels see them: with the rotated part)
        proj = seqops.gemm_nt(h, self.w_in)                                       # fp32 [q | latent, rotated key part | gate]
        self.side = (proj, self.side_col0)
        seqops.latent_store(proj, H * d, self.dkv_norm, self.eps, self.rank, batch, self.cache, rot=self.rot, freq=self.freq,
                            interleaved=self.rot_layout == "pairs", q_col0=0, heads=H, qdim=d, rot_gain=self.rot_gain)
        gate = proj if self.has_gate else None
        prompt = batch.n_ctx > 0 and self.prompt_kernel and h.dtype == torch.bfloat16 and max(d, self.vdim) <= 256
        a = torch.empty((batch.n_tok, H * self.vdim), dtype=h.dtype, device=h.device)
        if prompt:
            # portions: keys and values of their contexts (as far back as the window reaches) up-projected once (K = C W_uk^T, V^T = W_uv C^T,
            # gathered from the pages), then the matrix-core kernel; single tokens stay on the latent-space kernel below
            _, _, ctx_rows, n_ctx = batch.context(self.window)
            flat = self.cache.view(-1, r)
            k = torch.empty((n_ctx, H * d), dtype=h.dtype, device=h.device)
            vt = torch.empty((H * self.vdim, n_ctx), dtype=h.dtype, device=h.device)
            seqops.gemm_nt_gather(flat, ctx_rows, self.w_uk, None, n_ctx, H * d, k)
            seqops.gemm_nt_gather(self.w_uv, None, flat, ctx_rows, H * self.vdim, n_ctx, vt)
            seqops.latent_attention_prompt(proj, 0, gate, H * d + r, k, vt, self.sink, batch, self.scale, H, d, self.vdim, a, window=self.window)
        if not prompt or batch.n_single:
            seqops.latent_attention(proj, 0, gate, H * d + r, self.w_uk, self.w_uv, self.sink, self.cache, batch, self.scale, H, d, self.vdim,
                                    out=a, single_only=prompt, mfma=self.decode_mfma, window=self.window)
        return seqops.gemm_nt(a, self.w_o)


class Mamba2Mixer:
    """Selective state-space mixer (scalar decay per head, state n_state x vdim per head, B / C shared by the heads of a group), with the
    causal short convolution over x | B | C, the skip term, and the gated grouped RMS norm before the output projection.
    Tensors under `prefix`: in (2*inner + 2*groups*n_state + heads, width) laid out [z | x | B | C | dt], conv (channels, taps), conv.b,
    dt_bias, A_log, D (heads each), norm (inner), o (width, inner)."""

    def __init__(self, name, width, heads, vdim, n_state, groups, taps, norm_groups, eps):
        if heads % groups or (heads * vdim) % norm_groups:
            raise ZLError("mamba2: heads must divide by groups, heads * vdim by norm_groups")
        self.name, self.width, self.heads, self.vdim, self.n_state, self.groups = name, width, heads, vdim, n_state, groups
        self.taps, self.norm_groups, self.eps = taps, norm_groups, float(eps)
        self.inner = heads * vdim
        self.channels = self.inner + 2 * groups * n_state
        self.scan_segment = None          # tokens per segment of a long portion (None: seqops.scan_segment; 0: never in segments)

    def load(self, get, prefix, dtype, device):
        W = self.width
        self.w_in = _mat(get, prefix + "in", (self.inner + self.channels + self.heads, W), dtype, device)
        self.conv_w = _mat(get, prefix + "conv", (self.channels, self.taps), torch.float32, device)
        self.conv_b = _vec(get, prefix + "conv.b", self.channels, device)
        self.dt_bias = _vec(get, prefix + "dt_bias", self.heads, device)
        self.a_log = _vec(get, prefix + "A_log", self.heads, device)
        self.d = _vec(get, prefix + "D", self.heads, device)
        self.norm_w = _vec(get, prefix + "norm", self.inner, device)
        self.w_o = _mat(get, prefix + "o", (W, self.inner), dtype, device)
        return self

    def init_random(self, gen, dtype, device):
        W = self.width
        self.w_in = _rand(gen, (self.inner + self.channels + self.heads, W), W ** -0.5, dtype, device)
        self.conv_w = _rand(gen, (self.channels, self.taps), 0.5, torch.float32, device)
        self.conv_b = torch.zeros(self.channels, device=device)
        self.dt_bias = torch.zeros(self.heads, device=device)
        self.a_log = torch.zeros(self.heads, device=device)
        self.d = torch.ones(self.heads, device=device)
        self.norm_w = torch.ones(self.inner, device=device)
        self.w_o = _rand(gen, (W, self.inner), self.inner ** -0.5, dtype, device)
        return self

    def bind(self, cache, dtype):
        self.tail = cache.add_state(self.name + ".conv", (self.taps - 1, self.channels)) if self.taps > 1 else None
        self.state = cache.add_state(self.name + ".ssm", (self.heads, self.n_state, self.vdim))

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.w_o))

    def forward(self, h, batch):
        proj = seqops.gemm_nt(h, self.w_in)                                       # fp32 [z | x | B | C | dt]
        xbc = seqops.conv_silu(proj, self.inner, self.conv_w, self.conv_b, self.tail, batch)
        y = seqops.ssm_scan(xbc, proj, self.inner + self.channels, self.dt_bias, self.a_log, self.d, self.state, self.heads, self.vdim,
                            self.n_state, self.groups, batch, seg_len=self.scan_segment)
        g = seqops.gated_group_norm(y, proj, 0, self.norm_w, self.eps, self.norm_groups, h.dtype)
        return seqops.gemm_nt(g, self.w_o)


class PolyNormFF:
    """Dense feed-forward down(act(up h)) with the PolyNorm activation: a N(z) + b N(z^2) + c N(z^3) + e, N = division by the row's root
    mean square.  Tensors: up (ff, width), down (width, ff), act (4: a, b, c, e)."""

    def __init__(self, width, ff, eps):
        self.width, self.ff, self.eps = width, ff, float(eps)

    def load(self, get, prefix, dtype, device):
        self.w_up = _mat(get, prefix + "up", (self.ff, self.width), dtype, device)
        self.w_down = _mat(get, prefix + "down", (self.width, self.ff), dtype, device)
        self.coef = [float(v) for v in get(prefix + "act").to(torch.float32).reshape(4)]
        return self

    def init_random(self, gen, dtype, device):
        self.w_up = _rand(gen, (self.ff, self.width), self.width ** -0.5, dtype, device)
        self.w_down = _rand(gen, (self.width, self.ff), self.ff ** -0.5, dtype, device)
        self.coef = [1.0, 0.5, 0.25, 0.0]
        return self

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_up, self.w_down))

    def forward(self, h):
        z = seqops.gemm_nt(h, self.w_up)
        return seqops.gemm_nt(seqops.polynorm(z, self.coef, self.eps, h.dtype), self.w_down)


def rotary_frequencies(n_rot, base, divide=1.0, device="cpu"):
    """base^(-2i / n_rot) / divide for the n_rot / 2 pairs, worked out in float64 and rounded once to fp32"""
    i = torch.arange(n_rot // 2, dtype=torch.float64)
    return (torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / n_rot) / float(divide)).to(torch.float32).to(device)


def scaled_frequencies(n_rot, base, scaling=None, device="cpu"):
    """(frequencies fp32 (n_rot / 2), gain) of a rotation whose frequencies are rescaled for contexts longer than the `original` one
    (scaling = {factor, original, fast, slow}; None: the plain frequencies and gain 1).  A pair that turns more than `fast` times over
    `original` positions keeps its frequency f_i = base^(-2i / n_rot), one that turns less than `slow` times gets f_i / factor, and
    between the two pair indices lo = floor(index(fast)), hi = ceil(index(slow)) -- index(t) = n_rot ln(original / (2 pi t)) / (2 ln base),
    clamped to the head -- the two are blended linearly in i.  cos and sin are multiplied by the gain 0.1 ln(factor) + 1.  Worked out in
    float64, rounded once."""
    if not scaling:
        return rotary_frequencies(n_rot, base, 1.0, device), 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def index(turns):
        return n_rot * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index(float(scaling["fast"]))), 0)
    hi = min(math.ceil(index(float(scaling["slow"]))), n_rot - 1)
    i = torch.arange(n_rot // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / n_rot)
    ramp = torch.clamp((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return (f / factor * ramp + f * (1.0 - ramp)).to(torch.float32).to(device), 0.1 * math.log(factor) + 1.0


def distance_bias_table(rel, far, longest, device):
    """The bias of every distance 0 .. L - 1 from a table `rel` (rows, heads) of bucketed distances: the first rows // 2 distances have a
    row each, larger ones share the other rows on a logarithmic scale that reaches the last row at the distance `far`
    (row = half + floor(ln(n / half) / ln(far / half) * (rows - half)), at most rows - 1).  Returns fp32 (heads, L), L = far + 1 -- every
    distance from `far` on has the last row, the kernels clamp -- or `longest` when no query ever looks that far."""
    rows, heads = rel.shape
    half = rows // 2
    if half < 1 or far <= half:
        raise ZLError("distance bias: the table needs two rows or more and a largest distance beyond its exact half")
    L = int(far) + 1 if longest <= 0 else min(int(far) + 1, int(longest))
    n = torch.arange(L, dtype=torch.float64)
    big = half + torch.floor(torch.log(torch.clamp(n, min=1.0) / half) / math.log(far / half) * (rows - half)).to(torch.int64)
    row = torch.where(n < half, n.to(torch.int64), torch.clamp(big, max=rows - 1))
    return rel.to(torch.float32)[row.to(rel.device)].t().contiguous().to(device)


def linear_slopes(heads, device):
    """2^(-8 (h + 1) / heads) for h = 0 .. heads - 1, worked out in float64 and rounded once to fp32"""
    h = torch.arange(heads, dtype=torch.float64)
    return torch.exp2(-8.0 * (h + 1.0) / heads).to(torch.float32).to(device)


class WindowAttention(SideRows):
    """Softmax attention with grouped key / value heads over a paged cache: rotary positions on the first `rot_dims` coordinates of every
    query and key head (pairs i, i + rot_dims / 2; every frequency divided by `rot_scaling`, or rescaled by the dictionary of that name, see
    scaled_frequencies), queries and keys divided by their root mean
    square afterwards (qk_norm), a sliding window of `window` positions (0: none), optionally
      * values turned by their own position over all vdim coordinates before they are cached and the heads' sums turned back by the query's
        position (rotate_values; frequencies from the same base, never scaled),
      * the heads' softmax weights mixed by a (heads, heads) matrix after the softmax (tensor `talk`),
      * a sigmoid gate per output coordinate computed from the mixer's input (tensor `g`), or per head (head_gate; tensor g (heads, width)),
      * keys and values borrowed from another layer's cache (kv_source: that layer's WindowAttention; then no k / v tensors),
      * rotated pairs that are neighbours (2i, 2i + 1) instead of (i, i + rot_dims / 2) (rope_interleaved),
      * biases on q, k, v (bias; tensors q.b, k.b, v.b) and a short causal convolution over time on every channel of q, k, v right after the
        projection (conv_taps > 0; tensors q.conv, k.conv, v.conv (channels, taps); the last taps - 1 projected rows are slot state),
      * the sequence's first keep_first keys visible behind the window, at their true positions,
      * a learned sink per head in the softmax denominator (tensor `sink`; no key, no value, not scaled),
      * values blended with ANOTHER such layer's values of the same token before they are cached, v <- (1 - lam) v + lam v_other with lam
        the scalar tensor `vmix` (v_mix_source: that layer's WindowAttention, which ran earlier in the same step),
      * a weight on the query / key norm shared by the heads (norm_weight; tensors q.norm, k.norm (dim)), a factor on the scores per head
        (head_scale; tensor `temp`), scores capped by softcap * tanh(. / softcap), a learned bias by the distance between query and key
        added after the cap (rel_far > 0; tensor `rel` (rows, heads), see distance_bias_table),
      * queries that only see the keys of their own chunk of `chunk` positions, chunks counted from position 0 of the sequence,
      * weights that are no softmax: weights="sigmoid" gives every visible key sigmoid(score + offset_h) (tensor `pb` (heads)), not
        normalised over the keys,
      * ONE norm over all query heads and one over all key heads, right after the projection (whole_norm; tensors q.norm (heads*dim), k.norm
        (kv_heads*dim)), queries multiplied by 1 + coef ln(floor((p + 1) / every) + 1) at position p (q_temp = (coef, every)),
      * a linear distance bias: slope_h (p - j) is taken off the score, slope_h = 2^(-8 (h + 1) / heads) (slope_bias).
    Tensors under `prefix`: q (heads*dim, width), k (kv_heads*dim, width), v (kv_heads*vdim, width), talk (heads, heads), g (heads*vdim, width),
    o (width, heads*vdim).  q | k | v | g are one product."""

    def __init__(self, name, width, heads, kv_heads, dim, vdim, scale, window, rot_dims, rot_base, rot_scaling, eps, qk_norm=True,
                 rotate_values=True, talk=True, gate=True, kv_source=None, rope_interleaved=False, bias=False, conv_taps=0, keep_first=0,
                 sink=False, v_mix=False, v_mix_source=None, norm_weight=False, head_scale=False, softcap=0.0, rel_far=0, chunk=0,
                 weights="softmax", whole_norm=False, q_temp=None, slope_bias=False, head_gate=False):
        if weights not in ("softmax", "sigmoid") or (weights == "sigmoid" and (sink or talk)) or (chunk and keep_first) or chunk < 0:
            raise ZLError("attention: sigmoid weights have no sink and no mixing; chunks keep no first keys")
        if norm_weight and not qk_norm:
            raise ZLError("attention: a norm weight needs the query / key norm")
        self.norm_weight, self.has_head_scale, self.softcap, self.rel_far, self.chunk = bool(norm_weight), bool(head_scale), float(softcap or 0.0), \
            int(rel_far or 0), int(chunk or 0)
        self.sigmoid = weights == "sigmoid"
        if whole_norm and (qk_norm or kv_source is not None) or (slope_bias and self.sigmoid):
            raise ZLError("attention: one norm over all heads excludes a norm per head and borrowed keys; sigmoid weights have no slopes")
        self.whole_norm, self.q_temp, self.slope_bias = bool(whole_norm), (None if q_temp is None else (float(q_temp[0]), int(q_temp[1]))), bool(slope_bias)
        self.slope = self.prep = self.proj_bias = None
        self.q_norm_w = self.k_norm_w = self.temp = self.rel = self.offset = self.form = None
        if heads % kv_heads or rot_dims % 2 or rot_dims > dim or (rotate_values and vdim % 2):
            raise ZLError("attention: heads must divide by kv_heads, rotated sizes must be even and fit the head")
        if kv_source is not None and (kv_source.kv_heads, kv_source.dim, kv_source.vdim) != (kv_heads, dim, vdim):
            raise ZLError("attention: a borrowed cache must have this layer's key / value shape")
        if kv_source is not None and (bias or conv_taps or v_mix):
            raise ZLError("attention: a layer that borrows keys and values has no key / value projections to bias, convolve or blend")
        if v_mix_source is not None and (v_mix_source.kv_heads * v_mix_source.vdim != kv_heads * vdim):
            raise ZLError("attention: blended values must have this layer's value shape")
        self.interleaved, self.has_bias, self.taps, self.keep_first = bool(rope_interleaved), bool(bias), int(conv_taps), int(keep_first)
        self.has_sink, self.v_mix, self.v_mix_source = bool(sink), bool(v_mix), v_mix_source
        self.sink = self.in_bias = self.conv_w = self.tail = self.last_values = None
        self.vmix_lambda = 0.0
        self.name, self.width, self.heads, self.kv_heads, self.dim, self.vdim = name, width, heads, kv_heads, dim, vdim
        self.scale, self.window, self.rot_dims, self.rot_base, self.rot_scaling = float(scale), int(window), rot_dims, float(rot_base), \
            dict(rot_scaling) if isinstance(rot_scaling, dict) else float(rot_scaling or 1.0)
        self.eps, self.qk_norm, self.rotate_values, self.has_talk, self.has_gate = float(eps), qk_norm, rotate_values, talk, gate or head_gate
        self.head_gate, self.rot_gain = bool(head_gate), 1.0
        self.kv_source = kv_source
        self.k_cache = self.v_cache = None
        self.prompt_kernel = True         # bf16 portions on the matrix-core kernel (False: everything on the plain kernel)
        self.n_splits = None              # workgroups per (token, head) of the plain kernel (None: enough to fill the chip)

    def _cols(self):
        H, G, d, v = self.heads, self.kv_heads, self.dim, self.vdim
        own = self.kv_source is None
        kq, vq = H * d, H * d + (G * d if own else 0)
        g0 = vq + (G * v if own else 0)
        return kq, vq, g0, g0 + (0 if not self.has_gate else H if self.head_gate else H * v)

    def _tables(self, device):
        self.qk_freq = None
        if self.rot_dims and isinstance(self.rot_scaling, dict):
            self.qk_freq, self.rot_gain = scaled_frequencies(self.rot_dims, self.rot_base, self.rot_scaling, device)
        elif self.rot_dims:
            self.qk_freq = rotary_frequencies(self.rot_dims, self.rot_base, self.rot_scaling, device)
        self.v_freq = rotary_frequencies(self.vdim, self.rot_base, 1.0, device) if self.rotate_values else None
        self.form = None
        if self.slope_bias:
            self.slope = linear_slopes(self.heads, device)
        if self.has_head_scale or self.softcap > 0 or self.rel is not None or self.chunk or self.sigmoid or self.slope is not None:
            self.form = seqops.score_form(self.heads, self.temp, self.softcap, self.rel, self.offset, self.chunk, self.sigmoid, self.slope)
        self.set_prep()

    def set_prep(self, extra=None):
        """what the cache-writing launch does besides rotation and norms per head; extra: see seqops.head_prep"""
        self.prep = None
        if self.whole_norm or self.q_temp or extra or self.rot_gain != 1.0:
            self.prep = seqops.head_prep(self.whole_norm, *((self.q_norm_w, self.k_norm_w) if self.whole_norm else (None, None)), self.q_temp, extra,
                                         self.rot_gain)

    def _load_form(self, get, prefix, device):
        d, H = self.dim, self.heads
        if self.norm_weight:
            self.q_norm_w, self.k_norm_w = _vec(get, prefix + "q.norm", d, device), _vec(get, prefix + "k.norm", d, device)
        if self.whole_norm:
            self.q_norm_w, self.k_norm_w = _vec(get, prefix + "q.norm", H * d, device), _vec(get, prefix + "k.norm", self.kv_heads * d, device)
        if self.has_head_scale:
            self.temp = _vec(get, prefix + "temp", H, device)
        if self.rel_far:
            rel = get(prefix + "rel")
            if rel.dim() != 2 or rel.shape[1] != H:
                raise ZLError(f"tensor {prefix}rel: shape {tuple(rel.shape)}, expected (rows, {H})")
            longest = min(x for x in (self.chunk, self.window) if x > 0) if (self.chunk or self.window) else 0
            self.rel = distance_bias_table(rel, self.rel_far, longest, device)
        if self.sigmoid:
            self.offset = _vec(get, prefix + "pb", H, device)

    def load(self, get, prefix, dtype, device):
        H, G, d, v, W = self.heads, self.kv_heads, self.dim, self.vdim, self.width
        parts = [_mat(get, prefix + "q", (H * d, W), dtype, device)]
        if self.kv_source is None:
            parts += [_mat(get, prefix + "k", (G * d, W), dtype, device), _mat(get, prefix + "v", (G * v, W), dtype, device)]
        if self.has_gate:
            parts.append(_mat(get, prefix + "g", (H if self.head_gate else H * v, W), dtype, device))
        self.w_in = torch.cat(parts, dim=0).contiguous()
        self.talk = _mat(get, prefix + "talk", (H, H), torch.float32, device) if self.has_talk else None
        self.w_o = _mat(get, prefix + "o", (W, H * v), dtype, device)
        names = ("q", "k", "v") if self.kv_source is None else ("q",)
        sizes = {"q": H * d, "k": G * d, "v": G * v}
        if self.has_bias:
            self.in_bias = torch.cat([_vec(get, prefix + n + ".b", sizes[n], device) for n in names]).contiguous()
        if self.taps:
            self.conv_w = torch.cat([_mat(get, prefix + n + ".conv", (sizes[n], self.taps), torch.float32, device) for n in names]).contiguous()
        self._place_bias()
        self.sink = _vec(get, prefix + "sink", H, device) if self.has_sink else None
        if self.v_mix:
            self.vmix_lambda = float(_vec(get, prefix + "vmix", 1, device)[0])
        self._load_form(get, prefix, device)
        self._tables(device)
        return self

    def init_random(self, gen, dtype, device):
        H, v, W = self.heads, self.vdim, self.width
        self.w_in = _rand(gen, (self._cols()[3], W), W ** -0.5, dtype, device)
        self.talk = (torch.eye(H, device=device) + 0.1 * torch.randn(H, H, generator=gen, device=device)) if self.has_talk else None
        self.w_o = _rand(gen, (W, H * v), (H * v) ** -0.5, dtype, device)
        C = self._cols()[2]
        if self.has_bias:
            self.in_bias = 0.1 * torch.randn(C, generator=gen, device=device)
        if self.taps:
            self.conv_w = torch.randn(C, self.taps, generator=gen, device=device) * self.taps ** -0.5
        self._place_bias()
        self.sink = torch.zeros(H, device=device) if self.has_sink else None
        self.vmix_lambda = 0.5 if self.v_mix else 0.0
        d = self.dim
        if self.norm_weight or self.whole_norm:
            nq, nk = (d, d) if self.norm_weight else (H * d, self.kv_heads * d)
            self.q_norm_w, self.k_norm_w = (1.0 + 0.1 * torch.randn(n, generator=gen, device=device) for n in (nq, nk))
        if self.has_head_scale:
            self.temp = 1.0 + 0.1 * torch.randn(H, generator=gen, device=device)
        if self.rel_far:
            longest = min(x for x in (self.chunk, self.window) if x > 0) if (self.chunk or self.window) else 0
            self.rel = distance_bias_table(0.5 * torch.randn(32, H, generator=gen, device=device), max(self.rel_far, 17), longest, device)
        if self.sigmoid:
            self.offset = -2.0 + 0.1 * torch.randn(H, generator=gen, device=device)
        self._tables(device)
        return self

    def _place_bias(self):
        """biases without a convolution join the product itself (its epilogue; the gate's columns get zeros)"""
        if self.has_bias and not self.taps:
            self.proj_bias = torch.zeros(self._cols()[3], device=self.in_bias.device)
            self.proj_bias[:self.in_bias.numel()] = self.in_bias

    def bind(self, cache, dtype):
        if self.kv_source is not None:                      # (the lender is an earlier layer: it is bound already)
            self.k_cache, self.v_cache = self.kv_source.k_cache, self.kv_source.v_cache
            return
        self.k_cache = cache.add_plane(self.name + ".k", (self.kv_heads * self.dim,), dtype)
        self.v_cache = cache.add_plane(self.name + ".v", (self.kv_heads * self.vdim,), dtype)      # (the kernels keep a page transposed)
        if self.taps > 1:
            self.tail = cache.add_state(self.name + ".conv", (self.taps - 1, self._cols()[2]))

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.w_o))

    def forward(self, h, batch):
        bias = self.proj_bias
        if bias is not None and self.side_col0 is not None and bias.numel() != self.w_in.shape[0]:
            bias = self.proj_bias = torch.cat([bias, torch.zeros(self.w_in.shape[0] - bias.numel(), device=bias.device)])
        proj = seqops.gemm_nt(h, self.w_in, bias=bias)                            # fp32 [q | k | v | gate]
        self.side = (proj, self.side_col0)
        return seqops.gemm_nt(self.attend(proj, 0, batch, h.dtype), self.w_o)

    def joint_in(self):
        return None, self.w_in, self.proj_bias

    def joint_out(self):
        return self.w_o, None

    def attend(self, proj, col0, batch, dtype, lead=None, out=None, out_scale=1.0):
        """everything between the two products, from the fp32 columns [q | k | v | gate] of proj that start at col0 (biases are in them unless
        a short convolution adds them); returns the output projection's input, times out_scale, in `out` when given"""
        H, G, d, v = self.heads, self.kv_heads, self.dim, self.vdim
        k0, v0, g0, _ = self._cols()
        own = self.kv_source is None
        # the short convolution gives a second buffer [q | k | v] (the gate stays in proj); otherwise q is rotated inside proj
        qkv, c0 = (seqops.short_conv(proj, col0, self.conv_w, self.in_bias, self.tail, batch), 0) if self.conv_w is not None else (proj, col0)
        blend = None
        if self.v_mix and self.v_mix_source is not None:
            src, col = self.v_mix_source.last_values
            blend = (src, col, self.vmix_lambda)
        self.last_values = (qkv, c0 + v0) if self.v_mix else None                 # (this step's values before blending, for a later layer)
        seqops.rope_norm_store(qkv, c0, c0 + k0, c0 + v0, H, G, d, v, self.qk_freq, self.rot_dims, self.v_freq, self.eps, self.qk_norm, batch,
                               self.k_cache if own else None, self.v_cache if own else None, interleaved=self.interleaved, vmix=blend,
                               q_norm_w=self.q_norm_w if self.norm_weight else None, k_norm_w=self.k_norm_w if self.norm_weight else None,
                               prep=self.prep)
        acc, ml, n_splits = seqops.window_attention(qkv, c0, self.k_cache, self.v_cache, batch, self.scale, self.window, H, G, d, v,
                                                    all_kv=self.has_talk, mfma=self.prompt_kernel, n_splits=self.n_splits,
                                                    keep_first=self.keep_first, form=self.form)
        return seqops.head_mix_gate(acc, ml, n_splits, self.talk, self.v_freq, proj if self.has_gate else None, col0 + g0, batch, H, G, v, dtype,
                                    sink=self.sink, plain_sum=self.sigmoid, gate_per_head=self.head_gate, out=out, out_scale=out_scale)


class DecayLinearAttention:
    """Linear attention with a fixed decay per head: q, k, v = act(projections); S_t = decay_h S_{t-1} + k_t v_t^T, o_t = S_t^T q_t per head,
    the state fp32 per sequence; then an RMS norm over `norm_groups` equal parts of the heads' outputs (1: all heads together, heads: each
    head alone) with an optional weight, a gate -- sigmoid or silu of a projection (gate_act) --, the output projection.  Optionally (a
    retention layer) q and k are rotated by their position over the first rot_dims coordinates of every head (pairs i, i + rot_dims / 2,
    angle p * rot_base^(-2i / rot_dims)) and the keys multiplied by key_scale (the recurrence is linear in k: applied to o, before its norm).
    Tensors under `prefix`: q, k (heads*dim, width), v, g (heads*vdim, width), norm (heads*vdim), o (width, heads*vdim)."""

    def __init__(self, name, width, heads, dim, vdim, decay, eps, act="silu", norm_groups=1, norm_weight=True, gate_act="sigmoid", rot_dims=0,
                 rot_base=10000.0, key_scale=1.0):
        if len(decay) != heads:
            raise ZLError("linear attention: one decay per head")
        if rot_dims % 2 or not 0 <= rot_dims <= dim or (rot_dims and act is not None):
            raise ZLError("linear attention: the rotated part is even and fits the head; rotated queries and keys have no activation")
        self.name, self.width, self.heads, self.dim, self.vdim = name, width, heads, dim, vdim
        self.decay_values, self.eps, self.act, self.norm_groups = [float(x) for x in decay], float(eps), act, norm_groups
        self.has_norm_weight, self.gate_act, self.key_scale = bool(norm_weight), gate_act, float(key_scale)
        self.rot_dims, self.rot_base = int(rot_dims), float(rot_base)
        self.scan_segment = None

    def _constants(self, device):
        self.decay = torch.tensor(self.decay_values, dtype=torch.float64).to(torch.float32).to(device)
        self.freq = rotary_frequencies(self.rot_dims, self.rot_base, 1.0, device) if self.rot_dims else None

    def load(self, get, prefix, dtype, device):
        H, d, v, W = self.heads, self.dim, self.vdim, self.width
        self.w_in = torch.cat([_mat(get, prefix + "q", (H * d, W), dtype, device), _mat(get, prefix + "k", (H * d, W), dtype, device),
                               _mat(get, prefix + "v", (H * v, W), dtype, device), _mat(get, prefix + "g", (H * v, W), dtype, device)], dim=0).contiguous()
        self.norm_w = _vec(get, prefix + "norm", H * v, device) if self.has_norm_weight else None
        self.w_o = _mat(get, prefix + "o", (W, H * v), dtype, device)
        self._constants(device)
        return self

    def init_random(self, gen, dtype, device):
        H, d, v, W = self.heads, self.dim, self.vdim, self.width
        self.w_in = _rand(gen, (2 * H * d + 2 * H * v, W), W ** -0.5, dtype, device)
        self.norm_w = torch.ones(H * v, device=device) if self.has_norm_weight else None
        self.w_o = _rand(gen, (W, H * v), (H * v) ** -0.5, dtype, device)
        self._constants(device)
        return self

    def bind(self, cache, dtype):
        self.state = cache.add_state(self.name + ".S", (self.heads, self.dim, self.vdim))

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.w_o))

    def rotated(self, col0):
        """the queries and keys behind col0 as heads to rotate in place (seqops.head_prep's `extra`); None without a rotation"""
        return (col0, 2 * self.heads, self.dim, self.rot_dims, self.freq) if self.rot_dims else None

    def forward(self, h, batch):
        proj = seqops.gemm_nt(h, self.w_in)                                       # fp32 [q | k | v | gate]
        if self.rot_dims:                                                         # (queries and keys alike: 2 heads groups of one launch)
            seqops.rope_norm_store(proj, 0, 0, 0, 2 * self.heads, 1, self.dim, 1, self.freq, self.rot_dims, None, self.eps, False, batch, None, None)
        return seqops.gemm_nt(self.attend(proj, 0, batch, h.dtype), self.w_o)

    def attend(self, proj, col0, batch, dtype):
        """everything between the two products but the rotation, from the fp32 columns [q | k | v | gate] of proj that start at col0"""
        H, d, v = self.heads, self.dim, self.vdim
        y = seqops.decay_scan(proj, col0, col0 + H * d, col0 + 2 * H * d, self.act == "silu", self.decay, None, None, False, self.state, H, d, v, batch,
                              seg_len=self.scan_segment)
        return seqops.linear_attn_finish(y, False, self.key_scale, None, 0.0, H, v, self.norm_groups, self.norm_w, self.eps, proj,
                                         col0 + 2 * H * d + H * v, dtype, gate_act=self.gate_act)


class ParallelMixers:
    """Two mixers side by side on the same input: the first `left` (WindowAttention), the second `right` (DecayLinearAttention).  Their input
    projections are ONE product [left | right]; one launch then norms, rotates and caches for both; their results join the residual with an
    RMS norm over the model width each, as the branches (y, weight, coef) that seqops.add_branches sums.
    Tensors under `prefix`: left.*, right.* (the mixers' own), left.out, right.out (width)."""
    parts = ("left", "right")

    def __init__(self, name, left, right, coef=0.5):
        if left.width != right.width or left.conv_w is not None or left.taps or left.kv_source is not None:
            raise ZLError("parallel mixers: one width; the left one projects its own keys and values and has no convolution")
        self.name, self.width, self.left, self.right, self.coef = name, left.width, left, right, float(coef)

    def _join(self):
        left, right = self.left, self.right
        self.w_in = torch.cat([left.w_in, right.w_in], dim=0).contiguous()
        self.col = left.w_in.shape[0]                                             # (where the right mixer's columns start)
        self.in_bias = None
        if left.proj_bias is not None:
            self.in_bias = torch.zeros(self.w_in.shape[0], device=self.w_in.device)
            self.in_bias[:self.col] = left.proj_bias
        left.w_in = right.w_in = None                                             # (the rows live in the joint matrix now)
        left.set_prep(right.rotated(self.col))
        return self

    def load(self, get, prefix, dtype, device):
        self.left.load(get, prefix + "left.", dtype, device)
        self.right.load(get, prefix + "right.", dtype, device)
        self.left_out, self.right_out = _vec(get, prefix + "left.out", self.width, device), _vec(get, prefix + "right.out", self.width, device)
        return self._join()

    def init_random(self, gen, dtype, device):
        self.left.init_random(gen, dtype, device)
        self.right.init_random(gen, dtype, device)
        self.left_out, self.right_out = (1.0 + 0.1 * torch.randn(self.width, generator=gen, device=device) for _ in range(2))
        return self._join()

    def bind(self, cache, dtype):
        self.left.bind(cache, dtype)
        self.right.bind(cache, dtype)

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.left.w_o, self.right.w_o))

    def branches(self, h, batch):
        proj = seqops.gemm_nt(h, self.w_in, bias=self.in_bias)                    # fp32 [left: q | k | v | right: q | k | v | gate]
        a = self.left.attend(proj, 0, batch, h.dtype)                             # (its first launch also rotates the right mixer's q and k)
        r = self.right.attend(proj, self.col, batch, h.dtype)
        return [(seqops.gemm_nt(a, self.left.w_o), self.left_out, self.coef), (seqops.gemm_nt(r, self.right.w_o), self.right_out, self.coef)]


class Mamba1Mixer:
    """Selective state-space mixer with a decay per channel and state: [x | z] = W_in h; x through a causal short convolution (with bias) and
    SiLU; [low | B | C] = W_x x; dt = softplus(W_dt low + bias) per channel; S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n with
    A = -exp(A_log), y_c = sum_n S[c, n] C_n + D_c x_c; (y * silu(z)) to the output projection.  The state and the convolution's last inputs
    are fp32 slot states.  The rows of `low` are padded to a multiple of 8 with zero rows (and W_dt with zero columns), so that the small
    product reads aligned rows.
    Tensors under `prefix`: in (2*inner, width), conv (inner, taps), conv.b (inner), x (rank + 2*n_state, inner), dt (inner, rank), dt.b
    (inner), A_log (inner, n_state), D (inner), o (width, inner)."""

    def __init__(self, name, width, inner, n_state, rank, taps):
        if min(inner, n_state, rank, taps) < 1:
            raise ZLError("mamba1: sizes must be positive")
        self.name, self.width, self.inner, self.n_state, self.rank, self.taps = name, width, inner, n_state, rank, taps
        self.low = (rank + 7) // 8 * 8
        self.scan_segment = None          # tokens per segment of a long portion (None: seqops.scan_segment; 0: never in segments)

    def _pack(self, w_x, w_dt, a_log):
        r, low = self.rank, self.low
        pad = torch.zeros((low - r, self.inner), dtype=w_x.dtype, device=w_x.device)
        self.w_x = torch.cat([w_x[:r], pad, w_x[r:]], dim=0).contiguous()
        self.w_dt = torch.zeros((self.inner, low), dtype=w_dt.dtype, device=w_dt.device)
        self.w_dt[:, :r] = w_dt
        # the rates as exponents of two, (n_state, inner): exp(dt A) = 2^(dt a2)
        self.a2 = (-torch.exp(a_log.double()) * math.log2(math.e)).to(torch.float32).t().contiguous()

    def load(self, get, prefix, dtype, device):
        C, N, R, W = self.inner, self.n_state, self.rank, self.width
        self.w_in = _mat(get, prefix + "in", (2 * C, W), dtype, device)
        self.conv_w = _mat(get, prefix + "conv", (C, self.taps), torch.float32, device)
        self.conv_b, self.dt_bias, self.d = (_vec(get, prefix + n, C, device) for n in ("conv.b", "dt.b", "D"))
        self._pack(_mat(get, prefix + "x", (R + 2 * N, C), dtype, device), _mat(get, prefix + "dt", (C, R), dtype, device),
                   _mat(get, prefix + "A_log", (C, N), torch.float32, device))
        self.w_o = _mat(get, prefix + "o", (W, C), dtype, device)
        return self

    def init_random(self, gen, dtype, device):
        C, N, R, W = self.inner, self.n_state, self.rank, self.width
        self.w_in = _rand(gen, (2 * C, W), W ** -0.5, dtype, device)
        self.conv_w = _rand(gen, (C, self.taps), self.taps ** -0.5, torch.float32, device)
        self.conv_b, self.d = torch.zeros(C, device=device), torch.ones(C, device=device)
        self.dt_bias = torch.full((C,), -3.0, device=device)
        self._pack(_rand(gen, (R + 2 * N, C), C ** -0.5, dtype, device), _rand(gen, (C, R), R ** -0.5, dtype, device),
                   torch.log(torch.arange(1, N + 1, device=device, dtype=torch.float32))[None, :].repeat(C, 1))
        self.w_o = _rand(gen, (W, C), C ** -0.5, dtype, device)
        return self

    def bind(self, cache, dtype):
        self.tail = cache.add_state(self.name + ".conv", (self.taps - 1, self.inner)) if self.taps > 1 else None
        self.state = cache.add_state(self.name + ".ssm", (self.n_state, self.inner))

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.w_x, self.w_dt, self.w_o))

    def branches(self, h, batch):
        return [(self.forward(h, batch), None, 1.0)]

    def forward(self, h, batch):
        C, N, low = self.inner, self.n_state, self.low
        proj = seqops.gemm_nt(h, self.w_in)                                       # fp32 [x | z]
        x, xt = seqops.short_conv(proj, 0, self.conv_w, None, self.tail, batch, act=True, bias=self.conv_b, also=h.dtype)
        small, u = seqops.gemm_nt(xt, self.w_x, lead=low)                         # fp32 [low, padded | B | C]; low once more in the serving format
        dt = seqops.gemm_nt(u, self.w_dt, bias=self.dt_bias, act="softplus")
        y = seqops.selective_scan(x, dt, small, low, low + N, proj, C, self.a2, self.d, self.state, batch, h.dtype, seg_len=self.scan_segment)
        return seqops.gemm_nt(y, self.w_o)


class GatedLinearAttention:
    """Linear attention with a learned decay per KEY CHANNEL and token: q = W_q h * dim^-1/2, k = W_k h, v = W_v h;
        alpha = sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)   (heads x dim, from a low-rank pair of projections)
        S_t = diag(alpha_t) S_{t-1} + k_t v_t^T,  o_t = S_t^T q_t   per head, S fp32 per sequence, from zero
    then each head's o divided by its root mean square over vdim, times a weight shared by the heads, times silu(W_g h), and the output
    projection.  The logarithm of the decay, the decay and the recurrence are fp32; the scale dim^-1/2 is applied to o (the recurrence is
    linear in q).  Tensors under `prefix`: q, k (heads*dim, width), v, g (heads*vdim, width), a1 (low, width), a2 (heads*dim, low), a2.b
    (heads*dim), norm (vdim), o (width, heads*vdim).  q | k | v | g | a1 are one product."""

    def __init__(self, name, width, heads, dim, vdim, tau, eps):
        if tau <= 0:
            raise ZLError("gated linear attention: tau > 0")
        self.name, self.width, self.heads, self.dim, self.vdim = name, width, heads, dim, vdim
        self.tau, self.eps = float(tau), float(eps)
        self.scan_segment = None

    def load(self, get, prefix, dtype, device):
        H, d, v, W = self.heads, self.dim, self.vdim, self.width
        a1 = get(prefix + "a1")
        self.low = int(a1.shape[0])
        self.w_in = torch.cat([_mat(get, prefix + "q", (H * d, W), dtype, device), _mat(get, prefix + "k", (H * d, W), dtype, device),
                               _mat(get, prefix + "v", (H * v, W), dtype, device), _mat(get, prefix + "g", (H * v, W), dtype, device),
                               _mat(get, prefix + "a1", (self.low, W), dtype, device)], dim=0).contiguous()
        self.w_a2 = _mat(get, prefix + "a2", (H * d, self.low), dtype, device)
        self.a2_bias = _vec(get, prefix + "a2.b", H * d, device)
        self.norm_w = _vec(get, prefix + "norm", v, device).repeat(H).contiguous()
        self.w_o = _mat(get, prefix + "o", (W, H * v), dtype, device)
        return self

    def init_random(self, gen, dtype, device, low=16):
        H, d, v, W = self.heads, self.dim, self.vdim, self.width
        self.low = low
        self.w_in = _rand(gen, (2 * H * d + 2 * H * v + low, W), W ** -0.5, dtype, device)
        self.w_a2 = _rand(gen, (H * d, low), low ** -0.5, dtype, device)
        self.a2_bias = torch.full((H * d,), 2.0, device=device)
        self.norm_w = torch.ones(H * v, device=device)
        self.w_o = _rand(gen, (W, H * v), (H * v) ** -0.5, dtype, device)
        return self

    def bind(self, cache, dtype):
        self.state = cache.add_state(self.name + ".S", (self.heads, self.dim, self.vdim))

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.w_a2, self.w_o))

    def forward(self, h, batch):
        H, d, v = self.heads, self.dim, self.vdim
        proj = seqops.gemm_nt(h, self.w_in)                                       # fp32 [q | k | v | gate | low-rank decay input]
        g0 = 2 * H * d + H * v
        alpha = seqops.lowrank_decay(proj, g0 + H * v, self.w_a2, self.a2_bias, self.tau)
        y = seqops.decay_scan(proj, 0, H * d, 2 * H * d, False, None, None, None, False, self.state, H, d, v, batch, seg_len=self.scan_segment,
                              decay_v=alpha)
        a = seqops.linear_attn_finish(y, False, d ** -0.5, None, 0.0, H, v, H, self.norm_w, self.eps, proj, g0, h.dtype, gate_act="silu")
        return seqops.gemm_nt(a, self.w_o)


class GatedDeltaRule:
    """Gated delta rule: q, k, v pass a short causal convolution per channel and SiLU, q and k become unit vectors per head (q times dim^-1/2);
    beta = sigmoid(W_b h) per head;
        S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q        per head, S (dim x vdim) fp32 per sequence, from zero
    with the decay g = exp(-exp(A_log) softplus(z + dt_bias)): decay="head": z = W_a h, a number per head; decay="channel": z = W_a2 (W_a1 h),
    a number per head and key channel.  Then each head's o is divided by its root mean square over vdim, times a weight shared by the heads,
    times gate_act of W_g h (gate="full") or of W_g2 (W_g1 h) (gate="lowrank"), and the output projection.  Several heads may share a query /
    key head.  The two second steps of low-rank pairs are ONE product with a block-diagonal matrix whose input is the LEADING columns of the
    first product, written once more in the serving format.
    Tensors under `prefix`: q, k (kv_heads*dim, width), v (heads*vdim, width), q.conv, k.conv, v.conv (channels, taps), b (heads, width), A_log
    (heads), dt_bias (heads | heads*dim), a (heads, width) or a1 (low, width), a2 (heads*dim, low), g (heads*vdim, width) or g1 (low, width),
    g2 (heads*vdim, low), norm (vdim), o (width, heads*vdim)."""
    UNIT_EPS = 1e-6                       # joins a head's sum of squares under the root

    def __init__(self, name, width, heads, kv_heads, dim, vdim, taps, eps, decay="head", gate="full", gate_act="silu"):
        if heads % kv_heads or min(heads, kv_heads, dim, vdim, taps) < 1:
            raise ZLError("delta rule: heads must divide by kv_heads, sizes must be positive")
        if decay not in ("head", "channel") or gate not in ("full", "lowrank") or gate_act not in ("silu", "sigmoid"):
            raise ZLError("delta rule: decay per head or channel, gate full or lowrank, silu or sigmoid")
        self.name, self.width, self.heads, self.kv_heads, self.dim, self.vdim, self.taps, self.eps = name, width, heads, kv_heads, dim, vdim, taps, float(eps)
        self.per_channel, self.lowrank_gate, self.gate_act = decay == "channel", gate == "lowrank", gate_act
        self.channels = 2 * kv_heads * dim + heads * vdim
        self.lead = self.w_low = None

    def _pairs(self):
        """[(first step's name, second step's name, outputs)] of the low-rank pairs"""
        out = [("a1", "a2", self.heads * self.dim)] if self.per_channel else []
        return out + ([("g1", "g2", self.heads * self.vdim)] if self.lowrank_gate else [])

    def _rows(self):
        """[(name, rows)] of the input projection behind the leading low-rank rows"""
        G, d, H, v = self.kv_heads, self.dim, self.heads, self.vdim
        return [("q", G * d), ("k", G * d), ("v", H * v), ("b", H)] + ([] if self.per_channel else [("a", H)]) + ([] if self.lowrank_gate else [("g", H * v)])

    def _set(self, mats, firsts, seconds, conv_w, a_log, dt_bias, norm, w_o, device):
        H, v = self.heads, self.vdim
        self.w_in = torch.cat(mats, dim=0).contiguous()
        if firsts:                        # the leading rows, padded to whole 16-byte pieces, and the block-diagonal second step
            low = sum(m.shape[0] for m in firsts)
            pad = (low + 7) // 8 * 8
            self.lead = torch.cat(firsts + [torch.zeros((pad - low, self.width), dtype=firsts[0].dtype, device=device)], dim=0).contiguous()
            self.w_low = torch.zeros((sum(m.shape[0] for m in seconds), pad), dtype=firsts[0].dtype, device=device)
            r = c = 0
            for m in seconds:
                self.w_low[r:r + m.shape[0], c:c + m.shape[1]] = m
                r, c = r + m.shape[0], c + m.shape[1]
        self.conv_w = conv_w.contiguous()
        self.rate = torch.exp(a_log.double()).to(torch.float32).contiguous()
        self.dt_bias, self.norm_w, self.w_o = dt_bias, norm.repeat(H).contiguous(), w_o
        return self

    def load(self, get, prefix, dtype, device):
        W, H, d, v = self.width, self.heads, self.dim, self.vdim
        firsts, seconds = [], []
        for one, two, n in self._pairs():
            low = int(get(prefix + one).shape[0])
            firsts.append(_mat(get, prefix + one, (low, W), dtype, device))
            seconds.append(_mat(get, prefix + two, (n, low), dtype, device))
        rows = self._rows()
        conv = torch.cat([_mat(get, prefix + n + ".conv", (r, self.taps), torch.float32, device) for n, r in rows[:3]], dim=0)
        return self._set([_mat(get, prefix + n, (r, W), dtype, device) for n, r in rows], firsts, seconds, conv, _vec(get, prefix + "A_log", H, device),
                         _vec(get, prefix + "dt_bias", H * d if self.per_channel else H, device), _vec(get, prefix + "norm", v, device),
                         _mat(get, prefix + "o", (W, H * v), dtype, device), device)

    def init_random(self, gen, dtype, device, low=None):
        W, H, d, v = self.width, self.heads, self.dim, self.vdim
        low = d if low is None else low
        firsts = [_rand(gen, (low, W), W ** -0.5, dtype, device) for _ in self._pairs()]
        seconds = [_rand(gen, (n, low), low ** -0.5, dtype, device) for _, _, n in self._pairs()]
        conv = torch.randn((self.channels, self.taps), generator=gen, device=device) * self.taps ** -0.5
        return self._set([_rand(gen, (r, W), W ** -0.5, dtype, device) for _, r in self._rows()], firsts, seconds, conv, torch.zeros(H, device=device),
                         torch.full((H * d if self.per_channel else H,), -3.0, device=device), torch.ones(v, device=device),
                         _rand(gen, (W, H * v), (H * v) ** -0.5, dtype, device), device)

    def bind(self, cache, dtype):
        self.tail = cache.add_state(self.name + ".conv", (self.taps - 1, self.channels)) if self.taps > 1 else None
        self.state = cache.add_state(self.name + ".S", (self.heads, self.vdim, self.dim))     # (a value column's numbers side by side)

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.lead, self.w_low, self.w_o) if t is not None)

    def joint_in(self):
        return self.lead, self.w_in, None

    def joint_out(self):
        return self.w_o, None

    def forward(self, h, batch):
        if self.lead is None:
            proj, lead, col0 = seqops.gemm_nt(h, self.w_in), None, 0
        else:
            col0 = self.lead.shape[0]
            proj, lead = seqops.gemm_nt(h, torch.cat([self.lead, self.w_in], dim=0), lead=col0)
        return seqops.gemm_nt(self.attend(proj, col0, batch, h.dtype, lead=lead), self.w_o)

    def attend(self, proj, col0, batch, dtype, lead=None, out=None, out_scale=1.0):
        """everything between the two products, from the fp32 columns [q | k | v | b | (a) | (g)] of proj that start at col0 and the low-rank
        columns `lead` in the serving format; returns the output projection's input, times out_scale, in `out` when given"""
        H, G, d, v = self.heads, self.kv_heads, self.dim, self.vdim
        b0 = col0 + self.channels
        z = seqops.gemm_nt(lead, self.w_low) if self.w_low is not None else None               # fp32 [decay input | gate], the low-rank ones
        dec, dec0 = (z, 0) if self.per_channel else (proj, b0 + H)
        gate, gate0 = (z, H * d if self.per_channel else 0) if self.lowrank_gate else (proj, b0 + (H if self.per_channel else 2 * H))
        qkv, gates, decay = seqops.delta_prep(proj, col0, self.conv_w, self.tail, H, G, d, v, d ** -0.5, self.UNIT_EPS, b0, dec, dec0, self.dt_bias,
                                               self.rate, self.per_channel, batch)
        y = seqops.delta_scan(qkv, gates, decay, self.state, H, G, d, v, batch)
        return seqops.linear_attn_finish(y, False, 1.0, None, 0.0, H, v, H, self.norm_w, self.eps, gate, gate0, dtype, gate_act=self.gate_act, out=out,
                                         out_scale=out_scale)


class JoinedSublayers:
    """Sub-layers that read the same input and whose results are added, sum_i scale_i * part_i(h) -- mixers and a feed-forward side by side on
    one norm -- as TWO products: the parts' input projections are the rows of one matrix, what they leave before their output projections
    stands side by side in one row, and one matrix of their output projections side by side multiplies and adds it all (the scales act on
    the fp32 numbers before they are rounded to that row).  A part offers
        joint_in() -> (lead rows or None, rows, bias or None)      its input projection; lead rows: outputs that are also wanted in the serving format
        joint_out() -> (matrix, bias or None)                       its output projection
        attend(proj, col0, batch, dtype, lead, out, out_scale)      everything between, from its columns of proj into its columns of the row
    parts: [(tensor prefix, part, scale)]; name + part names register the caches and states."""

    def __init__(self, width, parts):
        self.width, self.parts = width, [p for _, p, _ in parts]
        self.prefixes, self.scales = [n for n, _, _ in parts], [float(s) for _, _, s in parts]
        if any(p.width != width for p in self.parts):
            raise ZLError("joined sub-layers: one width")

    def load(self, get, prefix, dtype, device):
        for n, p in zip(self.prefixes, self.parts):
            p.load(get, prefix + n, dtype, device)
        return self._join()

    def init_random(self, gen, dtype, device):
        for p in self.parts:
            p.init_random(gen, dtype, device)
        return self._join()

    def _join(self):
        leads, rows, biases = zip(*[p.joint_in() for p in self.parts])
        self.n_lead = sum(m.shape[0] for m in leads if m is not None)
        self.w_in = torch.cat([m for m in leads if m is not None] + list(rows), dim=0).contiguous()
        self.in_bias = None
        if any(b is not None for b in biases):
            self.in_bias = torch.zeros(self.w_in.shape[0], device=self.w_in.device)
        self.lead_at, self.col0, lead_at, at = [], [], 0, self.n_lead
        for lead, r, b in zip(leads, rows, biases):
            self.lead_at.append(None if lead is None else (lead_at, lead_at + lead.shape[0]))
            self.col0.append(at)
            if b is not None:
                self.in_bias[at:at + b.numel()] = b
            lead_at, at = lead_at + (0 if lead is None else lead.shape[0]), at + r.shape[0]
        mats, biases = zip(*[p.joint_out() for p in self.parts])
        self.w_out = torch.cat(mats, dim=1).contiguous()
        self.out_at, at = [], 0
        for m in mats:
            self.out_at.append((at, at + m.shape[1]))
            at += m.shape[1]
        self.out_bias = None
        for b, s in zip(biases, self.scales):
            if b is not None:
                self.out_bias = b * s if self.out_bias is None else self.out_bias + b * s
        for p in self.parts:                                                      # (the rows live in the joint matrices now)
            for n in ("w_in", "lead", "w_gu", "w_o", "w_down"):
                if getattr(p, n, None) is not None:
                    setattr(p, n, None)
        return self

    def bind(self, cache, dtype):
        for p in self.parts:
            p.bind(cache, dtype)

    def weight_bytes(self):
        extra = [getattr(p, "w_low", None) for p in self.parts]
        return sum(t.numel() * t.element_size() for t in [self.w_in, self.w_out] + extra if t is not None)

    def forward(self, h, batch):
        proj, lead = seqops.gemm_nt(h, self.w_in, bias=self.in_bias, lead=self.n_lead) if self.n_lead else (seqops.gemm_nt(h, self.w_in, bias=self.in_bias), None)
        row = torch.empty((batch.n_tok, self.w_out.shape[1]), dtype=h.dtype, device=h.device)
        for p, s, c, l, (a, b) in zip(self.parts, self.scales, self.col0, self.lead_at, self.out_at):
            p.attend(proj, c, batch, h.dtype, lead=None if l is None else lead[:, l[0]:l[1]], out=row[:, a:b], out_scale=s)
        return seqops.gemm_nt(row, self.w_out, bias=self.out_bias)


class TokenSideInput:
    """A second embedding that enters the residual behind a layer: e = dim columns of a table, looked up by the token; y = W_proj (gelu_tanh(W_gate x)
    * e), in the tanh form, joins the residual with an RMS norm over the model width.  The activation and the product with e are in the
    first product's epilogue.  Tensors under `prefix`: gate (dim, width), proj (width, dim), norm (width)."""

    def __init__(self, width, dim, column):
        self.width, self.dim, self.column = width, dim, column

    def load(self, get, prefix, dtype, device):
        self.w_gate = _mat(get, prefix + "gate", (self.dim, self.width), dtype, device)
        self.w_proj = _mat(get, prefix + "proj", (self.width, self.dim), dtype, device)
        self.norm_w = _vec(get, prefix + "norm", self.width, device)
        return self

    def init_random(self, gen, dtype, device):
        self.w_gate = _rand(gen, (self.dim, self.width), self.width ** -0.5, dtype, device)
        self.w_proj = _rand(gen, (self.width, self.dim), self.dim ** -0.5, dtype, device)
        self.norm_w = 1.0 + 0.1 * torch.randn(self.width, generator=gen, device=device)
        return self

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_gate, self.w_proj))

    def branch(self, xt, table, tokens, coef):
        """xt: the residual in the serving format; table (vocab, columns); the branch that seqops.add_branches sums"""
        g = seqops.gemm_nt(xt, self.w_gate, out_dtype=xt.dtype, act="gelu_tanh", factor=(table, self.column, tokens))
        return seqops.gemm_nt(g, self.w_proj), self.norm_w, coef


class PlainFF(SideRows):
    """Dense feed-forward down(act(up h)) without biases and without a gate; act: "relu2" (the square of relu), "gelu_tanh" or "silu".
    Tensors under `prefix`: up (ff, width), down (width, ff)."""
    _side_matrix = "w_up"

    def __init__(self, width, ff, act="relu2"):
        if act not in seqops.UNARY_ACTS:
            raise ZLError(f"feed-forward: unknown activation {act!r}")
        self.width, self.ff, self.act = width, ff, act

    def load(self, get, prefix, dtype, device):
        self.w_up = _mat(get, prefix + "up", (self.ff, self.width), dtype, device)
        self.w_down = _mat(get, prefix + "down", (self.width, self.ff), dtype, device)
        return self

    def init_random(self, gen, dtype, device):
        self.w_up = _rand(gen, (self.ff, self.width), self.width ** -0.5, dtype, device)
        self.w_down = _rand(gen, (self.width, self.ff), self.ff ** -0.5, dtype, device)
        return self

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_up, self.w_down))

    def forward(self, h):
        if self.side_col0 is None:                                                # (the activation in the product's epilogue)
            return seqops.gemm_nt(seqops.gemm_nt(h, self.w_up, out_dtype=h.dtype, act=self.act), self.w_down)
        z = seqops.gemm_nt(h, self.w_up)                                          # fp32 [up | side rows]
        self.side = (z, self.side_col0)
        return seqops.gemm_nt(seqops.unary_act(z, h.dtype, kind=self.act, cols=self.ff), self.w_down)


class GatedFF:
    """Dense gated feed-forward down(act(gate h) * (up h)); act: "gelu_tanh" (the tanh form) or "silu"; bias: every projection has one (tensors
    gate.b, up.b (ff), down.b (width)).  Tensors under `prefix`: gate, up (ff, width), down (width, ff).  gate | up are one product."""
    in_bias = out_bias = None

    def __init__(self, width, ff, act="gelu_tanh", bias=False):
        if act not in ("gelu_tanh", "silu"):
            raise ZLError(f"feed-forward: unknown activation {act!r}")
        self.width, self.ff, self.act, self.has_bias = width, ff, act, bool(bias)

    def load(self, get, prefix, dtype, device):
        self.w_gu = torch.cat([_mat(get, prefix + "gate", (self.ff, self.width), dtype, device),
                               _mat(get, prefix + "up", (self.ff, self.width), dtype, device)], dim=0).contiguous()
        self.w_down = _mat(get, prefix + "down", (self.width, self.ff), dtype, device)
        if self.has_bias:
            self.in_bias = torch.cat([_vec(get, prefix + n + ".b", self.ff, device) for n in ("gate", "up")]).contiguous()
            self.out_bias = _vec(get, prefix + "down.b", self.width, device)
        return self

    def init_random(self, gen, dtype, device):
        self.w_gu = _rand(gen, (2 * self.ff, self.width), self.width ** -0.5, dtype, device)
        self.w_down = _rand(gen, (self.width, self.ff), self.ff ** -0.5, dtype, device)
        if self.has_bias:
            self.in_bias, self.out_bias = (0.1 * torch.randn(n, generator=gen, device=device) for n in (2 * self.ff, self.width))
        return self

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_gu, self.w_down))

    def forward(self, h):
        return seqops.gemm_nt(seqops.act_mul(seqops.gemm_nt(h, self.w_gu, bias=self.in_bias), h.dtype, kind=self.act), self.w_down, bias=self.out_bias)

    def bind(self, cache, dtype):
        pass

    def joint_in(self):
        return None, self.w_gu, self.in_bias

    def joint_out(self):
        return self.w_down, self.out_bias

    def attend(self, proj, col0, batch, dtype, lead=None, out=None, out_scale=1.0):
        """what lies between the two products, from the columns [gate | up] of proj that start at col0"""
        if out_scale != 1.0:
            raise ZLError("feed-forward: no output scale")
        return seqops.act_mul(proj, dtype, kind=self.act, col0=col0, ff=self.ff, out=out)


class MLSTMMixer:
    """Matrix memory with exponential gates (mLSTM): per head a log input gate i and a log forget gate f = log sigmoid(.), both capped by
    cap * tanh(. / cap), a running maximum m (from 0) that keeps the exponentials in range:
        m_t = max(f + m_{t-1}, i);  S_t = e^{f + m_{t-1} - m_t} S_{t-1} + e^{i - m_t} k v^T;  n_t the same with k alone
        o = S_t^T q / (max(|n_t . q|, e^{-m_t}) + 1e-6),  q scaled by dim^-1/2
    then each head divided by its root mean square, a weight over all heads, the sigmoid gate, the output projection.  S, n, m are fp32 per
    sequence; n rides in the scan as one more value column that is 1 for every token.
    Tensors under `prefix`: q, k (heads*dim, width), v, g (heads*vdim, width), i, f (heads, width), i.b, f.b (heads), norm (heads*vdim),
    o (width, heads*vdim)."""

    def __init__(self, name, width, heads, dim, vdim, gate_cap, eps, den_eps=1e-6):
        self.name, self.width, self.heads, self.dim, self.vdim = name, width, heads, dim, vdim
        self.cap, self.eps, self.den_eps = float(gate_cap), float(eps), float(den_eps)
        self.scan_segment = None

    def load(self, get, prefix, dtype, device):
        H, d, v, W = self.heads, self.dim, self.vdim, self.width
        self.w_in = torch.cat([_mat(get, prefix + "q", (H * d, W), dtype, device), _mat(get, prefix + "k", (H * d, W), dtype, device),
                               _mat(get, prefix + "v", (H * v, W), dtype, device), _mat(get, prefix + "g", (H * v, W), dtype, device),
                               _mat(get, prefix + "i", (H, W), dtype, device), _mat(get, prefix + "f", (H, W), dtype, device)], dim=0).contiguous()
        self.i_bias, self.f_bias = _vec(get, prefix + "i.b", H, device), _vec(get, prefix + "f.b", H, device)
        self.norm_w = _vec(get, prefix + "norm", H * v, device)
        self.w_o = _mat(get, prefix + "o", (W, H * v), dtype, device)
        return self

    def init_random(self, gen, dtype, device):
        H, d, v, W = self.heads, self.dim, self.vdim, self.width
        self.w_in = _rand(gen, (2 * H * d + 2 * H * v + 2 * H, W), W ** -0.5, dtype, device)
        self.i_bias = torch.zeros(H, device=device)
        self.f_bias = torch.full((H,), 3.0, device=device)
        self.norm_w = torch.ones(H * v, device=device)
        self.w_o = _rand(gen, (W, H * v), (H * v) ** -0.5, dtype, device)
        return self

    def bind(self, cache, dtype):
        self.state = cache.add_state(self.name + ".S", (self.heads, self.dim, self.vdim + 1))
        self.m_state = cache.add_state(self.name + ".m", (self.heads,))

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_in, self.w_o))

    def forward(self, h, batch):
        H, d, v = self.heads, self.dim, self.vdim
        proj = seqops.gemm_nt(h, self.w_in)                                       # fp32 [q | k | v | gate | i | f]
        g0 = 2 * H * d + H * v
        decay, gain, m = seqops.exp_gates(proj, g0 + H * v, g0 + H * v + H, self.i_bias, self.f_bias, self.cap, self.m_state, H, batch)
        y = seqops.decay_scan(proj, 0, H * d, 2 * H * d, False, None, decay, gain, True, self.state, H, d, v, batch, seg_len=self.scan_segment)
        a = seqops.linear_attn_finish(y, True, d ** -0.5, m, self.den_eps, H, v, H, self.norm_w, self.eps, proj, g0, h.dtype)
        return seqops.gemm_nt(a, self.w_o)


class RoutedExpertsFF(SideRows):
    """Mixture of gated feed-forward experts, down(silu(gate h) * (up h)), without biases.  The router gives one logit per expert and per
    IDENTITY output (the last `identity` of its outputs: their "expert" returns h itself); probabilities = softmax over all outputs; an
    output is chosen by probability + `correction`, within the `keep` best of `groups` equal groups of neighbouring outputs (a group scores
    by its best member); the `top` chosen outputs are weighted by their plain probabilities (renormalised only if `renorm`), times
    `weight_scale`.
    Tensors under `prefix`: router (experts + identity, width), correction (experts + identity), e<j>.gate / e<j>.up (ff, width),
    e<j>.down (width, ff).  Gate and up rows of all experts are stacked in blocks of 16 (16 gate rows, their 16 up rows), so that the grouped
    product's epilogue finishes the activation."""
    _side_matrix = "w_router"

    def __init__(self, width, ff, experts, top, identity=0, groups=1, keep=1, correction=True, renorm=False, score="softmax", group_top=1,
                 renorm_eps=0.0, act="silu", act_alpha=1.0, limit=0.0, weight_scale=1.0, router_bias=False, shared_ff=0, shared_gate=False):
        """score: "softmax" over all outputs, "sigmoid" of each logit, or "chosen" (the largest logits, weighted by a softmax over the chosen
        ones only); router_bias: tensor router.b (experts + identity) is added to the logits; shared_ff > 0: one more expert `shared` (the
        same form and activation, its own size) runs for every token and is added, times sigmoid(W_sg h) with shared_gate (tensor shared.sg
        (1, width)) -- its gate, gate and up rows ride in the router's product; group_top: a group scores by the sum of its group_top best choice
        scores; act: "silu" -- silu(gate) up --, or "swish_clamp" -- g sigmoid(act_alpha g) (u + 1) with g = min(gate, limit),
        u = clamp(up, -limit, limit)"""
        if score not in seqops.ROUTER_SCORES or act not in ("silu", "swish_clamp") or group_top < 1:
            raise ZLError("experts: unknown score function or activation")
        self.score, self.group_top, self.renorm_eps, self.act, self.act_alpha, self.limit = score, int(group_top), float(renorm_eps), act, \
            float(act_alpha), float(limit)
        self.weight_scale = float(weight_scale)
        self.has_router_bias, self.shared_ff, self.shared_gate = bool(router_bias), int(shared_ff), bool(shared_gate)
        self.router_b = self.w_shared_down = None
        total = experts + identity
        if groups < 1 or total % groups or not 1 <= keep <= groups or top > keep * (total // groups):
            raise ZLError("experts: groups must divide the router outputs, and the kept groups must hold `top` outputs")
        self.width, self.ff, self.experts, self.top, self.identity = width, ff, experts, top, identity
        self.groups, self.keep, self.has_correction, self.renorm = groups, keep, correction, renorm
        self.packed = ff % 16 == 0                       # gate / up rows in blocks of 16: what the gated epilogue reads
        self.fused_act = self.packed                     # (the grouped product's epilogue finishes the activation)
        self.few_rows = seqops.MOE_FEW_ROWS
        self.tile_m = None                # rows per expert tile of the grouped products (None: by the experts' average share)

    def _pack_gate_up(self, gate, up):
        if not self.packed:
            return torch.cat([gate, up], dim=0)
        f, w = gate.shape
        return torch.stack([gate.reshape(f // 16, 16, w), up.reshape(f // 16, 16, w)], dim=1).reshape(2 * f, w)

    def _join_shared(self, gate, up, down, sg):
        """the shared expert's rows join the router's product: [router | shared gates | shared ups | the shared expert's own gate]"""
        self.shared_col = self.w_router.shape[0]
        self.w_router = torch.cat([self.w_router, gate, up] + ([sg] if sg is not None else []), dim=0).contiguous()
        self.w_shared_down = down

    def load(self, get, prefix, dtype, device):
        E, f, W = self.experts, self.ff, self.width
        self.w_router = _mat(get, prefix + "router", (E + self.identity, W), dtype, device)
        self.correction = _vec(get, prefix + "correction", E + self.identity, device) if self.has_correction else None
        self.router_b = _vec(get, prefix + "router.b", E + self.identity, device) if self.has_router_bias else None
        if self.shared_ff:
            p, sf = prefix + "shared.", self.shared_ff
            self._join_shared(_mat(get, p + "gate", (sf, W), dtype, device), _mat(get, p + "up", (sf, W), dtype, device),
                              _mat(get, p + "down", (W, sf), dtype, device), _mat(get, p + "sg", (1, W), dtype, device) if self.shared_gate else None)
        self.w_gu = torch.empty((E, 2 * f, W), dtype=dtype, device=device)
        self.w_down = torch.empty((E, W, f), dtype=dtype, device=device)
        for e in range(E):
            p = f"{prefix}e{e}."
            self.w_gu[e] = self._pack_gate_up(_mat(get, p + "gate", (f, W), dtype, device), _mat(get, p + "up", (f, W), dtype, device))
            self.w_down[e] = _mat(get, p + "down", (W, f), dtype, device)
        return self

    def init_random(self, gen, dtype, device):
        E, f, W = self.experts, self.ff, self.width
        self.w_router = _rand(gen, (E + self.identity, W), W ** -0.5, dtype, device)
        self.correction = torch.zeros(E + self.identity, device=device) if self.has_correction else None
        self.router_b = torch.zeros(E + self.identity, device=device) if self.has_router_bias else None
        if self.shared_ff:
            sf = self.shared_ff
            self._join_shared(_rand(gen, (sf, W), W ** -0.5, dtype, device), _rand(gen, (sf, W), W ** -0.5, dtype, device),
                              _rand(gen, (W, sf), sf ** -0.5, dtype, device), _rand(gen, (1, W), W ** -0.5, dtype, device) if self.shared_gate else None)
        self.w_gu = _rand(gen, (E, 2 * f, W), W ** -0.5, dtype, device)
        self.w_down = _rand(gen, (E, W, f), f ** -0.5, dtype, device)
        return self

    def weight_bytes(self):
        return sum(t.numel() * t.element_size() for t in (self.w_router, self.w_gu, self.w_down, self.w_shared_down) if t is not None)

    def forward(self, h):
        logits = seqops.gemm_nt(h, self.w_router)                                 # fp32 sums of the products [router | shared expert | side rows]
        self.side = (logits, self.side_col0)
        ids, weights = seqops.moe_route(logits, self.correction, self.groups, self.keep, self.top, self.renorm, score=self.score,
                                        group_top=self.group_top, renorm_eps=self.renorm_eps, weight_scale=self.weight_scale,
                                        n_out=self.experts + self.identity, logit_bias=self.router_b)
        sorted_tok, slot_pos, tiles, max_tiles, sorted_exp, tm = seqops.moe_align(ids, self.experts, self.tile_m)
        n_slots = ids.numel()
        few = sorted_exp if n_slots <= self.few_rows else None                    # decode steps: weight rows streamed per (row, column)
        if self.fused_act:
            a = seqops.gemm_nt_grouped(h, sorted_tok, self.w_gu, tiles, max_tiles, n_slots, gated=True, out_dtype=h.dtype, row_expert=few, tile_m=tm,
                                       act=self.act, act_alpha=self.act_alpha, act_limit=self.limit)
        else:
            a = seqops.act_mul(seqops.gemm_nt_grouped(h, sorted_tok, self.w_gu, tiles, max_tiles, n_slots, row_expert=few, tile_m=tm), h.dtype,
                               kind=self.act, alpha=self.act_alpha, limit=self.limit, block=16 if self.packed else 0)
        y = seqops.gemm_nt_grouped(a, None, self.w_down, tiles, max_tiles, n_slots, row_expert=few, tile_m=tm)
        if not self.shared_ff:
            return seqops.moe_combine(y, slot_pos, ids, weights, h, self.experts)
        s = seqops.gemm_nt(seqops.act_mul(logits, h.dtype, kind=self.act, alpha=self.act_alpha, limit=self.limit, col0=self.shared_col, ff=self.shared_ff),
                           self.w_shared_down)
        return seqops.moe_combine(y, slot_pos, ids, weights, h, self.experts, shared=s, gate=logits if self.shared_gate else None,
                                  g_col=self.shared_col + 2 * self.shared_ff)
