"""A plain float64 restatement of the Suvapel design, one function per mechanism, whole sequences at a time, no cache and no batching.

It shares no code with zhilight_amd: the product path (suvapel.py, mixers.py, the kernels) is held against it.  `weights` is a mapping
name -> tensor with the names of the checkpoint ("l<i>.mix.q", "l<i>.mix.left.q.conv", "l<i>.mlp.gate.b", "side.embed", ...); `cfg` is the
dictionary of config.json.

Notation: T tokens at positions 0 .. T-1, h (T, width) a sub-layer's input, matrices stored (out, in).
"""
import math

import torch

F64 = torch.float64


def _w(weights, name):
    return weights[name].to(F64)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def tanh_norm(x, alpha, w, b):
    """no statistics of the row: tanh(alpha x) w + b"""
    return torch.tanh(alpha * x) * w + b


def model_norm(x, weights, name):
    return tanh_norm(x, _w(weights, name + ".alpha"), _w(weights, name), _w(weights, name + ".b"))


def causal_conv(u, w):
    """(T, C), w (C, taps): out[t, c] = sum_j w[c, j] u[t - taps + 1 + j, c], zeros before the start"""
    T, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F64), u])
    out = torch.zeros_like(u)
    for j in range(taps):
        out = out + pad[j:j + T] * w[:, j]
    return out


# ---- attention -------------------------------------------------------------------------------------------------------------------------
def frequencies(rot):
    """(f (dims / 2), gain): plain base^(-2i / dims) or rescaled for long contexts"""
    n, base, s = int(rot["dims"]), float(rot["base"]), rot.get("scaling")
    f = torch.tensor([base ** (-2.0 * i / n) for i in range(n // 2)], dtype=F64)
    if not s:
        return f, 1.0
    at = lambda turns: n * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(at(s["fast"])), 0), min(math.ceil(at(s["slow"])), n - 1)
    out = []
    for i in range(n // 2):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f[i] / s["factor"] * r + f[i] * (1.0 - r))
    return torch.stack(out), 0.1 * math.log(s["factor"]) + 1.0


def rotate_half(x, pos, f, gain):
    """x (T, heads, dim): coordinates i and i + n/2 (n = 2 len(f)) turned by pos * f_i, the others unchanged"""
    half = f.shape[0]
    a = pos.to(F64)[:, None, None] * f
    c, s = torch.cos(a) * gain, torch.sin(a) * gain
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], dim=-1)


def visible(T, size, keep_first):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    if not size:
        return j <= i
    return (j <= i) & ((i - j < size) | (j < keep_first))


def softmax_attention(q, k, v, scale, mask):
    """q (T, H, d), k (T, G, d), v (T, G, vd): query head h reads key / value head h // (H / G)"""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        s = (q[:, h] @ k[:, h // rep].T) * scale
        s = torch.where(mask, s, torch.full_like(s, -math.inf))
        out[:, h] = torch.softmax(s, dim=-1) @ v[:, h // rep]
    return out


def attention(h, weights, p, m):
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_conv(h @ _w(weights, p + n).T, _w(weights, p + n + ".conv")) for n in "qkv")
    q, k, v = q.reshape(T, H, d), k.reshape(T, G, d), v.reshape(T, G, vd)
    f, gain = frequencies(m["rot"])
    pos = torch.arange(T)
    q, k = rotate_half(q, pos, f, gain), rotate_half(k, pos, f, gain)
    o = softmax_attention(q, k, v, m["scale"], visible(T, m["mask"]["size"], m["mask"].get("keep_first", 0)))
    o = o * sigmoid(h @ _w(weights, p + "g").T)[:, :, None]
    return o.reshape(T, H * vd) @ _w(weights, p + "o").T


# ---- gated delta rule ------------------------------------------------------------------------------------------------------------------
def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, beta, g):
    """q, k, g (T, H, d), v (T, H, vd), beta (T, H): S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q"""
    T, H, d = k.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def delta_mixer(h, weights, p, m, eps, per_channel):
    """per_channel: a decay per head and key channel from a low-rank pair, a sigmoid output gate from another; otherwise a decay per head, a
    silu output gate"""
    T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ _w(weights, p + n).T, _w(weights, p + n + ".conv"))) for n in "qkv")
    spread = torch.arange(H) // (H // G)
    q, k = unit_vector(q.reshape(T, G, d))[:, spread] * d ** -0.5, unit_vector(k.reshape(T, G, d))[:, spread]
    beta = sigmoid(h @ _w(weights, p + "b").T)
    rate = torch.exp(_w(weights, p + "A_log"))
    if per_channel:
        z = (h @ _w(weights, p + "a1").T) @ _w(weights, p + "a2").T + _w(weights, p + "dt_bias")
        g = torch.exp(-rate[None, :, None] * softplus(z.reshape(T, H, d)))
        gate = sigmoid((h @ _w(weights, p + "g1").T) @ _w(weights, p + "g2").T)
    else:
        g = torch.exp(-rate * softplus(h @ _w(weights, p + "a").T + _w(weights, p + "dt_bias")))[:, :, None].expand(T, H, d)
        gate = silu(h @ _w(weights, p + "g").T)
    o = delta_recurrence(q, k, v.reshape(T, H, vd), beta, g)
    o = unit_rms(o, eps) * _w(weights, p + "norm") * gate.reshape(T, H, vd)
    return o.reshape(T, H * vd) @ _w(weights, p + "o").T


# ---- feed-forward, per-layer token input -----------------------------------------------------------------------------------------------
def dense_ff(h, weights, p):
    gate = h @ _w(weights, p + "gate").T + _w(weights, p + "gate.b")
    up = h @ _w(weights, p + "up").T + _w(weights, p + "up.b")
    return (silu(gate) * up) @ _w(weights, p + "down").T + _w(weights, p + "down.b")


def token_side(x, e, weights, p, mult, eps):
    """x + mult * N(proj(gelu(gate x) * e)), N an RMS norm with a weight"""
    y = (gelu_tanh(x @ _w(weights, p + "gate").T) * e) @ _w(weights, p + "proj").T
    return x + mult * unit_rms(y, eps) * _w(weights, p + "norm")


# ---- the model -------------------------------------------------------------------------------------------------------------------------
def mixer(h, weights, p, layer, eps):
    m = layer["mixer"]
    if layer["type"] == "delta":
        return delta_mixer(h, weights, p, m, eps, per_channel=False)
    return m["left_scale"] * attention(h, weights, p + "left.", m["left"]) + \
        m["right_scale"] * delta_mixer(h, weights, p + "right.", m["right"], eps, per_channel=True)


def forward(tokens, weights, cfg, keep=None):
    """tokens (T) -> logits (T, vocab); keep: a list that receives the residual after every layer"""
    eps, mult, dim = cfg["norm"]["eps"], cfg["residual_mult"], cfg["token_side"]["dim"]
    tokens = torch.as_tensor(tokens, dtype=torch.int64)
    x = _w(weights, "embed")[tokens]
    side = _w(weights, "side.embed")[tokens]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = model_norm(x, weights, p + "norm1")
        y = mixer(h, weights, p + "mix.", layer, eps)
        if layer.get("mlp") is not None:
            y = y + dense_ff(h, weights, p + "mlp.")
        x = x + mult * y
        x = token_side(x, side[:, i * dim:(i + 1) * dim], weights, p + "side.", mult, eps)
        if keep is not None:
            keep.append(x.clone())
    return model_norm(x, weights, "final.norm") @ _w(weights, "head").T


# ---- test weights ------------------------------------------------------------------------------------------------------------------------
def random_weights(cfg, seed=0):
    """every tensor the configuration asks for, bf16-representable values (both serving formats start from the same numbers).  Key
    projections and convolutions lean towards the queries': a sequence's first delta-rule output is (q . k) v over its own root mean square, whose
    SIGN hangs on a product that random matrices let come close to zero."""
    g = torch.Generator().manual_seed(seed)
    W, sd = cfg["width"], {}

    def mat(name, rows, cols, std=None):
        sd[name] = (torch.randn(rows, cols, generator=g) * (std if std is not None else cols ** -0.5)).to(torch.bfloat16)

    def vec(name, n, std=0.2, mean=0.0):
        sd[name] = (mean + std * torch.randn(n, generator=g)).to(torch.bfloat16)

    def norm(name):
        vec(name, W, 0.2, 1.0)
        vec(name + ".b", W, 0.2)
        sd[name + ".alpha"] = torch.tensor(0.4 + 0.4 * float(torch.rand(1, generator=g))).to(torch.bfloat16)

    def conv(name, rows, taps):
        sd[name] = (0.4 * torch.randn(rows, taps, generator=g)).to(torch.bfloat16)
        sd[name][:, -1] += 0.7

    def delta(p, m, per_channel):
        H, G, d, e, low = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m.get("low", 10)
        for n, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
            mat(p + n, rows, W, 1.5 * W ** -0.5)
            conv(p + n + ".conv", rows, m["conv"])
        sd[p + "k"] = (0.9 * sd[p + "q"].float() + 0.4 * sd[p + "k"].float()).to(torch.bfloat16)
        sd[p + "k.conv"] = (sd[p + "q.conv"].float() + 0.2 * sd[p + "k.conv"].float()).to(torch.bfloat16)
        mat(p + "b", H, W)
        sd[p + "A_log"] = (torch.rand(H, generator=g) * 2.5 - 1.5).to(torch.bfloat16)
        vec(p + "norm", e, 0.2, 1.0)
        if per_channel:
            mat(p + "a1", low, W)
            mat(p + "a2", H * d, low)
            vec(p + "dt_bias", H * d, 1.2, -3.0)
            mat(p + "g1", low, W)
            mat(p + "g2", H * e, low)
        else:
            mat(p + "a", H, W)
            vec(p + "dt_bias", H, 1.0, -3.0)
            mat(p + "g", H * e, W)
        mat(p + "o", W, H * e)

    mat("embed", cfg["vocab"], W, 1.0)
    mat("side.embed", cfg["vocab"], len(cfg["layers"]) * cfg["token_side"]["dim"], 1.0)
    mat("head", cfg["vocab"], W)
    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        norm(p + "norm1")
        if l["type"] == "delta":
            delta(p + "mix.", m, False)
        else:
            a = m["left"]
            H, G, d, e = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * e)):
                mat(p + "mix.left." + n, rows, W)
                conv(p + "mix.left." + n + ".conv", rows, a["conv"])
            mat(p + "mix.left.g", H, W)
            mat(p + "mix.left.o", W, H * e)
            delta(p + "mix.right.", m["right"], True)
        if l.get("mlp") is not None:
            ff = l["mlp"]["ff"]
            for n in ("gate", "up"):
                mat(p + "mlp." + n, ff, W)
                vec(p + "mlp." + n + ".b", ff, 0.3)
            mat(p + "mlp.down", W, ff)
            vec(p + "mlp.down.b", W, 0.3)
        dim = cfg["token_side"]["dim"]
        mat(p + "side.gate", dim, W)
        mat(p + "side.proj", W, dim)
        vec(p + "side.norm", W, 0.2, 1.0)
    return sd
