"""A plain float64 restatement of the Zasazen design, one function per mechanism, whole sequences at a time, no cache and no batching.

It shares no code with zhilight_amd: the product path (zasazen.py, mixers.py, the kernels) is held against it.  `weights` is a mapping
name -> tensor with the names of the checkpoint ("l<i>.mix.in", "l<i>.mix.left.q", "l<i>.mlp.e<j>.gate", "loop.in", ...); `cfg` is the
dictionary of config.json.

Notation: T tokens at positions 0 .. T-1, h (T, width) a sub-layer's input, matrices stored (out, in).
"""
import math

import torch

F64 = torch.float64


def _w(weights, name):
    return weights[name].to(F64)


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis"""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- selective state space -----------------------------------------------------------------------------------------------------------
def causal_conv(u, w, b):
    """(T, C): out[t, c] = b[c] + sum_k w[c, k] u[t - (taps - 1) + k, c], zeros before the start"""
    T, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=F64), u])
    out = b[None, :].expand(T, -1).clone()
    for k in range(taps):
        out = out + pad[k:k + T] * w[:, k]
    return out


def selective_scan(x, dt, A, B, C, D):
    """x, dt (T, inner), A (inner, N) negative, B, C (T, N), D (inner):
    S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;  y_c = sum_n S[c, n] C_n + D_c x_c"""
    S = torch.zeros_like(A)
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        out[t] = (S * C[t][None, :]).sum(-1) + D * x[t]
    return out


def mamba1_mixer(h, weights, p, m, eps):
    inner, N, R = m["inner"], m["state"], m["dt_rank"]
    xz = h @ _w(weights, p + "in").T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, _w(weights, p + "conv"), _w(weights, p + "conv.b")))
    low = x @ _w(weights, p + "x").T
    dt = softplus(low[:, :R] @ _w(weights, p + "dt").T + _w(weights, p + "dt.b"))
    y = selective_scan(x, dt, -torch.exp(_w(weights, p + "A_log")), low[:, R:R + N], low[:, R + N:], _w(weights, p + "D"))
    return (y * silu(z)) @ _w(weights, p + "o").T


# ---- attention with a linear distance bias ---------------------------------------------------------------------------------------------
def slopes(H):
    return [2.0 ** (-8.0 * (a + 1) / H) for a in range(H)]


def query_temperature(T, coef, every):
    p = torch.arange(T)
    return 1.0 + coef * torch.log((p + 1).div(every, rounding_mode="floor").to(F64) + 1.0)


def sloped_attention(q, k, v, scale):
    """q (T, H, d), k (T, G, d), v (T, G, e), causal; head a reads kv head a // (H / G); softmax over q.k * scale - slope_a (i - j)"""
    T, H, _ = q.shape
    G = k.shape[1]
    i = torch.arange(T, dtype=F64)
    dist = i[:, None] - i[None, :]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * scale - slopes(H)[a] * dist
        out[:, a] = torch.softmax(s.masked_fill(dist < 0, -math.inf), -1) @ v[:, g]
    return out


def left_branch(h, weights, p, m, eps):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ _w(weights, p + n).T + _w(weights, p + n + ".b") for n in ("q", "k", "v"))
    q, k = rms_norm(q, _w(weights, p + "q.norm"), eps), rms_norm(k, _w(weights, p + "k.norm"), eps)
    t = m.get("q_temp")
    if t:
        q = q * query_temperature(T, float(t["coef"]), int(t["every"]))[:, None]
    o = sloped_attention(q.reshape(T, H, d), k.reshape(T, G, d), v.reshape(T, G, e), float(m["scale"]))
    return o.reshape(T, H * e) @ _w(weights, p + "o").T


# ---- retention -------------------------------------------------------------------------------------------------------------------------
def rotate_half(x, dims, base):
    """x (T, heads, size): coordinate i < dims/2 pairs with i + dims/2, the pair at position p turned by p * base^(-2i/dims)"""
    if not dims:
        return x
    out = x.clone()
    f = torch.pow(torch.tensor(float(base), dtype=F64), -2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    ang = torch.arange(x.shape[0], dtype=F64)[:, None] * f[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    out[..., :dims // 2] = u * c - v * s
    out[..., dims // 2:dims] = v * c + u * s
    return out


def retention(q, k, v, decay):
    """q, k (T, H, d), v (T, H, e): S <- decay_a S + k v^T, o = S^T q per head"""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    a = torch.tensor([float(x) for x in decay], dtype=F64)[:, None, None]
    for t in range(T):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out


def right_branch(h, weights, p, m, eps):
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m["vdim"]
    rot = m.get("rot") or {}
    q, k = ((rotate_half((h @ _w(weights, p + n).T).reshape(T, H, d), int(rot.get("dims", 0)), rot.get("base", 1.0))) for n in ("q", "k"))
    v = (h @ _w(weights, p + "v").T).reshape(T, H, e)
    o = unit_rms(retention(q, k * d ** -0.5, v, m["decay"]), eps).reshape(T, H * e)
    return (o * silu(h @ _w(weights, p + "g").T)) @ _w(weights, p + "o").T


def parallel_mixer(h, weights, p, m, eps):
    left = rms_norm(left_branch(h, weights, p + "left.", m["left"], eps), _w(weights, p + "left.out"), eps)
    right = rms_norm(right_branch(h, weights, p + "right.", m["right"], eps), _w(weights, p + "right.out"), eps)
    return 0.5 * (left + right)


# ---- feed-forwards ---------------------------------------------------------------------------------------------------------------------
def dense_ff(h, weights, p):
    return gelu_tanh(h @ _w(weights, p + "up").T) @ _w(weights, p + "down").T


def gated_ff(h, weights, p):
    return (silu(h @ _w(weights, p + "gate").T) * (h @ _w(weights, p + "up").T)) @ _w(weights, p + "down").T


def route(h, weights, p, top, margins=None):
    """(ids (T, top), weights (T, top)): the largest logits (with the router's bias), a softmax over the chosen ones.  margins (a list)
    receives the smallest gap between the last chosen and the first unchosen logit"""
    z = h @ _w(weights, p + "router").T + _w(weights, p + "router.b")
    order = z.sort(-1, descending=True)
    if margins is not None and top < z.shape[1]:
        margins.append(float((order.values[:, top - 1] - order.values[:, top]).min()))
    return order.indices[:, :top], torch.softmax(order.values[:, :top], -1)


def experts_ff(h, weights, p, f, margins=None):
    ids, wts = route(h, weights, p, int(f["router"]["top"]), margins)
    out = torch.zeros(h.shape[0], _w(weights, p + "e0.down").shape[0], dtype=F64)
    for t in range(h.shape[0]):
        for c in range(ids.shape[1]):
            out[t] += wts[t, c] * gated_ff(h[t], weights, p + "e%d." % int(ids[t, c]))
    if f.get("shared"):
        gate = 1.0 / (1.0 + torch.exp(-(h @ _w(weights, p + "shared.sg").T)))
        out = out + gate * gated_ff(h, weights, p + "shared.")
    return out


# ---- layers ----------------------------------------------------------------------------------------------------------------------------
MIXERS = {"mamba1": mamba1_mixer, "parallel": parallel_mixer}


def layer(x, weights, i, l, eps, margins=None):
    p = f"l{i}."
    y = MIXERS[l["type"]](rms_norm(x, _w(weights, p + "norm1"), eps), weights, p + "mix.", l["mixer"], eps)
    f = l.get("mlp")
    if f is None:
        return x + y
    h = rms_norm(x, _w(weights, p + "norm2"), eps)
    return x + (y + (dense_ff(h, weights, p + "mlp.") if f["kind"] == "dense" else experts_ff(h, weights, p + "mlp.", f, margins)))


def runs(cfg):
    """[(layer, pass)]: the layers before the loop, the looped ones `times` times in a row, the rest; pass is None outside the loop"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    return [(i, None) for i in range(a)] + [(i, t) for t in range(int(loop["times"])) for i in range(a, b)] + [(i, None) for i in range(b, n)]


def model(tokens, weights, cfg, keep_layers=None, margins=None):
    """logits (T, vocab) of one sequence; keep_layers: a list that receives x after every layer run; margins: see route"""
    eps = float(cfg["norm"]["eps"])
    x0 = _w(weights, "embed")[torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    x = x0
    for i, t in runs(cfg):
        if t is not None and i == int(cfg["loop"]["start"]):
            x = torch.cat([x, x0], -1) @ _w(weights, "loop.in").T + _w(weights, "loop.step")[t]
        x = layer(x, weights, i, cfg["layers"][i], eps, margins)
        if keep_layers is not None:
            keep_layers.append(x)
    return rms_norm(x, _w(weights, "final.norm"), eps) @ _w(weights, "head").T


# ---- test weights ------------------------------------------------------------------------------------------------------------------------
def random_weights(cfg, seed=0, fixed_choice=False):
    """every tensor the configuration asks for, bf16-representable values (both serving formats start from the same numbers).
    fixed_choice: the routers read ONE reserved coordinate of the residual only -- coordinate 0 of the embedding holds a number whose sign
    and size the token decides, no sub-layer writes to it and the loop's entry copies it -- with evenly spaced multiples per expert, so
    that the order of the logits is one fixed order or its reverse, with wide gaps: no choice is a close call under a rounded router input.
    The retention's key matrices then also lean towards its query matrices: a sequence's first output is (q . k) v / rms, whose SIGN hangs on
    a product that random matrices let come close to zero."""
    g = torch.Generator().manual_seed(seed)
    W, scale = cfg["width"], float(cfg["embedding"]["scale"])
    sd = {}

    def mat(name, rows, cols, std=None):
        sd[name] = (torch.randn(rows, cols, generator=g) * (std if std is not None else cols ** -0.5)).to(torch.bfloat16)

    def vec(name, n, std=0.2, mean=0.0):
        sd[name] = (mean + std * torch.randn(n, generator=g)).to(torch.bfloat16)

    mat("embed", cfg["vocab"], W, 1.5 / scale)
    if fixed_choice:
        size = (4.0 + 4.0 * torch.rand(cfg["vocab"], generator=g)) / scale
        sd["embed"][:, 0] = torch.where(torch.arange(cfg["vocab"]) % 3 == 0, -size, size).to(torch.bfloat16)
    mat("head", cfg["vocab"], W)
    vec("final.norm", W, 0.2, 1.0)
    if cfg.get("loop"):
        mat("loop.in", W, 2 * W)
        mat("loop.step", int(cfg["loop"]["times"]), W, 0.3)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        vec(p + "norm1", W, 0.2, 1.0)
        if l["type"] == "mamba1":
            C, N, R = m["inner"], m["state"], m["dt_rank"]
            mat(p + "mix.in", 2 * C, W)
            mat(p + "mix.conv", C, m["conv"], m["conv"] ** -0.5)
            vec(p + "mix.conv.b", C, 0.3)
            mat(p + "mix.x", R + 2 * N, C, 1.5 * C ** -0.5)
            mat(p + "mix.dt", C, R)
            vec(p + "mix.dt.b", C, 1.2, -1.5)
            sd[p + "mix.A_log"] = (torch.rand(C, N, generator=g) * 4.0 - 2.5).to(torch.bfloat16)
            vec(p + "mix.D", C, 0.3, 1.0)
            mat(p + "mix.o", W, C)
        else:
            a, r = m["left"], m["right"]
            H, G, d, e = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * e)):
                mat(p + "mix.left." + n, rows, W)
                vec(p + "mix.left." + n + ".b", rows, 0.5)
            vec(p + "mix.left.q.norm", H * d, 0.3, 1.3)
            vec(p + "mix.left.k.norm", G * d, 0.3, 1.3)
            mat(p + "mix.left.o", W, H * e)
            H, d, e = r["heads"], r["dim"], r["vdim"]
            for n, rows in (("q", H * d), ("k", H * d), ("v", H * e), ("g", H * e)):
                mat(p + "mix.right." + n, rows, W)
            if fixed_choice:
                sd[p + "mix.right.k"] = (0.8 * sd[p + "mix.right.q"].float() + 0.5 * sd[p + "mix.right.k"].float()).to(torch.bfloat16)
            mat(p + "mix.right.o", W, H * e)
            vec(p + "mix.left.out", W, 0.2, 1.0)
            vec(p + "mix.right.out", W, 0.2, 0.8)
        f = l.get("mlp")
        if f is None:
            continue
        vec(p + "norm2", W, 0.2, 0.9)
        if f["kind"] == "dense":
            mat(p + "mlp.up", f["ff"], W)
            mat(p + "mlp.down", W, f["ff"])
            continue
        E = f["router"]["experts"]
        mat(p + "mlp.router", E, W, 2.0 * W ** -0.5)
        vec(p + "mlp.router.b", E, 0.5)
        if fixed_choice:
            q = torch.zeros(E, W)
            q[:, 0] = 1.6 * torch.randperm(E, generator=g).double() - 0.8 * E
            sd[p + "mlp.router"] = q.to(torch.bfloat16)
            sd[p + "mlp.router.b"] = (0.1 * sd[p + "mlp.router.b"].float()).to(torch.bfloat16)
        names = [(f"e{j}.", f["expert"]["ff"]) for j in range(E)] + ([("shared.", f["shared"]["ff"])] if f.get("shared") else [])
        for n, ff in names:
            mat(p + "mlp." + n + "gate", ff, W)
            mat(p + "mlp." + n + "up", ff, W)
            mat(p + "mlp." + n + "down", W, ff)
        if f.get("shared"):
            mat(p + "mlp.shared.sg", 1, W)
    if fixed_choice:
        for name, t in sd.items():
            if name.endswith((".mix.o", ".left.o", ".right.o", ".down")):
                t[:1] = 0.0
        if "loop.in" in sd:
            sd["loop.in"][0] = 0.0
            sd["loop.in"][0, W] = 1.0
            sd["loop.step"][:, 0] = 0.0
    return sd
