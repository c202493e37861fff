"""Plain, slow Tebasun in float64: the yardstick of the Tebasun tests.

One function per mechanism, straight from the equations, token by token
where there is a recurrence. Works on the raw checkpoint (tensor name ->
tensor, unpadded) and the raw config dict, and shares no code with
distllm_amd.
"""

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-abs(z))) + torch.clamp(z, min=0)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi)
                                     * (z + 0.044715 * z ** 3)))


def rms(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def unit(x, eps=1e-6):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + eps)


def dyt(x, t, name):
    return torch.tanh(t[name + ".alpha"] * x) * t[name] + t[name + ".b"]


def embedding(t, tokens, scale):
    return t["embed"][tokens] * scale


def causal_conv(x, w):
    """x [T, C], w [C, taps]; the last column is the current token's."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for back in range(taps):
        if back < T:
            out[back:] += x[: T - back] * w[:, taps - 1 - back]
    return out


# ---- rotary attention ------------------------------------------------------

def frequencies(rot):
    """-> frequency of every pair, and the factor on cos and sin."""
    n, base = rot["dims"], rot["base"]
    f = [base ** (-2 * i / n) for i in range(n // 2)]
    s = rot.get("scaling")
    if s is None:
        return torch.tensor(f, dtype=F64), 1.0

    def dim(turns):
        return n * math.log(s["original"] / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(dim(s["fast"])), 0)
    hi = min(math.ceil(dim(s["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0), 1)
        out.append(fi / s["factor"] * ramp + fi * (1 - ramp))
    return (torch.tensor(out, dtype=F64),
            0.1 * math.log(s["factor"]) + 1)


def rotate(x, pos, rot):
    """x [T, heads, dim] at positions pos [T]."""
    f, mult = frequencies(rot)
    half = rot["dims"] // 2
    a = pos.to(F64)[:, None] * f
    c, s = torch.cos(a)[:, None] * mult, torch.sin(a)[:, None] * mult
    u, v = x[..., :half], x[..., half: 2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def attention(h, t, pre, m, eps):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ t[pre + "q"].T + t[pre + "q.b"]).view(T, H, d)
    v = (h @ t[pre + "k"].T + t[pre + "k.b"]).view(T, G, d)
    pos = torch.arange(T)
    q = rotate(rms(q, t[pre + "q.norm"], eps), pos, m["rot"])
    k = rotate(rms(v, t[pre + "k.norm"], eps), pos, m["rot"])
    out = torch.zeros(T, H, d, dtype=h.dtype)
    for n in range(H):
        g = n // (H // G)
        s = q[:, n] @ k[:, g].T * m["scale"]
        s = torch.where(pos[None] <= pos[:, None], s, -math.inf)
        out[:, n] = softmax_with_sink(s, t[pre + "sink"][n]) @ v[:, g]
    return out.reshape(T, -1) @ t[pre + "o"].T + t[pre + "o.b"]


def softmax_with_sink(s, sink):
    """Rows of weights; the sink takes its share of the denominator."""
    top = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


# ---- delta rule with a decay per key channel -------------------------------

def delta_inputs(h, t, pre, m):
    """-> q, k [T, H, dim], v [T, H, vdim], beta [T, H], g [T, H, dim]."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]

    def short(name):
        return silu(causal_conv(h @ t[pre + name].T,
                                t[pre + name + ".conv"]))

    own = torch.arange(H) // (H // G)
    q = unit(short("q").view(T, G, -1))[:, own] * m["dim"] ** -0.5
    k = unit(short("k").view(T, G, -1))[:, own]
    v = short("v").view(T, H, -1)
    beta = sigmoid(h @ t[pre + "b"].T)
    a = h @ t[pre + "a1"].T @ t[pre + "a2"].T + t[pre + "dt_bias"]
    g = torch.exp(-torch.exp(t[pre + "A_log"])[:, None]
                  * softplus(a).view(T, H, -1))
    return q, k, v, beta, g


def delta_step(S, q, k, v, beta, g):
    """One token of one head; S [dim, vdim]. -> state, read-out."""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + k[:, None] * u[None]
    return S, S.T @ q


def delta(h, t, pre, m, eps):
    T, H = h.shape[0], m["heads"]
    q, k, v, beta, g = delta_inputs(h, t, pre, m)
    o = torch.zeros(T, H, m["vdim"], dtype=h.dtype)
    for n in range(H):
        S = torch.zeros(m["dim"], m["vdim"], dtype=h.dtype)
        for i in range(T):
            S, o[i, n] = delta_step(S, q[i, n], k[i, n], v[i, n],
                                    beta[i, n], g[i, n])
    gate = sigmoid(h @ t[pre + "g1"].T @ t[pre + "g2"].T)
    o = rms(o, t[pre + "norm"], eps).reshape(T, -1) * gate
    return o @ t[pre + "o"].T


def parallel(h, t, pre, m, eps):
    return (m["left_scale"] * attention(h, t, pre + "left.", m["left"], eps)
            + m["right_scale"] * delta(h, t, pre + "right.", m["right"],
                                       eps))


# ---- real-gated linear recurrent unit --------------------------------------

def lru_gates(u, t, pre):
    """-> log of the decay and input gate, [T, width]."""
    def blockwise(name):
        w = t[pre + name]                                  # [B, s, s]
        z = (w[None] @ u.view(u.shape[0], w.shape[0], -1, 1))[..., 0]
        return sigmoid(z + t[pre + name + ".b"]).reshape(u.shape)

    return -8 * blockwise("ra") * softplus(t[pre + "lam"]), blockwise("ri")


def rglru(h, t, pre, m, eps):
    y = gelu_tanh(h @ t[pre + "y"].T + t[pre + "y.b"])
    u = causal_conv(h @ t[pre + "x"].T + t[pre + "x.b"], t[pre + "conv"]) \
        + t[pre + "conv.b"]
    log_a, i = lru_gates(u, t, pre)
    a = torch.exp(log_a)
    drive = torch.sqrt(1 - a * a) * i * u
    S = torch.zeros(u.shape[1], dtype=h.dtype)
    out = torch.zeros_like(u)
    for n in range(h.shape[0]):
        S = a[n] * S + drive[n]
        out[n] = S
    return (out * y) @ t[pre + "o"].T


# ---- the rest of a layer ---------------------------------------------------

def dense(h, t, pre):
    return (silu(h @ t[pre + "gate"].T) * (h @ t[pre + "up"].T)) \
        @ t[pre + "down"].T


def side(x, t, i, dim, tokens, eps):
    """What the per-layer token input adds to x."""
    pre = f"l{i}.side."
    e = t["side.embed"][tokens][:, i * dim: (i + 1) * dim]
    y = (gelu_tanh(x @ t[pre + "gate"].T) * e) @ t[pre + "proj"].T
    return rms(y, t[pre + "norm"], eps)


MIXERS = {"parallel": parallel, "rglru": rglru}


def layer(x, t, cfg, i, tokens):
    entry, eps, pre = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    x = x + MIXERS[entry["type"]](dyt(x, t, pre + "norm1"), t, pre + "mix.",
                                  entry["mixer"], eps)
    if entry["mlp"] is not None:
        x = x + dense(dyt(x, t, pre + "norm2"), t, pre + "mlp.")
    return x + side(x, t, i, cfg["token_side"]["dim"], tokens, eps)


def layer_runs(cfg):
    """(layer, pass it starts or None) in running order."""
    loop, runs = cfg["loop"], []
    runs += [(i, None) for i in range(loop["start"])]
    for p in range(loop["times"]):
        runs += [(i, p if i == loop["start"] else None)
                 for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"],
                                            len(cfg["layers"]))]


@torch.no_grad()
def forward(cfg, tensors, tokens, trace=None):
    """Logits [T, vocab] of one sequence; trace collects the residual
    stream after every layer run."""
    t = {k: v.to(F64) for k, v in tensors.items()}
    tokens = torch.as_tensor(tokens)
    x0 = embedding(t, tokens, cfg["embedding"]["scale"])
    x = x0
    for i, start in layer_runs(cfg):
        if start is not None:
            if start > 0:
                x = x + x0
            x = x + t["loop.step"][start]
        x = layer(x, t, cfg, i, tokens)
        if trace is not None:
            trace.append(x.clone())
    return dyt(x, t, "final.norm") @ t["embed"].T


# ---- small configurations and weights --------------------------------------

def rotation(dims=8, base=1000.0, factor=4.0, original=16, fast=4.0,
             slow=0.5):
    return {"base": base, "dims": dims,
            "scaling": {"factor": factor, "fast": fast,
                        "original": original, "slow": slow}}


def dense_mlp(ff=48):
    return {"kind": "dense", "ff": ff}


def parallel_layer(mlp, heads=4, kv_heads=2, dim=16, rot=None, scale=0.4,
                   left_scale=0.7, right_scale=0.9, right=None):
    right = {"heads": 3, "kv_heads": 3, "dim": 12, "vdim": 20, "conv": 4,
             **(right or {})}
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                 "vdim": dim, "rot": rot or rotation(), "scale": scale},
        "left_scale": left_scale, "right": right,
        "right_scale": right_scale}}


def rglru_layer(mlp, width=40, blocks=2, conv=4):
    return {"type": "rglru", "mlp": mlp,
            "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def make_config(layers, width=48, vocab=67, loop=(0, 1, 1), side=6,
                scale=3.0, eps=1e-5):
    return {"architecture": "Tebasun", "embedding": {"scale": scale},
            "layers": layers,
            "loop": dict(zip(("start", "stop", "times"), loop)),
            "norm": {"eps": eps}, "token_side": {"dim": side},
            "vocab": vocab, "width": width}


def make_tensors(cfg, seed=0, gain=1.0, ranks=(5, 7)):
    """Random bf16 weights; `gain` scales the matrices, `ranks` are the
    inner sizes of the decay's and the gate's pairs of products."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    n, sd = len(cfg["layers"]), cfg["token_side"]["dim"]
    t = {}

    def mat(name, rows, cols, k=1.0):
        t[name] = torch.randn(rows, cols, generator=g) * (
            gain * k / math.sqrt(cols))

    def vec(name, *shape, mean=0.0, spread=0.3):
        t[name] = mean + torch.randn(*shape, generator=g) * spread

    def norm(name):
        vec(name, W, mean=1.0)
        vec(name + ".b", W, spread=0.1)
        t[name + ".alpha"] = 0.5 + torch.rand((), generator=g)

    t["embed"] = torch.randn(V, W, generator=g) / cfg["embedding"]["scale"]
    t["side.embed"] = torch.randn(V, n * sd, generator=g)
    vec("loop.step", cfg["loop"]["times"], W)
    norm("final.norm")
    for i, entry in enumerate(cfg["layers"]):
        p, m = f"l{i}.", entry["mixer"]
        norm(p + "norm1")
        if entry["type"] == "parallel":
            a, q = m["left"], p + "mix.left."
            for nm, h in (("q", a["heads"]), ("k", a["kv_heads"])):
                mat(q + nm, h * a["dim"], W)
                vec(q + nm + ".b", h * a["dim"])
                vec(q + nm + ".norm", a["dim"], mean=1.2)
            vec(q + "sink", a["heads"], mean=0.5, spread=1.0)
            mat(q + "o", W, a["heads"] * a["dim"])
            vec(q + "o.b", W)
            a, q = m["right"], p + "mix.right."
            H, G, d, v = (a["heads"], a["kv_heads"], a["dim"], a["vdim"])
            for nm, rows in (("q", G * d), ("k", G * d), ("v", H * v)):
                mat(q + nm, rows, W)
                t[q + nm + ".conv"] = torch.randn(
                    rows, a["conv"], generator=g) / math.sqrt(a["conv"])
            mat(q + "b", H, W)
            vec(q + "A_log", H, mean=-0.7)
            vec(q + "norm", v, mean=1.0)
            mat(q + "a1", ranks[0], W)
            mat(q + "a2", H * d, ranks[0])
            vec(q + "dt_bias", H * d, mean=-2.0, spread=1.5)
            mat(q + "g1", ranks[1], W)
            mat(q + "g2", H * v, ranks[1], 2.0)
            mat(q + "o", W, H * v)
        else:
            q, wd, B = p + "mix.", m["width"], m["blocks"]
            for nm in "yx":
                mat(q + nm, wd, W)
                vec(q + nm + ".b", wd)
            t[q + "conv"] = torch.randn(wd, m["conv"], generator=g) \
                / math.sqrt(m["conv"])
            vec(q + "conv.b", wd)
            s = wd // B
            for nm in ("ra", "ri"):
                t[q + nm] = torch.randn(B, s, s, generator=g) \
                    / math.sqrt(s)
                vec(q + nm + ".b", B, s)
            vec(q + "lam", wd, mean=-2.5, spread=1.5)
            mat(q + "o", W, wd)
        if entry["mlp"] is not None:
            norm(p + "norm2")
            ff = entry["mlp"]["ff"]
            mat(p + "mlp.gate", ff, W)
            mat(p + "mlp.up", ff, W)
            mat(p + "mlp.down", W, ff)
        mat(p + "side.gate", sd, W)
        mat(p + "side.proj", W, sd)
        vec(p + "side.norm", W, mean=0.6)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}
