"""Plain, slow Bufulorn in float64: the yardstick of the Bufulorn tests.

One function per mechanism, straight from the equations. Works on the raw
checkpoint (tensor name -> tensor, unpadded) and the raw config dict, and
shares no code with distllm_amd.
"""

import math

import torch


def layer_norm(x, w, b, eps):
    mean = x.mean(-1, keepdim=True)
    var = ((x - mean) ** 2).mean(-1, keepdim=True)
    return (x - mean) / torch.sqrt(var + eps) * w + b


def rms(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-abs(z))) + torch.clamp(z, min=0)


def softmax(s):
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def embedding(t, tokens):
    return t["embed"][tokens] + t["pos"][: len(tokens)]


# ---- attention -------------------------------------------------------------

def visible(i, j, size):
    """Whether query position i sees key position j."""
    return (j <= i) & (i // size == j // size)


def distance_bias(i, j, r1, r2):
    return r1 * torch.log1p(r2 * (i - j).to(torch.float64))


def keys_values(h, t, pre, m, eps):
    """[T, width] -> normed keys [T, G, dim], values [T, G, vdim]."""
    G = m["kv_heads"]
    k = (h @ t[pre + "k"].T + t[pre + "k.b"]).view(-1, G, m["dim"])
    v = (h @ t[pre + "v"].T + t[pre + "v.b"]).view(-1, G, m["vdim"])
    return rms(k, t[pre + "k.norm"], eps), v


def attention(h, kv, t, pre, m, eps):
    """h [T, width] (mixer input), kv: keys_values of the owning layer."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    k, v = kv
    q = (h @ t[pre + "q"].T + t[pre + "q.b"]).view(T, H, m["dim"])
    q = rms(q, t[pre + "q.norm"], eps)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    seen = visible(i, j, m["mask"]["size"])
    out = torch.zeros(T, H, m["vdim"], dtype=h.dtype)
    for n in range(H):
        s = q[:, n] @ k[:, n // (H // G)].T * m["scale"]
        s = m["softcap"] * torch.tanh(s / m["softcap"])
        s = s - distance_bias((i - j).clamp(min=0), 0, t[pre + "r1"][n],
                              t[pre + "r2"][n])
        s = torch.where(seen, s, -math.inf)
        out[:, n] = softmax(s) @ v[:, n // (H // G)]
    return (out.reshape(T, -1) * sigmoid(h @ t[pre + "g"].T)) @ t[pre + "o"].T


# ---- delta rule ------------------------------------------------------------

def short_conv(x, w):
    """Causal convolution per channel: x [T, C], w [C, taps]."""
    taps = w.shape[1]
    x = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=x.dtype), x])
    T = x.shape[0] - taps + 1
    return sum(x[a: a + T] * w[:, a] for a in range(taps))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def decay(a, A_log, dt_bias):
    return torch.exp(-torch.exp(A_log) * softplus(a + dt_bias))


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, e], g, beta [T, H] -> [T, H, e]."""
    S = torch.zeros(q.shape[1], q.shape[2], v.shape[2], dtype=q.dtype)
    out = []
    for n in range(q.shape[0]):
        S = g[n, :, None, None] * S
        u = beta[n, :, None] * (v[n] - (S * k[n, :, :, None]).sum(1))
        S = S + k[n, :, :, None] * u[:, None]
        out.append((S * q[n, :, :, None]).sum(1))
    return torch.stack(out)


def delta(h, t, pre, m, eps):
    T, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def proj(n):
        return silu(short_conv(h @ t[pre + n].T, t[pre + n + ".conv"]))

    q = unit(proj("q").view(T, G, d)) * d ** -0.5
    k = unit(proj("k").view(T, G, d))
    v = proj("v").view(T, H, e)
    own = torch.arange(H) // (H // G)
    g = decay(h @ t[pre + "a"].T, t[pre + "A_log"], t[pre + "dt_bias"])
    o = delta_rule(q[:, own], k[:, own], v, g, sigmoid(h @ t[pre + "b"].T))
    o = rms(o, t[pre + "norm"], eps)
    return (o.reshape(T, -1) * silu(h @ t[pre + "g"].T)) @ t[pre + "o"].T


# ---- feed-forward ----------------------------------------------------------

def xielu(z, p, q):
    pos = softplus(p) * z * z + z / 2
    neg = (0.5 + softplus(q)) * (torch.expm1(z.clamp(max=0)) - z) + z / 2
    return torch.where(z > 0, pos, neg)


def dense(h, t, pre):
    p, q = t[pre + "act"]
    return xielu(h @ t[pre + "up"].T, p, q) @ t[pre + "down"].T


def choose(s, top, count, keep):
    """Indices of the chosen experts from the scores [experts] of a token."""
    per = len(s) // count
    best = sorted(range(count),
                  key=lambda c: -float(s[c * per: (c + 1) * per].max()))
    allowed = [e for c in best[:keep] for e in range(c * per, (c + 1) * per)]
    return sorted(allowed, key=lambda e: -float(s[e]))[:top]


def expert(h, t, pre):
    return (silu(h @ t[pre + "gate"].T) * (h @ t[pre + "up"].T)) \
        @ t[pre + "down"].T


def moe(h, t, pre, r):
    s = softmax(h @ t[pre + "router"].T)
    out = torch.zeros_like(h)
    chosen = [choose(row, r["top"], r["groups"]["count"],
                     r["groups"]["keep"]) for row in s]
    for e in range(r["experts"]):
        rows = [n for n, c in enumerate(chosen) if e in c]
        if rows:
            out[rows] += s[rows, e, None] * expert(h[rows], t, f"{pre}e{e}.")
    return out


# ---- model -----------------------------------------------------------------

def forward(config, tensors, tokens, trace=None):
    """Logits [T, vocab] of one sequence; `trace`, when given, collects
    the residual stream after every layer."""
    t = {k: v.to(torch.float64) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = embedding(t, torch.as_tensor(tokens))
    kv = {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        if layer["type"] == "attention":
            if m.get("kv_from") is None:
                kv[i] = keys_values(x, t, p + "mix.", m, eps)
            y = attention(x, kv[m.get("kv_from", i)], t, p + "mix.", m, eps)
        else:
            y = delta(x, t, p + "mix.", m, eps)
        x = x + layer_norm(y, t[p + "norm1"], t[p + "norm1.b"], eps)
        f = layer.get("mlp")
        if f is not None:
            y = (dense(x, t, p + "mlp.") if f["kind"] == "dense"
                 else moe(x, t, p + "mlp.", f["router"]))
            x = x + layer_norm(y, t[p + "norm2"], t[p + "norm2.b"], eps)
        if trace is not None:
            trace.append(x)
    x = layer_norm(x, t["final.norm"], t["final.norm.b"], eps)
    return x @ t["head"].T


# ---- random models ---------------------------------------------------------

def make_config(layers, width=48, vocab=97, eps=1e-5, max_positions=512):
    return {"architecture": "Bufulorn", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "max_positions": max_positions,
            "layers": layers}


def dense_mlp(ff=56):
    return {"kind": "dense", "ff": ff}


def moe_mlp(ff=40, experts=6, top=2, count=3, keep=2):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top,
                       "groups": {"count": count, "keep": keep}}}


def attention_layer(mlp, heads=4, kv_heads=2, dim=16, vdim=24, size=20,
                    scale=0.25, softcap=20.0, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "mask": {"size": size}, "scale": scale, "softcap": softcap}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def delta_layer(mlp, heads=4, kv_heads=2, dim=16, vdim=24, conv=4):
    return {"type": "delta", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                      "vdim": vdim, "conv": conv}}


def make_tensors(config, seed=0, gain=1.0, router=5.0):
    """Random weights of a config, rounded to bfloat16 so that every dtype
    under test starts from the same numbers. `gain` scales the queries:
    larger values make attention peaky, so that a wrong key shows. So does
    `router` with the routers' choices."""
    g = torch.Generator().manual_seed(seed)
    W, V = config["width"], config["vocab"]
    t = {}

    def lin(name, out, inp, s=1.0):
        t[name] = torch.randn(out, inp, generator=g) * (s / math.sqrt(inp))

    def vec(name, n, mid=1.0, spread=0.3):
        t[name] = mid + spread * torch.randn(n, generator=g)

    def bias(name, n):
        vec(name + ".b", n, 0.0, 0.3)

    t["embed"] = torch.randn(V, W, generator=g)
    t["pos"] = 0.7 * torch.randn(config["max_positions"], W, generator=g)
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.mix.", layer["mixer"]
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        if layer["type"] == "attention":
            lin(p + "q", H * d, W), bias(p + "q", H * d)
            vec(p + "q.norm", d, gain)
            if m.get("kv_from") is None:
                lin(p + "k", G * d, W), bias(p + "k", G * d)
                lin(p + "v", G * e, W), bias(p + "v", G * e)
                vec(p + "k.norm", d)
            t[p + "r1"] = torch.rand(H, generator=g) * 2
            t[p + "r2"] = torch.rand(H, generator=g)
        else:
            for n, c in (("q", G * d), ("k", G * d), ("v", H * e)):
                lin(p + n, c, W)
                t[p + n + ".conv"] = torch.randn(c, m["conv"], generator=g) \
                    / math.sqrt(m["conv"])
            lin(p + "b", H, W), lin(p + "a", H, W)
            vec(p + "A_log", H, -1.5), vec(p + "dt_bias", H, -1.0)
            vec(p + "norm", e)
        lin(p + "g", H * e, W)
        lin(p + "o", W, H * e)
        vec(f"l{i}.norm1", W), bias(f"l{i}.norm1", W)
        f, p = layer["mlp"], f"l{i}.mlp."
        if f is None:
            continue
        vec(f"l{i}.norm2", W), bias(f"l{i}.norm2", W)
        if f["kind"] == "dense":
            lin(p + "up", f["ff"], W, 2.0)
            lin(p + "down", W, f["ff"])
            vec(p + "act", 2, 0.2, 0.5)
        else:
            for n in range(f["router"]["experts"]):
                lin(f"{p}e{n}.gate", f["expert"]["ff"], W, 2.0)
                lin(f"{p}e{n}.up", f["expert"]["ff"], W)
                lin(f"{p}e{n}.down", W, f["expert"]["ff"])
            lin(p + "router", f["router"]["experts"], W, router)
    vec("final.norm", W), bias("final.norm", W)
    lin("head", V, W)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}
