"""Plain, slow Kanotar in float64: the yardstick of the Kanotar tests.

One function per mechanism, one token at a time where that is the
clearest form, straight from the equations. Works on the raw checkpoint
(tensor name -> tensor, unpadded) and the raw config dict, and shares
no code with distllm_amd.
"""

import math

import torch


def rms(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def visible(i, size):
    """Key positions that query position i sees: the last `size`
    positions up to and including i."""
    return range(max(0, i - size + 1), i + 1)


def softmax(s):
    e = torch.exp(s - s.max())
    return e / e.sum()


def latent(h, t, pre, eps):
    """[T, width] -> the cached latents [T, kv_rank]."""
    return rms(h @ t[pre + "dkv"].T, t[pre + "dkv.norm"], eps)


def queries(h, t, pre, heads, dim, eps):
    cq = rms(h @ t[pre + "dq"].T, t[pre + "dq.norm"], eps)
    return (cq @ t[pre + "uq"].T).view(-1, heads, dim)


def latent_attention(h, c, t, pre, m, eps):
    """h [T, width] (mixer input), c [T, kv_rank] -> [T, width]."""
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = queries(h, t, pre, H, d, eps)
    k = (c @ t[pre + "uk"].T).view(-1, H, d)
    v = (c @ t[pre + "uv"].T).view(-1, H, dv)
    out = torch.zeros(h.shape[0], H, dv, dtype=h.dtype)
    for i in range(h.shape[0]):
        js = list(visible(i, m["mask"]["size"]))
        for n in range(H):
            p = softmax(k[js, n] @ q[i, n] * m["scale"])
            out[i, n] = p @ v[js, n]
    return out.reshape(h.shape[0], H * dv) @ t[pre + "o"].T


def clamped_glu(h, t, pre, limit):
    g = torch.clamp(h @ t[pre + "gate"].T, max=limit)
    u = torch.clamp(h @ t[pre + "up"].T, -limit, limit)
    y = g / (1 + torch.exp(-1.702 * g)) * (u + 1)
    return y @ t[pre + "down"].T


def forward(config, tensors, tokens, trace=None):
    """Logits [T, vocab] of one sequence; `trace`, when given, collects
    the residual stream after every layer."""
    t = {k: v.to(torch.float64) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = t["embed"][torch.as_tensor(tokens)]
    latents = {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = rms(x, t[p + "norm1"], eps)
        if m.get("kv_from") is None:
            latents[i] = latent(h, t, p + "mix.", eps)
            c = latents[i]
        else:
            c = latents[m["kv_from"]]
        y = latent_attention(h, c, t, p + "mix.", m, eps)
        x = x + rms(y, t[p + "norm1b"], eps)
        if layer.get("mlp") is not None:
            y = clamped_glu(rms(x, t[p + "norm2"], eps), t, p + "mlp.",
                            layer["mlp"]["limit"])
            x = x + rms(y, t[p + "norm2b"], eps)
        if trace is not None:
            trace.append(x)
    h = rms(x, t["final.norm"], eps)
    return h @ t["head"].T * config["logit_scale"]


def make_config(layers, width=48, vocab=97, eps=1e-5, logit_scale=0.7):
    return {"architecture": "Kanotar", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": layers}


def make_layer(heads=3, dim=16, vdim=24, q_rank=20, kv_rank=32, size=8,
               scale=0.3, kv_from=None, ff=56, limit=1.5):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank,
         "kv_rank": kv_rank, "scale": scale, "mask": {"size": size}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m,
            "mlp": (None if ff is None
                    else {"kind": "dense", "ff": ff, "limit": limit})}


def make_tensors(config, seed=0, gain=1.0):
    """Random weights of a config, rounded to bfloat16 so that every
    dtype under test starts from the same numbers. `gain` scales the
    query up-projection: larger values make attention peaky, so that a
    wrong key shows."""
    g = torch.Generator().manual_seed(seed)
    W, V = config["width"], config["vocab"]
    t = {}

    def lin(name, out, inp, s=1.0):
        t[name] = torch.randn(out, inp, generator=g) * (s / math.sqrt(inp))

    def vec(name, n):
        t[name] = 1 + 0.3 * torch.randn(n, generator=g)

    t["embed"] = torch.randn(V, W, generator=g)
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        for n in ("norm1", "norm1b"):
            vec(p + n, W)
        lin(p + "mix.dq", m["q_rank"], W)
        vec(p + "mix.dq.norm", m["q_rank"])
        lin(p + "mix.uq", m["heads"] * m["dim"], m["q_rank"], gain)
        if m.get("kv_from") is None:
            lin(p + "mix.dkv", m["kv_rank"], W)
            vec(p + "mix.dkv.norm", m["kv_rank"])
        lin(p + "mix.uk", m["heads"] * m["dim"], m["kv_rank"])
        lin(p + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"])
        lin(p + "mix.o", W, m["heads"] * m["vdim"])
        if layer["mlp"] is not None:
            for n in ("norm2", "norm2b"):
                vec(p + n, W)
            ff = layer["mlp"]["ff"]
            lin(p + "mlp.gate", ff, W, 2.0)
            lin(p + "mlp.up", ff, W, 2.0)
            lin(p + "mlp.down", W, ff)
    vec("final.norm", W)
    lin("head", V, W)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}
