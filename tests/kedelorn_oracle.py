"""Plain, slow Kedelorn in float64: the yardstick of the Kedelorn tests.

One function per mechanism, straight from the equations, token by token
where there is a recurrence. Works on the raw checkpoint (tensor name ->
tensor, unpadded) and the raw config dict, and shares no code with
distllm_amd.
"""

import math

import torch

from tebasun_oracle import rotate, sigmoid, silu, softmax_with_sink

F64 = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """Weights are stored around zero."""
    return rms(x, eps) * (1 + w)


# ---- retention -------------------------------------------------------------

def retention_step(S, q, k, v, decay):
    """One token of one head; S [dim, vdim]. -> state, read-out."""
    S = decay * S + k[:, None] * v[None]
    return S, S.T @ q


def retention(h, t, pre, m, eps, caches):
    T, H = h.shape[0], m["heads"]
    pos = torch.arange(T)
    q = rotate((h @ t[pre + "q"].T).view(T, H, m["dim"]), pos, m["rot"])
    k = rotate((h @ t[pre + "k"].T).view(T, H, m["dim"]), pos, m["rot"])
    k = k * m["dim"] ** -0.5
    v = (h @ t[pre + "v"].T).view(T, H, m["vdim"])
    o = torch.zeros(T, H, m["vdim"], dtype=h.dtype)
    for n in range(H):
        S = torch.zeros(m["dim"], m["vdim"], dtype=h.dtype)
        for i in range(T):
            S, o[i, n] = retention_step(S, q[i, n], k[i, n], v[i, n],
                                        m["decay"][n])
    y = rms(o, eps).reshape(T, -1) * silu(h @ t[pre + "g"].T)
    return y @ t[pre + "o"].T


# ---- latent attention ------------------------------------------------------

def latents(h, t, pre, m, eps):
    """What a token leaves behind: the latent and the rotated key part."""
    z = h @ t[pre + "dkv"].T
    c = rms(z[:, : m["kv_rank"]], eps) * t[pre + "dkv.norm"]
    r = rotate(z[:, None, m["kv_rank"]:], torch.arange(len(z)), m["rot"])
    return c, r[:, 0]


def latent_attention(h, t, pre, m, eps, caches):
    T, H, d, r = h.shape[0], m["heads"], m["dim"], m["rot_dim"]
    if m.get("kv_from") is None:
        caches.append(latents(h, t, pre, m, eps))
    else:
        caches.append(caches[m["kv_from"]])
    c, kr = caches[-1]
    pos = torch.arange(T)
    q = (h @ t[pre + "q"].T).view(T, H, d + r)
    qr = rotate(q[..., d:], pos, m["rot"])
    k = (c @ t[pre + "uk"].T).view(T, H, d)
    v = (c @ t[pre + "uv"].T).view(T, H, m["vdim"])
    gate = sigmoid(h @ t[pre + "g"].T)
    out = torch.zeros(T, H, m["vdim"], dtype=h.dtype)
    for n in range(H):
        s = (q[:, n, :d] @ k[:, n].T + qr[:, n] @ kr.T) * m["scale"]
        s = torch.where(pos[None] <= pos[:, None], s, -math.inf)
        w = softmax_with_sink(s, t[pre + "sink"][n])
        out[:, n] = w @ v[:, n] * gate[:, n, None]
    return out.reshape(T, -1) @ t[pre + "o"].T


# ---- routed experts --------------------------------------------------------

def expert(h, t, pre):
    return torch.clamp(h @ t[pre + "up"].T, min=0) ** 2 @ t[pre + "down"].T


def route(h, t, pre, r):
    """-> the chosen experts [T, top] and their weights."""
    s = sigmoid(h @ t[pre + "router"].T)
    ids = (s + t[pre + "correction"]).topk(r["top"], -1).indices
    return ids, s.gather(1, ids) * r["scale"]


def moe(h, t, pre, mlp):
    ids, w = route(h, t, pre, mlp["router"])
    out = torch.zeros_like(h)
    for i in range(len(h)):
        for e, x in zip(ids[i].tolist(), w[i]):
            out[i] += x * expert(h[i], t, f"{pre}e{e}.")
    if mlp.get("shared") is not None:
        out = out + expert(h, t, pre + "shared.") * sigmoid(
            h @ t[pre + "shared.sg"].T)
    return out


# ---- streams ---------------------------------------------------------------

def read(X, t, hc):
    """X [streams, T, width] -> what a sublayer reads."""
    return (t[hc + "in"][:, None, None] * X).sum(0)


def write(X, y, t, hc):
    """The streams after a sublayer's output y; mix is [from, to]."""
    mixed = (t[hc + "mix"][:, :, None, None] * X[:, None]).sum(0)
    return mixed + t[hc + "out"][:, None, None] * y


MIXERS = {"retention": retention, "latent_attention": latent_attention}


def layer(X, t, cfg, i, caches):
    entry, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    if entry["type"] != "latent_attention":
        caches.append(None)
    h = norm(read(X, t, p + "hc1."), t[p + "norm1"], eps)
    X = write(X, MIXERS[entry["type"]](h, t, p + "mix.", entry["mixer"], eps,
                                       caches), t, p + "hc1.")
    if entry["mlp"] is not None:
        h = norm(read(X, t, p + "hc2."), t[p + "norm2"], eps)
        X = write(X, moe(h, t, p + "mlp.", entry["mlp"]), t, p + "hc2.")
    return X


@torch.no_grad()
def forward(cfg, tensors, tokens, trace=None):
    """Logits [T, vocab] of one sequence; trace collects the sum of the
    streams after every layer."""
    t = {k: v.to(F64) for k, v in tensors.items()}
    X = t["embed"][torch.as_tensor(tokens)].expand(cfg["streams"], -1, -1)
    caches = []
    for i in range(len(cfg["layers"])):
        X = layer(X, t, cfg, i, caches)
        if trace is not None:
            trace.append(X.sum(0))
    x = norm(X.sum(0), t["final.norm"], cfg["norm"]["eps"])
    return x @ t["head"].T


# ---- small configurations and weights --------------------------------------

def yarn(dims=8, base=1000.0, factor=4.0, original=16, fast=4.0, slow=0.5):
    return {"base": base, "dims": dims,
            "scaling": {"factor": factor, "fast": fast,
                        "original": original, "slow": slow}}


def moe_mlp(ff=20, experts=6, top=2, scale=1.7, shared=28):
    mlp = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": experts, "scale": scale, "top": top}}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return mlp


def retention_layer(mlp, heads=3, dim=12, vdim=20, rot=None, decay=None):
    decay = decay or [1 - 2.0 ** (-2 - 5 * n / heads) for n in range(heads)]
    return {"type": "retention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "decay": decay,
        "rot": rot or {"base": 300.0, "dims": 8}}}


def latent_layer(mlp, heads=4, dim=16, rot_dim=8, vdim=12, kv_rank=24,
                 rot=None, scale=0.5, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "kv_rank": kv_rank, "rot": rot or yarn(rot_dim), "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mlp": mlp, "mixer": m}


def make_config(layers, width=48, vocab=67, streams=3, eps=2e-5):
    return {"architecture": "Kedelorn", "layers": layers,
            "norm": {"eps": eps}, "streams": streams, "vocab": vocab,
            "width": width}


def make_tensors(cfg, seed=0, gain=1.0):
    """Random bf16 weights; `gain` scales the matrices."""
    g = torch.Generator().manual_seed(seed)
    W, V, s = cfg["width"], cfg["vocab"], cfg["streams"]
    t = {}

    def mat(name, rows, cols, k=1.0):
        t[name] = torch.randn(rows, cols, generator=g) * (
            gain * k / math.sqrt(cols))

    def vec(name, *shape, mean=0.0, spread=0.3):
        t[name] = mean + torch.randn(*shape, generator=g) * spread

    t["embed"] = torch.randn(V, W, generator=g)
    mat("head", V, W)
    vec("final.norm", W)
    for i, entry in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", entry["mixer"], entry["mlp"]
        H, q = m["heads"], p + "mix."
        for j in ("1", "2") if mlp is not None else ("1",):
            vec(p + "norm" + j, W)
            vec(p + f"hc{j}.in", s, mean=1 / s)
            vec(p + f"hc{j}.out", s, mean=0.8)
            t[p + f"hc{j}.mix"] = torch.eye(s) * 0.8 \
                + torch.randn(s, s, generator=g) * 0.3 / math.sqrt(s)
        if entry["type"] == "retention":
            for nm, d in (("q", "dim"), ("k", "dim"), ("v", "vdim"),
                          ("g", "vdim")):
                mat(q + nm, H * m[d], W)
            mat(q + "o", W, H * m["vdim"])
        else:
            r = m["kv_rank"]
            mat(q + "q", H * (m["dim"] + m["rot_dim"]), W)
            if m.get("kv_from") is None:
                mat(q + "dkv", r + m["rot_dim"], W)
                vec(q + "dkv.norm", r, mean=1.0)
            mat(q + "uk", H * m["dim"], r)
            mat(q + "uv", H * m["vdim"], r, 1.5)
            vec(q + "sink", H, mean=0.5, spread=1.0)
            mat(q + "g", H, W)
            mat(q + "o", W, H * m["vdim"], 1.5)
        if mlp is None:
            continue
        q, E = p + "mlp.", mlp["router"]["experts"]
        ffs = {f"e{e}": mlp["expert"]["ff"] for e in range(E)}
        if mlp.get("shared") is not None:
            ffs["shared"] = mlp["shared"]["ff"]
            mat(q + "shared.sg", 1, W)
        for nm, ff in ffs.items():
            mat(q + nm + ".up", ff, W)
            mat(q + nm + ".down", W, ff, 0.7)
        mat(q + "router", E, W, 1.5)
        vec(q + "correction", E, spread=0.2)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}
