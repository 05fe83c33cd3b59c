"""Plain, slow implementation of the Zokanex decoder, one function per
mechanism, written from the equations and sharing no code with the engine.

Everything works on one whole sequence at a time (no cache, no batching):
`forward(cfg, weights, tokens)` returns the logits at every position and the
residual after every layer. `cfg` is the parsed config.json dictionary and
`weights` maps checkpoint tensor names to tensors. All arithmetic runs in
`dtype` (float64 by default).
"""
from __future__ import annotations

import json
import math
import os
import struct

import torch


# ---- small pieces -----------------------------------------------------------
def rms_unit(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi)
                                       * (z + 0.044715 * z ** 3)))


def linear(x, w):
    return x @ w.T


def rotate(x, positions, base, dims):
    """x [T, heads, D]: entries i and i + dims/2 of the first `dims` turn by
    position * base^(-2i/dims); the rest stays."""
    if not dims:
        return x
    y = x.clone()
    half = dims // 2
    for i in range(half):
        a = positions.to(x.dtype) * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        y[:, :, i] = u * c - v * s
        y[:, :, i + half] = v * c + u * s
    return y


# ---- attention --------------------------------------------------------------
def sees_window(T, size):
    """[T, T]: position i sees the `size` positions that end with itself
    (size 0: every earlier one)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    return ok & (i - j < size) if size else ok


def attend(q, k, v, scale, visible):
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H, Dv]; query head h
    reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = q[:, h] @ k[:, h // per].T * scale
        s = s.masked_fill(~visible, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, h // per]
    return out


def attention_keys_values(h, w, p, m, eps):
    """What the layer's cache holds: normed and turned keys, values."""
    T, G = h.shape[0], m["kv_heads"]
    k = linear(h, w[p + "k"]).view(T, G, m["dim"])
    k = rms_norm(k, w[p + "k.norm"], eps)
    rot = m.get("rot") or dict(base=1.0, dims=0)
    k = rotate(k, torch.arange(T), rot["base"], rot["dims"])
    return k, linear(h, w[p + "v"]).view(T, G, m["vdim"])


def mixer_attention(h, w, p, m, eps, kv):
    """kv: (keys, values) of this layer or of the layer it borrows from."""
    T, H = h.shape[0], m["heads"]
    q = linear(h, w[p + "q"]).view(T, H, m["dim"])
    q = rms_norm(q, w[p + "q.norm"], eps)
    rot = m.get("rot") or dict(base=1.0, dims=0)
    q = rotate(q, torch.arange(T), rot["base"], rot["dims"])
    o = attend(q, kv[0], kv[1], m["scale"],
               sees_window(T, (m.get("mask") or {}).get("size", 0)))
    return linear(o.reshape(T, -1), w[p + "o"])


# ---- retention --------------------------------------------------------------
def retention_core(q, k, v, decay, state=None):
    """q, k [T, H, D], v [T, H, Dv]; S <- decay_h S + k v^T, o = S^T q. Returns
    (o [T, H, Dv], last state [H, D, Dv])."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None else state
    a = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
    out = []
    for t in range(T):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def mixer_retention(h, w, p, m, eps):
    T, H, D = h.shape[0], m["heads"], m["dim"]
    rot = m.get("rot") or dict(base=1.0, dims=0)

    def turned(name):
        z = linear(h, w[p + name]).view(T, H, D)
        return rotate(z, torch.arange(T), rot["base"], rot["dims"])
    v = linear(h, w[p + "v"]).view(T, H, m["vdim"])
    o, _ = retention_core(turned("q"), turned("k") * D ** -0.5, v, m["decay"])
    o = rms_unit(o, eps).reshape(T, -1) * silu(linear(h, w[p + "g"]))
    return linear(o, w[p + "o"])


# ---- feed-forwards ----------------------------------------------------------
def ff_dense(h, w, f):
    return linear(gelu_tanh(linear(h, w[f + "gate"])) * linear(h, w[f + "up"]),
                  w[f + "down"])


def expert(h, w, e):
    return linear(silu(linear(h, w[e + "gate"])) * linear(h, w[e + "up"]),
                  w[e + "down"])


def route(z, r):
    """Router logits [experts] of one token -> list of (expert, weight)."""
    s = torch.sigmoid(z).tolist()
    n = len(s)
    g = r.get("groups") or {}
    count, keep = g.get("count", 1), g.get("keep", 1)
    size = n // count
    score = []
    for i in range(count):
        best = sorted(s[i * size:(i + 1) * size], reverse=True)[:2]
        score.append((-sum(best), i))
    eligible = {i for _, i in sorted(score)[:keep]}
    order = sorted((-s[e], e) for e in range(n) if e // size in eligible)
    return [(e, s[e] * r.get("scale", 1.0)) for _, e in order[:r["top"]]]


def choice_margin(z, r):
    """How clear the choice of one token is: the smallest score difference
    between a kept and a dropped group, or a chosen and a passed-over expert
    (infinite where nothing is dropped)."""
    s = torch.sigmoid(z)
    g = r.get("groups") or dict(count=1, keep=1)
    s = s.view(g["count"], -1)
    pair = s.topk(min(2, s.shape[1]), -1).values.sum(-1)
    pair, order = pair.sort(descending=True)
    gap = math.inf
    if g["keep"] < g["count"]:
        gap = float(pair[g["keep"] - 1] - pair[g["keep"]])
    s = s[order[:g["keep"]]].reshape(-1).sort(descending=True).values
    if len(s) > r["top"]:
        gap = min(gap, float(s[r["top"] - 1] - s[r["top"]]))
    return gap


def ff_moe(h, w, f, mlp, margin=None):
    """margin [T]: lowered to the tokens' choice margins."""
    out = torch.zeros_like(h)
    z = linear(h, w[f + "router"])
    for t in range(h.shape[0]):
        if margin is not None:
            margin[t] = min(float(margin[t]), choice_margin(z[t],
                                                            mlp["router"]))
        for e, a in route(z[t], mlp["router"]):
            out[t] += a * expert(h[t:t + 1], w, f"{f}e{e}.")[0]
    if mlp.get("shared"):
        out = out + expert(h, w, f + "shared.") \
            * torch.sigmoid(linear(h, w[f + "shared.sg"]))
    return out


# ---- the stack --------------------------------------------------------------
def forward(cfg, weights, tokens, dtype=torch.float64):
    """-> (logits [T, vocab], residual after every layer [layers, T, W], choice
    margin of every token over all routers [T])."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v)
         for k, v in weights.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = cfg["norm"]["eps"]
    x = w["embed"][tokens] * (cfg.get("embedding") or {}).get("scale", 1.0)
    kept, after = {}, []
    margin = torch.full((len(tokens),), math.inf)
    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        if lc["type"] == "retention":
            y = mixer_retention(h, w, p + "mix.", m, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                src = i
                kept[i] = attention_keys_values(h, w, p + "mix.", m, eps)
            y = mixer_attention(h, w, p + "mix.", m, eps, kept[src])
        mlp = lc.get("mlp")
        if mlp:
            y = y + (ff_dense(h, w, p + "mlp.") if mlp["kind"] == "dense"
                     else ff_moe(h, w, p + "mlp.", mlp, margin))
        x = x + y
        after.append(x)
    return linear(rms_norm(x, w["final.norm"], eps), w["head"]), \
        torch.stack(after), margin


# ---- test models: configurations, random checkpoints, model folders ---------
def dense(ff=12):
    return dict(kind="dense", ff=ff)


def moe(ff=6, experts=6, top=2, count=3, keep=2, scale=1.25, shared=10):
    mlp = dict(kind="moe", expert=dict(ff=ff),
               router=dict(experts=experts, top=top, scale=scale,
                           groups=dict(count=count, keep=keep)))
    if shared:
        mlp["shared"] = dict(ff=shared)
    return mlp


def attention(heads=4, kv_heads=2, dim=8, vdim=6, dims=4, size=7, base=100.0,
              scale=None, kv_from=None, mlp="dense"):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
             rot=dict(base=base, dims=dims),
             scale=scale if scale is not None else 1.3 * dim ** -0.5)
    if size:
        m["mask"] = dict(size=size)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention", mixer=m,
                mlp=dense() if mlp == "dense" else mlp)


def retention(heads=2, dim=6, vdim=5, dims=4, base=100.0, decay=None,
              mlp="dense"):
    return dict(type="retention", mlp=dense() if mlp == "dense" else mlp,
                mixer=dict(heads=heads, dim=dim, vdim=vdim,
                           rot=dict(base=base, dims=dims),
                           decay=decay or [1.0 - 0.4 ** (h + 1)
                                           for h in range(heads)]))


def make_config(width=24, vocab=50, eps=1e-4, scale=1.7, layers=None):
    return dict(architecture="Zokanex", vocab=vocab, width=width,
                norm=dict(eps=eps), embedding=dict(scale=scale),
                layers=layers or [attention(), retention(mlp=moe())])


def make_weights(cfg, seed=0):
    """Random bf16-representable weights (fp32 tensors) for a config."""
    gen = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def rnd(*shape, std=None):
        std = std if std is not None else 1.0 / math.sqrt(shape[-1])
        return (torch.randn(*shape, generator=gen) * std).bfloat16().float()

    def about(mean, *shape, spread=0.3):
        return (mean + spread * torch.randn(shape, generator=gen)) \
            .bfloat16().float()

    out = {"embed": rnd(cfg["vocab"], W, std=1.0),
           "final.norm": about(1.2, W), "head": rnd(cfg["vocab"], W)}

    def put_ff(f, ff, std=1.0):
        out[f + "gate"] = rnd(ff, W, std=std / math.sqrt(W))
        out[f + "up"] = rnd(ff, W, std=std / math.sqrt(W))
        out[f + "down"] = rnd(W, ff)

    for i, lc in enumerate(cfg["layers"]):
        p, mc = f"l{i}.", lc["mixer"]
        m = p + "mix."
        H, D, dv = mc["heads"], mc["dim"], mc["vdim"]
        out[p + "norm1"] = about(1.0, W)
        out[m + "q"] = rnd(H * D, W)
        if lc["type"] == "attention":
            G = mc["kv_heads"]
            out[m + "q.norm"] = about(1.1, D)
            if "kv_from" not in mc:
                out[m + "k"], out[m + "v"] = rnd(G * D, W), rnd(G * dv, W)
                out[m + "k.norm"] = about(1.1, D)
        else:
            out[m + "k"], out[m + "v"] = rnd(H * D, W), rnd(H * dv, W)
            out[m + "g"] = rnd(H * dv, W)
        out[m + "o"] = rnd(W, H * dv)
        mlp, f = lc.get("mlp"), p + "mlp."
        if not mlp:
            continue
        if mlp["kind"] == "dense":
            put_ff(f, mlp["ff"])
            continue
        out[f + "router"] = rnd(mlp["router"]["experts"], W,
                                std=2.0 / math.sqrt(W))
        for j in range(mlp["router"]["experts"]):
            put_ff(f"{f}e{j}.", mlp["expert"]["ff"], 1.5)
        if mlp.get("shared"):
            put_ff(f + "shared.", mlp["shared"]["ff"], 1.5)
            out[f + "shared.sg"] = rnd(1, W, std=2.0 / math.sqrt(W))
    return out


def write_model_dir(folder, cfg, tensors):
    """config.json and a bf16 safetensors file (8-byte header length, JSON
    header, raw data)."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, t in tensors.items():
        raw = t.to(torch.bfloat16).contiguous().view(torch.int16).numpy() \
            .tobytes()
        header[name] = dict(dtype="BF16", shape=list(t.shape),
                            data_offsets=[at, at + len(raw)])
        blobs.append(raw)
        at += len(raw)
    js = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(js)))
        f.write(js)
        for b in blobs:
            f.write(b)
    return folder


def rel_err(got, want):
    """Per row: rms of the mean-free difference over the rms of `want`."""
    got, want = got.to(torch.float64), want.to(torch.float64)
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    ref = want - want.mean(-1, keepdim=True)
    return torch.sqrt((d ** 2).mean(-1)) / torch.sqrt((ref ** 2).mean())
