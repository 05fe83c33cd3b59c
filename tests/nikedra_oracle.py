"""Plain, slow implementation of the Nikedra decoder, one function per
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
    """w: a vector over the last axis, or one number for all of it."""
    return rms_unit(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def linear(x, w, b=None):
    y = x @ w.T
    return y if b is None else y + b


def causal_conv(x, w, b=None):
    """x [T, C], w [C, taps], last column = the current token; zeros before
    the start."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            src = t - taps + 1 + j
            if src >= 0:
                y[t] += w[:, j] * x[src]
    return y if b is None else y + b


# ---- rotary positions -------------------------------------------------------
def rotary(rot, dtype=torch.float64):
    """Frequencies and the cos/sin multiplier. `scaling` stretches the slow
    pairs by `factor` with a linear ramp over the pair index."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc, mult = rot.get("scaling"), 1.0
    if sc:
        def index_of(turns):
            return dims * math.log(sc["original"] / (2 * math.pi * turns)) \
                / (2 * math.log(base))
        lo = max(math.floor(index_of(sc["fast"])), 0)
        hi = min(math.ceil(index_of(sc["slow"])), dims - 1)
        for i in range(dims // 2):
            r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f[i] = f[i] / sc["factor"] * r + f[i] * (1.0 - r)
        mult = 0.1 * math.log(sc["factor"]) + 1.0
    return torch.tensor(f, dtype=dtype), mult


def rotate(x, freqs, mult, dims):
    """x [T, H, D]: entry i < dims/2 of every head turns with entry i +
    dims/2 by the angle position * f_i."""
    if dims == 0:
        return x
    ang = torch.arange(x.shape[0], dtype=freqs.dtype)[:, None] * freqs
    c, s = (torch.cos(ang) * mult)[:, None], (torch.sin(ang) * mult)[:, None]
    half = dims // 2
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


# ---- attention --------------------------------------------------------------
def sees_window(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    m = j <= i
    return m if not size else m & (i - j < size)


def sees_chunk(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    m = j <= i
    return m if not size else m & (i // size == j // size)


def attend(q, k, v, scale, mask):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; softmax over visible keys."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        p = torch.softmax(s.masked_fill(~mask, float("-inf")), -1)
        out[:, h] = p @ v[:, h // per]
    return out


def mask_size(m):
    return (m.get("mask") or {}).get("size", 0)


def mixer_latent_attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, d, rd, dv, r = (m[x] for x in ("heads", "dim", "rot_dim", "vdim",
                                      "kv_rank"))
    q = linear(h, w[pre + "q"]).view(T, H, d + rd)
    dkv = linear(h, w[pre + "dkv"])
    c = rms_norm(dkv[:, :r], w[pre + "dkv.norm"], eps)
    f, mult = rotary(m["rot"], h.dtype)
    qr = rotate(q[..., d:], f, mult, int(m["rot"]["dims"]))
    kr = rotate(dkv[:, None, r:], f, mult, int(m["rot"]["dims"]))
    k = linear(c, w[pre + "uk"]).view(T, H, d)
    v = linear(c, w[pre + "uv"]).view(T, H, dv)
    o = attend(torch.cat([q[..., :d], qr], -1),
               torch.cat([k, kr.expand(T, H, rd)], -1), v, m["scale"],
               sees_window(T, mask_size(m)))
    o = o.reshape(T, H * dv) * torch.sigmoid(linear(h, w[pre + "g"]))
    return linear(o, w[pre + "o"])


def mixer_chunked_attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, G, D, dv = (m[x] for x in ("heads", "kv_heads", "dim", "vdim"))
    q = linear(h, w[pre + "q"]).view(T, H, D)
    k = linear(h, w[pre + "k"]).view(T, G, D)
    v = linear(h, w[pre + "v"]).view(T, G, dv)
    rot = m.get("rot")
    if rot:
        f, mult = rotary(rot, h.dtype)
        q = rotate(q, f, mult, int(rot["dims"]))
        k = rotate(k, f, mult, int(rot["dims"]))
    o = attend(q, k, v, m["scale"], sees_chunk(T, mask_size(m)))
    o = o * torch.sigmoid(linear(h, w[pre + "g"]))[:, :, None]
    return linear(o.reshape(T, H * dv), w[pre + "o"])


# ---- recurrences ------------------------------------------------------------
def delta_core(q, k, v, beta, g):
    """q, k [T, H, D] (ready to use), v [T, H, Dv], beta [T, H], g [T, H, D]
    -> o [T, H, Dv], final state [H, D, Dv]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def mixer_channel_delta(h, w, pre, m, eps):
    T = h.shape[0]
    H, G, D, dv = (m[x] for x in ("heads", "kv_heads", "dim", "vdim"))
    per = H // G
    q, k, v = (silu(causal_conv(linear(h, w[pre + n]), w[f"{pre}{n}.conv"]))
               for n in "qkv")
    q = (unit(q.view(T, G, D)) * D ** -0.5).repeat_interleave(per, 1)
    k = unit(k.view(T, G, D)).repeat_interleave(per, 1)
    beta = torch.sigmoid(linear(h, w[pre + "b"]))
    a = linear(linear(h, w[pre + "a1"]), w[pre + "a2"]) + w[pre + "dt_bias"]
    g = torch.exp(-torch.exp(w[pre + "A_log"])[None, :, None]
                  * softplus(a).view(T, H, D))
    o, _ = delta_core(q, k, v.view(T, H, dv), beta, g)
    o = rms_norm(o, w[pre + "norm"], eps).reshape(T, H * dv)
    o = o * torch.sigmoid(linear(linear(h, w[pre + "g1"]), w[pre + "g2"]))
    return linear(o, w[pre + "o"])


def ssm_core(x, B, C, dt, A_log, D_skip):
    """x [T, H, P], B and C [T, H, N], dt [T, H] -> y [T, H, P]."""
    T, H, P = x.shape
    S = torch.zeros(H, B.shape[-1], P, dtype=x.dtype)
    y = torch.zeros_like(x)
    for t in range(T):
        a = torch.exp(-torch.exp(A_log) * dt[t])
        S = a[:, None, None] * S + (dt[t][:, None] * B[t])[:, :, None] \
            * x[t][:, None, :]
        y[t] = (S * C[t][:, :, None]).sum(1) + D_skip[:, None] * x[t]
    return y


def mixer_state_space(h, w, pre, m, eps):
    T = h.shape[0]
    H, P, N, G = (m[x] for x in ("heads", "vdim", "state", "groups"))
    inner = H * P
    z, xbc, dt = torch.split(linear(h, w[pre + "in"]),
                             [inner, inner + 2 * G * N, H], -1)
    xbc = silu(causal_conv(xbc, w[pre + "conv"], w[pre + "conv.b"]))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    dt = softplus(dt + w[pre + "dt_bias"])
    y = ssm_core(x.view(T, H, P),
                 B.view(T, G, N).repeat_interleave(H // G, 1),
                 C.view(T, G, N).repeat_interleave(H // G, 1), dt,
                 w[pre + "A_log"], w[pre + "D"]).reshape(T, inner)
    y = y * silu(z)
    parts = m["norm_groups"]
    y = rms_unit(y.view(T, parts, inner // parts), eps).reshape(T, inner)
    return linear(y * w[pre + "norm"], w[pre + "o"])


def mixer_parallel(h, w, pre, m, eps):
    a = mixer_chunked_attention(h, w, pre + "left.", m["left"], eps)
    b = mixer_state_space(h, w, pre + "right.", m["right"], eps)
    return 0.5 * (rms_norm(a, w[pre + "left.out"], eps)
                  + rms_norm(b, w[pre + "right.out"], eps))


MIXERS = {"latent_attention": mixer_latent_attention,
          "channel_delta": mixer_channel_delta, "parallel": mixer_parallel}


# ---- feed-forwards ----------------------------------------------------------
def clamped_gate(g, u, limit):
    g = torch.clamp(g, max=limit)
    u = torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def ff_dense(h, w, pre, mlp):
    g = linear(h, w[pre + "gate"], w[pre + "gate.b"])
    u = linear(h, w[pre + "up"], w[pre + "up.b"])
    return linear(clamped_gate(g, u, mlp["limit"]), w[pre + "down"],
                  w[pre + "down.b"])


def route(h, w, pre, r):
    s = torch.sigmoid(linear(h, w[pre + "router"]))
    wt, ids = s.topk(r["top"], -1)
    return ids, wt


def ff_moe(h, w, pre, mlp):
    ids, wt = route(h, w, pre, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(ids[t].tolist(), wt[t]):
            z = linear(a * h[t:t + 1], w[f"{pre}e{e}.up"])
            out[t] += linear(gelu_erf(z), w[f"{pre}e{e}.down"])[0]
    return out


def feed_forward(h, w, pre, mlp):
    return (ff_moe if mlp["kind"] == "moe" else ff_dense)(h, w, pre, mlp)


# ---- the stack --------------------------------------------------------------
def run_layer(x, cfg, w, i):
    lc, eps, p = cfg["layers"][i], cfg["norm"]["eps"], f"l{i}."
    h = rms_norm(x, w[p + "norm1"], eps)
    h = h + causal_conv(h, w[p + "canon1"])
    y = MIXERS[lc["type"]](h, w, p + "mix.", lc["mixer"], eps)
    if lc.get("mlp"):
        y = y + feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.",
                             lc["mlp"])
    return x + y


def depth_average(results, weights):
    return sum(a * r for a, r in zip(weights, results))


def forward(cfg, weights, tokens, dtype=torch.float64):
    """-> (logits [T, vocab], residual after every layer [layers, T, W])."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v)
         for k, v in weights.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    eps = cfg["norm"]["eps"]
    x = rms_norm(w["embed"][tokens], w["embed.norm"], eps)
    results, after = [x], []
    for i in range(len(cfg["layers"])):
        results.append(run_layer(x, cfg, w, i))
        x = depth_average(results, w[f"l{i}.dwa"])
        after.append(x)
    hid = rms_norm(x, w["final.norm"], eps)
    return hid @ w["head"].T * cfg["logit_scale"], torch.stack(after)


# ---- test models: configurations, random checkpoints, model folders ---------
def dense(ff=12, limit=1.0):
    return dict(kind="dense", ff=ff, limit=limit)


def moe(ff=6, experts=5, top=2):
    return dict(kind="moe", expert=dict(ff=ff),
                router=dict(experts=experts, top=top))


def latent(heads=2, dim=6, rot_dim=4, vdim=5, rank=8, size=5, base=100.0,
           scale=None, mlp="dense"):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=rank,
             rot=dict(base=base, dims=rot_dim),
             scale=scale if scale is not None else (dim + rot_dim) ** -0.5)
    if size:
        m["mask"] = dict(size=size)
    return dict(type="latent_attention", mixer=m,
                mlp=dense() if mlp == "dense" else mlp)


def delta(heads=4, kv_heads=2, dim=6, vdim=5, conv=4, mlp="dense"):
    return dict(type="channel_delta", mlp=dense() if mlp == "dense" else mlp,
                mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
                           conv=conv))


YARN = dict(factor=4.0, fast=8.0, original=64, slow=1.0)


def parallel(heads=4, kv_heads=2, dim=8, vdim=6, dims=4, size=7, base=100.0,
             scaling=YARN, scale=None, s_heads=4, s_vdim=5, state=6, groups=2,
             norm_groups=2, conv=3, mlp="dense"):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim,
                scale=scale if scale is not None else dim ** -0.5)
    if dims:
        left["rot"] = dict(base=base, dims=dims)
        if scaling:
            left["rot"]["scaling"] = dict(scaling)
    if size:
        left["mask"] = dict(size=size)
    right = dict(heads=s_heads, vdim=s_vdim, state=state, groups=groups,
                 norm_groups=norm_groups, conv=conv)
    return dict(type="parallel", mixer=dict(left=left, right=right),
                mlp=dense() if mlp == "dense" else mlp)


def make_config(width=24, vocab=50, eps=1e-5, taps=3, logit_scale=0.7,
                layers=None):
    return dict(architecture="Nikedra", vocab=vocab, width=width,
                norm=dict(eps=eps), canon=dict(taps=taps),
                logit_scale=logit_scale,
                layers=layers or [delta(), parallel(mlp=moe()), latent()])


def make_weights(cfg, seed=0, ranks=(3, 4)):
    """Random bf16-representable weights (fp32 tensors) for a config; ranks:
    inner sizes of the decay's and the gate's low-rank projections."""
    gen = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def rnd(*shape, std=None):
        std = std if std is not None else 1.0 / math.sqrt(shape[-1])
        return (torch.randn(*shape, generator=gen) * std).bfloat16().float()

    def about(mean, *shape, spread=0.2):
        return (mean + spread * torch.randn(shape, generator=gen)) \
            .bfloat16().float()

    out = {"embed": rnd(cfg["vocab"], W, std=1.0), "embed.norm": about(1.0),
           "final.norm": about(1.3), "head": rnd(cfg["vocab"], W)}

    def put_attention(m, a):
        H, G, D, dv = (a[x] for x in ("heads", "kv_heads", "dim", "vdim"))
        out[m + "q"] = rnd(H * D, W, std=1.5 / math.sqrt(W))
        out[m + "k"] = rnd(G * D, W, std=1.5 / math.sqrt(W))
        out[m + "v"] = rnd(G * dv, W)
        out[m + "g"] = rnd(H, W)
        out[m + "o"] = rnd(W, H * dv)

    def put_state_space(m, s):
        H, P, N, G = (s[x] for x in ("heads", "vdim", "state", "groups"))
        inner, ch = H * P, H * P + 2 * G * N
        out[m + "in"] = rnd(inner + ch + H, W)
        out[m + "conv"] = rnd(ch, s["conv"])
        out[m + "conv.b"] = rnd(ch, std=0.2)
        out[m + "dt_bias"] = about(-1.0, H, spread=0.5)
        out[m + "A_log"] = about(-0.5, H, spread=0.5)
        out[m + "D"] = about(1.0, H)
        out[m + "norm"] = about(1.0, inner)
        out[m + "o"] = rnd(W, inner)

    for i, lc in enumerate(cfg["layers"]):
        p, mc = f"l{i}.", lc["mixer"]
        m = p + "mix."
        out[p + "norm1"] = about(0.9)
        out[p + "canon1"] = rnd(W, cfg["canon"]["taps"], std=0.4)
        # the newest result weighs most, the earlier ones visibly
        out[p + "dwa"] = torch.cat([rnd(i + 1, std=0.25), about(1.0, 1)])
        if lc["type"] == "parallel":
            put_attention(m + "left.", mc["left"])
            put_state_space(m + "right.", mc["right"])
            out[m + "left.out"] = about(1.0, W)
            out[m + "right.out"] = about(1.0, W)
        elif lc["type"] == "latent_attention":
            H, d, rd, dv, r = (mc[x] for x in ("heads", "dim", "rot_dim",
                                               "vdim", "kv_rank"))
            out[m + "q"] = rnd(H * (d + rd), W, std=1.5 / math.sqrt(W))
            out[m + "dkv"] = rnd(r + rd, W, std=1.5 / math.sqrt(W))
            out[m + "dkv.norm"] = about(1.0, r)
            out[m + "uk"], out[m + "uv"] = rnd(H * d, r), rnd(H * dv, r)
            out[m + "g"], out[m + "o"] = rnd(H * dv, W), rnd(W, H * dv)
        else:
            H, G, D, dv = (mc[x] for x in ("heads", "kv_heads", "dim",
                                           "vdim"))
            for n, c in (("q", G * D), ("k", G * D), ("v", H * dv)):
                out[m + n] = rnd(c, W)
                out[f"{m}{n}.conv"] = rnd(c, mc["conv"])
            out[m + "b"] = rnd(H, W)
            out[m + "A_log"] = about(-1.0, H, spread=0.5)
            out[m + "norm"] = about(1.0, dv)
            out[m + "a1"] = rnd(ranks[0], W)
            out[m + "a2"] = rnd(H * D, ranks[0])
            out[m + "dt_bias"] = about(-1.5, H * D, spread=1.0)
            out[m + "g1"] = rnd(ranks[1], W)
            out[m + "g2"] = rnd(H * dv, ranks[1])
            out[m + "o"] = rnd(W, H * dv)
        mlp, f = lc.get("mlp"), p + "mlp."
        if not mlp:
            continue
        out[p + "norm2"] = about(1.1)
        if mlp["kind"] == "dense":
            for n, (a, b) in (("gate", (mlp["ff"], W)), ("up", (mlp["ff"], W)),
                              ("down", (W, mlp["ff"]))):
                out[f + n], out[f + n + ".b"] = rnd(a, b), rnd(a, std=0.3)
        else:
            out[f + "router"] = rnd(mlp["router"]["experts"], W,
                                    std=2.0 / math.sqrt(W))
            ff = mlp["expert"]["ff"]
            for j in range(mlp["router"]["experts"]):
                out[f"{f}e{j}.up"] = rnd(ff, W, std=2.0 / math.sqrt(W))
                out[f"{f}e{j}.down"] = rnd(W, ff)
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
