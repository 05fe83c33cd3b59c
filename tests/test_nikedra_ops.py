"""The mechanisms of the Nikedra decoder one at a time: the op layer
(xllm_service_amd.ops.hybrid; fp32 torch on the CPU, HIP kernels under the gpu
marker, fp32 and bf16 storage) against the plain functions of
tests/nikedra_oracle.py. Inputs are made so that a fault shows: one key whose
score stands out just inside or just outside a window or a chunk, decays that
keep one key channel and forget the others, gate values on both sides of the
clamps, layer results of very different sizes in the depth average."""
import math

import pytest
import torch

import nikedra_oracle as no
from xllm_service_amd.models.mixers import scaled_rope_frequencies
from xllm_service_amd.models.moe import RoutedExperts
from xllm_service_amd.ops import hybrid as hops

F64 = torch.float64
TARGETS = [("cpu", torch.float32),
           pytest.param(("cuda", torch.float32), marks=pytest.mark.gpu),
           pytest.param(("cuda", torch.bfloat16), marks=pytest.mark.gpu)]
BS = 16                                    # page size of the engine's pool


def _tol(target):
    return 2e-5 if target[1] == torch.float32 else 2e-2


def _close(got, want, target, what="", scale=1.0):
    got, want = got.detach().cpu().to(F64), want.to(F64)
    err = float((got - want).abs().max() / max(float(want.abs().max()), 1e-9))
    assert err < _tol(target) * scale, (what, err)


def _rnd(g, *shape, dtype=torch.float32, std=1.0):
    """Random values that bf16 holds exactly (so both storage types see the
    same inputs as the fp64 functions)."""
    return (torch.randn(*shape, generator=g) * std).bfloat16().to(dtype)


def _i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


# ------------------------------------------------- depth average, activations
@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("W", [20, 257, 1288])
@pytest.mark.parametrize("f32", [False, True])
def test_depth_average_with_two_norms(target, W, f32):
    """A chain of layers: entry (a normed row, no weights), a plain mixer
    output, two normed halves, with and without a feed-forward."""
    dev, dt = target
    g = torch.Generator().manual_seed(W)
    T, levels, eps = 5, 6, 1e-5

    def d(t):
        return None if t is None else t.to(dev)
    hist = torch.full((levels, T, W), float("nan"), device=dev)
    e = _rnd(g, T, W, dtype=dt, std=3.0)
    ge, g1, g2 = (torch.tensor([v]) for v in (0.7, 1.3, -0.4))
    h1, h2 = hops.depth_mix_norm(None, hist, 0, d(e), d(ge), None, None, 1.0,
                                 None, None, d(g1), d(g2), eps, dt)
    x = no.rms_norm(e.to(F64), 0.7, eps)
    results = [x]
    _close(hist[0], x, target if dt == torch.float32 else
           ("", torch.float32), "entry", 5)
    _close(h1, no.rms_norm(x, 1.3, eps), target, "entry h1")
    _close(h2, no.rms_norm(x, -0.4, eps), target, "entry h2")
    xd = torch.full((T, W), float("nan"), device=dev)
    for lv in range(1, levels):
        halves, has_f = lv % 2 == 0, lv != 3
        m1, m2 = (_rnd(g, T, W, dtype=dt, std=10.0 ** (lv - 3))
                  for _ in range(2))
        w1, w2 = (1.0 + 0.5 * torch.randn(W, generator=g) for _ in range(2))
        f = _rnd(g, T, W, dtype=torch.float32 if f32 else dt)
        dwa = torch.randn(lv + 1, generator=g)
        if halves:
            parts = (d(m1), d(w1), d(m2), d(w2), 0.5)
            y = 0.5 * (no.rms_norm(m1.to(F64), w1.to(F64), eps)
                       + no.rms_norm(m2.to(F64), w2.to(F64), eps))
        else:
            parts = (d(m1), None, None, None, 1.0)
            y = m1.to(F64)
        last = lv == levels - 1
        h1, h2 = hops.depth_mix_norm(
            hist[0] if lv == 1 else xd, hist, lv, *parts,
            d(f) if has_f else None, d(dwa), d(g1), None if last else d(g2),
            eps, dt, xd)
        results.append(x + y + (f.to(F64) if has_f else 0.0))
        x = no.depth_average(results, dwa.to(F64))
        _close(hist[lv], results[-1], ("", torch.float32), ("kept", lv), 5)
        _close(xd, x, ("", torch.float32), ("x", lv), 5)
        _close(h1, no.rms_norm(x, 1.3, eps), target, ("h1", lv))
        assert (h2 is None) == last
        if h2 is not None:
            _close(h2, no.rms_norm(x, -0.4, eps), target, ("h2", lv))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("F", [5, 12, 352])
@pytest.mark.parametrize("limit", [0.5, 7.0])
def test_clamped_gate(target, F, limit):
    """The gate has no lower bound, the up half has both."""
    dev, dt = target
    g = torch.Generator().manual_seed(F)
    x = _rnd(g, 7, 2 * F, dtype=dt, std=3.0)
    x[0, 0], x[0, F] = 40.0, -40.0
    x[1, 0], x[1, F] = -9.0, 40.0
    x[2, 0], x[2, F] = -0.75, -1.0
    want = no.clamped_gate(x[:, :F].to(F64), x[:, F:].to(F64), limit)
    _close(hops.clamped_glu(x.to(dev), limit, 1.702, 1.0), want, target)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("F", [3, 8, 130])
def test_scaled_gelu(target, F):
    dev, dt = target
    g = torch.Generator().manual_seed(F)
    x = _rnd(g, 12, F, dtype=dt, std=2.0)
    s = torch.rand(12, generator=g)
    _close(hops.gelu_scaled(x.to(dev)), no.gelu_erf(x.to(F64)), target)
    _close(hops.gelu_scaled(x.to(dev), s.to(dev)),
           no.gelu_erf(x.to(F64) * s.to(F64)[:, None]), target)
    # four tokens, three experts; token 2 chose experts 0 and 2 ...
    ids = torch.tensor([[1, 0], [0, 1], [2, 0], [1, 2]], dtype=torch.int32)
    wts = torch.rand(4, 2, generator=g)
    want = torch.zeros(3, 4, F, dtype=F64)
    for t in range(4):
        for e, a in zip(ids[t].tolist(), wts[t]):
            want[e, t] = no.gelu_erf(a.to(F64) * x.view(3, 4, F)[e, t].to(F64))
    got = hops.gelu_scaled(x.view(3, 4, F).to(dev), None, ids.to(dev),
                           wts.to(dev))
    _close(got, want, target, "routed")


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("T", [9, 300])
@pytest.mark.parametrize("experts,top", [(5, 2), (4, 1), (3, 3), (1, 1)])
def test_experts_with_weighted_inputs(target, T, experts, top):
    """All execution shapes (dense batched, padded batched, expert by
    expert: most tokens alike) against one expert call per choice."""
    dev, dt = target
    g = torch.Generator().manual_seed(10 * experts + top)
    W, ff = 24, 16
    w = {"router": _rnd(g, experts, W, std=0.5)}
    m = RoutedExperts(W, ff, experts, top, 1, 1, dt, gated=False,
                      weight_input=True)
    with torch.no_grad():
        m.router.copy_(w["router"])
    for e in range(experts):
        w[f"e{e}.up"] = _rnd(g, ff, W, std=0.6)
        w[f"e{e}.down"] = _rnd(g, W, ff, std=0.3)
        m.load_expert(e, w[f"e{e}.up"], w[f"e{e}.down"])
    m = m.to(dev)
    mlp = dict(router=dict(top=top))
    for skew in (False, True):
        h = torch.randn(T, W, generator=g)
        if skew:
            h[: 2 * T // 3] = h[0] + 0.01 * h[: 2 * T // 3]
        h = h.bfloat16().to(dt)
        want = no.ff_moe(h.to(F64), {k: v.to(F64) for k, v in w.items()}, "",
                         mlp)
        m.dense_max_tokens = 64
        with torch.no_grad():
            got = m(h.to(dev))
            m.dense_max_tokens = 0 if T <= 64 else 10 ** 6   # the other shape
            again = m(h.to(dev))
        for what, y in (("auto", got), ("other", again)):
            bad = no.rel_err(y.cpu(), want) > \
                (1e-4 if dt == torch.float32 else 0.1)
            assert int(bad.sum()) <= T // 40, (what, skew, int(bad.sum()))


# --------------------------------------------------------- turns and stores
YARN = dict(factor=4.0, original=64, fast=4.0, slow=1.0)


def test_frequency_ramp():
    """The ramp between the pairs that turn fast and slow, for constants
    that put its ends inside, outside and on one pair."""
    for rot in (dict(base=100.0, dims=16, scaling=YARN),
                dict(base=1e6, dims=64, scaling=dict(factor=8.0, fast=32.0,
                                                     original=512, slow=1.0)),
                dict(base=50.0, dims=6, scaling=dict(factor=2.0, fast=1.0,
                                                     original=2, slow=1.0)),
                dict(base=50.0, dims=2, scaling=dict(factor=2.0, fast=64.0,
                                                     original=64, slow=0.5)),
                dict(base=100.0, dims=8)):
        f, mult = scaled_rope_frequencies(rot)
        want, wm = no.rotary(rot)
        assert torch.allclose(f, want, rtol=1e-12) and abs(mult - wm) < 1e-12
        if rot.get("scaling"):
            assert mult > 1.0


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("D,rot", [(12, 8), (64, 64), (10, 2), (128, 96)])
def test_half_layout_turn_with_multiplier(target, D, rot):
    """Queries and keys at positions up to 3000 turned in the half layout by
    stretched frequencies, cos and sin times the multiplier; the in-place
    turn of a part of every head gives the same."""
    dev, dt = target
    g = torch.Generator().manual_seed(D)
    H, G, T = 4, 2, 6
    freqs, mult = scaled_rope_frequencies(dict(base=100.0, dims=rot,
                                               scaling=YARN))
    pos = torch.tensor([0, 1, 2, 63, 700, 3000])
    q, k, v = _rnd(g, T, H * D, dtype=dt), _rnd(g, T, G * D, dtype=dt), \
        _rnd(g, T, G * 3, dtype=dt)

    def turn(z, n):
        full = torch.zeros(3001, n, D, dtype=F64)
        full[pos] = z.to(F64).view(T, n, D)
        return no.rotate(full, freqs, mult, rot)[pos]
    kc = torch.zeros(1, G, BS, D, dtype=dt, device=dev)
    vc = torch.zeros(1, G, BS, 3, dtype=dt, device=dev)
    slots = torch.tensor([3, 0, 9, 1, 15, 7], device=dev)
    qn = hops.rope_headnorm_store(
        q.to(dev), k.to(dev), v.to(dev), pos.to(dev), freqs.to(dev), rot,
        False, False, 1e-5, H, G, kc, vc, slots, mult)
    _close(qn.view(T, H, D), turn(q, H), target, "q")
    _close(kc[0][:, slots].transpose(0, 1), turn(k, G), target, "k")
    assert torch.equal(vc[0][:, slots].transpose(0, 1).reshape(T, -1).cpu(), v)
    # heads of [plain part of 5 | turned part]
    big = _rnd(g, T, H, 5 + D, dtype=dt)
    want = big.to(F64).clone()
    want[..., 5:] = turn(big[..., 5:].reshape(T, -1), H)
    got = hops.rope_interleaved_(big.to(dev), pos.to(dev), freqs.to(dev), mult,
                                 5, rot, pairs=False)
    _close(got, want, target, "in place")
    # a latent row: normed part | turned part (half layout)
    r = 7
    dkv, w = _rnd(g, T, r + D, dtype=dt), 1.0 + 0.3 * torch.randn(
        r, generator=g)
    cache = torch.zeros(1, BS, r + D, dtype=dt, device=dev)
    hops.latent_kv_store(dkv.to(dev), w.to(dev), 1e-5, pos.to(dev),
                         freqs.to(dev), mult, rot, cache, slots, r, False)
    rows = cache[0, slots]
    _close(rows[:, :r], no.rms_norm(dkv[:, :r].to(F64), w.to(F64), 1e-5),
           target, "latent")
    _close(rows[:, r:], turn(dkv[:, r:], 1)[:, 0], target, "latent tail")


# ----------------------------------------------------------------- attention
def _paged(rows, dev, dt, seed, spare=3):
    """Scatter tensors [L, G, D] over shuffled pages [blocks, G, 16, D] whose
    other rows hold stale values; returns the caches and the block table."""
    L = rows[0].shape[0]
    nblk = (L + BS - 1) // BS
    g = torch.Generator().manual_seed(seed)
    order = torch.randperm(nblk + spare, generator=g)[:nblk]
    out = []
    for z in rows:
        c = torch.randn(nblk + spare, z.shape[1], BS, z.shape[2],
                        generator=g).to(dt)
        for j in range(L):
            c[order[j // BS], :, j % BS] = z[j].to(dt)
        out.append(c.to(dev))
    return out, order.to(torch.int32)


def _chunk_case(target, H, G, D, Dv, L, asked, size, standout, seed,
                decode=False):
    """The positions `asked` (a range ending at or before L) of a sequence
    query; key `standout` has a score far above the rest for every one."""
    dev, dt = target
    g = torch.Generator().manual_seed(seed)
    q, k, v = (_rnd(g, L, H, D, std=0.5), _rnd(g, L, G, D, std=0.5),
               _rnd(g, L, G, Dv))
    if standout is not None:
        k[standout] = 0.0
        k[standout, :, 0] = 8.0
        q[:, :, 0] = 4.0
    scale = 1.0 / math.sqrt(D)
    a, b = asked
    want = no.attend(q.to(F64), k.to(F64), v.to(F64), scale,
                     no.sees_chunk(L, size))[a:b]
    (kc, vc), table = _paged([k, v], dev, dt, seed)
    out = torch.empty(b - a, H, Dv, dtype=torch.float32, device=dev)
    qq = q[a:b].reshape(b - a, H * D).to(dt).to(dev)
    kw = dict(window=size, chunked=True)
    if decode:
        n = b - a                       # every query a decode row, one batch
        hops.capped_attn(qq, kc, vc, table[None].repeat(n, 1).to(dev), None,
                         _i32(list(range(a + 1, b + 1)), dev), H, scale, 0.0,
                         out, **kw)
    else:
        hops.capped_attn(qq, kc, vc, table[None].to(dev),
                         _i32([0, b - a], dev), _i32([b], dev), H, scale, 0.0,
                         out, **kw)
    return out, want


SHAPES = [(4, 2, 8, 6), (6, 2, 64, 64), (4, 1, 128, 48), (2, 2, 64, 72),
          (3, 3, 10, 10), (5, 5, 192, 200)]


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("H,G,D,Dv", SHAPES)
def test_chunk_edges(target, decode, H, G, D, Dv):
    """Queries on both sides of a chunk's edge; a standout key on the last
    place of the earlier chunk, on the first and on the middle of the
    later."""
    size, L = 40, 130
    for edge in (40, 80, 120):
        for standout in (edge - 1, edge, edge + 2, edge - size):
            got, want = _chunk_case(target, H, G, D, Dv, L,
                                    (edge - 2, min(edge + 5, L)), size,
                                    standout, edge + standout, decode)
            _close(got, want, target, (edge, standout))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("size", [1, 2, 15, 16, 17, 31, 32, 33, 64, 100, 500])
def test_chunks_at_page_and_tile_borders(target, decode, size):
    L = 100
    for a, b in ((0, 1), (0, 40), (60, 100), (size - 1, size + 1)):
        if b > L:
            continue
        got, want = _chunk_case(target, 4, 2, 64, 64, L, (a, b), size, None,
                                size + a, decode)
        _close(got, want, target, (a, b, size))


@pytest.mark.parametrize("target", TARGETS)
def test_chunk_decode_over_context_partitions(target, monkeypatch):
    monkeypatch.setenv("XLLM_CAPPED_PARTS", "5")
    for size, standout in ((300, 600), (300, 599), (257, 771), (1000, 3)):
        got, want = _chunk_case(target, 4, 2, 64, 32, 820, (815, 820), size,
                                standout, size, True)
        _close(got, want, target, (size, standout))


def _latent_case(target, H, r, rd, L, asked, window, standout, seed,
                 decode=False):
    """Queries folded to the width of the cached rows [c | turned key]; the
    row `standout` is scored far above the rest through its tail."""
    dev, dt = target
    g = torch.Generator().manual_seed(seed)
    rows = _rnd(g, L, r + rd, std=0.5)
    q = _rnd(g, L, H, r + rd, std=0.5)
    if standout is not None:
        rows[standout, r:] = 0.0
        rows[standout, -1] = 8.0
        q[:, :, -1] = 4.0
    a, b = asked
    mask = no.sees_window(L, window)
    want = torch.stack([
        no.attend(q[:, h:h + 1].to(F64), rows[:, None].to(F64),
                  rows[:, None, :r].to(F64), 0.4, mask)[a:b, 0]
        for h in range(H)], 1)
    (cache,), table = _paged([rows[:, None]], dev, dt, seed)
    cache = cache[:, 0].contiguous()
    out = torch.empty(b - a, H, r, dtype=torch.float32, device=dev)
    qq = q[a:b].to(dt).contiguous().to(dev)
    if decode:
        n = b - a
        hops.latent_attn(qq, cache, table[None].repeat(n, 1).to(dev), None,
                         _i32(list(range(a + 1, b + 1)), dev), 0.4, r, out,
                         window)
    else:
        hops.latent_attn(qq, cache, table[None].to(dev),
                         _i32([0, b - a], dev), _i32([b], dev), 0.4, r, out,
                         window)
    return out, want


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("H,r,rd", [(2, 9, 4), (4, 88, 24), (20, 64, 16),
                                    (3, 200, 40), (2, 512, 64), (40, 40, 8)])
def test_latent_window_edges(target, decode, H, r, rd):
    L, window = 150, 37
    for standout in (149 - window + 1, 149 - window, 149 - window - 3, 149,
                     0, 112):
        got, want = _latent_case(target, H, r, rd, L, (146, 150), window,
                                 standout, r + standout, decode)
        _close(got, want, target, standout)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("window", [0, 1, 15, 16, 17, 32, 33, 64, 500])
def test_latent_windows_at_page_and_tile_borders(target, decode, window):
    for a, b in ((0, 1), (0, 50), (60, 100)):
        got, want = _latent_case(target, 4, 64, 32, 100, (a, b), window, None,
                                 window + a, decode)
        _close(got, want, target, (a, b, window))


@pytest.mark.parametrize("target", TARGETS)
def test_latent_window_decode_over_partitions(target, monkeypatch):
    monkeypatch.setenv("XLLM_LATENT_PARTS", "7")
    for window, standout in ((400, 420), (400, 419), (33, 787), (0, 5)):
        got, want = _latent_case(target, 4, 64, 32, 820, (818, 820), window,
                                 standout, window, True)
        _close(got, want, target, (window, standout))


# --------------------------------------------------------------- recurrences
def _delta_inputs(g, T, H, G, D, Dv, dt):
    return (_rnd(g, T, G * D, dtype=dt), _rnd(g, T, G * D, dtype=dt),
            _rnd(g, T, H * Dv, dtype=dt), _rnd(g, T, H, dtype=dt, std=2.0),
            _rnd(g, T, H * D, dtype=dt, std=2.0))


def _delta_want(q, k, v, b, a, A_log, dt_bias, H, G, D, Dv):
    T, per = q.shape[0], H // G
    q, k, v, b, a = (z.to(F64) for z in (q, k, v, b, a))
    q = (no.unit(q.view(T, G, D)) * D ** -0.5).repeat_interleave(per, 1)
    k = no.unit(k.view(T, G, D)).repeat_interleave(per, 1)
    g = torch.exp(-torch.exp(A_log.to(F64))[None, :, None]
                  * no.softplus(a + dt_bias.to(F64)).view(T, H, D))
    return no.delta_core(q, k, v.view(T, H, Dv), torch.sigmoid(b), g)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 6, 5), (1, 1, 16, 16),
                                      (3, 3, 40, 12), (4, 2, 64, 64),
                                      (2, 1, 256, 32), (2, 2, 1, 4),
                                      (32, 8, 32, 64)])
def test_channel_decay_through_portions_and_slots(target, H, G, D, Dv):
    """A sequence fed in portions (down to one and two tokens) must give what
    the whole gives; its slot held another sequence's state before; a row
    without a slot runs from zero and stores nothing."""
    dev, dt = target
    g = torch.Generator().manual_seed(H * D + Dv)
    T = 45
    q, k, v, b, a = _delta_inputs(g, T, H, G, D, Dv, dt)
    A_log = torch.randn(H, generator=g) * 0.5 - 1.0
    dt_bias = torch.randn(H * D, generator=g)
    want, S_end = _delta_want(q, k, v, b, a, A_log, dt_bias, H, G, D, Dv)
    dq, dk, dv, db, da = (x.to(dev) for x in (q, k, v, b, a))
    for cuts in ([T], [1, 2, 17, 1, 1, 16, 7], [2] * 5 + [33, 1, 1]):
        state = torch.randn(3, H, D, Dv, generator=g).to(dev)   # stale
        before = state.clone()
        out = torch.empty(T, H, Dv, device=dev)
        at = 0
        for n in cuts:
            rows = slice(at, at + n)
            single = n == 1 and at > 0
            if single:
                slots, cu, ctx = [1], None, [at]
                sel, o = rows, out[rows]
            else:                  # a second request without a slot rides along
                slots, cu, ctx = [1, -1], [0, n, n + 2], [at, 5]
                sel = list(range(at, at + n)) + [0, 1]
                o = torch.empty(n + 2, H, Dv, device=dev)
            hops.delta_rule(dq[sel], dk[sel], dv[sel], db[sel], da[sel],
                            dt_bias.to(dev), A_log.to(dev), state,
                            _i32(slots, dev), None if cu is None
                            else _i32(cu, dev), _i32(ctx, dev), G, o)
            if not single:
                out[rows] = o[:n]
            at += n
        _close(out, want, target, cuts, 5)
        _close(state[1], S_end, target, ("state", cuts), 5)
        assert torch.equal(state[0], before[0]) and \
            torch.equal(state[2], before[2])


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("H,G,D,Dv", [(2, 1, 40, 12), (4, 2, 64, 64),
                                      (2, 2, 128, 128), (3, 1, 16, 100)])
def test_channel_decay_long_chunks(target, H, G, D, Dv):
    """Chunks long enough for the piece-parallel passes, from a zero state
    and from a carried one, beside a short request; slow and fast decays
    beside each other in one head."""
    dev, dt = target
    g = torch.Generator().manual_seed(D + Dv)
    T = 650
    q, k, v, b, a = _delta_inputs(g, T, H, G, D, Dv, dt)
    A_log = torch.randn(H, generator=g) * 0.5 - 2.0
    dt_bias = torch.linspace(-9.0, 3.0, H * D)[torch.randperm(
        H * D, generator=g)]
    want, S_end = _delta_want(q, k, v, b, a, A_log, dt_bias, H, G, D, Dv)
    dq, dk, dv, db, da = (x.to(dev) for x in (q, k, v, b, a))
    for cuts in ([T], [37, T - 37]):
        state = torch.randn(3, H, D, Dv, generator=g).to(dev)   # stale
        out = torch.empty(T, H, Dv, device=dev)
        at = 0
        for n in cuts:
            sel = list(range(5)) + list(range(at, at + n))
            o = torch.empty(n + 5, H, Dv, device=dev)
            hops.delta_rule(dq[sel], dk[sel], dv[sel], db[sel], da[sel],
                            dt_bias.to(dev), A_log.to(dev), state,
                            _i32([-1, 2], dev), _i32([0, 5, n + 5], dev),
                            _i32([0, at], dev), G, o, max_q_len=n)
            out[at:at + n] = o[5:]
            at += n
        _close(out, want, target, cuts, 10)
        _close(state[2], S_end, target, ("state", cuts), 10)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("cols", ["1", "4"])
def test_one_channel_remembers(target, cols, monkeypatch):
    """Channel 0 keeps what it holds, every other channel forgets at once: a
    value written at the first token under a key along channel 0 is read
    back 300 tokens later, in a prompt and in decoding."""
    monkeypatch.setenv("XLLM_DELTA_COLS", cols)
    dev, dt = target
    H, D, Dv, T = 2, 32, 48, 300
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.zeros(T, H * D), torch.zeros(T, H * D),
               _rnd(g, T, H * Dv))
    q.view(T, H, D)[:, :, 0] = 1.0
    k.view(T, H, D)[0, :, 0] = 1.0
    k.view(T, H, D)[1:, :, 1:] = _rnd(g, T - 1, H, D - 1)
    b = torch.full((T, H), 30.0)                      # beta = 1
    a = torch.zeros(T, H * D)
    dt_bias = torch.full((H, D), 60.0)
    dt_bias[:, 0] = -60.0
    q, k, v, b, a = (z.to(dt).to(dev) for z in (q, k, v, b, a))
    dt_bias, A_log = dt_bias.reshape(-1).to(dev), torch.zeros(H, device=dev)
    state = torch.zeros(1, H, D, Dv, device=dev)
    out = torch.empty(T, H, Dv, device=dev)
    n = T - 3
    hops.delta_rule(q[:n], k[:n], v[:n], b[:n], a[:n], dt_bias, A_log, state,
                    _i32([0], dev), _i32([0, n], dev), _i32([0], dev), H,
                    out[:n])
    for t in range(n, T):
        s = slice(t, t + 1)
        hops.delta_rule(q[s], k[s], v[s], b[s], a[s], dt_bias, A_log, state,
                        _i32([0], dev), None, _i32([t], dev), H, out[s])
    want = (v[0].view(H, Dv).cpu().to(F64) * D ** -0.5).expand(T, H, Dv)
    _close(out, want, target)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("C,taps", [(10, 4), (7, 3), (256, 2), (24, 1),
                                    (6, 6)])
def test_input_convolution(target, C, taps):
    """h + conv(h) through portions shorter than the filter and decoded rows,
    in slots that held other sequences; the decode rows move the state
    themselves."""
    dev, dt = target
    g = torch.Generator().manual_seed(C + taps)
    T = 23
    xs = [_rnd(g, T, C, dtype=dt) for _ in range(2)]
    w = _rnd(g, C, taps, dtype=dt)
    wants = [x.to(F64) + no.causal_conv(x.to(F64), w.to(F64)) for x in xs]
    state = torch.randn(4, taps - 1, C, generator=g).to(dt).to(dev)
    before = state.clone()
    got = [[], []]
    at = [0, 0]
    for step in ([2, 1], [1, 2], [1, 1], [5, 7], [1, 1], [2, 9], [11, 2]):
        decode = step == [1, 1]
        rows = [x[p:p + n] for x, p, n in zip(xs, at, step)]
        out = torch.empty(sum(step), C, dtype=dt, device=dev)
        y = hops.short_conv(
            torch.cat(rows).to(dev), w.to(dev), None, state, 0,
            _i32([3, 1], dev), None if decode
            else _i32([0, step[0], sum(step)], dev), _i32(at, dev), 1, C,
            add_input=True, advance=True, out=out)
        assert y is out
        got[0].append(y[:step[0]])
        got[1].append(y[step[0]:])
        at = [p + n for p, n in zip(at, step)]
    assert at == [T, T]
    for i in range(2):
        _close(torch.cat(got[i]), wants[i], target, i)
    assert torch.equal(state[0], before[0]) and torch.equal(state[2],
                                                            before[2])
    if taps > 1:
        k = taps - 1
        assert torch.equal(state[3].cpu(), xs[0][-k:])
        assert torch.equal(state[1].cpu(), xs[1][-k:])
    # a row without a slot (batch padding) reads and stores nothing
    s2 = state.clone()
    hops.short_conv(xs[0][:2].to(dev), w.to(dev), None, s2, 0,
                    _i32([-1, -1], dev), None, _i32([9, 9], dev), 1, C,
                    add_input=True, advance=True)
    assert torch.equal(s2, state)
