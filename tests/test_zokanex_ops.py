"""The mechanisms of the Zokanex decoder one at a time: the op layer
(xllm_service_amd.ops.hybrid; fp32 torch on the CPU, HIP kernels under the gpu
marker, fp32 and bf16 storage) against the plain functions of
tests/zokanex_oracle.py. Inputs are made so that a fault shows: one key whose
score stands out just inside or just outside a window, head norm weights that
differ within a rotary pair, an early key that only a slow head remembers,
lengths around the edges of pages and chunks."""
import math

import pytest
import torch

import zokanex_oracle as zo
from xllm_service_amd.models.mixers import banded_rope_frequencies
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
    assert got.shape == want.shape, (what, got.shape, want.shape)
    err = float((got - want).abs().max() / max(float(want.abs().max()), 1e-9))
    assert err < _tol(target) * scale, (what, err)


EXACT = ("", torch.float32)                # fp32 whatever the storage type


def _rnd(g, *shape, dtype=torch.float32, std=1.0):
    """Random values that bf16 holds exactly (so both storage types see the
    same inputs as the fp64 functions)."""
    return (torch.randn(*shape, generator=g) * std).bfloat16().to(dtype)


def _i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


def _inside(rows, cols, dtype, dev, lead=3, tail=5):
    """A [rows, cols] view in the middle of a wider tensor of NaNs."""
    big = torch.full((rows, lead + cols + tail), float("nan"), dtype=dtype,
                     device=dev)
    return big, big[:, lead:lead + cols]


# ------------------------------------------------------------ row-wise steps
@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("W", [20, 257, 1288])
def test_embedding_row_and_its_norm(target, W):
    dev, dt = target
    g = torch.Generator().manual_seed(W)
    table, w = _rnd(g, 9, W, dtype=dt), 1.0 + torch.rand(W, generator=g)
    ids = torch.tensor([8, 0, 3, 3, 7])
    for rows, idx in ((table, ids), (table, None)):
        x, h = hops.embed_norm(rows.to(dev),
                               None if idx is None else idx.to(dev), 1.75,
                               w.to(dev), 1e-3, dt)
        want = (table if idx is None else table[idx]).to(F64) * 1.75
        assert x.dtype == torch.float32
        _close(x, want, EXACT)
        _close(h, zo.rms_norm(want, w.to(F64), 1e-3), target)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("W", [20, 257, 1288])
@pytest.mark.parametrize("top", [0, 1, 3])
def test_joint_residual_update(target, W, top):
    """The sublayers' sum and the weighted expert rows (one of them absent)
    join the fp32 residual, and its norm follows."""
    dev, dt = target
    g = torch.Generator().manual_seed(W + top)
    T = 6
    x, y = torch.randn(T, W, generator=g) * 3.0, _rnd(g, T, W, dtype=dt)
    w = 1.0 + torch.rand(W, generator=g)
    want, experts = x.to(F64) + y.to(F64), None
    if top:
        e = _rnd(g, 11, W, dtype=dt, std=2.0)
        rows = torch.randint(0, 11, (T, top), generator=g).to(torch.int32)
        wts = torch.rand(T, top, generator=g)
        rows[2, 0] = -1
        for t in range(T):
            for k in range(top):
                if rows[t, k] >= 0:
                    want[t] += wts[t, k].to(F64) * e[rows[t, k]].to(F64)
        experts = (e.to(dev), rows.to(dev), wts.to(dev))
    xd = x.to(dev)
    h = hops.join_norm_(xd, y.to(dev), experts, w.to(dev), 1e-4)
    _close(xd, want, EXACT)
    _close(h, zo.rms_norm(want, w.to(F64), 1e-4), target)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("F", [3, 24, 352])
@pytest.mark.parametrize("gelu", [False, True])
@pytest.mark.parametrize("gated", [False, True])
def test_gate_of_row_views(target, F, gelu, gated):
    """Parts of one wide row in, a part of another out; nothing else there
    is touched."""
    dev, dt = target
    g = torch.Generator().manual_seed(F)
    T = 7
    p = _rnd(g, T, 2 + 2 * F + 1 + 3, dtype=dt, std=2.0)
    p[0, 2], p[1, 2] = 30.0, -30.0
    a, b, s = p[:, 2:2 + F], p[:, 2 + F:2 + 2 * F], p[:, 2 + 2 * F:3 + 2 * F]
    act = zo.gelu_tanh if gelu else zo.silu
    want = act(a.to(F64)) * b.to(F64)
    if gated:
        want = want * torch.sigmoid(s.to(F64))
    pd = p.to(dev)
    big, out = _inside(T, F, dt, dev)
    hops.glu_rows(pd[:, 2:2 + F], pd[:, 2 + F:2 + 2 * F], out, gelu=gelu,
                  row_gate=pd[:, 2 + 2 * F:3 + 2 * F] if gated else None)
    _close(out, want, target)
    assert torch.isnan(big[:, :3]).all() and torch.isnan(big[:, 3 + F:]).all()


@pytest.mark.parametrize("target", TARGETS)
def test_table_of_turns(target):
    """cos | sin stay exact where an angle is large."""
    dev, _ = target
    pos = torch.tensor([0, 1, 777, 1000003])
    f = banded_rope_frequencies(dict(base=5e5, dims=10))
    got = hops.rope_table(pos.to(dev), f.to(dev)).cpu().to(F64)
    for t, p in enumerate(pos.tolist()):
        for i in range(5):
            a = math.fmod(p * 5e5 ** (-2.0 * i / 10), 2 * math.pi)
            assert abs(float(got[t, i]) - math.cos(a)) < 1e-6
            assert abs(float(got[t, 5 + i]) - math.sin(a)) < 1e-6


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("tabled", [False, True])
@pytest.mark.parametrize("D,rot", [(12, 8), (64, 64), (10, 2), (128, 96),
                                   (6, 0), (200, 200)])
def test_head_norm_before_the_turn(target, D, rot, tabled):
    """Weighted norm per head first, then the half-layout turn; keys and
    values to their slots (one token has none), or queries alone."""
    dev, dt = target
    g = torch.Generator().manual_seed(D + rot)
    H, G, T, eps = 4, 2, 6, 1e-2
    pos = torch.tensor([0, 1, 2, 63, 700, 3000])
    freqs = banded_rope_frequencies(dict(base=100.0, dims=rot)) if rot \
        else torch.zeros(0, dtype=F64)
    q, k, v = _rnd(g, T, H * D, dtype=dt), _rnd(g, T, G * D, dtype=dt), \
        _rnd(g, T, G * 3, dtype=dt)
    qw, kw = (0.5 + torch.rand(D, generator=g) for _ in range(2))

    def prep(z, n, w):
        z = zo.rms_norm(z.to(F64).view(T, n, D), w.to(F64), eps)
        return zo.rotate(z, pos, 100.0, rot)
    kc = torch.zeros(1, G, BS, D, dtype=dt, device=dev)
    vc = torch.zeros(1, G, BS, 3, dtype=dt, device=dev)
    slots = torch.tensor([3, 0, -1, 1, 15, 7], device=dev)
    table = hops.rope_table(pos.to(dev), freqs.to(dev)) if tabled and rot \
        else None
    args = (pos.to(dev), freqs.to(dev), rot, False, False, eps, H, G, kc, vc,
            slots, 1.0, qw.to(dev))
    qn = hops.rope_headnorm_store(q.to(dev), k.to(dev), v.to(dev), *args,
                                  kw.to(dev), table)
    _close(qn.view(T, H, D), prep(q, H, qw), target, "q")
    has = slots.cpu() >= 0
    where = slots[has.to(dev)]
    _close(kc[0][:, where].transpose(0, 1), prep(k, G, kw)[has], target, "k")
    assert torch.equal(vc[0][:, where].transpose(0, 1).reshape(5, -1).cpu(),
                       v[has])
    assert float(kc[0, :, 2].abs().max()) == 0.0
    before = kc.clone(), vc.clone()
    alone = hops.rope_headnorm_store(q.to(dev), None, None, *args, None, table)
    assert torch.equal(alone, qn)
    assert torch.equal(before[0], kc) and torch.equal(before[1], vc)


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


def _window_case(target, H, G, D, Dv, L, asked, size, standout, seed,
                 decode=False, lead=8):
    """The positions `asked` (a range) of a sequence query; key `standout`
    has a score far above the rest. The result goes into the middle of wider
    rows of the model dtype."""
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
    want = zo.attend(q.to(F64), k.to(F64), v.to(F64), scale,
                     zo.sees_window(L, size))[a:b]
    (kc, vc), table = _paged([k, v], dev, dt, seed)
    n = b - a
    big, out = _inside(n, H * Dv, dt, dev, lead, 8)
    qq = q[a:b].reshape(n, H * D).to(dt).to(dev)
    if decode:                          # every query a decode row, one batch
        hops.capped_attn(qq, kc, vc, table[None].repeat(n, 1).to(dev), None,
                         _i32(list(range(a + 1, b + 1)), dev), H, scale, 0.0,
                         out, window=size)
    else:
        hops.capped_attn(qq, kc, vc, table[None].to(dev), _i32([0, n], dev),
                         _i32([b], dev), H, scale, 0.0, out, window=size)
    assert torch.isnan(big[:, :lead]).all()
    assert torch.isnan(big[:, lead + H * Dv:]).all()
    return out.view(n, H, Dv) if out.is_contiguous() \
        else out.reshape(n, H, Dv), want


SHAPES = [(4, 2, 8, 6), (5, 1, 64, 40), (4, 1, 128, 48), (2, 2, 64, 72),
          (3, 3, 10, 10), (5, 5, 192, 200)]


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("H,G,D,Dv", SHAPES)
def test_window_edges_into_joint_rows(target, decode, H, G, D, Dv):
    """A standout key on the last place the window holds, on the next one,
    and on the query itself."""
    size, L = 40, 130
    for i in (45, 64, 128):
        for standout in (i - size, i - size + 1, i):
            got, want = _window_case(target, H, G, D, Dv, L, (i - 1, i + 2),
                                     size, standout, i + standout, decode)
            _close(got, want, target, (i, standout))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("size", [0, 1, 2, 15, 16, 17, 31, 32, 33, 64, 500])
def test_windows_at_page_and_tile_borders(target, decode, size):
    L = 100
    for (a, b), lead in (((0, 1), 8), ((0, 40), 3), ((60, 100), 8)):
        got, want = _window_case(target, 4, 2, 64, 64, L, (a, b), size, None,
                                 size + a, decode, lead)
        _close(got, want, target, (a, b, size))


@pytest.mark.parametrize("target", TARGETS)
def test_window_decode_over_context_partitions(target, monkeypatch):
    monkeypatch.setenv("XLLM_CAPPED_PARTS", "5")
    for size, standout in ((300, 700 - 300), (300, 700 - 299), (0, 3)):
        got, want = _window_case(target, 6, 2, 64, 48, 702, (700, 702), size,
                                 standout, size, True)
        _close(got, want, target, (size, standout))


# ----------------------------------------------------------------- retention
def _retention_ref(q, k, v, gate, decay, base, rot, eps, state=None, start=0):
    """Oracle's normed and gated outputs and last state of rows that begin at
    position `start`."""
    T = q.shape[0]
    pos = torch.arange(start, start + T)
    D = q.shape[2]
    qq = zo.rotate(q.to(F64), pos, base, rot)
    kk = zo.rotate(k.to(F64), pos, base, rot) * D ** -0.5
    o, S = zo.retention_core(qq, kk, v.to(F64), decay, state)
    o = zo.rms_unit(o, eps).reshape(T, -1)
    return o * zo.silu(gate.to(F64)), S


class _Seq:
    """One sequence's random projections, rows as they leave a wide GEMM."""

    def __init__(self, g, T, H, D, Dv, dt):
        self.q, self.k = _rnd(g, T, H, D, dtype=dt), _rnd(g, T, H, D, dtype=dt)
        self.v = _rnd(g, T, H, Dv, dtype=dt)
        self.gate = _rnd(g, T, H * Dv, dtype=dt)

    def rows(self, a, b):
        n = b - a
        return torch.cat([self.q[a:b].reshape(n, -1), self.k[a:b].reshape(n, -1),
                          self.v[a:b].reshape(n, -1), self.gate[a:b]], 1)


def _run(target, rows, pos, H, D, Dv, rot, base, decay, state, slots, cu, ctx,
         eps):
    dev, dt = target
    f = banded_rope_frequencies(dict(base=base, dims=rot)) if rot \
        else torch.zeros(0, dtype=F64)
    p = rows.to(dev)
    a, b = H * D, H * Dv
    big, out = _inside(p.shape[0], b, dt, dev, 8, 4)
    hops.retention(p[:, :a], p[:, a:2 * a], p[:, 2 * a:2 * a + b],
                   p[:, 2 * a + b:], hops.rope_table(pos.to(dev), f.to(dev)),
                   D ** -0.5, torch.tensor(decay, device=dev), state,
                   _i32(slots, dev), None if cu is None else _i32(cu, dev),
                   _i32(ctx, dev), eps, out)
    assert torch.isnan(big[:, :8]).all() and torch.isnan(big[:, 8 + b:]).all()
    return out


RSHAPES = [(2, 6, 5, 4), (3, 32, 32, 32), (2, 64, 40, 48), (2, 128, 128, 128),
           (1, 96, 200, 64), (2, 256, 64, 8), (1, 7, 130, 2), (4, 16, 8, 0)]


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("H,D,Dv,rot", RSHAPES)
def test_retention_through_portions_and_decoding(target, H, D, Dv, rot):
    """Portions around the chunk size and down to two tokens, then decoded
    rows, from a slot that held another sequence's state."""
    dev, dt = target
    g = torch.Generator().manual_seed(D + Dv)
    base, eps = 50.0, 1e-3
    decay = [1.0 - 0.6 ** (2 * h + 1) for h in range(H)]
    cuts = [63, 2, 64, 65, 3, 130, 1, 1, 2, 1]
    n = sum(cuts)
    s = _Seq(g, n, H, D, Dv, dt)
    want, last = _retention_ref(s.q, s.k, s.v, s.gate, decay, base, rot, eps)
    state = torch.randn(3, H, D, Dv, generator=g).to(dev)
    other = state[[0, 2]].clone()
    at = 0
    for c in cuts:
        pos = torch.arange(at, at + c)
        got = _run(target, s.rows(at, at + c), pos, H, D, Dv, rot, base, decay,
                   state, [1], None if c == 1 else [0, c], [at], eps)
        _close(got, want[at:at + c], target, (at, c), 2.0)
        at += c
    _close(state[1], last, EXACT, "state", 3.0)
    assert torch.equal(state[[0, 2]], other)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("H,D,Dv,rot", [(2, 32, 32, 16), (3, 20, 12, 20),
                                        (1, 64, 136, 64)])
def test_retention_of_unequal_batches(target, H, D, Dv, rot):
    """Prompt portions of very different lengths in one call (fresh ones,
    continued ones, one without a slot), then decoded rows of some of them
    beside a row without a slot."""
    dev, dt = target
    g = torch.Generator().manual_seed(H)
    base, eps = 1e4, 1e-5
    decay = [0.97, 1.0, 0.2][:H]
    lens = [1, 200, 64, 2, 129]
    first = [0, 70, 0, 0, 1]                   # tokens that came earlier
    slot = [4, 0, -1, 2, 3]
    seqs = [_Seq(g, a + b + 1, H, D, Dv, dt) for a, b in zip(lens, first)]
    state = torch.randn(6, H, D, Dv, generator=g).to(dev)
    want, kept = [], []
    for i, (s, a, b) in enumerate(zip(seqs, lens, first)):
        if b:
            st = _retention_ref(s.q[:b], s.k[:b], s.v[:b], s.gate[:b], decay,
                                base, rot, eps)[1]
            state[slot[i]] = st.float().to(dev)
            st = state[slot[i]].cpu().to(F64)
        else:
            st = None
        y, S = _retention_ref(s.q[b:], s.k[b:], s.v[b:], s.gate[b:], decay,
                              base, rot, eps, st, b)
        want.append(y)
        kept.append(S)
    rows = torch.cat([s.rows(b, b + a) for s, a, b in zip(seqs, lens, first)])
    pos = torch.cat([torch.arange(b, b + a) for a, b in zip(lens, first)])
    cu = [0]
    for a in lens:
        cu.append(cu[-1] + a)
    got = _run(target, rows, pos, H, D, Dv, rot, base, decay, state, slot, cu,
               first, eps)
    for i, a in enumerate(lens):
        _close(got[cu[i]:cu[i + 1]], want[i][:a], target, ("portion", i), 2.0)
    # one more token each; the sequence without a slot starts from zero
    order = [3, 2, 1, 0]
    rows = torch.cat([seqs[i].rows(first[i] + lens[i], first[i] + lens[i] + 1)
                      for i in order])
    pos = torch.tensor([first[i] + lens[i] for i in order])
    got = _run(target, rows, pos, H, D, Dv, rot, base, decay, state,
               [slot[i] for i in order], None, pos.tolist(), eps)
    for j, i in enumerate(order):
        if slot[i] >= 0:
            _close(got[j], want[i][-1], target, ("decoded", i), 2.0)
            _close(state[slot[i]], kept[i], EXACT, ("state", i), 3.0)
    s, t = seqs[2], lens[2]
    y, _ = _retention_ref(s.q[t:], s.k[t:], s.v[t:], s.gate[t:], decay, base,
                          rot, eps, None, t)
    _close(got[1], y[0], target, "no slot", 2.0)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("back", [63, 64, 65, 700])
def test_a_slow_head_remembers_a_far_key(target, back):
    """One key answers the last query; everything between is orthogonal to
    it. The head with decay 0.999 recalls its value, the fast one does not."""
    dev, dt = target
    H, D, Dv, T = 2, 16, 8, back + 1
    g = torch.Generator().manual_seed(back)
    s = _Seq(g, T, H, D, Dv, dt)
    s.k[..., 0] = 0.0
    s.q.zero_()
    s.q[..., 0] = 4.0
    s.k[0] = 0.0
    s.k[0, :, 0] = 2.0
    decay = [0.999, 0.5]
    want, last = _retention_ref(s.q, s.k, s.v, s.gate, decay, 1e4, 0, 1e-8)
    state = torch.zeros(1, H, D, Dv, device=dev)
    cuts = [T] if back < 100 else [back - 66, 64, 3]
    assert sum(cuts) == T
    at = 0
    for c in cuts:
        got = _run(target, s.rows(at, at + c), torch.arange(at, at + c), H, D,
                   Dv, 0, 1e4, decay, state, [0], [0, c], [at], 1e-8)
        at += c
    slow = zo.rms_unit(s.v[0, 0].to(F64), 1e-8) * zo.silu(
        s.gate[-1, :Dv].to(F64))
    _close(got[-1, :Dv], slow, target, "recalled", 50 if dt == torch.float32
           else 1.0)
    _close(got[-1], want[-1], target, "both", 2.0)
    _close(state[0], last, EXACT, "state", 3.0)


@pytest.mark.parametrize("target", TARGETS)
def test_long_portion_in_one_call(target):
    """Many chunks (the scan's unrolled part and its rest)."""
    dev, dt = target
    H, D, Dv, rot, T = 2, 24, 16, 24, 64 * 19 + 7
    g = torch.Generator().manual_seed(1)
    s = _Seq(g, T, H, D, Dv, dt)
    decay = [0.995, 0.9]
    want, last = _retention_ref(s.q, s.k, s.v, s.gate, decay, 1e5, rot, 1e-5)
    state = torch.zeros(1, H, D, Dv, device=dev)
    got = _run(target, s.rows(0, T), torch.arange(T), H, D, Dv, rot, 1e5,
               decay, state, [0], [0, T], [0], 1e-5)
    _close(got, want, target, "", 3.0)
    _close(state[0], last, EXACT, "state", 3.0)


# ------------------------------------------------------------------- experts
ROUTES = [dict(experts=6, top=2, scale=1.25, groups=dict(count=3, keep=2)),
          dict(experts=6, top=3, scale=0.5, groups=dict(count=2, keep=1)),
          dict(experts=4, top=1, scale=1.0, groups=dict(count=4, keep=2)),
          dict(experts=5, top=5, scale=2.0),
          dict(experts=1, top=1, scale=3.0, groups=dict(count=1, keep=1))]


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("r", ROUTES)
def test_route_with_groups_and_scale(target, r):
    dev, _ = target
    g = torch.Generator().manual_seed(r["experts"])
    T, W = 40, 16
    h, w = _rnd(g, T, W), _rnd(g, r["experts"], W, std=0.5)
    gr = r.get("groups") or dict(count=1, keep=1)
    ids, wts = hops.moe_route(h.to(dev), w.to(dev), r["top"], gr["count"],
                              gr["keep"], scale=r["scale"])
    z = h.to(F64) @ w.to(F64).T
    for t in range(T):
        want = zo.route(z[t], r)
        assert ids[t].tolist() == [e for e, _ in want], t
        _close(wts[t], torch.tensor([a for _, a in want]), EXACT)


def test_group_of_two_good_experts_beats_one_with_the_best():
    """The best single expert sits in a group whose second is poor."""
    z = torch.tensor([[3.0, -5.0, 1.5, 1.2, -1.0, -1.0]])
    ids, wts = hops.moe_route(z, torch.eye(6), 2, 3, 1, scale=2.0)
    assert ids.tolist() == [[2, 3]]
    _close(wts[0], 2.0 * torch.sigmoid(torch.tensor([1.5, 1.2])), EXACT)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("T", [9, 300])
@pytest.mark.parametrize("r", ROUTES)
def test_experts_in_every_execution_shape(target, T, r):
    """Dense batched, padded batched, expert by expert: the dispatched rows
    and weights summed by the residual update."""
    dev, dt = target
    g = torch.Generator().manual_seed(T + r["experts"])
    W, ff = 24, 16
    w = {"router": _rnd(g, r["experts"], W, std=0.5)}
    gr = r.get("groups") or dict(count=1, keep=1)
    m = RoutedExperts(W, ff, r["experts"], r["top"], gr["count"], gr["keep"],
                      dt, scale=r["scale"])
    with torch.no_grad():
        m.router.copy_(w["router"])
    for e in range(r["experts"]):
        for n, shape in (("gate", (ff, W)), ("up", (ff, W)),
                         ("down", (W, ff))):
            w[f"e{e}.{n}"] = _rnd(g, *shape, std=0.4)
        m.load_expert(e, w[f"e{e}.up"], w[f"e{e}.down"], w[f"e{e}.gate"])
    m = m.to(dev)
    one = torch.ones(W, device=dev)
    for skew in (False, True):
        h = torch.randn(T, W, generator=g)
        if skew:
            h[: 2 * T // 3] = h[0] + 0.01 * h[: 2 * T // 3]
        h = h.bfloat16().to(dt)
        want = zo.ff_moe(h.to(F64), {k: v.to(F64) for k, v in w.items()}, "",
                         dict(router=r))
        for limit in (64, 0 if T <= 64 else 10 ** 6):
            m.dense_max_tokens = limit
            x = torch.zeros(T, W, device=dev)
            with torch.no_grad():
                hops.join_norm_(x, torch.zeros(T, W, dtype=dt, device=dev),
                                m.dispatch(h.to(dev)), one, 1e-5)
                again = m(h.to(dev))
            for y in (x, again):
                bad = zo.rel_err(y.cpu(), want) > \
                    (1e-4 if dt == torch.float32 else 0.1)
                assert int(bad.sum()) <= T // 40, (skew, limit, int(bad.sum()))
