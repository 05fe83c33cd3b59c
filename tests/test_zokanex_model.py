"""The Zokanex decoder through the engine against the plain oracle
(tests/zokanex_oracle.py). Every test makes its own small configuration and
random checkpoint, writes it as a model folder, and loads it with
LLMEngine(folder): config reader, safetensors loader, cache manager, batching
and kernels are all the product's. CPU path always; the HIP path (fp32 and
bf16, decode through captured graphs) under the gpu marker."""
import functools

import pytest
import torch

import zokanex_oracle as zo
from xllm_service_amd.engine.engine import LLMEngine
from xllm_service_amd.engine.sampling import SamplingParams
from zokanex_oracle import attention, dense, make_config, make_weights, moe, \
    rel_err, retention, write_model_dir

TARGETS = [("cpu", torch.float32),
           pytest.param(("cuda", torch.float32), marks=pytest.mark.gpu),
           pytest.param(("cuda", torch.bfloat16), marks=pytest.mark.gpu)]


def _variants():
    return {
        # both mixers, own and borrowed keys (not only the neighbour's, also
        # through another window), dense and routed feed-forwards
        "mixed": make_config(layers=[
            retention(mlp=moe()), attention(size=7), attention(
                size=12, kv_from=1, mlp=moe(experts=4, top=1, count=2, keep=1)),
            retention(heads=3, dim=8, vdim=9, dims=8, mlp=None),
            attention(heads=3, kv_heads=3, dims=8, size=5, mlp=moe(shared=0)),
            attention(size=3, kv_from=1, mlp=None)]),
        # nothing optional: no windows, no turn, no feed-forward, no scale of
        # the embedding; odd widths, one key head for all
        "plain": make_config(width=20, scale=1.0, layers=[
            attention(heads=3, kv_heads=1, dim=7, vdim=3, dims=2, size=0,
                      mlp=None),
            retention(heads=5, dim=3, vdim=7, dims=0, mlp=None),
            attention(heads=6, kv_heads=2, dim=5, vdim=11, dims=0, size=0,
                      mlp=dense(5)),
            retention(heads=1, dim=10, vdim=1, dims=2,
                      mlp=moe(experts=3, top=2, count=1, keep=1, scale=1.0,
                              shared=3))]),
        # everything that can be 1
        "ones": make_config(width=16, scale=1.0, layers=[
            attention(heads=1, kv_heads=1, dim=2, vdim=1, dims=2, size=1,
                      scale=1.0, mlp=moe(ff=1, experts=1, top=1, count=1,
                                         keep=1, scale=1.0, shared=1)),
            retention(heads=1, dim=1, vdim=1, dims=0, decay=[1.0],
                      mlp=dense(1)),
            attention(heads=1, kv_heads=1, dim=2, vdim=1, dims=2, size=1,
                      kv_from=0, mlp=moe(ff=3, experts=3, top=3, count=3,
                                         keep=3))]),
        # windows at a page's size and around it, borrowed through others
        "edges": make_config(width=32, scale=0.3, layers=[
            attention(heads=4, dim=8, vdim=8, dims=8, size=16),
            attention(heads=4, dim=8, vdim=8, dims=8, size=17, kv_from=0),
            retention(decay=[0.999, 0.5], mlp=moe(ff=8, top=3)),
            attention(heads=2, dim=8, vdim=8, dims=8, size=15, kv_from=0,
                      base=100.0, mlp=moe(scale=2.0)),
            attention(size=33, base=1e4)]),
        # head widths of the matrix-core attention classes and of the wide
        # retention kernels, rows wider than one tile batch
        "large": make_config(width=128, vocab=200, eps=2e-6, layers=[
            attention(heads=4, kv_heads=2, dim=64, vdim=40, dims=48, size=33,
                      base=1e4, mlp=moe(ff=48, experts=12, top=3, count=4,
                                        keep=2, shared=56)),
            retention(heads=3, dim=72, vdim=56, dims=40, base=1e4,
                      mlp=dense(192)),
            attention(heads=2, kv_heads=2, dim=128, vdim=72, dims=128, size=70,
                      base=1e5, mlp=None),
            attention(heads=8, kv_heads=2, dim=64, vdim=40, dims=48, size=90,
                      base=1e4, kv_from=0, mlp=dense(96)),
            retention(heads=2, dim=48, vdim=160, dims=16, base=1e3,
                      decay=[0.98, 0.9995],
                      mlp=moe(ff=32, experts=5, top=2, count=1, keep=1))]),
    }


@functools.lru_cache(maxsize=None)
def _model(name, tmp_root):
    cfg = _variants()[name]
    w = make_weights(cfg, seed=sum(map(ord, name)))
    folder = write_model_dir(f"{tmp_root}/{name}", cfg, w)
    return cfg, w, folder


@pytest.fixture(scope="module")
def root(tmp_path_factory):
    return str(tmp_path_factory.mktemp("zokanex_models"))


def _tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


@functools.lru_cache(maxsize=None)
def _oracle(name, tmp_root, n, seed):
    cfg, w, _ = _model(name, tmp_root)
    out, _, margin = zo.forward(cfg, w, _tokens(cfg, n, seed))
    return out, margin


def _engine(folder, target, blocks=64, slots=4, **kw):
    dev, dt = target
    return LLMEngine(folder, device=dev, dtype=dt, max_num_seqs=slots,
                     max_kv_blocks=blocks, max_model_len=blocks * 16,
                     enable_graphs=dev == "cuda", swap_space_mb=0, **kw)


def _check(got, want, target, what=""):
    """fp32: every row close, but for a rare row where two experts' choice
    scores nearly tie. bf16: rounding-sized error; rows whose choice hangs on
    less than bf16 rounding of the router's input (want = (logits, choice
    margins)) may differ."""
    clear = slice(None)
    if isinstance(want, tuple):
        want, margin = want
        clear = margin > (1e-5 if target[1] == torch.float32 else 0.01)
    e = rel_err(got, want)[clear]
    if target[1] == torch.float32:
        assert float(e.median()) < 1e-4, (what, float(e.median()))
        assert int((e > 5e-4).sum()) <= len(e) // 40, (what, e)
    else:
        assert float(e.median()) < 0.06, (what, float(e.median()))
        assert float((e > 0.15).float().mean()) <= 0.1, (what, e)


def _run_portions(eng, rid, toks, cuts, end=True):
    """Feed toks in portions of the given sizes; logits at every position."""
    out, at = [], 0
    for n in cuts:
        last = at + n == len(toks)
        out.append(eng.score_step([(rid, toks[at:at + n], list(range(n)))],
                                  finished=[rid] if (last and end) else []))
        at += n
    assert at == len(toks)
    return torch.cat(out)


NAMES = ["mixed", "plain", "ones", "edges", "large"]


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompt(root, target, name):
    cfg, w, folder = _model(name, root)
    eng = _engine(folder, target)
    for n, seed in ((1, 1), (2, 2), (67, 3)):   # first tokens, past a page
        toks = _tokens(cfg, n, seed)
        got = _run_portions(eng, f"w{n}", toks, [n])
        _check(got, _oracle(name, root, n, seed), target, (name, n))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", NAMES)
def test_residual_after_every_layer(root, target, name):
    """Hook the residual after every layer of one prompt."""
    cfg, w, folder = _model(name, root)
    eng = _engine(folder, target)
    toks = _tokens(cfg, 21, 5)
    seen = []
    hooks = [b.register_forward_hook(lambda m, i, o: seen.append(
        i[0].detach().float().cpu().clone())) for b in eng.model.blocks]
    eng.score_step([("a", toks, [0])], finished=["a"])
    for h in hooks:
        h.remove()
    trail = zo.forward(cfg, w, toks)[1]
    assert len(seen) == len(trail) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(seen, trail)):
        err = (a.double() - b).norm(dim=-1) / b.norm(dim=-1).mean()
        if target[1] == torch.float32:
            assert float(err.max()) < 2e-4, (name, i, float(err.max()))
        else:
            assert float(err.median()) < 0.04, (name, i, float(err.median()))
            assert float((err > 0.15).float().mean()) <= 0.1, (name, i, err)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", NAMES)
def test_prefill_then_token_by_token(root, target, name):
    cfg, w, folder = _model(name, root)
    eng = _engine(folder, target)
    n = 40
    toks = _tokens(cfg, n, 7)
    want = _oracle(name, root, n, 7)
    for first in (1, 2, 15, 16, 17):
        got = _run_portions(eng, f"d{first}", toks, [first] + [1] * (n - first))
        _check(got, want, target, (name, first))


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["mixed", "edges", "large"])
def test_portions_of_many_sizes(root, target, name):
    cfg, w, folder = _model(name, root)
    eng = _engine(folder, target)
    n = 150
    toks = _tokens(cfg, n, 8)
    want = _oracle(name, root, n, 8)
    for cuts in ([2] * 10 + [16, 15, 17, 2, 64, 3, 1, 1, 11],
                 [63, 2, 64, 1, 2, 2, 16],
                 [65, 31, 33, 1, 1, 17, 2]):
        assert sum(cuts) == n
        got = _run_portions(eng, "p", toks, cuts)
        _check(got, want, target, cuts)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["edges", "large"])
def test_long_prompt_and_long_decoding(root, target, name):
    """A prompt of many pages, then decoding across several more: windows
    slide and chunks begin and end over decoded tokens, states run on."""
    cfg, w, folder = _model(name, root)
    eng = _engine(folder, target)
    n = 330
    toks = _tokens(cfg, n, 9)
    got = _run_portions(eng, "l", toks, [200] + [1] * (n - 200))
    _check(got, _oracle(name, root, n, 9), target)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("borrowed", [False, True])
def test_what_a_layer_cannot_see_changes_nothing(tmp_path, target, borrowed):
    """One attention layer that adds to the residual: another token just
    outside the window of a late position leaves its logits as they are to
    the last bit, one just inside changes them; through a prompt cut inside
    the window and through decoded tokens. borrowed: the keys belong to an
    earlier layer with a narrower window that adds nothing itself."""
    size, n = 24, 60
    layers = [attention(size=size, mlp=None)]
    if borrowed:
        layers = [attention(size=5, mlp=None),
                  attention(size=size, kv_from=0, mlp=None)]
    edge = n - size
    cfg = make_config(width=16, layers=layers)
    w = make_weights(cfg, seed=3)
    if borrowed:
        w["l0.mix.o"] *= 0.0
    eng = _engine(write_model_dir(str(tmp_path), cfg, w), target)
    base = _tokens(cfg, n, 4)

    def last_row(toks, cuts, rid):
        return _run_portions(eng, rid, toks, cuts)[-1]
    for j, cuts in enumerate(([n], [edge + 3, n - edge - 3],
                              [7] + [1] * (n - 7))):
        ref = last_row(base, cuts, f"r{j}")
        for at, seen in ((edge - 1, False), (edge, True)):
            toks = list(base)
            toks[at] = (toks[at] + 7) % cfg["vocab"]
            diff = float((last_row(toks, cuts, f"c{j}{at}") - ref).abs().max())
            assert (diff > 1e-3) if seen else diff == 0.0, (cuts, at, diff)
    _check(ref[None], zo.forward(cfg, w, base)[0][-1:], target)


@pytest.mark.parametrize("target", TARGETS)
def test_an_early_token_reaches_far_through_the_states(tmp_path, target):
    """A retention layer that hardly decays: the first token still shows 200
    positions later, in a slot used before."""
    cfg = make_config(width=16, layers=[retention(decay=[0.9999, 0.9995],
                                                  mlp=None)])
    w = make_weights(cfg, seed=5)
    eng = _engine(write_model_dir(str(tmp_path), cfg, w), target, slots=1)
    rows = []
    for first in (1, 2):
        toks = [first] + _tokens(cfg, 199, 4)
        got = _run_portions(eng, f"k{first}", toks, [130, 2] + [1] * 68)
        _check(got, zo.forward(cfg, w, toks)[0], target)
        rows.append(got[-1])
    assert float((rows[0] - rows[1]).abs().max()) > 1e-3


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["mixed", "edges", "large"])
def test_unequal_batch_with_reused_pages(root, target, name):
    """A pool far smaller than the sum of all requests: requests come and go
    in mixed batches (prompt portions beside single tokens), later ones land
    on freed pages and slots that still hold the earlier ones' keys and
    states. Every request must match its own run alone."""
    cfg, w, folder = _model(name, root)
    lens = dict(a=70, b=3, c=33, d=50, e=18, f=41)
    toks = {k: _tokens(cfg, n, 20 + i) for i, (k, n) in enumerate(lens.items())}
    want = {k: _oracle(name, root, n, 20 + i)
            for i, (k, n) in enumerate(lens.items())}
    eng = _engine(folder, target, blocks=10, slots=3)   # 160 tokens of pages
    plan = [
        [("a", 30), ("b", 2)],
        [("a", 1), ("b", 1), ("c", 17)],
        [("a", 16), ("c", 16)],                 # b done: its page is free
        [("a", 1), ("d", 2)],                   # d on b's page
        [("a", 22), ("d", 1)],                  # a done (70)
        [("d", 31), ("e", 18)],                 # c done earlier; e on a's pages
        [("d", 1), ("f", 5)],
        [("d", 15), ("f", 1)],
        [("f", 35)],
    ]
    at = {k: 0 for k in lens}
    got = {k: [] for k in lens}
    for step in plan:
        entries, done = [], []
        for k, n in step:
            entries.append((k, toks[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == lens[k]:
                done.append(k)
        out = eng.score_step(entries, finished=done)
        o = 0
        for k, n in step:
            got[k].append(out[o:o + n])
            o += n
    assert at == lens
    assert eng.block_manager.num_free == 10
    for k in lens:
        _check(torch.cat(got[k]), want[k], target, k)


@pytest.mark.parametrize("target", TARGETS)
@pytest.mark.parametrize("name", ["mixed", "large"])
def test_greedy_generation_through_scheduler(root, target, name):
    """generate(): continuous batching with chunked prompts (a 16-token step
    budget), three unequal prompts on two batch rows, greedy sampling. The
    oracle continues each prompt alone; a step whose two best oracle logits
    are closer than the dtype's noise ends the comparison."""
    cfg, w, folder = _model(name, root)
    dev, dt = target
    eng = LLMEngine(folder, device=dev, dtype=dt, max_num_seqs=2,
                    max_kv_blocks=32, max_model_len=256,
                    max_batched_tokens=16, enable_graphs=dev == "cuda",
                    swap_space_mb=0)
    prompts = [_tokens(cfg, n, 40 + n) for n in (37, 5, 20)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=6, ignore_eos=True))
    margin = 1e-3 if dt == torch.float32 else 0.15
    for p, out in zip(prompts, outs):
        assert len(out) == 6
        seq = list(p)
        for tok in out:
            top = zo.forward(cfg, w, seq)[0][-1].topk(2)
            if float(top.values[0] - top.values[1]) < margin:
                break
            assert tok == int(top.indices[0])
            seq.append(tok)
    assert eng.block_manager.num_free == 32


def test_preset_generates_through_the_engine():
    """The named preset (random weights)."""
    eng = LLMEngine("zokanex-tiny", device="cpu", max_num_seqs=2,
                    max_kv_blocks=16, max_model_len=128, swap_space_mb=0)
    assert len(eng.model.blocks) == 4 and len(eng.runner.kv_caches) == 4
    a = eng.generate([[1, 2, 3, 4, 5, 6, 7], [9, 8]],
                     SamplingParams(max_tokens=4, ignore_eos=True))
    b = eng.generate([[9, 8]], SamplingParams(max_tokens=4, ignore_eos=True))
    assert [len(x) for x in a] == [4, 4] and a[1] == b[0]


def test_trace_replay_command(root, tmp_path):
    """bin/trace_run on a model folder: steps on stdin, logits in files, a
    pool of 128 tokens used by three requests in turn."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np
    cfg, w, folder = _model("mixed", root)
    toks = {k: _tokens(cfg, n, 60 + n) for k, n in (("a", 40), ("b", 9),
                                                     ("c", 30))}
    steps = [
        dict(step=0, entries=[dict(id="a", tokens=toks["a"][:33], want=[0, 32]),
                              dict(id="b", tokens=toks["b"][:8], want=[])],
             end=[]),
        dict(step=1, entries=[dict(id="a", tokens=toks["a"][33:34], want=[0]),
                              dict(id="b", tokens=toks["b"][8:], want=[0])],
             end=["b"]),
        dict(step=2, entries=[dict(id="c", tokens=toks["c"][:2], want=[1])],
             end=[]),
        dict(step=3, entries=[dict(id="a", tokens=toks["a"][34:], want=[5]),
                              dict(id="c", tokens=toks["c"][2:], want=[27])],
             end=["a", "c"]),
    ]
    exe = os.path.join(os.path.dirname(os.path.dirname(
        os.path.abspath(__file__))), "bin", "trace_run")
    out = tmp_path / "out"
    p = subprocess.run(
        [sys.executable, exe, "--model", folder, "--dtype", "float32", "--out",
         str(out), "--max-tokens", "128", "--slots", "2", "--device", "cpu"],
        input="".join(json.dumps(x) + "\n" for x in steps), text=True,
        capture_output=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.split("\n") if l.startswith("done")] == [
        f"done {i}" for i in range(4)]
    full = {k: zo.forward(cfg, w, t)[0] for k, t in toks.items()}
    want = {0: [full["a"][0], full["a"][32]], 1: [full["a"][33], full["b"][8]],
            2: [full["c"][1]], 3: [full["a"][39], full["c"][29]]}
    for i, rows in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4")
                               .reshape(len(rows), -1).copy())
        _check(got, torch.stack(rows), ("cpu", torch.float32), i)


def test_config_is_checked(tmp_path):
    bad = make_config()
    bad["layers"][0]["type"] = "something"
    with pytest.raises(ValueError):
        LLMEngine(write_model_dir(str(tmp_path / "t"), bad, {}), device="cpu")
    bad = make_config()
    bad["layers"][0]["mlp"]["kind"] = "other"
    with pytest.raises(ValueError):
        LLMEngine(write_model_dir(str(tmp_path / "k"), bad, {}), device="cpu")
    for j, layers in enumerate((
            [attention(kv_from=0)],                          # itself
            [retention(), attention(kv_from=0)],             # no keys there
            [attention(), attention(kv_from=0), attention(kv_from=1)],
            [attention(), attention(kv_from=0, dim=10)])):
        with pytest.raises(ValueError):
            LLMEngine(write_model_dir(str(tmp_path / f"b{j}"),
                                      make_config(layers=layers), {}),
                      device="cpu")
    bad = make_config(layers=[retention(heads=3, decay=[0.5, 0.6])])
    with pytest.raises(ValueError):
        LLMEngine(write_model_dir(str(tmp_path / "n"), bad, {}), device="cpu")
    ok = make_config()
    w = make_weights(ok)
    del w["l0.mix.k.norm"]
    with pytest.raises(KeyError):
        LLMEngine(write_model_dir(str(tmp_path / "m"), ok, w), device="cpu")
    w = make_weights(ok)
    w["l0.mix.v"] = torch.zeros(3, ok["width"])
    with pytest.raises((ValueError, RuntimeError)):
        LLMEngine(write_model_dir(str(tmp_path / "u"), ok, w), device="cpu")
    w = make_weights(ok)
    w["l1.mlp.e0.up"] = torch.zeros(3, 3)
    with pytest.raises((ValueError, RuntimeError)):
        LLMEngine(write_model_dir(str(tmp_path / "e"), ok, w), device="cpu")
    w = make_weights(ok)
    w["l9.norm1"] = torch.ones(1)
    with pytest.raises(ValueError):
        LLMEngine(write_model_dir(str(tmp_path / "x"), ok, w), device="cpu")


def test_a_stack_without_pages(tmp_path):
    """Retention layers only: nothing is kept per token, the default block
    pool stays finite and generation runs."""
    cfg = make_config(layers=[retention(), retention(mlp=moe())])
    folder = write_model_dir(str(tmp_path), cfg, make_weights(cfg))
    eng = LLMEngine(folder, device="cpu", max_num_seqs=2, max_model_len=64,
                    swap_space_mb=0)
    out = eng.generate([[1, 2, 3]], SamplingParams(max_tokens=3,
                                                   ignore_eos=True))
    assert len(out[0]) == 3
