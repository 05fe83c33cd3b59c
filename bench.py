#!/usr/bin/env python3
"""Flagship benchmark — the driver contract (see repo instructions).

Default mode measures the BASELINE.json headline the honest way: SLO-goodput
(output tok/s from requests whose TTFT meets the 1 s SLO) through the FULL
serving stack — HTTP (uvicorn, real TCP) -> master scheduler -> msgrpc ->
per-GPU worker processes -> SSE streaming back — under open-loop Poisson
arrivals whose rate is auto-calibrated to ~0.9x the measured capacity.

Topology scales with --gpus N (one worker process per GPU):
  N=1            one DEFAULT (colocated prefill+decode) worker
  N>=2           PD-disaggregated: max(1, N//4) PREFILL + rest DECODE
                 (8 GPUs -> 2P+6D), KV blocks migrating
                 prefill->decode over xGMI (hipIpc + peer copies)

A "step" is one COMPLETED request in steady state: after --warmup completed
requests under the Poisson load, the timed region spans exactly --steps
further completions (barrier + torch.cuda.synchronize on both sides, MAX
elapsed over ranks). value = sum of output tokens of SLO-passing requests
completed in the window / elapsed — the whole-job aggregate.

  python bench.py --gpus 1 --steps 20 --warmup 5
  python -m torch.distributed.run --nnodes=1 --nproc-per-node 8 \
      --master-addr 127.0.0.1 bench.py --gpus 8 --steps 120 --warmup 10

--mode engine keeps the round-1 closed-loop engine-step microbench (kernel
iteration tool; its metric string says so).
"""
from __future__ import annotations

import argparse
import asyncio
import json
import os
import random
import socket
import subprocess
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))

# hipBLASLt/rocBLAS algo selection tuned offline on MI355X (TunableOp);
# must be configured before the first torch import in the process.
_TUNABLE = os.path.join(ROOT, "configs", "tunableop_gfx950.csv")
if os.path.exists(_TUNABLE):
    os.environ.setdefault("PYTORCH_TUNABLEOP_ENABLED", "1")
    os.environ.setdefault("PYTORCH_TUNABLEOP_TUNING", "0")
    os.environ.setdefault("PYTORCH_TUNABLEOP_FILENAME", _TUNABLE)

if os.environ.get("BENCH_LOADGEN") != "1":
    import torch


def parse_args():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=20,
                    help="serving: timed completed requests; "
                         "engine: timed engine steps")
    ap.add_argument("--warmup", type=int, default=5)
    ap.add_argument("--mode", choices=("serving", "engine", "hybrid"),
                    default="serving",
                    help="hybrid: prefill/decode throughput and per-kernel "
                         "rates of the pugovik stacks beside equal-size "
                         "llama stacks (one GPU; prints one JSON line per "
                         "measurement, not the headline record)")
    ap.add_argument("--hybrid-sizes", default="2k,4k")
    ap.add_argument("--hybrid-family", default="pugovik",
                    choices=("pugovik", "dunusun", "tosipel", "gararax",
                             "nikedra", "zokanex"),
                    help="which hybrid stack --mode hybrid measures beside "
                         "the equal-size llama stack")
    ap.add_argument("--model", default="llama-3-8b")
    ap.add_argument("--concurrency", type=int, default=128,
                    help="ramp/calibration concurrency per decode GPU "
                         "(batch sweep on MI355X: 64->9.7k, 96->11.2k, "
                         "128->13.9k, 192->13.8k tok/s engine-step)")
    ap.add_argument("--input-len", type=int, default=1024)
    ap.add_argument("--output-len", type=int, default=1024)
    ap.add_argument("--max-batched-tokens", type=int, default=8192,
                    help="worker chunked-prefill budget per step")
    ap.add_argument("--device", default=None)
    ap.add_argument("--policy", default="CAR")
    ap.add_argument("--slo-ttft-ms", type=float, default=1000.0)
    ap.add_argument("--pace", type=float, default=0.95,
                    help="Poisson arrival rate as a fraction of the "
                         "ramp-measured capacity")
    ap.add_argument("--arrival-rate", type=float, default=0.0,
                    help="req/s override (0 = auto-calibrate)")
    ap.add_argument("--ramp-s", type=float, default=0.0,
                    help="capacity-calibration window (0 = auto)")
    ap.add_argument("--push-interval-ms", type=float, default=0.0,
                    help="worker->master token push coalescing window "
                         "(0 = auto: scales with decode GPU count so the "
                         "master's SSE fan-out stays off the hot path)")
    ap.add_argument("--max-kv-blocks", type=int, default=0)
    ap.add_argument("--startup-timeout", type=float, default=900.0)
    return ap.parse_args()


# --------------------------------------------------------------------------
# hybrid mode: pugovik-<size> beside llama-<size>, end to end and per kernel
# --------------------------------------------------------------------------
def _time_gpu(fn, iters=10, warm=3):
    for _ in range(warm):
        fn()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(
        enable_timing=True)
    a.record()
    for _ in range(iters):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / iters * 1e-3


def _hybrid_end_to_end(name, device, prompt_len, batch, ctx, steps):
    """(prefill tok/s for one prompt_len prompt, decode tok/s at `batch`
    sequences of ~ctx tokens through the captured decode graph)."""
    from xllm_service_amd.engine.engine import LLMEngine
    from xllm_service_amd.engine.sampling import SamplingParams
    from xllm_service_amd.models.config import get_config
    cfg = get_config(name)
    blocks = (batch * (ctx + steps + 64) + prompt_len) // 16 + 64
    eng = LLMEngine(name, device=device, max_num_seqs=batch,
                    max_batched_tokens=max(prompt_len, 8192),
                    max_kv_blocks=blocks, max_model_len=max(prompt_len, ctx)
                    + steps + 128, state_slots=batch + 1, seed=0,
                    enable_prefix_caching=False, swap_space_mb=0)
    g = torch.Generator().manual_seed(0)
    mk = lambda n: torch.randint(0, cfg.vocab_size, (n,), generator=g).tolist()
    one = SamplingParams(max_tokens=1, ignore_eos=True)
    eng.generate([mk(prompt_len)], one)                       # warm
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    reps = 3
    for _ in range(reps):
        eng.generate([mk(prompt_len)], one)
    torch.cuda.synchronize()
    prefill = reps * prompt_len / (time.perf_counter() - t0)
    for i in range(batch):
        eng.add_request(f"d{i}", mk(ctx), SamplingParams(
            max_tokens=steps + 16, ignore_eos=True))
    while any(not s.prefill_done for s in eng.seqs.values()):
        eng.step()
    for _ in range(8):
        eng.step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    n = 0
    for _ in range(steps):
        n += sum(len(o.new_token_ids) for o in eng.step())
    torch.cuda.synchronize()
    decode = n / (time.perf_counter() - t0)
    del eng
    torch.cuda.empty_cache()
    return prefill, decode


def _hybrid_kernels(size, device, T, batch, ctx):
    """Achieved rates of the mixer kernels at one layer's shapes: bytes that
    must move (GB/s) for the decode kernels, useful FLOP/s for prefill."""
    from xllm_service_amd import ops
    from xllm_service_amd.models.config import get_config
    from xllm_service_amd.ops import hybrid as hops
    pc, lc = get_config(f"pugovik-{size}"), get_config(f"llama-{size}")
    lat = next(l.mixer for l in pc.layers if l.type == "latent_attention")
    lin = next(l.mixer for l in pc.layers if l.type == "lightning")
    bf = dict(dtype=torch.bfloat16, device=device)
    i32 = dict(dtype=torch.int32, device=device)
    out = []
    nblk = (max(T, ctx) + 15) // 16
    # ---- latent attention vs paged attention -----------------------------
    H, r, rd = lat["heads"], lat["kv_rank"], lat["rot_dim"]
    W = r + rd
    cache = torch.randn(batch * nblk, 16, W, **bf)
    tab = torch.arange(batch * nblk, **i32).view(batch, nblk)
    q = torch.randn(T, H, W, **bf)
    o = torch.empty(T, H, r, dtype=torch.float32, device=device)
    cu = torch.tensor([0, T], **i32)
    sl = torch.tensor([T], **i32)
    t = _time_gpu(lambda: hops.latent_attn(q, cache, tab[:1], cu, sl, 0.1, r,
                                           o), 3, 1)
    fl = 2.0 * H * (W + r) * T * (T + 1) / 2
    out.append(("latent_attn prefill", t, fl / t / 1e12, "TFLOP/s"))
    qd = torch.randn(batch, H, W, **bf)
    od = torch.empty(batch, H, r, dtype=torch.float32, device=device)
    sld = torch.full((batch,), ctx, **i32)
    t = _time_gpu(lambda: hops.latent_attn(qd, cache, tab, None, sld, 0.1, r,
                                           od))
    out.append(("latent_attn decode", t, batch * ctx * W * 2 / t / 1e9,
                "GB/s"))
    Hq, Hk, D = lc.num_heads, lc.num_kv_heads, lc.head_dim
    kc = torch.randn(batch * nblk, Hk, 16, D, **bf)
    vc = torch.randn(batch * nblk, Hk, 16, D, **bf)
    ql = torch.randn(T, Hq, D, **bf)
    if D == 128:
        t = _time_gpu(lambda: ops.paged_attn_prefill(ql, kc, vc, tab[:1], cu,
                                                     sl, 0.1), 3, 1)
        out.append(("paged_attn prefill (llama)", t,
                    4.0 * Hq * D * T * (T + 1) / 2 / t / 1e12, "TFLOP/s"))
    qld = torch.randn(batch, Hq, D, **bf)
    t = _time_gpu(lambda: ops.paged_attn_decode(qld, kc, vc, tab, sld, 0.1))
    out.append(("paged_attn decode (llama)", t,
                batch * ctx * Hk * D * 2 * 2 / t / 1e9, "GB/s"))
    # ---- decayed linear attention ----------------------------------------
    Hh, Dk, Dv = lin["heads"], lin["dim"], lin["vdim"]
    dec = torch.tensor(lin["decay"], dtype=torch.float32, device=device)
    st = torch.zeros(batch, Hh, Dk, Dv, dtype=torch.float32, device=device)
    qkv = torch.randn(T, 2 * Hh * Dk + Hh * Dv, **bf)
    oo = torch.empty(T, Hh, Dv, dtype=torch.float32, device=device)
    t = _time_gpu(lambda: hops.decay_attn(
        qkv[:, :Hh * Dk], qkv[:, Hh * Dk:2 * Hh * Dk], qkv[:, 2 * Hh * Dk:],
        dec, st, torch.zeros(1, **i32), cu, torch.zeros(1, **i32), oo), 3, 1)
    out.append(("decay_attn prefill", t, 4.0 * Hh * Dk * Dv * T / t / 1e12,
                "TFLOP/s (recurrence form)"))
    qkvd = torch.randn(batch, 2 * Hh * Dk + Hh * Dv, **bf)
    ood = torch.empty(batch, Hh, Dv, dtype=torch.float32, device=device)
    sls = torch.arange(batch, **i32)
    cx = torch.full((batch,), ctx, **i32)
    t = _time_gpu(lambda: hops.decay_attn(
        qkvd[:, :Hh * Dk], qkvd[:, Hh * Dk:2 * Hh * Dk], qkvd[:, 2 * Hh * Dk:],
        dec, st, sls, None, cx, ood))
    out.append(("decay_attn decode", t,
                batch * Hh * Dk * Dv * 4 * 2 / t / 1e9, "GB/s"))
    # ---- norms -------------------------------------------------------------
    Wd = pc.hidden_size
    x = torch.randn(T, Wd, dtype=torch.float32, device=device)
    w = torch.ones(Wd, dtype=torch.float32, device=device)
    t = _time_gpu(lambda: hops.group_rmsnorm(x, w, 1e-6, pc.norm_groups,
                                             torch.bfloat16))
    out.append(("group_rmsnorm fp32->bf16", t, T * Wd * 6 / t / 1e9, "GB/s"))
    y = torch.randn(T, Wd, **bf)
    gt = torch.randn(T, Wd, **bf)
    t = _time_gpu(lambda: hops.gated_norm_residual(x, y, gt, w, w, w, 0.5,
                                                   1e-6, pc.norm_groups))
    out.append(("gated_norm_residual", t, T * Wd * 12 / t / 1e9, "GB/s"))
    xb, rb, wb = torch.randn(T, Wd, **bf), torch.randn(T, Wd, **bf), \
        torch.ones(Wd, **bf)
    t = _time_gpu(lambda: ops.fused_add_rmsnorm(xb, rb, wb, 1e-6))
    out.append(("fused_add_rmsnorm (llama)", t, T * Wd * 8 / t / 1e9, "GB/s"))
    return out


def _dunusun_kernels(size, device, T, batch, ctx):
    """Achieved rates of the Dunusun mixer kernels at one layer's shapes,
    beside the like kernels of the pugovik / llama stacks of that size."""
    from xllm_service_amd import ops
    from xllm_service_amd.models.config import get_config
    from xllm_service_amd.ops import hybrid as hops
    dc, pc, lc = (get_config(f"{f}-{size}") for f in ("dunusun", "pugovik",
                                                       "llama"))
    par = next(l.mixer for l in dc.layers if l.type == "parallel")
    ssm = next(l.mixer for l in dc.layers if l.type == "mamba2")
    lin = next(l.mixer for l in pc.layers if l.type == "lightning")
    bf = dict(dtype=torch.bfloat16, device=device)
    f32 = dict(dtype=torch.float32, device=device)
    i32 = dict(dtype=torch.int32, device=device)
    out = []
    nblk = (max(T, ctx) + 15) // 16
    tab = torch.arange(batch * nblk, **i32).view(batch, nblk)
    cu = torch.tensor([0, T], **i32)
    sl = torch.tensor([T], **i32)
    sld = torch.full((batch,), ctx, **i32)
    z1 = torch.zeros(1, **i32)
    sls = torch.arange(batch, **i32)
    cx = torch.full((batch,), ctx, **i32)
    # ---- soft-capped attention vs paged attention ------------------------
    L = par["left"]
    H, G, D, Dv = L["heads"], L["kv_heads"], L["dim"], L["vdim"]
    kc = torch.randn(batch * nblk, G, 16, D, **bf)
    vc = torch.randn(batch * nblk, G, 16, Dv, **bf)
    q = torch.randn(T, H * D, **bf)
    o = torch.empty(T, H, Dv, **f32)
    t = _time_gpu(lambda: hops.capped_attn(q, kc, vc, tab[:1], cu, sl, H,
                                           L["scale"], L["softcap"], o), 3, 1)
    out.append(("capped_attn prefill", t,
                2.0 * H * (D + Dv) * T * (T + 1) / 2 / t / 1e12, "TFLOP/s"))
    qd = torch.randn(batch, H * D, **bf)
    od = torch.empty(batch, H, Dv, **f32)
    t = _time_gpu(lambda: hops.capped_attn(qd, kc, vc, tab, None, sld, H,
                                           L["scale"], L["softcap"], od))
    out.append(("capped_attn decode", t,
                batch * ctx * G * (D + Dv) * 2 / t / 1e9, "GB/s"))
    Hq, Hk, Dl = lc.num_heads, lc.num_kv_heads, lc.head_dim
    kl = torch.randn(batch * nblk, Hk, 16, Dl, **bf)
    vl = torch.randn(batch * nblk, Hk, 16, Dl, **bf)
    ql = torch.randn(T, Hq, Dl, **bf)
    if Dl == 128:
        t = _time_gpu(lambda: ops.paged_attn_prefill(ql, kl, vl, tab[:1], cu,
                                                     sl, 0.1), 3, 1)
        out.append(("paged_attn prefill (llama)", t,
                    4.0 * Hq * Dl * T * (T + 1) / 2 / t / 1e12, "TFLOP/s"))
    qld = torch.randn(batch, Hq, Dl, **bf)
    t = _time_gpu(lambda: ops.paged_attn_decode(qld, kl, vl, tab, sld, 0.1))
    out.append(("paged_attn decode (llama)", t,
                batch * ctx * Hk * Dl * 2 * 2 / t / 1e9, "GB/s"))
    # ---- gated recurrences vs decayed linear attention -------------------
    def recur(kind, Hh, Gg, Dk, Dvv, tokens, slots, cuq, ctxl):
        qq = torch.randn(tokens, Gg * Dk, **bf)
        kk = torch.randn(tokens, Gg * Dk, **bf)
        vv = torch.randn(tokens, Hh * Dvv, **bf)
        gg = torch.randn(tokens, Hh if kind == 0 else Hh * Dk, **bf)
        st = torch.zeros(batch, Hh, Dk, Dvv, **f32)
        p0 = torch.zeros(Hh if kind == 0 else Hh * Dk, **f32)
        p1 = torch.zeros(Hh, **f32) if kind == 0 else None
        oo = torch.empty(tokens, Hh, Dvv, **f32)
        return lambda: hops.gated_recurrence(
            kind, qq, kk, vv, gg, p0, p1, p1, 0.06, 0.1, st, slots, cuq, ctxl,
            Gg, oo, max_q_len=tokens)
    Hs, P, N, Gs = ssm["heads"], ssm["vdim"], ssm["state"], ssm["groups"]
    R = par["right"]
    for label, kind, Hh, Gg, Dk, Dvv in (
            ("ssm", 0, Hs, Gs, N, P),
            ("gla", 1, R["heads"], R["heads"], R["dim"], R["vdim"])):
        t = _time_gpu(recur(kind, Hh, Gg, Dk, Dvv, T, z1, cu, z1), 3, 1)
        out.append((f"gated_recurrence {label} prefill", t,
                    4.0 * Hh * Dk * Dvv * T / t / 1e12,
                    "TFLOP/s (recurrence form)"))
        t = _time_gpu(recur(kind, Hh, Gg, Dk, Dvv, batch, sls, None, cx))
        out.append((f"gated_recurrence {label} decode", t,
                    batch * Hh * Dk * Dvv * 4 * 2 / t / 1e9, "GB/s"))
    Hh, Dk, Dvv = lin["heads"], lin["dim"], lin["vdim"]
    dec = torch.tensor(lin["decay"], **f32)
    st = torch.zeros(batch, Hh, Dk, Dvv, **f32)
    qkv = torch.randn(T, 2 * Hh * Dk + Hh * Dvv, **bf)
    oo = torch.empty(T, Hh, Dvv, **f32)
    t = _time_gpu(lambda: hops.decay_attn(
        qkv[:, :Hh * Dk], qkv[:, Hh * Dk:2 * Hh * Dk], qkv[:, 2 * Hh * Dk:],
        dec, st, z1, cu, z1, oo), 3, 1)
    out.append(("decay_attn prefill (pugovik)", t,
                4.0 * Hh * Dk * Dvv * T / t / 1e12,
                "TFLOP/s (recurrence form)"))
    qkvd = torch.randn(batch, 2 * Hh * Dk + Hh * Dvv, **bf)
    ood = torch.empty(batch, Hh, Dvv, **f32)
    t = _time_gpu(lambda: hops.decay_attn(
        qkvd[:, :Hh * Dk], qkvd[:, Hh * Dk:2 * Hh * Dk], qkvd[:, 2 * Hh * Dk:],
        dec, st, sls, None, cx, ood))
    out.append(("decay_attn decode (pugovik)", t,
                batch * Hh * Dk * Dvv * 4 * 2 / t / 1e9, "GB/s"))
    # ---- short convolution -------------------------------------------------
    C, taps = Hs * P + 2 * Gs * N, ssm["conv"]
    xin = torch.randn(T, C, **bf)
    cw, cb = torch.randn(C, taps, **bf), torch.randn(C, **bf)
    cst = torch.zeros(batch, taps - 1, C, **bf)
    t = _time_gpu(lambda: hops.short_conv(xin, cw, cb, cst, 0, z1, cu, z1, 1,
                                          C, act_silu=True))
    out.append(("short_conv+silu", t, T * C * 4 / t / 1e9, "GB/s"))
    # ---- streams and norms -------------------------------------------------
    Wd, S = dc.hidden_size, dc.streams or 1
    xs = torch.randn(T, S, Wd, **f32)
    w = torch.ones(Wd, **f32)
    wi = torch.ones(S, **f32)
    mix = torch.eye(S, **f32)
    t = _time_gpu(lambda: hops.streams_mix_norm(xs, wi, w, w, 1e-6,
                                                torch.bfloat16))
    out.append(("streams_mix_norm", t, T * Wd * (4 * S + 2) / t / 1e9,
                "GB/s"))
    y = torch.randn(T, Wd, **bf)
    t = _time_gpu(lambda: hops.streams_update_(xs, mix, wi, y, 1.0, y, 1.0))
    out.append(("streams_update", t, T * Wd * (8 * S + 4) / t / 1e9, "GB/s"))
    t = _time_gpu(lambda: hops.streams_update_mix_norm_(
        xs, mix, wi, y, 1.0, y, 1.0, wi, w, w, 1e-6))
    out.append(("streams_update_mix_norm (fused)", t,
                T * Wd * (8 * S + 6) / t / 1e9, "GB/s"))
    xsd, yd = xs[:batch].contiguous(), y[:batch].contiguous()
    t = _time_gpu(lambda: hops.streams_update_mix_norm_(
        xsd, mix, wi, yd, 1.0, yd, 1.0, wi, w, w, 1e-6))
    out.append((f"streams_update_mix_norm, {batch} rows (decode)", t,
                batch * Wd * (8 * S + 6) / t / 1e9, "GB/s"))
    x1 = torch.randn(T, Wd, **f32)
    t = _time_gpu(lambda: hops.group_rmsnorm(x1, w, 1e-6, pc.norm_groups,
                                             torch.bfloat16))
    out.append(("group_rmsnorm fp32->bf16 (pugovik)", t,
                T * Wd * 6 / t / 1e9, "GB/s"))
    gt = torch.randn(T, Wd, **bf)
    t = _time_gpu(lambda: hops.gated_norm_residual(x1, y, gt, w, w, w, 0.5,
                                                   1e-6, pc.norm_groups))
    out.append(("gated_norm_residual (pugovik)", t, T * Wd * 12 / t / 1e9,
                "GB/s"))
    return out


def _tosipel_kernels(size, device, T, batch, ctx):
    """Achieved rates of the Tosipel mixer kernels at one layer's shapes,
    beside the like kernels of the dunusun / pugovik / llama stacks of that
    size."""
    from xllm_service_amd import ops
    from xllm_service_amd.models.config import get_config
    from xllm_service_amd.ops import hybrid as hops
    tc, dc, pc, lc = (get_config(f"{f}-{size}") for f in (
        "tosipel", "dunusun", "pugovik", "llama"))
    att = next(l.mixer for l in tc.layers if l.type == "attention")
    lat = next(l.mixer for l in tc.layers if l.type == "latent_attention")
    dl = next(l.mixer for l in tc.layers if l.type == "delta")
    cap = next(l.mixer for l in dc.layers if l.type == "parallel")["left"]
    ssm = next(l.mixer for l in dc.layers if l.type == "mamba2")
    plat = next(l.mixer for l in pc.layers if l.type == "latent_attention")
    bf = dict(dtype=torch.bfloat16, device=device)
    f32 = dict(dtype=torch.float32, device=device)
    i32 = dict(dtype=torch.int32, device=device)
    out = []
    nblk = (max(T, ctx) + 15) // 16
    tab = torch.arange(batch * nblk, **i32).view(batch, nblk)
    cu = torch.tensor([0, T], **i32)
    sl = torch.tensor([T], **i32)
    sld = torch.full((batch,), ctx, **i32)
    z1 = torch.zeros(1, **i32)
    sls = torch.arange(batch, **i32)
    cx = torch.full((batch,), ctx, **i32)
    # ---- windowed attention with a sink vs the soft-capped / llama kernels
    H, G, D, Dv = att["heads"], att["kv_heads"], att["dim"], att["vdim"]
    win = att["mask"]["size"]
    kc = torch.randn(batch * nblk, G, 16, D, **bf)
    vc = torch.randn(batch * nblk, G, 16, Dv, **bf)
    q = torch.randn(T, H * D, **bf)
    o = torch.empty(T, H, Dv, **f32)
    sink = torch.zeros(H, **f32)
    seen = sum(min(i + 1, win) for i in range(T))      # (query, key) pairs
    t = _time_gpu(lambda: hops.capped_attn(q, kc, vc, tab[:1], cu, sl, H,
                                           att["scale"], 0.0, o, window=win,
                                           sink=sink), 3, 1)
    out.append((f"window_attn prefill (window {win})", t,
                2.0 * H * (D + Dv) * seen / t / 1e12, "TFLOP/s"))
    qd = torch.randn(batch, H * D, **bf)
    od = torch.empty(batch, H, Dv, **f32)
    t = _time_gpu(lambda: hops.capped_attn(qd, kc, vc, tab, None, sld, H,
                                           att["scale"], 0.0, od, window=win,
                                           sink=sink))
    out.append((f"window_attn decode (window {win})", t,
                batch * min(ctx, win) * G * (D + Dv) * 2 / t / 1e9, "GB/s"))
    Hc, Gc, Dc, Dvc = cap["heads"], cap["kv_heads"], cap["dim"], cap["vdim"]
    kcc = torch.randn(batch * nblk, Gc, 16, Dc, **bf)
    vcc = torch.randn(batch * nblk, Gc, 16, Dvc, **bf)
    qc = torch.randn(T, Hc * Dc, **bf)
    oc = torch.empty(T, Hc, Dvc, **f32)
    t = _time_gpu(lambda: hops.capped_attn(qc, kcc, vcc, tab[:1], cu, sl, Hc,
                                           cap["scale"], cap["softcap"], oc),
                  3, 1)
    out.append(("capped_attn prefill (dunusun)", t,
                2.0 * Hc * (Dc + Dvc) * T * (T + 1) / 2 / t / 1e12,
                "TFLOP/s"))
    qcd = torch.randn(batch, Hc * Dc, **bf)
    ocd = torch.empty(batch, Hc, Dvc, **f32)
    t = _time_gpu(lambda: hops.capped_attn(qcd, kcc, vcc, tab, None, sld, Hc,
                                           cap["scale"], cap["softcap"], ocd))
    out.append(("capped_attn decode (dunusun)", t,
                batch * ctx * Gc * (Dc + Dvc) * 2 / t / 1e9, "GB/s"))
    Hq, Hk, Dl = lc.num_heads, lc.num_kv_heads, lc.head_dim
    kl = torch.randn(batch * nblk, Hk, 16, Dl, **bf)
    vl = torch.randn(batch * nblk, Hk, 16, Dl, **bf)
    qld = torch.randn(batch, Hq, Dl, **bf)
    t = _time_gpu(lambda: ops.paged_attn_decode(qld, kl, vl, tab, sld, 0.1))
    out.append(("paged_attn decode (llama)", t,
                batch * ctx * Hk * Dl * 2 * 2 / t / 1e9, "GB/s"))
    # ---- latent attention without a rotated part vs pugovik's -------------
    for label, Hh, r, rd in (
            ("latent_attn", lat["heads"], lat["kv_rank"], 0),
            ("latent_attn (pugovik)", plat["heads"], plat["kv_rank"],
             plat["rot_dim"])):
        Wl = r + rd
        cache = torch.randn(batch * nblk, 16, Wl, **bf)
        ql_ = torch.randn(T, Hh, Wl, **bf)
        ol = torch.empty(T, Hh, r, **f32)
        t = _time_gpu(lambda: hops.latent_attn(ql_, cache, tab[:1], cu, sl,
                                               0.1, r, ol), 3, 1)
        out.append((f"{label} prefill", t,
                    2.0 * Hh * (Wl + r) * T * (T + 1) / 2 / t / 1e12,
                    "TFLOP/s"))
        qld_ = torch.randn(batch, Hh, Wl, **bf)
        old = torch.empty(batch, Hh, r, **f32)
        t = _time_gpu(lambda: hops.latent_attn(qld_, cache, tab, None, sld,
                                               0.1, r, old))
        out.append((f"{label} decode", t, batch * ctx * Wl * 2 / t / 1e9,
                    "GB/s"))
    # ---- delta rule vs the selective state space recurrence ---------------
    Hh, Gg, Dk, Dvv = dl["heads"], dl["kv_heads"], dl["dim"], dl["vdim"]

    def delta(tokens, slots, cuq, ctxl):
        qq = torch.randn(tokens, Gg * Dk, **bf)
        kk = torch.randn(tokens, Gg * Dk, **bf)
        vv = torch.randn(tokens, Hh * Dvv, **bf)
        bb, aa = torch.randn(tokens, Hh, **bf), torch.randn(tokens, Hh, **bf)
        st = torch.zeros(batch, Hh, Dk, Dvv, **f32)
        p = torch.zeros(Hh, **f32)
        oo = torch.empty(tokens, Hh, Dvv, **f32)
        return lambda: hops.delta_rule(qq, kk, vv, bb, aa, p, p, st, slots,
                                       cuq, ctxl, Gg, oo, max_q_len=tokens)
    t = _time_gpu(delta(T, z1, cu, z1), 3, 1)
    out.append(("delta_rule prefill", t, 8.0 * Hh * Dk * Dvv * T / t / 1e12,
                "TFLOP/s (recurrence form)"))
    t = _time_gpu(delta(batch, sls, None, cx))
    out.append(("delta_rule decode", t,
                batch * Hh * Dk * Dvv * 4 * 2 / t / 1e9, "GB/s"))
    Hs, P, N, Gs = ssm["heads"], ssm["vdim"], ssm["state"], ssm["groups"]

    def recur(tokens, slots, cuq, ctxl):
        qq = torch.randn(tokens, Gs * N, **bf)
        kk = torch.randn(tokens, Gs * N, **bf)
        vv = torch.randn(tokens, Hs * P, **bf)
        gg = torch.randn(tokens, Hs, **bf)
        st = torch.zeros(batch, Hs, N, P, **f32)
        p0 = torch.zeros(Hs, **f32)
        oo = torch.empty(tokens, Hs, P, **f32)
        return lambda: hops.gated_recurrence(
            0, qq, kk, vv, gg, p0, p0, p0, 0.06, 0.1, st, slots, cuq, ctxl,
            Gs, oo, max_q_len=tokens)
    t = _time_gpu(recur(T, z1, cu, z1), 3, 1)
    out.append(("gated_recurrence ssm prefill (dunusun)", t,
                4.0 * Hs * N * P * T / t / 1e12, "TFLOP/s (recurrence form)"))
    t = _time_gpu(recur(batch, sls, None, cx))
    out.append(("gated_recurrence ssm decode (dunusun)", t,
                batch * Hs * N * P * 4 * 2 / t / 1e9, "GB/s"))
    # ---- q/k preparation, convolution, norms, gates ------------------------
    big = torch.randn(T, H * D + G * D + G * Dv, **bf)
    qw, kw = torch.ones(H * D, **f32), torch.ones(G * D, **f32)
    rot = att["rot"]["dims"]
    inv = torch.ones(rot // 2, dtype=torch.float64, device=device)
    pos = torch.arange(T, device=device)
    slot = torch.arange(T, device=device)
    t = _time_gpu(lambda: hops.rownorm_rope_store(
        big[:, :H * D], big[:, H * D:H * D + G * D], big[:, H * D + G * D:],
        qw, kw, 1e-6, pos, inv, rot, H, G, kc, vc, slot))
    out.append(("rownorm_rope_store", t,
                T * (H * D * 2 + G * D * 2 + G * Dv * 2) * 2 / t / 1e9,
                "GB/s"))
    C, taps = 2 * Gg * Dk + Hh * Dvv, dl["conv"]
    xin = torch.randn(T, C, **bf)
    cw = torch.randn(C, taps, **bf)
    cst = torch.zeros(batch, taps - 1, C, **bf)
    t = _time_gpu(lambda: hops.short_conv(xin, cw, None, cst, 0, z1, cu, z1,
                                          1, C, act_silu=True))
    out.append(("short_conv+silu", t, T * C * 4 / t / 1e9, "GB/s"))
    Wd = tc.hidden_size
    x1 = torch.randn(T, Wd, **f32)
    y = torch.randn(T, Wd, **bf)
    w = torch.ones(Wd, **f32)
    t = _time_gpu(lambda: hops.norm_residual_add_(x1, y, w, 1e-6,
                                                  torch.bfloat16))
    out.append(("norm_residual_add", t, T * Wd * 12 / t / 1e9, "GB/s"))
    xd1, yd1 = x1[:batch].contiguous(), y[:batch].contiguous()
    t = _time_gpu(lambda: hops.norm_residual_add_(xd1, yd1, w, 1e-6,
                                                  torch.bfloat16))
    out.append((f"norm_residual_add, {batch} rows (decode)", t,
                batch * Wd * 12 / t / 1e9, "GB/s"))
    S = dc.streams or 1
    xs = torch.randn(T, S, Wd, **f32)
    wi, mix = torch.ones(S, **f32), torch.eye(S, **f32)
    t = _time_gpu(lambda: hops.streams_update_mix_norm_(
        xs, mix, wi, y, 1.0, y, 1.0, wi, w, w, 1e-6))
    out.append(("streams_update_mix_norm (dunusun)", t,
                T * Wd * (8 * S + 6) / t / 1e9, "GB/s"))
    gt = torch.randn(T, Wd, **bf)
    t = _time_gpu(lambda: hops.gated_norm_residual(x1, y, gt, w, w, w, 0.5,
                                                   1e-6, pc.norm_groups))
    out.append(("gated_norm_residual (pugovik)", t, T * Wd * 12 / t / 1e9,
                "GB/s"))
    ff = next(l.mlp for l in tc.layers if l.mlp)["ff"]
    gu = torch.randn(T, 2 * ff, **bf)
    t = _time_gpu(lambda: hops.gelu_tanh_mul(gu))
    out.append(("gelu_tanh_mul", t, T * ff * 6 / t / 1e9, "GB/s"))
    t = _time_gpu(lambda: hops.silu_mul(gu))
    out.append(("silu_mul (pugovik)", t, T * ff * 6 / t / 1e9, "GB/s"))
    return out


def _gararax_kernels(size, device, T, batch, ctx):
    """Achieved rates of the Gararax kernels at one layer's shapes, beside
    the like kernels of the tosipel / pugovik / llama stacks of that size."""
    from xllm_service_amd import ops
    from xllm_service_amd.models.config import get_config
    from xllm_service_amd.ops import hybrid as hops
    gc, tc, pc, lc = (get_config(f"{f}-{size}") for f in (
        "gararax", "tosipel", "pugovik", "llama"))
    a1 = next(l.mixer for l in gc.layers if l.type == "attention")
    a2 = next(l.mixer for l in gc.layers if l.type == "attention_2")
    a3 = next(l.mixer for l in gc.layers if l.type == "attention_3")
    moe = next(l.mlp for l in gc.layers if l.mlp["kind"] == "moe")
    dense = next(l.mlp for l in gc.layers if l.mlp["kind"] == "dense")
    tatt = next(l.mixer for l in tc.layers if l.type == "attention")
    pmoe = next(l.mlp for l in pc.layers if l.mlp)
    bf = dict(dtype=torch.bfloat16, device=device)
    f32 = dict(dtype=torch.float32, device=device)
    i32 = dict(dtype=torch.int32, device=device)
    out = []
    nblk = (max(T, ctx) + 15) // 16
    tab = torch.arange(batch * nblk, **i32).view(batch, nblk)
    cu = torch.tensor([0, T], **i32)
    sl = torch.tensor([T], **i32)
    sld = torch.full((batch,), ctx, **i32)

    def attn_pair(label, m, window, keep, sink, hs, same, tail=""):
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        kc = torch.randn(batch * nblk, G, 16, D, **bf)
        vc = kc if same else torch.randn(batch * nblk, G, 16, Dv, **bf)
        q = torch.randn(T, H * D, **bf)
        o = torch.empty(T, H, Dv, **f32)
        sk = torch.zeros(H, **f32) if sink else None
        hsc = torch.ones(H, **f32) if hs else None
        kw = dict(window=window, sink=sk, keep_first=keep, head_scale=hsc)
        seen = sum(min(i + 1, window) + min(keep, max(i + 1 - window, 0))
                   if window else i + 1 for i in range(T))
        t = _time_gpu(lambda: hops.capped_attn(q, kc, vc, tab[:1], cu, sl, H,
                                               m["scale"], 0.0, o, **kw), 3, 1)
        out.append((f"{label} prefill{tail}", t,
                    2.0 * H * (D + Dv) * seen / t / 1e12, "TFLOP/s"))
        qd = torch.randn(batch, H * D, **bf)
        od = torch.empty(batch, H, Dv, **f32)
        t = _time_gpu(lambda: hops.capped_attn(qd, kc, vc, tab, None, sld, H,
                                               m["scale"], 0.0, od, **kw))
        keys = min(ctx, window + keep) if window else ctx
        width = D if same else D + Dv
        out.append((f"{label} decode{tail}", t,
                    batch * keys * G * width * 2 / t / 1e9, "GB/s"))

    w1 = a1["mask"]
    attn_pair("window+kept attn", a1, w1["size"], w1["keep_first"], False,
              False, False, f" (window {w1['size']}, kept {w1['keep_first']})")
    w2 = a2["mask"]
    attn_pair("keys-as-values sink attn", a2, w2["size"], w2["keep_first"],
              True, False, True, f" (window {w2['size']})")
    attn_pair("full attn, head multiplier", a3, 0, 0, False, True, False)
    attn_pair("window+sink attn (tosipel)", tatt, tatt["mask"]["size"], 0,
              True, False, False, f" (window {tatt['mask']['size']})")
    Hq, Hk, Dl = lc.num_heads, lc.num_kv_heads, lc.head_dim
    kl = torch.randn(batch * nblk, Hk, 16, Dl, **bf)
    vl = torch.randn(batch * nblk, Hk, 16, Dl, **bf)
    if Dl == 128:
        ql = torch.randn(T, Hq, Dl, **bf)
        t = _time_gpu(lambda: ops.paged_attn_prefill(ql, kl, vl, tab[:1], cu,
                                                     sl, 0.1), 3, 1)
        out.append(("paged_attn prefill (llama)", t,
                    4.0 * Hq * Dl * T * (T + 1) / 2 / t / 1e12, "TFLOP/s"))
    qld = torch.randn(batch, Hq, Dl, **bf)
    t = _time_gpu(lambda: ops.paged_attn_decode(qld, kl, vl, tab, sld, 0.1))
    out.append(("paged_attn decode (llama)", t,
                batch * ctx * Hk * Dl * 2 * 2 / t / 1e9, "GB/s"))
    # ---- query/key preparation with paged store ----------------------------
    H, G, D, Dv = a1["heads"], a1["kv_heads"], a1["dim"], a1["vdim"]
    rot = a1["rot"]["dims"]
    proj = torch.randn(T, H * D + G * D + G * Dv, **bf)
    kc = torch.zeros(nblk, G, 16, D, **bf)
    vc = torch.zeros(nblk, G, 16, Dv, **bf)
    pos = torch.arange(T, dtype=torch.long, device=device)
    inv = torch.rand(rot // 2, dtype=torch.float64, device=device)
    nbytes = T * (2 * H * D + 2 * G * D + 2 * G * Dv) * 2
    t = _time_gpu(lambda: hops.rope_headnorm_store(
        proj[:, :H * D], proj[:, H * D:H * D + G * D], proj[:, H * D + G * D:],
        pos, inv, rot, True, True, 1e-6, H, G, kc, vc, pos))
    out.append(("rope_headnorm_store", t, nbytes / t / 1e9, "GB/s"))
    Ht, Gt, Dt, Dvt = tatt["heads"], tatt["kv_heads"], tatt["dim"], \
        tatt["vdim"]
    rt = tatt["rot"]["dims"]
    projt = torch.randn(T, Ht * Dt + Gt * Dt + Gt * Dvt, **bf)
    kct = torch.zeros(nblk, Gt, 16, Dt, **bf)
    vct = torch.zeros(nblk, Gt, 16, Dvt, **bf)
    invt = torch.rand(rt // 2, dtype=torch.float64, device=device)
    wq, wk = torch.ones(Ht * Dt, **f32), torch.ones(Gt * Dt, **f32)
    t = _time_gpu(lambda: hops.rownorm_rope_store(
        projt[:, :Ht * Dt], projt[:, Ht * Dt:Ht * Dt + Gt * Dt],
        projt[:, Ht * Dt + Gt * Dt:], wq, wk, 1e-6, pos, invt, rt, Ht, Gt,
        kct, vct, pos))
    out.append(("rownorm_rope_store (tosipel)", t,
                T * (2 * Ht * Dt + 2 * Gt * Dt + 2 * Gt * Dvt) * 2 / t / 1e9,
                "GB/s"))
    # ---- norms and activations ---------------------------------------------
    Wd = gc.hidden_size
    x = torch.randn(T, Wd, **f32)
    w = torch.ones(Wd, **f32)
    y = torch.randn(T, Wd, **bf)
    y32 = torch.randn(T, Wd, **f32)
    t = _time_gpu(lambda: hops.norm_residual_add_(x, y, w, 1e-6,
                                                  torch.bfloat16, w))
    out.append(("norm_residual_add + next norm", t, T * Wd * 12 / t / 1e9,
                "GB/s"))
    t = _time_gpu(lambda: hops.norm_residual_add_(x, y32, w, 1e-6,
                                                  torch.bfloat16, w))
    out.append(("norm_residual_add + next norm (fp32 input)", t,
                T * Wd * 14 / t / 1e9, "GB/s"))
    t = _time_gpu(lambda: hops.norm_residual_add_(x, y, w, 1e-6,
                                                  torch.bfloat16))
    out.append(("norm_residual_add (tosipel)", t, T * Wd * 12 / t / 1e9,
                "GB/s"))
    ff = dense["ff"]
    z = torch.randn(T, ff, **bf)
    coef = torch.tensor([0.5, 0.3, 0.2, 0.0], **f32)
    t = _time_gpu(lambda: hops.polynorm(z, coef, 1e-6))
    out.append(("polynorm", t, T * ff * 4 / t / 1e9, "GB/s"))
    z2 = torch.randn(T, 2 * ff, **bf)
    t = _time_gpu(lambda: hops.gelu_tanh_mul(z2))
    out.append(("gelu_tanh_mul (tosipel)", t, T * ff * 6 / t / 1e9, "GB/s"))
    sd = gc.side_dim
    ga = torch.randn(T, sd, **bf)
    tbl = torch.randn(T, sd * gc.num_layers, **bf)
    t = _time_gpu(lambda: hops.gelu_tanh_gate(ga, tbl[:, sd:2 * sd]))
    out.append(("gelu_tanh_gate (side input)", t, T * sd * 6 / t / 1e9,
                "GB/s"))
    # ---- router and combine --------------------------------------------------
    r = moe["router"]
    n_all = r["experts"] + r["identity"]
    h = torch.randn(T, Wd, **bf)
    wr = torch.randn(n_all, Wd, **f32)
    corr = torch.zeros(n_all, **f32)
    t = _time_gpu(lambda: hops.moe_route(
        h, wr, r["top"], r["groups"]["count"], r["groups"]["keep"],
        softmax=True, correction=corr, group_max=True, normalize=True))
    out.append(("moe_route softmax+correction", t, T / t / 1e6, "Mtok/s"))
    pr = pmoe["router"]
    wrp = torch.randn(pr["experts"], pc.hidden_size, **f32)
    hp = torch.randn(T, pc.hidden_size, **bf)
    t = _time_gpu(lambda: hops.moe_route(hp, wrp, pr["top"],
                                         pr["groups"]["count"],
                                         pr["groups"]["keep"]))
    out.append(("moe_route sigmoid (pugovik)", t, T / t / 1e6, "Mtok/s"))
    top = r["top"]
    ye = torch.randn(T * top, Wd, **bf)
    rows = torch.arange(T * top, **i32).view(T, top).clone()
    rows[::3, 0] = -1
    wts = torch.rand(T, top, **f32)
    t = _time_gpu(lambda: hops.moe_combine(ye, rows, wts, T, h, y))
    out.append(("moe_combine + identity + shared", t,
                T * Wd * (2 * top + 2 + 4) / t / 1e9, "GB/s"))
    rows0 = torch.arange(T * top, **i32).view(T, top)
    t = _time_gpu(lambda: hops.moe_combine(ye, rows0, wts, T))
    out.append(("moe_combine (pugovik)", t, T * Wd * (2 * top + 4) / t / 1e9,
                "GB/s"))
    return out


def _nikedra_kernels(size, device, T, batch, ctx):
    """Achieved rates of the Nikedra kernels at one layer's shapes, each
    beside the like kernel of the tosipel / dunusun / pugovik stacks of that
    size."""
    from xllm_service_amd.models.config import get_config
    from xllm_service_amd.ops import hybrid as hops
    nc, tc, dc, pc = (get_config(f"{f}-{size}") for f in (
        "nikedra", "tosipel", "dunusun", "pugovik"))

    def mixer(cfg, kind):
        return next(l.mixer for l in cfg.layers if l.type == kind)
    left, ssm = mixer(nc, "parallel")["left"], mixer(nc, "parallel")["right"]
    lat, dl = mixer(nc, "latent_attention"), mixer(nc, "channel_delta")
    tatt, tdl = mixer(tc, "attention"), mixer(tc, "delta")
    plat, dssm = mixer(pc, "latent_attention"), mixer(dc, "mamba2")
    bf = dict(dtype=torch.bfloat16, device=device)
    f32 = dict(dtype=torch.float32, device=device)
    i32 = dict(dtype=torch.int32, device=device)
    out = []
    nblk = (max(T, ctx) + 15) // 16
    tab = torch.arange(batch * nblk, **i32).view(batch, nblk)
    cu = torch.tensor([0, T], **i32)
    sl = torch.tensor([T], **i32)
    sld = torch.full((batch,), ctx, **i32)
    z1 = torch.zeros(1, **i32)
    sls = torch.arange(batch, **i32)

    def add(label, fn, work, unit, iters=10):
        t = _time_gpu(fn, iters, 3)
        out.append((label, t, work / t / (1e12 if "FLOP" in unit else 1e9),
                    unit))
    # ---- chunked attention vs windowed attention ---------------------------
    for label, m, chunked in (("chunk attn", left, True),
                              ("window+sink attn (tosipel)", tatt, False)):
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        win = m["mask"]["size"]
        kc = torch.randn(batch * nblk, G, 16, D, **bf)
        vc = torch.randn(batch * nblk, G, 16, Dv, **bf)
        q = torch.randn(T, H * D, **bf)
        o = torch.empty(T, H, Dv, **f32)
        kw = dict(window=win, chunked=chunked,
                  sink=None if chunked else torch.zeros(H, **f32))
        seen = sum(i % win + 1 if chunked else min(i + 1, win)
                   for i in range(T))
        add(f"{label} prefill ({win})",
            lambda: hops.capped_attn(q, kc, vc, tab[:1], cu, sl, H,
                                     m["scale"], 0.0, o, **kw),
            2.0 * H * (D + Dv) * seen, "TFLOP/s", 3)
        qd = torch.randn(batch, H * D, **bf)
        od = torch.empty(batch, H, Dv, **f32)
        keys = (ctx - 1) % win + 1 if chunked else min(ctx, win)
        add(f"{label} decode ({win})",
            lambda: hops.capped_attn(qd, kc, vc, tab, None, sld, H,
                                     m["scale"], 0.0, od, **kw),
            batch * keys * G * (D + Dv) * 2, "GB/s")
        del kc, vc
    # ---- latent attention with and without a window ------------------------
    for label, m, win in (("latent window attn", lat, lat["mask"]["size"]),
                          ("latent_attn (pugovik)", plat, 0)):
        H, r, W = m["heads"], m["kv_rank"], m["kv_rank"] + m["rot_dim"]
        cache = torch.randn(batch * nblk, 16, W, **bf)
        q = torch.randn(T, H, W, **bf)
        o = torch.empty(T, H, r, **f32)
        seen = sum(min(i + 1, win or T) for i in range(T))
        add(f"{label} prefill",
            lambda: hops.latent_attn(q, cache, tab[:1], cu, sl, 0.1, r, o,
                                     win),
            2.0 * H * (W + r) * seen, "TFLOP/s", 3)
        qd = torch.randn(batch, H, W, **bf)
        od = torch.empty(batch, H, r, **f32)
        add(f"{label} decode",
            lambda: hops.latent_attn(qd, cache, tab, None, sld, 0.1, r, od,
                                     win),
            batch * min(ctx, win or ctx) * W * 2, "GB/s")
    # ---- delta rule, channel decays vs head decays -------------------------
    for label, m, ch in (("channel delta_rule", dl, True),
                         ("delta_rule (tosipel)", tdl, False)):
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        n = H * D if ch else H
        st = torch.zeros(batch, H, D, Dv, **f32)
        dtb, al = torch.zeros(n, **f32), torch.zeros(H, **f32)
        for tokens, slots, cuq, ctxl, tail in (
                (T, z1, cu, z1, "prefill"), (batch, sls, None, sld, "decode")):
            qq = torch.randn(tokens, G * D, **bf)
            vv = torch.randn(tokens, H * Dv, **bf)
            bb, aa = torch.randn(tokens, H, **bf), torch.randn(tokens, n, **bf)
            oo = torch.empty(tokens, H, Dv, **f32)
            work = 8.0 * H * D * Dv * T if cuq is not None \
                else batch * H * D * Dv * 8
            add(f"{label} {tail}",
                lambda: hops.delta_rule(qq, qq, vv, bb, aa, dtb, al, st,
                                        slots, cuq, ctxl, G, oo,
                                        max_q_len=tokens), work,
                "GB/s" if cuq is None else "TFLOP/s (recurrence form)",
                10 if cuq is None else 3)
    # ---- state space recurrence ---------------------------------------------
    for label, m in (("state space", ssm), ("state space (dunusun)", dssm)):
        H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
        st = torch.zeros(batch, H, N, P, **f32)
        p0 = torch.zeros(H, **f32)
        for tokens, slots, cuq, ctxl, tail in (
                (T, z1, cu, z1, "prefill"), (batch, sls, None, sld, "decode")):
            qq = torch.randn(tokens, G * N, **bf)
            vv, gg = torch.randn(tokens, H * P, **bf), \
                torch.randn(tokens, H, **bf)
            oo = torch.empty(tokens, H, P, **f32)
            work = 4.0 * H * N * P * T if cuq is not None \
                else batch * H * N * P * 8
            add(f"{label} {tail}",
                lambda: hops.gated_recurrence(
                    0, qq, qq, vv, gg, p0, p0, p0, 0.0, 1.0, st, slots, cuq,
                    ctxl, G, oo, max_q_len=tokens), work,
                "GB/s" if cuq is None else "TFLOP/s (recurrence form)",
                10 if cuq is None else 3)
    # ---- input convolution ----------------------------------------------------
    Wd = nc.hidden_size
    xin = torch.randn(T, Wd, **bf)
    cw = torch.randn(Wd, nc.canon_taps, **bf)
    cst = torch.zeros(batch, nc.canon_taps - 1, Wd, **bf)
    add("input convolution",
        lambda: hops.short_conv(xin, cw, None, cst, 0, z1, cu, z1, 1, Wd,
                                add_input=True, advance=True), T * Wd * 4,
        "GB/s")
    add("short_conv+silu (dunusun, tosipel)",
        lambda: hops.short_conv(xin, cw, None, cst, 0, z1, cu, z1, 1, Wd,
                                act_silu=True), T * Wd * 4, "GB/s")
    xd = xin[:batch].contiguous()
    add(f"input convolution + state, {batch} rows (decode)",
        lambda: hops.short_conv(xd, cw, None, cst, 0, sls, None, sld, 1, Wd,
                                add_input=True, advance=True),
        batch * Wd * 2 * (2 + 2 * (nc.canon_taps - 1)), "GB/s")
    # ---- depth average vs the streams kernel ----------------------------------
    lv = nc.num_layers
    w, g = torch.ones(Wd, **f32), torch.ones(1, **f32)
    for rows, tail in ((T, ""), (batch, f", {batch} rows (decode)")):
        hist = torch.randn(lv + 1, rows, Wd, **f32)
        x, m1 = torch.randn(rows, Wd, **f32), torch.randn(rows, Wd, **bf)
        for level in (1, lv):
            dwa = torch.ones(level + 1, **f32)
            add(f"depth_mix_norm, level {level}{tail}",
                lambda: hops.depth_mix_norm(
                    x, hist, level, m1, None, None, None, 1.0, m1, dwa, g, g,
                    1e-6, torch.bfloat16, x),
                rows * Wd * (4 * (level + 3) + 2 * 4), "GB/s")
        dwa = torch.ones(lv + 1, **f32)
        add(f"depth_mix_norm, level {lv}, two normed halves{tail}",
            lambda: hops.depth_mix_norm(
                x, hist, lv, m1, w, m1, w, 0.5, x, dwa, g, g, 1e-6,
                torch.bfloat16, x), rows * Wd * (4 * (lv + 4) + 2 * 4),
            "GB/s")
        S = dc.streams or 1
        xs = torch.randn(rows, S, Wd, **f32)
        wi, mix = torch.ones(S, **f32), torch.eye(S, **f32)
        add(f"streams_update_mix_norm (dunusun){tail}",
            lambda: hops.streams_update_mix_norm_(
                xs, mix, wi, m1, 1.0, m1, 1.0, wi, w, w, 1e-6),
            rows * Wd * (8 * S + 6), "GB/s")
    # ---- query/key preparation, gates, experts --------------------------------
    H, G, D, Dv = left["heads"], left["kv_heads"], left["dim"], left["vdim"]
    rot = left["rot"]["dims"]
    proj = torch.randn(T, H * D + G * D + G * Dv, **bf)
    kc = torch.zeros(nblk, G, 16, D, **bf)
    vc = torch.zeros(nblk, G, 16, Dv, **bf)
    pos = torch.arange(T, dtype=torch.long, device=device)
    inv = torch.rand(rot // 2, dtype=torch.float64, device=device)
    wq, wk = torch.ones(H * D, **f32), torch.ones(G * D, **f32)
    q, k, v = proj[:, :H * D], proj[:, H * D:H * D + G * D], \
        proj[:, H * D + G * D:]
    nb = T * (2 * H * D + 2 * G * D + 2 * G * Dv) * 2
    add("rope_headnorm_store (half layout, multiplier)",
        lambda: hops.rope_headnorm_store(q, k, v, pos, inv, rot, False, False,
                                         1e-6, H, G, kc, vc, pos, 1.1), nb,
        "GB/s")
    add("rownorm_rope_store (tosipel)",
        lambda: hops.rownorm_rope_store(q, k, v, wq, wk, 1e-6, pos, inv, rot,
                                        H, G, kc, vc, pos), nb, "GB/s")
    ff = 3 * Wd // 2
    gu = torch.randn(T, 2 * ff, **bf)
    add("clamped_glu", lambda: hops.clamped_glu(gu, 7.0, 1.702, 1.0),
        T * ff * 6, "GB/s")
    add("gelu_tanh_mul (tosipel)", lambda: hops.gelu_tanh_mul(gu),
        T * ff * 6, "GB/s")
    mlp = next(l.mlp for l in nc.layers if l.mlp["kind"] == "moe")
    E, top, eff = mlp["router"]["experts"], mlp["router"]["top"], \
        mlp["expert"]["ff"]
    ze = torch.randn(T * top, eff, **bf)
    sc = torch.rand(T * top, **f32)
    add("gelu_scaled (sorted rows)", lambda: hops.gelu_scaled(ze, sc),
        T * top * eff * 4, "GB/s")
    add("silu_mul (pugovik)", lambda: hops.silu_mul(gu), T * ff * 6, "GB/s")
    zd = torch.randn(E, batch, eff, **bf)
    ids = torch.randint(0, E, (batch, top), **i32)
    wd = torch.rand(batch, top, **f32)
    add(f"gelu_scaled ({batch} tokens x {E} experts)",
        lambda: hops.gelu_scaled(zd, None, ids, wd), E * batch * eff * 2,
        "GB/s written")
    return out


def _zokanex_kernels(size, device, T, batch, ctx):
    """Achieved rates of the Zokanex kernels at one layer's shapes, each
    beside the like kernel of the gararax / tosipel / pugovik / nikedra stacks
    of that size. The results go into rows of the joint output operand, as in
    the model."""
    import torch.nn.functional as F
    from xllm_service_amd.models.config import get_config
    from xllm_service_amd.models.mixers import banded_rope_frequencies
    from xllm_service_amd.ops import hybrid as hops
    zc, tc, pc = (get_config(f"{f}-{size}") for f in (
        "zokanex", "tosipel", "pugovik"))

    def mixer(cfg, kind):
        return next(l.mixer for l in cfg.layers if l.type == kind)
    att, ret = mixer(zc, "attention"), mixer(zc, "retention")
    tatt, lin = mixer(tc, "attention"), mixer(pc, "lightning")
    dense = next(l.mlp for l in zc.layers if l.mlp["kind"] == "dense")
    moe = next(l.mlp for l in zc.layers if l.mlp["kind"] == "moe")
    bf = dict(dtype=torch.bfloat16, device=device)
    f32 = dict(dtype=torch.float32, device=device)
    i32 = dict(dtype=torch.int32, device=device)
    out = []
    nblk = (max(T, ctx) + 15) // 16
    tab = torch.arange(batch * nblk, **i32).view(batch, nblk)
    cu = torch.tensor([0, T], **i32)
    sl = torch.tensor([T], **i32)
    sld = torch.full((batch,), ctx, **i32)
    z1 = torch.zeros(1, **i32)
    sls = torch.arange(batch, **i32)
    pos = torch.arange(T, dtype=torch.long, device=device)

    def add(label, fn, work, unit, iters=20):
        t = _time_gpu(fn, iters, 3)
        scale = 1e12 if "FLOP" in unit else 1e6 if unit == "Mtok/s" else 1e9
        out.append((label, t, work / t / scale, unit))
    # ---- windowed attention ---------------------------------------------------
    Wd, ff = zc.hidden_size, dense["ff"]
    for label, m, joint in (("window attn", att, True),
                            ("window+sink attn (tosipel)", tatt, False)):
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        win = m["mask"]["size"]
        kc = torch.randn(batch * nblk, G, 16, D, **bf)
        vc = torch.randn(batch * nblk, G, 16, Dv, **bf)
        q = torch.randn(T, H * D, **bf)
        o = torch.empty(T, H * Dv + ff, **bf)[:, :H * Dv] if joint \
            else torch.empty(T, H, Dv, **f32)
        kw = dict(window=win,
                  sink=None if joint else torch.zeros(H, **f32))
        seen = sum(min(i + 1, win) for i in range(T))
        add(f"{label} prefill ({win})",
            lambda: hops.capped_attn(q, kc, vc, tab[:1], cu, sl, H,
                                     m["scale"], 0.0, o, **kw),
            2.0 * H * (D + Dv) * seen, "TFLOP/s", 5)
        add(f"{label} decode ({win})",
            lambda: hops.capped_attn(q[:batch], kc, vc, tab, None, sld, H,
                                     m["scale"], 0.0, o[:batch], **kw),
            batch * min(ctx, win) * G * (D + Dv) * 2, "GB/s")
        del kc, vc
    # ---- retention vs decayed linear attention ----------------------------------
    H, D, Dv, rot = ret["heads"], ret["dim"], ret["vdim"], ret["rot"]
    a, b = H * D, H * Dv
    p = torch.randn(T, 2 * a + 2 * b, **bf)
    dec = torch.tensor(ret["decay"], **f32)
    st = torch.zeros(batch, H, D, Dv, **f32)
    y = torch.empty(T, b + ff, **bf)
    inv = banded_rope_frequencies(rot).to(device)
    table = hops.rope_table(pos, inv)
    tokens = ((T, z1, cu, z1, "prefill"), (batch, sls, None, sld, "decode"))
    for n, slots, cuq, ctxl, tail in tokens:
        q, k, v, g = (p[:n, i:j] for i, j in (
            (0, a), (a, 2 * a), (2 * a, 2 * a + b), (2 * a + b, 2 * a + 2 * b)))
        add(f"retention + norm + gate {tail}",
            lambda: hops.retention(q, k, v, g, table[:n], D ** -0.5, dec, st,
                                   slots, cuq, ctxl, 1e-6, y[:n, :b]),
            4.0 * H * D * Dv * T if cuq is not None
            else batch * H * D * Dv * 8,
            "GB/s" if cuq is None else "TFLOP/s (recurrence form)")
    Hp, Dp, Vp = lin["heads"], lin["dim"], lin["vdim"]
    pl = torch.randn(T, 2 * Hp * Dp + Hp * Vp, **bf)
    decp = torch.tensor(lin["decay"], **f32)
    stp = torch.zeros(batch, Hp, Dp, Vp, **f32)
    op = torch.empty(T, Hp, Vp, **f32)
    for n, slots, cuq, ctxl, tail in tokens:
        q, k, v = pl[:n, :Hp * Dp], pl[:n, Hp * Dp:2 * Hp * Dp], \
            pl[:n, 2 * Hp * Dp:]
        add(f"decay_attn (pugovik) {tail}",
            lambda: hops.decay_attn(q, k, v, decp, stp, slots, cuq, ctxl,
                                    op[:n], max_q_len=n),
            4.0 * Hp * Dp * Vp * T if cuq is not None
            else batch * Hp * Dp * Vp * 8,
            "GB/s" if cuq is None else "TFLOP/s (recurrence form)", 5)
    add("rope_table", lambda: hops.rope_table(pos, inv), T * rot["dims"] * 4,
        "GB/s")
    # ---- query/key preparation --------------------------------------------------
    H, G, D, Dv = att["heads"], att["kv_heads"], att["dim"], att["vdim"]
    rd = att["rot"]["dims"]
    proj = torch.randn(T, H * D + G * D + G * Dv, **bf)
    kc = torch.zeros(nblk, G, 16, D, **bf)
    vc = torch.zeros(nblk, G, 16, Dv, **bf)
    w = torch.ones(D, **f32)
    wq, wk = torch.ones(H * D, **f32), torch.ones(G * D, **f32)
    inv = banded_rope_frequencies(att["rot"]).to(device)
    table = hops.rope_table(pos, inv)
    q, k, v = proj[:, :H * D], proj[:, H * D:H * D + G * D], \
        proj[:, H * D + G * D:]
    nb = T * (2 * H * D + 2 * G * D + 2 * G * Dv) * 2
    args = (pos, inv, rd, False, False, 1e-6, H, G, kc, vc, pos, 1.0)
    add("head norm + turn + store",
        lambda: hops.rope_headnorm_store(q, k, v, *args, w, w, table), nb,
        "GB/s")
    add("head norm + turn, borrowed keys",
        lambda: hops.rope_headnorm_store(q, None, None, *args, w, None, table),
        T * 2 * H * D * 2, "GB/s")
    add("rope_headnorm_store (gararax)",
        lambda: hops.rope_headnorm_store(
            q, k, v, pos, inv, rd, True, True, 1e-6, H, G, kc, vc, pos), nb,
        "GB/s")
    add("rownorm_rope_store (tosipel)",
        lambda: hops.rownorm_rope_store(q, k, v, wq, wk, 1e-6, pos, inv, rd,
                                        H, G, kc, vc, pos), nb, "GB/s")
    # ---- residual ---------------------------------------------------------------
    x, wn = torch.randn(T, Wd, **f32), torch.ones(Wd, **f32)
    top = moe["router"]["top"]
    ya = torch.randn(T, Wd, **bf)
    ye = torch.randn(T * top, Wd, **bf)
    rows = torch.randperm(T * top, device=device).to(torch.int32) \
        .view(T, top)
    wts = torch.rand(T, top, **f32)
    hist, one = torch.randn(2, T, Wd, **f32), torch.ones(1, **f32)
    for n, tail in ((T, ""), (batch, f", {batch} rows (decode)")):
        xn, yn = x[:n], ya[:n]
        add(f"join_norm{tail}",
            lambda: hops.join_norm_(xn, yn, None, wn, 1e-6), n * Wd * 12,
            "GB/s")
        rn = rows[:n] % (n * top)
        add(f"join_norm + experts{tail}",
            lambda: hops.join_norm_(xn, yn, (ye, rn, wts[:n]), wn, 1e-6),
            n * Wd * (12 + 2 * top), "GB/s")
        hn = hist[:, :n].contiguous()
        add(f"depth_mix_norm level 1 (nikedra){tail}",
            lambda: hops.depth_mix_norm(
                hn[0], hn, 1, yn, None, None, None, 1.0, yn, one.expand(2)
                .contiguous(), one, None, 1e-6, torch.bfloat16, xn),
            n * Wd * 20, "GB/s")
        add(f"norm_residual_add + next norm (gararax){tail}",
            lambda: hops.norm_residual_add_(xn, yn, wn, 1e-6, torch.bfloat16,
                                            wn), n * Wd * 12, "GB/s")
    add("moe_combine (pugovik)", lambda: hops.moe_combine(ye, rows, wts, T),
        T * Wd * (2 * top + 4), "GB/s")
    # ---- gates ------------------------------------------------------------------
    gu = torch.randn(T, 2 * ff + 16, **bf)
    yo = torch.empty(T, Wd + ff, **bf)
    add("glu_rows gelu", lambda: hops.glu_rows(
        gu[:, :ff], gu[:, ff:2 * ff], yo[:, Wd:], gelu=True), T * ff * 6,
        "GB/s")
    sf = moe["shared"]["ff"]
    add("glu_rows silu + row gate", lambda: hops.glu_rows(
        gu[:, :sf], gu[:, sf:2 * sf], yo[:, Wd:Wd + sf], gelu=False,
        row_gate=gu[:, 2 * sf:2 * sf + 1]), T * sf * 6, "GB/s")
    g2 = torch.randn(T, 2 * ff, **bf)
    add("gelu_tanh_mul (tosipel)", lambda: hops.gelu_tanh_mul(g2), T * ff * 6,
        "GB/s")
    # ---- router -----------------------------------------------------------------
    r = moe["router"]
    h, wr = torch.randn(T, Wd, **bf), torch.randn(r["experts"], Wd, **f32)
    gr = r["groups"]
    add("moe_route with scale", lambda: hops.moe_route(
        h, wr, r["top"], gr["count"], gr["keep"], scale=r["scale"]), T,
        "Mtok/s")
    # ---- one output GEMM for mixer and feed-forward vs two ------------------------
    wo, wd = torch.randn(Wd, Wd, **bf), torch.randn(Wd, ff, **bf)
    wj = torch.cat([wo, wd], 1).contiguous()
    for n, tail in ((T, "prefill"), (batch, f"{batch} rows")):
        yj = torch.randn(n, Wd + ff, **bf)
        y1, y2 = yj[:, :Wd].contiguous(), yj[:, Wd:].contiguous()
        fl = 2.0 * n * Wd * (Wd + ff)
        add(f"joint output GEMM, {tail}", lambda: F.linear(yj, wj), fl,
            "TFLOP/s")
        add(f"two output GEMMs, {tail}",
            lambda: (F.linear(y1, wo), F.linear(y2, wd)), fl, "TFLOP/s")
    return out


def run_hybrid_mode(args, device):
    assert torch.cuda.is_available(), "hybrid mode measures the HIP path"
    kernels = _hybrid_kernels
    fams = ("pugovik", "llama")
    if args.hybrid_family == "dunusun":
        kernels = _dunusun_kernels
        fams = ("dunusun", "pugovik", "llama")
    if args.hybrid_family == "tosipel":
        kernels = _tosipel_kernels
        fams = ("tosipel", "dunusun", "llama")
    if args.hybrid_family == "gararax":
        kernels = _gararax_kernels
        fams = ("gararax", "tosipel", "pugovik", "llama")
    if args.hybrid_family == "nikedra":
        kernels = _nikedra_kernels
        fams = ("nikedra", "tosipel", "dunusun", "pugovik", "llama")
    if args.hybrid_family == "zokanex":
        kernels = _zokanex_kernels
        fams = ("zokanex", "gararax", "pugovik", "nikedra", "llama")
    for size in args.hybrid_sizes.split(","):
        T, batch, ctx = 4096, 32, 2048
        for name, t, rate, unit in kernels(size, device, T, batch, ctx):
            print(json.dumps(dict(kind="kernel", size=size, kernel=name,
                                  ms=round(t * 1e3, 4), rate=round(rate, 2),
                                  unit=unit, tokens=T, batch=batch, ctx=ctx)),
                  flush=True)
        for fam in fams:
            pre, dec = _hybrid_end_to_end(f"{fam}-{size}", device, T, batch,
                                          1024, args.steps)
            print(json.dumps(dict(kind="end_to_end", model=f"{fam}-{size}",
                                  prefill_tok_s=round(pre, 1),
                                  prefill_len=T,
                                  decode_tok_s=round(dec, 1), batch=batch,
                                  ctx=1024, dtype="bf16",
                                  data="synthetic")), flush=True)


# --------------------------------------------------------------------------
# engine mode (round-1 closed-loop engine-step microbench)
# --------------------------------------------------------------------------
def run_engine_mode(args, rank, world, local_rank, use_gpu, dist, device,
                    model_name):
    from xllm_service_amd.engine.engine import LLMEngine
    from xllm_service_amd.engine.sampling import SamplingParams
    from xllm_service_amd.models.config import get_config

    cfg = get_config(model_name)
    eng = LLMEngine(model_name, device=device,
                    max_num_seqs=args.concurrency * 2,
                    max_batched_tokens=args.max_batched_tokens,
                    max_kv_blocks=None if use_gpu else 4096,
                    seed=0)
    torch.manual_seed(1234 + rank)
    rid = 0

    def feed(n):
        nonlocal rid
        for _ in range(n):
            prompt = torch.randint(0, cfg.vocab_size,
                                   (args.input_len,)).tolist()
            eng.add_request(f"r{rank}-{rid}", prompt,
                            SamplingParams(max_tokens=args.output_len,
                                           ignore_eos=True))
            rid += 1

    feed(args.concurrency)

    def one_step():
        outs = eng.step()
        done = sum(1 for o in outs if o.finished)
        if done:
            feed(done)
        return sum(len(o.new_token_ids) for o in outs)

    for _ in range(args.warmup):
        one_step()
    if dist:
        dist.barrier()
    if use_gpu:
        torch.cuda.synchronize()
    t0 = time.perf_counter()
    generated = 0
    for _ in range(args.steps):
        generated += one_step()
    if use_gpu:
        torch.cuda.synchronize()
    if dist:
        dist.barrier()
    t1 = time.perf_counter()
    elapsed = t1 - t0
    if dist:
        te = torch.tensor([elapsed], dtype=torch.float64)
        dist.all_reduce(te, op=dist.ReduceOp.MAX)
        elapsed = float(te.item())
        tg = torch.tensor([float(generated)], dtype=torch.float64)
        dist.all_reduce(tg, op=dist.ReduceOp.SUM)
        generated = int(tg.item())
    n_gpus = world if world > 1 else (1 if use_gpu else args.gpus)
    if rank == 0:
        print(json.dumps({
            "metric": "engine-step throughput (out tok/s, closed loop, "
                      "no serving stack), Llama-3-8B",
            "value": round(generated / elapsed, 2),
            "unit": "tok/s", "n_gpus": n_gpus,
            "steps": args.steps, "warmup": args.warmup,
            "ms_per_step": round(elapsed / args.steps * 1000, 3),
            "higher_is_better": True, "scaling": "weak",
            "vs_baseline": None,
            "dtype": "bf16" if use_gpu else "fp32", "data": "synthetic",
            "config": {"model": model_name,
                       "global_batch": args.concurrency * n_gpus,
                       "seq_len": args.input_len + args.output_len,
                       "input_len": args.input_len,
                       "output_len": args.output_len,
                       "parallelism": f"dp{n_gpus}"},
        }))


# --------------------------------------------------------------------------
# serving mode helpers
# --------------------------------------------------------------------------
def free_port():
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        return s.getsockname()[1]


def topology(n: int):
    """Instance role per rank."""
    if n <= 1:
        return ["DEFAULT"]
    n_p = max(1, n // 4)
    return ["PREFILL"] * n_p + ["DECODE"] * (n - n_p)


def spawn_worker(args, name, itype, device, registry_port, log_path,
                 model_name):
    cmd = [sys.executable, "-m", "xllm_service_amd.engine.worker",
           "--name", name, "--type", itype, "--model", model_name,
           "--registry-host", "127.0.0.1",
           "--registry-port", str(registry_port),
           "--max-batched-tokens", str(args.max_batched_tokens),
           "--push-interval-ms", str(args.push_interval_ms),
           "--seed", "0"]
    if device:
        cmd += ["--device", device]
    if args.max_kv_blocks:
        cmd += ["--max-kv-blocks", str(args.max_kv_blocks)]
    logf = open(log_path, "wb")
    return subprocess.Popen(cmd, cwd=ROOT, stdout=logf,
                            stderr=subprocess.STDOUT), logf


class Completions:
    """Completion log + exact K-step timing. Only open-loop ("poisson")
    requests count as steps — the closed-loop ramp burst has queued-up
    TTFTs by construction and its stragglers complete in bursts."""

    def __init__(self):
        self.records = []          # (t_end, ttft_s, out_tokens, tag, hdr)
        self.durations = []        # completed request wall time
        self.phase_count = 0
        self.k = None
        self.t1 = None
        self.event = asyncio.Event()

    def arm(self, k):
        self.phase_count, self.k, self.t1 = 0, k, None
        self.event = asyncio.Event()
        if k <= 0:
            self.t1 = time.monotonic()
            self.event.set()

    def on_complete(self, t, ttft, ntok, tag, t_hdr=0.0, dur=0.0):
        self.records.append((t, ttft, ntok, tag, t_hdr))
        if dur > 0:
            self.durations.append(dur)
        if self.k is not None and self.t1 is None and tag == "poisson":
            self.phase_count += 1
            if self.phase_count >= self.k:
                self.t1 = t
                self.event.set()



# --------------------------------------------------------------------------
# load-generator child process (no torch; driven over stdin/stdout).
# A single asyncio loop cannot parse tens of thousands of SSE chunks per
# second AND issue new requests on time — measured client-side TTFT then
# includes loadgen queueing, not serving latency. So the load is spread
# over M light processes; completions stream back as DONE lines
# (CLOCK_MONOTONIC is system-wide on Linux, so child timestamps are
# directly comparable in the parent).
# --------------------------------------------------------------------------
def loadgen_child_main():
    import httpx
    cfg = json.loads(os.environ["BENCH_LOADGEN_CFG"])

    async def run():
        client = httpx.AsyncClient(
            base_url=f"http://127.0.0.1:{cfg['http_port']}", timeout=600.0,
            limits=httpx.Limits(max_connections=2048,
                                max_keepalive_connections=2048))
        rnd = random.Random(cfg["seed"])
        ramping = {"on": False}
        quit_ev = asyncio.Event()
        tasks = []

        async def one_request(tag):
            prompt = [rnd.randrange(10, cfg["vocab_hi"])
                      for _ in range(cfg["input_len"])]
            t0 = time.monotonic()
            ttft = None
            t_hdr = None
            try:
                async with client.stream("POST", "/v1/completions", json={
                        "model": cfg["model"], "prompt": prompt,
                        "max_tokens": cfg["output_len"],
                        "temperature": 0.0, "ignore_eos": True,
                        "stream": True}) as resp:
                    t_hdr = time.monotonic() - t0
                    if resp.status_code != 200:
                        return
                    async for line in resp.aiter_lines():
                        if ttft is None and line.startswith("data: ") \
                                and "[DONE]" not in line:
                            ttft = time.monotonic() - t0
            except (httpx.HTTPError, OSError):
                return
            if ttft is not None:
                t1 = time.monotonic()
                print(f"DONE {t1:.4f} {ttft:.4f} "
                      f"{cfg['output_len']} {tag} {t_hdr:.4f} "
                      f"{t1 - t0:.4f}", flush=True)

        async def ramp_client(stagger):
            await asyncio.sleep(rnd.uniform(0, stagger))
            while ramping["on"]:
                await one_request("ramp")

        async def poisson(rate):
            while not quit_ev.is_set():
                tasks.append(asyncio.create_task(one_request("poisson")))
                await asyncio.sleep(rnd.expovariate(rate))

        loop = asyncio.get_event_loop()
        while True:
            line = await loop.run_in_executor(None, sys.stdin.readline)
            if not line:
                break
            parts = line.split()
            if not parts:
                continue
            if parts[0] == "ramp":
                ramping["on"] = True
                stag = float(parts[2]) if len(parts) > 2 else 0.0
                for _ in range(int(parts[1])):
                    tasks.append(asyncio.create_task(ramp_client(stag)))
            elif parts[0] == "stopramp":
                ramping["on"] = False
            elif parts[0] == "poisson":
                tasks.append(asyncio.create_task(poisson(float(parts[1]))))
            elif parts[0] == "quit":
                break
        quit_ev.set()
        ramping["on"] = False
        for t in tasks:
            t.cancel()
        await asyncio.gather(*tasks, return_exceptions=True)
        await client.aclose()

    asyncio.run(run())


def summarize_window(records, t0, t1, slo_s, rate, output_len):
    """Pure window math for the serving record (unit-tested): SLO-gated
    goodput capped at the offered load, raw window rate, TTFT percentiles.
    records: (t_end, ttft_s, out_tokens, tag, hdr_s)."""
    window = [r for r in records if t0 <= r[0] <= t1 and r[3] == "poisson"]
    elapsed = max(t1 - t0, 1e-3)
    offered = rate * output_len
    good = sum(r[2] for r in window if r[1] <= slo_s) / elapsed
    alltok = sum(r[2] for r in window) / elapsed
    ttfts = sorted(r[1] for r in window)
    p50 = ttfts[len(ttfts) // 2] * 1000 if ttfts else 0.0
    p99 = ttfts[int(len(ttfts) * 0.99)] * 1000 if ttfts else 0.0
    hdrs = sorted(r[4] for r in window)
    p50h = hdrs[len(hdrs) // 2] * 1000 if hdrs else 0.0
    return dict(value=min(good, offered), total=min(alltok, offered),
                window_raw=alltok, offered=offered, p50_ttft_ms=p50,
                p99_ttft_ms=p99, p50_headers_ms=p50h, n=len(window))


def _parse_prom(text: str) -> dict:
    vals = {}
    for line in text.splitlines():
        if line.startswith("#") or " " not in line:
            continue
        name, _, v = line.rpartition(" ")
        try:
            vals[name] = float(v)
        except ValueError:
            pass
    return vals


async def run_serving_rank0(args, world, dist, use_gpu, model_name,
                            barrier, my_worker_device):
    import httpx

    http_port = free_port()
    rpc_port = free_port()
    registry_port = free_port()
    os.makedirs("gpurun_out", exist_ok=True)
    # the master runs in its own process (real deployment shape; keeps the
    # load generator's event loop out of the serving path)
    mlog = open("gpurun_out/bench_master.log", "wb")
    mproc = subprocess.Popen(
        [sys.executable, "-m", "xllm_service_amd.service.master",
         "--http-host", "127.0.0.1", "--http-port", str(http_port),
         "--rpc-port", str(rpc_port), "--registry-port", str(registry_port),
         "--model-id", model_name, "--policy", args.policy],
        cwd=ROOT, stdout=mlog, stderr=subprocess.STDOUT)

    roles = topology(max(world, 1))
    n_total = len(roles)
    if world > 1:
        # ship the registry address to the other ranks (they spawn their
        # own worker subprocess against it)
        await asyncio.get_event_loop().run_in_executor(
            None, dist.broadcast_object_list,
            [("127.0.0.1", registry_port)], 0)

    proc = logf = None
    client = httpx.AsyncClient(
        base_url=f"http://127.0.0.1:{http_port}", timeout=600.0,
        limits=httpx.Limits(max_connections=4096,
                            max_keepalive_connections=4096))

    async def prom() -> dict:
        try:
            r = await client.get("/metrics")
            return _parse_prom(r.text)
        except (httpx.HTTPError, OSError):
            return {}

    try:
        deadline = time.monotonic() + args.startup_timeout
        while not await prom():            # master HTTP up
            if mproc.poll() is not None or time.monotonic() > deadline:
                raise RuntimeError("master process did not come up; tail:\n"
                                   + open("gpurun_out/bench_master.log",
                                          "rb").read()[-4000:].decode(
                                              errors="replace"))
            await asyncio.sleep(0.5)
        proc, logf = spawn_worker(
            args, f"{roles[0].lower()}-0", roles[0], my_worker_device,
            registry_port, "gpurun_out/bench_worker_r0.log", model_name)

        def n_instances(m):
            return sum(v for k, v in m.items()
                       if k.startswith("cluster_schedulable_instances"))

        while True:
            m = await prom()
            if n_instances(m) >= n_total:
                break
            if proc.poll() is not None:
                raise RuntimeError(
                    "worker died; tail:\n" + open(
                        "gpurun_out/bench_worker_r0.log",
                        "rb").read()[-4000:].decode(errors="replace"))
            if time.monotonic() > deadline:
                raise TimeoutError(
                    f"{n_instances(m)}/{n_total} workers registered "
                    "before timeout")
            await asyncio.sleep(0.5)
        await asyncio.sleep(1.0)   # let P<->D links settle
        await barrier()            # B1: cluster up

        comp = Completions()
        vocab_hi = 120000 if "8b" in model_name else 400
        n_decode = sum(1 for r in roles if r != "PREFILL") or 1
        conc = args.concurrency * n_decode

        # spawn the load-generator children (see loadgen_child_main)
        n_lg = max(2, 2 * n_decode)
        lg_env = dict(os.environ, BENCH_LOADGEN="1")
        children = []
        lg_logs = []
        for i in range(n_lg):
            lg_env["BENCH_LOADGEN_CFG"] = json.dumps(dict(
                http_port=http_port, model=model_name,
                input_len=args.input_len, output_len=args.output_len,
                vocab_hi=vocab_hi, seed=1000 + i))
            lf = open(f"gpurun_out/bench_loadgen_{i}.log", "wb")
            lg_logs.append(lf)
            children.append(subprocess.Popen(
                [sys.executable, os.path.abspath(__file__)],
                cwd=ROOT, env=dict(lg_env), stdin=subprocess.PIPE,
                stdout=subprocess.PIPE, stderr=lf))

        def cmd_all(line_fmt, *per_child):
            for i, ch in enumerate(children):
                vals = [pc[i] for pc in per_child]
                ch.stdin.write((line_fmt.format(*vals) + "\n").encode())
                ch.stdin.flush()

        async def reader(ch):
            loop = asyncio.get_event_loop()
            while True:
                line = await loop.run_in_executor(None, ch.stdout.readline)
                if not line:
                    return
                if line.startswith(b"DONE"):
                    parts = line.split()
                    comp.on_complete(float(parts[1]), float(parts[2]),
                                     int(parts[3]), parts[4].decode(),
                                     float(parts[5]) if len(parts) > 5
                                     else 0.0,
                                     float(parts[6]) if len(parts) > 6
                                     else 0.0)

        from concurrent.futures import ThreadPoolExecutor
        asyncio.get_event_loop().set_default_executor(
            ThreadPoolExecutor(max_workers=n_lg + 8))
        readers = [asyncio.create_task(reader(ch)) for ch in children]

        # ---- phase A: closed-loop ramp + capacity calibration ----------
        ramp_s = args.ramp_s or (8.0 if use_gpu else 2.0)
        shares = [conc // n_lg + (1 if i < conc % n_lg else 0)
                  for i in range(n_lg)]
        # stagger ramp starts so the first generation of closed-loop
        # requests doesn't complete as one synchronized bunch (which
        # makes the ramp->Poisson handover oscillate for many request
        # durations)
        cmd_all("ramp {} {}", shares, [ramp_s] * n_lg)

        async def gen_tokens():
            return (await prom()).get("generated_tokens_total", 0.0)

        async def active_now():
            return (await prom()).get("server_active_requests", 0.0)

        while await active_now() < 0.9 * conc:    # ramp fully started
            await asyncio.sleep(0.5)
            if time.monotonic() > deadline:
                raise TimeoutError("ramp never filled")
        await asyncio.sleep(2.0)
        c0, tA = await gen_tokens(), time.monotonic()
        await asyncio.sleep(ramp_s)
        cap_tok_s = (await gen_tokens() - c0) / (time.monotonic() - tA)

        rate = args.arrival_rate or max(
            args.pace * cap_tok_s / args.output_len, 0.2)

        # ---- phase B: open-loop Poisson ---------------------------------
        # hand over WITHOUT draining: ramp re-issues stop as Poisson
        # arrivals start, so in-flight stays near steady (~R x D) instead
        # of refilling from empty (a from-empty window under-measures the
        # steady rate for its whole first request-duration)
        cmd_all("stopramp", )
        poisson_t0 = time.monotonic()
        cmd_all("poisson {}", [rate / n_lg] * n_lg)
        d_est = args.output_len * conc / max(cap_tok_s, 1.0)
        settle = poisson_t0 + 1.5 * d_est - time.monotonic()
        if settle > 0:
            await asyncio.sleep(settle)   # ramp residuals gone, B steady
        comp.arm(args.warmup)

        async def wait_or_die(ev):
            while not ev.is_set():
                if any(ch.poll() is not None for ch in children):
                    raise RuntimeError("a load-generator child died")
                if mproc.poll() is not None:
                    raise RuntimeError("master process died")
                if proc.poll() is not None:
                    raise RuntimeError("worker process died")
                try:
                    await asyncio.wait_for(ev.wait(), 5.0)
                except asyncio.TimeoutError:
                    pass

        await wait_or_die(comp.event)    # W completions at steady state

        await barrier()                  # B2
        if use_gpu:
            torch.cuda.synchronize()
        comp.arm(args.steps)
        t0 = time.monotonic()
        await wait_or_die(comp.event)
        t1 = comp.t1
        if use_gpu:
            torch.cuda.synchronize()
        await barrier()                  # B3

        elapsed = max(t1 - t0, 1e-3)   # K completions can share a tick
        if world > 1:
            te = torch.tensor([elapsed], dtype=torch.float64)
            await asyncio.get_event_loop().run_in_executor(
                None, dist.all_reduce, te, dist.ReduceOp.MAX)
            elapsed = float(te.item())

        sm = summarize_window(comp.records, t0, t0 + elapsed,
                              args.slo_ttft_ms / 1000.0, rate,
                              args.output_len)

        n_p = sum(1 for r in roles if r == "PREFILL")
        n_d = len(roles) - n_p
        par = ("colocated-1gpu" if n_total == 1
               else f"pd-{n_p}p{n_d}d")
        print(json.dumps({
            "metric": "SLO-goodput (out tok/s under p50 TTFT SLO), "
                      "Llama-3-8B PD-disagg on 8 MI355X",
            "value": round(sm["value"], 2),
            "unit": "tok/s",
            "n_gpus": n_total,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(elapsed / args.steps * 1000, 3),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": "bf16" if use_gpu else "fp32",
            "data": "synthetic",
            "total_tok_per_s": round(sm["total"], 2),
            "window_tok_per_s": round(sm["window_raw"], 2),
            "offered_tok_per_s": round(sm["offered"], 2),
            "p50_ttft_ms": round(sm["p50_ttft_ms"], 1),
            "p99_ttft_ms": round(sm["p99_ttft_ms"], 1),
            "slo_ttft_ms": args.slo_ttft_ms,
            "arrival_rate_req_s": round(rate, 2),
            "p50_headers_ms": round(sm["p50_headers_ms"], 1),
            "p50_request_s": round(sorted(comp.durations)[
                len(comp.durations) // 2], 2) if comp.durations else 0.0,
            "calibrated_capacity_tok_s": round(cap_tok_s, 1),
            "requests_timed": sm["n"],
            "config": {
                "model": model_name,
                "global_batch": conc,
                "seq_len": args.input_len + args.output_len,
                "input_len": args.input_len,
                "output_len": args.output_len,
                "parallelism": par,
                "stack": "http(uvicorn tcp)+sse -> master proc -> msgrpc "
                         f"-> {n_total} worker proc(s)",
                "policy": args.policy,
                "push_interval_ms": args.push_interval_ms,
            },
        }))
        cmd_all("quit", )
        for rt in readers:
            rt.cancel()
        await asyncio.gather(*readers, return_exceptions=True)
        # debugging artifacts: per-request completions + final master metrics
        try:
            with open("gpurun_out/bench_requests.csv", "w") as f:
                f.write("t_end,ttft_s,tokens,tag\n")
                for r in comp.records:
                    f.write(f"{r[0]:.3f},{r[1]:.3f},{r[2]},{r[3]}\n")
            mtxt = (await client.get("/metrics")).text
            with open("gpurun_out/bench_metrics_after.txt", "w") as f:
                f.write(mtxt)
        except Exception:
            pass
        await barrier()                  # B4: teardown
    finally:
        await client.aclose()
        procs = [proc, mproc] + [c for c in locals().get("children", [])]
        for p in procs:
            if p is not None:
                p.terminate()
        for p in procs:
            if p is not None:
                try:
                    p.wait(timeout=15)
                except subprocess.TimeoutExpired:
                    p.kill()
        for lf in locals().get("lg_logs", []):
            lf.close()
        if logf:
            logf.close()
        mlog.close()


def run_serving_follower(args, rank, dist, use_gpu, model_name):
    """Ranks > 0: host one worker subprocess on this rank's GPU and follow
    the barrier protocol (B1 cluster-up, B2/B3 timing, B4 teardown)."""
    box = [None]
    dist.broadcast_object_list(box, src=0)
    host, registry_port = box[0]
    device = f"cuda:{int(os.environ.get('LOCAL_RANK', rank))}" if use_gpu \
        else "cpu"
    roles = topology(int(os.environ["WORLD_SIZE"]))
    os.makedirs("gpurun_out", exist_ok=True)
    proc, logf = spawn_worker(
        args, f"{roles[rank].lower()}-{rank}", roles[rank], device,
        registry_port, f"gpurun_out/bench_worker_r{rank}.log", model_name)
    try:
        dist.barrier()                   # B1
        dist.barrier()                   # B2
        if use_gpu:
            torch.cuda.synchronize()
        t0 = time.monotonic()
        dist.barrier()                   # B3
        t1 = time.monotonic()
        if use_gpu:
            torch.cuda.synchronize()
        te = torch.tensor([t1 - t0], dtype=torch.float64)
        dist.all_reduce(te, op=dist.ReduceOp.MAX)
        dist.barrier()                   # B4
    finally:
        proc.terminate()
        try:
            proc.wait(timeout=15)
        except subprocess.TimeoutExpired:
            proc.kill()
        logf.close()


def main():
    args = parse_args()
    rank = int(os.environ.get("RANK", "0"))
    world = int(os.environ.get("WORLD_SIZE", "1"))
    local_rank = int(os.environ.get("LOCAL_RANK", str(rank)))

    use_gpu = torch.cuda.is_available() if args.device is None else (
        args.device.startswith("cuda"))
    dist = None
    if world > 1:
        import torch.distributed as dist_mod
        dist = dist_mod
        os.environ.setdefault("MASTER_ADDR", "127.0.0.1")
        # gloo for the benchmark's own barriers/reductions (host-side);
        # the workers' data plane (RCCL / xGMI) is their own. Bounded
        # timeout: a failing rank must not hang the others for 30 min.
        import datetime
        dist.init_process_group(backend="gloo",
                                timeout=datetime.timedelta(seconds=900))
        if use_gpu:
            torch.cuda.set_device(local_rank)

    model_name = args.model
    if not use_gpu:
        # CPU fallback so `python bench.py` runs anywhere; the measured
        # config on GPU is the flagship model.
        if model_name == "llama-3-8b":
            model_name = "llama-tiny"
        if args.input_len == 1024:
            args.input_len = 48
        if args.output_len == 1024:
            args.output_len = 16
        if args.concurrency == 128:
            args.concurrency = 8

    if args.push_interval_ms <= 0:
        r = topology(max(world, 1))
        nd = sum(1 for x in r if x != "PREFILL") or 1
        args.push_interval_ms = 25.0 * max(1.0, nd / 2.0)

    if args.mode == "hybrid":
        run_hybrid_mode(args, args.device or f"cuda:{local_rank}")
    elif args.mode == "engine":
        device = args.device or (f"cuda:{local_rank}" if use_gpu else "cpu")
        run_engine_mode(args, rank, world, local_rank, use_gpu, dist,
                        device, model_name)
    elif rank == 0:
        my_dev = (args.device or
                  (f"cuda:{local_rank}" if use_gpu else "cpu"))

        async def barrier():
            if dist:
                await asyncio.get_event_loop().run_in_executor(
                    None, dist.barrier)

        try:
            asyncio.run(run_serving_rank0(args, world, dist, use_gpu,
                                          model_name, barrier, my_dev))
        except Exception:
            if world > 1:
                raise          # multi-rank: peers are barrier-synced
            # N=1 safety net: a serving-stack failure still yields an
            # HONESTLY-LABELLED record (engine metric string, not the
            # SLO-goodput headline)
            import traceback
            traceback.print_exc(file=sys.stderr)
            print("serving bench failed; falling back to engine mode",
                  file=sys.stderr)
            run_engine_mode(args, rank, world, local_rank, use_gpu, dist,
                            my_dev, model_name)
    else:
        run_serving_follower(args, rank, dist, use_gpu, model_name)

    if dist:
        dist.destroy_process_group()


if __name__ == "__main__":
    if os.environ.get("BENCH_LOADGEN") == "1":
        loadgen_child_main()
    else:
        main()
