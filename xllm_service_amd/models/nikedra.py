"""Nikedra: a hybrid decoder on the paged-cache / state-slot engine.

Each layer has one sequence mixer — latent attention over a sliding window, a
delta rule with one decay per head and key channel, or chunked softmax
attention beside a selective state space mixer — and an optional feed-forward
that reads the same residual:

    h  = norm1(x);  h <- h + conv(h)                 (short, over time)
    X' = x + mixer(h) + ff(norm2(x))                 kept as X_(i+1)
    x  <- sum_{j <= i+1} dwa_j X_j                   X_0 = normed embedding

The norms divide by the root mean square and multiply by ONE number. Every
layer keeps the convolution's last inputs beside what its mixer keeps. The
results X_j of a step live only inside that step: [layers + 1, tokens, width]
in fp32. One kernel per layer adds the sublayers' outputs (the halves of a
parallel mixer normed on the way), keeps X_(i+1), forms the weighted sum and
writes the next layer's two normed inputs.

Feed-forwards: dense with a clamped gate, g sigmoid(1.702 g) (u + 1) with
g <= limit, |u| <= limit, all projections biased; or routed experts without a
gate (exact GELU) chosen by sigmoid scores that multiply the expert's INPUT.

fp32: residual and layer results, norms, rotary angles, scores and softmax,
decays, both recurrences and their states, router. Model dtype: GEMMs,
convolutions, gates, activations. Everything a mixer reads from its input
comes out of ONE merged projection per layer. The logit scale is folded into
the number of the final norm.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from xllm_service_amd.engine.cache_spec import CacheGroup
from xllm_service_amd.engine.metadata import AttnMetadata
from xllm_service_amd.models.config import NikedraConfig
from xllm_service_amd.models.mixers import (GatedDeltaRule, GroupedAttention,
                                            InputConvolution, LatentAttention,
                                            ParallelMixer,
                                            SelectiveStateSpace)
from xllm_service_amd.models.moe import RoutedExperts
from xllm_service_amd.ops import hybrid as hops

GATE_SLOPE = 1.702          # sigmoid slope of the dense feed-forward's gate
UP_SHIFT = 1.0              # added to its up-projection


def _f32(*shape, fill=1.0):
    return nn.Parameter(torch.full(shape, fill, dtype=torch.float32))


def _window(m: dict) -> int:
    return int((m.get("mask") or {}).get("size", 0))


def make_mixer(kind: str, m: dict, width: int, eps: float, dtype,
               ranks: Dict[str, int]):
    """ranks: inner sizes of the delta layer's two low-rank projections."""
    if kind == "latent_attention":
        return LatentAttention(
            width, m["heads"], m["dim"], m["rot_dim"], m["vdim"],
            m["kv_rank"], m["scale"], m.get("rot"), eps, None, dtype,
            window=_window(m), rot_pairs=False)
    if kind == "channel_delta":
        return GatedDeltaRule(
            width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"],
            eps, dtype, decay_rank=ranks.get("a1", m.get("decay_rank", 16)),
            gate_rank=ranks.get("g1", m.get("gate_rank", 16)),
            gate_silu=False)
    if kind == "parallel":
        L, R = m["left"], m["right"]
        left = GroupedAttention(
            width, L["heads"], L["kv_heads"], L["dim"], L["vdim"],
            L.get("rot"), False, L["scale"], _window(L), 0, eps, dtype,
            head_gated=True, chunked=True, yarn=True)
        right = SelectiveStateSpace(
            width, R["heads"], R["vdim"], R["state"], R["groups"],
            R["norm_groups"], R["conv"], eps, dtype)
        return ParallelMixer(left, right, 0.5, 0.5, normed=width)
    raise ValueError(f"unknown mixer type {kind!r}")


class ClampedGateFF(nn.Module):
    """down(clamped_glu(gate h, up h)), all three biased."""

    def __init__(self, width: int, ff: int, limit: float, dtype):
        super().__init__()
        self.limit = float(limit)
        self.gate_up = nn.Parameter(torch.empty(2 * ff, width, dtype=dtype))
        self.gate_up_b = nn.Parameter(torch.zeros(2 * ff, dtype=dtype))
        self.down = nn.Parameter(torch.empty(width, ff, dtype=dtype))
        self.down_b = nn.Parameter(torch.zeros(width, dtype=dtype))

    def forward(self, h):
        z = F.linear(h, self.gate_up, self.gate_up_b)
        return F.linear(hops.clamped_glu(z, self.limit, GATE_SLOPE, UP_SHIFT),
                        self.down, self.down_b)


class NikedraBlock(nn.Module):
    def __init__(self, cfg: NikedraConfig, index: int, ranks: Dict[str, int],
                 dtype):
        super().__init__()
        lc = cfg.layers[index]
        W, eps = cfg.hidden_size, cfg.rms_eps
        self.eps, self.dtype, self.index = eps, dtype, index
        self.conv = InputConvolution(W, cfg.canon_taps, dtype)
        self.mixer = make_mixer(lc.type, lc.mixer, W, eps, dtype, ranks)
        self.in_proj = nn.Parameter(torch.empty(self.mixer.in_width, W,
                                                dtype=dtype))
        self.norm1 = _f32(1)
        self.dwa = _f32(index + 2)
        self.ff = None
        if lc.mlp is not None:
            self.norm2 = _f32(1)
            if lc.mlp["kind"] == "dense":
                self.ff = ClampedGateFF(W, lc.mlp["ff"], lc.mlp["limit"],
                                        dtype)
            else:
                r = lc.mlp["router"]
                self.ff = RoutedExperts(
                    W, lc.mlp["expert"]["ff"], r["experts"], r["top"], 1, 1,
                    dtype, gated=False, weight_input=True)

    def cache_spec(self):
        return CacheGroup((self.conv.cache_spec(), self.mixer.cache_spec()))

    @property
    def g2(self):
        return self.norm2 if self.ff is not None else None

    def forward(self, x_in, x, hist, h1, h2, positions, cache, meta, aux,
                next_g1, next_g2):
        """x_in: fp32 residual; x: where the new residual goes (may be x_in);
        hist: fp32 layer results; h1/h2: the normed inputs of mixer and
        feed-forward. Returns the new residual's two normed forms."""
        h = self.conv(h1, cache[0], meta, aux)
        y = self.mixer(F.linear(h, self.in_proj), positions, cache[1], meta,
                       aux)
        f = self.ff(h2) if self.ff is not None else None
        m = self.mixer
        if isinstance(y, tuple):
            parts = (y[0], m.left_norm, y[1], m.right_norm, m.scales[0])
        else:
            parts = (y, None, None, None, 1.0)
        return hops.depth_mix_norm(x_in, hist, self.index + 1, *parts, f,
                                   self.dwa, next_g1, next_g2, self.eps,
                                   self.dtype, x)


class NikedraForCausalLM(nn.Module):
    def __init__(self, cfg: NikedraConfig, dtype=torch.bfloat16):
        super().__init__()
        self.cfg, self.dtype = cfg, dtype
        W, n = cfg.hidden_size, cfg.num_layers
        self.embed = nn.Embedding(cfg.vocab_size, W, dtype=dtype)
        self.embed_norm = _f32(1)
        ranks = self._low_ranks(cfg)
        self.blocks = nn.ModuleList(
            [NikedraBlock(cfg, i, ranks.get(i, {}), dtype) for i in range(n)])
        # holds logit_scale * the checkpoint's number
        self.final_norm = _f32(1)
        self.lm_head = nn.Parameter(torch.empty(cfg.vocab_size, W,
                                                dtype=dtype))

    @staticmethod
    def _low_ranks(cfg: NikedraConfig) -> Dict[int, Dict[str, int]]:
        """The inner sizes of the delta layers' low-rank projections are
        tensor shapes, not config entries: read them from the checkpoint
        header when there is one."""
        if not cfg.model_dir:
            return {}
        from xllm_service_amd.models.loader import safetensors_shapes
        shapes = safetensors_shapes(cfg.model_dir)
        return {i: {n: int(shapes[f"l{i}.mix.{n}"][0]) for n in ("a1", "g1")
                    if f"l{i}.mix.{n}" in shapes}
                for i in range(cfg.num_layers)}

    def cache_specs(self):
        return [b.cache_spec() for b in self.blocks]

    # ---- weights -----------------------------------------------------------
    def load_weights(self, tensors: Dict[str, torch.Tensor]) -> None:
        """Checkpoint names: embed, embed.norm, final.norm, head, and per
        layer l<i>.{norm1,norm2,canon1,dwa}, l<i>.mlp.{gate,up,down}(.b) or
        l<i>.mlp.{router,e<j>.{up,down}}, and l<i>.mix.* (latent attention: q,
        dkv, dkv.norm, uk, uv, g, o; channel delta: q, k, v (each with
        .conv), b, a1, a2, g1, g2, A_log, dt_bias, norm, o; parallel:
        left.{q,k,v,g,o,out}, right.{in,conv,conv.b,dt_bias,A_log,D,norm,o,
        out}). Linear weights are [out, in]."""
        used = set()

        def take(name):
            if name not in tensors:
                raise KeyError(f"checkpoint lacks {name!r}")
            used.add(name)
            return tensors[name]

        def put(param, value, times=None):
            if tuple(param.shape) != tuple(value.shape):
                raise ValueError(f"shape mismatch: {tuple(value.shape)} "
                                 f"for {tuple(param.shape)}")
            with torch.no_grad():
                if times is not None:
                    value = value.float() * times
                param.copy_(value.to(param.dtype))

        def number(name):
            return take(name).reshape(1)

        put(self.embed.weight, take("embed"))
        put(self.embed_norm, number("embed.norm"))
        put(self.final_norm, number("final.norm"), self.cfg.logit_scale)
        put(self.lm_head, take("head"))
        for i, blk in enumerate(self.blocks):
            p = f"l{i}."
            m, mx = p + "mix.", blk.mixer
            put(blk.norm1, number(p + "norm1"))
            put(blk.conv.w, take(p + "canon1"))
            put(blk.dwa, take(p + "dwa"))
            if isinstance(mx, LatentAttention):
                put(blk.in_proj, torch.cat([take(m + n)
                                            for n in ("q", "dkv", "g")], 0))
                put(mx.dkv_norm, take(m + "dkv.norm"))
                H, r = mx.heads, mx.kv_rank
                put(mx.w_uk, take(m + "uk").view(H, mx.dim, r))
                put(mx.w_uv_t,
                    take(m + "uv").view(H, mx.vdim, r).transpose(1, 2))
                put(mx.o_proj, take(m + "o"))
            elif isinstance(mx, GatedDeltaRule):
                put(blk.in_proj, torch.cat(
                    [take(m + n) for n in ("q", "k", "v", "g1", "b", "a1")],
                    0))
                put(mx.conv_w, torch.cat(
                    [take(f"{m}{n}.conv") for n in "qkv"], 0))
                put(mx.a2, take(m + "a2"))
                put(mx.g2, take(m + "g2"))
                put(mx.A_log, take(m + "A_log"))
                put(mx.dt_bias, take(m + "dt_bias"))
                put(mx.out_norm, take(m + "norm"))
                put(mx.o_proj, take(m + "o"))
            else:
                lp, rp, R = m + "left.", m + "right.", mx.right
                put(blk.in_proj, torch.cat(
                    [take(lp + n) for n in "qkvg"] + [take(rp + "in")], 0))
                put(mx.left.o_proj, take(lp + "o"))
                put(mx.left_norm, take(lp + "out"))
                put(R.conv_w, take(rp + "conv"))
                put(R.conv_b, take(rp + "conv.b"))
                put(R.dt_bias, take(rp + "dt_bias"))
                put(R.A_log, take(rp + "A_log"))
                put(R.D, take(rp + "D"))
                put(R.out_norm, take(rp + "norm"))
                put(R.o_proj, take(rp + "o"))
                put(mx.right_norm, take(rp + "out"))
            ff, f = blk.ff, p + "mlp."
            if ff is None:
                continue
            put(blk.norm2, number(p + "norm2"))
            if isinstance(ff, ClampedGateFF):
                put(ff.gate_up, torch.cat([take(f + "gate"),
                                           take(f + "up")], 0))
                put(ff.gate_up_b, torch.cat([take(f + "gate.b"),
                                             take(f + "up.b")], 0))
                put(ff.down, take(f + "down"))
                put(ff.down_b, take(f + "down.b"))
            else:
                put(ff.router, take(f + "router"))
                for j in range(ff.experts):
                    ff.load_expert(j, take(f"{f}e{j}.up"),
                                   take(f"{f}e{j}.down"))
        extra = set(tensors) - used
        if extra:
            raise ValueError(f"unused checkpoint tensors: {sorted(extra)[:8]}")

    def random_init(self, seed: int = 0):
        dev = next(self.parameters()).device
        gen = torch.Generator(device=dev).manual_seed(seed)

        def randn(shape):
            return torch.randn(shape, generator=gen, device=dev,
                               dtype=torch.float32)
        with torch.no_grad():
            for name, p in self.named_parameters():
                leaf = name.rsplit(".", 1)[-1]
                if leaf == "dt_bias":
                    p.copy_(-2.0 + 0.5 * randn(p.shape))
                elif leaf == "A_log":
                    p.copy_(-1.0 + 0.5 * randn(p.shape))
                elif leaf in ("conv_w", "w"):
                    p.copy_((randn(p.shape) * 0.4).to(p.dtype))
                elif leaf in ("conv_b", "gate_up_b", "down_b"):
                    p.copy_((0.1 * randn(p.shape)).to(p.dtype))
                elif leaf == "dwa":
                    p.copy_(0.1 * randn(p.shape))
                    p[-1] += 1.0
                elif leaf == "final_norm":
                    p.fill_(self.cfg.logit_scale)
                elif p.dtype == torch.float32 and p.dim() == 1:
                    p.copy_(1.0 + 0.1 * randn(p.shape))
                elif leaf == "weight":                 # embedding table
                    p.copy_(randn(p.shape).to(p.dtype))
                else:
                    # expert matrices are kept [expert, in, out]
                    fan = p.shape[-2 if leaf in ("w_in", "w_down") else -1]
                    p.copy_((randn(p.shape) / math.sqrt(fan)).to(p.dtype))

    # ---- forward -----------------------------------------------------------
    def forward(self, input_ids, positions, kv_caches: List,
                meta: AttnMetadata,
                inputs_embeds: Optional[torch.Tensor] = None):
        e = inputs_embeds if inputs_embeds is not None \
            else self.embed(input_ids)
        T, W = e.shape
        n = len(self.blocks)
        aux = {}
        if meta.num_decode_tokens:
            aux["decode_ctx_lens"] = meta.decode_seq_lens - 1
        hist = torch.empty(n + 1, T, W, dtype=torch.float32, device=e.device)
        x = torch.empty(T, W, dtype=torch.float32, device=e.device)

        def after(i):                    # the norms that read the residual
            if i < n:
                return self.blocks[i].norm1, self.blocks[i].g2
            return self.final_norm, None
        h1, h2 = hops.depth_mix_norm(
            None, hist, 0, e, self.embed_norm, None, None, 1.0, None, None,
            *after(0), self.cfg.rms_eps, self.dtype)
        for i, blk in enumerate(self.blocks):
            h1, h2 = blk(hist[0] if i == 0 else x, x, hist, h1, h2, positions,
                         kv_caches[i], meta, aux, *after(i + 1))
        return h1

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.lm_head)
