"""Zokanex: a hybrid decoder on the paged-cache / state-slot engine.

Every layer has ONE norm; its sequence mixer and its optional feed-forward
read the same normed residual and are added to it together:

    h = rms(x) w;   x <- x + mixer(h) + ff(h)          x_0 = scale * embedding

`attention`  grouped heads, weighted RMS norm of every query and key head,
             half-layout rotary positions after it, a sliding window; a layer
             may read the keys and values an earlier layer cached
`retention`  linear attention with one fixed decay per head and rotary
             positions, unit head norm, SiLU gate; fp32 state in a slot

Feed-forwards: dense down(gelu_tanh(gate h) * up h), or routed experts
(sigmoid scores, group limiting by the two best members, raw scores times a
constant as weights) beside a shared expert scaled by one sigmoid number per
token.

Because both sublayers read h, all they read from it comes out of ONE GEMM
(rows [mixer | feed-forward gate | up | shared gate number]; with experts the
feed-forward rows are the shared expert's). Because their outputs are added,
both leave through ONE GEMM as well: the mixer's heads and the feed-forward's
activations are written side by side into one row and the output matrices
stand side by side ([W, heads + ff]), so the sum is formed in the GEMM's fp32
accumulators. The shared expert's number is applied to its activations (the
down-projection is linear). What follows - adding that sum and the weighted
expert outputs to the residual, and the next layer's norm - is one kernel.

fp32: residual, norms, rotary angles, scores and softmax, the retention
recurrence with its turned queries and keys, its state and head norm, router.
Model dtype: GEMMs, gates, activations, cached keys and values.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from xllm_service_amd.engine.metadata import AttnMetadata
from xllm_service_amd.models.config import ZokanexConfig
from xllm_service_amd.models.mixers import GroupedAttention, Retention
from xllm_service_amd.models.moe import RoutedExperts
from xllm_service_amd.ops import hybrid as hops

PAD = 16                    # rows of the input matrix come in such multiples


def _f32(*shape, fill=1.0):
    return nn.Parameter(torch.full(shape, fill, dtype=torch.float32))


def make_mixer(kind: str, m: dict, width: int, eps: float, dtype):
    if kind == "attention":
        return GroupedAttention(
            width, m["heads"], m["kv_heads"], m["dim"], m["vdim"],
            m.get("rot"), False, m["scale"],
            (m.get("mask") or {}).get("size", 0), 0, eps, dtype,
            head_norm=True, kv_from=m.get("kv_from"), project=False)
    if kind == "retention":
        return Retention(width, m["heads"], m["dim"], m["vdim"], m["decay"],
                         m.get("rot"), eps, dtype, project=False)
    raise ValueError(f"unknown mixer type {kind!r}")


class ZokanexBlock(nn.Module):
    def __init__(self, cfg: ZokanexConfig, index: int, dtype):
        super().__init__()
        lc = cfg.layers[index]
        W, eps = cfg.hidden_size, cfg.rms_eps
        self.eps, self.dtype = eps, dtype
        self.norm1 = _f32(W)
        self.mixer = make_mixer(lc.type, lc.mixer, W, eps, dtype)
        self.experts, self.ff = None, 0    # ff: the part inside the two GEMMs
        mlp = lc.mlp
        if mlp is not None and mlp["kind"] == "dense":
            self.ff = int(mlp["ff"])
        elif mlp is not None:
            r = mlp["router"]
            g = r.get("groups") or {}
            self.experts = RoutedExperts(
                W, mlp["expert"]["ff"], r["experts"], r["top"],
                g.get("count", 1), g.get("keep", 1), dtype,
                scale=r.get("scale", 1.0))
            self.ff = int((mlp.get("shared") or {}).get("ff", 0))
        self.gated = self.experts is not None and self.ff > 0
        self.ff_at = self.mixer.in_width
        self.rows = self.ff_at + 2 * self.ff + int(self.gated)
        self.in_proj = nn.Parameter(torch.zeros(
            -(-self.rows // PAD) * PAD, W, dtype=dtype))
        self.out_proj = nn.Parameter(torch.empty(
            W, self.mixer.o_width + self.ff, dtype=dtype))

    def forward(self, x, h, positions, cache, meta, aux, next_w):
        """x: fp32 residual (updated in place); h: its norm in the model
        dtype. Returns the new residual's norm with next_w."""
        proj = F.linear(h, self.in_proj)
        o, f, at = self.mixer.o_width, self.ff, self.ff_at
        y = torch.empty(h.shape[0], o + f, dtype=h.dtype, device=h.device)
        self.mixer.heads_out(proj, positions, cache, meta, aux, y[:, :o])
        if f:
            hops.glu_rows(
                proj[:, at:at + f], proj[:, at + f:at + 2 * f], y[:, o:],
                gelu=self.experts is None,
                row_gate=proj[:, at + 2 * f:at + 2 * f + 1] if self.gated
                else None)
        routed = self.experts.dispatch(h) if self.experts is not None else None
        return hops.join_norm_(x, F.linear(y, self.out_proj), routed, next_w,
                               self.eps)


class ZokanexForCausalLM(nn.Module):
    def __init__(self, cfg: ZokanexConfig, dtype=torch.bfloat16):
        super().__init__()
        self.cfg, self.dtype = cfg, dtype
        W = cfg.hidden_size
        self.embed = nn.Embedding(cfg.vocab_size, W, dtype=dtype)
        self.blocks = nn.ModuleList(
            [ZokanexBlock(cfg, i, dtype) for i in range(cfg.num_layers)])
        self.final_norm = _f32(W)
        self.lm_head = nn.Parameter(torch.empty(cfg.vocab_size, W,
                                                dtype=dtype))

    def cache_specs(self):
        return [b.mixer.cache_spec() for b in self.blocks]

    # ---- weights -----------------------------------------------------------
    def load_weights(self, tensors: Dict[str, torch.Tensor]) -> None:
        """Checkpoint names: embed, final.norm, head, and per layer l<i>.norm1,
        l<i>.mix.{q,k,v,o} with {q.norm,k.norm} (attention; without k, v,
        k.norm where another layer's keys are read) or g (retention), and
        l<i>.mlp.{gate,up,down} or l<i>.mlp.{router,e<j>.{gate,up,down},
        shared.{gate,up,down,sg}}. Linear weights are [out, in]."""
        used = set()

        def take(name):
            if name not in tensors:
                raise KeyError(f"checkpoint lacks {name!r}")
            used.add(name)
            return tensors[name]

        def put(param, value):
            if tuple(param.shape) != tuple(value.shape):
                raise ValueError(f"shape mismatch: {tuple(value.shape)} "
                                 f"for {tuple(param.shape)}")
            with torch.no_grad():
                param.copy_(value.to(param.dtype))

        put(self.embed.weight, take("embed"))
        put(self.final_norm, take("final.norm"))
        put(self.lm_head, take("head"))
        for i, blk in enumerate(self.blocks):
            p = f"l{i}."
            m, mx, ex = p + "mix.", blk.mixer, blk.experts
            put(blk.norm1, take(p + "norm1"))
            if isinstance(mx, Retention):
                names = "qkvg"
            else:
                names = "q" if mx.kv_from is not None else "qkv"
                put(mx.q_norm, take(m + "q.norm"))
                if mx.k_norm is not None:
                    put(mx.k_norm, take(m + "k.norm"))
            into = [take(m + n) for n in names]
            out = [take(m + "o")]
            if blk.ff:
                f = p + ("mlp." if ex is None else "mlp.shared.")
                into += [take(f + "gate"), take(f + "up")]
                if blk.gated:
                    into.append(take(f + "sg"))
                out.append(take(f + "down"))
            put(blk.in_proj[:blk.rows], torch.cat(into, 0))
            put(blk.out_proj, torch.cat(out, 1))
            if ex is not None:
                f = p + "mlp."
                put(ex.router, take(f + "router"))
                for j in range(ex.experts):
                    e = f"{f}e{j}."
                    ex.load_expert(j, take(e + "up"), take(e + "down"),
                                   take(e + "gate"))
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
                if p.dtype == torch.float32 and p.dim() == 1:
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
        aux = {}
        if meta.num_decode_tokens:
            aux["decode_ctx_lens"] = meta.decode_seq_lens - 1
        eps = self.cfg.rms_eps
        norms = [b.norm1 for b in self.blocks] + [self.final_norm]
        src = (self.embed.weight, input_ids) if inputs_embeds is None \
            else (inputs_embeds, None)
        x, h = hops.embed_norm(*src, self.cfg.embed_scale, norms[0], eps,
                               self.dtype)
        for i, blk in enumerate(self.blocks):
            h = blk(x, h, positions, kv_caches[i], meta, aux, norms[i + 1])
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.lm_head)
