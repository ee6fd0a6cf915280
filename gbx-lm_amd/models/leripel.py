"""Leripel: a decoder-only stack of PARALLEL layers with routed experts whose config.json lists its layers one by one.

A layer run reads one RMS norm of the residual stream, ``h = norm1(x)``, feeds it to its mixer and (optionally) its feed-forward, and
adds both outputs together: ``x += mixer(h) + ff(h)``.  Mixer kinds: ``retention`` (linear attention with a fixed decay per head) and
``mamba2`` (state space duality), both models/recurrent_mixers.py, and ``attention`` (grouped-query softmax attention inside chunks,
models/sink_attention.py:ChunkedAttention).  Feed-forward: routed silu experts behind a softmax router with expert groups
(models/switch_layers.py:DenseRoutedGLU), optionally with an expert that every token takes, weighted by a sigmoid per token.  Config
``loop`` runs the layers ``start .. stop-1`` ``times`` times in a row with the same weights; every run has a cache of its own, and in
front of every pass the stream becomes ``W_in [x ; embedding]``.

Everything that reads ``h`` as a matrix product is ONE product: the mixer's projections and the shared expert's gate and up rows; the
shared gate is one more row of the (fp32) router.  Everything that ends in the stream as a matrix product is one product too: the
mixer's context and the shared expert's hidden row (already times its gate) lie side by side in front of ``W_o | W_down``.  The layer
ends in one launch that adds this product and the weighted experts to the stream and forms the next layer's norm
(models/residual.py:layer_update_).  Every size and constant is read per layer from the config.  The stream is fp32; matrix products
run in the activation dtype (bf16 as stored, or fp32 when the model is loaded with ``dtype=torch.float32``).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional

import torch
import torch.nn.functional as F
from torch import nn

from ..batching import StepBatch
from .base import BaseModelArgs
from .feed_forward import glu_
from .recurrent_mixers import Retention, StateSpaceDual
from .residual import StreamRMSNorm, layer_update_
from .sink_attention import ChunkedAttention
from .step_model import RaggedStepModel, loop_runs
from .switch_layers import DenseRoutedGLU


@dataclass
class ModelArgs(BaseModelArgs):
    architecture: str
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, Any]
    loop: Optional[Dict[str, int]] = None

    @property
    def model_type(self) -> str:
        return self.architecture.lower()


def _mixer(args: ModelArgs, spec: Dict[str, Any]) -> nn.Module:
    kind, m, eps = spec["type"], spec["mixer"], args.norm["eps"]
    if kind == "retention":
        return Retention(args.width, m["heads"], m["dim"], m["vdim"], m["decay"], eps, own_projections=False)
    if kind == "mamba2":
        return StateSpaceDual(args.width, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"], eps, own_projections=False)
    if kind == "attention":
        rot = m.get("rot") or {}
        return ChunkedAttention(args.width, m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"], rot.get("dims", 0), rot.get("base", 10000.0),
                                (m.get("mask") or {}).get("size"), m["scale"], own_projections=False)
    raise ValueError(f"Leripel: unknown mixer type {kind!r}")


def _routed(args: ModelArgs, spec: Optional[Dict[str, Any]]) -> Optional[DenseRoutedGLU]:
    if spec is None:
        return None
    if spec.get("kind", "moe") != "moe":
        raise ValueError(f"Leripel: unknown feed-forward kind {spec.get('kind')!r}")
    r, g = spec["router"], spec["router"].get("groups")
    return DenseRoutedGLU(args.width, spec["expert"]["ff"], r["experts"], r["top"], groups=None if not g else (g["count"], g["keep"]),
                          gate_row=bool(spec.get("shared")))


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


class Layer(nn.Module):
    def __init__(self, args: ModelArgs, spec: Dict[str, Any]):
        super().__init__()
        self.norm1 = StreamRMSNorm(args.width, args.norm["eps"])
        self.mixer = _mixer(args, spec)
        self.routed = _routed(args, spec.get("mlp"))
        self.shared_ff = spec["mlp"]["shared"]["ff"] if self.routed is not None and self.routed.gate_row else 0
        self.off_ff = _pad8(self.mixer.ctx_width)                     # the shared expert's hidden row starts here, behind the context
        self.inp = nn.Linear(args.width, _pad8(self.mixer.in_rows + 2 * self.shared_ff), bias=False)
        self.o = nn.Linear(self.off_ff + _pad8(self.shared_ff), args.width, bias=False)
        for p in self.parameters():
            p.requires_grad_(False)

    def forward(self, x: torch.Tensor, h: torch.Tensor, batch: StepBatch, cache, next_norm: Optional[StreamRMSNorm],
                image: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        """``h`` = this layer's norm of the fp32 stream ``x``.  Updates ``x`` in place (and leaves its image in ``image``); returns the next
        run's norm of it if ``next_norm`` is given."""
        t, n, ff = h.shape[0], self.mixer.ctx_width, self.shared_ff
        y = F.linear(h, self.inp.weight)
        full = n % 8 == 0 and ff % 8 == 0                             # no empty channels between the parts
        rows = (torch.empty if full else torch.zeros)((t, self.o.in_features), dtype=h.dtype, device=h.device)
        self.mixer.mix(y[:, :self.mixer.in_rows], batch, cache, rows[:, :n])
        cand = w = None
        if self.routed is not None:
            cand, w = self.routed(h)
        if ff:
            glu_(y[:, self.mixer.in_rows:self.mixer.in_rows + 2 * ff], "silu", row_scale=w[:, self.routed.top], out=rows[:, self.off_ff:self.off_ff + ff])
        return layer_update_(x, F.linear(rows, self.o.weight), cand, w, next_norm, image)


class LeripelModel(nn.Module):
    def __init__(self, args: ModelArgs):
        super().__init__()
        self.embed_tokens = nn.Embedding(args.vocab, args.width)
        self.embed_tokens.weight.requires_grad_(False)
        self.layers = nn.ModuleList(Layer(args, spec) for spec in args.layers)
        self.norm = StreamRMSNorm(args.width, args.norm["eps"])
        if args.loop:
            self.loop_in = nn.Linear(2 * args.width, args.width, bias=False)
            self.loop_in.weight.requires_grad_(False)

    def embed(self, tokens: torch.Tensor, image: Optional[torch.Tensor]) -> torch.Tensor:
        """fp32 [T, W]; ``image`` [T, W] (activation dtype, any row stride) gets the same rows."""
        w = self.embed_tokens.weight
        if tokens.is_cuda:
            from .. import mixer_ops as M
            return M.embed_scaled(w, tokens, 1.0, image=False if image is None else image)[0]
        rows = w[tokens]
        if image is not None:
            image.copy_(rows)
        return rows.float()


class Model(RaggedStepModel):
    def __init__(self, args: ModelArgs):
        super().__init__(args)
        self.model = LeripelModel(args)
        self._runs = loop_runs(len(args.layers), args.loop)

    @property
    def layer_runs(self) -> List[int]:
        return [i for i, _ in self._runs]

    def forward_tokens(self, tokens: torch.Tensor, batch: StepBatch, caches) -> torch.Tensor:
        """One ragged step: tokens [T] -> fp32 stream [T, width] after the last layer run.  Positions are NOT advanced here."""
        layers, runs, width = self.model.layers, self._runs, self.args.width
        dt = self.lm_head.weight.dtype
        pair = None                                                   # x | embedding: the input of the product in front of a pass
        if any(enters for _, enters in runs):
            pair = torch.empty((tokens.numel(), 2 * width), dtype=dt, device=tokens.device)
        x = self.model.embed(tokens, None if pair is None else pair[:, width:])
        h = None
        for n, ((i, enters), cache) in enumerate(zip(runs, caches)):
            layer = layers[i]
            if enters:
                if n == 0:
                    pair[:, :width].copy_(pair[:, width:])
                h = layer_update_(x, F.linear(pair, self.model.loop_in.weight), None, None, layer.norm1, replace=True)
            elif n == 0:
                h = layer.norm1(x, dt)
            after = runs[n + 1] if n + 1 < len(runs) else None
            leaves = after is not None and after[1]                   # a pass starts next: it reads the stream's image, not a norm of it
            h = layer(x, h, batch, cache, None if after is None or leaves else layers[after[0]].norm1, pair[:, :width] if leaves else None)
            if self.trace_layers is not None:
                self.trace_layers.append(x.clone())
        return x

    def sanitize(self, weights: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint names -> module paths.  Matrices that read the same input are stacked, those whose products are added lie side by
        side, experts are stacked; what only enters 32-bit arithmetic (norms, router, temperatures, biases, rates) becomes fp32."""
        out: Dict[str, torch.Tensor] = {}
        f32 = lambda t: t.float()
        out["model.embed_tokens.weight"] = weights["embed"]
        out["model.norm.weight"] = f32(weights["final.norm"])
        out["lm_head.weight"] = weights["head"]
        if self.args.loop:
            out["model.loop_in.weight"] = weights["loop.in"]
        for i, spec in enumerate(self.args.layers):
            p, t = f"l{i}.", f"model.layers.{i}."
            layer = self.model.layers[i]
            mixer, m = layer.mixer, p + "mix."
            out[t + "norm1.weight"] = f32(weights[p + "norm1"])
            if spec["type"] == "mamba2":
                parts = [weights[m + "in"]]
                out[t + "mixer.conv"] = weights[m + "conv"].t().contiguous()
                out[t + "mixer.conv_bias"], out[t + "mixer.dt_bias"] = f32(weights[m + "conv.b"]), f32(weights[m + "dt_bias"])
                out[t + "mixer.rate"], out[t + "mixer.skip"] = torch.exp(f32(weights[m + "A_log"])), f32(weights[m + "D"])
                out[t + "mixer.out_norm"] = f32(weights[m + "norm"])
            else:
                parts = [weights[m + nm] for nm in ("q", "k", "v", "g")]
                if spec["type"] == "retention":
                    out[t + "mixer.decay"] = mixer.decay
                else:
                    out[t + "mixer.freq"], out[t + "mixer.temp"] = mixer.freq, f32(weights[m + "temp"])
            ff, f = layer.shared_ff, p + "mlp."
            inp = torch.zeros(layer.inp.weight.shape, dtype=parts[0].dtype, device=parts[0].device)
            o = torch.zeros(layer.o.weight.shape, dtype=parts[0].dtype, device=parts[0].device)
            rows = torch.cat(parts)
            inp[:rows.shape[0]] = rows
            o[:, :mixer.ctx_width] = weights[m + "o"]
            if ff:
                inp[mixer.in_rows:mixer.in_rows + 2 * ff] = torch.cat([weights[f + "shared.gate"], weights[f + "shared.up"]])
                o[:, layer.off_ff:layer.off_ff + ff] = weights[f + "shared.down"]
            out[t + "inp.weight"], out[t + "o.weight"] = inp, o
            if layer.routed is not None:
                n_e = layer.routed.num_experts
                router = [f32(weights[f + "router"])] + ([f32(weights[f + "shared.sg"])] if ff else [])
                out[t + "routed.router"] = torch.cat(router)
                out[t + "routed.gate_up"] = torch.stack([torch.cat([weights[f + f"e{e}.gate"], weights[f + f"e{e}.up"]]) for e in range(n_e)])
                out[t + "routed.down"] = torch.stack([weights[f + f"e{e}.down"] for e in range(n_e)])
        return out
