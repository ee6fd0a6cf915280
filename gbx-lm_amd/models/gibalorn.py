"""Gibalorn: a decoder-only stack of pre-norm layers with routed experts whose config.json lists its layers one by one.

A layer run:  x += mixer(norm1(x)),  then (unless the layer has no feed-forward)  x += experts(norm2(x)).  Mixer kinds:
``latent_attention`` (keys and values of all heads from one cached latent row per token, queries through a latent of their own, an
output gate per channel) and ``attention`` (grouped-query attention whose values are the key projections before their rotation, one
added to the softmax denominator), both models/sink_attention.py, and ``mamba2`` (state space duality,
models/recurrent_mixers.py:StateSpaceDual).  Feed-forward: experts ``down(relu(up h)^2)`` behind a sigmoid router whose weight
multiplies the expert's INPUT (models/switch_layers.py:DenseRoutedGLU).  Config ``loop`` runs the layers ``start .. stop-1`` ``times``
times in a row with the same weights; every run has a cache of its own, and in front of every pass but the first the embedding rows are
added to the stream again.

Every sublayer boundary is one launch (models/residual.py:layer_update_): the stream's update -- by the mixer's output, or by the sum
of the chosen experts' outputs and, where a pass ends in front of another one, the embedding rows -- and the norm the next sublayer
reads.  Every size and constant is read per layer from the config.  The stream is fp32; matrix products run in the activation dtype
(bf16 as stored, or fp32 when the model is loaded with ``dtype=torch.float32``).
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

import torch
from torch import nn

from ..batching import StepBatch
from .base import BaseModelArgs
from .recurrent_mixers import StateSpaceDual
from .residual import StreamRMSNorm, layer_update_
from .sink_attention import LatentAttention, SharedKeyValueAttention
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
    rot = m.get("rot") or {}
    if kind == "latent_attention":
        if rot.get("dims", m["rot_dim"]) != m["rot_dim"]:
            raise ValueError("Gibalorn: a latent mixer rotates exactly its rot_dim part")
        return LatentAttention(args.width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], rot.get("base", 10000.0), None, m["scale"], eps,
                               sink=False, q_rank=m["q_rank"], interleaved=True, gate_channels=True)
    if kind == "attention":
        if m.get("vdim", m["dim"]) != m["dim"]:
            raise ValueError("Gibalorn: the values of an attention mixer are its keys, so they have one size")
        return SharedKeyValueAttention(args.width, m["heads"], m.get("kv_heads", m["heads"]), m["dim"], rot.get("dims", 0), rot.get("base", 10000.0), m["scale"])
    if kind == "mamba2":
        return StateSpaceDual(args.width, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"], eps)
    raise ValueError(f"Gibalorn: unknown mixer type {kind!r}")


def _routed(args: ModelArgs, spec: Optional[Dict[str, Any]]) -> Optional[DenseRoutedGLU]:
    if spec is None:
        return None
    if spec.get("kind", "moe") != "moe":
        raise ValueError(f"Gibalorn: unknown feed-forward kind {spec.get('kind')!r}")
    return DenseRoutedGLU(args.width, spec["expert"]["ff"], spec["router"]["experts"], spec["router"]["top"], scoring="sigmoid", activation="relu2",
                          weigh_input=True, corrected=False)


class Layer(nn.Module):
    def __init__(self, args: ModelArgs, spec: Dict[str, Any]):
        super().__init__()
        self.norm1 = StreamRMSNorm(args.width, args.norm["eps"])
        self.mixer = _mixer(args, spec)
        self.routed = _routed(args, spec.get("mlp"))
        self.norm2 = None if self.routed is None else StreamRMSNorm(args.width, args.norm["eps"])

    def forward(self, x: torch.Tensor, h: torch.Tensor, batch: StepBatch, cache, next_norm: Optional[StreamRMSNorm],
                extra: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        """``h`` = this layer's norm1 of the fp32 stream ``x``.  Updates ``x`` in place, adds ``extra`` (rows that join the stream behind this
        run) and returns the next run's norm of the result, or None without ``next_norm``."""
        y = self.mixer(h, batch, cache)
        if self.routed is None:
            return layer_update_(x, y, None, None, next_norm, extra=extra)
        cand, _ = self.routed(layer_update_(x, y, None, None, self.norm2))
        return layer_update_(x, None, cand, None, next_norm, extra=extra)


class GibalornModel(nn.Module):
    def __init__(self, args: ModelArgs):
        super().__init__()
        self.embed_tokens = nn.Embedding(args.vocab, args.width)
        self.embed_tokens.weight.requires_grad_(False)
        self.layers = nn.ModuleList(Layer(args, spec) for spec in args.layers)
        self.norm = StreamRMSNorm(args.width, args.norm["eps"])

    def embed(self, tokens: torch.Tensor, keep: bool) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
        """(fp32 stream [T, W], the rows once more in the activation dtype if they are to be kept)."""
        w = self.embed_tokens.weight
        rows = torch.empty((tokens.numel(), w.shape[1]), dtype=w.dtype, device=w.device) if keep else None
        if tokens.is_cuda:
            from .. import mixer_ops as M
            return M.embed_scaled(w, tokens, 1.0, image=rows if keep else False)[0], rows
        if keep:
            rows.copy_(w[tokens])
        return w[tokens].float(), rows


class Model(RaggedStepModel):
    def __init__(self, args: ModelArgs):
        super().__init__(args)
        self.model = GibalornModel(args)
        self._runs = []                                               # (layer, the embedding joins the stream in front of this run)
        entered = False
        for i, enters in loop_runs(len(args.layers), args.loop):
            self._runs.append((i, enters and entered))
            entered = entered or enters

    @property
    def layer_runs(self) -> List[int]:
        return [i for i, _ in self._runs]

    def forward_tokens(self, tokens: torch.Tensor, batch: StepBatch, caches) -> torch.Tensor:
        """One ragged step: tokens [T] -> fp32 stream [T, width] after the last layer run.  Positions are NOT advanced here."""
        layers, runs = self.model.layers, self._runs
        x, rows = self.model.embed(tokens, any(again for _, again in runs))
        h = layers[runs[0][0]].norm1(x, self.lm_head.weight.dtype) if runs else None
        for n, ((i, _), cache) in enumerate(zip(runs, caches)):
            after, again = runs[n + 1] if n + 1 < len(runs) else (None, False)
            norm = None if after is None else layers[after].norm1
            if self.trace_layers is None or not again:
                h = layers[i](x, h, batch, cache, norm, rows if again else None)
                if self.trace_layers is not None:
                    self.trace_layers.append(x.clone())
            else:                                                     # the trace holds the stream before the embedding joins it
                layers[i](x, h, batch, cache, None, None)
                self.trace_layers.append(x.clone())
                h = layer_update_(x, rows, None, None, norm)
        return x

    def sanitize(self, weights: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
        """Checkpoint names -> module paths.  Matrices that read the same input are stacked, experts too; what only enters 32-bit arithmetic
        (norms, router, biases, rates) becomes fp32; tables the modules computed from the config are kept as they are."""
        out: Dict[str, torch.Tensor] = {}
        f32 = lambda t: t.float()
        out["model.embed_tokens.weight"] = weights["embed"]
        out["model.norm.weight"] = f32(weights["final.norm"])
        out["lm_head.weight"] = weights["head"]
        for i, spec in enumerate(self.args.layers):
            p, t = f"l{i}.", f"model.layers.{i}."
            layer = self.model.layers[i]
            mixer, m, to = layer.mixer, p + "mix.", t + "mixer."
            out[t + "norm1.weight"] = f32(weights[p + "norm1"])
            if spec["type"] == "latent_attention":
                fused = mixer.fuse_weights(weights[m + "dq"], weights[m + "dkv"], weights[m + "g"], weights[m + "uk"], weights[m + "uv"])
                out.update({to + k: v for k, v in fused.items()})
                out[to + "uq.weight"] = weights[m + "uq"]
                out[to + "q_norm"], out[to + "latent_norm"], out[to + "freq"] = f32(weights[m + "dq.norm"]), f32(weights[m + "dkv.norm"]), mixer.freq
            elif spec["type"] == "attention":
                out[to + "inp.weight"] = mixer.fuse_weights(weights[m + "q"], weights[m + "k"])
                out[to + "freq"], out[to + "sink"] = mixer.freq, mixer.sink
            else:
                inp = torch.zeros(mixer.inp.weight.shape, dtype=weights[m + "in"].dtype, device=weights[m + "in"].device)
                inp[:weights[m + "in"].shape[0]] = weights[m + "in"]
                out[to + "inp.weight"], out[to + "conv"] = inp, weights[m + "conv"].t().contiguous()
                out[to + "conv_bias"], out[to + "dt_bias"] = f32(weights[m + "conv.b"]), f32(weights[m + "dt_bias"])
                out[to + "rate"], out[to + "skip"] = torch.exp(f32(weights[m + "A_log"])), f32(weights[m + "D"])
                out[to + "out_norm"] = f32(weights[m + "norm"])
            out[to + "o.weight"] = weights[m + "o"]
            if layer.routed is not None:
                f, n_e = p + "mlp.", layer.routed.num_experts
                out[t + "norm2.weight"] = f32(weights[p + "norm2"])
                out[t + "routed.router"] = f32(weights[f + "router"])
                out[t + "routed.gate_up"] = torch.stack([weights[f + f"e{e}.up"] for e in range(n_e)])
                out[t + "routed.down"] = torch.stack([weights[f + f"e{e}.down"] for e in range(n_e)])
        return out
