"""Dogulorn: a small decoder whose layers mix latent attention (no positions, sliding window, caches shared between
layers) and gated-delta-rule recurrences, with a 32-bit residual stream normed on both sides of every sublayer, a clamped
gated MLP, a token-pair embedding and a per-layer token input.

The configuration (``config.json``) lists the layers one by one; tensor names are ``l<i>.mix.*`` / ``l<i>.mlp.*`` /
``l<i>.side.*`` beside ``embed``, ``bigram``, ``side.embed``, ``final.norm`` and ``head``.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Any, Iterable, Optional, Union

import torch

from . import ops
from .kv_cache import LatentCacheSpec
from .layers import _init_weight, get_forward_context
from .mixers import (ClampedGluMLP, GatedDelta, GatedDeltaConfig, LatentAttention, LatentAttentionConfig, TokenSideInput)
from .state_cache import StateSpec
from .text_model import TokenDecoder

GLU_ALPHA = 1.702       # slope of the gate's sigmoid, fixed by the design


@dataclass
class DogulornLayerConfig:
    mixer: Union[LatentAttentionConfig, GatedDeltaConfig]
    ff: int = 0                       # 0: no feed-forward
    limit: float = 0.0


@dataclass
class DogulornConfig:
    vocab_size: int
    hidden_size: int
    layers: list[DogulornLayerConfig] = field(default_factory=list)
    rms_norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    bigram_buckets: int = 1
    bigram_mul_prev: int = 0
    bigram_mul_cur: int = 0
    token_side_dim: int = 0
    name: str = "dogulorn"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def embedding_size(self) -> int:
        return self.hidden_size

    @classmethod
    def from_dict(cls, d: dict) -> "DogulornConfig":
        layers = []
        for i, entry in enumerate(d["layers"]):
            m, mlp = entry["mixer"], entry.get("mlp")
            if entry["type"] == "latent_attention":
                mask = m.get("mask")
                mixer: Any = LatentAttentionConfig(
                    heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), q_rank=int(m["q_rank"]),
                    kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), window=int(mask["size"]) if mask else None,
                    kv_from=None if m.get("kv_from") is None else int(m["kv_from"]))
            elif entry["type"] == "delta":
                mixer = GatedDeltaConfig(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]),
                                         vdim=int(m["vdim"]), conv=int(m["conv"]))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {entry['type']!r}")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            layers.append(DogulornLayerConfig(mixer, int(mlp["ff"]) if mlp else 0, float(mlp["limit"]) if mlp else 0.0))
        bg = d["embedding"]["bigram"]
        cfg = cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers, rms_norm_eps=float(d["norm"]["eps"]),
                  embedding_scale=float(d["embedding"]["scale"]), bigram_buckets=int(bg["buckets"]),
                  bigram_mul_prev=int(bg["mul_prev"]), bigram_mul_cur=int(bg["mul_cur"]),
                  token_side_dim=int(d["token_side"]["dim"]))
        cfg.validate()
        return cfg

    @classmethod
    def from_json(cls, path: str) -> "DogulornConfig":
        with open(os.path.join(path, "config.json") if os.path.isdir(path) else path) as f:
            return cls.from_dict(json.load(f))

    def validate(self) -> None:
        for i, layer in enumerate(self.layers):
            m = layer.mixer
            if not isinstance(m, LatentAttentionConfig):
                continue
            if m.window is not None and m.window < 1:
                raise ValueError(f"layer {i}: a window holds at least the token itself")
            if m.kv_from is None:
                continue
            src = self.layers[m.kv_from].mixer if 0 <= m.kv_from < i else None
            if not isinstance(src, LatentAttentionConfig) or src.kv_from is not None or src.kv_rank != m.kv_rank:
                raise ValueError(f"layer {i}: kv_from {m.kv_from} is not an earlier latent-attention layer with a cache of its "
                                 "own and the same rank")


class DogulornDecoderLayer:
    def __init__(self, cfg: DogulornConfig, index: int, dtype, device, generator=None):
        lc = cfg.layers[index]
        w, eps = cfg.hidden_size, cfg.rms_norm_eps
        self.eps = eps
        cls = LatentAttention if isinstance(lc.mixer, LatentAttentionConfig) else GatedDelta
        self.mixer = cls(lc.mixer, w, eps, dtype, device, generator)
        self.mlp = ClampedGluMLP(w, lc.ff, lc.limit, GLU_ALPHA, dtype, device, generator) if lc.ff else None
        self.side = TokenSideInput(w, cfg.token_side_dim, index, dtype, device, generator)
        ones = lambda: torch.ones(w, dtype=dtype, device=device)   # noqa: E731
        self.norm1, self.norm1b = ones(), ones()
        self.norm2, self.norm2b = (ones(), ones()) if self.mlp else (None, None)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield p + "norm1", self.norm1
        yield p + "norm1b", self.norm1b
        if self.mlp:
            yield p + "norm2", self.norm2
            yield p + "norm2b", self.norm2b
            yield from self.mlp.named_weights(p + "mlp.")
        yield from self.mixer.named_weights(p + "mix.")
        yield from self.side.named_weights(p + "side.")

    def __call__(self, x: torch.Tensor, h: torch.Tensor, md, side_table: torch.Tensor, ids: torch.Tensor, next_norm: torch.Tensor):
        """x: the fp32 stream, updated in place; h: its pre-norm for the mixer.  Returns the pre-norm of what follows."""
        y = self.mixer(h, md, True)
        h = ops.residual_norm(x, y, self.norm1b, self.norm2, self.eps)
        if self.mlp:
            h = ops.residual_norm(x, self.mlp(h, True), self.norm2b, None, self.eps)
        return ops.residual_norm(x, self.side(h, side_table, ids, True), self.side.norm, next_norm, self.eps)


class DogulornForCausalLM(TokenDecoder):
    """Takes token ids (and each request's state slot) from the step's metadata; returns final-normed hidden rows."""

    def __init__(self, cfg: DogulornConfig, dtype=torch.bfloat16, device=None, seed: Optional[int] = 0):
        super().__init__(cfg, dtype, device)
        gen = self.generator(seed)
        w, v = cfg.hidden_size, cfg.vocab_size
        self.embed = _init_weight(v, w, dtype, device, gen, std=1.0)
        self.bigram = _init_weight(cfg.bigram_buckets + 1, w, dtype, device, gen, std=1.0)
        self.side_embed = _init_weight(v, cfg.num_hidden_layers * cfg.token_side_dim, dtype, device, gen, std=1.0)
        self.layers = [DogulornDecoderLayer(cfg, i, dtype, device, gen) for i in range(cfg.num_hidden_layers)]
        self.final_norm = torch.ones(w, dtype=dtype, device=device)
        self.head = _init_weight(v, w, dtype, device, gen, std=w ** -0.5)
        self.last_token: Optional[torch.Tensor] = None

    # ---- caches -------------------------------------------------------------------
    def kv_cache_specs(self, block_size: int) -> dict[int, LatentCacheSpec]:
        """layer -> its cache; layers that read another layer's cache have none"""
        specs = {}
        for i, layer in enumerate(self.layers):
            if isinstance(layer.mixer, LatentAttention) and layer.mixer.cfg.kv_from is None:
                specs[i] = layer.mixer.kv_cache_spec(block_size)
        return specs

    def bind_kv_caches(self, caches: dict[int, torch.Tensor]) -> None:
        for i, layer in enumerate(self.layers):
            if isinstance(layer.mixer, LatentAttention):
                src = layer.mixer.cfg.kv_from
                layer.mixer.cache = caches[i if src is None else src]

    def prefill_windows(self) -> list[int]:
        """windows of the layers whose prompt attention runs on a gathered context"""
        return sorted({layer.mixer.window for layer in self.layers if isinstance(layer.mixer, LatentAttention)})

    def state_specs(self) -> list[StateSpec]:
        specs = [StateSpec((), torch.int64)]          # the previous token
        for layer in self.layers:
            if isinstance(layer.mixer, GatedDelta):
                specs.extend(layer.mixer.state_specs())
        return specs

    def bind_states(self, tensors: list[torch.Tensor]) -> None:
        it = iter(tensors)
        self.last_token = next(it)
        for layer in self.layers:
            if isinstance(layer.mixer, GatedDelta):
                layer.mixer.bind_state(next(it), next(it))

    @property
    def is_recurrent(self) -> bool:
        return any(isinstance(layer.mixer, GatedDelta) for layer in self.layers)

    # ---- forward --------------------------------------------------------------------
    def forward(self, input_ids=None, positions=None, intermediate_tensors=None, inputs_embeds=None, **kwargs):
        cfg, md = self.config, get_forward_context().attn_metadata
        if input_ids is None or md is None:
            raise ValueError("token ids and the step's metadata are required")
        x, h = ops.pair_embed_norm(self.embed, self.bigram, self.layers[0].norm1, input_ids, md.prev_ids, md.prev_slots,
                                   self.last_token, positions, cfg.embedding_scale, cfg.bigram_mul_prev, cfg.bigram_mul_cur,
                                   cfg.rms_norm_eps)
        for i, layer in enumerate(self.layers):
            nxt = self.layers[i + 1].norm1 if i + 1 < len(self.layers) else self.final_norm
            h = layer(x, h, md, self.side_embed, input_ids, nxt)
            if self.residual_tap is not None:
                self.residual_tap.append(x.clone())
        return h

    __call__ = forward

    # ---- weights ----------------------------------------------------------------------
    def named_weights(self) -> Iterable[tuple[str, torch.Tensor]]:
        """checkpoint name -> parameter (a row block of a fused one where the checkpoint stores the pieces apart)"""
        yield "embed", self.embed
        yield "bigram", self.bigram
        yield "side.embed", self.side_embed
        for i, layer in enumerate(self.layers):
            yield from layer.named_weights(f"l{i}.")
        yield "final.norm", self.final_norm
        yield "head", self.head

    def weights_changed(self) -> None:
        for layer in self.layers:
            if isinstance(layer.mixer, LatentAttention):
                layer.mixer.weights_changed()
