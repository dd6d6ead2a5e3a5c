"""Bodopel: a small decoder of windowed attention layers whose heads mix their softmax weights, with soft-capped scores, a
log-distance bias, a learned position vector per token, a short causal filter in front of every sublayer, squared-relu
feed-forwards and a run of layers that is looped with its weights shared, each pass adding a vector of its own to the
stream.  The residual stream is 32-bit.

The configuration (``config.json``) lists the layers one by one; tensor names are ``l<i>.norm1`` / ``l<i>.canon1`` /
``l<i>.mix.*`` / ``l<i>.norm2`` / ``l<i>.canon2`` / ``l<i>.mlp.*`` beside ``embed``, ``pos``, ``loop.step``, ``final.norm``
and ``head``.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Any, Iterable, Optional

import torch

from . import ops
from .kv_cache import KVCacheSpec
from .layers import _init_weight, get_forward_context
from .mixers import InputConv, LayerMemory, SquaredReluMLP, TalkingAttention, TalkingAttentionConfig
from .state_cache import StateSpec
from .text_model import LoopConfig, TokenDecoder, layer_runs

NORM_SHIFT = 1.0        # norm weights of the stream are stored as their distance from one


@dataclass
class BodopelLayerConfig:
    mixer: TalkingAttentionConfig
    ff: int = 0                       # 0: no feed-forward


@dataclass
class BodopelConfig:
    vocab_size: int
    hidden_size: int
    max_positions: int
    layers: list[BodopelLayerConfig] = field(default_factory=list)
    rms_norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    taps: int = 1
    loop: Optional[LoopConfig] = None
    name: str = "bodopel"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def embedding_size(self) -> int:
        return self.hidden_size

    @property
    def runs(self) -> list[tuple[int, Optional[int]]]:
        """(layer, pass of the loop that starts with it), in the order the layers run"""
        return layer_runs(len(self.layers), self.loop)

    @classmethod
    def from_dict(cls, d: dict) -> "BodopelConfig":
        layers = []
        for i, entry in enumerate(d["layers"]):
            m, mlp = entry["mixer"], entry.get("mlp")
            if entry["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer type {entry['type']!r}")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            mask, cap = m.get("mask"), m.get("softcap")
            layers.append(BodopelLayerConfig(TalkingAttentionConfig(
                heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
                window=int(mask["size"]) if mask else None, softcap=float(cap) if cap is not None else 0.0), int(mlp["ff"]) if mlp else 0))
        lp = d.get("loop")
        cfg = cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), max_positions=int(d["max_positions"]), layers=layers,
                  rms_norm_eps=float(d["norm"]["eps"]), embedding_scale=float(d["embedding"]["scale"]), taps=int(d["canon"]["taps"]),
                  loop=LoopConfig(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None)
        cfg.validate()
        return cfg

    @classmethod
    def from_json(cls, path: str) -> "BodopelConfig":
        with open(os.path.join(path, "config.json") if os.path.isdir(path) else path) as f:
            return cls.from_dict(json.load(f))

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a model has at least one layer")
        if self.taps < 1:
            raise ValueError("a filter has at least the tap of the row itself")
        if self.max_positions < 1:
            raise ValueError("a position table has at least one row")
        if self.loop is not None:
            self.loop.validate(len(self.layers))


class BodopelDecoderLayer:
    def __init__(self, cfg: BodopelConfig, index: int, dtype, device, generator=None):
        lc, w = cfg.layers[index], cfg.hidden_size
        self.norm1 = torch.zeros(w, dtype=dtype, device=device)
        self.conv1 = InputConv(w, cfg.taps, dtype, device, generator)
        self.mixer = TalkingAttention(lc.mixer, w, cfg.rms_norm_eps, dtype, device, generator)
        self.mlp: Optional[SquaredReluMLP] = None
        self.norm2: Optional[torch.Tensor] = None
        self.conv2: Optional[InputConv] = None
        if lc.ff:
            self.mlp = SquaredReluMLP(w, lc.ff, dtype, device, generator)
            self.norm2 = torch.zeros(w, dtype=dtype, device=device)
            self.conv2 = InputConv(w, cfg.taps, dtype, device, generator)

    @property
    def convs(self) -> list[InputConv]:
        return [self.conv1] + ([self.conv2] if self.conv2 else [])

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield p + "norm1", self.norm1
        yield p + "canon1", self.conv1.weight.t()
        yield from self.mixer.named_weights(p + "mix.")
        if self.mlp:
            yield p + "norm2", self.norm2
            yield p + "canon2", self.conv2.weight.t()
            yield from self.mlp.named_weights(p + "mlp.")


class BodopelForCausalLM(TokenDecoder):
    """Takes token ids (and each request's state slot) from the step's metadata; returns final-normed hidden rows."""

    def __init__(self, cfg: BodopelConfig, dtype=torch.bfloat16, device=None, seed: Optional[int] = 0):
        super().__init__(cfg, dtype, device)
        gen = self.generator(seed)
        w, v = cfg.hidden_size, cfg.vocab_size
        self.embed = _init_weight(v, w, dtype, device, gen, std=1.0)
        self.pos = _init_weight(cfg.max_positions, w, dtype, device, gen, std=1.0)
        self.loop_step = _init_weight(cfg.loop.times, w, dtype, device, gen, std=1.0) if cfg.loop else None
        self.layers = [BodopelDecoderLayer(cfg, i, dtype, device, gen) for i in range(cfg.num_hidden_layers)]
        self.final_norm = torch.zeros(w, dtype=dtype, device=device)
        self.head = _init_weight(v, w, dtype, device, gen, std=w ** -0.5)
        self.runs = cfg.runs
        # every pass of a looped layer has its own cache and state
        self.memory = [LayerMemory() for _ in self.runs]
        self.rings: list[list[ops.ConvRing]] = []

    # ---- caches -------------------------------------------------------------------
    def kv_cache_specs(self, block_size: int) -> dict[int, KVCacheSpec]:
        """layer run -> its cache"""
        return {r: self.layers[i].mixer.kv_cache_spec(block_size) for r, (i, _) in enumerate(self.runs)}

    def bind_kv_caches(self, caches: dict[int, Any]) -> None:
        for r, kv in caches.items():
            self.memory[r].bind_kv(kv)

    def prefill_windows(self) -> list[int]:
        """windows of the layers whose prompt attention runs on a gathered context"""
        return sorted({layer.mixer.window for layer in self.layers})

    def state_specs(self) -> list[StateSpec]:
        return [s for i, _ in self.runs for c in self.layers[i].convs for s in c.state_specs()]

    def bind_states(self, tensors: list[torch.Tensor]) -> None:
        it = iter(tensors)
        self.rings = [[c.bind(it) for c in self.layers[i].convs] for i, _ in self.runs]

    @property
    def is_recurrent(self) -> bool:
        return bool(self.state_specs())

    # ---- forward --------------------------------------------------------------------
    def forward(self, input_ids=None, positions=None, intermediate_tensors=None, inputs_embeds=None, **kwargs):
        cfg, md = self.config, get_forward_context().attn_metadata
        if input_ids is None or md is None:
            raise ValueError("token ids and the step's metadata are required")
        eps, w, t = cfg.rms_norm_eps, cfg.hidden_size, input_ids.shape[0]
        x = torch.empty(t, w, dtype=torch.float32, device=self.embed.device)
        one_row_each = md.num_decodes == md.num_reqs == t

        def into(norm, ring, put):
            """norm of the stream, then the sublayer's filter: in the same launch when every row is a request's only one"""
            h = torch.empty(t, w, dtype=self.dtype, device=x.device)
            if ring is None:
                return put(norm, h, {})
            if one_row_each:
                return put(norm, h, {"conv": ring, "slots": md.state_rows})
            return ops.input_conv(put(norm, h, {}), ring, md.state_rows, md.query_start_loc, md.seq_lens, md.num_reqs, md.max_query_len)

        def add(y, step=None):
            def put(norm, h, conv):
                return ops.residual_add_norm_conv(x, y, norm, eps, h, NORM_SHIFT, step, positions=positions, **conv)
            return put

        def pass_row(r):     # what is added to the stream ahead of run r
            start = self.runs[r][1] if r < len(self.runs) else None
            return None if start is None else self.loop_step[start]

        h = into(self.layers[self.runs[0][0]].norm1, self.rings[0][0],
                 lambda norm, h, conv: ops.embed_pos_norm(self.embed, input_ids, x, norm, eps, h, positions, cfg.embedding_scale, self.pos,
                                                          pass_row(0), NORM_SHIFT, **conv))
        for r, (i, _) in enumerate(self.runs):
            layer, rings = self.layers[i], self.rings[r]
            y = layer.mixer(h, md, self.memory[r], True)
            if layer.mlp:
                y = layer.mlp(into(layer.norm2, rings[1], add(y)), True)
            step = pass_row(r + 1)
            if r + 1 < len(self.runs):
                h = into(self.layers[self.runs[r + 1][0]].norm1, self.rings[r + 1][0], add(y, step))
            else:
                h = into(self.final_norm, None, add(y))
            if self.residual_tap is not None:
                self.residual_tap.append(x.clone() if step is None else x - step.float())
        return h

    __call__ = forward

    # ---- weights ----------------------------------------------------------------------
    def named_weights(self) -> Iterable[tuple[str, torch.Tensor]]:
        """checkpoint name -> parameter (a row block of a fused one where the checkpoint stores the pieces apart)"""
        yield "embed", self.embed
        yield "pos", self.pos
        if self.loop_step is not None:
            yield "loop.step", self.loop_step
        for i, layer in enumerate(self.layers):
            yield from layer.named_weights(f"l{i}.")
        yield "final.norm", self.final_norm
        yield "head", self.head
