"""Lifuzen: a small decoder whose layers run mixer and feed-forward side by side, each on a norm of its own of the same stream.
Mixers are a state-space recurrence, or attention whose values are its keys, with short filters, partial rotary positions, normed
heads and a sink; feed-forwards are routed experts of squared relu whose scores scale what an expert reads.  A run of layers may be
looped with its weights shared, each pass adding a vector of its own and, from the second on, the embedding output to the stream.
Logits come from the embedding table, soft-capped.  The residual stream is 32-bit.

The configuration (``config.json``) lists the layers one by one; tensor names are ``l<i>.norm1`` / ``l<i>.mix.*`` / ``l<i>.norm2`` /
``l<i>.mlp.*`` beside ``embed``, ``loop.step`` and ``final.norm``.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Any, Iterable, Optional, Union

import torch

from . import ops
from .kv_cache import KVCacheSpec
from .layers import _init_weight, get_forward_context
from .mixers import KeyValueAttention, KeyValueAttentionConfig, LayerMemory, StateSpace, StateSpaceConfig
from .moe import RoutedExperts
from .state_cache import StateSpec
from .text_model import LoopConfig, TokenDecoder, layer_runs

NORM_SHIFT = 1.0        # norm weights of the stream are stored as their distance from one
SINK = 0.0              # score of the sink


@dataclass
class ExpertsConfig:
    experts: int
    top: int
    ff: int


@dataclass
class LifuzenLayerConfig:
    mixer: Union[StateSpaceConfig, KeyValueAttentionConfig]
    mlp: Optional[ExpertsConfig] = None


@dataclass
class LifuzenConfig:
    vocab_size: int
    hidden_size: int
    layers: list[LifuzenLayerConfig] = field(default_factory=list)
    rms_norm_eps: float = 1e-6
    residual_mult: float = 1.0
    logit_softcap: Optional[float] = None
    loop: Optional[LoopConfig] = None
    name: str = "lifuzen"

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
    def from_dict(cls, d: dict) -> "LifuzenConfig":
        layers = []
        for i, entry in enumerate(d["layers"]):
            m, mlp = entry["mixer"], entry.get("mlp")
            if entry["type"] == "mamba2":
                mixer: Any = StateSpaceConfig(heads=int(m["heads"]), groups=int(m["groups"]), state=int(m["state"]), vdim=int(m["vdim"]),
                                              conv=int(m["conv"]), norm_groups=int(m["norm_groups"]))
            elif entry["type"] == "attention":
                if int(m.get("vdim", m["dim"])) != int(m["dim"]):
                    raise ValueError(f"layer {i}: values are the keys, so vdim {m['vdim']} must be dim {m['dim']}")
                rot = m.get("rot") or {"dims": 0, "base": 1.0}
                mixer = KeyValueAttentionConfig(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), conv=int(m["conv"]),
                                                scale=float(m["scale"]), rot_dims=int(rot["dims"]), rot_base=float(rot["base"]), sink=SINK)
            else:
                raise ValueError(f"layer {i}: unknown mixer type {entry['type']!r}")
            if mlp is not None and mlp.get("kind") != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
            layers.append(LifuzenLayerConfig(mixer, ExpertsConfig(experts=int(mlp["router"]["experts"]), top=int(mlp["router"]["top"]),
                                                                  ff=int(mlp["expert"]["ff"])) if mlp else None))
        lp, cap = d.get("loop"), d.get("logit_softcap")
        cfg = cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers, rms_norm_eps=float(d["norm"]["eps"]),
                  residual_mult=float(d["residual_mult"]), logit_softcap=float(cap) if cap is not None else None,
                  loop=LoopConfig(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None)
        cfg.validate()
        return cfg

    @classmethod
    def from_json(cls, path: str) -> "LifuzenConfig":
        with open(os.path.join(path, "config.json") if os.path.isdir(path) else path) as f:
            return cls.from_dict(json.load(f))

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a model has at least one layer")
        if self.logit_softcap is not None and not self.logit_softcap > 0:
            raise ValueError("the logits' soft cap must be positive")
        if self.loop is not None:
            self.loop.validate(len(self.layers))


class LifuzenDecoderLayer:
    def __init__(self, cfg: LifuzenConfig, index: int, dtype, device, generator=None):
        lc, w = cfg.layers[index], cfg.hidden_size
        mixer_cls = StateSpace if isinstance(lc.mixer, StateSpaceConfig) else KeyValueAttention
        self.norm1 = torch.zeros(w, dtype=dtype, device=device)
        self.mixer = mixer_cls(lc.mixer, w, cfg.rms_norm_eps, dtype, device, generator)
        self.norm2: Optional[torch.Tensor] = None
        self.experts: Optional[RoutedExperts] = None
        if lc.mlp:
            self.norm2 = torch.zeros(w, dtype=dtype, device=device)
            self.experts = RoutedExperts(w, lc.mlp.experts, lc.mlp.top, lc.mlp.ff, dtype, device, generator, act="relu_squared",
                                         scores="sigmoid", bias=False, weigh_input=True)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield p + "norm1", self.norm1
        yield from self.mixer.named_weights(p + "mix.")
        if self.experts:
            yield p + "norm2", self.norm2
            yield from self.experts.named_weights(p + "mlp.")


class LifuzenForCausalLM(TokenDecoder):
    """Takes token ids (and each request's state slot) from the step's metadata; returns final-normed hidden rows."""

    def __init__(self, cfg: LifuzenConfig, dtype=torch.bfloat16, device=None, seed: Optional[int] = 0):
        super().__init__(cfg, dtype, device)
        gen = self.generator(seed)
        w, v = cfg.hidden_size, cfg.vocab_size
        self.embed = _init_weight(v, w, dtype, device, gen, std=1.0)
        self.head = self.embed
        self.logit_softcap = cfg.logit_softcap
        self.loop_step = _init_weight(cfg.loop.times, w, dtype, device, gen, std=1.0) if cfg.loop else None
        self.layers = [LifuzenDecoderLayer(cfg, i, dtype, device, gen) for i in range(cfg.num_hidden_layers)]
        self.final_norm = torch.zeros(w, dtype=dtype, device=device)
        self.unread_weights = frozenset(f"l{i}.norm2" for i, layer in enumerate(self.layers) if not layer.experts)
        self.runs = cfg.runs
        self.memory = [LayerMemory() for _ in self.runs]      # every pass of a looped layer has its own cache and state

    # ---- caches -------------------------------------------------------------------
    def kv_cache_specs(self, block_size: int) -> dict[int, KVCacheSpec]:
        """layer run -> its cache; runs of layers without attention have none"""
        specs = {r: self.layers[i].mixer.kv_cache_spec(block_size) for r, (i, _) in enumerate(self.runs)}
        return {r: s for r, s in specs.items() if s is not None}

    def bind_kv_caches(self, caches: dict[int, Any]) -> None:
        for r, kv in caches.items():
            self.memory[r].bind_kv(kv)

    def state_specs(self) -> list[StateSpec]:
        return [s for i, _ in self.runs for s in self.layers[i].mixer.state_specs()]

    def bind_states(self, tensors: list[torch.Tensor]) -> None:
        it = iter(tensors)
        for mem, (i, _) in zip(self.memory, self.runs):
            mem.states = [next(it) for _ in self.layers[i].mixer.state_specs()]

    @property
    def is_recurrent(self) -> bool:
        return bool(self.state_specs())

    # ---- forward --------------------------------------------------------------------
    def forward(self, input_ids=None, positions=None, intermediate_tensors=None, inputs_embeds=None, **kwargs):
        cfg, md = self.config, get_forward_context().attn_metadata
        if input_ids is None or md is None:
            raise ValueError("token ids and the step's metadata are required")
        w, t = cfg.hidden_size, input_ids.shape[0]
        x = torch.empty(t, w, dtype=torch.float32, device=self.embed.device)

        def into(r, y=None, experts=None):
            """the stream with what comes ahead of run ``r``, and the norms that run reads; behind the last run the final norm"""
            last = r == len(self.runs)
            layer, start = (None, None) if last else (self.layers[self.runs[r][0]], self.runs[r][1])
            w1, w2 = (self.final_norm, None) if last else (layer.norm1, layer.norm2)
            h1 = torch.empty(t, w, dtype=self.dtype, device=x.device)
            h2 = torch.empty_like(h1) if w2 is not None else None
            ops.stream_norm2(x, y, w1, w2, cfg.rms_norm_eps, h1, h2, NORM_SHIFT, cfg.residual_mult, experts,
                             self.embed if y is None or start else None, input_ids, None if start is None else self.loop_step[start])
            if self.residual_tap is not None and y is not None:      # the stream as the layer leaves it
                s = x.clone()
                if start is not None:
                    s -= self.loop_step[start].float() + (self.embed[input_ids].float() if start else 0)
                self.residual_tap.append(s)
            return h1, h2

        h1, h2 = into(0)
        for r, (i, _) in enumerate(self.runs):
            layer = self.layers[i]
            experts = layer.experts(h2) if layer.experts else None
            h1, h2 = into(r + 1, layer.mixer(h1, md, self.memory[r], True), experts)
        return h1

    __call__ = forward

    # ---- weights ----------------------------------------------------------------------
    def named_weights(self) -> Iterable[tuple[str, torch.Tensor]]:
        """checkpoint name -> parameter (a block of a fused one where the checkpoint stores the pieces apart)"""
        yield "embed", self.embed
        if self.loop_step is not None:
            yield "loop.step", self.loop_step
        for i, layer in enumerate(self.layers):
            yield from layer.named_weights(f"l{i}.")
        yield "final.norm", self.final_norm
