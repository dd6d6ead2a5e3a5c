"""Pupopel: a small decoder whose layers run mixer and feed-forward side by side on one normed row.  Mixers are the gated
delta rule with a decay per key channel, or attention (normed heads, query temperature, distance bias, sink) beside decayed
linear attention; feed-forwards are dense or routed with a shared expert; a run of layers may be looped with its weights
shared, every pass entering through a product of the stream and the embedding output.  The residual stream is 32-bit.

The configuration (``config.json``) lists the layers one by one; tensor names are ``l<i>.norm1`` / ``l<i>.mix.*`` /
``l<i>.mlp.*`` beside ``embed``, ``loop.in``, ``final.norm`` and ``head``.  The ranks of the delta layers' low-rank products
are given by the tensors alone.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Any, Iterable, Optional, Union

import torch

from . import ops
from .kv_cache import KVCacheSpec
from .layers import _DEFER_REDUCE, _init_weight, get_forward_context
from .mixers import (ChannelDelta, ChannelDeltaConfig, DenseGlu, LayerMemory, LightningAttention, LightningConfig, ParallelMixers,
                     SharedProjections, SinkAttention, SinkAttentionConfig, StepInfo, Sublayer)
from .moe import RoutedExperts
from .state_cache import StateSpec
from .text_model import LoopConfig, TokenDecoder, layer_runs

NORM_SHIFT = 1.0        # norm weights of the stream are stored as their distance from one
DENSE_ACT, EXPERT_ACT = "gelu_tanh", "silu"


def head_slopes(heads: int) -> list[float]:
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


@dataclass
class ParallelConfig:
    left: SinkAttentionConfig
    right: LightningConfig
    left_scale: float
    right_scale: float


@dataclass
class MoEFeedForwardConfig:
    experts: int
    top: int
    ff: int
    shared_ff: int = 0                # 0: no shared expert


@dataclass
class PupopelLayerConfig:
    mixer: Union[ChannelDeltaConfig, ParallelConfig]
    mlp: Union[None, int, MoEFeedForwardConfig] = None       # int: width of a dense feed-forward


@dataclass
class PupopelConfig:
    vocab_size: int
    hidden_size: int
    layers: list[PupopelLayerConfig] = field(default_factory=list)
    rms_norm_eps: float = 1e-6
    loop: Optional[LoopConfig] = None
    name: str = "pupopel"

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def embedding_size(self) -> int:
        return self.hidden_size

    @property
    def runs(self) -> list[tuple[int, bool]]:
        """(layer, whether a pass of the loop starts with it), in the order the layers run"""
        return [(i, start is not None) for i, start in layer_runs(len(self.layers), self.loop)]

    @classmethod
    def from_dict(cls, d: dict, shapes: Optional[dict] = None) -> "PupopelConfig":
        """``shapes``: the checkpoint's tensor shapes; without them a delta layer's ranks are its ``decay_rank`` / ``gate_rank``
        entries, or its head size."""
        layers = []
        for i, entry in enumerate(d["layers"]):
            m, mlp = entry["mixer"], entry.get("mlp")
            if entry["type"] == "channel_delta":
                rank = {n: (shapes or {}).get(f"l{i}.mix.{n}1", (m.get(key, m["dim"]),))[0] for n, key in (("a", "decay_rank"), ("g", "gate_rank"))}
                mixer: Any = ChannelDeltaConfig(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                                                conv=int(m["conv"]), decay_rank=int(rank["a"]), gate_rank=int(rank["g"]))
            elif entry["type"] == "parallel":
                a, r = m["left"], m["right"]
                t = a.get("q_temp") or {"coef": 0.0, "every": 1}
                if int(t["every"]) != t["every"] or t["every"] < 1:
                    raise ValueError(f"layer {i}: q_temp.every must be a positive whole number of tokens")
                left = SinkAttentionConfig(heads=int(a["heads"]), kv_heads=int(a["kv_heads"]), dim=int(a["dim"]), vdim=int(a["vdim"]),
                                           scale=float(a["scale"]), slopes=head_slopes(int(a["heads"])), temp_coef=float(t["coef"]),
                                           temp_every=int(t["every"]))
                right = LightningConfig(heads=int(r["heads"]), dim=int(r["dim"]), vdim=int(r["vdim"]), decay=[float(x) for x in r["decay"]])
                mixer = ParallelConfig(left, right, float(m["left_scale"]), float(m["right_scale"]))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {entry['type']!r}")
            if mlp is None:
                ff: Any = None
            elif mlp["kind"] == "dense":
                ff = int(mlp["ff"])
            elif mlp["kind"] == "moe":
                shared = mlp.get("shared")
                ff = MoEFeedForwardConfig(experts=int(mlp["router"]["experts"]), top=int(mlp["router"]["top"]), ff=int(mlp["expert"]["ff"]),
                                          shared_ff=int(shared["ff"]) if shared else 0)
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layers.append(PupopelLayerConfig(mixer, ff))
        lp = d.get("loop")
        cfg = cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), layers=layers, rms_norm_eps=float(d["norm"]["eps"]),
                  loop=LoopConfig(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None)
        cfg.validate()
        return cfg

    @classmethod
    def from_checkpoint(cls, d: dict, shapes: dict) -> "PupopelConfig":
        return cls.from_dict(d, shapes)

    @classmethod
    def from_json(cls, path: str) -> "PupopelConfig":
        with open(os.path.join(path, "config.json") if os.path.isdir(path) else path) as f:
            return cls.from_dict(json.load(f))

    def validate(self) -> None:
        if not self.layers:
            raise ValueError("a model has at least one layer")
        if self.loop is not None:
            self.loop.validate(len(self.layers))


class PupopelDecoderLayer:
    def __init__(self, cfg: PupopelConfig, index: int, dtype, device, generator=None):
        lc, w, eps = cfg.layers[index], cfg.hidden_size, cfg.rms_norm_eps
        self.norm1 = torch.zeros(w, dtype=dtype, device=device)
        args = (w, eps, dtype, device, generator)
        if isinstance(lc.mixer, ChannelDeltaConfig):
            self.mixer: Sublayer = ChannelDelta(lc.mixer, *args, prefix="mix.")
        else:
            self.mixer = ParallelMixers({
                "left": SinkAttention(lc.mixer.left, *args, prefix="mix.left.", out_scale=lc.mixer.left_scale),
                "right": LightningAttention(lc.mixer.right, *args, prefix="mix.right.", out_scale=lc.mixer.right_scale)})
        moe = lc.mlp if isinstance(lc.mlp, MoEFeedForwardConfig) else None
        self.experts = RoutedExperts(w, moe.experts, moe.top, moe.ff, dtype, device, generator) if moe else None
        self.glu: Optional[DenseGlu] = None
        if moe is None and lc.mlp:
            self.glu = DenseGlu(lc.mlp, DENSE_ACT, "mlp.")
        elif moe is not None and moe.shared_ff:
            self.glu = DenseGlu(moe.shared_ff, EXPERT_ACT, "mlp.shared.")
        subs = [self.mixer] + ([self.glu] if self.glu else [])
        self.proj = SharedProjections(w, [b for s in subs for b in s.ins], [b for s in subs for b in s.outs], dtype, device, generator)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield p + "norm1", self.norm1
        for name, w in self.proj.named_weights():
            yield p + name, w
        yield from self.mixer.named_weights(p + "mix.")
        if self.experts:
            yield from self.experts.named_weights(p + "mlp.")

    def __call__(self, h: torch.Tensor, step: StepInfo, memory: LayerMemory):
        """h: the normed row.  Returns what the residual add takes: the output product and the routed experts' rows."""
        experts = self.experts(h) if self.experts else None
        x = self.proj.project(h)
        buf, y = self.proj.buffers(h.shape[0])
        ni, no = len(self.mixer.ins), len(self.mixer.outs)
        self.mixer.run(x[:ni], y[:no], step, memory)
        if self.glu:
            self.glu.run(x[ni:], y[no:], step, memory)
        return self.proj.out(buf, True), experts


class PupopelForCausalLM(TokenDecoder):
    """Takes token ids (and each request's state slot) from the step's metadata; returns final-normed hidden rows."""

    def __init__(self, cfg: PupopelConfig, dtype=torch.bfloat16, device=None, seed: Optional[int] = 0):
        super().__init__(cfg, dtype, device)
        gen = self.generator(seed)
        w, v = cfg.hidden_size, cfg.vocab_size
        self.embed = _init_weight(v, w, dtype, device, gen, std=1.0)
        self.loop_in = _init_weight(w, 2 * w, dtype, device, gen, std=(2 * w) ** -0.5) if cfg.loop else None
        self.layers = [PupopelDecoderLayer(cfg, i, dtype, device, gen) for i in range(cfg.num_hidden_layers)]
        self.final_norm = torch.zeros(w, dtype=dtype, device=device)
        self.head = _init_weight(v, w, dtype, device, gen, std=w ** -0.5)
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
        eps, w, t = cfg.rms_norm_eps, cfg.hidden_size, input_ids.shape[0]
        x = torch.empty(t, w, dtype=torch.float32, device=self.embed.device)
        new = lambda *s: torch.empty(*s, dtype=self.dtype, device=x.device)   # noqa: E731
        both = new(t, 2 * w) if cfg.loop else None       # [stream, embedding output]: what a pass enters through
        starts = [s for _, s in self.runs] + [False]
        norms = [self.layers[i].norm1 for i, _ in self.runs] + [self.final_norm]
        step = StepInfo(md, positions)

        def target(r):      # (what run r's predecessor leaves for it: weight of its norm, row buffer)
            return (None, both[:, :w]) if starts[r] else (norms[r], new(t, w))

        pre, h = target(0)
        ops.embed_norm(self.embed, input_ids, x, pre, eps, h, both[:, w:] if cfg.loop else None, NORM_SHIFT)
        for r, (i, start) in enumerate(self.runs):
            if start:
                h = ops.residual_add_norm(x, stream_linear(both, self.loop_in), norms[r], eps, new(t, w), w_shift=NORM_SHIFT, start=True)
            y, experts = self.layers[i](h, step, self.memory[r])
            pre, h = target(r + 1)
            ops.residual_add_norm(x, y, pre, eps, h, experts, NORM_SHIFT)
            if self.residual_tap is not None:
                self.residual_tap.append(x.clone())
        return h

    __call__ = forward

    # ---- weights ----------------------------------------------------------------------
    def named_weights(self) -> Iterable[tuple[str, torch.Tensor]]:
        """checkpoint name -> parameter (a block of a fused one where the checkpoint stores the pieces apart)"""
        yield "embed", self.embed
        if self.loop_in is not None:
            yield "loop.in", self.loop_in
        for i, layer in enumerate(self.layers):
            yield from layer.named_weights(f"l{i}.")
        yield "final.norm", self.final_norm
        yield "head", self.head


def stream_linear(x: torch.Tensor, weight: torch.Tensor):
    """x weight^T for a 32-bit stream: sums leave in fp32 (or as the streaming kernel's fp32 partials)"""
    if x.dtype == torch.float32:
        return torch.nn.functional.linear(x, weight)
    m, (n, k) = x.shape[0], weight.shape
    if _DEFER_REDUCE and m <= 256 and ops.linear_supported(m, n, k, x.dtype):
        part = ops.linear_partials(x, weight)
        if part is not None:
            return part
    return torch.mm(x, weight.t(), out_dtype=torch.float32)
