"""Sequence mixers and small blocks of decoders with a 32-bit residual stream: latent attention without positions
(its cache row shared by all heads, optionally by several layers), the gated delta rule with a decay per head or per key
channel, attention with a distance bias and a sink, decayed linear attention, several mixers side by side, attention whose
heads mix their softmax weights, a short filter in front of a sublayer, a state-space recurrence, and attention whose values are its
keys.  Constants that a design fixes are parameters here; the layers know nothing of the model they are in.

Two kinds: mixers that own their projections (``LatentAttention``, ``GatedDelta``, ``TalkingAttention``, ``StateSpace``,
``KeyValueAttention``: rows in, rows out), and mixers for layers whose sublayers all read one normed row and add up (``ChannelDelta``, ``SinkAttention``, ``LightningAttention``,
``ParallelMixers``, ``DenseGlu``): such a layer has ONE input product and ONE output product (``SharedProjections``), and a
sublayer names its blocks of both, turning columns of the first into columns the second reads.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Iterable, Iterator, Optional, Sequence

import torch
import torch.nn.functional as F

from . import ops
from .kv_cache import KVCacheSpec, LatentCacheSpec, normalize_layer_kv
from .layers import AttentionMetadata, _apply_linear, _init_weight, fused_gate_up_silu, fused_up_relu_squared, tuned_linear
from .state_cache import StateSpec


def _pad16(n: int) -> int:
    return -(-n // 16) * 16


class ReplicatedLinear:
    """y = x W^T, not sharded; routed like the decoder's other linears.  ``parts`` names row blocks of the weight that a
    checkpoint stores apart; rows past their sum (padding to a multiple of 16) stay zero.  ``biased``: the parts that have a
    bias (stored as ``<part>.b``); the others' stays zero."""

    def __init__(self, in_features: int, parts: dict[str, int], dtype, device, generator=None, pad: bool = False,
                 biased: Sequence[str] = ()):
        self.parts, self.biased = parts, biased
        n = sum(parts.values())
        self.out_features = n
        self.weight = _init_weight(_pad16(n) if pad else n, in_features, dtype, device, generator, std=in_features ** -0.5)
        if pad:
            self.weight[n:].zero_()
        self.bias = torch.zeros(self.weight.shape[0], dtype=dtype, device=device) if biased else None

    def named(self, prefix: str) -> Iterable[tuple[str, torch.Tensor]]:
        r = 0
        for name, n in self.parts.items():
            yield prefix + name, self.weight[r:r + n]
            if name in self.biased:
                yield prefix + name + ".b", self.bias[r:r + n]
            r += n

    def __call__(self, x: torch.Tensor, defer_reduce: bool = False):
        return _apply_linear(self, x, self.bias, defer_reduce)


@dataclass
class LatentAttentionConfig:
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: Optional[int] = None      # tokens a query sees, itself included; None: all before it
    kv_from: Optional[int] = None     # layer whose cache this layer reads (it writes none of its own)


class LatentAttention:
    """q through a latent, k and v of every head from the cached latent row (``csrc/latent_attn.hip``)."""

    def __init__(self, cfg: LatentAttentionConfig, width: int, eps: float, dtype, device, generator=None):
        self.cfg, self.eps, self.dtype = cfg, eps, dtype
        self.window = cfg.window if cfg.window is not None else 2**31 - 1
        own = cfg.kv_from is None
        self.down = ReplicatedLinear(width, {"dq": cfg.q_rank, **({"dkv": cfg.kv_rank} if own else {})}, dtype, device, generator)
        self.uq = ReplicatedLinear(cfg.q_rank, {"uq": cfg.heads * cfg.dim}, dtype, device, generator)
        self.uk = ReplicatedLinear(cfg.kv_rank, {"uk": cfg.heads * cfg.dim}, dtype, device, generator)
        self.uv = ReplicatedLinear(cfg.kv_rank, {"uv": cfg.heads * cfg.vdim}, dtype, device, generator)
        self.o = ReplicatedLinear(cfg.heads * cfg.vdim, {"o": width}, dtype, device, generator)
        self.dq_norm = torch.ones(cfg.q_rank, dtype=dtype, device=device)
        self.dkv_norm = torch.ones(cfg.kv_rank, dtype=dtype, device=device) if own else None
        self.cache: Optional[torch.Tensor] = None
        self._uk_t: Optional[torch.Tensor] = None

    def kv_cache_spec(self, block_size: int) -> Optional[LatentCacheSpec]:
        return LatentCacheSpec(block_size, self.cfg.kv_rank, self.dtype) if self.cfg.kv_from is None else None

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        for lin in (self.down, self.uq, self.uk, self.uv, self.o):
            yield from lin.named(p)
        yield p + "dq.norm", self.dq_norm
        if self.dkv_norm is not None:
            yield p + "dkv.norm", self.dkv_norm

    def __call__(self, h: torch.Tensor, md: AttentionMetadata, defer_reduce: bool = False):
        c = self.cfg
        cq = ops.latent_norm_cache(self.down(h), self.dq_norm, self.dkv_norm, self.cache, md.slot_mapping, self.eps)
        q = self.uq(cq)
        nd, total = md.num_decodes, q.shape[0]
        o = torch.empty(total, c.heads * c.vdim, dtype=q.dtype, device=q.device)
        if nd:
            self._decode(q[:nd], o[:nd], md)
        if nd < total:
            self._prefill(q, o, md)
        return self.o(o, defer_reduce)

    def weights_changed(self) -> None:
        self._uk_t = None

    def _absorb_weight(self) -> torch.Tensor:
        """W_uk per head transposed, [H, rank, dim]: the absorb product then reads rows"""
        if self._uk_t is None:
            c = self.cfg
            self._uk_t = self.uk.weight.view(c.heads, c.dim, c.kv_rank).transpose(1, 2).contiguous()
        return self._uk_t

    def _rows(self, q: torch.Tensor, o: torch.Tensor, md: AttentionMetadata, row0: int) -> None:
        """rows [row0, T) through the kernel that takes any sizes and types"""
        c = self.cfg
        qa = ops.head_gemm(q, self.uk.weight.view(c.heads, c.dim, c.kv_rank), transposed=True)
        oa = ops.latent_attn_rows(qa, self.cache, md.block_table, md.seq_lens, md.query_start_loc, c.heads, self.window, c.scale,
                                  row0=row0)
        o[row0:] = ops.head_gemm(oa[row0:], self.uv.weight.view(c.heads, c.vdim, c.kv_rank))

    def _decode(self, q: torch.Tensor, o: torch.Tensor, md: AttentionMetadata) -> None:
        c = self.cfg
        if not ops.latent_decode_supported(self.dtype, c.kv_rank, c.dim, c.vdim, self.cache.shape[1]):
            return self._rows(q, o, md, 0)
        qa = ops.head_gemm_nt(q, self._absorb_weight())
        oa = ops.latent_decode(qa, self.cache, md.block_table, md.seq_lens, c.heads, self.window, md.max_seq_len, c.scale)
        ops.head_gemm_nt(oa, self.uv.weight.view(c.heads, c.vdim, c.kv_rank), o)

    def _prefill(self, q: torch.Tensor, o: torch.Tensor, md: AttentionMetadata) -> None:
        c, nd = self.cfg, md.num_decodes
        if not ops.latent_prefill_supported(self.dtype, c.kv_rank, c.dim, c.vdim):
            return self._rows(q, o, md, nd)
        start, rows = md.prefill_ctx[self.window]
        table, lens, qsl = md.block_table[nd:], md.seq_lens[nd:], md.query_start_loc[nd:]
        key = (self.cache.data_ptr(), self.window)      # layers that share a cache share its gathered rows
        ctx = md.step_cache.get(key)
        if ctx is None:
            ctx = md.step_cache[key] = ops.latent_gather(self.cache, start, rows, table, lens, qsl, self.window)
        # K by rows, V transposed: the attention kernel reads both along its k dimension
        ops.latent_prefill(o, q, F.linear(ctx, self.uk.weight), F.linear(self.uv.weight, ctx), start, lens, qsl, md.max_query_len,
                           c.heads, self.window, c.scale)


@dataclass
class GatedDeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                         # taps of the short convolutions


class GatedDelta:
    """Gated delta rule with short convolutions (``csrc/gated_delta.hip``)."""

    def __init__(self, cfg: GatedDeltaConfig, width: int, eps: float, dtype, device, generator=None):
        if cfg.heads % cfg.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.cfg, self.eps, self.dtype = cfg, eps, dtype
        kd, hv = cfg.kv_heads * cfg.dim, cfg.heads * cfg.vdim
        self.proj = ReplicatedLinear(width, {"q": kd, "k": kd, "v": hv, "g": hv, "b": cfg.heads, "a": cfg.heads}, dtype, device,
                                     generator, pad=True)
        self.o = ReplicatedLinear(hv, {"o": width}, dtype, device, generator)
        self.channels = 2 * kd + hv
        self.conv_w = _init_weight(self.channels, cfg.conv, dtype, device, generator, std=0.5)
        self.a_log = torch.zeros(cfg.heads, dtype=torch.float32, device=device)
        self.dt_bias = torch.zeros(cfg.heads, dtype=torch.float32, device=device)
        self.norm = torch.ones(cfg.vdim, dtype=dtype, device=device)
        self.state: Optional[torch.Tensor] = None
        self.ring: Optional[torch.Tensor] = None

    def state_specs(self) -> list[StateSpec]:
        c = self.cfg
        return [StateSpec((c.heads, c.dim, c.vdim), torch.float32), StateSpec((c.conv, self.channels), self.dtype)]

    def bind_state(self, state: torch.Tensor, ring: torch.Tensor) -> None:
        self.state, self.ring = state, ring

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        c = self.cfg
        yield from self.proj.named(p)
        yield from self.o.named(p)
        kd = c.kv_heads * c.dim
        for name, lo, hi in (("q", 0, kd), ("k", kd, 2 * kd), ("v", 2 * kd, self.channels)):
            yield p + name + ".conv", self.conv_w[lo:hi]
        yield p + "A_log", self.a_log
        yield p + "dt_bias", self.dt_bias
        yield p + "norm", self.norm

    def __call__(self, h: torch.Tensor, md: AttentionMetadata, defer_reduce: bool = False):
        c = self.cfg
        proj = self.proj(h)
        out = torch.empty(h.shape[0], c.heads * c.vdim, dtype=self.dtype, device=h.device)
        args = (proj, self.conv_w, self.a_log, self.dt_bias, self.norm, self.state, self.ring, md.state_rows, md.query_start_loc,
                md.seq_lens, c.kv_heads, self.eps, out)
        nd = md.num_decodes
        if nd:
            ops.gated_delta_step(*args, 0, nd, update_ring=False)
        if nd < md.num_reqs:
            ops.gated_delta_chunked(*args, nd, md.num_reqs - nd, nd, md.max_query_len)
        return self.o(out, defer_reduce)


class ClampedGluMLP:
    """down(g sigmoid(alpha g) (u + 1)) on a clamped gate and up projection"""

    def __init__(self, width: int, ff: int, limit: float, alpha: float, dtype, device, generator=None):
        self.limit, self.alpha = limit, alpha
        self.gate_up = ReplicatedLinear(width, {"gate": ff, "up": ff}, dtype, device, generator)
        self.down = ReplicatedLinear(ff, {"down": width}, dtype, device, generator)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield from self.gate_up.named(p)
        yield from self.down.named(p)

    def __call__(self, h: torch.Tensor, defer_reduce: bool = False):
        act = fused_gate_up_silu(self.gate_up, h, (self.alpha, self.limit))     # decode batches: one launch
        if act is None:
            act = ops.clamped_glu(self.gate_up(h), self.alpha, self.limit)
        return self.down(act, defer_reduce)


class TokenSideInput:
    """proj(gelu_tanh(gate x) * (the layer's slice of a per-token table)); the caller norms and adds it"""

    def __init__(self, width: int, dim: int, layer: int, dtype, device, generator=None):
        self.offset = layer * dim
        self.gate = ReplicatedLinear(width, {"gate": dim}, dtype, device, generator)
        self.proj = ReplicatedLinear(dim, {"proj": width}, dtype, device, generator)
        self.norm = torch.ones(width, dtype=dtype, device=device)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield from self.gate.named(p)
        yield from self.proj.named(p)
        yield p + "norm", self.norm

    def __call__(self, x: torch.Tensor, table: torch.Tensor, ids: torch.Tensor, defer_reduce: bool = False):
        return self.proj(ops.gelu_lookup_mul(self.gate(x), table, ids, self.offset), defer_reduce)


@dataclass
class TalkingAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None      # tokens a query sees, itself included; None: all before it
    softcap: float = 0.0              # 0: none


class TalkingAttention:
    """Grouped-query attention whose heads mix their softmax weights, with soft-capped scores, a distance bias of
    r1 ln(1 + r2 distance), q and k each normed over all heads at once, and a gate on the concatenated heads
    (``csrc/talking_attn.hip``, ``csrc/talking_attn_mfma.hip``)."""

    def __init__(self, cfg: TalkingAttentionConfig, width: int, eps: float, dtype, device, generator=None):
        if cfg.heads % cfg.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if cfg.window is not None and cfg.window < 1:
            raise ValueError("a window holds at least the token itself")
        if cfg.softcap < 0:
            raise ValueError("the soft cap must be positive")
        self.cfg, self.eps, self.dtype = cfg, eps, dtype
        self.window = cfg.window if cfg.window is not None else 2**31 - 1
        big = max(cfg.dim, cfg.vdim)
        # heads are laid out to the sizes the matrix-core kernels are built for
        self.head_dim = -(-big // 8) * 8 if dtype != torch.bfloat16 or big > 128 else 64 if big <= 64 else 128
        nq, nk, nv, ng = cfg.heads * cfg.dim, cfg.kv_heads * cfg.dim, cfg.kv_heads * cfg.vdim, cfg.heads * cfg.vdim
        self.qkv, self.gated = nq + nk + nv, ng
        self.proj = ReplicatedLinear(width, {"q": nq, "k": nk, "v": nv, "g": ng}, dtype, device, generator, pad=True,
                                     biased=("q", "k", "v"))
        self.o = ReplicatedLinear(ng, {"o": width}, dtype, device, generator)
        self.q_norm, self.k_norm = _vec(nq, dtype, device), _vec(nk, dtype, device)
        self.r1, self.r2 = _vec(cfg.heads, torch.float32, device), _vec(cfg.heads, torch.float32, device)
        self.talk = torch.eye(cfg.heads, dtype=torch.float32, device=device)
        self.heads = ops.TalkingHeads(self.talk, self.r1, self.r2, cfg.scale, cfg.softcap, self.window, cfg.vdim)

    def kv_cache_spec(self, block_size: int) -> KVCacheSpec:
        return KVCacheSpec(block_size, self.cfg.kv_heads, self.head_dim, self.dtype)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield from self.proj.named(p)
        yield from self.o.named(p)
        yield p + "q.norm", self.q_norm
        yield p + "k.norm", self.k_norm
        yield p + "r1", self.r1
        yield p + "r2", self.r2
        yield p + "talk", self.talk

    def __call__(self, h: torch.Tensor, md: AttentionMetadata, memory: "LayerMemory", defer_reduce: bool = False):
        c = self.cfg
        kc, vc = memory.kv
        x = self.proj(h)
        q = ops.row_norm_cache(x[:, :self.qkv], self.q_norm, self.k_norm, kc, vc, md.slot_mapping, c.heads, c.dim, c.vdim, self.eps)
        gate = x[:, self.qkv:self.qkv + self.gated]
        out = torch.empty(h.shape[0], self.gated, dtype=self.dtype, device=h.device)
        args = (out, q, kc, vc)
        if not ops.talking_attn_supported(self.dtype, c.heads, c.kv_heads, self.head_dim, c.vdim, kc.shape[1], c.softcap):
            ops.talking_attn_rows(*args, md.block_table, md.seq_lens, md.query_start_loc, self.heads, gate)
            return self.o(out, defer_reduce)
        nd, n = md.num_decodes, md.num_reqs
        if nd:
            ops.talking_decode(*args, md.block_table, md.seq_lens, md.query_start_loc, self.heads, md.max_seq_len, nd, gate)
        if nd < n:      # the portions' row offsets count from the step's first row, so the operands go whole
            start, rows = md.prefill_ctx[self.window]
            ops.talking_prefill(*args, md.block_table[nd:n], md.seq_lens[nd:n], md.query_start_loc[nd:n + 1], self.heads, start, rows,
                                md.max_query_len, gate)
        return self.o(out, defer_reduce)


@dataclass
class StateSpaceConfig:
    heads: int
    groups: int                       # of heads that share B and C
    state: int
    vdim: int
    conv: int                         # taps of the short filters
    norm_groups: int                  # equal parts of the gated row that are normed apart

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state


class StateSpace:
    """State-space recurrence with a scalar decay per head and token, short filters in front of it and a gated norm behind it
    (``csrc/state_space.hip``)."""

    def __init__(self, cfg: StateSpaceConfig, width: int, eps: float, dtype, device, generator=None):
        if cfg.heads % cfg.groups or cfg.inner % cfg.norm_groups:
            raise ValueError("heads must be a multiple of groups, and their columns of norm_groups")
        if cfg.conv < 1:
            raise ValueError("a filter has at least the tap of the row itself")
        self.cfg, self.eps, self.dtype = cfg, eps, dtype
        # z | x | B | C | step sizes
        self.proj = ReplicatedLinear(width, {"in": cfg.inner + cfg.channels + cfg.heads}, dtype, device, generator, pad=True)
        self.o = ReplicatedLinear(cfg.inner, {"o": width}, dtype, device, generator)
        self.conv_w = _init_weight(cfg.channels, cfg.conv, dtype, device, generator, std=0.5)
        self.conv_b = _vec(cfg.channels, dtype, device, 0.0)
        self.dt_bias, self.a_log = _vec(cfg.heads, torch.float32, device, 0.0), _vec(cfg.heads, torch.float32, device, 0.0)
        self.d = _vec(cfg.heads, torch.float32, device)
        self.norm = _vec(cfg.inner, dtype, device)

    def kv_cache_spec(self, block_size: int) -> Optional[KVCacheSpec]:
        return None

    def state_specs(self) -> list[StateSpec]:
        c = self.cfg
        return [StateSpec((c.heads, c.state, c.vdim), torch.float32), StateSpec((c.conv, c.channels), self.dtype)]

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield from self.proj.named(p)
        yield from self.o.named(p)
        yield p + "conv", self.conv_w
        yield p + "conv.b", self.conv_b
        yield p + "dt_bias", self.dt_bias
        yield p + "A_log", self.a_log
        yield p + "D", self.d
        yield p + "norm", self.norm

    def __call__(self, h: torch.Tensor, md: AttentionMetadata, memory: "LayerMemory", defer_reduce: bool = False):
        c = self.cfg
        x = self.proj(h)
        out = torch.empty(h.shape[0], c.inner, dtype=self.dtype, device=h.device)
        at = c.inner + c.channels
        args = (x[:, c.inner:at], x[:, :c.inner], x[:, at:at + c.heads], self.conv_w, self.conv_b, self.dt_bias, self.a_log, self.d,
                self.norm, *memory.states, md.state_rows, md.query_start_loc, md.seq_lens, c.groups, c.norm_groups, self.eps, out)
        nd = md.num_decodes
        if nd:
            ops.state_space(*args, 0, nd, 0, nd, 1, chunked=False)
        if nd < md.num_reqs:
            ops.state_space(*args, nd, md.num_reqs - nd, nd, h.shape[0] - nd, md.max_query_len)
        return self.o(out, defer_reduce)


@dataclass
class KeyValueAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    conv: int                         # taps of the short filters
    scale: float
    rot_dims: int = 0                 # leading dimensions of a head that turn with the position, in neighbouring pairs
    rot_base: float = 10000.0
    sink: Optional[float] = None      # score of one more term of the softmax's denominator; None: no such term


class KeyValueAttention:
    """Grouped-query attention whose values are its keys as the short filter leaves them; queries and keys turn with the position
    and are then normed per head, without weights (``csrc/conv_rope.hip`` and the paged-attention kernels)."""

    def __init__(self, cfg: KeyValueAttentionConfig, width: int, eps: float, dtype, device, generator=None):
        if cfg.heads % cfg.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if cfg.scale <= 0:
            raise ValueError("the score scale must be positive")
        if cfg.conv < 1:
            raise ValueError("a filter has at least the tap of the row itself")
        if cfg.rot_dims % 2 or not 0 <= cfg.rot_dims <= cfg.dim:
            raise ValueError("rotary dimensions come in pairs, no more than a head has")
        self.cfg, self.eps, self.dtype = cfg, eps, dtype
        # heads are laid out to the sizes the matrix-core kernels are built for
        self.head_dim = -(-cfg.dim // 8) * 8 if dtype != torch.bfloat16 or cfg.dim > 128 else 64 if cfg.dim <= 64 else 128
        nq, nk = cfg.heads * cfg.dim, cfg.kv_heads * cfg.dim
        self.nq, self.channels = nq, nq + nk
        self.proj = ReplicatedLinear(width, {"q": nq, "k": nk}, dtype, device, generator, pad=True)
        self.conv_w = _init_weight(self.channels, cfg.conv, dtype, device, generator, std=0.5)
        self.o = _init_weight(width, cfg.heads * self.head_dim, dtype, device, generator, std=nq ** -0.5)
        self.o.view(width, cfg.heads, self.head_dim)[:, :, cfg.dim:].zero_()
        freq = [cfg.rot_base ** (-2.0 * i / cfg.rot_dims) for i in range(cfg.rot_dims // 2)]
        self.inv_freq = torch.tensor(freq, dtype=torch.float32, device=device) if freq else None
        self.sinks = None if cfg.sink is None else _vec(cfg.heads, torch.float32, device, cfg.sink)

    def kv_cache_spec(self, block_size: int) -> Optional[KVCacheSpec]:
        return KVCacheSpec(block_size, self.cfg.kv_heads, self.head_dim, self.dtype, self.cfg.heads)

    def state_specs(self) -> list[StateSpec]:
        return [StateSpec((self.cfg.conv, self.channels), self.dtype)]

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield from self.proj.named(p)
        yield p + "q.conv", self.conv_w[:self.nq]
        yield p + "k.conv", self.conv_w[self.nq:]
        w = self.o.view(self.o.shape[0], self.cfg.heads, self.head_dim)[:, :, :self.cfg.dim]
        yield p + "o", self.o if self.head_dim == self.cfg.dim else w

    def __call__(self, h: torch.Tensor, md: AttentionMetadata, memory: "LayerMemory", defer_reduce: bool = False):
        c, (kc, vc) = self.cfg, memory.kv
        x = self.proj(h)[:, :self.channels]
        q = torch.empty(h.shape[0], c.heads * self.head_dim, dtype=self.dtype, device=h.device)
        args = (x, self.conv_w, memory.states[0], q, kc, vc, self.inv_freq, md.state_rows, md.query_start_loc, md.seq_lens, md.slot_mapping,
                c.heads, c.dim, self.eps)
        nd, n = md.num_decodes, md.num_reqs
        if nd:
            ops.conv_rope_cache(*args, 0, nd, 1)
        if nd < n:
            ops.conv_rope_cache(*args, nd, n - nd, md.max_query_len)
        out = torch.empty_like(q)
        if not ops.paged_attn_bias_supported(self.dtype, self.head_dim, kc.shape[1]):
            ops.attn_rows(out, q, kc, vc, md.block_table, md.seq_lens, md.query_start_loc, c.scale, sinks=self.sinks)
        else:
            if nd:
                ops.paged_attn_decode(out[:nd], q[:nd], kc, vc, md.block_table[:nd], md.seq_lens[:nd], md.max_seq_len, c.scale,
                                      workspace=md.decode_workspace, sinks=self.sinks)
            if nd < n:      # the portions' row offsets count from the step's first row, so q and out go whole
                ops.paged_attn_prefill(out, q, kc, vc, md.block_table[nd:n], md.seq_lens[nd:n], md.query_start_loc[nd:n + 1],
                                       md.max_query_len, c.scale, max_seq_len=md.max_seq_len, sinks=self.sinks)
        return tuned_linear(out, self.o, defer_reduce=defer_reduce)


class InputConv:
    """h + a causal filter per channel over h: what a sublayer reads in place of h (``csrc/residual_norm.hip``)"""

    def __init__(self, width: int, taps: int, dtype, device, generator=None):
        if taps < 1:
            raise ValueError("a filter has at least the tap of the row itself")
        self.width, self.taps, self.dtype = width, taps, dtype
        self.weight = _init_weight(taps, width, dtype, device, generator, std=0.5 * taps ** -0.5)

    def state_specs(self) -> list[StateSpec]:
        return [StateSpec((self.taps - 1, self.width), self.dtype)] if self.taps > 1 else []

    def bind(self, it: Iterator[torch.Tensor]) -> ops.ConvRing:
        """one layer run's filter, its ring taken from the run's state tensors"""
        return ops.ConvRing(self.weight, next(it) if self.taps > 1 else None)


class SquaredReluMLP:
    """down(relu(up h)^2)"""

    def __init__(self, width: int, ff: int, dtype, device, generator=None):
        self.up = ReplicatedLinear(width, {"up": ff}, dtype, device, generator)
        self.down = ReplicatedLinear(ff, {"down": width}, dtype, device, generator)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield from self.up.named(p)
        yield from self.down.named(p)

    def __call__(self, h: torch.Tensor, defer_reduce: bool = False):
        act = fused_up_relu_squared(self.up, h)       # decode batches: no launch of its own for the activation
        if act is None:
            act = ops.relu_squared(self.up(h))
        return self.down(act, defer_reduce)


# ------------------------------------------------------------------------------------------ sublayers side by side
@dataclass
class InBlock:
    """Neighbouring rows of the shared input product, stored apart in the checkpoint: name -> rows"""

    parts: dict[str, int]

    @property
    def size(self) -> int:
        return sum(self.parts.values())


@dataclass
class OutBlock:
    """Columns of the shared output product: ``groups`` groups of ``width`` columns, laid out ``pitch`` apart"""

    name: str
    groups: int
    width: int
    pitch: int

    @property
    def size(self) -> int:
        return self.groups * self.pitch


class SharedProjections:
    """The input and output product of a layer whose sublayers read the same row and whose outputs add up.  Blocks start on
    multiples of eight (16-byte rows for the kernels that read and write them); what lies between them is zero."""

    ALIGN = 8

    def __init__(self, width: int, ins: Sequence[InBlock], outs: Sequence[OutBlock], dtype, device, generator=None):
        self.ins, self.outs = list(ins), list(outs)
        self.in_at, n = self._place([b.size for b in self.ins])
        self.out_at, k = self._place([b.size for b in self.outs])
        self.gaps = k != sum(b.groups * b.width for b in self.outs)
        self.inp = ReplicatedLinear(width, {"in": n}, dtype, device, generator, pad=True)
        real = sum(b.groups * b.width for b in self.outs)
        self.out = ReplicatedLinear(k, {"out": width}, dtype, device, generator)
        self.out.weight.mul_((k / real) ** 0.5)
        keep = torch.zeros(k, dtype=torch.bool, device=device)
        for b, a in zip(self.outs, self.out_at):
            keep[a:a + b.size].view(b.groups, b.pitch)[:, :b.width] = True
        self.out.weight[:, ~keep] = 0
        used = torch.zeros(self.inp.weight.shape[0], dtype=torch.bool, device=device)
        for b, a in zip(self.ins, self.in_at):
            used[a:a + b.size] = True
        self.inp.weight[~used] = 0

    def _place(self, sizes: Sequence[int]) -> tuple[list[int], int]:
        at, n = [], 0
        for s in sizes:
            at.append(n)
            n += -(-s // self.ALIGN) * self.ALIGN
        return at, n

    def named_weights(self) -> Iterable[tuple[str, torch.Tensor]]:
        for b, a in zip(self.ins, self.in_at):
            for name, n in b.parts.items():
                yield name, self.inp.weight[a:a + n]
                a += n
        for b, a in zip(self.outs, self.out_at):
            w = self.out.weight[:, a:a + b.size].view(-1, b.groups, b.pitch)[:, :, :b.width]
            yield b.name, w if b.pitch != b.width else self.out.weight[:, a:a + b.size]

    def project(self, h: torch.Tensor) -> list[torch.Tensor]:
        """a view per input block"""
        y = self.inp(h)
        return [y[:, a:a + b.size] for b, a in zip(self.ins, self.in_at)]

    def buffers(self, rows: int) -> tuple[torch.Tensor, list[torch.Tensor]]:
        """the output product's operand and a view per block (sublayers fill whole blocks; gaps between blocks stay zero)"""
        w = self.out.weight
        exact = sum(b.size for b in self.outs) == w.shape[1]
        buf = (torch.empty if exact else torch.zeros)(rows, w.shape[1], dtype=w.dtype, device=w.device)
        return buf, [buf[:, a:a + b.size] for b, a in zip(self.outs, self.out_at)]


@dataclass
class StepInfo:
    """what a sublayer needs of the step besides its own rows"""

    md: AttentionMetadata
    positions: torch.Tensor


class Sublayer:
    """``ins`` / ``outs``: its blocks of the shared products (names below the layer's prefix).  ``run`` fills its output views
    from its input views; ``memory`` holds its cache and state tensors of this layer run."""

    ins: list[InBlock]
    outs: list[OutBlock]

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        """parameters outside the shared products"""
        return ()

    def kv_cache_spec(self, block_size: int) -> Optional[KVCacheSpec]:
        return None

    def state_specs(self) -> list[StateSpec]:
        return []

    def run(self, x: list[torch.Tensor], y: list[torch.Tensor], step: StepInfo, memory: "LayerMemory") -> None:
        raise NotImplementedError


@dataclass
class LayerMemory:
    """one layer run's cache and state tensors (a layer that runs several times has one of these per run)"""

    kv: Optional[tuple[torch.Tensor, torch.Tensor]] = None
    states: list[torch.Tensor] = field(default_factory=list)

    def bind_kv(self, layer_kv) -> None:
        self.kv = normalize_layer_kv(layer_kv)


def _vec(n: int, dtype, device, value: float = 1.0) -> torch.Tensor:
    return torch.full((n,), value, dtype=dtype, device=device)


@dataclass
class ChannelDeltaConfig(GatedDeltaConfig):
    """decay (one per head and key channel) and output gate come through products of low rank"""

    decay_rank: int = 0
    gate_rank: int = 0


class ChannelDelta(Sublayer):
    """Gated delta rule with one decay per head and key channel (``csrc/gated_delta.hip``)."""

    def __init__(self, cfg: ChannelDeltaConfig, width: int, eps: float, dtype, device, generator=None, prefix: str = ""):
        if cfg.heads % cfg.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.cfg, self.eps, self.dtype = cfg, eps, dtype
        kd, hd, hv = cfg.kv_heads * cfg.dim, cfg.heads * cfg.dim, cfg.heads * cfg.vdim
        p = prefix
        self.ins = [InBlock({p + "q": kd, p + "k": kd, p + "v": hv}), InBlock({p + "a1": cfg.decay_rank, p + "g1": cfg.gate_rank}),
                    InBlock({p + "b": cfg.heads})]
        self.outs = [OutBlock(p + "o", 1, hv, hv)]
        self.channels = 2 * kd + hv
        self.conv_w = _init_weight(self.channels, cfg.conv, dtype, device, generator, std=0.5)
        # both second factors in one product, block-diagonal: [a1 h; g1 h] -> [decay; gate]
        self.gate_at = -(-hd // 8) * 8
        self.low = torch.zeros(self.gate_at + hv, cfg.decay_rank + cfg.gate_rank, dtype=dtype, device=device)
        self._low_blocks = {"a2": self.low[:hd, :cfg.decay_rank], "g2": self.low[self.gate_at:, cfg.decay_rank:]}
        for w in self._low_blocks.values():
            w.copy_(_init_weight(*w.shape, dtype, device, generator, std=w.shape[1] ** -0.5))
        self.a_log = _vec(cfg.heads, torch.float32, device, 0.0)
        self.dt_bias = _vec(hd, torch.float32, device, 0.0)
        self.norm = _vec(cfg.vdim, dtype, device)

    def state_specs(self) -> list[StateSpec]:
        c = self.cfg
        return [StateSpec((c.heads, c.dim, c.vdim), torch.float32), StateSpec((c.conv, self.channels), self.dtype)]

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        kd = self.cfg.kv_heads * self.cfg.dim
        for name, lo, hi in (("q", 0, kd), ("k", kd, 2 * kd), ("v", 2 * kd, self.channels)):
            yield p + name + ".conv", self.conv_w[lo:hi]
        for name, w in self._low_blocks.items():
            yield p + name, w
        yield p + "A_log", self.a_log
        yield p + "dt_bias", self.dt_bias
        yield p + "norm", self.norm

    def run(self, x, y, step, memory) -> None:
        c, md = self.cfg, step.md
        qkv, low, beta = x
        both = tuned_linear(low, self.low)
        hd = c.heads * c.dim
        args = (qkv, self.conv_w, self.a_log, self.dt_bias, self.norm, *memory.states, md.state_rows, md.query_start_loc, md.seq_lens,
                c.kv_heads, self.eps, y[0])
        kw = dict(gate=both[:, self.gate_at:], beta=beta, decay=both[:, :hd], sigmoid_gate=True)
        nd = md.num_decodes
        if nd:
            ops.gated_delta_step(*args, 0, nd, update_ring=False, **kw)
        if nd < md.num_reqs:
            ops.gated_delta_chunked(*args, nd, md.num_reqs - nd, nd, md.max_query_len, **kw)


@dataclass
class SinkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    slopes: Optional[list[float]] = None      # per head, taken off per token of distance; None: no distance bias
    temp_coef: float = 0.0                    # q times 1 + coef ln(floor((p + 1) / every) + 1)
    temp_every: int = 1


class SinkAttention(Sublayer):
    """Grouped-query attention with normed heads, a query temperature, a distance bias and a sink (``csrc/biased_attn.hip`` and
    the paged-attention kernels)."""

    def __init__(self, cfg: SinkAttentionConfig, width: int, eps: float, dtype, device, generator=None, prefix: str = "",
                 out_scale: float = 1.0):
        if cfg.heads % cfg.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        if cfg.scale <= 0:
            raise ValueError("the score scale must be positive")
        self.cfg, self.eps, self.dtype, self.out_scale = cfg, eps, dtype, out_scale
        big = max(cfg.dim, cfg.vdim)
        # heads are laid out to the sizes the matrix-core kernels are built for
        self.head_dim = -(-big // 8) * 8 if dtype != torch.bfloat16 or big > 128 else 64 if big <= 64 else 128
        p = prefix
        self.ins = [InBlock({p + "q": cfg.heads * cfg.dim, p + "k": cfg.kv_heads * cfg.dim, p + "v": cfg.kv_heads * cfg.vdim})]
        self.outs = [OutBlock(p + "o", cfg.heads, cfg.vdim, self.head_dim)]
        self.q_norm, self.k_norm = _vec(cfg.dim, dtype, device), _vec(cfg.dim, dtype, device)
        self.sink = _vec(cfg.heads, torch.float32, device, 0.0)
        self.slopes = None if cfg.slopes is None else torch.tensor(cfg.slopes, dtype=torch.float32, device=device)

    def kv_cache_spec(self, block_size: int) -> KVCacheSpec:
        return KVCacheSpec(block_size, self.cfg.kv_heads, self.head_dim, self.dtype, self.cfg.heads)

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield p + "q.norm", self.q_norm
        yield p + "k.norm", self.k_norm
        yield p + "sink", self.sink

    def run(self, x, y, step, memory) -> None:
        c, md = self.cfg, step.md
        kc, vc = memory.kv
        q = ops.head_norm_cache(x[0], self.q_norm, self.k_norm, kc, vc, md.slot_mapping, step.positions, c.heads, c.dim, c.vdim, self.eps,
                                c.temp_coef, c.temp_every)
        out, nd = y[0], md.num_decodes
        bias = dict(slopes=self.slopes, sinks=self.sink, out_scale=self.out_scale)
        if not ops.paged_attn_bias_supported(self.dtype, self.head_dim, kc.shape[1]):
            ops.attn_rows(out, q, kc, vc, md.block_table, md.seq_lens, md.query_start_loc, c.scale, **bias)
            return
        if nd:
            ops.paged_attn_decode(out[:nd], q[:nd], kc, vc, md.block_table[:nd], md.seq_lens[:nd], md.max_seq_len, c.scale,
                                  workspace=md.decode_workspace, **bias)
        if nd < md.num_reqs:      # the portions' row offsets count from the step's first row, so q and out go whole
            ops.paged_attn_prefill(out, q, kc, vc, md.block_table[nd:md.num_reqs], md.seq_lens[nd:md.num_reqs],
                                   md.query_start_loc[nd:md.num_reqs + 1], md.max_query_len, c.scale, max_seq_len=md.max_seq_len, **bias)


@dataclass
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: list[float]


class LightningAttention(Sublayer):
    """Decayed linear attention, its heads normed together and gated (``csrc/lightning_attn.hip``)."""

    def __init__(self, cfg: LightningConfig, width: int, eps: float, dtype, device, generator=None, prefix: str = "",
                 out_scale: float = 1.0):
        if len(cfg.decay) != cfg.heads or any(d <= 0 for d in cfg.decay):
            raise ValueError(f"one positive decay per head ({cfg.heads}), got {cfg.decay}")
        self.cfg, self.eps, self.dtype, self.out_scale = cfg, eps, dtype, out_scale
        hd, hv = cfg.heads * cfg.dim, cfg.heads * cfg.vdim
        p = prefix
        self.ins = [InBlock({p + "q": hd, p + "k": hd, p + "v": hv}), InBlock({p + "g": hv})]
        self.outs = [OutBlock(p + "o", 1, hv, hv)]
        self.norm = _vec(hv, dtype, device)
        self.decay = torch.tensor(cfg.decay, dtype=torch.float32, device=device)
        self.log2_decay = torch.tensor([math.log2(d) for d in cfg.decay], dtype=torch.float32, device=device)

    def state_specs(self) -> list[StateSpec]:
        c = self.cfg
        return [StateSpec((c.heads, c.dim, c.vdim), torch.float32)]

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        yield p + "norm", self.norm

    def run(self, x, y, step, memory) -> None:
        md, nd = step.md, step.md.num_decodes
        args = (x[0], x[1], self.norm, self.decay, self.log2_decay, memory.states[0], md.state_rows, md.query_start_loc, md.seq_lens,
                self.eps, y[0])
        if nd:
            ops.lightning_attn(*args, 0, nd, 0, nd, 1, self.out_scale, chunked=False)
        if nd < md.num_reqs:
            ops.lightning_attn(*args, nd, md.num_reqs - nd, nd, x[0].shape[0] - nd, md.max_query_len, self.out_scale)


class ParallelMixers(Sublayer):
    """Mixers that read the same row and whose outputs (each scaled by its own ``out_scale``) add up; name -> mixer"""

    def __init__(self, mixers: dict[str, Sublayer]):
        self.mixers = mixers
        self.ins = [b for m in mixers.values() for b in m.ins]
        self.outs = [b for m in mixers.values() for b in m.outs]

    def kv_cache_spec(self, block_size: int) -> Optional[KVCacheSpec]:
        specs = [s for s in (m.kv_cache_spec(block_size) for m in self.mixers.values()) if s is not None]
        if len(specs) > 1:
            raise NotImplementedError("one of the mixers side by side may keep a KV cache")
        return specs[0] if specs else None

    def state_specs(self) -> list[StateSpec]:
        return [s for m in self.mixers.values() for s in m.state_specs()]

    def named_weights(self, p: str) -> Iterable[tuple[str, torch.Tensor]]:
        for name, m in self.mixers.items():
            yield from m.named_weights(f"{p}{name}.")

    def run(self, x, y, step, memory) -> None:
        i = o = s = 0
        for m in self.mixers.values():
            ni, no, ns = len(m.ins), len(m.outs), len(m.state_specs())
            m.run(x[i:i + ni], y[o:o + no], step, LayerMemory(memory.kv, memory.states[s:s + ns]))
            i, o, s = i + ni, o + no, s + ns


class DenseGlu(Sublayer):
    """down(act(gate) * up)"""

    def __init__(self, ff: int, act: str, prefix: str = ""):
        self.ff, self.act = ff, act
        # gate and up on 16-byte rows of their own: two blocks
        self.ins = [InBlock({prefix + "gate": ff}), InBlock({prefix + "up": ff})]
        self.outs = [OutBlock(prefix + "down", 1, ff, ff)]

    def run(self, x, y, step, memory) -> None:
        ops.glu(y[0], x[0], x[1], self.act)
