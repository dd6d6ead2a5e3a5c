"""Sequence mixers and small blocks of decoders with a 32-bit residual stream: latent attention without positions
(its cache row shared by all heads, optionally by several layers) and the gated delta rule.  Constants that a design
fixes are parameters here; the layers know nothing of the model they are in.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Iterable, Optional

import torch
import torch.nn.functional as F

from . import ops
from .kv_cache import LatentCacheSpec
from .layers import AttentionMetadata, _apply_linear, _init_weight, fused_gate_up_silu
from .state_cache import StateSpec


def _pad16(n: int) -> int:
    return -(-n // 16) * 16


class ReplicatedLinear:
    """y = x W^T, not sharded; routed like the decoder's other linears.  ``parts`` names row blocks of the weight that a
    checkpoint stores apart; rows past their sum (padding to a multiple of 16) stay zero."""

    def __init__(self, in_features: int, parts: dict[str, int], dtype, device, generator=None, pad: bool = False):
        self.parts = parts
        n = sum(parts.values())
        self.out_features = n
        self.weight = _init_weight(_pad16(n) if pad else n, in_features, dtype, device, generator, std=in_features ** -0.5)
        if pad:
            self.weight[n:].zero_()
        self.bias = None

    def named(self, prefix: str) -> Iterable[tuple[str, torch.Tensor]]:
        r = 0
        for name, n in self.parts.items():
            yield prefix + name, self.weight[r:r + n]
            r += n

    def __call__(self, x: torch.Tensor, defer_reduce: bool = False):
        return _apply_linear(self, x, None, defer_reduce)


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
