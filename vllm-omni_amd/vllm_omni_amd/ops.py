"""Torch-tensor wrappers over the C ABI.  Plumbing only: no arithmetic happens here.

Every function launches on torch's *current* stream (so it is hipGraph-capturable under
``torch.cuda.graph``) and raises on non-GPU tensors — there is no CPU path in the product.
Reference call sites these stand in for are cited in include/vllm_omni_amd.h.
"""
from __future__ import annotations

import ctypes
import os
from typing import Optional, Sequence, Union

import torch

from . import _C
from ._C import check, lib

_DT = {torch.float16: _C.MI_DTYPE_F16, torch.bfloat16: _C.MI_DTYPE_BF16, torch.float32: _C.MI_DTYPE_F32}


def _dt(t: torch.dtype) -> int:
    try:
        return _DT[t]
    except KeyError:
        raise TypeError(f"unsupported dtype {t}") from None


def _gpu(*ts: Optional[torch.Tensor]) -> None:
    for t in ts:
        if t is not None and not t.is_cuda:
            raise RuntimeError(
                "vllm_omni_amd ops run only on the GPU (HIP kernels); got a CPU tensor. "
                "There is no CPU fallback by design."
            )


# the raw handle of torch's current stream without building a torch.cuda.Stream object per launch (an eager
# prefill chunk is ~500 launches; the object form measured 5-6 us of host time per call, this one well under 1)
_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)
_cur_device = getattr(torch._C, "_cuda_getDevice", None)


def _stream() -> int:
    if _raw_stream is not None and _cur_device is not None:
        return _raw_stream(_cur_device())
    return torch.cuda.current_stream().cuda_stream


def _p(t: Optional[torch.Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


def _cache_strides(kc: torch.Tensor, vc: torch.Tensor):
    """k_cache / v_cache are views shaped [num_blocks, block_size, kv_heads, head_dim]."""
    if kc.dim() != 4 or vc.shape != kc.shape or kc.stride() != vc.stride() or kc.stride(3) != 1:
        raise ValueError("k_cache/v_cache must be [num_blocks, block_size, kv_heads, head_dim] views "
                         "with identical strides and contiguous head_dim")
    return kc.stride(0), kc.stride(1), kc.stride(2)


# --------------------------------------------------------------------------- A4
def reshape_and_cache(k: torch.Tensor, v: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                      slot_mapping: torch.Tensor) -> None:
    """cache[slot] = (k, v)[token] for slot >= 0.  k, v: [T, kv_heads, head_dim] (or flattened)."""
    _gpu(k, v, k_cache, v_cache, slot_mapping)
    nb, bs, h, d = k_cache.shape
    t = k.shape[0]
    if slot_mapping.dtype != torch.int64 or slot_mapping.numel() < t:
        raise ValueError("slot_mapping must be int64 with >= num_tokens entries")
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    check("mi_reshape_and_cache", lib.mi_reshape_and_cache(
        _p(k), _p(v), _p(k_cache), _p(v_cache), _p(slot_mapping), t, h, d, bs,
        k.stride(0), v.stride(0), cb, ct, ch, _dt(k.dtype), _stream()))


# --------------------------------------------------------------------- A7/A7b/A4
def rope_neox_and_cache(q: torch.Tensor, k: torch.Tensor, v: Optional[torch.Tensor],
                        positions: torch.Tensor, cos_sin_cache: torch.Tensor, head_dim: int,
                        k_cache: Optional[torch.Tensor] = None, v_cache: Optional[torch.Tensor] = None,
                        slot_mapping: Optional[torch.Tensor] = None,
                        mrope_section: Optional[torch.Tensor] = None,
                        q_norm_weight: Optional[torch.Tensor] = None,
                        k_norm_weight: Optional[torch.Tensor] = None, norm_eps: float = 1e-6) -> None:
    """In-place (q/k-norm ->) neox RoPE on q [T, nq*d], k [T, nkv*d]; optional KV-cache write.

    positions int64 [T] or [3, T] (then ``mrope_section`` is an int32 *host* tensor of 3 entries);
    cos_sin_cache fp32 [max_position, rot_dim].
    """
    _gpu(q, k, v, positions, cos_sin_cache, k_cache, v_cache, slot_mapping, q_norm_weight, k_norm_weight)
    t = q.shape[0]
    nq = q.shape[-1] // head_dim if q.dim() == 2 else q.shape[1]
    nkv = k.shape[-1] // head_dim if k.dim() == 2 else k.shape[1]
    if positions.dtype != torch.int64 or cos_sin_cache.dtype != torch.float32:
        raise TypeError("positions must be int64 and cos_sin_cache float32")
    max_pos, rot_dim = cos_sin_cache.shape
    sec = None
    row_stride = 0
    if positions.dim() == 2:
        if mrope_section is None:
            raise ValueError("positions is [3, T]: mrope_section required")
        sec = (ctypes.c_int32 * 3)(*[int(x) for x in mrope_section])
        row_stride = positions.stride(0)
        if positions.stride(1) != 1:
            raise ValueError("positions rows must be contiguous")
    bs = cb = ct = ch = 0
    if k_cache is not None:
        cb, ct, ch = _cache_strides(k_cache, v_cache)
        bs = k_cache.shape[1]
        if slot_mapping is None or slot_mapping.dtype != torch.int64:
            raise ValueError("slot_mapping (int64) required with k_cache")
    check("mi_rope_neox_and_cache", lib.mi_rope_neox_and_cache(
        _p(q), _p(k), _p(v), _p(positions), row_stride,
        ctypes.cast(sec, ctypes.c_void_p) if sec is not None else None,
        _p(cos_sin_cache), max_pos, rot_dim, _p(q_norm_weight), _p(k_norm_weight), float(norm_eps),
        _p(k_cache), _p(v_cache), _p(slot_mapping), t, nq, nkv, head_dim, bs,
        q.stride(0), k.stride(0), v.stride(0) if v is not None else 0, cb, ct, ch,
        _dt(q.dtype), _stream()))


def embed_codes(ids: torch.Tensor, table: torch.Tensor, out_a: torch.Tensor, out_b: Optional[torch.Tensor] = None,
                ids_out: Optional[torch.Tensor] = None) -> None:
    """``out_a[t] = out_b[t] = table[ids[t]]``, ``ids_out[t] = ids[t]`` in one launch (``mi_embed_codes``): the code
    predictor's per-step glue.  ``out_*`` [T, E] row views (any row stride), ``ids_out`` int64 [T] (any stride)."""
    _gpu(ids, table, out_a, out_b, ids_out)
    if ids.dtype != torch.int64 or ids.dim() != 1 or not ids.is_contiguous():
        raise TypeError("ids must be contiguous int64 [T]")
    if table.dim() != 2 or not table.is_contiguous() or out_a.dtype != table.dtype or out_a.stride(-1) != 1:
        raise ValueError("table must be contiguous [V, E]; outputs rows of the same dtype")
    if ids_out is not None and (ids_out.dtype != torch.int64 or ids_out.dim() != 1):
        raise TypeError("ids_out must be int64 [T]")
    check("mi_embed_codes", lib.mi_embed_codes(
        _p(out_a), _p(out_b), _p(ids_out), _p(table), _p(ids), ids.shape[0], table.shape[1], table.shape[0],
        out_a.stride(0), out_b.stride(0) if out_b is not None else 0, ids_out.stride(0) if ids_out is not None else 0,
        _stream()))


def block_attention_supported(num_q_heads: int, num_kv_heads: int, head_dim: int, block_size: int, rot_dim: int) -> bool:
    return (head_dim == 128 and rot_dim == 128 and block_size <= 64 and num_q_heads % num_kv_heads == 0
            and num_q_heads // num_kv_heads in (1, 2, 4, 8))


def rope_cache_attend_block(out: torch.Tensor, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                            positions: Union[torch.Tensor, int], cos_sin_cache: torch.Tensor, head_dim: int,
                            k_cache: torch.Tensor, v_cache: torch.Tensor, block_ids: torch.Tensor, scale: float,
                            q_norm_weight: Optional[torch.Tensor] = None, k_norm_weight: Optional[torch.Tensor] = None,
                            norm_eps: float = 1e-6, max_position_bound: Optional[int] = None) -> torch.Tensor:
    """(q/k-norm ->) RoPE -> K/V append -> attention in ONE launch for sequences that live in one KV block each
    (``mi_rope_cache_attend_block``): row t's new token sits at ``positions[t]`` of block ``block_ids[t]`` and attends
    over tokens 0..positions[t] of it.  ``block_ids`` int32 [T] (any stride: a block-table column).
    ``positions``: int64 [T] on the device with ``max_position_bound`` >= every entry (default block_size - 1), or a
    host int when every row sits at the same position (the code predictor's lock-step sequences)."""
    _gpu(out, q, k, v, cos_sin_cache, k_cache, v_cache, block_ids, q_norm_weight, k_norm_weight)
    if isinstance(positions, int):
        bound, positions = positions, None
    else:
        _gpu(positions)
        if positions.dtype != torch.int64 or positions.dim() != 1:
            raise TypeError("positions must be int64 [T] (or a host int)")
        bound = k_cache.shape[1] - 1 if max_position_bound is None else int(max_position_bound)
    if cos_sin_cache.dtype != torch.float32:
        raise TypeError("cos_sin_cache must be float32")
    if block_ids.dtype != torch.int32 or block_ids.dim() != 1:
        raise TypeError("block_ids must be int32 [T]")
    t = q.shape[0]
    nq, nkv = q.shape[-1] // head_dim, k.shape[-1] // head_dim
    max_pos, rot_dim = cos_sin_cache.shape
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    check("mi_rope_cache_attend_block", lib.mi_rope_cache_attend_block(
        _p(out), _p(q), _p(k), _p(v), _p(positions), bound, _p(cos_sin_cache), max_pos, rot_dim, _p(q_norm_weight),
        _p(k_norm_weight), float(norm_eps), _p(k_cache), _p(v_cache), _p(block_ids), block_ids.stride(0), t, nq, nkv,
        head_dim, k_cache.shape[1], out.stride(0), q.stride(0), k.stride(0), v.stride(0), cb, ct, ch, float(scale),
        _dt(q.dtype), _stream()))
    return out


def rope_cache_attend_block_splitk(part: "SplitKPartials", num_q_heads: int, num_kv_heads: int, head_dim: int,
                                   positions: Union[torch.Tensor, int], cos_sin_cache: torch.Tensor, k_cache: torch.Tensor,
                                   v_cache: torch.Tensor, block_ids: torch.Tensor, scale: float,
                                   q_norm_weight: Optional[torch.Tensor] = None,
                                   k_norm_weight: Optional[torch.Tensor] = None, norm_eps: float = 1e-6,
                                   max_position_bound: Optional[int] = None) -> torch.Tensor:
    """``rope_cache_attend_block`` fed by the split-K partials of ``qkv_proj`` (``linear_partials``): returns the
    attention output [T, nq*d]; bit-identical to ``linear`` + ``rope_cache_attend_block``."""
    _gpu(cos_sin_cache, k_cache, v_cache, block_ids, q_norm_weight, k_norm_weight)
    part._live()
    if part.n != (num_q_heads + 2 * num_kv_heads) * head_dim:
        raise ValueError("partials row is not [q heads | k heads | v heads]")
    if isinstance(positions, int):
        bound, positions = positions, None
    else:
        _gpu(positions)
        if positions.dtype != torch.int64 or positions.dim() != 1:
            raise TypeError("positions must be int64 [T] (or a host int)")
        bound = k_cache.shape[1] - 1 if max_position_bound is None else int(max_position_bound)
    if cos_sin_cache.dtype != torch.float32 or block_ids.dtype != torch.int32 or block_ids.dim() != 1:
        raise TypeError("cos_sin_cache must be float32, block_ids int32 [T]")
    max_pos, rot_dim = cos_sin_cache.shape
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    out = torch.empty(part.m, num_q_heads * head_dim, dtype=part.dtype, device=part.device)
    check("mi_rope_cache_attend_block_splitk", lib.mi_rope_cache_attend_block_splitk(
        _p(out), _p(part.part), part.split, _p(part.bias), _p(positions), bound, _p(cos_sin_cache), max_pos, rot_dim,
        _p(q_norm_weight), _p(k_norm_weight), float(norm_eps), _p(k_cache), _p(v_cache), _p(block_ids), block_ids.stride(0),
        part.m, num_q_heads, num_kv_heads, head_dim, k_cache.shape[1], out.stride(0), cb, ct, ch, float(scale),
        _dt(part.dtype), _stream()))
    return out


class CpStack:
    """Host handle of the code predictor's one-launch layer stack (``mi_cp_stack_decode``, csrc/cp_stack.hip): the
    pointer tables of the layers' weights and private KV caches (the tensors are kept alive here) and the workspace
    that carries the activations between the launch's phases and its grid-barrier state.

    ``layers``: per layer a dict with ``qkv, o, gate_up, down, input_norm, post_norm, q_norm, k_norm`` (device tensors of
    the compute dtype) and ``k_cache, v_cache`` ([num_blocks, block_size, kv_heads, 128] views); ``max_rows``: the largest
    batch a call may bring."""

    _KEYS = ("qkv", "o", "gate_up", "down", "input_norm", "post_norm", "q_norm", "k_norm", "k_cache", "v_cache")

    def __init__(self, layers: Sequence[dict], final_norm: torch.Tensor, cos_sin_cache: torch.Tensor, num_q_heads: int,
                 num_kv_heads: int, head_dim: int, norm_eps: float, scale: float, max_rows: int):
        import ctypes

        first = layers[0]
        _gpu(final_norm, cos_sin_cache, *[t for layer in layers for t in (layer[k] for k in self._KEYS)])
        self.dtype = first["qkv"].dtype
        self.hidden = int(first["qkv"].shape[1])
        self.inter = int(first["down"].shape[1])
        self.nq, self.nkv, self.head_dim = int(num_q_heads), int(num_kv_heads), int(head_dim)
        self.eps, self.scale = float(norm_eps), float(scale)
        self.max_rows = int(max_rows)
        for layer in layers:
            if (tuple(layer["qkv"].shape) != ((self.nq + 2 * self.nkv) * self.head_dim, self.hidden)
                    or tuple(layer["o"].shape) != (self.hidden, self.nq * self.head_dim)
                    or tuple(layer["gate_up"].shape) != (2 * self.inter, self.hidden)
                    or tuple(layer["down"].shape) != (self.hidden, self.inter)):
                raise ValueError("layer weights do not have the stack's shapes")
            for k in self._KEYS[:8]:
                if layer[k].dtype != self.dtype or not layer[k].is_contiguous():
                    raise TypeError(f"{k}: contiguous {self.dtype} expected")
            if layer["k_cache"].stride() != first["k_cache"].stride() or layer["k_cache"].shape != first["k_cache"].shape:
                raise ValueError("the layers' KV caches must share one layout")
        self._cb, self._ct, self._ch = _cache_strides(first["k_cache"], first["v_cache"])
        self.block_size = int(first["k_cache"].shape[1])
        self._keep = (list(layers), final_norm, cos_sin_cache)
        n = len(layers)
        arr = ctypes.c_void_p * n
        self._tables = {k: arr(*[layer[k].data_ptr() for layer in layers]) for k in self._KEYS}
        self.num_layers = n
        self.final_norm, self.cos_sin = final_norm, cos_sin_cache
        nbytes = int(lib.mi_cp_stack_workspace_bytes(self.max_rows, self.hidden, self.nq, self.nkv, self.inter))
        if nbytes <= 0:
            raise ValueError("unsupported code-predictor stack geometry")
        self.workspace = torch.zeros(nbytes, dtype=torch.uint8, device=final_norm.device)
        self._ws_bytes = nbytes
        self._fresh = True

    def decode(self, out: torch.Tensor, x: torch.Tensor, block_ids: torch.Tensor, position: int) -> torch.Tensor:
        """One pass: x [rows, hidden] -> out [rows, hidden] (final-norm output), every row's new token at ``position`` of
        the KV block ``block_ids[row]``."""
        _gpu(out, x, block_ids)
        rows = int(x.shape[0])
        if rows > self.max_rows:
            raise ValueError(f"{rows} rows exceed the workspace's {self.max_rows}")
        if x.dtype != self.dtype or out.dtype != self.dtype or not x.is_contiguous() or not out.is_contiguous():
            raise TypeError("x / out must be contiguous tensors of the stack's dtype")
        if tuple(x.shape) != (rows, self.hidden) or tuple(out.shape) != (rows, self.hidden):
            raise ValueError("x / out must be [rows, hidden]")
        if block_ids.dtype != torch.int32 or block_ids.dim() != 1 or block_ids.shape[0] < rows:
            raise TypeError("block_ids must be int32 [rows]")
        t = self._tables
        check("mi_cp_stack_decode", lib.mi_cp_stack_decode(
            _p(out), _p(x), t["qkv"], t["o"], t["gate_up"], t["down"], t["input_norm"], t["post_norm"], t["q_norm"], t["k_norm"],
            _p(self.final_norm), t["k_cache"], t["v_cache"], _p(block_ids), block_ids.stride(0), _p(self.cos_sin),
            self.cos_sin.shape[0], int(position), rows, self.hidden, self.nq, self.nkv, self.head_dim, self.inter,
            self.num_layers, self.block_size, self._cb, self._ct, self._ch, self.eps, self.scale, _p(self.workspace),
            self._ws_bytes, 0, _dt(self.dtype), _stream()))   # the workspace was zeroed at allocation
        return out

    def status(self) -> int:
        """0 = every grid barrier of every launch so far completed (synchronises)."""
        return int(self.workspace[self._ws_bytes - 256:self._ws_bytes - 252].view(torch.int32).item())


# --------------------------------------------------------------------------- A5
# Default decode mode (see include/vllm_omni_amd.h, flags): True = P may be rounded to the cache dtype
# before P.V, as the reference's TRITON_ATTN kernel does -> matrix-core kernel where built (head_dim 128,
# block >= 16), dot2 VALU kernel elsewhere.  False = exact mode (P kept fp32, VALU kernel).
DECODE_PACKED_PV = True
DECODE_NONTEMPORAL = True   # nt cache policy on the K/V stream: +8 % measured (profiles/)


def _decode_flags(packed_pv: Optional[bool], force_valu: bool) -> int:
    return ((_C.MI_DECODE_PACKED_PV if (DECODE_PACKED_PV if packed_pv is None else packed_pv) else 0)
            | (_C.MI_DECODE_FORCE_VALU if force_valu else 0))


def decode_auto_partition(num_seqs: int, num_kv_heads: int, max_seq_len: int, block_size: int = 16,
                          requested: int = 0, packed_pv: Optional[bool] = None, force_valu: bool = False,
                          head_dim: int = 128) -> int:
    """Partition size a decode call will really use: ``requested``, or the auto choice — the fewest partitions that
    leave >= 512 waves (1024 at head_dim 64), ONE (direct output, no merge launch) once sequences x KV heads reach that;
    any multiple of 32 tokens for the matrix-core kernel, capped at 64 blocks for the VALU kernel (``packed_pv`` False /
    ``force_valu``)."""
    return int(lib.mi_paged_attn_decode_effective_partition(num_seqs, num_kv_heads, max_seq_len, head_dim, block_size,
                                                            requested, _decode_flags(packed_pv, force_valu)))


def decode_workspace_bytes(num_seqs: int, num_q_heads: int, head_dim: int, max_seq_len: int,
                           partition_size: int) -> int:
    return int(lib.mi_paged_attn_decode_workspace_bytes(num_seqs, num_q_heads, head_dim, max_seq_len,
                                                        partition_size))


# Workspaces whose counter region (the first MI_DECODE_COUNTER_BYTES) this module has zeroed: only on those does a
# decode call ask for the fused merge (the kernel leaves the counters at zero, so once is enough).  Keyed by the
# tensor OBJECT (a weak reference): a recycled address of a freed tensor can never pass for a prepared one.
_DECODE_WS_READY: dict = {}   # id(tensor) -> weakref(tensor)   (tensors compare element-wise: no WeakSet)


def _decode_ws_ready(ws: Optional[torch.Tensor]) -> bool:
    r = _DECODE_WS_READY.get(id(ws)) if ws is not None else None
    return r is not None and r() is ws


def new_decode_workspace(nbytes: int, device) -> torch.Tensor:
    """A decode workspace (``decode_workspace_bytes``) with its arrival-counter region zeroed: what
    ``paged_attn_decode`` needs to merge the context partitions inside the attention launch itself."""
    import weakref

    ws = torch.empty(max(int(nbytes), 16), dtype=torch.uint8, device=device)
    ws[:min(ws.numel(), _C.MI_DECODE_COUNTER_BYTES)].zero_()
    key = id(ws)
    _DECODE_WS_READY[key] = weakref.ref(ws, lambda _r, k=key: _DECODE_WS_READY.pop(k, None))
    return ws


# OFF by default: measured SLOWER than the separate merge kernel on every shape tried (profiles/r03c_decode_fused_ab.log:
# 391 against 363 us at B 256 / ctx 4096, 56 against 46 us at the 1/8-size shard shapes) — every wave now ends with a
# store-acknowledge wait and an atomic round trip while it still holds its LDS slot (5 waves per CU), which costs more
# streaming time than the 5-7 us merge launch it saves.  Kept (bit-identical, tested) for shapes with few, long waves.
DECODE_FUSED_MERGE = os.environ.get("VLLM_OMNI_AMD_DECODE_FUSED_MERGE", "0") == "1"
# RoPE + KV write of a pure-decode step inside the attention launch (rope_cache_paged_attn_decode); "0": two launches (A/B)
ROPE_DECODE_FUSION = os.environ.get("VLLM_OMNI_AMD_ROPE_DECODE_FUSION", "1") != "0"


def _head_vectors(nq: int, *ts: Optional[torch.Tensor]) -> None:
    for t in ts:
        if t is not None and (t.dtype != torch.float32 or t.numel() != nq or not t.is_contiguous()):
            raise ValueError(f"expected {nq} contiguous fp32 values")


def paged_attn_decode(out: torch.Tensor, q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                      block_table: torch.Tensor, seq_lens: torch.Tensor, max_seq_len: int, scale: float,
                      partition_size: int = 0, workspace: Optional[torch.Tensor] = None,
                      packed_pv: Optional[bool] = None, force_valu: bool = False,
                      nontemporal: Optional[bool] = None, rounded_p: bool = False,
                      fused_merge: Optional[bool] = None, _skip_merge: bool = False, slopes: Optional[torch.Tensor] = None,
                      sinks: Optional[torch.Tensor] = None, out_scale: float = 1.0) -> torch.Tensor:
    """out[s, h] = softmax(q[s,h] . K^T * scale) . V over the paged cache (one query per sequence).

    q, out: [S, nq*d] (or [S, nq, d]); block_table int32 [S, max_blocks]; seq_lens int32 [S].
    ``max_seq_len`` is a host-side upper bound of seq_lens (sizes the launch).
    ``out`` may be fp32 for parity measurement.  ``packed_pv`` (None = module default
    ``DECODE_PACKED_PV``): P.V on 16-bit operands — the MFMA kernel (P carried as a hi + lo pair of
    cache-dtype values, inside the fp32-P tolerance) where it is built, the dot2 VALU form elsewhere;
    ``force_valu`` keeps the VALU kernel; ``rounded_p`` asks the MFMA kernel for the single-rounding
    P of flash kernels (A/B measurements only).  ``fused_merge`` (None = on for workspaces made by
    ``new_decode_workspace``): the context partitions are merged inside the attention launch by the last-arriving
    wave of each (sequence, head group) instead of a second kernel — same bits.  Returns ``out``.
    ``slopes`` / ``sinks`` (fp32 [nq]): a distance bias (score - slope * (position - key position)) and one more term
    exp(sink) of the softmax's denominator, and the output times ``out_scale``; bf16 and the default mode only.
    """
    _gpu(out, q, k_cache, v_cache, block_table, seq_lens, workspace, slopes, sinks)
    nb, bs, hkv, d = k_cache.shape
    s = q.shape[0]
    nq = q.numel() // (s * d) if s else 0
    if block_table.dtype != torch.int32 or seq_lens.dtype != torch.int32:
        raise TypeError("block_table and seq_lens must be int32")
    if block_table.stride(1) != 1:
        raise ValueError("block_table rows must be contiguous")
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    if s == 0:
        return out
    partition_size = decode_auto_partition(s, hkv, max_seq_len, bs, partition_size, packed_pv, force_valu, head_dim=d)
    need = decode_workspace_bytes(s, nq, d, max_seq_len, partition_size)
    if need and (workspace is None or workspace.numel() * workspace.element_size() < need):
        workspace = new_decode_workspace(need, q.device)
    ready = _decode_ws_ready(workspace)
    if fused_merge is None:
        fused_merge = DECODE_FUSED_MERGE and ready
    elif fused_merge and not ready:
        raise ValueError("fused_merge needs a workspace from ops.new_decode_workspace (zeroed arrival counters)")
    if slopes is None and sinks is None and out_scale != 1.0:
        raise ValueError("out_scale goes with a distance bias or a sink")
    if slopes is not None or sinks is not None:
        _head_vectors(nq, slopes, sinks)
        if force_valu or rounded_p or packed_pv is False or out.dtype != q.dtype:
            raise ValueError("a distance bias or a sink runs in the default mode only")
        check("mi_paged_attn_decode_biased", lib.mi_paged_attn_decode_biased(
            _p(out), _p(q), _p(k_cache), _p(v_cache), _p(block_table), _p(seq_lens), _p(slopes), _p(sinks), float(out_scale), s, nq, hkv, d, bs,
            block_table.stride(0), int(max_seq_len), float(scale), q.stride(0), out.stride(0), cb, ct, ch, int(partition_size),
            _p(workspace), workspace.numel() * workspace.element_size() if workspace is not None else 0, _dt(q.dtype), _stream()))
        return out
    check("mi_paged_attn_decode", lib.mi_paged_attn_decode(
        _p(out), _p(q), _p(k_cache), _p(v_cache), _p(block_table), _p(seq_lens), s, nq, hkv, d, bs,
        block_table.stride(0), int(max_seq_len), float(scale), q.stride(0), out.stride(0), cb, ct, ch,
        int(partition_size), _p(workspace),
        workspace.numel() * workspace.element_size() if workspace is not None else 0,
        _dt(q.dtype), _dt(out.dtype),
        (_C.MI_DECODE_PACKED_PV if (DECODE_PACKED_PV if packed_pv is None else packed_pv) else 0)
        | (_C.MI_DECODE_FORCE_VALU if force_valu else 0)
        | (_C.MI_DECODE_ROUNDED_P if rounded_p else 0)
        | (_C.MI_DECODE_FUSED_MERGE if fused_merge else 0)
        | (_C.MI_DECODE_SKIP_MERGE if _skip_merge else 0)   # bench.py's kernel-only timing; never set by the product
        | (_C.MI_DECODE_NONTEMPORAL if (DECODE_NONTEMPORAL if nontemporal is None else nontemporal) else 0),
        _stream()))
    return out


def rope_decode_fusable(q: torch.Tensor, k_cache: torch.Tensor, positions: torch.Tensor, rot_dim: int,
                        partition_size: int, num_seqs: int, max_seq_len: int) -> bool:
    """Whether ``rope_cache_paged_attn_decode`` covers this call: the production decode kernel (matrix cores, nt
    streams, hi + lo P), full rotary, 1-D positions."""
    nb, bs, hkv, d = k_cache.shape
    if not (DECODE_PACKED_PV and DECODE_NONTEMPORAL and ROPE_DECODE_FUSION) or positions.dim() != 1 or rot_dim != d or bs < 16:
        return False
    ps = decode_auto_partition(num_seqs, hkv, max_seq_len, bs, partition_size, None, False, head_dim=d)
    return ps % 32 == 0


def rope_cache_paged_attn_decode(out: torch.Tensor, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                                 positions: torch.Tensor, cos_sin_cache: torch.Tensor, k_cache: torch.Tensor,
                                 v_cache: torch.Tensor, slot_mapping: torch.Tensor, block_table: torch.Tensor,
                                 seq_lens: torch.Tensor, max_seq_len: int, scale: float, partition_size: int = 0,
                                 workspace: Optional[torch.Tensor] = None, _skip_merge: bool = False,
                                 q_norm_weight: Optional[torch.Tensor] = None, k_norm_weight: Optional[torch.Tensor] = None,
                                 norm_eps: float = 1e-6) -> torch.Tensor:
    """``rope_neox_and_cache`` + ``paged_attn_decode`` of a pure-decode step in ONE launch (same bits): q is rotated in
    registers (the tensor keeps its un-rotated values), the token's rotated k and its v are written to the cache by the
    wave that owns the sequence's last context partition.  q [S, nq*d], k / v [S, nkv*d]: views of the qkv row."""
    _gpu(out, q, k, v, positions, cos_sin_cache, k_cache, v_cache, slot_mapping, block_table, seq_lens, workspace,
         q_norm_weight, k_norm_weight)
    if (q_norm_weight is None) != (k_norm_weight is None):
        raise ValueError("q_norm_weight and k_norm_weight come together")
    nb, bs, hkv, d = k_cache.shape
    s = q.shape[0]
    if s == 0:
        return out
    nq = q.numel() // (s * d)
    if block_table.dtype != torch.int32 or seq_lens.dtype != torch.int32:
        raise TypeError("block_table and seq_lens must be int32")
    if positions.dtype != torch.int64 or slot_mapping.dtype != torch.int64 or cos_sin_cache.dtype != torch.float32:
        raise TypeError("positions / slot_mapping must be int64 and cos_sin_cache float32")
    if positions.dim() != 1 or block_table.stride(1) != 1:
        raise ValueError("1-D positions and contiguous block_table rows required")
    max_pos, rot_dim = cos_sin_cache.shape
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    partition_size = decode_auto_partition(s, hkv, max_seq_len, bs, partition_size, None, False, head_dim=d)
    need = decode_workspace_bytes(s, nq, d, max_seq_len, partition_size)
    if need and (workspace is None or workspace.numel() * workspace.element_size() < need):
        workspace = new_decode_workspace(need, q.device)
    fused_merge = DECODE_FUSED_MERGE and _decode_ws_ready(workspace)
    check("mi_rope_cache_paged_attn_decode", lib.mi_rope_cache_paged_attn_decode(
        _p(out), _p(q), _p(k), _p(v), _p(positions), _p(cos_sin_cache), max_pos, rot_dim, _p(q_norm_weight),
        _p(k_norm_weight), float(norm_eps), _p(k_cache), _p(v_cache),
        _p(slot_mapping), _p(block_table), _p(seq_lens), s, nq, hkv, d, bs, block_table.stride(0), int(max_seq_len),
        float(scale), q.stride(0), k.stride(0), v.stride(0), out.stride(0), cb, ct, ch, int(partition_size), _p(workspace),
        workspace.numel() * workspace.element_size() if workspace is not None else 0, _dt(q.dtype), _dt(out.dtype),
        _C.MI_DECODE_PACKED_PV | _C.MI_DECODE_NONTEMPORAL | (_C.MI_DECODE_FUSED_MERGE if fused_merge else 0)
        | (_C.MI_DECODE_SKIP_MERGE if _skip_merge else 0), _stream()))
    return out


# --------------------------------------------------------------------------- A6
_PREFILL_WS: dict = {}   # device -> grow-only fp32 workspace of the split-context prefill (never captured in a graph)


def paged_attn_prefill(out: torch.Tensor, q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                       block_table: torch.Tensor, seq_lens: torch.Tensor, query_start_loc: torch.Tensor,
                       max_query_len: int, scale: float, max_seq_len: Optional[int] = None,
                       segments: int = 0, slopes: Optional[torch.Tensor] = None,
                       sinks: Optional[torch.Tensor] = None, out_scale: float = 1.0) -> torch.Tensor:
    """Varlen causal attention of query chunks against the paged cache (chunked prefill).

    ``max_seq_len`` (host upper bound of ``seq_lens``) lets a launch that would leave most CUs idle — the ragged last
    chunk of a long prompt, a TP shard with one KV head — split every tile's context into segments run by separate
    workgroups and merged afterwards (``mi_paged_attn_prefill_split``).  Without it nothing is split.
    ``segments``: 0 automatic, 1 never, n > 1 force n (tests).  ``slopes`` / ``sinks`` /
    ``out_scale``: as in ``paged_attn_decode``."""
    _gpu(out, q, k_cache, v_cache, block_table, seq_lens, query_start_loc, slopes, sinks)
    nb, bs, hkv, d = k_cache.shape
    t = q.shape[0]
    nq = q.numel() // (t * d) if t else 0
    s = seq_lens.shape[0]
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    if t == 0 or s == 0:
        return out
    ws, ws_bytes, msl = None, 0, 0
    if max_seq_len is not None and segments != 1:
        msl = int(max_seq_len)
        ws_bytes = int(lib.mi_paged_attn_prefill_workspace_bytes(t, s, int(max_query_len), msl, nq, hkv, d, int(segments)))
        if ws_bytes:
            ws = _PREFILL_WS.get(q.device)
            if ws is None or ws.numel() * 4 < ws_bytes:
                ws = _PREFILL_WS[q.device] = torch.empty((ws_bytes + 3) // 4, dtype=torch.float32, device=q.device)
    tail = (s, t, int(max_query_len), nq, hkv, d, bs, block_table.stride(0), float(scale), q.stride(0), out.stride(0), cb, ct, ch,
            _dt(q.dtype), msl, int(segments) if ws is not None else 1, _p(ws), ws.numel() * 4 if ws is not None else 0, _stream())
    head = (_p(out), _p(q), _p(k_cache), _p(v_cache), _p(block_table), _p(seq_lens), _p(query_start_loc))
    if slopes is not None or sinks is not None:
        _head_vectors(nq, slopes, sinks)
        check("mi_paged_attn_prefill_biased", lib.mi_paged_attn_prefill_biased(*head, _p(slopes), _p(sinks), float(out_scale), *tail))
    else:
        if out_scale != 1.0:
            raise ValueError("out_scale goes with a distance bias or a sink")
        check("mi_paged_attn_prefill_split", lib.mi_paged_attn_prefill_split(*head, *tail))
    return out


# --------------------------------------------------------------------------- A8
def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    _gpu(x, weight, out)
    x2 = x.view(-1, x.shape[-1])
    if out is None:
        out = torch.empty_like(x)
    o2 = out.view(-1, x.shape[-1])
    check("mi_rms_norm", lib.mi_rms_norm(_p(o2), _p(x2), _p(weight), float(eps), x2.shape[0], x2.shape[1],
                                          x2.stride(0), o2.stride(0), _dt(x.dtype), _stream()))
    return out


def fused_add_rms_norm(x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor, eps: float) -> None:
    """In place: residual <- x + residual; x <- rmsnorm(residual) * weight."""
    _gpu(x, residual, weight)
    x2 = x.view(-1, x.shape[-1])
    r2 = residual.view(-1, x.shape[-1])
    check("mi_fused_add_rms_norm", lib.mi_fused_add_rms_norm(
        _p(x2), _p(r2), _p(weight), float(eps), x2.shape[0], x2.shape[1], x2.stride(0), r2.stride(0),
        _dt(x.dtype), _stream()))


# --------------------------------------------------------------------------- A9
def silu_and_mul(x: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    _gpu(x, out)
    inter = x.shape[-1] // 2
    x2 = x.view(-1, x.shape[-1])
    if out is None:
        out = torch.empty(*x.shape[:-1], inter, dtype=x.dtype, device=x.device)
    o2 = out.view(-1, inter)
    check("mi_silu_and_mul", lib.mi_silu_and_mul(_p(o2), _p(x2), x2.shape[0], inter, x2.stride(0),
                                                  o2.stride(0), _dt(x.dtype), _stream()))
    return out


# -------------------------------------------------------------------------- A11
def mask_logits_argmax(logits: torch.Tensor, ranges: Sequence[tuple[int, int]] = (), col: int = -1,
                       ids: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Set up to two [lo, hi) column ranges and one column to -1e9 in place; greedy argmax."""
    _gpu(logits, ids)
    if len(ranges) > 2:
        raise ValueError("at most two masked ranges")
    r = list(ranges) + [(0, 0)] * (2 - len(ranges))
    t, v = logits.shape
    if ids is None:
        ids = torch.empty(t, dtype=torch.int64, device=logits.device)
    check("mi_mask_logits_argmax", lib.mi_mask_logits_argmax(
        _p(logits), _p(ids), t, v, logits.stride(0), r[0][0], r[0][1], r[1][0], r[1][1], int(col),
        _dt(logits.dtype), _stream()))
    return ids


def sample_tokens(logits: torch.Tensor, temperature: torch.Tensor, seed: torch.Tensor, offset: torch.Tensor,
                  top_k: Optional[torch.Tensor] = None, top_p: Optional[torch.Tensor] = None,
                  rep_penalty: Optional[torch.Tensor] = None, seen_bitmap: Optional[torch.Tensor] = None,
                  seen_row: Optional[torch.Tensor] = None, update_seen: bool = True,
                  ids: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Penalty -> temperature -> top-k -> top-p -> exponential-race draw, one launch (N2).

    temperature/top_p/rep_penalty fp32 [rows]; top_k/seen_row int32 [rows]; seed/offset int64 [rows] (bit
    patterns of the uint64 Philox key and draw counter); seen_bitmap int32 [state rows, words]."""
    _gpu(logits, temperature, seed, offset, top_k, top_p, rep_penalty, seen_bitmap, seen_row, ids)
    t, v = logits.shape
    if temperature.dtype != torch.float32 or seed.dtype != torch.int64 or offset.dtype != torch.int64:
        raise TypeError("temperature must be float32, seed/offset int64")
    for name, x, dt in (("top_k", top_k, torch.int32), ("top_p", top_p, torch.float32),
                        ("rep_penalty", rep_penalty, torch.float32), ("seen_bitmap", seen_bitmap, torch.int32),
                        ("seen_row", seen_row, torch.int32)):
        if x is not None and x.dtype != dt:
            raise TypeError(f"{name} must be {dt}")
    if ids is None:
        ids = torch.empty(t, dtype=torch.int64, device=logits.device)
    check("mi_sample_tokens", lib.mi_sample_tokens(
        _p(ids), _p(logits), t, v, logits.stride(0), _dt(logits.dtype), _p(temperature), _p(top_k), _p(top_p),
        _p(rep_penalty), _p(seen_bitmap), _p(seen_row), seen_bitmap.shape[1] if seen_bitmap is not None else 0,
        1 if update_seen else 0, _p(seed), _p(offset), _stream()))
    return ids


def sample_tokens_embed(logits: torch.Tensor, temperature: torch.Tensor, seed: torch.Tensor, offset: torch.Tensor,
                        top_k: Optional[torch.Tensor], top_p: Optional[torch.Tensor], table: torch.Tensor,
                        out_a: torch.Tensor, out_b: Optional[torch.Tensor] = None, ids_out: Optional[torch.Tensor] = None,
                        ids: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``sample_tokens`` (no repetition penalty) + ``embed_codes`` in one launch: the drawn id's row of ``table`` goes to
    ``out_a[r]`` (and ``out_b[r]``), the id also to ``ids_out[r]`` (any stride).  The code predictor's per-step draw."""
    _gpu(logits, temperature, seed, offset, top_k, top_p, table, out_a, out_b, ids_out, ids)
    t, v = logits.shape
    if temperature.dtype != torch.float32 or seed.dtype != torch.int64 or offset.dtype != torch.int64:
        raise TypeError("temperature must be float32, seed/offset int64")
    if (top_k is not None and top_k.dtype != torch.int32) or (top_p is not None and top_p.dtype != torch.float32):
        raise TypeError("top_k must be int32, top_p float32")
    if table.dim() != 2 or table.shape[0] < v or not table.is_contiguous() or table.element_size() != 2:
        raise ValueError("table must be a contiguous 16-bit [>= vocab, dim] tensor")
    dim = table.shape[1]
    for o in (out_a, out_b):
        if o is not None and (tuple(o.shape) != (t, dim) or o.dtype != table.dtype or o.stride(1) != 1):
            raise ValueError("out_a / out_b must be [rows, dim] of the table's dtype with contiguous rows")
    if ids_out is not None and (ids_out.dtype != torch.int64 or ids_out.dim() != 1 or ids_out.shape[0] != t):
        raise TypeError("ids_out must be int64 [rows]")
    if ids is None:
        ids = torch.empty(t, dtype=torch.int64, device=logits.device)
    check("mi_sample_tokens_embed", lib.mi_sample_tokens_embed(
        _p(ids), _p(logits), t, v, logits.stride(0), _dt(logits.dtype), _p(temperature), _p(top_k), _p(top_p), _p(seed),
        _p(offset), _p(table), dim, _p(out_a), out_a.stride(0), _p(out_b), out_b.stride(0) if out_b is not None else 0,
        _p(ids_out), ids_out.stride(0) if ids_out is not None else 0, _stream()))
    return ids


def talker_decode_embeds(out: torch.Tensor, embed_table: torch.Tensor, token_ids: torch.Tensor,
                         reply_rows: Optional[torch.Tensor] = None, reply_idx: Optional[torch.Tensor] = None) -> torch.Tensor:
    """out[t] = embed_table[token_ids[t]] (+ reply_rows[reply_idx[t]] where reply_idx[t] >= 0)."""
    _gpu(out, embed_table, token_ids, reply_rows, reply_idx)
    t = token_ids.shape[0]
    if token_ids.dtype != torch.int64 or (reply_idx is not None and reply_idx.dtype != torch.int64):
        raise TypeError("token_ids / reply_idx must be int64")
    check("mi_talker_decode_embeds", lib.mi_talker_decode_embeds(
        _p(out), _p(embed_table), _p(token_ids), _p(reply_rows), _p(reply_idx), t, embed_table.shape[1],
        embed_table.shape[0], reply_rows.shape[0] if reply_rows is not None else 0, out.stride(0),
        _dt(embed_table.dtype), _stream()))
    return out


# -------------------------------------------------------------------------- A13
def dynamic_int8_quant(x: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """Dynamic symmetric per-row int8 quantisation (int8_config.py:323-342): (int8 [rows, hidden], fp32 scale [rows])."""
    _gpu(x)
    x2 = x.view(-1, x.shape[-1])
    xq = torch.empty(x2.shape, dtype=torch.int8, device=x.device)
    xs = torch.empty(x2.shape[0], dtype=torch.float32, device=x.device)
    rc = lib.mi_int8_quant_rows(_p(xq), _p(xs), _p(x2), x2.shape[0], x2.shape[1], x2.stride(0), _dt(x.dtype), _stream())
    if rc == _C.MI_ERR_UNSUPPORTED:   # odd widths / alignments: the scalar kernel
        rc = lib.mi_dynamic_int8_quant(_p(xq), _p(xs), _p(x2), x2.shape[0], x2.shape[1], x2.stride(0), _dt(x.dtype),
                                       _stream())
    check("mi_dynamic_int8_quant", rc)
    return xq, xs


class QuantizedActs:
    """A W8A8 activation on its way into a linear layer: int8 rows + one fp32 scale per row, produced by the op in
    front of the linear (``rms_norm_int8``) instead of a separate quantisation launch."""

    __slots__ = ("xq", "xs", "lead", "dtype")

    def __init__(self, xq: torch.Tensor, xs: torch.Tensor, lead: tuple, dtype: torch.dtype):
        self.xq, self.xs, self.lead, self.dtype = xq, xs, lead, dtype


def rms_norm_int8(x: torch.Tensor, weight: torch.Tensor, eps: float, residual: Optional[torch.Tensor] = None) -> QuantizedActs:
    """RMSNorm (``residual`` None) or fused residual-add RMSNorm (``residual`` updated in place; ``x`` untouched) whose
    output leaves as the W8A8 activation — same bits as the norm followed by ``dynamic_int8_quant``, one launch."""
    _gpu(x, weight, residual)
    x2 = x.view(-1, x.shape[-1])
    r2 = residual.view(-1, x.shape[-1]) if residual is not None else None
    xq = torch.empty(x2.shape, dtype=torch.int8, device=x.device)
    xs = torch.empty(x2.shape[0], dtype=torch.float32, device=x.device)
    check("mi_rms_norm_int8", lib.mi_rms_norm_int8(_p(xq), _p(xs), _p(x2), _p(r2), _p(weight), float(eps), x2.shape[0],
                                                   x2.shape[1], x2.stride(0), r2.stride(0) if r2 is not None else 0,
                                                   _dt(x.dtype), _stream()))
    return QuantizedActs(xq, xs, tuple(x.shape[:-1]), x.dtype)


def int8_gemm_dequant(xq: torch.Tensor, x_scale: torch.Tensor, wq: torch.Tensor, w_scale: torch.Tensor,
                      bias: Optional[torch.Tensor], out_dtype: torch.dtype) -> torch.Tensor:
    _gpu(xq, x_scale, wq, w_scale, bias)
    m, k = xq.shape
    n = wq.shape[0]
    out = torch.empty(m, n, dtype=out_dtype, device=xq.device)
    check("mi_int8_gemm_dequant", lib.mi_int8_gemm_dequant(
        _p(out), _p(xq), _p(x_scale), _p(wq), _p(w_scale), _p(bias), m, n, k, out.stride(0),
        _dt(out_dtype), _stream()))
    return out


def int8_dequant(acc: torch.Tensor, x_scale: torch.Tensor, w_scale: torch.Tensor, bias: Optional[torch.Tensor],
                 out_dtype: torch.dtype) -> torch.Tensor:
    _gpu(acc, x_scale, w_scale, bias)
    m, n = acc.shape
    out = torch.empty(m, n, dtype=out_dtype, device=acc.device)
    check("mi_int8_dequant", lib.mi_int8_dequant(_p(out), _p(acc), _p(x_scale), _p(w_scale), _p(bias), m, n,
                                                  acc.stride(0), out.stride(0), _dt(out_dtype), _stream()))
    return out


_LINEAR_WS: dict = {}
_LINEAR_CNT: dict = {}   # device -> zeroed arrival counters of the in-launch split-K reduce (every launch leaves them zero)
# "1": split-K linears reduce inside their launch (mi_linear_fused_reduce: the last-arriving slice sums the slabs, same
# bits).  Built, tested, and measured SLOWER than the separate reduce launch at the shard shapes (down_proj at 128 rows
# x TP 4: 19.5 against 18.7 us; o_proj 11.1 / 10.7 — the last arriver's write-through, counter round trip and slab
# re-read cost more than the ~3.8 us launch they replace: profiles/r04i_fused_reduce.log), so it is opt-in.
LINEAR_FUSED_REDUCE = os.environ.get("VLLM_OMNI_AMD_LINEAR_FUSED_REDUCE", "0") == "1"
_LINEAR_WS_RETIRED: list = []   # outgrown workspaces stay allocated: a captured hipGraph may still write to them


def linear_supported(m: int, n: int, k: int, dtype: torch.dtype) -> bool:
    """Shape envelope of ``mi_linear`` (decode batches): rows <= 512 (two row blocks of 256 above 256), k a multiple
    of 128, n of 16."""
    return 0 < m <= 512 and k % 128 == 0 and n % 16 == 0 and dtype in (torch.bfloat16, torch.float16)


def linear(x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """y = x W^T (+ b) for a decode batch (<= 512 rows) by the weight-streaming kernel of csrc/skinny_gemm.hip;
    stands in for the library GEMM behind vLLM's ColumnParallelLinear / RowParallelLinear on the decode path."""
    _gpu(x, weight, bias)
    x2 = x.reshape(-1, x.shape[-1])
    if x2.stride(-1) != 1:
        x2 = x2.contiguous()
    m, k = x2.shape
    n = weight.shape[0]
    if weight.shape[1] != k or not weight.is_contiguous() or weight.dtype != x.dtype:
        raise ValueError("weight must be a contiguous [n, k] tensor of x's dtype")
    out = torch.empty(m, n, dtype=x.dtype, device=x.device)
    need = lib.mi_linear_workspace_bytes(m, n, k)
    ws = _linear_workspace(x.device, need) if need else None
    if need and LINEAR_FUSED_REDUCE:   # split-K: the reduce rides in the launch (last-arriving slice), same bits
        cnt = _LINEAR_CNT.get(x.device)
        if cnt is None:
            cnt = _LINEAR_CNT[x.device] = torch.zeros(_C.MI_LINEAR_COUNTER_BYTES // 4, dtype=torch.int32, device=x.device)
        check("mi_linear_fused_reduce", lib.mi_linear_fused_reduce(
            _p(out), _p(x2), _p(weight), _p(bias), m, n, k, x2.stride(0), out.stride(0), _p(ws), ws.numel(), _p(cnt),
            cnt.numel() * 4, _dt(x.dtype), _stream()))
        return out.view(*x.shape[:-1], n)
    check("mi_linear", lib.mi_linear(_p(out), _p(x2), _p(weight), _p(bias), m, n, k, x2.stride(0), out.stride(0),
                                     _p(ws) if need else None, ws.numel() if need else 0, _dt(x.dtype), _stream()))
    return out.view(*x.shape[:-1], n)


class SplitKPartials:
    """fp32 partials [split, m, n] of a split-K ``linear`` whose reduction has been left to the consumer: the fused
    residual-add + RMSNorm that follows (``fused_add_rms_norm_splitk``) or ``materialize()``.  The partials live in
    the shared workspace: they must be consumed before the next split-K linear on this device (checked)."""

    __slots__ = ("part", "split", "m", "n", "bias", "dtype", "lead", "device", "_gen")

    def __init__(self, part, split, m, n, bias, dtype, lead, device, gen):
        self.part, self.split, self.m, self.n, self.bias, self.dtype = part, split, m, n, bias, dtype
        self.lead, self.device, self._gen = lead, device, gen

    def _live(self) -> None:
        if _LINEAR_GEN.get(self.device) != self._gen:
            raise RuntimeError("split-K partials were overwritten by a later linear before they were reduced")

    def materialize(self) -> torch.Tensor:
        self._live()
        out = torch.empty(self.m, self.n, dtype=self.dtype, device=self.device)
        check("mi_linear_reduce", lib.mi_linear_reduce(_p(out), _p(self.part), self.split, _p(self.bias), self.m, self.n,
                                                       out.stride(0), _dt(self.dtype), _stream()))
        return out.view(*self.lead, self.n)


_LINEAR_GEN: dict = {}


def _linear_workspace(device, need: int) -> torch.Tensor:
    ws = _LINEAR_WS.get(device)
    if ws is None or ws.numel() < need:
        if ws is not None:
            _LINEAR_WS_RETIRED.append(ws)
        ws = _LINEAR_WS[device] = torch.empty(need, dtype=torch.uint8, device=device)
    _LINEAR_GEN[device] = _LINEAR_GEN.get(device, 0) + 1
    return ws


def linear_partials(x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor] = None) -> Optional[SplitKPartials]:
    """The streaming kernel of ``linear`` without its reduce launch, or None when this shape's plan has no split-K
    (nothing to defer).  Reduce with ``fused_add_rms_norm_splitk`` or ``.materialize()``."""
    _gpu(x, weight, bias)
    x2 = x.reshape(-1, x.shape[-1])
    if x2.stride(-1) != 1:
        x2 = x2.contiguous()
    m, k = x2.shape
    n = weight.shape[0]
    if weight.shape[1] != k or not weight.is_contiguous() or weight.dtype != x.dtype:
        raise ValueError("weight must be a contiguous [n, k] tensor of x's dtype")
    need = lib.mi_linear_workspace_bytes(m, n, k)
    if not need:
        return None
    ws = _linear_workspace(x.device, need)
    split = ctypes.c_int32(0)
    check("mi_linear_partials", lib.mi_linear_partials(_p(x2), _p(weight), m, n, k, x2.stride(0), _p(ws), ws.numel(),
                                                       ctypes.byref(split), _dt(x.dtype), _stream()))
    return SplitKPartials(ws, split.value, m, n, bias, x.dtype, tuple(x.shape[:-1]), x.device, _LINEAR_GEN[x.device])


def fused_add_rms_norm_splitk(p: SplitKPartials, residual: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """residual <- rnd(sum of the partials (+ bias)) + residual (in place); returns rmsnorm(residual) * weight — the
    reduce of a split-K ``linear`` folded into the fused-add RMSNorm behind it, bit-identical to the two apart."""
    _gpu(residual, weight)
    p._live()
    r2 = residual.view(-1, residual.shape[-1])
    if r2.shape != (p.m, p.n):
        raise ValueError("residual shape does not match the partials")
    out = torch.empty(p.m, p.n, dtype=p.dtype, device=p.device)
    check("mi_fused_add_rms_norm_splitk", lib.mi_fused_add_rms_norm_splitk(
        _p(out), _p(p.part), p.split, _p(p.bias), _p(r2), _p(weight), float(eps), p.m, p.n, out.stride(0), r2.stride(0),
        _dt(p.dtype), _stream()))
    return out.view(*p.lead, p.n)


def rope_neox_and_cache_splitk(part: SplitKPartials, num_q_heads: int, num_kv_heads: int, head_dim: int,
                               positions: torch.Tensor, cos_sin_cache: torch.Tensor, k_cache: torch.Tensor,
                               v_cache: torch.Tensor, slot_mapping: torch.Tensor,
                               mrope_section: Optional[torch.Tensor] = None,
                               q_norm_weight: Optional[torch.Tensor] = None,
                               k_norm_weight: Optional[torch.Tensor] = None, norm_eps: float = 1e-6) -> torch.Tensor:
    """``rope_neox_and_cache`` fed by the split-K partials of ``qkv_proj`` (``linear_partials``): returns the rotated
    q [T, nq*d]; k and v go to the cache only.  Bit-identical to ``linear`` + ``rope_neox_and_cache``."""
    _gpu(positions, cos_sin_cache, k_cache, v_cache, slot_mapping, q_norm_weight, k_norm_weight)
    part._live()
    if part.n != (num_q_heads + 2 * num_kv_heads) * head_dim:
        raise ValueError("partials row is not [q heads | k heads | v heads]")
    if positions.dtype != torch.int64 or cos_sin_cache.dtype != torch.float32 or slot_mapping.dtype != torch.int64:
        raise TypeError("positions / slot_mapping must be int64 and cos_sin_cache float32")
    max_pos, rot_dim = cos_sin_cache.shape
    sec = None
    row_stride = 0
    if positions.dim() == 2:
        if mrope_section is None:
            raise ValueError("positions is [3, T]: mrope_section required")
        sec = (ctypes.c_int32 * 3)(*[int(x) for x in mrope_section])
        row_stride = positions.stride(0)
        if positions.stride(1) != 1:
            raise ValueError("positions rows must be contiguous")
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    q_out = torch.empty(part.m, num_q_heads * head_dim, dtype=part.dtype, device=part.device)
    check("mi_rope_neox_and_cache_splitk", lib.mi_rope_neox_and_cache_splitk(
        _p(q_out), _p(part.part), part.split, _p(part.bias), _p(positions), row_stride,
        ctypes.cast(sec, ctypes.c_void_p) if sec is not None else None, _p(cos_sin_cache), max_pos, rot_dim,
        _p(q_norm_weight), _p(k_norm_weight), float(norm_eps), _p(k_cache), _p(v_cache), _p(slot_mapping), part.m,
        num_q_heads, num_kv_heads, head_dim, k_cache.shape[1], q_out.stride(0), cb, ct, ch, _dt(part.dtype), _stream()))
    return q_out


def linear_silu_mul(x: torch.Tensor, weight: torch.Tensor, clamped: Optional[tuple[float, float]] = None) -> torch.Tensor:
    """silu(x Wg^T) * (x Wu^T) for a decode batch, weight = [gate rows; up rows] — ``gate_up_proj`` and the
    ``SiluAndMul`` behind it (qwen2_old.py:65-68) in one launch; the [m, 2 I] intermediate never reaches memory.
    ``clamped`` (alpha, limit): the activation of ``clamped_glu`` instead."""
    _gpu(x, weight)
    x2 = x.reshape(-1, x.shape[-1])
    if x2.stride(-1) != 1:
        x2 = x2.contiguous()
    m, k = x2.shape
    if weight.shape[0] % 2 or weight.shape[1] != k or not weight.is_contiguous() or weight.dtype != x.dtype:
        raise ValueError("weight must be a contiguous [2 * inter, k] tensor of x's dtype")
    inter = weight.shape[0] // 2
    out = torch.empty(m, inter, dtype=x.dtype, device=x.device)
    if clamped is not None:
        check("mi_linear_clamped_glu", lib.mi_linear_clamped_glu(
            _p(out), _p(x2), _p(weight), m, inter, k, x2.stride(0), out.stride(0), float(clamped[0]), float(clamped[1]),
            _dt(x.dtype), _stream()))
        return out.view(*x.shape[:-1], inter)
    check("mi_linear_silu_mul", lib.mi_linear_silu_mul(_p(out), _p(x2), _p(weight), m, inter, k, x2.stride(0),
                                                       out.stride(0), _dt(x.dtype), _stream()))
    return out.view(*x.shape[:-1], inter)



INT8_TILE_ROWS = 512   # rows one launch of the tiled W8A8 kernel takes


def int8_linear_supported(m: int, n: int, k: int) -> bool:
    """Shape envelope of ONE launch of the tiled W8A8 kernel (csrc/skinny_gemm.hip on int8 rows)."""
    return 0 < m <= INT8_TILE_ROWS and k % 128 == 0 and n % 16 == 0 and k > 0


def int8_linear(x: torch.Tensor, wq: torch.Tensor, w_scale: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """W8A8 linear of the reference's scheme (vllm_omni/quantization/int8_config.py:323-342: dynamic symmetric
    per-token activation scale, per-output-channel weight scale): hand-written per-token quantisation kernel, then
    ONE launch of the tiled int8 kernel — LDS-DMA ring, `v_mfma_i32_16x16x64_i8`, dequantisation + bias in the
    epilogue (``mi_int8_linear``; split-K shapes add its small reduce launch).  Prefill chunks (more than 512 rows)
    take the library contraction with the in-tree dequantisation epilogue (``torch._int_mm`` + ``mi_int8_dequant``),
    tiny weights the simple MFMA kernel ``mi_int8_gemm_dequant`` — the measured policy is spelled out below;
    ``VLLM_OMNI_AMD_INT8`` = ``library`` / ``simple`` / ``tiled`` forces one path (cross-checks, A/B runs).  Integer
    sums are exact on every path, so all three agree bit for bit."""
    if isinstance(x, QuantizedActs):
        xq, xs, lead, dtype = x.xq, x.xs, x.lead, x.dtype
    else:
        xq, xs = dynamic_int8_quant(x.reshape(-1, x.shape[-1]))
        lead, dtype = tuple(x.shape[:-1]), x.dtype
    m, k = xq.shape
    n = wq.shape[0]
    mode = os.environ.get("VLLM_OMNI_AMD_INT8", "kernel")
    lib_ok = m > 16 and k % 8 == 0 and n % 8 == 0
    tiled_ok = int8_linear_supported(min(m, INT8_TILE_ROWS), n, k)
    # Policy from profiles/r03_int8_linear_bench.log (all paths give the same bits, so this is speed only):
    #   <= 512 rows: the tiled kernel (24-48 us against 27-86 library, 33-263 simple at the S-A shapes, 256 rows) —
    #      except weights of <= 2 M elements at >= 256 rows (the S-B attention / expert shapes), where the simple MFMA
    #      kernel has less fixed cost (12.7 against 16.6 us);
    #   more rows (prefill chunks): the library contraction + the in-tree dequantisation epilogue (60 / 163 us against
    #      150 / 307 us for the tiled kernel run in 512-row blocks and 252 / 931 us for the simple kernel at 2048 rows);
    #      the tiled kernel in row blocks where the library cannot take the shape; the simple kernel last.
    if mode == "library" and lib_ok:
        y = int8_dequant(torch._int_mm(xq, wq.t()), xs, w_scale, bias, dtype)
    elif mode == "simple":
        y = int8_gemm_dequant(xq, xs, wq, w_scale, bias, dtype)
    elif m <= INT8_TILE_ROWS and tiled_ok and not (m >= 256 and n * k <= (1 << 21) and mode != "tiled"):
        y = int8_linear_q(xq, xs, wq, w_scale, bias, dtype)
    elif m > INT8_TILE_ROWS and lib_ok and mode != "tiled":
        y = int8_dequant(torch._int_mm(xq, wq.t()), xs, w_scale, bias, dtype)
    elif m > INT8_TILE_ROWS and tiled_ok:
        y = torch.empty(m, n, dtype=dtype, device=xq.device)   # rows of a GEMM are independent: same bits as one launch
        for r0 in range(0, m, INT8_TILE_ROWS):
            r1 = min(r0 + INT8_TILE_ROWS, m)
            int8_linear_q(xq[r0:r1], xs[r0:r1], wq, w_scale, bias, dtype, out=y[r0:r1])
    else:
        y = int8_gemm_dequant(xq, xs, wq, w_scale, bias, dtype)
    return y.view(*lead, n)


def int8_linear_q(xq: torch.Tensor, xs: torch.Tensor, wq: torch.Tensor, w_scale: torch.Tensor,
                  bias: Optional[torch.Tensor], out_dtype: torch.dtype, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The tiled W8A8 kernel on already-quantised activations (xq int8 [m, k], xs fp32 [m])."""
    _gpu(xq, xs, wq, w_scale, bias, out)
    m, k = xq.shape
    n = wq.shape[0]
    if wq.shape[1] != k or not wq.is_contiguous() or xq.stride(1) != 1:
        raise ValueError("wq must be a contiguous int8 [n, k] tensor; xq rows must be contiguous")
    if out is None:
        out = torch.empty(m, n, dtype=out_dtype, device=xq.device)
    elif out.shape != (m, n) or out.dtype != out_dtype or out.stride(1) != 1:
        raise ValueError("out must be an [m, n] tensor of out_dtype with contiguous rows")
    need = lib.mi_int8_linear_workspace_bytes(m, n, k)
    ws = _linear_workspace(xq.device, need) if need else None
    check("mi_int8_linear", lib.mi_int8_linear(_p(out), _p(xq), _p(xs), _p(wq), _p(w_scale), _p(bias), m, n, k,
                                               xq.stride(0), out.stride(0), _p(ws) if need else None,
                                               ws.numel() if need else 0, _dt(out_dtype), _stream()))
    return out


class Int8SplitKPartials:
    """Exact int32 partials [split, m, n] of a split-K W8A8 projection whose reduction + dequantisation has been left
    to the fused-add RMSNorm behind it (``fused_add_rms_norm_splitk_int8``) or ``materialize()``; same workspace
    discipline as ``SplitKPartials``."""

    __slots__ = ("part", "split", "m", "n", "xs", "ws", "bias", "dtype", "lead", "device", "_gen")

    def __init__(self, part, split, m, n, xs, ws, bias, dtype, lead, device, gen):
        self.part, self.split, self.m, self.n, self.xs, self.ws = part, split, m, n, xs, ws
        self.bias, self.dtype, self.lead, self.device, self._gen = bias, dtype, lead, device, gen

    def _live(self) -> None:
        if _LINEAR_GEN.get(self.device) != self._gen:
            raise RuntimeError("split-K partials were overwritten by a later linear before they were reduced")

    def materialize(self) -> torch.Tensor:
        """The 16-bit projection output (what mi_int8_linear would have returned): reduce + dequant on the device."""
        self._live()
        z = torch.zeros(self.m, self.n, dtype=self.dtype, device=self.device)      # residual = 0: x + 0 = x exactly
        one = torch.ones(self.n, dtype=self.dtype, device=self.device)
        check("mi_fused_add_rms_norm_splitk_int8", lib.mi_fused_add_rms_norm_splitk_int8(
            _p(torch.empty_like(z)), None, _p(self.part), self.split, _p(self.xs), _p(self.ws), _p(self.bias), _p(z),
            _p(one), 1e-6, self.m, self.n, z.stride(0), z.stride(0), _dt(self.dtype), _stream()))
        return z.view(*self.lead, self.n)


def int8_linear_partials(x, wq: torch.Tensor, w_scale: torch.Tensor, bias: Optional[torch.Tensor]) -> Optional[Int8SplitKPartials]:
    """The split-K W8A8 kernel without its reduce launch, or None when this shape has no split-K plan (decided BEFORE
    the activation is quantised: the caller's fallback quantises it itself)."""
    n, k = wq.shape
    m = x.xq.shape[0] if isinstance(x, QuantizedActs) else x.numel() // x.shape[-1]
    if not int8_linear_supported(m, n, k):
        return None
    need = lib.mi_int8_linear_workspace_bytes(m, n, k)
    if not need:
        return None
    if isinstance(x, QuantizedActs):
        xq, xs, lead, dtype = x.xq, x.xs, x.lead, x.dtype
    else:
        xq, xs = dynamic_int8_quant(x.reshape(-1, x.shape[-1]))
        lead, dtype = tuple(x.shape[:-1]), x.dtype
    ws = _linear_workspace(xq.device, need)
    split = ctypes.c_int32(0)
    check("mi_int8_linear_partials", lib.mi_int8_linear_partials(_p(xq), _p(wq), m, n, k, xq.stride(0), _p(ws), ws.numel(),
                                                                 ctypes.byref(split), _stream()))
    return Int8SplitKPartials(ws, split.value, m, n, xs, w_scale, bias, dtype, lead, xq.device, _LINEAR_GEN[xq.device])


def fused_add_rms_norm_splitk_int8(p: Int8SplitKPartials, residual: torch.Tensor, weight: torch.Tensor, eps: float,
                                   quant: bool = False):
    """residual <- rnd(dequant(sum of the int32 partials) (+ bias)) + residual (in place); returns
    rmsnorm(residual) * weight — as a 16-bit tensor, or (quant) as the next W8A8 linear's ``QuantizedActs``."""
    _gpu(residual, weight)
    p._live()
    r2 = residual.view(-1, residual.shape[-1])
    if r2.shape != (p.m, p.n):
        raise ValueError("residual shape does not match the partials")
    dev = residual.device
    if quant:
        out = torch.empty(p.m, p.n, dtype=torch.int8, device=dev)
        qs = torch.empty(p.m, dtype=torch.float32, device=dev)
    else:
        out = torch.empty(p.m, p.n, dtype=p.dtype, device=dev)
        qs = None
    check("mi_fused_add_rms_norm_splitk_int8", lib.mi_fused_add_rms_norm_splitk_int8(
        _p(out), _p(qs), _p(p.part), p.split, _p(p.xs), _p(p.ws), _p(p.bias), _p(r2), _p(weight), float(eps), p.m, p.n,
        out.stride(0), r2.stride(0), _dt(p.dtype), _stream()))
    if quant:
        return QuantizedActs(out, qs, p.lead, p.dtype)
    return out.view(*p.lead, p.n)


def int8_linear_silu_mul(x: torch.Tensor, wq: torch.Tensor, w_scale: torch.Tensor) -> torch.Tensor:
    """``act_fn(gate_up_proj(x))`` with W8A8 weights in one GEMM launch (+ the activation quantisation in front)."""
    if isinstance(x, QuantizedActs):
        xq, xs, lead, dtype = x.xq, x.xs, x.lead, x.dtype
    else:
        xq, xs = dynamic_int8_quant(x.reshape(-1, x.shape[-1]))
        lead, dtype = tuple(x.shape[:-1]), x.dtype
    m, k = xq.shape
    inter = wq.shape[0] // 2
    out = torch.empty(m, inter, dtype=dtype, device=xq.device)
    for r0 in range(0, m, INT8_TILE_ROWS):   # one launch per 512 rows (prefill chunks): rows are independent
        r1 = min(r0 + INT8_TILE_ROWS, m)
        check("mi_int8_linear_silu_mul", lib.mi_int8_linear_silu_mul(
            _p(out[r0:r1]), _p(xq[r0:r1]), _p(xs[r0:r1]), _p(wq), _p(w_scale), r1 - r0, inter, k, xq.stride(0),
            out.stride(0), _dt(dtype), _stream()))
    return out.view(*lead, inter)


# --------------------------------------------------------------------------- N4: fused sparse MoE
def moe_route(router_logits: torch.Tensor, top_k: int, norm_topk_prob: bool, round_to: Optional[torch.dtype] = None,
              want_counts: bool = True, bias: Optional[torch.Tensor] = None, sigmoid: bool = False):
    """-> (topk_ids int32 [T, k], topk_weights fp32 [T, k], expert_counts int32 [E] or None).  ``want_counts=False``:
    no per-expert counting and no launch to zero the counters (``fused_moe``: the grouping counts the ids itself).
    ``bias`` (fp32 [E]) is added to the logits.  ``norm_topk_prob``: a softmax over the chosen logits only (``sigmoid``: each
    logit's sigmoid instead of the softmax, divided by the chosen ones' sum)."""
    _gpu(router_logits, bias)
    t, e = router_logits.shape
    _head_vectors(e, bias)
    ids = torch.empty(t, top_k, dtype=torch.int32, device=router_logits.device)
    w = torch.empty(t, top_k, dtype=torch.float32, device=router_logits.device)
    counts = torch.empty(e, dtype=torch.int32, device=router_logits.device) if want_counts else None
    check("mi_moe_route", lib.mi_moe_route(_p(ids), _p(w), _p(counts), _p(router_logits), _p(bias), t, e, router_logits.stride(0),
                                           int(top_k), 1 if norm_topk_prob else 0, int(sigmoid), _dt(router_logits.dtype),
                                           -1 if round_to is None else _dt(round_to), _stream()))
    return ids, w, counts


def _moe_align(ids: torch.Tensor, num_experts: int, max_rows: int, rows_per_tile: int):
    """(token, choice) pairs grouped by expert in tiles: -> sorted_pairs, row_of_pair, tile_expert, num_tiles"""
    i32 = dict(dtype=torch.int32, device=ids.device)
    out = (torch.empty(max_rows, **i32), torch.empty(ids.numel(), **i32), torch.empty(max_rows // rows_per_tile, **i32),
           torch.empty(1, **i32))
    check("mi_moe_align", lib.mi_moe_align(*map(_p, out), _p(ids), None, ids.numel(), num_experts, max_rows, rows_per_tile, _stream()))
    return out


def fused_moe(x: torch.Tensor, router_logits: torch.Tensor, w_gate_up: torch.Tensor, w_down: torch.Tensor, top_k: int,
              norm_topk_prob: bool = False, shared_out: Optional[torch.Tensor] = None,
              shared_gate_weight: Optional[torch.Tensor] = None, routing=None,
              rows_per_tile: int = 0) -> torch.Tensor:
    """Sparse-MoE layer output for x [T, H]: route -> align -> gated expert GEMM -> down expert GEMM ->
    weighted combine (+ sigmoid-gated shared expert output computed by the caller).  w_gate_up [E, 2I, H] (gate rows
    then up rows), w_down [E, H, I].  ``routing`` = (ids int32, weights fp32) skips the router (tests)."""
    _gpu(x, router_logits, w_gate_up, w_down, None if callable(shared_out) else shared_out, shared_gate_weight)
    t, h = x.shape
    e, two_i, _ = w_gate_up.shape
    i = two_i // 2
    dev = x.device
    if routing is None:
        ids, w, _ = moe_route(router_logits, top_k, norm_topk_prob, round_to=x.dtype, want_counts=False)
    else:
        ids, w = routing
    rpt = rows_per_tile or int(lib.mi_moe_rows_per_tile(t, top_k, e))
    max_rows = int(lib.mi_moe_max_rows(t, top_k, e, rpt))
    sorted_pairs, row_of_pair, tile_expert, num_tiles = _moe_align(ids, e, max_rows, rpt)   # counts the ids itself
    act = torch.empty(max_rows, i, dtype=x.dtype, device=dev)
    part = torch.empty(max_rows, h, dtype=x.dtype, device=dev)
    dt = _dt(x.dtype)
    check("mi_moe_expert_gemm", lib.mi_moe_expert_gemm(
        _p(act), _p(x), _p(w_gate_up), _p(sorted_pairs), _p(tile_expert), _p(num_tiles), max_rows // rpt, _C.MI_MOE_GATED, None, i, h, top_k,
        x.stride(0), act.stride(0), w_gate_up.stride(0), rpt, dt, _stream()))
    check("mi_moe_expert_gemm", lib.mi_moe_expert_gemm(
        _p(part), _p(act), _p(w_down), _p(sorted_pairs), _p(tile_expert), _p(num_tiles), max_rows // rpt, _C.MI_MOE_PLAIN, None, h, i, top_k,
        act.stride(0), part.stride(0), w_down.stride(0), rpt, dt, _stream()))
    out = torch.empty_like(x)
    if callable(shared_out):      # the caller computed it beside this path (another stream): join here
        shared_out = shared_out()
        _gpu(shared_out)
    check("mi_moe_combine", lib.mi_moe_combine(
        _p(out), _p(part), _p(row_of_pair), _p(w), _p(shared_out), _p(x), _p(shared_gate_weight), t, h, top_k,
        part.stride(0), out.stride(0), x.stride(0), shared_out.stride(0) if shared_out is not None else 0, dt, _stream()))
    return out


# ------------------------------------------------- 32-bit residual stream, latent attention, gated delta rule
def _rows(t: torch.Tensor) -> tuple[int, int]:
    """(row stride, columns) of a 2-D tensor with contiguous rows"""
    if t.dim() != 2 or t.stride(1) != 1:
        raise ValueError("expected a 2-D tensor with contiguous rows")
    return t.stride(0), t.shape[1]


def _i32(*ts: Optional[torch.Tensor]) -> None:
    for t in ts:
        if t is not None and (t.dtype != torch.int32 or not t.is_contiguous()):
            raise TypeError("expected a contiguous int32 tensor")


def _i64(*ts: Optional[torch.Tensor]) -> None:
    for t in ts:
        if t is not None and (t.dtype != torch.int64 or not t.is_contiguous()):
            raise TypeError("expected a contiguous int64 tensor")


def residual_norm(x: torch.Tensor, y: Union[torch.Tensor, "SplitKPartials"], w_post: torch.Tensor,
                  w_pre: Optional[torch.Tensor], eps: float, want_h: bool = True) -> Optional[torch.Tensor]:
    """``x += rms_norm(y; w_post)`` in place (x fp32 [T, W]); returns ``rms_norm(x; w_pre)``, or x cast to w_post's dtype
    when ``w_pre`` is None.  ``y`` may be the split-K partials of the linear in front."""
    part = isinstance(y, SplitKPartials)
    if part:
        y._live()
        if y.bias is not None:
            raise ValueError("residual_norm takes partials of a linear without bias")
    src = y.part if part else y
    _gpu(x, src, w_post, w_pre)
    xs, width = _rows(x)
    rows = x.shape[0]
    if x.dtype != torch.float32 or w_post.numel() != width or (w_pre is not None and (w_pre.numel() != width or w_pre.dtype != w_post.dtype)):
        raise ValueError("residual_norm: fp32 stream and weights of its width")
    if part:
        if (y.m, y.n) != (rows, width):
            raise ValueError("partials of another shape")
        ys = width
    else:
        ys, yw = _rows(y)
        if y.shape[0] != rows or yw != width or y.dtype != w_post.dtype:
            raise ValueError("sublayer output of another shape or dtype")
    h = torch.empty(rows, width, dtype=w_post.dtype, device=x.device) if want_h else None
    check("mi_residual_norm", lib.mi_residual_norm(
        _p(x), _p(src), y.split if part else 0, _p(w_post), _p(w_pre), _p(h), float(eps), rows, width, xs, ys,
        width, _dt(w_post.dtype), _stream()))
    return h


def pair_embed_norm(table: torch.Tensor, pairs: torch.Tensor, w_pre: torch.Tensor, ids: torch.Tensor,
                    prev_ids: Optional[torch.Tensor], slots: torch.Tensor, last_token: torch.Tensor, positions: torch.Tensor,
                    scale: float, mul_prev: int, mul_cur: int, eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """Scaled token row + pair row (``pairs`` [buckets + 1, W]) -> (x fp32, rms_norm(x; w_pre))."""
    _gpu(table, pairs, w_pre, ids, prev_ids, slots, last_token, positions)
    _i64(ids, prev_ids, last_token, positions)
    _i32(slots)
    t, (vocab, width) = ids.shape[0], table.shape
    if slots.numel() < t or positions.numel() < t or (prev_ids is not None and prev_ids.numel() < t):
        raise ValueError("pair_embed_norm: index arrays shorter than the rows")
    if pairs.shape[1] != width or w_pre.numel() != width or not (table.is_contiguous() and pairs.is_contiguous()):
        raise ValueError("pair_embed_norm: tables of different widths")
    x = torch.empty(t, width, dtype=torch.float32, device=table.device)
    h = torch.empty(t, width, dtype=table.dtype, device=table.device)
    check("mi_pair_embed_norm", lib.mi_pair_embed_norm(
        _p(x), _p(h), _p(table), _p(pairs), _p(w_pre), _p(ids), _p(prev_ids), _p(slots), _p(last_token), _p(positions),
        float(scale), int(mul_prev), int(mul_cur), pairs.shape[0] - 1, float(eps), t, width, vocab, width, width,
        _dt(table.dtype), _stream()))
    return x, h


def gelu_lookup_mul(z: torch.Tensor, table: torch.Tensor, ids: torch.Tensor, offset: int) -> torch.Tensor:
    """``gelu_tanh(z) * table[ids, offset : offset + z.shape[1]]``"""
    _gpu(z, table, ids)
    _i64(ids)
    zs, dim = _rows(z)
    ts, cols = _rows(table)
    if offset + dim > cols or ids.numel() < z.shape[0] or table.dtype != z.dtype:
        raise ValueError("gelu_lookup_mul: slice outside the table, or dtypes differ")
    out = torch.empty(z.shape[0], dim, dtype=z.dtype, device=z.device)
    check("mi_gelu_lookup_mul", lib.mi_gelu_lookup_mul(_p(out), _p(z), _p(table), _p(ids), z.shape[0], dim, zs, ts, int(offset),
                                                       table.shape[0], _dt(z.dtype), _stream()))
    return out


def clamped_glu(gate_up: torch.Tensor, alpha: float, limit: float) -> torch.Tensor:
    """[T, 2 F] gate | up -> [T, F]: g sigmoid(alpha g) (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit)"""
    _gpu(gate_up)
    gs, two = _rows(gate_up)
    t, ff = gate_up.shape[0], two // 2
    out = torch.empty(t, ff, dtype=gate_up.dtype, device=gate_up.device)
    check("mi_clamped_glu", lib.mi_clamped_glu(_p(out), _p(gate_up), t, ff, gs, ff, float(alpha), float(limit),
                                               _dt(gate_up.dtype), _stream()))
    return out


def latent_norm_cache(x: torch.Tensor, q_weight: torch.Tensor, c_weight: Optional[torch.Tensor], cache: Optional[torch.Tensor],
                      slot_mapping: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    """Row = query latent | new cache latent: returns the normed query latent, writes the normed cache rows
    (``cache`` [blocks, block_size, rank]) at their slots.  ``c_weight`` None: no cache half."""
    _gpu(x, q_weight, c_weight, cache, slot_mapping)
    xs, cols = _rows(x)
    t, nq = x.shape[0], q_weight.numel()
    nc = 0 if c_weight is None else c_weight.numel()
    if cols < nq + nc or q_weight.dtype != x.dtype:
        raise ValueError("latent_norm_cache: row shorter than its two halves")
    bs = cb = ct = 0
    if nc:
        _i64(slot_mapping)
        if cache.dim() != 3 or cache.shape[2] != nc or cache.stride(2) != 1 or cache.dtype != x.dtype or slot_mapping.numel() < t:
            raise ValueError("latent_norm_cache: cache [blocks, block_size, rank] of x's dtype, one slot per row")
        bs, cb, ct = cache.shape[1], cache.stride(0), cache.stride(1)
    out = torch.empty(t, nq, dtype=x.dtype, device=x.device)
    check("mi_latent_norm_cache", lib.mi_latent_norm_cache(
        _p(x), xs, _p(q_weight), nq, _p(out), _p(c_weight), nc, _p(cache) if nc else None, _p(slot_mapping) if nc else None,
        bs, cb, ct, float(eps), t, _dt(x.dtype), _stream()))
    return out


def head_gemm(x: torch.Tensor, w: torch.Tensor, transposed: bool = False) -> torch.Tensor:
    """``y[t, h] = w[h] @ x[t, h]`` for x [T, H * K] and w [H, N, K] (``transposed``: w [H, K, N], used as w[h]^T)."""
    _gpu(x, w)
    xs, cols = _rows(x)
    hh, a, b = w.shape
    n, k = (b, a) if transposed else (a, b)
    if cols != hh * k or w.dtype != x.dtype:
        raise ValueError("head_gemm: x [T, heads * k] and w of one dtype")
    y = torch.empty(x.shape[0], hh * n, dtype=x.dtype, device=x.device)
    sn, sk = (w.stride(2), w.stride(1)) if transposed else (w.stride(1), w.stride(2))
    check("mi_head_gemm", lib.mi_head_gemm(_p(y), _p(x), _p(w), x.shape[0], hh, n, k, hh * n, xs, w.stride(0), sn, sk,
                                           _dt(x.dtype), _stream()))
    return y


def _latent_cache(cache: torch.Tensor, rank: int) -> tuple[int, int, int]:
    if cache.dim() != 3 or cache.shape[2] != rank or cache.stride(2) != 1:
        raise ValueError("latent cache must be [blocks, block_size, rank] with contiguous rows")
    return cache.shape[1], cache.stride(0), cache.stride(1)


def latent_attn_rows(q: torch.Tensor, cache: torch.Tensor, block_table: torch.Tensor, seq_lens: torch.Tensor,
                     query_start_loc: torch.Tensor, heads: int, window: int, scale: float, row0: int = 0,
                     out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Absorbed latent attention of rows [row0, T) of ``q`` [T, heads * rank]; any sizes and dtypes."""
    _gpu(q, cache, block_table, seq_lens, query_start_loc)
    _i32(seq_lens, query_start_loc)
    rank = q.shape[1] // heads
    bs, cb, ct = _latent_cache(cache, rank)
    if not q.is_contiguous() or cache.dtype != q.dtype or block_table.dtype != torch.int32 or block_table.stride(1) != 1:
        raise ValueError("latent_attn_rows: contiguous q of the cache's dtype, int32 block table")
    out = torch.empty_like(q) if out is None else out
    check("mi_latent_attn_rows", lib.mi_latent_attn_rows(
        _p(out), _p(q), _p(cache), _p(block_table), _p(seq_lens), _p(query_start_loc), row0, q.shape[0] - row0,
        seq_lens.shape[0], heads, rank, bs, min(int(window), 2**31 - 1), float(scale), cb, ct, block_table.stride(0),
        _dt(q.dtype), _stream()))
    return out


def latent_decode_supported(dtype: torch.dtype, kv_rank: int, dim: int, vdim: int, block_size: int) -> bool:
    return (dtype == torch.bfloat16 and kv_rank % 8 == 0 and kv_rank <= 512 and dim % 8 == 0 and vdim % 4 == 0
            and block_size & (block_size - 1) == 0)


def latent_prefill_supported(dtype: torch.dtype, kv_rank: int, dim: int, vdim: int) -> bool:
    return dtype == torch.bfloat16 and kv_rank % 8 == 0 and dim % 8 == 0 and vdim % 8 == 0 and max(dim, vdim) <= 256


def head_gemm_nt(x: torch.Tensor, w: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``head_gemm`` for w [H, N, K] on the matrix cores (bf16, K a multiple of 8, N of 4)."""
    _gpu(x, w, out)
    xs, cols = _rows(x)
    hh, n, k = w.shape
    if cols != hh * k or w.dtype != torch.bfloat16 or x.dtype != torch.bfloat16 or not w.is_contiguous():
        raise ValueError("head_gemm_nt: bf16 x [T, heads * k] and contiguous w [heads, n, k]")
    y = torch.empty(x.shape[0], hh * n, dtype=x.dtype, device=x.device) if out is None else out
    check("mi_head_gemm_nt", lib.mi_head_gemm_nt(_p(y), _p(x), _p(w), x.shape[0], hh, n, k, y.stride(0), xs, n * k, _stream()))
    return y


def latent_decode(q: torch.Tensor, cache: torch.Tensor, block_table: torch.Tensor, seq_lens: torch.Tensor, heads: int, window: int,
                  max_seq_len: int, scale: float) -> torch.Tensor:
    """Absorbed latent attention of one query per request, ``q`` [R, heads * rank] bf16."""
    _gpu(q, cache, block_table, seq_lens)
    _i32(seq_lens)
    n, rank = q.shape[0], q.shape[1] // heads
    bs, cb, ct = _latent_cache(cache, rank)
    if not q.is_contiguous() or q.dtype != torch.bfloat16 or cache.dtype != torch.bfloat16 or block_table.dtype != torch.int32:
        raise TypeError("latent_decode: contiguous bf16 q, bf16 cache, int32 block table")
    if seq_lens.shape[0] < n or block_table.shape[0] < n or block_table.stride(1) != 1:
        raise ValueError("latent_decode: one block-table row and length per query")
    window = min(int(window), 2**31 - 1)
    need = lib.mi_latent_decode_workspace_bytes(n, heads, rank, window, max_seq_len)
    ws = torch.empty(need, dtype=torch.uint8, device=q.device) if need else None
    out = torch.empty_like(q)
    check("mi_latent_decode", lib.mi_latent_decode(
        _p(out), _p(q), _p(cache), _p(block_table), _p(seq_lens), n, heads, rank, bs, window, max_seq_len, float(scale), cb, ct,
        block_table.stride(0), _p(ws), need, _stream()))
    return out


def latent_gather(cache: torch.Tensor, ctx_start: torch.Tensor, ctx_rows: int, block_table: torch.Tensor, seq_lens: torch.Tensor,
                  query_start_loc: torch.Tensor, window: int) -> torch.Tensor:
    """[ctx_rows, rank]: per request the cache rows its portion can see, 64-row aligned, zero padded."""
    _gpu(cache, ctx_start, block_table, seq_lens, query_start_loc)
    _i32(ctx_start, seq_lens, query_start_loc)
    rank, n = cache.shape[2], seq_lens.shape[0]
    bs, cb, ct = _latent_cache(cache, rank)
    if cache.dtype != torch.bfloat16 or ctx_start.shape[0] < n + 1 or query_start_loc.shape[0] < n + 1 or block_table.shape[0] < n:
        raise ValueError("latent_gather: bf16 cache and one entry per request")
    ctx = torch.empty(ctx_rows, rank, dtype=cache.dtype, device=cache.device)
    check("mi_latent_gather", lib.mi_latent_gather(
        _p(ctx), _p(cache), _p(ctx_start), _p(block_table), _p(seq_lens), _p(query_start_loc), n, ctx_rows, rank, bs,
        min(int(window), 2**31 - 1), cb, ct, block_table.stride(0), _stream()))
    return ctx


def latent_prefill(out: torch.Tensor, q: torch.Tensor, k: torch.Tensor, vt: torch.Tensor, ctx_start: torch.Tensor,
                   seq_lens: torch.Tensor, query_start_loc: torch.Tensor, max_query_len: int, heads: int, window: int,
                   scale: float) -> torch.Tensor:
    """Windowed attention of prompt portions: q [T, heads * dim], k [ctx, heads * dim], vt [heads * vdim, ctx] -> out rows."""
    _gpu(out, q, k, vt, ctx_start, seq_lens, query_start_loc)
    _i32(ctx_start, seq_lens, query_start_loc)
    qs, qc = _rows(q)
    ks, kc = _rows(k)
    vs, vc = _rows(vt)
    os_, oc = _rows(out)
    n = seq_lens.shape[0]
    if qc != kc or vt.shape[0] != oc or vc != k.shape[0] or qc % heads or oc % heads or out.shape[0] < q.shape[0]:
        raise ValueError("latent_prefill: sizes do not fit")
    if any(t.dtype != torch.bfloat16 for t in (out, q, k, vt)) or ctx_start.shape[0] < n + 1 or query_start_loc.shape[0] < n + 1:
        raise TypeError("latent_prefill: bf16 operands and one entry per request")
    check("mi_latent_prefill", lib.mi_latent_prefill(
        _p(out), _p(q), _p(k), _p(vt), _p(ctx_start), _p(seq_lens), _p(query_start_loc), n, max_query_len, heads, qc // heads,
        oc // heads, min(int(window), 2**31 - 1), float(scale), os_, qs, ks, vs, _stream()))
    return out


def gated_delta_step(proj: torch.Tensor, conv_w: torch.Tensor, a_log: torch.Tensor, dt_bias: torch.Tensor, norm_w: torch.Tensor,
                     state: torch.Tensor, ring: torch.Tensor, slots: torch.Tensor, query_start_loc: torch.Tensor,
                     seq_lens: torch.Tensor, kv_heads: int, eps: float, out: torch.Tensor, req0: int, num_reqs: int,
                     update_ring: bool = True, gate: Optional[torch.Tensor] = None, beta: Optional[torch.Tensor] = None,
                     decay: Optional[torch.Tensor] = None, sigmoid_gate: bool = False) -> torch.Tensor:
    """Gated delta rule of requests [req0, req0 + num_reqs), token by token.  ``state`` fp32 [slots, H, D, V], ``ring``
    [slots, taps, channels]; ``out`` [T, H * V] receives the requests' rows.  ``proj`` holds rows q | k | v, and behind them
    gate | b | a where these do not come as tensors of their own; ``decay`` [T, H] or, one per key channel, [T, H * D]
    (``dt_bias`` has as many)."""
    a = _delta_args(proj, conv_w, a_log, dt_bias, norm_w, state, ring, slots, query_start_loc, seq_lens, kv_heads, eps, out, req0,
                    num_reqs, gate, beta, decay, sigmoid_gate)
    check("mi_gated_delta_step", lib.mi_gated_delta_step(ctypes.byref(a), int(update_ring), _dt(proj.dtype), _stream()))
    return out


def gated_delta_chunked(proj, conv_w, a_log, dt_bias, norm_w, state, ring, slots, query_start_loc, seq_lens, kv_heads: int,
                        eps: float, out: torch.Tensor, req0: int, num_reqs: int, row0: int, max_query_len: int, gate=None, beta=None,
                        decay=None, sigmoid_gate: bool = False) -> torch.Tensor:
    """The same for prompt portions (requests [req0, req0 + num_reqs) own the rows from ``row0`` to the end of ``proj``), 64
    tokens at a time on the fp32 matrix cores; sizes outside its envelope (dim or vdim > 256) go token by token."""
    a = _delta_args(proj, conv_w, a_log, dt_bias, norm_w, state, ring, slots, query_start_loc, seq_lens, kv_heads, eps, out, req0,
                    num_reqs, gate, beta, decay, sigmoid_gate)
    rows = proj.shape[0] - row0
    need = lib.mi_gated_delta_chunked_workspace_bytes(rows, num_reqs, a.heads, a.dim, a.vdim, a.channel_decay)
    if not need:
        check("mi_gated_delta_step", lib.mi_gated_delta_step(ctypes.byref(a), 1, _dt(proj.dtype), _stream()))
        return out
    ws = torch.empty(need, dtype=torch.uint8, device=proj.device)
    check("mi_gated_delta_chunked", lib.mi_gated_delta_chunked(ctypes.byref(a), row0, rows, max_query_len, _p(ws), need,
                                                               _dt(proj.dtype), _stream()))
    return out


def _delta_args(proj, conv_w, a_log, dt_bias, norm_w, state, ring, slots, query_start_loc, seq_lens, kv_heads, eps, out, req0, num_reqs,
                gate, beta, decay, sigmoid_gate) -> "_C.GatedDeltaArgs":
    _gpu(proj, conv_w, a_log, dt_bias, norm_w, state, ring, slots, query_start_loc, seq_lens, out, gate, beta, decay)
    _i32(slots, query_start_loc, seq_lens)
    ps, cols = _rows(proj)
    os_, oc = _rows(out)
    _, hh, d, v = state.shape
    taps, ch = ring.shape[1], ring.shape[2]
    at = ch                       # what is not given apart follows q | k | v in the rows of ``proj``
    views = []
    for t, n in ((gate, hh * v), (beta, hh), (decay, hh)):
        if t is None:
            t = proj[:, at:at + n]
            at += n
        views.append(t)
    gate, beta, decay = views
    channel = d > 1 and decay.shape[1] == hh * d      # one key channel: the same thing
    if cols < at or out.shape[0] < proj.shape[0]:
        raise ValueError("gated_delta: projection rows [q | k | v | gate | b | a], one output row each")
    if not (state.is_contiguous() and ring.is_contiguous() and conv_w.is_contiguous()):
        raise ValueError("gated_delta: contiguous state, ring and conv weights")
    if state.dtype != torch.float32 or a_log.dtype != torch.float32 or dt_bias.dtype != torch.float32:
        raise TypeError("recurrent state, A_log and dt_bias are fp32")
    if (ch != 2 * kv_heads * d + hh * v or tuple(conv_w.shape) != (ch, taps) or oc != hh * v or norm_w.numel() != v
            or a_log.numel() != hh or dt_bias.numel() != (hh * d if channel else hh)):
        raise ValueError("gated_delta: sizes do not fit")
    if any(t.shape[0] < proj.shape[0] or t.stride(1) != 1 or t.shape[1] != n
           for t, n in ((gate, hh * v), (beta, hh), (decay, hh * d if channel else hh))):
        raise ValueError("gated_delta: gate, b and decay rows do not fit")
    if any(t.dtype != proj.dtype for t in (conv_w, norm_w, ring, out, gate, beta, decay)):
        raise TypeError("gated_delta: one activation dtype")
    if req0 + num_reqs > seq_lens.shape[0] or slots.shape[0] < req0 + num_reqs or query_start_loc.shape[0] < req0 + num_reqs + 1:
        raise ValueError("gated_delta: request range outside the metadata")
    return _C.GatedDeltaArgs(_p(proj), _p(gate), _p(beta), _p(decay), _p(conv_w), _p(norm_w), _p(a_log), _p(dt_bias), _p(state), _p(ring),
                             _p(slots), _p(query_start_loc), _p(seq_lens), _p(out), ps, gate.stride(0), beta.stride(0), decay.stride(0),
                             os_, req0, num_reqs, hh, kv_heads, d, v, taps, int(channel), int(sigmoid_gate), float(eps))


# ------------------------------------------------- layers with mixer and feed-forward side by side
class ExpertRows:
    """Output rows of routed experts, one per (token, choice), and how they sum up: ``residual_add_norm`` does it.  ``weights``
    None: every row counts once (``top`` choices a token)."""

    def __init__(self, part: torch.Tensor, weights: Optional[torch.Tensor], row_of_pair: Optional[torch.Tensor], top: Optional[int] = None):
        self.part, self.weights, self.row_of_pair = part, weights, row_of_pair
        self.top = weights.shape[1] if weights is not None else top

    def check(self, rows: int, width: int, dtype) -> int:
        """row stride of ``part``, after a look at the sizes"""
        _gpu(self.part, self.row_of_pair, self.weights)
        ps, pw = _rows(self.part)
        ww = self.weights
        if pw != width or self.part.dtype != dtype or (ww is not None and (ww.shape[0] != rows or ww.dtype != torch.float32
                                                                           or not ww.is_contiguous())):
            raise ValueError("expert rows of another shape or dtype")
        if self.row_of_pair is None and self.part.shape[0] < rows * self.top:
            raise ValueError("one row per pair expected")
        if self.row_of_pair is not None and self.row_of_pair.numel() < rows * self.top:
            raise ValueError("a row per pair expected")
        _i32(self.row_of_pair)
        return ps


def residual_add_norm(x: torch.Tensor, y: Union[torch.Tensor, "SplitKPartials"], w_pre: Optional[torch.Tensor], eps: float,
                      h: torch.Tensor, experts: Optional[ExpertRows] = None, w_shift: float = 0.0, start: bool = False) -> torch.Tensor:
    """``x += y (+ the experts' rows)`` in place (x fp32 [T, W]; ``start``: x = y instead), then ``h`` = x / rms(x) * (w_pre +
    w_shift), or x cast when ``w_pre`` is None.  ``y``: rows of h's dtype, fp32 rows, or split-K partials."""
    part = isinstance(y, SplitKPartials)
    if part:
        y._live()
        if y.bias is not None:
            raise ValueError("residual_add_norm takes partials of a linear without bias")
    src = y.part if part else y
    _gpu(x, src, w_pre, h)
    xs, width = _rows(x)
    hs, hw = _rows(h)
    rows = x.shape[0]
    if x.dtype != torch.float32 or hw != width or h.shape[0] < rows or (w_pre is not None and (w_pre.numel() != width or w_pre.dtype != h.dtype)):
        raise ValueError("residual_add_norm: fp32 stream, h and weights of its width")
    if part:
        if (y.m, y.n) != (rows, width):
            raise ValueError("partials of another shape")
        split, ys = y.split, width
    else:
        ys, yw = _rows(y)
        if y.shape[0] != rows or yw != width or y.dtype not in (h.dtype, torch.float32):
            raise ValueError("layer output of another shape or dtype")
        split = 1 if y.dtype == torch.float32 and h.dtype != torch.float32 else 0
    top, rp, ww, ps, prt = 0, None, None, 0, None
    if experts is not None:
        prt, rp, ww, top = experts.part, experts.row_of_pair, experts.weights, experts.top
        if ww is None:
            raise ValueError("residual_add_norm takes weighted experts' rows")
        ps = experts.check(rows, width, h.dtype)
    check("mi_residual_add_norm", lib.mi_residual_add_norm(
        _p(x), _p(src), split, _p(prt), _p(rp), _p(ww), top, _p(w_pre), float(w_shift), _p(h), int(start), float(eps), rows, width, xs,
        ys, hs, ps, _dt(h.dtype), _stream()))
    return h


def embed_norm(table: torch.Tensor, ids: torch.Tensor, x: torch.Tensor, w_pre: Optional[torch.Tensor], eps: float, h: torch.Tensor,
               copy: Optional[torch.Tensor] = None, w_shift: float = 0.0) -> None:
    """x = table[ids] (fp32), ``copy`` = the same in the table's dtype, ``h`` as in ``residual_add_norm``"""
    _gpu(table, ids, x, w_pre, h, copy)
    _i64(ids)
    xs, width = _rows(x)
    hs, hw = _rows(h)
    cs, cw = _rows(copy) if copy is not None else (0, width)
    rows = x.shape[0]
    if x.dtype != torch.float32 or not table.is_contiguous() or (table.shape[1], hw, cw) != (width,) * 3 or ids.numel() != rows:
        raise ValueError("embed_norm: sizes do not fit")
    if h.shape[0] < rows or (copy is not None and copy.shape[0] < rows) or (w_pre is not None and w_pre.numel() != width):
        raise ValueError("embed_norm: sizes do not fit")
    if any(t is not None and t.dtype != table.dtype for t in (h, copy, w_pre)):
        raise TypeError("embed_norm: one dtype")
    check("mi_embed_norm", lib.mi_embed_norm(_p(x), _p(h), _p(copy), _p(table), _p(w_pre), float(w_shift), _p(ids), float(eps), rows, width,
                                             table.shape[0], xs, hs, cs, _dt(table.dtype), _stream()))


def glu(out: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, act: str) -> torch.Tensor:
    """``out = act(gate) * up``; act "silu" or "gelu_tanh".  gate and up are column blocks of one matrix."""
    _gpu(out, gate, up)
    gs, ff = _rows(gate)
    us, uf = _rows(up)
    os_, of = _rows(out)
    if gs != us or not ff == uf == of or not gate.shape[0] == up.shape[0] == out.shape[0] or not gate.dtype == up.dtype == out.dtype:
        raise ValueError("glu: gate, up and out of one shape, gate and up of one row stride")
    check("mi_glu", lib.mi_glu(_p(out), _p(gate), _p(up), gate.shape[0], ff, gs, os_,
                               {"silu": _C.MI_ACT_SILU, "gelu_tanh": _C.MI_ACT_GELU_TANH}[act], _dt(gate.dtype), _stream()))
    return out


def head_norm_cache(x: torch.Tensor, q_weight: Optional[torch.Tensor], k_weight: Optional[torch.Tensor], k_cache: torch.Tensor,
                    v_cache: torch.Tensor, slot_mapping: torch.Tensor, positions: torch.Tensor, num_q_heads: int, dim: int, vdim: int,
                    eps: float, temp_coef: float = 0.0, temp_every: int = 1) -> torch.Tensor:
    """Rows q | k | v: per-head norms, the query temperature, K / V cache write; returns q, heads laid out as in the cache."""
    _gpu(x, q_weight, k_weight, k_cache, v_cache, slot_mapping, positions)
    _i64(slot_mapping, positions)
    xs, cols = _rows(x)
    rows = x.shape[0]
    _, bs, g, hd = k_cache.shape
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    if cols != (num_q_heads + g) * dim + g * vdim or slot_mapping.numel() < rows or positions.numel() < rows:
        raise ValueError("head_norm_cache: sizes do not fit")
    for w in (q_weight, k_weight):
        if w is not None and (w.numel() != dim or w.dtype != x.dtype):
            raise ValueError("head_norm_cache: norm weights of one head's size")
    if x.dtype != k_cache.dtype:
        raise TypeError("cache and activations share a dtype")
    q = torch.empty(rows, num_q_heads * hd, dtype=x.dtype, device=x.device)
    check("mi_head_norm_cache", lib.mi_head_norm_cache(
        _p(x), xs, _p(q_weight), _p(k_weight), _p(q), q.stride(0), _p(k_cache), _p(v_cache), _p(slot_mapping), _p(positions), rows,
        num_q_heads, g, dim, vdim, hd, bs, cb, ct, ch, float(temp_coef), int(temp_every), float(eps), _dt(x.dtype), _stream()))
    return q


def attn_rows(out: torch.Tensor, q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_table: torch.Tensor,
              seq_lens: torch.Tensor, query_start_loc: torch.Tensor, scale: float, slopes: Optional[torch.Tensor] = None,
              sinks: Optional[torch.Tensor] = None, row0: int = 0, out_scale: float = 1.0) -> torch.Tensor:
    """Causal attention of rows [row0, T), any sizes and types; ``slopes`` / ``sinks`` as in ``paged_attn_decode``."""
    _gpu(out, q, k_cache, v_cache, block_table, seq_lens, query_start_loc, slopes, sinks)
    _i32(seq_lens, query_start_loc)
    _, bs, g, hd = k_cache.shape
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    qs, qc = _rows(q)
    os_, oc = _rows(out)
    nq = qc // hd
    if qc != nq * hd or oc != qc or out.shape[0] < q.shape[0] or block_table.dtype != torch.int32 or block_table.stride(1) != 1:
        raise ValueError("attn_rows: sizes do not fit")
    if not q.dtype == out.dtype == k_cache.dtype:
        raise TypeError("attn_rows: one dtype")
    _head_vectors(nq, slopes, sinks)
    check("mi_attn_rows", lib.mi_attn_rows(
        _p(out), _p(q), _p(k_cache), _p(v_cache), _p(block_table), _p(seq_lens), _p(query_start_loc), _p(slopes), _p(sinks), float(out_scale), row0,
        q.shape[0] - row0, seq_lens.shape[0], nq, g, hd, bs, float(scale), qs, os_, cb, ct, ch, block_table.stride(0), _dt(q.dtype),
        _stream()))
    return out


def paged_attn_bias_supported(dtype: torch.dtype, head_dim: int, block_size: int) -> bool:
    """whether the matrix-core paged-attention kernels take a distance bias and a sink at these sizes"""
    return dtype == torch.bfloat16 and head_dim in (64, 128) and block_size >= 16 and block_size & (block_size - 1) == 0


def lightning_attn(qkv: torch.Tensor, gate: torch.Tensor, norm_w: torch.Tensor, decay: torch.Tensor, log2_decay: torch.Tensor,
                   state: torch.Tensor, slots: torch.Tensor, query_start_loc: torch.Tensor, seq_lens: torch.Tensor, eps: float,
                   out: torch.Tensor, req0: int, num_reqs: int, row0: int, rows: int, max_query_len: int, mul: float = 1.0,
                   chunked: bool = True) -> torch.Tensor:
    """Decayed linear attention of requests [req0, req0 + num_reqs), which own rows [row0, row0 + rows).  ``state`` fp32 [slots,
    H, D, V]; ``chunked``: 64 tokens at a time (sizes outside that form go token by token)."""
    _gpu(qkv, gate, norm_w, decay, log2_decay, state, slots, query_start_loc, seq_lens, out)
    _i32(slots, query_start_loc, seq_lens)
    ps, cols = _rows(qkv)
    gs, gc = _rows(gate)
    os_, oc = _rows(out)
    _, hh, d, v = state.shape
    if cols != hh * (2 * d + v) or gc != hh * v or oc != hh * v or norm_w.numel() != hh * v or decay.numel() != hh or log2_decay.numel() != hh:
        raise ValueError("lightning_attn: sizes do not fit")
    if any(t.dtype != torch.float32 for t in (state, decay, log2_decay)) or not state.is_contiguous():
        raise TypeError("lightning_attn: contiguous fp32 state and decays")
    if any(t.dtype != qkv.dtype for t in (gate, norm_w, out)):
        raise TypeError("lightning_attn: one activation dtype")
    if min(qkv.shape[0], gate.shape[0], out.shape[0]) < row0 + rows:
        raise ValueError("lightning_attn: rows outside the tensors")
    if req0 + num_reqs > seq_lens.shape[0] or slots.shape[0] < req0 + num_reqs or query_start_loc.shape[0] < req0 + num_reqs + 1:
        raise ValueError("lightning_attn: request range outside the metadata")
    need = lib.mi_lightning_workspace_bytes(rows, num_reqs, hh, d, v, 1) if chunked else 0
    chunked = need > 0
    if not chunked:
        need = lib.mi_lightning_workspace_bytes(rows, num_reqs, hh, d, v, 0)
    ws = torch.empty(max(need, 1), dtype=torch.uint8, device=qkv.device)
    a = _C.LightningArgs(_p(qkv), _p(gate), _p(norm_w), _p(decay), _p(log2_decay), _p(state), _p(slots), _p(query_start_loc), _p(seq_lens),
                         _p(out), ps, gs, os_, req0, num_reqs, hh, d, v, float(eps), float(mul))
    check("mi_lightning_attn", lib.mi_lightning_attn(ctypes.byref(a), row0, rows, max_query_len, int(chunked), _p(ws), need,
                                                     _dt(qkv.dtype), _stream()))
    return out


def moe_router_logits(h: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """h weight^T, sums and result in fp32 (a library product; ``moe_route`` adds a bias)"""
    _gpu(h, weight)
    if h.dtype == torch.float32:
        return torch.nn.functional.linear(h, weight)
    return torch.mm(h, weight.t(), out_dtype=torch.float32)


def moe_expert_rows(x: torch.Tensor, ids: torch.Tensor, weights: torch.Tensor, w_up: torch.Tensor, w_down: torch.Tensor,
                    act: str = "silu_gated", weigh_input: bool = False) -> ExpertRows:
    """Experts on the rows routed to them, not yet summed: grouped matrix-core products where the sizes allow, the any-size
    kernel (fp32, odd sizes) elsewhere.  ``act`` "silu_gated": ``w_up`` holds gate, then up rows; "relu_squared": up rows only.
    ``weigh_input`` (relu_squared): the weights scale what an expert reads, the rows then sum up as they are."""
    _gpu(x, ids, weights, w_up, w_down)
    _i32(ids)
    t, h = x.shape
    top = ids.shape[1]
    gated = act == "silu_gated"
    if act not in ("silu_gated", "relu_squared") or (gated and weigh_input):
        raise ValueError(f"moe_expert_rows: act {act!r}, weigh_input {weigh_input} is not built")
    form = _C.MI_MOE_GATED if gated else _C.MI_MOE_RELU_SQUARED
    pw = weights if weigh_input else None
    if tuple(weights.shape) != (t, top) or weights.dtype != torch.float32 or not weights.is_contiguous():
        raise ValueError("moe_expert_rows: one fp32 weight per choice")
    e, ups, k = w_up.shape
    i = ups // 2 if gated else ups
    xs = _rows(x)[0]
    if k != h or tuple(w_down.shape) != (e, h, i) or not w_up.is_contiguous() or not w_down.is_contiguous() or w_up.dtype != x.dtype:
        raise ValueError("moe_expert_rows: expert weights do not fit")
    dt, dev = _dt(x.dtype), x.device
    if x.dtype == torch.bfloat16 and h % 8 == 0 and i % 8 == 0 and xs % 8 == 0:
        guard = h % 128 or i % (64 if gated else 128)
        rpt = int(lib.mi_moe_rows_per_tile(t, top, e))
        rpt = min(rpt, 64) if guard else rpt
        max_rows = int(lib.mi_moe_max_rows(t, top, e, rpt))
        sorted_pairs, row_of_pair, tile_expert, num_tiles = _moe_align(ids, e, max_rows, rpt)
        mid = torch.empty(max_rows, i, dtype=x.dtype, device=dev)
        part = torch.empty(max_rows, h, dtype=x.dtype, device=dev)
        for out, a, w, f, s, n, kk in ((mid, x, w_up, form, pw, i, h), (part, mid, w_down, _C.MI_MOE_PLAIN, None, h, i)):
            check("mi_moe_expert_gemm", lib.mi_moe_expert_gemm(
                _p(out), _p(a), _p(w), _p(sorted_pairs), _p(tile_expert), _p(num_tiles), max_rows // rpt, f, _p(s), n, kk, top, a.stride(0),
                out.stride(0), w.stride(0), rpt, dt, _stream()))
        return ExpertRows(part, None if weigh_input else weights, row_of_pair, top)
    mid = torch.empty(t * top, i, dtype=x.dtype, device=dev)
    part = torch.empty(t * top, h, dtype=x.dtype, device=dev)
    for out, a, w, f, s, n, kk in ((mid, x, w_up, form, pw, i, h), (part, mid, w_down, _C.MI_MOE_PLAIN, None, h, i)):
        check("mi_moe_pair_gemm", lib.mi_moe_pair_gemm(_p(out), _p(a), _p(w), _p(ids), t * top, e, f, _p(s), n, kk, top, a.stride(0),
                                                       out.stride(0), w.stride(0), dt, _stream()))
    return ExpertRows(part, None if weigh_input else weights, None, top)


# ------------------------------------------------- a filter in front of every sublayer, heads that mix their softmax weights
class ConvRing:
    """The filter of one sublayer in one layer run: ``weight`` [taps, width] (the last one for the row itself) and the ring of
    every state slot's last taps - 1 rows [slots, taps - 1, width] (None when taps is 1)."""

    def __init__(self, weight: torch.Tensor, ring: Optional[torch.Tensor]):
        taps, width = weight.shape
        if not weight.is_contiguous():
            raise ValueError("filter weights must be contiguous")
        if taps > 1 and (ring is None or tuple(ring.shape[1:]) != (taps - 1, width) or not ring.is_contiguous() or ring.dtype != weight.dtype):
            raise ValueError("a ring of taps - 1 rows per slot, in the weights' dtype")
        self.weight, self.ring, self.taps, self.width = weight, ring, taps, width


def _conv_rows(conv: Optional[ConvRing], slots, positions, rows: int, width: int, dtype):
    """C arguments (weight, ring, slots, positions, taps) of the one-token form"""
    if conv is None:
        return None, None, None, None, 0
    _gpu(conv.weight, conv.ring, slots, positions)
    _i32(slots)
    _i64(positions)
    if conv.width != width or conv.weight.dtype != dtype or slots.numel() < rows or positions.numel() < rows:
        raise ValueError("filter of another width or dtype, or too few slots and positions")
    return _p(conv.weight), _p(conv.ring), _p(slots), _p(positions), conv.taps


def residual_add_norm_conv(x: torch.Tensor, y: Union[torch.Tensor, "SplitKPartials"], w_pre: Optional[torch.Tensor], eps: float,
                           h: torch.Tensor, w_shift: float = 0.0, add_row: Optional[torch.Tensor] = None,
                           conv: Optional[ConvRing] = None, slots: Optional[torch.Tensor] = None,
                           positions: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``residual_add_norm`` with a row ``add_row`` added to every row's stream, and the filter over ``h`` of rows that are
    their sequences' only new ones (``slots``, ``positions`` per row)."""
    part = isinstance(y, SplitKPartials)
    if part:
        y._live()
        if y.bias is not None:
            raise ValueError("partials of a linear without bias")
    src = y.part if part else y
    _gpu(x, src, w_pre, h, add_row)
    xs, width = _rows(x)
    hs, hw = _rows(h)
    rows = x.shape[0]
    if x.dtype != torch.float32 or hw != width or h.shape[0] < rows:
        raise ValueError("residual_add_norm_conv: fp32 stream, h of its width")
    for w in (w_pre, add_row):
        if w is not None and (w.numel() != width or w.dtype != h.dtype or not w.is_contiguous()):
            raise ValueError("residual_add_norm_conv: weights of the stream's width in h's dtype")
    if part:
        if (y.m, y.n) != (rows, width):
            raise ValueError("partials of another shape")
        split, ys = y.split, width
    else:
        ys, yw = _rows(y)
        if y.shape[0] != rows or yw != width or y.dtype not in (h.dtype, torch.float32):
            raise ValueError("layer output of another shape or dtype")
        split = 1 if y.dtype == torch.float32 and h.dtype != torch.float32 else 0
    cw, ring, sl, pos, taps = _conv_rows(conv, slots, positions, rows, width, h.dtype)
    check("mi_residual_add_norm_conv", lib.mi_residual_add_norm_conv(
        _p(x), _p(src), split, _p(add_row), _p(w_pre), float(w_shift), _p(h), cw, ring, sl, pos, taps, float(eps), rows, width, xs, ys, hs,
        _dt(h.dtype), _stream()))
    return h


def embed_pos_norm(table: torch.Tensor, ids: torch.Tensor, x: torch.Tensor, w_pre: Optional[torch.Tensor], eps: float, h: torch.Tensor,
                   positions: torch.Tensor, scale: float = 1.0, pos_table: Optional[torch.Tensor] = None,
                   add_row: Optional[torch.Tensor] = None, w_shift: float = 0.0, conv: Optional[ConvRing] = None,
                   slots: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x = scale * table[ids] + pos_table[positions] + add_row (fp32); ``h`` as in ``residual_add_norm_conv``"""
    _gpu(table, ids, x, w_pre, h, positions, pos_table, add_row)
    _i64(ids, positions)
    xs, width = _rows(x)
    hs, hw = _rows(h)
    rows = x.shape[0]
    if x.dtype != torch.float32 or not table.is_contiguous() or (table.shape[1], hw) != (width, width) or h.shape[0] < rows \
            or ids.numel() != rows or positions.numel() < rows:
        raise ValueError("embed_pos_norm: sizes do not fit")
    for w in (w_pre, add_row):
        if w is not None and (w.numel() != width or not w.is_contiguous()):
            raise ValueError("embed_pos_norm: sizes do not fit")
    if pos_table is not None and (pos_table.shape[1] != width or not pos_table.is_contiguous()):
        raise ValueError("embed_pos_norm: position table of another width")
    if any(t is not None and t.dtype != table.dtype for t in (h, w_pre, pos_table, add_row)):
        raise TypeError("embed_pos_norm: one dtype")
    cw, ring, sl, _, taps = _conv_rows(conv, slots, positions, rows, width, h.dtype)
    check("mi_embed_pos_norm", lib.mi_embed_pos_norm(
        _p(x), _p(h), _p(table), float(scale), _p(pos_table), _p(positions), pos_table.shape[0] if pos_table is not None else 0,
        _p(add_row), _p(w_pre), float(w_shift), _p(ids), cw, ring, sl, taps, float(eps), rows, width, table.shape[0], xs, hs,
        _dt(table.dtype), _stream()))
    return h


def input_conv(h: torch.Tensor, conv: ConvRing, slots: torch.Tensor, query_start_loc: torch.Tensor, seq_lens: torch.Tensor,
               num_reqs: int, max_query_len: int, req0: int = 0) -> torch.Tensor:
    """h plus the filter over it, for portions of any length; leaves each request's last rows in its ring"""
    _gpu(h, conv.weight, conv.ring, slots, query_start_loc, seq_lens)
    _i32(slots, query_start_loc, seq_lens)
    hs, width = _rows(h)
    if conv.width != width or conv.weight.dtype != h.dtype:
        raise ValueError("filter of another width or dtype")
    if min(slots.numel(), seq_lens.numel(), query_start_loc.numel() - 1) < req0 + num_reqs:
        raise ValueError("input_conv: request range outside the metadata")
    out = torch.empty(h.shape[0], width, dtype=h.dtype, device=h.device)
    check("mi_input_conv", lib.mi_input_conv(
        _p(out), _p(h), _p(conv.weight), _p(conv.ring), _p(slots), _p(query_start_loc), _p(seq_lens), req0, num_reqs, max_query_len,
        conv.taps, width, hs, out.stride(0), _dt(h.dtype), _stream()))
    return out


def relu_squared(z: Union[torch.Tensor, "SplitKPartials"]) -> torch.Tensor:
    """relu(z)^2; ``z`` may be the split-K partials of a linear without bias"""
    if isinstance(z, SplitKPartials):
        z._live()
        if z.bias is not None:
            raise ValueError("partials of a linear without bias")
        src, split, rows, ff, zs, dtype = z.part, z.split, z.m, z.n, z.n, z.dtype
    else:
        zs, ff = _rows(z)
        src, split, rows, dtype = z, 0, z.shape[0], z.dtype
    _gpu(src)
    out = torch.empty(rows, ff, dtype=dtype, device=src.device)
    check("mi_relu_squared", lib.mi_relu_squared(_p(out), _p(src), split, rows, ff, zs, out.stride(0), _dt(dtype), _stream()))
    return out


def linear_relu_squared(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """relu(x W^T)^2 for a decode batch by the weight-streaming kernel of ``linear``"""
    _gpu(x, weight)
    xs, k = _rows(x)
    m, n = x.shape[0], weight.shape[0]
    if weight.shape[1] != k or not weight.is_contiguous() or weight.dtype != x.dtype:
        raise ValueError("weight must be a contiguous [n, k] tensor of x's dtype")
    out = torch.empty(m, n, dtype=x.dtype, device=x.device)
    need = lib.mi_linear_workspace_bytes(m, n, k)
    ws = _linear_workspace(x.device, need) if need else None
    check("mi_linear_relu_squared", lib.mi_linear_relu_squared(_p(out), _p(x), _p(weight), m, n, k, xs, out.stride(0), _p(ws),
                                                               ws.numel() if need else 0, _dt(x.dtype), _stream()))
    return out


def row_norm_cache(x: torch.Tensor, q_weight: Optional[torch.Tensor], k_weight: Optional[torch.Tensor], k_cache: torch.Tensor,
                   v_cache: torch.Tensor, slot_mapping: torch.Tensor, num_q_heads: int, dim: int, vdim: int, eps: float) -> torch.Tensor:
    """Rows q | k | v: q and k each normed over all heads at once, K / V cache write; returns q, heads laid out as in the cache."""
    _gpu(x, q_weight, k_weight, k_cache, v_cache, slot_mapping)
    _i64(slot_mapping)
    xs, cols = _rows(x)
    rows = x.shape[0]
    _, bs, g, hd = k_cache.shape
    cb, ct, ch = _cache_strides(k_cache, v_cache)
    if cols != (num_q_heads + g) * dim + g * vdim or slot_mapping.numel() < rows or max(dim, vdim) > hd:
        raise ValueError("row_norm_cache: sizes do not fit")
    for w, n in ((q_weight, num_q_heads * dim), (k_weight, g * dim)):
        if w is not None and (w.numel() != n or w.dtype != x.dtype):
            raise ValueError("row_norm_cache: norm weights of the projection's size")
    if x.dtype != k_cache.dtype:
        raise TypeError("cache and activations share a dtype")
    q = torch.empty(rows, num_q_heads * hd, dtype=x.dtype, device=x.device)
    check("mi_row_norm_cache", lib.mi_row_norm_cache(
        _p(x), xs, _p(q_weight), _p(k_weight), _p(q), q.stride(0), _p(k_cache), _p(v_cache), _p(slot_mapping), rows, num_q_heads, g, dim,
        vdim, hd, bs, cb, ct, ch, float(eps), _dt(x.dtype), _stream()))
    return q


class TalkingHeads:
    """What attention with mixed heads needs besides its operands: fp32 ``talk`` [H, H], ``r1`` / ``r2`` [H] (or None), scale,
    soft cap (0: none), window, value size."""

    def __init__(self, talk: torch.Tensor, r1: Optional[torch.Tensor], r2: Optional[torch.Tensor], scale: float, softcap: float,
                 window: int, vdim: int):
        h = talk.shape[0]
        if talk.dtype != torch.float32 or tuple(talk.shape) != (h, h) or not talk.is_contiguous():
            raise ValueError("talk: contiguous fp32 [heads, heads]")
        if (r1 is None) != (r2 is None):
            raise ValueError("r1 and r2 go together")
        _head_vectors(h, r1, r2)
        self.talk, self.r1, self.r2, self.scale, self.softcap, self.vdim = talk, r1, r2, float(scale), float(softcap), int(vdim)
        self.heads, self.window = h, min(int(window), 2**31 - 1)


def _talking_args(out, q, kc, vc, table, seq_lens, qsl, th: TalkingHeads, gate, n: int):
    _gpu(out, q, kc, vc, table, seq_lens, qsl, th.talk, th.r1, th.r2, gate)
    _i32(seq_lens, qsl)
    _, bs, g, hd = kc.shape
    cb, ct, ch = _cache_strides(kc, vc)
    qs, qc = _rows(q)
    os_, oc = _rows(out)
    if qc != th.heads * hd or oc != th.heads * th.vdim or table.dtype != torch.int32 or table.stride(1) != 1:
        raise ValueError("talking attention: sizes do not fit")
    if not q.dtype == out.dtype == kc.dtype or (gate is not None and gate.dtype != q.dtype):
        raise TypeError("talking attention: one dtype")
    gs = 0
    if gate is not None:
        gs, gc = _rows(gate)
        if gc != oc or gate.shape[0] < out.shape[0]:
            raise ValueError("talking attention: a gate per output value")
    if min(table.shape[0], seq_lens.numel(), qsl.numel() - 1) < n:
        raise ValueError("talking attention: one metadata entry per request")
    return _C.TalkingAttnArgs(_p(out), _p(q), _p(kc), _p(vc), _p(table), _p(seq_lens), _p(qsl), _p(th.r1), _p(th.r2), _p(th.talk), _p(gate),
                              qs, os_, gs, cb, ct, ch, table.stride(0), th.heads, g, hd, th.vdim, bs, th.window, th.scale, th.softcap)


def talking_attn_rows(out: torch.Tensor, q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_table: torch.Tensor,
                      seq_lens: torch.Tensor, query_start_loc: torch.Tensor, th: TalkingHeads, gate: Optional[torch.Tensor] = None,
                      row0: int = 0) -> torch.Tensor:
    """Attention with mixed heads of rows [row0, T), any sizes and types"""
    n = seq_lens.shape[0]
    a = _talking_args(out, q, k_cache, v_cache, block_table, seq_lens, query_start_loc, th, gate, n)
    if out.shape[0] < q.shape[0]:
        raise ValueError("talking_attn_rows: sizes do not fit")
    check("mi_talking_attn_rows", lib.mi_talking_attn_rows(ctypes.byref(a), row0, q.shape[0] - row0, n, _dt(q.dtype), _stream()))
    return out


def talking_attn_supported(dtype: torch.dtype, heads: int, kv_heads: int, head_dim: int, vdim: int, block_size: int, softcap: float) -> bool:
    """whether the matrix-core forms take these sizes"""
    return dtype == torch.bfloat16 and bool(lib.mi_talking_attn_supported(heads, kv_heads, head_dim, vdim, block_size, float(softcap)))


def talking_decode(out: torch.Tensor, q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_table: torch.Tensor,
                   seq_lens: torch.Tensor, query_start_loc: torch.Tensor, th: TalkingHeads, max_seq_len: int, num_reqs: int,
                   gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One row per request: rows and requests [0, num_reqs)"""
    a = _talking_args(out, q, k_cache, v_cache, block_table, seq_lens, query_start_loc, th, gate, num_reqs)
    if min(q.shape[0], out.shape[0]) < num_reqs:
        raise ValueError("talking_decode: sizes do not fit")
    need = lib.mi_talking_decode_workspace_bytes(num_reqs, th.heads, k_cache.shape[2], th.vdim, th.window, max_seq_len)
    ws = torch.empty(max(need, 1), dtype=torch.uint8, device=q.device)
    check("mi_talking_decode", lib.mi_talking_decode(ctypes.byref(a), num_reqs, max_seq_len, _p(ws), need, _stream()))
    return out


def talking_prefill(out: torch.Tensor, q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_table: torch.Tensor,
                    seq_lens: torch.Tensor, query_start_loc: torch.Tensor, th: TalkingHeads, ctx_start: torch.Tensor, ctx_rows: int,
                    max_query_len: int, gate: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Prompt portions: metadata of the portions alone, row offsets counted from the step's first row; ``ctx_start``: where a
    portion's visible context starts among ``ctx_rows`` gathered rows (multiples of 64)."""
    n = seq_lens.shape[0]
    a = _talking_args(out, q, k_cache, v_cache, block_table, seq_lens, query_start_loc, th, gate, n)
    _gpu(ctx_start)
    _i32(ctx_start)
    if out.shape[0] < q.shape[0] or ctx_start.numel() < n + 1:
        raise ValueError("talking_prefill: sizes do not fit")
    rows, g, hd = q.shape[0], k_cache.shape[2], k_cache.shape[3]
    need = lib.mi_talking_prefill_workspace_bytes(rows, th.heads, g, hd, ctx_rows)
    ws = torch.empty(max(need, 1), dtype=torch.uint8, device=q.device)
    check("mi_talking_prefill", lib.mi_talking_prefill(ctypes.byref(a), _p(ctx_start), ctx_rows, n, rows, max_query_len, _p(ws), need,
                                                       _stream()))
    return out


# ------------------------------------------------- state-space layers, attention whose values are its keys
def stream_norm2(x: torch.Tensor, y: Union[torch.Tensor, "SplitKPartials", None], w1: torch.Tensor, w2: Optional[torch.Tensor], eps: float,
                 h1: torch.Tensor, h2: Optional[torch.Tensor] = None, w_shift: float = 0.0, mult: float = 1.0,
                 experts: Optional[ExpertRows] = None, table: Optional[torch.Tensor] = None, ids: Optional[torch.Tensor] = None,
                 add_row: Optional[torch.Tensor] = None) -> None:
    """``x += mult * (y + the experts' rows)`` in place (x fp32 [T, W]; ``y`` None: x starts from zero), then ``x += table[ids] +
    add_row`` where given, then ``h1`` / ``h2`` = x / rms(x) * (w1 / w2 + w_shift).  ``y`` as in ``residual_add_norm``."""
    part = isinstance(y, SplitKPartials)
    if part:
        y._live()
        if y.bias is not None:
            raise ValueError("stream_norm2 takes partials of a linear without bias")
    src = y.part if part else y
    _gpu(x, src, w1, w2, h1, h2, table, ids, add_row)
    xs, width = _rows(x)
    rows = x.shape[0]
    if x.dtype != torch.float32 or (w2 is None) != (h2 is None) or (y is None and (table is None or experts is not None)):
        raise ValueError("stream_norm2: an fp32 stream that starts from the table or takes a layer's output; one output per norm")
    strides = []
    for h, w in ((h1, w1), (h2, w2)):
        if h is None:
            strides.append(0)
            continue
        hs, hw = _rows(h)
        if hw != width or h.shape[0] < rows or w.numel() != width or not w.dtype == h.dtype == h1.dtype:
            raise ValueError("stream_norm2: norm rows and weights of the stream's width")
        strides.append(hs)
    split, ys = 0, 0
    if part:
        if (y.m, y.n) != (rows, width):
            raise ValueError("partials of another shape")
        split, ys = y.split, width
    elif y is not None:
        ys, yw = _rows(y)
        if y.shape[0] != rows or yw != width or y.dtype not in (h1.dtype, torch.float32):
            raise ValueError("layer output of another shape or dtype")
        split = 1 if y.dtype == torch.float32 and h1.dtype != torch.float32 else 0
    prt, rp, ww, top, ps = None, None, None, 0, 0
    if experts is not None:
        prt, rp, ww, top = experts.part, experts.row_of_pair, experts.weights, experts.top
        ps = experts.check(rows, width, h1.dtype)
    if table is not None:
        _i64(ids)
        if not table.is_contiguous() or table.shape[1] != width or table.dtype != h1.dtype or ids is None or ids.numel() < rows:
            raise ValueError("stream_norm2: an embedding table of the stream's width, an id per row")
    if add_row is not None and (add_row.numel() != width or add_row.dtype != h1.dtype or not add_row.is_contiguous()):
        raise ValueError("stream_norm2: a row of the stream's width")
    check("mi_stream_norm2", lib.mi_stream_norm2(
        _p(x), _p(src), split, _p(prt), _p(rp), _p(ww), top, float(mult), _p(table), _p(ids) if table is not None else None,
        table.shape[0] if table is not None else 0, _p(add_row), _p(w1), _p(w2), float(w_shift), _p(h1), _p(h2), float(eps), rows, width, xs,
        ys, ps, strides[0], strides[1], _dt(h1.dtype), _stream()))


def _step_requests(slots, query_start_loc, seq_lens, req0: int, num_reqs: int, what: str) -> None:
    _i32(slots, query_start_loc, seq_lens)
    if req0 < 0 or min(seq_lens.shape[0], slots.shape[0], query_start_loc.shape[0] - 1) < req0 + num_reqs:
        raise ValueError(f"{what}: request range outside the metadata")


def conv_rope_cache(x: torch.Tensor, conv_w: torch.Tensor, ring: torch.Tensor, q_out: torch.Tensor, k_cache: torch.Tensor,
                    v_cache: torch.Tensor, inv_freq: Optional[torch.Tensor], slots: torch.Tensor, query_start_loc: torch.Tensor,
                    seq_lens: torch.Tensor, slot_mapping: torch.Tensor, num_q_heads: int, dim: int, eps: float, req0: int, num_reqs: int,
                    max_query_len: int, update_ring: bool = True) -> torch.Tensor:
    """Rows q | k of requests [req0, req0 + num_reqs): causal filter per channel, value row = the filtered k, rotary on neighbouring
    pairs, unweighted norm per head, K / V cache write; q to ``q_out``, heads laid out as in the cache.  ``ring`` [slots, taps,
    channels]; ``inv_freq`` fp32 [rotary dimensions / 2] (None: no rotation)."""
    _gpu(x, conv_w, ring, q_out, k_cache, v_cache, inv_freq, slots, query_start_loc, seq_lens, slot_mapping)
    _step_requests(slots, query_start_loc, seq_lens, req0, num_reqs, "conv_rope_cache")
    _i64(slot_mapping)
    xs, cols = _rows(x)
    qs, qc = _rows(q_out)
    _, bs, g, hd = k_cache.shape
    cb, ct, chs = _cache_strides(k_cache, v_cache)
    ch, taps = (num_q_heads + g) * dim, conv_w.shape[1]
    if cols != ch or tuple(conv_w.shape) != (ch, taps) or tuple(ring.shape[1:]) != (taps, ch) or qc != num_q_heads * hd or hd < dim:
        raise ValueError("conv_rope_cache: sizes do not fit")
    if q_out.shape[0] < x.shape[0] or slot_mapping.numel() < x.shape[0]:
        raise ValueError("conv_rope_cache: one output row and one slot per row")
    if not conv_w.is_contiguous() or not ring.is_contiguous() or any(t.dtype != x.dtype for t in (conv_w, ring, q_out, k_cache)):
        raise TypeError("conv_rope_cache: one dtype, contiguous filter and ring")
    pairs = 0
    if inv_freq is not None:
        pairs = inv_freq.numel()
        _head_vectors(pairs, inv_freq)
    a = _C.ConvRopeCacheArgs(_p(x), _p(conv_w), _p(ring), _p(q_out), _p(k_cache), _p(v_cache), _p(inv_freq), _p(slots), _p(query_start_loc),
                             _p(seq_lens), _p(slot_mapping), xs, qs, cb, ct, chs, req0, num_reqs, max_query_len, num_q_heads, g, dim, hd, bs,
                             2 * pairs, taps, int(update_ring), float(eps))
    check("mi_conv_rope_cache", lib.mi_conv_rope_cache(ctypes.byref(a), _dt(x.dtype), _stream()))
    return q_out


def state_space(xbc: torch.Tensor, z: torch.Tensor, dt: torch.Tensor, conv_w: torch.Tensor, conv_b: torch.Tensor, dt_bias: torch.Tensor,
                a_log: torch.Tensor, d: torch.Tensor, norm_w: torch.Tensor, state: torch.Tensor, ring: torch.Tensor, slots: torch.Tensor,
                query_start_loc: torch.Tensor, seq_lens: torch.Tensor, groups: int, norm_groups: int, eps: float, out: torch.Tensor,
                req0: int, num_reqs: int, row0: int, rows: int, max_query_len: int, chunked: bool = True) -> torch.Tensor:
    """State-space recurrence of requests [req0, req0 + num_reqs), which own rows [row0, row0 + rows).  ``xbc``, ``z`` and ``dt``
    are column blocks of one matrix; ``state`` fp32 [slots, H, N, V]; ``ring`` [slots, taps, channels].  ``chunked``: 64 tokens at a
    time (fp32 and sizes outside that form go token by token)."""
    _gpu(xbc, z, dt, conv_w, conv_b, dt_bias, a_log, d, norm_w, state, ring, slots, query_start_loc, seq_lens, out)
    _step_requests(slots, query_start_loc, seq_lens, req0, num_reqs, "state_space")
    ps, ch = _rows(xbc)
    os_, oc = _rows(out)
    _, hh, n, v = state.shape
    taps = ring.shape[1]
    if _rows(z) != (ps, hh * v) or _rows(dt) != (ps, hh):
        raise ValueError("state_space: x | B | C, z and dt are column blocks of one matrix")
    if ch != hh * v + 2 * groups * n or hh % groups or (hh * v) % norm_groups or oc != hh * v or norm_w.numel() != hh * v:
        raise ValueError("state_space: sizes do not fit")
    if tuple(conv_w.shape) != (ch, taps) or conv_b.numel() != ch or ring.shape[2] != ch or any(t.numel() != hh for t in (dt_bias, a_log, d)):
        raise ValueError("state_space: sizes do not fit")
    if any(t.dtype != torch.float32 for t in (state, dt_bias, a_log, d)):
        raise TypeError("state_space: state, step bias, A_log and D are fp32")
    if any(t.dtype != xbc.dtype for t in (z, dt, conv_w, conv_b, norm_w, ring, out)):
        raise TypeError("state_space: one activation dtype")
    if not all(t.is_contiguous() for t in (state, ring, conv_w, conv_b, norm_w, dt_bias, a_log, d)):
        raise ValueError("state_space: contiguous state and weights")
    if min(xbc.shape[0], z.shape[0], dt.shape[0], out.shape[0]) < row0 + rows:
        raise ValueError("state_space: rows outside the tensors")
    ad = _dt(xbc.dtype)
    need = lib.mi_state_space_workspace_bytes(rows, num_reqs, hh, groups, n, v, 1, ad) if chunked else 0
    chunked = need > 0
    if not chunked:
        need = lib.mi_state_space_workspace_bytes(rows, num_reqs, hh, groups, n, v, 0, ad)
    ws = torch.empty(max(need, 1), dtype=torch.uint8, device=xbc.device)
    a = _C.StateSpaceArgs(_p(xbc), _p(z), _p(dt), _p(conv_w), _p(conv_b), _p(norm_w), _p(dt_bias), _p(a_log), _p(d), _p(state), _p(ring),
                          _p(slots), _p(query_start_loc), _p(seq_lens), _p(out), ps, os_, req0, num_reqs, hh, groups, n, v, taps, norm_groups,
                          float(eps))
    check("mi_state_space", lib.mi_state_space(ctypes.byref(a), row0, rows, max_query_len, int(chunked), _p(ws), need, ad, _stream()))
    return out


def soft_cap_argmax(logits: torch.Tensor, cap: float, ids: Optional[torch.Tensor] = None, greedy: bool = True) -> Optional[torch.Tensor]:
    """``logits`` = cap tanh(logits / cap) in place; with ``greedy`` also the first index of every row's maximum."""
    _gpu(logits, ids)
    stride, vocab = _rows(logits)
    t = logits.shape[0]
    if greedy and ids is None:
        ids = torch.empty(t, dtype=torch.int64, device=logits.device)
    if not greedy:
        ids = None
    _i64(ids)
    if ids is not None and ids.numel() < t:
        raise ValueError("soft_cap_argmax: an id per row")
    check("mi_soft_cap_argmax", lib.mi_soft_cap_argmax(_p(logits), _p(ids), float(cap), t, vocab, stride, _dt(logits.dtype), _stream()))
    return ids
