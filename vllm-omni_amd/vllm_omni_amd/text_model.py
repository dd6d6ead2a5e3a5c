"""What decoders that take token ids share: the runner's view of such a model, logits, checkpoint loading, looped layers."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Iterable, Optional

import torch

from . import ops
from .layers import tuned_linear


@dataclass
class LoopConfig:
    """layers start .. stop - 1 run ``times`` times in a row"""

    start: int
    stop: int
    times: int

    def validate(self, layers: int) -> None:
        if not (0 <= self.start < self.stop <= layers and self.times >= 1):
            raise ValueError(f"loop {self.start}..{self.stop} x {self.times} does not fit {layers} layers")


def layer_runs(n: int, loop: Optional[LoopConfig]) -> list[tuple[int, Optional[int]]]:
    """(layer, pass of the loop that starts with it or None), in the order ``n`` layers run"""
    if loop is None:
        return [(i, None) for i in range(n)]
    passes = [(i, t if i == loop.start else None) for t in range(loop.times) for i in range(loop.start, loop.stop)]
    return [(i, None) for i in range(loop.start)] + passes + [(i, None) for i in range(loop.stop, n)]


class TokenDecoder:
    """Subclasses set ``head`` and yield their parameters from ``named_weights``: (checkpoint name, tensor), the tensor a row or
    column block of a fused parameter where the checkpoint stores the pieces apart.  A block of three dimensions is a
    two-dimensional checkpoint tensor whose columns fall into groups (heads laid out further apart than they are wide)."""

    consumes_token_ids = True
    extra_dtypes = (torch.float32,)      # runs in true 32-bit as well
    has_preprocess = False
    has_postprocess = False
    prefer_model_sampler = False
    head: torch.Tensor
    logit_softcap: Optional[float] = None      # logits are cap tanh(logits / cap)
    unread_weights: frozenset = frozenset()    # names a checkpoint may hold although nothing reads them

    def __init__(self, cfg: Any, dtype, device):
        from .distributed import get_tensor_model_parallel_world_size

        if get_tensor_model_parallel_world_size() > 1:
            raise NotImplementedError("this model runs data-parallel only (tp_size 1)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"this model runs in bfloat16 or float32, not {dtype}")
        self.config, self.dtype, self.device = cfg, dtype, device
        self.residual_tap: Optional[list] = None      # a list collects the stream after every layer (inspection)

    def generator(self, seed: Optional[int]) -> Optional[torch.Generator]:
        if seed is None:
            return None
        gen = torch.Generator(device=self.device)
        gen.manual_seed(seed)
        return gen

    def named_weights(self) -> Iterable[tuple[str, torch.Tensor]]:
        raise NotImplementedError

    def weights_changed(self) -> None:
        """after a load: what was derived from parameters is stale"""

    def prefill_windows(self) -> list[int]:
        """windows of the layers whose prompt attention runs on a gathered context"""
        return []

    def compute_logits(self, hidden_states: torch.Tensor) -> torch.Tensor:
        logits = tuned_linear(hidden_states, self.head)
        if self.logit_softcap is not None:
            ops.soft_cap_argmax(logits, self.logit_softcap, greedy=False)
        return logits

    def compute_logits_and_greedy(self, hidden_states: torch.Tensor, ids: Optional[torch.Tensor] = None):
        if self.logit_softcap is not None:
            logits = tuned_linear(hidden_states, self.head)
            return logits, ops.soft_cap_argmax(logits, self.logit_softcap, ids)
        logits = self.compute_logits(hidden_states)
        return logits, ops.mask_logits_argmax(logits, ids=ids)

    def load_weights(self, weights) -> set[str]:
        params = dict(self.named_weights())
        loaded: set[str] = set()
        for name, w in (weights.items() if isinstance(weights, dict) else weights):
            dst = params.get(name)
            if dst is None and name in self.unread_weights:
                continue
            if dst is None:
                raise KeyError(f"checkpoint tensor maps to no parameter: {name!r}")
            want = tuple(dst.shape) if dst.dim() < 3 else (dst.shape[0], dst.shape[1] * dst.shape[2])
            if want != tuple(w.shape):
                raise ValueError(f"{name}: checkpoint shape {tuple(w.shape)}, parameter {want}")
            dst.copy_(w.view(dst.shape).to(dst.dtype))
            loaded.add(name)
        self.weights_changed()
        return loaded

    def weight_bytes(self) -> int:
        return sum(w.numel() * w.element_size() for _, w in self.named_weights())

    def quantize_int8(self) -> None:
        raise ValueError("int8 quantization is not built for this model")
