"""Single-process engine: a checkpoint folder behind the scheduler, the worker and the model runner.

``LLMEngine.generate`` is the ordinary serving loop (schedule -> execute -> sample -> update); ``run_portions`` runs a step
whose tokens are given, through the same scheduler bookkeeping, caches, state slots and kernels.
"""
from __future__ import annotations

import os
from typing import Any, Iterable, Iterator, Optional, Sequence

import torch

from .compat import torch_dtype
from .registry import config_from_dir
from .sched_output import Request, RequestStatus, SamplingParams
from .scheduler import StandaloneARScheduler
from .worker import GPUARWorker, WorkerConfig


def checkpoint_tensors(path: str) -> Iterator[tuple[str, torch.Tensor]]:
    """(name, tensor) of every ``*.safetensors`` file of a folder, one tensor in memory at a time."""
    from safetensors import safe_open

    files = sorted(f for f in os.listdir(path) if f.endswith(".safetensors"))
    if not files:
        raise FileNotFoundError(f"no *.safetensors in {path}")
    for name in files:
        with safe_open(os.path.join(path, name), framework="pt") as f:
            for key in f.keys():
                yield key, f.get_tensor(key)


class _SchedulerConfig:
    """the fields ``StandaloneARScheduler`` reads"""

    def __init__(self, c: WorkerConfig):
        self.scheduler_config = {"max_num_seqs": c.max_num_seqs, "max_num_batched_tokens": c.max_num_batched_tokens}
        self.cache_config = {"block_size": c.block_size, "enable_prefix_caching": c.enable_prefix_caching}
        self.model_config = {"max_model_len": c.max_model_len}


class LLMEngine:
    def __init__(self, model: Any, dtype="bfloat16", max_num_seqs: int = 64, max_model_len: int = 4096,
                 max_num_batched_tokens: int = 8192, block_size: int = 16, num_blocks: Optional[int] = None,
                 gpu_memory_utilization: float = 0.9, enforce_eager: bool = False, seed: int = 0,
                 enable_prefix_caching: bool = False, weights: Optional[Iterable] = None):
        """``model``: a checkpoint folder, or a configuration (random weights unless ``weights`` is given).  ``num_blocks``:
        KV blocks besides the reserved null block; default: what the memory budget holds."""
        if isinstance(model, str):
            config = config_from_dir(model)
            weights = checkpoint_tensors(model) if weights is None else weights
        else:
            config = model
        if getattr(config, "max_positions", None):      # a learned position per token: no sequence is longer than the table
            max_model_len = min(max_model_len, config.max_positions)
        wc = WorkerConfig(model_config=config, dtype=torch_dtype(dtype), gpu_memory_utilization=gpu_memory_utilization,
                          block_size=block_size, max_num_seqs=max_num_seqs, max_model_len=max_model_len,
                          max_num_batched_tokens=max(max_num_batched_tokens, max_num_seqs), enforce_eager=enforce_eager,
                          engine_output_type="text", seed=seed, enable_prefix_caching=enable_prefix_caching)
        self.config = wc
        self.worker = GPUARWorker(wc)
        self.worker.init_device()
        self.worker.load_model()
        if weights is not None:
            loaded = self.model.load_weights(weights)
            missing = [n for n, _ in self.model.named_weights() if n not in loaded]
            if missing:
                raise ValueError(f"checkpoint lacks {len(missing)} tensors: {', '.join(missing[:5])} ...")
        if num_blocks is None:
            # room past this is never used: every live request at its longest
            num_blocks = min(self.worker.determine_num_available_blocks() - 1, max_num_seqs * -(-max_model_len // block_size))
        self.worker.initialize_cache(num_blocks + 1)
        self.scheduler = StandaloneARScheduler(_SchedulerConfig(wc), num_blocks=num_blocks + 1)

    @property
    def runner(self):
        return self.worker.model_runner

    @property
    def model(self):
        return self.worker.get_model()

    # ---- serving ------------------------------------------------------------------
    def add_request(self, request_id: str, prompt_token_ids: Sequence[int], params: Optional[SamplingParams] = None,
                    eos_token_id: Optional[int] = None) -> None:
        if not prompt_token_ids or len(prompt_token_ids) >= self.config.max_model_len:
            raise ValueError(f"a prompt of 1..{self.config.max_model_len - 1} tokens, got {len(prompt_token_ids)}")
        vocab = self.config.model_config.vocab_size
        if any(not 0 <= int(t) < vocab for t in prompt_token_ids):
            raise ValueError(f"prompt token outside the vocabulary of {vocab}")
        self.scheduler.add_request(Request(request_id, [int(t) for t in prompt_token_ids], params or SamplingParams(),
                                           eos_token_id=eos_token_id))

    def step(self) -> list:
        """One scheduling step; the ``EngineCoreOutput``s of the requests that got tokens or finished."""
        so = self.scheduler.schedule()
        out = self.worker.execute_model(so)
        if out is None:
            out = self.worker.sample_tokens()
        return [o for outs in self.scheduler.update_from_output(so, out).values() for o in outs.outputs]

    def generate(self, prompts: Sequence[Sequence[int]], params: Optional[SamplingParams] = None,
                 eos_token_id: Optional[int] = None) -> list[list[int]]:
        """Token ids generated for every prompt."""
        ids = [f"gen-{i}" for i in range(len(prompts))]
        out: dict[str, list[int]] = {i: [] for i in ids}
        for rid, p in zip(ids, prompts):
            self.add_request(rid, p, params, eos_token_id)
        while self.scheduler.get_num_unfinished_requests():
            for o in self.step():
                out[o.request_id].extend(o.new_token_ids)
        self.step()     # hands the last finished ids to the runner: their state slots and rows are free again
        return [out[i] for i in ids]

    # ---- given tokens ---------------------------------------------------------------
    def run_portions(self, portions: dict[str, Sequence[int]], wanted: Optional[dict[str, list[int]]] = None,
                     finished: Sequence[str] = ()) -> Optional[torch.Tensor]:
        """Run exactly these next tokens of these requests as one batch; logits (fp32, device) at the ``wanted`` places of
        the portions, or None.  ``finished`` requests give back what they hold after the step."""
        vocab = self.config.model_config.vocab_size
        for rid, toks in portions.items():
            if any(not 0 <= int(t) < vocab for t in toks):
                raise ValueError(f"request {rid}: token outside the vocabulary of {vocab}")
        logits = None
        if portions:
            so = self.scheduler.schedule_portions({r: [int(t) for t in ts] for r, ts in portions.items()})
            self.worker.execute_model(so)
            wanted = {r: list(p) for r, p in (wanted or {}).items() if len(p)}
            if wanted:
                logits = self.runner.logits_at(wanted)
            self.runner.discard_step()
        if finished:
            self.scheduler.finish_requests(list(finished), RequestStatus.FINISHED_STOPPED)
        return logits
