"""Owns the model, the cache and the states of one GPU and turns a scheduled batch into one forward pass and one sampled
token per sequence (counterpart of electrock_infer/engine/model_runner.py:92-236, single process: the reference's
shared-memory fan-out to tensor-parallel ranks has nothing to do on one GPU)."""
from typing import List, Optional

import torch

from ..utils.loader import load_model
from .batch import make_ragged
from .config import EngineConfig
from .decode_graph import DecodeGraphs
from .model import BatchContext, Sampler
from .registry import build_model
from .sequence import Sequence


class ModelRunner:

    def __init__(self, config: EngineConfig):
        self.config = config
        self.block_size = config.kvcache_block_size
        self.device = torch.device(config.device)
        torch.cuda.set_device(self.device)
        with torch.device(self.device):
            self.model = build_model(config)
        if config.model_dir is not None:
            load_model(self.model, config.model_dir, device=str(self.device))
        else:
            self.model.init_random_weights(config.seed)
        self.sampler = Sampler()
        self.ragged = getattr(self.model, "ragged_batches", False)      # takes RaggedBatch (batch.py)
        if hasattr(self.model, "reserve_workspace"):
            self.model.reserve_workspace(self.device, config.max_num_batched_tokens)
        self.allocate_kv_cache()

    def allocate_kv_cache(self) -> None:
        """The model's cache for as many blocks as configured, or as fit into the device memory left under
        gpu_memory_utilization (model_runner.py:92-110) behind the state slots."""
        config = self.config
        block_bytes, slot_bytes = self.model.cache_bytes(self.block_size)
        if config.num_kvcache_blocks <= 0:
            free, total = torch.cuda.mem_get_info(self.device)
            budget = int(total * config.gpu_memory_utilization) - (total - free) - slot_bytes * config.num_state_slots
            if budget < block_bytes:
                raise RuntimeError("no device memory left for the KV cache")
            # what max_num_seqs sequences of max_model_len tokens can ever use is enough
            most = config.max_num_seqs * (-(-config.max_model_len // self.block_size))
            config.num_kvcache_blocks = min(budget // block_bytes, most) if block_bytes else most
        # (one block and one slot more than the planner hands out, for the unused rows of padded decode steps)
        extra = 1 if self.ragged else 0
        self.model.allocate_cache(config.num_kvcache_blocks + extra, self.block_size, config.num_state_slots + extra, self.device)
        self.graphs = DecodeGraphs(self) if self.ragged and config.decode_graphs else None

    # ---- batch preparation ----
    def _to_device(self, values, dtype) -> torch.Tensor:
        return torch.tensor(values, dtype=dtype, pin_memory=True).to(self.device, non_blocking=True)

    def _block_tables(self, seqs: List[Sequence]) -> torch.Tensor:
        width = max(len(s.block_table) for s in seqs)
        return self._to_device([s.block_table + [0] * (width - len(s.block_table)) for s in seqs], torch.int64)

    def check_slots(self, seqs: List[Sequence]) -> None:
        if self.config.num_state_slots > 0 and any(not 0 <= s.state_slot < self.config.num_state_slots for s in seqs):
            raise ValueError("a sequence of this model needs a state slot")

    def prepare_ragged(self, seqs: List[Sequence], rows: Optional[List[int]] = None):
        """The planned portions of any batch, for models that take RaggedBatch; ``rows``: batch rows whose logits are
        wanted (default: the last one of every sequence)."""
        self.check_slots(seqs)
        chunk = self.model.chunk_tokens(sum(s.num_scheduled_tokens for s in seqs))
        return make_ragged(seqs, self.block_size, chunk, self.device, rows)

    def prepare_prefill(self, seqs: List[Sequence]):
        """Feed every sequence's planned portion behind its computed tokens; the cache slots follow from the block
        table."""
        input_ids, positions, slots, q_lens, k_lens, last = [], [], [], [], [], []
        for seq in seqs:
            start, n = seq.num_computed_tokens, seq.num_computed_tokens + seq.num_scheduled_tokens
            input_ids.extend(seq[start:n])
            positions.extend(range(start, n))
            q_lens.append(n - start)
            k_lens.append(n)
            for pos in range(start, n):
                slots.append(seq.block_table[pos // self.block_size] * self.block_size + pos % self.block_size)
            last.append(len(input_ids) - 1)
        need_tables = any(k != q for q, k in zip(q_lens, k_lens))
        ctx = BatchContext(True, self._to_device(slots, torch.int64), q_lens, k_lens,
                           block_tables=self._block_tables(seqs) if need_tables else None,
                           last_token_index=self._to_device(last, torch.int64))
        return self._to_device(input_ids, torch.int64), self._to_device(positions, torch.int64), ctx

    def prepare_decode(self, seqs: List[Sequence]):
        """One token per sequence: the last one sampled, at position len - 1, into the last slot of its table."""
        input_ids = [s.last_token for s in seqs]
        positions = [len(s) - 1 for s in seqs]
        slots = [s.block_table[-1] * self.block_size + s.last_block_num_tokens - 1 for s in seqs]
        ctx = BatchContext(False, self._to_device(slots, torch.int64), [], [], block_tables=self._block_tables(seqs),
                           context_lens=self._to_device([len(s) for s in seqs], torch.int64))
        # the same for every layer of the step: key j of a sequence counts if j < its context length
        keys = ctx.block_tables.shape[1] * self.block_size
        ctx.decode_mask = (torch.arange(keys, device=self.device)[None, :] < ctx.context_lens[:, None])[:, None, None, :]
        return self._to_device(input_ids, torch.int64), self._to_device(positions, torch.int64), ctx

    # ---- one step ----
    @torch.inference_mode()
    def run_model(self, input_ids, positions, ctx: BatchContext) -> torch.Tensor:
        return self.model.compute_logits(self.model(input_ids, positions, ctx), ctx)

    @torch.inference_mode()
    def run_ragged(self, seqs: List[Sequence], rows: Optional[List[int]] = None) -> torch.Tensor:
        """Logits [wanted, vocab] of one forward pass over the planned portions.  A decode step is the replay of a
        recorded graph where one can be had (the result is overwritten by the next replay of that graph)."""
        if self.graphs is not None and rows is None and all(s.num_scheduled_tokens == 1 for s in seqs):
            logits = self.graphs.run(seqs)
            if logits is not None:
                return logits
        batch = self.prepare_ragged(seqs, rows)
        return self.model.compute_logits(self.model(batch), batch)

    def logits(self, seqs: List[Sequence], is_prefill: bool) -> torch.Tensor:
        """Logits behind the last fed token of every sequence."""
        if self.ragged:
            return self.run_ragged(seqs)
        return self.run_model(*(self.prepare_prefill(seqs) if is_prefill else self.prepare_decode(seqs)))

    def portion_logits(self, seqs: List[Sequence], rows: List[int]) -> torch.Tensor:
        """Logits of chosen rows of the planned portions (rows count through the batch)."""
        if self.ragged:
            return self.run_ragged(seqs, rows)
        input_ids, positions, ctx = self.prepare_prefill(seqs)
        ctx.last_token_index = self._to_device(rows, torch.int64)
        return self.run_model(input_ids, positions, ctx)

    def run(self, seqs: List[Sequence], is_prefill: bool, return_logits: bool = False):
        logits = self.logits(seqs, is_prefill)
        if all(s.temperature == 0 for s in seqs):
            token_ids = logits.argmax(dim=-1).tolist()
        else:
            temperatures = self._to_device([s.temperature for s in seqs], torch.float32)
            token_ids = self.sampler(logits, temperatures).tolist()
        return (token_ids, logits) if return_logits else token_ids
