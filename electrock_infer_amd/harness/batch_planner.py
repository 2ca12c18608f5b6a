"""Which requests run in the next step.

Policy (the reference's, electrock_infer/engine/scheduler.py:24-74): requests that wait are started first, in
arrival order, for as long as the step's token budget, its sequence budget and the free KV blocks allow; only a
step that could start none is a decode step of the running requests, oldest first, in which a request that needs
a block when none is free takes it from the youngest running request (which goes back to the head of the waiting
line and is prefilled again later, prompt and completion so far), or gives way itself when it is the last one.

With ``prefill_portion`` set, a prompt is computed in portions of at most so many tokens: a request then stays in the
prefill steps until its last portion, whose step samples its first token; a prompt longer than a step's token budget
becomes possible.  Requests of models with a recurrent state also hold a state slot from admission to release.

Construction (this build's own): the running requests are a plain list in admission order and a step is planned
into a ``Plan`` record; the decode planner walks that list by index and evicts from its tail.
"""
from collections import deque
from dataclasses import dataclass, field
from typing import Deque, List

from .config import EngineConfig
from .kv_pool import KVBlockPool, StateSlotPool
from .sequence import Sequence, SequenceStatus


@dataclass
class Plan:
    seqs: List[Sequence] = field(default_factory=list)
    is_prefill: bool = False
    fresh_tokens: int = 0          # prefill: tokens that are not served from the prefix cache


class BatchPlanner:

    def __init__(self, config: EngineConfig):
        self.max_seqs = config.max_num_seqs
        self.max_tokens = config.max_num_batched_tokens
        self.eos = config.eos
        self.portion = config.prefill_portion
        self.pool = KVBlockPool(config.num_kvcache_blocks, config.kvcache_block_size, reuse_prefix=config.reuse_prefix)
        self.slots = StateSlotPool(config.num_state_slots) if config.num_state_slots > 0 else None
        self.waiting: Deque[Sequence] = deque()
        self.running: List[Sequence] = []
        self.num_preemptions = 0

    def submit(self, seq: Sequence) -> None:
        self.waiting.append(seq)

    def idle(self) -> bool:
        return not self.waiting and not self.running

    # ---- planning ----
    def _schedule(self, plan: Plan, seq: Sequence) -> None:
        """Feed the request's next portion (all that is left of it, unless portions are set)."""
        left = len(seq) - seq.num_computed_tokens
        seq.num_scheduled_tokens = min(left, self.portion, self.max_tokens - plan.fresh_tokens) if self.portion > 0 else left
        plan.seqs.append(seq)

    def _admit(self, seq: Sequence) -> None:
        self.pool.admit(seq)
        if self.slots is not None:
            self.slots.take(seq)
        seq.prefilling = True
        # everything found in the prefix cache: still feed the last token
        seq.num_computed_tokens = min(seq.num_cached_tokens, len(seq) - 1)

    def _may_start(self, plan: Plan, seq: Sequence) -> bool:
        if self.slots is not None and self.slots.num_free == 0:
            return False
        room = plan.fresh_tokens < self.max_tokens if self.portion > 0 else plan.fresh_tokens + len(seq) <= self.max_tokens
        return len(plan.seqs) < self.max_seqs and room and self.pool.fits(seq)

    def _plan_prefill(self) -> Plan:
        plan = Plan(is_prefill=True)
        if self.portion > 0:                              # prompts under way go on first
            for seq in self.running:
                if seq.prefilling:
                    if len(plan.seqs) == self.max_seqs or plan.fresh_tokens >= self.max_tokens:
                        break
                    self._schedule(plan, seq)
                    plan.fresh_tokens += seq.num_scheduled_tokens
        started = 0
        for seq in list(self.waiting):                    # arrival order; the first one that does not fit ends the batch
            if not self._may_start(plan, seq):
                break
            self._admit(seq)
            self._schedule(plan, seq)
            plan.fresh_tokens += seq.num_scheduled_tokens if self.portion > 0 else len(seq) - seq.num_cached_tokens
            started += 1
        for _ in range(started):
            seq = self.waiting.popleft()
            seq.status = SequenceStatus.RUNNING
            self.running.append(seq)
        return plan

    def _plan_decode(self) -> Plan:
        plan = Plan(is_prefill=False)
        keep, i = self.running, 0
        while i < len(keep) and len(plan.seqs) < self.max_seqs:
            seq = keep[i]
            while not self.pool.can_grow(seq) and len(keep) > i + 1:
                self._evict(keep.pop())                   # the youngest gives its blocks
            if self.pool.can_grow(seq):
                self.pool.grow(seq)
                seq.num_scheduled_tokens = 1
                plan.seqs.append(seq)
                i += 1
            else:
                self._evict(keep.pop(i))                  # nobody behind it: it goes itself
        if not plan.seqs:
            raise RuntimeError("the KV cache cannot hold a single running request")
        return plan

    def plan(self) -> Plan:
        p = self._plan_prefill() if self.waiting or self.portion > 0 else Plan()
        return p if p.seqs else self._plan_decode()

    def release(self, seq: Sequence) -> None:
        """Give back what the request holds."""
        self.pool.release(seq)
        if self.slots is not None:
            self.slots.give_back(seq)
        seq.num_computed_tokens = seq.num_scheduled_tokens = 0
        seq.prefilling = False

    def _evict(self, seq: Sequence) -> None:
        seq.status = SequenceStatus.WAITING
        self.release(seq)
        self.waiting.appendleft(seq)
        self.num_preemptions += 1

    # ---- after the step ----
    def _is_done(self, seq: Sequence, token_id: int) -> bool:
        if token_id == self.eos and not seq.ignore_eos:
            return True
        return seq.num_completion_tokens == seq.max_tokens or len(seq) == seq.max_total_tokens

    def commit(self, seqs: List[Sequence], token_ids: List[int]) -> List[Sequence]:
        """Append the sampled tokens (a prompt's portion that was not its last one has none); requests that end here
        leave the running list and give their blocks back.  Returns them."""
        ended = []
        for seq, token_id in zip(seqs, token_ids):
            seq.num_computed_tokens += seq.num_scheduled_tokens
            seq.num_scheduled_tokens = 0
            if seq.num_computed_tokens < len(seq):
                continue
            seq.prefilling = False
            seq.append_token(token_id)
            if self._is_done(seq, token_id):
                seq.status = SequenceStatus.FINISHED
                self.release(seq)
                ended.append(seq)
        if ended:
            gone = {id(s) for s in ended}
            self.running = [s for s in self.running if id(s) not in gone]
        return ended
