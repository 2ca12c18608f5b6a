"""What the kernels of libelectrock_decoder.so need to know about the batch of one forward pass: a ragged list of
portions, one per sequence, each the next tokens of its sequence.  A decode step is the case of one token each."""
from dataclasses import dataclass
from typing import List, Optional

import torch

from .sequence import Sequence


@dataclass
class RaggedBatch:
    """All tensors are int32 views of one device buffer, filled by one copy."""
    buffer: torch.Tensor
    n_seqs: int
    max_q: int                      # longest portion
    max_context: int                # longest context, this step's tokens included
    table_width: int
    n_chunks: int
    chunk_tokens: int
    padded_keys: int                # all contexts behind each other, each padded to a multiple of 64
    tokens: torch.Tensor            # [T]
    positions: torch.Tensor         # [T]
    cache_rows: torch.Tensor        # [T] row of the paged cache that takes the token
    q_begin: torch.Tensor           # [n_seqs + 1]
    starts: torch.Tensor            # [n_seqs]
    state_slots: torch.Tensor       # [n_seqs]
    tables: torch.Tensor            # [n_seqs, table_width]
    chunks: torch.Tensor            # [n_chunks, 4] pieces of portions of at most chunk_tokens: sequence, row, tokens, 0
    seq_chunks: torch.Tensor        # [n_seqs + 1]
    k_lens: torch.Tensor            # [n_seqs] context length, this step's tokens included
    k_begin: torch.Tensor           # [n_seqs + 1] first of a sequence's padded keys
    logit_rows: torch.Tensor        # rows whose logits are wanted


@dataclass
class DecodePadding:
    """A fixed shape for decode steps: ``batch`` sequences of one token, tables of ``table_width`` blocks.  Rows beyond the
    real sequences are first tokens of sequences whose cache row and state nobody else uses."""
    batch: int
    table_width: int
    scratch_block: int
    scratch_slot: int


def make_ragged(seqs: List[Sequence], block_size: int, chunk_tokens: int, device, rows: Optional[List[int]] = None,
                padding: Optional[DecodePadding] = None, into: Optional[RaggedBatch] = None) -> RaggedBatch:
    """Describe the planned portions of ``seqs``; ``rows``: batch rows whose logits are wanted (default: the last row of
    every portion).  ``into``: an earlier batch of the same ``padding``, whose buffer is overwritten."""
    tokens, positions, cache_rows, q_begin, chunks, seq_chunks, last = [], [], [], [0], [], [0], []
    for i, s in enumerate(seqs):
        start, n = s.num_computed_tokens, s.num_scheduled_tokens
        if n <= 0 or start + n > len(s) or len(s.block_table) * block_size < start + n:
            raise ValueError("a portion needs tokens, and blocks that hold them")
        row = q_begin[-1]
        tokens.extend(s[start:start + n])
        positions.extend(range(start, start + n))
        cache_rows.extend(s.block_table[p // block_size] * block_size + p % block_size for p in range(start, start + n))
        for at in range(0, n, chunk_tokens):
            chunks += [i, row + at, min(chunk_tokens, n - at), 0]
        q_begin.append(row + n)
        seq_chunks.append(len(chunks) // 4)
        last.append(row + n - 1)
    starts = [s.num_computed_tokens for s in seqs]
    counts = [s.num_scheduled_tokens for s in seqs]
    slots = [s.state_slot for s in seqs]
    contexts = [a + n for a, n in zip(starts, counts)]
    extra = 0
    if padding is not None:
        extra = padding.batch - len(seqs)
        if extra < 0 or any(n != 1 for n in counts):
            raise ValueError("padding is for decode steps of at most its batch")
        for i in range(len(seqs), padding.batch):
            chunks += [i, i, 1, 0]
        tokens, positions = tokens + [0] * extra, positions + [0] * extra
        cache_rows = cache_rows + [padding.scratch_block * block_size] * extra
        q_begin, seq_chunks, last = list(range(padding.batch + 1)), list(range(padding.batch + 1)), list(range(padding.batch))
        starts, slots, contexts = starts + [0] * extra, slots + [padding.scratch_slot] * extra, contexts + [1] * extra
    k_begin = [0]
    for c in contexts:
        k_begin.append(k_begin[-1] + -(-c // 64) * 64)
    width = max(-(-c // block_size) for c in contexts)
    if padding is not None:
        if width > padding.table_width:
            raise ValueError("a context does not fit the padding's tables")
        width = padding.table_width
    tables = []
    for s, c in zip(seqs, contexts):
        used = s.block_table[:-(-c // block_size)]
        tables += used + [0] * (width - len(used))
    for _ in range(extra):
        tables += [padding.scratch_block] + [0] * (width - 1)
    wanted = last if rows is None else rows
    parts = {"tokens": tokens, "positions": positions, "cache_rows": cache_rows, "q_begin": q_begin, "starts": starts,
             "state_slots": slots, "tables": tables, "chunks": chunks, "seq_chunks": seq_chunks,
             "k_lens": contexts, "k_begin": k_begin, "logit_rows": wanted}
    flat, at = [], {}
    for name, values in parts.items():
        flat += [0] * (-len(flat) % 4)                  # 16-byte aligned views
        at[name] = (len(flat), len(values))
        flat += values
    host = torch.tensor(flat, dtype=torch.int32, pin_memory=torch.device(device).type == "cuda")
    if into is not None:
        into.buffer.copy_(host, non_blocking=True)
        return into
    dev = host.to(device, non_blocking=True)
    view = {name: dev[a:a + n] for name, (a, n) in at.items()}
    n_seqs = len(starts)
    view["tables"] = view["tables"].view(n_seqs, width)
    view["chunks"] = view["chunks"].view(-1, 4)
    return RaggedBatch(buffer=dev, n_seqs=n_seqs, max_q=max(counts, default=1),
                       max_context=padding.table_width * block_size if padding is not None else max(contexts),
                       table_width=width, n_chunks=len(chunks) // 4, chunk_tokens=chunk_tokens, padded_keys=k_begin[-1], **view)
