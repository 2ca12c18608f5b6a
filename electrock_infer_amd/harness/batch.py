"""What the kernels of libelectrock_decoder.so need to know about the batch of one forward pass: a ragged list of
portions, one per sequence, each the next tokens of its sequence.  A decode step is the case of one token each."""
from dataclasses import dataclass
from typing import List, Optional

import torch

from .sequence import Sequence


@dataclass
class RaggedBatch:
    """All tensors are int32 views of one device buffer, filled by one copy."""
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


def make_ragged(seqs: List[Sequence], block_size: int, chunk_tokens: int, device, rows: Optional[List[int]] = None) -> RaggedBatch:
    """Describe the planned portions of ``seqs``; ``rows``: batch rows whose logits are wanted (default: the last row of
    every portion)."""
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
    contexts = [a + n for a, n in zip(starts, counts)]
    k_begin = [0]
    for c in contexts:
        k_begin.append(k_begin[-1] + -(-c // 64) * 64)
    width = max(-(-c // block_size) for c in contexts)
    tables = []
    for s, c in zip(seqs, contexts):
        used = s.block_table[:-(-c // block_size)]
        tables += used + [0] * (width - len(used))
    wanted = last if rows is None else rows
    parts = {"tokens": tokens, "positions": positions, "cache_rows": cache_rows, "q_begin": q_begin, "starts": starts,
             "state_slots": [s.state_slot for s in seqs], "tables": tables, "chunks": chunks, "seq_chunks": seq_chunks,
             "k_lens": contexts, "k_begin": k_begin, "logit_rows": wanted}
    flat, at = [], {}
    for name, values in parts.items():
        flat += [0] * (-len(flat) % 4)                  # 16-byte aligned views
        at[name] = (len(flat), len(values))
        flat += values
    host = torch.tensor(flat, dtype=torch.int32, pin_memory=torch.device(device).type == "cuda")
    dev = host.to(device, non_blocking=True)
    view = {name: dev[a:a + n] for name, (a, n) in at.items()}
    view["tables"] = view["tables"].view(len(seqs), width)
    view["chunks"] = view["chunks"].view(-1, 4)
    return RaggedBatch(n_seqs=len(seqs), max_q=max(counts), max_context=max(contexts), table_width=width,
                       n_chunks=len(chunks) // 4, chunk_tokens=chunk_tokens, padded_keys=k_begin[-1], **view)
