"""Decode steps as HIP graphs: the forward pass of a padded batch of single tokens is recorded once per (batch size, table
width) and replayed with new contents of its one integer buffer, so that a step costs the host one copy and one launch.

A graph is kept only if it passes two tests when it is recorded.  It may hold no memset node (a library call may record
one; such nodes are not reliable in replays), and on a batch of nothing but padding -- first tokens of sequences that
start from nothing -- several replays, with the program's own work in between, must equal the eager result bit for bit.
Otherwise that shape runs eagerly.
"""
import ctypes
from typing import Dict, List, Optional, Tuple

import torch

from .batch import DecodePadding, RaggedBatch, make_ragged
from .sequence import Sequence

_NODE_MEMSET = 2        # hipGraphNodeTypeMemset


def memset_nodes(graph: torch.cuda.CUDAGraph) -> int:
    """Memset nodes of a graph that was recorded with keep_graph=True."""
    hip = ctypes.CDLL("libamdhip64.so")
    raw, count = ctypes.c_void_p(graph.raw_cuda_graph()), ctypes.c_size_t(0)
    if hip.hipGraphGetNodes(raw, None, ctypes.byref(count)) != 0:
        raise RuntimeError("hipGraphGetNodes failed")
    nodes = (ctypes.c_void_p * count.value)()
    if hip.hipGraphGetNodes(raw, nodes, ctypes.byref(count)) != 0:
        raise RuntimeError("hipGraphGetNodes failed")
    kinds = []
    for node in nodes:
        kind = ctypes.c_int(-1)
        if hip.hipGraphNodeGetType(ctypes.c_void_p(node), ctypes.byref(kind)) != 0:
            raise RuntimeError("hipGraphNodeGetType failed")
        kinds.append(kind.value)
    return kinds.count(_NODE_MEMSET)


class _Recorded:

    def __init__(self, graph: torch.cuda.CUDAGraph, batch: RaggedBatch, padding: DecodePadding, logits: torch.Tensor):
        self.graph, self.batch, self.padding, self.logits = graph, batch, padding, logits


class DecodeGraphs:

    BATCHES = (1, 2, 4, 8, 12, 16, 24, 32, 48, 64, 96, 128, 192, 256)
    MIN_WIDTH = 8           # table widths are powers of two from here on

    def __init__(self, runner):
        self.runner = runner
        self.recorded: Dict[Tuple[int, int], Optional[_Recorded]] = {}     # None: this shape runs eagerly
        self.pool = None
        self.replays = 0

    def shape_of(self, seqs: List[Sequence]) -> Optional[Tuple[int, int]]:
        batch = next((b for b in self.BATCHES if b >= len(seqs)), None)
        if batch is None:
            return None
        need, width = max(-(-(s.num_computed_tokens + 1) // self.runner.block_size) for s in seqs), self.MIN_WIDTH
        while width < need:
            width *= 2
        return batch, width

    def run(self, seqs: List[Sequence]) -> Optional[torch.Tensor]:
        """Logits [len(seqs), vocab], or None if the step has to run eagerly."""
        shape = self.shape_of(seqs)
        if shape is None:
            return None
        if shape not in self.recorded:
            self.recorded[shape] = self._record(*shape)
        r = self.recorded[shape]
        if r is None:
            return None
        self.runner.check_slots(seqs)
        self._fill(seqs, r.padding, r.batch)
        r.graph.replay()
        self.replays += 1
        return r.logits[:len(seqs)]

    def _fill(self, seqs, padding: DecodePadding, into: Optional[RaggedBatch] = None) -> RaggedBatch:
        runner = self.runner
        return make_ragged(seqs, runner.block_size, runner.model.chunk_tokens(1), runner.device, padding=padding, into=into)

    # (outside inference mode: a recording leaves tensors behind in torch's generator that later recordings write to)
    @torch.inference_mode(False)
    @torch.no_grad()
    def _record(self, batch_size: int, width: int) -> Optional[_Recorded]:
        runner, model = self.runner, self.runner.model
        padding = DecodePadding(batch_size, width, runner.config.num_kvcache_blocks, runner.config.num_state_slots)
        batch = self._fill([], padding)
        step = lambda: model.compute_logits(model(batch), batch)
        side = torch.cuda.Stream(device=runner.device)
        side.wait_stream(torch.cuda.current_stream(runner.device))
        with torch.cuda.stream(side):       # libraries set themselves up outside the recording
            step()
            eager = step().clone()
        torch.cuda.current_stream(runner.device).wait_stream(side)
        torch.cuda.synchronize(runner.device)
        graph = torch.cuda.CUDAGraph(keep_graph=True)
        with torch.cuda.graph(graph, pool=self.pool, stream=side):
            logits = step()
        if memset_nodes(graph) > 0:
            return None
        graph.instantiate()
        self.pool = self.pool or graph.pool()
        for _ in range(3):
            logits.fill_(float("nan"))
            graph.replay()
            torch.cuda.synchronize(runner.device)
            if not torch.equal(logits, eager):
                return None
            step()
        return _Recorded(graph, batch, padding, logits)
