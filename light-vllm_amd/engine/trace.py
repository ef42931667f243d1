"""Trace replay: given token ids go through a model step by step and the logits asked for come back.

The replay composes the steps (which requests, how many new tokens each) in place of the scheduling policy; everything
else is the engine's own: block and state-slot managers, input builder, worker step, caches, kernels.  Nothing is
sampled."""
from typing import Dict, List, Optional, Tuple

import torch

from .config import CacheConfig, SchedulerConfig
from .input_builder import token_rows
from .llm_engine import LLMEngine
from .sequence import Sequence, SequenceGroup, SequenceStatus

MAX_LIVE_REQUESTS = 4


class TraceReplay:

    def __init__(self, model_config, max_tokens: int, device: str = "cuda:0", max_live: int = MAX_LIVE_REQUESTS,
                 block_size: int = 16):
        """`max_tokens`: the most tokens that live requests hold at any time, each count rounded up to a multiple of 64."""
        blocks = -(-max_tokens // block_size)
        cc = CacheConfig(block_size=block_size, num_gpu_blocks=blocks, num_cpu_blocks=0, num_state_slots=max_live)
        sc = SchedulerConfig(max_num_batched_tokens=max(max_tokens, 64), max_num_seqs=max_live,
                             max_model_len=max(max_tokens, 64), use_v2_block_manager=True, chunked_prefill_enabled=True)
        self.engine = LLMEngine(model_config, cc, sc, device=device, use_hip_graph=False)
        self.groups: Dict[str, SequenceGroup] = {}
        self._next_id = 0

    def _group(self, request_id: str, tokens: List[int]) -> SequenceGroup:
        g = self.groups.get(request_id)
        if g is None:
            seq = Sequence(self._next_id, tokens, self.engine.cache_config.block_size)
            self._next_id += 1
            g = self.groups[request_id] = SequenceGroup(request_id, [seq])
        else:
            for t in tokens:
                g.seqs[0].append_token_id(t)
        return g

    def step(self, entries: List[Tuple[str, List[int], List[int]]]) -> Optional[torch.Tensor]:
        """entries: (request id, its next tokens, places among them whose logits are wanted).  Returns float32
        [wanted, vocab] on the CPU in the order of the entries and of their places, None when nothing is wanted."""
        vocab = self.engine.model_config.vocab_size
        for rid, tokens, want in entries:
            if not tokens or not all(0 <= t < vocab for t in tokens) or not all(0 <= w < len(tokens) for w in want):
                raise ValueError(f"request {rid}: empty portion, token out of the vocabulary or place out of the portion")
        if len({rid for rid, _, _ in entries}) != len(entries):
            raise ValueError("a request may appear once in a step")
        eng = self.engine
        sched = eng.scheduler.schedule_exact([(self._group(rid, tokens), len(tokens)) for rid, tokens, _ in entries])
        first_row = {m.request_id: row for _, m, row, _, _, _ in
                     token_rows(sched.seq_group_metadata_list, eng.cache_config.block_size, None)}
        rows = [first_row[rid] + w for rid, _, want in entries for w in want]
        with torch.cuda.stream(eng.stream):
            logits = eng.worker.execute_logits(eng.input_builder(sched), rows)
            out = logits.float().cpu() if logits is not None else None
        eng.stream.synchronize()
        for s in sched.scheduled_seq_groups:
            s.seq_group.update_num_computed_tokens(s.token_chunk_size)
        return out

    def end(self, request_id: str) -> None:
        """The request is finished: its blocks and its state slot are given back."""
        g = self.groups.pop(request_id)
        g.seqs[0].status = SequenceStatus.FINISHED_STOPPED
        self.engine.scheduler.free_seq(g.seqs[0])
        self.engine.scheduler.free_finished_request([request_id])
