"""The serving engine around a step model: paged block allocation, step building, continuous batching with chunked
prompts, and generation.

  BlockAllocator   free lists of cache blocks (block tables hold first-slot ids: block * block_size) and of the state
                   slots of recurrent layers
  Sequence         token ids, how many of them the cache holds, its blocks and its state slot
  StepBuilder      entries (sequence, new tokens) -> tokens, positions, InputParameters of ONE batch
  Scheduler        which sequences bring how many tokens into the next step
  LLMEngine        the loop: schedule -> ModelRunner.forward -> sample -> finish

A step model is anything with forward(tokens, positions, params, return_logits=True) -> logits: DagupelStep,
VebusunStep, LlamaDecodeStep.
"""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Deque, Dict, List, Optional, Sequence as Seq, Tuple

import numpy as np
import torch

from .layers import InputParameters, Portion
from .model_runner import ModelRunner, ModelRunnerOptions
from .sampling import Sampler, SamplingParams


class OutOfBlocks(RuntimeError):
    """The cache pool has no free block (or state slot) left."""


class BlockAllocator:
    """n_states: recurrent state slots, one per live sequence (0: the model keeps none)."""

    def __init__(self, n_blocks: int, block_size: int, n_states: int = 0):
        if block_size < 1 or block_size & (block_size - 1):
            raise ValueError("block_size is a power of two")
        self.n_blocks, self.block_size, self.n_states = n_blocks, block_size, n_states
        self._free: Deque[int] = deque(range(n_blocks))
        self._free_states: Deque[int] = deque(range(n_states))

    @property
    def n_free(self) -> int:
        return len(self._free)

    def blocks_for(self, n_tokens: int) -> int:
        return (n_tokens + self.block_size - 1) // self.block_size

    def allocate(self, n: int) -> List[int]:
        if n > len(self._free):
            raise OutOfBlocks(f"{n} cache blocks wanted, {len(self._free)} free")
        return [self._free.popleft() for _ in range(n)]

    def free(self, blocks: Seq[int]) -> None:
        self._free.extend(blocks)

    @property
    def n_free_states(self) -> int:
        return len(self._free_states)

    def can_admit(self, n_tokens: int) -> bool:
        """Room for a new sequence of n_tokens tokens?"""
        return self.blocks_for(n_tokens) <= self.n_free and (not self.n_states or bool(self._free_states))

    def allocate_state(self) -> int:
        if not self._free_states:
            raise OutOfBlocks(f"all {self.n_states} state slots are taken")
        return self._free_states.popleft()

    def free_state(self, slot: int) -> None:
        self._free_states.append(slot)


@dataclass
class Sequence:
    id: object
    tokens: List[int]
    n_cached: int = 0                 # tokens whose keys the cache holds
    blocks: List[int] = field(default_factory=list)
    state: Optional[int] = None       # slot of its recurrent state
    n_prompt: int = 0
    sampler: Optional[Sampler] = None

    def reserve(self, allocator: BlockAllocator, n_tokens: int) -> None:
        """Blocks for the first n_tokens tokens, and a state slot where the model keeps state."""
        need = allocator.blocks_for(n_tokens) - len(self.blocks)
        if need > 0:
            self.blocks += allocator.allocate(need)
        if allocator.n_states and self.state is None:
            self.state = allocator.allocate_state()

    def release(self, allocator: BlockAllocator) -> None:
        allocator.free(self.blocks)
        if self.state is not None:
            allocator.free_state(self.state)
        self.blocks, self.state, self.n_cached = [], None, 0


@dataclass
class Step:
    """One batch, ready for the model.  Entry i of the call that built it starts at row row0[i]."""
    tokens: torch.Tensor
    positions: torch.Tensor
    params: InputParameters
    row0: List[int]
    order: List[int]    # order[k] = the entry that is k-th in the batch

    def rows(self, i: int, places: Seq[int]) -> List[int]:
        return [self.row0[i] + p for p in places]


class StepBuilder:
    """portion_min (of the model): entries that bring at least so many tokens go behind the others and are described
    as portions; None: the model serves every row alike."""

    def __init__(self, allocator: BlockAllocator, device, portion_min: Optional[int] = None):
        self.allocator, self.device, self.portion_min = allocator, device, portion_min

    def build(self, entries: Seq[Tuple[Sequence, int]], logit_rows: Optional[Dict[int, Seq[int]]] = None) -> Step:
        """entries: (sequence, number of its next tokens).  logit_rows: entry -> places among its new tokens whose
        logits are wanted, entries in their given order; None = the last of every sequence, in batch order."""
        B = self.allocator.block_size
        n_new = [n for _, n in entries]
        for seq, n in entries:
            if n < 1 or seq.n_cached + n > len(seq.tokens):
                raise ValueError(f"sequence {seq.id}: {n} new tokens of {len(seq.tokens) - seq.n_cached}")
        is_portion = [self.portion_min is not None and n >= self.portion_min for n in n_new]
        order = sorted(range(len(entries)), key=lambda i: is_portion[i])   # (stable)
        tokens, pos, slots, table, bcu, q_cu, kv_cu, portions = [], [], [], [], [0], [0], [0], []
        row0 = [0] * len(entries)
        for i in order:
            seq, n = entries[i]
            c = seq.n_cached
            seq.reserve(self.allocator, c + n)
            blocks = np.asarray(seq.blocks[:self.allocator.blocks_for(c + n)], dtype=np.int32) * B
            p = np.arange(c, c + n, dtype=np.int32)
            row0[i] = q_cu[-1]
            tokens.append(np.asarray(seq.tokens[c:c + n], dtype=np.int32))
            pos.append(p)
            slots.append(blocks[p // B] + p % B)
            table.append(blocks)
            if is_portion[i]:
                portions.append(Portion(row0[i], n, c + n, blocks))
            bcu.append(bcu[-1] + blocks.size)
            q_cu.append(q_cu[-1] + n)
            kv_cu.append(kv_cu[-1] + c + n)
        arrays = [np.concatenate(tokens), np.concatenate(pos), np.concatenate(slots), np.concatenate(table),
                  np.asarray(bcu), np.asarray(q_cu), np.asarray(kv_cu)]
        if self.allocator.n_states:
            arrays.append(np.asarray([entries[i][0].state for i in order]))
        if logit_rows is not None:
            arrays.append(np.asarray([row0[i] + p for i in range(len(entries)) for p in logit_rows.get(i, ())], dtype=np.int32))
        # one transfer; every array starts on a 16-byte boundary of it
        sizes = [a.size for a in arrays]
        at = np.concatenate([[0], np.cumsum([(n + 3) // 4 * 4 for n in sizes])]).astype(np.int64)
        packed = np.zeros(int(at[-1]), dtype=np.int32)
        for a, s in zip(arrays, at):
            packed[s:s + a.size] = a
        dev = torch.from_numpy(packed).to(self.device)
        d = [dev[int(s):int(s) + n] for s, n in zip(at, sizes)]
        kv_lens = np.diff(kv_cu)
        state_slots = d[7] if self.allocator.n_states else None
        params = InputParameters(q_cu_seq_lens=d[5], kv_cu_seq_lens=d[6], new_cache_slots=d[2], block_tables=d[3],
                                 cu_block_lens=d[4], q_max_seq_len=max(n_new), kv_max_seq_len=int(kv_lens.max()),
                                 kv_total_len=int(kv_cu[-1]), logit_rows=d[-1] if logit_rows is not None else None,
                                 portions=portions, state_slots=state_slots)
        return Step(d[0], d[1], params, row0, order)

    @staticmethod
    def commit(entries: Seq[Tuple[Sequence, int]]) -> None:
        for seq, n in entries:
            seq.n_cached += n


class Scheduler:
    """Continuous batching: every running sequence's next token first, then prompts in order of arrival, cut to what
    is left of the step's token budget.  When the pool runs dry the youngest sequence gives its blocks back and
    starts over later (its tokens are kept)."""

    def __init__(self, allocator: BlockAllocator, max_seqs: int, max_step_tokens: int):
        self.allocator, self.max_seqs, self.max_step_tokens = allocator, max_seqs, max_step_tokens
        self.waiting: Deque[Sequence] = deque()
        self.running: List[Sequence] = []     # oldest first

    def add(self, seq: Sequence) -> None:
        self.waiting.append(seq)

    def finish(self, seq: Sequence) -> None:
        self.running.remove(seq)
        seq.release(self.allocator)

    def _preempt(self) -> Sequence:
        seq = self.running.pop()
        seq.release(self.allocator)
        self.waiting.appendleft(seq)
        return seq

    def schedule(self) -> List[Tuple[Sequence, int]]:
        budget = self.max_step_tokens
        entries: List[Tuple[Sequence, int]] = []
        preempted = False
        # single next tokens before portions of prompts, each oldest first
        for seq in sorted(self.running, key=lambda s: len(s.tokens) - s.n_cached > 1):
            if seq not in self.running or budget == 0:
                continue
            n = min(len(seq.tokens) - seq.n_cached, budget)
            while True:
                try:
                    seq.reserve(self.allocator, seq.n_cached + n)
                    break
                except OutOfBlocks:
                    victim = self._preempt()
                    preempted = True
                    gone = [e for e in entries if e[0] is victim]
                    entries = [e for e in entries if e[0] is not victim]
                    budget += sum(e[1] for e in gone)
                    if victim is seq:
                        break
            if seq in self.running:
                entries.append((seq, n))
                budget -= n
        while self.waiting and not preempted and budget > 0 and len(self.running) < self.max_seqs:
            seq = self.waiting[0]
            if not self.allocator.can_admit(len(seq.tokens)):
                break   # (a lone request always fits: LLMEngine.add_request)
            n = min(len(seq.tokens), budget)
            seq.reserve(self.allocator, n)
            self.running.append(self.waiting.popleft())
            entries.append((seq, n))
            budget -= n
        return entries


@dataclass
class EngineOptions:
    max_seqs: int = 64
    max_step_tokens: int = 2048
    graph_batch_sizes: List[int] = field(default_factory=list)   # decode batches captured into hipGraphs
    graph_max_seq_len: int = 2048


class LLMEngine:
    def __init__(self, model, n_blocks: int, block_size: int, device="cuda", options: Optional[EngineOptions] = None):
        self.model, self.device = model, torch.device(device)
        self.options = o = options or EngineOptions()
        self.allocator = BlockAllocator(n_blocks, block_size, getattr(model, "n_states", 0))
        self.builder = StepBuilder(self.allocator, self.device, getattr(model, "portion_min", None))
        self.scheduler = Scheduler(self.allocator, o.max_seqs, o.max_step_tokens)
        self.runner = ModelRunner(model, self.device, ModelRunnerOptions(
            block_size=block_size, cuda_graph_max_seq_len=o.graph_max_seq_len, cuda_graph_batch_sizes=list(o.graph_batch_sizes)),
            return_logits=True)
        shape = getattr(model, "shape", None)
        self.max_positions = getattr(model, "max_positions", None) or shape.max_position
        self.vocab = getattr(model, "vocab", None) or shape.vocab
        self._next_id = 0

    def capture_graphs(self) -> None:
        """Warm-up: one graph per decode batch size.  The capture runs write to the cache, so call it before serving."""
        for bs in sorted(self.options.graph_batch_sizes):
            self.runner.capture_cuda_graphs(bs)

    def run_entries(self, entries: Seq[Tuple[Sequence, int]], logit_rows: Optional[Dict[int, Seq[int]]] = None):
        """One step of the model over `entries`; the cache holds their tokens afterwards.  -> (Step, logits)."""
        step = self.builder.build(entries, logit_rows)
        logits = self.runner.forward(step.tokens, step.positions, step.params)
        self.builder.commit(entries)
        return step, logits

    def check_tokens(self, tokens: Seq[int], at: int = 0) -> None:
        if at + len(tokens) > self.max_positions:
            raise ValueError(f"{at + len(tokens)} tokens exceed the model's {self.max_positions} positions")
        if len(tokens) and not (0 <= min(tokens) and max(tokens) < self.vocab):
            raise ValueError(f"token ids are 0 .. {self.vocab - 1}")

    def add_request(self, prompt: Seq[int], params: SamplingParams) -> Sequence:
        if not prompt:
            raise ValueError("the prompt is empty")
        self.check_tokens(prompt)
        total = min(len(prompt) + params.max_tokens, self.max_positions)
        if self.allocator.blocks_for(total) > self.allocator.n_blocks:
            raise ValueError(f"{total} tokens do not fit the cache pool")
        seq = Sequence(self._next_id, [int(t) for t in prompt], n_prompt=len(prompt), sampler=Sampler(params, self.device))
        self._next_id += 1
        self.scheduler.add(seq)
        return seq

    def step(self) -> List[Sequence]:
        """One scheduled step; the sequences that finished in it."""
        entries = self.scheduler.schedule()
        if not entries:
            return []
        step, logits = self.run_entries(entries)
        done = []
        for k, i in enumerate(step.order):
            seq = entries[i][0]
            if seq.n_cached < len(seq.tokens):
                continue   # (a portion of a prompt: nothing to sample yet)
            p = seq.sampler.params
            token = seq.sampler.sample(logits[k])
            seq.tokens.append(token)
            if token in p.stop_ids or len(seq.tokens) - seq.n_prompt >= p.max_tokens or len(seq.tokens) >= self.max_positions:
                done.append(seq)
        for seq in done:
            self.scheduler.finish(seq)
        return done

    def generate(self, prompts: Seq[Seq[int]], params: SamplingParams) -> List[List[int]]:
        """Token ids in, generated token ids out."""
        seqs = [self.add_request(p, params) for p in prompts]
        left = set(s.id for s in seqs)
        while left:
            left -= {s.id for s in self.step()}
        return [s.tokens[s.n_prompt:] for s in seqs]
