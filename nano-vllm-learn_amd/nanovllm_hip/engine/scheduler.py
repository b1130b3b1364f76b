"""Which tokens run in the next step.

Two policies over the same queues (FCFS, at most max_num_seqs sequences, at most max_num_batched_tokens tokens a step):
  prefill first (nanovllm/engine/scheduler.py:27-89)  whole prompts while any wait and fit, otherwise one token of every running sequence
  mixed          for models whose step takes portions of prompts beside single tokens: every running sequence's next tokens first, then
                 portions of waiting prompts up to the token budget
A running sequence that finds no block for its next token makes the youngest running one give up its blocks and state (scheduler.py:60-89) and
start over from its own tokens later."""
from collections import deque


class Scheduler:
    def __init__(self, block_manager, state_slots=None, max_num_seqs=512, max_num_batched_tokens=16384, mixed=False):
        self.block_manager, self.state_slots = block_manager, state_slots
        self.max_num_seqs, self.max_num_batched_tokens, self.mixed = max_num_seqs, max_num_batched_tokens, mixed
        self.waiting, self.running = deque(), []

    def add(self, seq):
        self.waiting.append(seq)

    def unfinished(self):
        return bool(self.waiting or self.running)

    def acquire(self, seq, num_tokens):
        """Blocks for the sequence's first `num_tokens` tokens and a state slot; all or nothing."""
        if self.state_slots is not None and not self.state_slots.allocate(seq):
            return False
        if self.block_manager.grow(seq, num_tokens):
            return True
        if self.state_slots is not None and not seq.block_table:
            self.state_slots.deallocate(seq)
        return False

    def _acquire_whole(self, seq):
        """Blocks for the prompt and, while the pool has them, for everything the sequence will generate: a block table that never changes
        gives every decode step the same launch geometry."""
        return self.acquire(seq, len(seq) + seq.max_tokens - seq.num_completion_tokens) or self.acquire(seq, len(seq))

    def release(self, seq):
        self.block_manager.deallocate(seq)                      # (num_cached_tokens back to zero)
        if self.state_slots is not None:
            self.state_slots.deallocate(seq)

    def decoding(self):
        """The running sequences, when nothing but their next tokens can run: every one has only its newest token left to feed."""
        if not self.running or any(len(s) - s.num_cached_tokens != 1 for s in self.running):
            return []
        return [] if self.waiting and self._admissible(self.waiting[0]) else self.running

    def _admissible(self, seq):
        free = len(self.block_manager.free_block_ids)
        bs = self.block_manager.block_size
        slot = self.state_slots is None or seq.state_slot >= 0 or bool(self.state_slots.free)
        return len(self.running) < self.max_num_seqs and slot and free * bs >= min(len(seq), self.max_num_batched_tokens)

    def _preempt(self, seq):
        self.running.remove(seq)
        self.release(seq)
        self.waiting.appendleft(seq)

    def schedule(self):
        """[(sequence, tokens of it that run now)] with blocks and slots in place."""
        batch, budget = [], self.max_num_batched_tokens
        if not self.mixed:
            while self.waiting and len(self.running) < self.max_num_seqs and len(self.waiting[0]) <= budget and self._acquire_whole(self.waiting[0]):
                seq = self.waiting.popleft()
                self.running.append(seq)
                batch.append((seq, len(seq)))
                budget -= len(seq)
            if batch:
                return batch
        for seq in list(self.running):
            if seq not in self.running or budget <= 0:          # (given up for an older one above)
                continue
            n = min(len(seq) - seq.num_cached_tokens, budget)
            while not self.acquire(seq, seq.num_cached_tokens + n):
                victim = self.running[-1]
                self._preempt(victim)
                batch = [(s, k) for s, k in batch if s is not victim]
                if victim is seq:
                    break
            else:
                batch.append((seq, n))
                budget -= n
        if self.mixed:
            while self.waiting and budget > 0 and len(self.running) < self.max_num_seqs:
                seq = self.waiting[0]
                n = min(len(seq) - seq.num_cached_tokens, budget)
                if not self.acquire(seq, seq.num_cached_tokens + n):
                    break
                self.waiting.popleft()
                self.running.append(seq)
                batch.append((seq, n))
                budget -= n
        if not batch:
            raise RuntimeError("out of memory: KV cache blocks exhausted" if len(self.waiting) <= 1 or self.waiting[0].num_tokens <= self.max_num_batched_tokens
                               else "a prompt exceeds max_num_batched_tokens")
        return batch

    def finish(self, seq):
        self.running.remove(seq)
        self.release(seq)
