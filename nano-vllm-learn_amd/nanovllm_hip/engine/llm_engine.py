"""generate() over the scheduler, the block manager, the state slots and the runner (nanovllm/engine/llm_engine.py:94-143,
scheduler.py:27-89).  Greedy sampling (bench_my.py uses temperature 0, ignore_eos, fixed max_tokens), so control flow is
value-independent: once only next tokens of running sequences are left to feed, they run as a device-resident graph session."""
from __future__ import annotations

from ..models import load_config
from .block_manager import BlockManager, StateSlots
from .model_runner import ModelRunner, greedy_tokens
from .scheduler import Scheduler
from .sequence import Sequence

MIN_SESSION_STEPS = 8         # fewer steps than this do not pay for capturing a graph


class LLMEngine:
    def __init__(self, cfg, num_kvcache_blocks, max_num_batched_tokens=16384, max_num_seqs=512,
                 max_model_len=4096, enforce_eager=False, device=None, seed=0, warmup=False, weights=None):
        self.cfg = cfg
        self.max_num_batched_tokens = max_num_batched_tokens
        self.max_num_seqs = max_num_seqs
        self.enforce_eager = enforce_eager
        self.runner = ModelRunner(cfg, num_kvcache_blocks, device=device, max_model_len=max_model_len, seed=seed, weights=weights, max_num_seqs=max_num_seqs)
        self.block_manager = BlockManager(num_kvcache_blocks, cfg.kvcache_block_size)
        self.state_slots = StateSlots(max_num_seqs) if self.runner.state else None
        self.scheduler = Scheduler(self.block_manager, self.state_slots, max_num_seqs, max_num_batched_tokens, mixed=self.runner.mixed_batches)
        if warmup:                                                   # the reference always warms up (model_runner.py:52)
            self.runner.warmup_model(max_num_batched_tokens, max_num_seqs)

    @classmethod
    def from_folder(cls, path, config_overrides=None, **kw):
        """Engine for a model folder (config.json, *.safetensors); the architecture it names picks the model."""
        return cls(load_config(path, **(config_overrides or {})), weights=path, **kw)

    def sequence(self, token_ids, max_tokens=64):
        return Sequence(token_ids, max_tokens=max_tokens, block_size=None if self.cfg.kvcache_block_size == Sequence.block_size else self.cfg.kvcache_block_size)

    def prefill(self, seqs, reserve_tokens):
        """Run every waiting sequence through prefill in FCFS batches; appends the first generated token."""
        waiting = list(seqs)
        while waiting:
            batch, ntok = [], 0
            while waiting and len(batch) < self.max_num_seqs and ntok + len(waiting[0]) <= self.max_num_batched_tokens:
                s = waiting.pop(0)
                self.block_manager.allocate(s, reserve_tokens=reserve_tokens)
                if self.state_slots is not None and not self.state_slots.allocate(s):
                    raise RuntimeError("out of state slots")
                batch.append(s)
                ntok += len(s)
            if not batch:
                raise RuntimeError("a prompt exceeds max_num_batched_tokens")
            if self.runner.mixed_batches:
                tokens = self._sample(self.runner.run_step([(s, len(s)) for s in batch]))
            else:
                tokens = self.runner.run(batch, True)
            for s, t in zip(batch, tokens):
                s.append_token(t)

    def _sample(self, logits):
        tokens = greedy_tokens(logits).tolist()
        self.runner.raise_if_device_failed()
        return tokens

    # ------------------------------------------------------------------ token-level use (no sampling)
    def feed(self, portions, want=None):
        """Run given tokens: portions = [(sequence, tokens of it to run)], want = places whose logits are asked for.  Blocks and state slots are
        taken as needed and given back by release(); models with mixed batches only."""
        for seq, n in portions:
            if not self.scheduler.acquire(seq, seq.num_cached_tokens + n):
                raise RuntimeError("out of memory: cache blocks or state slots exhausted")
        return self.runner.run_step(portions, want)

    def release(self, seq):
        self.scheduler.release(seq)

    # ------------------------------------------------------------------ generation
    def step(self):
        """One scheduled batch; appends a token to every sequence whose tokens are all in."""
        batch = self.scheduler.schedule()
        if self.runner.mixed_batches:
            done = [s.num_cached_tokens + n == len(s) for s, n in batch]
            logits = self.runner.run_step(batch, [[n - 1] if d else [] for (_, n), d in zip(batch, done)])
            seqs = [s for (s, _), d in zip(batch, done) if d]
            tokens = self._sample(logits) if seqs else []
        else:
            seqs = [s for s, _ in batch]
            tokens = self.runner.run(seqs, seqs[0].num_cached_tokens == 0)
            for s in seqs:
                s.num_cached_tokens = len(s)
        self._append(seqs, tokens)

    def _append(self, seqs, tokens):
        for s, t in zip(seqs, tokens):
            s.append_token(t)
        for s in seqs:
            if s.finished:
                self.scheduler.finish(s)

    def _decode_session(self):
        """Run the decoding sequences together until the first one finishes, as one graph session; False when that is not possible."""
        seqs = list(self.scheduler.decoding())
        if self.enforce_eager or not seqs:
            return False
        n = min(s.max_tokens - s.num_completion_tokens for s in seqs)
        if n < MIN_SESSION_STEPS or not all(self.scheduler.acquire(s, len(s) + n) for s in seqs):
            return False
        sess = self.runner.decode_session(seqs, n)
        sess.step(n)
        sess.finish()
        for s in seqs:
            s.num_cached_tokens = len(s) - 1
        self._append(seqs, [])
        return True

    def generate(self, prompt_token_ids, max_tokens):
        """Greedy-generate tokens for every prompt (max_tokens: one number, or one per prompt); returns the completion token ids."""
        counts = max_tokens if isinstance(max_tokens, (list, tuple)) else [max_tokens] * len(prompt_token_ids)
        seqs = [self.sequence(p, n) for p, n in zip(prompt_token_ids, counts)]
        for s in seqs:
            if len(s) + s.max_tokens > self.runner.max_model_len + 1:
                raise ValueError(f"prompt of {len(s)} tokens + {s.max_tokens} exceeds max_model_len {self.runner.max_model_len}")
            self.scheduler.add(s)
        while self.scheduler.unfinished():
            if not self._decode_session():
                self.step()
        return [s.completion_token_ids for s in seqs]
