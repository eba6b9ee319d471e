"""Continuous batching over the ragged engine (the SplitFuse composition its `put` / `query` contract is made for).

Every step is one ragged batch of at most `token_budget` tokens: one token of every running sequence first, then
portions of the waiting prompts, the last one cut to what is left. A request is admitted once the cache can hold it to
its end, next to everything admitted before, so no running sequence is ever evicted; its blocks and state slot go back
when it ends."""
from collections import OrderedDict, deque

import torch

from ..sampling import sample_tokens


class _Request:

    def __init__(self, key, prompt, max_new_tokens, eos):
        self.key = key
        self.prompt = torch.as_tensor(prompt, dtype=torch.long).reshape(-1)
        self.max_new_tokens = int(max_new_tokens)
        self.eos = set(eos) if isinstance(eos, (list, tuple, set)) else ({eos} if eos is not None else set())
        self.uid = None
        self.done = 0           # prompt tokens already in the cache
        self.out = []

    def blocks(self, block_size):
        return -(-(self.prompt.numel() + self.max_new_tokens) // block_size)


class RaggedScheduler:

    def __init__(self, engine, token_budget=None, do_sample=False, temperature=1.0, top_k=0, top_p=1.0, seed=None):
        self.engine = engine
        self._sm = engine._config.state_manager
        self.token_budget = min(token_budget or self._sm.max_ragged_batch_size, self._sm.max_ragged_batch_size)
        self._sampling = (do_sample, temperature, top_k, top_p)
        self._generator = None
        if do_sample:
            self._generator = torch.Generator(device=engine._device)
            self._generator.manual_seed(seed if seed is not None else int(torch.initial_seed()) % 2**31)
        self._waiting, self._live = deque(), OrderedDict()
        self._next_uid = max([u for u in engine._state_manager.tracked_sequences if isinstance(u, int)], default=-1) + 1
        self._capacity = engine._state_manager.free_blocks
        self.outputs = {}

    @property
    def pending(self):
        return bool(self._waiting or self._live)

    def add(self, key, prompt, max_new_tokens, eos_token_id=None):
        r = _Request(key, prompt, max_new_tokens, eos_token_id)
        if r.prompt.numel() == 0:
            raise ValueError("empty prompt")
        total = r.prompt.numel() + r.max_new_tokens
        if total > self._sm.max_context or r.blocks(self.engine._state_manager.block_size) > self._capacity:
            raise ValueError(f"a request of {total} tokens does not fit the engine (max_context "
                             f"{self._sm.max_context}, {self._capacity} free cache blocks)")
        if r.max_new_tokens <= 0:
            self.outputs[key] = []
            return
        self._waiting.append(r)

    def _admit(self):
        mgr = self.engine._state_manager
        held = sum(r.blocks(mgr.block_size) for r in self._live.values())
        while self._waiting:
            r = self._waiting[0]
            if len(self._live) >= min(self._sm.max_ragged_sequence_count, self.token_budget) or \
                    held + r.blocks(mgr.block_size) > self._capacity:
                break
            fresh = sum(1 for x in self._live.values() if mgr.get_sequence(x.uid) is None)
            if mgr.n_tracked_sequences + fresh >= self._sm.max_tracked_sequences or \
                    (mgr.free_slots is not None and fresh >= mgr.free_slots):
                break
            r.uid = self._next_uid
            self._next_uid += 1
            held += r.blocks(mgr.block_size)
            self._live[r.uid] = self._waiting.popleft()
        if self._waiting and not self._live:
            raise RuntimeError("the engine has no room for another sequence")

    def step(self):
        """Run one batch; returns the (key, token) pairs it produced."""
        self._admit()
        budget = self.token_budget
        uids, toks = [], []
        for r in self._live.values():
            if r.out:
                uids.append(r.uid)
                toks.append(torch.tensor([r.out[-1]]))
                budget -= 1
        for r in self._live.values():
            left = r.prompt.numel() - r.done
            n = min(left, budget)
            if not r.out and n > 0:
                uids.append(r.uid)
                toks.append(r.prompt[r.done:r.done + n])
                r.done += n
                budget -= n
        if not uids:
            return []
        # logits of the sequences that have their whole prompt in the cache now
        ready = [self._live[u].done == self._live[u].prompt.numel() for u in uids]
        logits = self.engine.put(uids, toks, logit_positions=[[t.numel() - 1] if ok else [] for t, ok in zip(toks, ready)])
        new = sample_tokens(logits, *self._sampling, self._generator).tolist() if any(ready) else []
        produced = []
        for u, tok in zip([u for u, ok in zip(uids, ready) if ok], new):
            r = self._live[u]
            r.out.append(tok)
            produced.append((r.key, tok))
            if len(r.out) >= r.max_new_tokens or tok in r.eos:
                self.outputs[r.key] = r.out
                self.engine.flush(u)
                del self._live[u]
        return produced
