"""Continuous batching over an engine.Model: requests are admitted while sequences and pages are free, every step carries one token of each running request next to
portions of the prompts that are still being read, and finished requests give their sequence back. Greedy sampling on the device; the tokens a step produced are fed to
the next one without passing through the host, which reads them `lag` steps late."""
from collections import deque

import torch

from .lib import PM355Error


class Request:
    def __init__(self, prompt, n_predict, rid=None):
        if not len(prompt):
            raise PM355Error("a request needs at least one prompt token")
        self.prompt, self.n_predict, self.id = list(prompt), n_predict, rid
        self.seq, self.read, self.issued, self.tokens = None, 0, 0, []       # tokens read of the prompt, tokens asked of the device, tokens known

    @property
    def done(self):
        return len(self.tokens) >= self.n_predict


class Scheduler:
    """step_tokens: most tokens per step; portion: most prompt tokens of one request per step. A request is admitted when the pages for its whole length are free (minus what
    the running ones may still take), so that a step never runs out of cache."""

    def __init__(self, model, step_tokens=2048, portion=512, lag=1, keep_logits=False):
        self.model, self.step_tokens, self.portion, self.lag, self.keep_logits = model, step_tokens, portion, lag, keep_logits
        self.waiting, self.running, self.finished = deque(), [], []
        self.reserved, self.pending, self.logits = 0, deque(), {}

    def submit(self, prompt, n_predict, rid=None):
        r = Request(prompt, n_predict, rid)
        info = self.model.pool_info()
        if self._pages(r, info) > info.n_pages or len(r.prompt) + n_predict > info.max_seq_tokens:
            raise PM355Error("the request is longer than the cache")
        self.waiting.append(r)
        return r

    @staticmethod
    def _pages(r, info):
        return -(-(len(r.prompt) + max(r.n_predict - 1, 0)) // info.page_tokens)

    def _admit(self):
        info = self.model.pool_info()
        while self.waiting and self.waiting[0].n_predict < 1:
            self.finished.append(self.waiting.popleft())
        free = info.free_seqs
        while self.waiting and free > 0:
            r = self.waiting[0]
            need = self._pages(r, info)
            if self.reserved + need > info.n_pages:
                break
            self.waiting.popleft()
            r.seq = self.model.seq_new()
            self.reserved += need
            free -= 1
            self.running.append(r)

    def _retire(self, keep):
        """read back the tokens of all steps but the last `keep`"""
        while len(self.pending) > keep:
            rows, host, ev, logits = self.pending.popleft()
            ev.synchronize()
            for i, r in enumerate(rows):
                r.tokens.append(int(host[i]))
                if logits is not None:
                    self.logits.setdefault(id(r), []).append(logits[i].cpu())
        for r in [r for r in self.running if r.done]:
            self.running.remove(r)
            self.model.seq_free(r.seq)
            self.reserved -= self._pages(r, self.model.pool_info())
            self.finished.append(r)

    def step(self):
        """One batch; False when nothing is left to do."""
        self._admit()
        entries, rows, budget = [], [], self.step_tokens
        for r in self.running:                             # tokens first: prompts fill what is left of the step
            if r.read == len(r.prompt) and r.issued < r.n_predict and budget:
                entries.append((r.seq, None, (0,)))
                rows.append(r)
                budget -= 1
        for r in self.running:
            n = min(len(r.prompt) - r.read, self.portion, budget)
            if n > 0:
                last = r.read + n == len(r.prompt)
                entries.append((r.seq, r.prompt[r.read:r.read + n], (n - 1,) if last else ()))
                r.read += n
                budget -= n
                if last:
                    rows.append(r)
        if not entries:
            self._retire(0)
            return bool(self.waiting or self.running)
        for r in rows:
            r.issued += 1
        n = len(rows)
        slot = self._slot(n)
        self.model.batch(entries, logits=slot["logits"], argmax=slot["argmax"])
        slot["host"].copy_(slot["argmax"], non_blocking=True)
        slot["event"].record()
        if n:
            self.pending.append((rows, slot["host"], slot["event"], None if slot["logits"] is None else slot["logits"][:n].clone()))
        self._retire(self.lag)
        return True

    def _slot(self, n):
        """output buffers, one more set than steps in flight; the same ones come round again, so that the engine's captured graphs fit"""
        if not hasattr(self, "_ring"):
            self._ring, self._turn = {}, 0
        self._turn = (self._turn + 1) % (self.lag + 2)
        key = (self._turn, max(n, 1))
        if key not in self._ring:
            dev = self.model.dev
            self._ring[key] = dict(argmax=torch.zeros(max(n, 1), dtype=torch.int32, device=dev), host=torch.zeros(max(n, 1), dtype=torch.int32, pin_memory=True),
                                   event=torch.cuda.Event(), logits=torch.empty(max(n, 1), self.model.n_vocab, device=dev) if self.keep_logits else None)
        return self._ring[key]

    def run(self):
        """until every submitted request is finished; returns them in the order they ended"""
        while self.step():
            pass
        return self.finished


def generate(model, prompts, n_predict, **kw):
    """greedy continuations of several prompts (lists of token ids), batched"""
    s = Scheduler(model, **kw)
    rs = [s.submit(p, n_predict) for p in prompts]
    s.run()
    return [r.tokens for r in rs]
