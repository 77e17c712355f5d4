"""Serving on a cache of shared cells: requests as sequences, steps that mix prompt portions and single tokens, greedy sampling.

Stepper maps requests to sequences and runs given tokens; Scheduler decides what each step holds (continuous batching: every running
request decodes one token per step, the rest of the token budget goes to waiting prompts, portion by portion)."""
import collections

import numpy as np

MAX_SEQS = 31              # sequence ids of the shared cache a server may hand out


class Stepper:
    """Requests by name on the sequences of one model (Model.kv_cells_*)."""

    def __init__(self, model, n_cells, max_live=MAX_SEQS):
        self.m = model
        self.n_cells = n_cells
        model.kv_cells_init(n_cells)
        self.free = list(range(min(max_live, MAX_SEQS)))[::-1]
        self.seq, self.pos = {}, {}

    @property
    def free_cells(self):
        return self.n_cells - sum(self.pos.values())

    def admit(self, rid):
        if not self.free:
            raise RuntimeError("no free sequence: too many live requests")
        self.seq[rid], self.pos[rid] = self.free.pop(), 0

    def end(self, rid):
        """Gives back the request's cells and its sequence."""
        s = self.seq.pop(rid)
        del self.pos[rid]
        self.m.kv_cells_seq_rm(s, -1, -1)
        self.free.append(s)

    def run(self, entries, logits=True, greedy=False):
        """entries: (request, its next tokens, places among them that are wanted).  One batch.  Returns (logits [wanted, vocab] or None,
        greedy next tokens or None) in the order of the entries and their places."""
        tokens, positions, masks, want = [], [], [], []
        for rid, toks, places in entries:
            if rid not in self.seq:
                self.admit(rid)
            base, p, s = len(tokens), self.pos[rid], self.seq[rid]
            tokens.extend(toks)
            positions.extend(range(p, p + len(toks)))
            masks.extend([1 << s] * len(toks))
            want.extend(base + k for k in places)
        if not tokens:
            return (np.empty((0, self.m.hp.n_vocab), np.float32) if logits else None), (np.empty(0, np.int32) if greedy else None)
        nxt, lg = self.m.kv_cells_step(tokens, positions, masks, want, want_logits=logits, want_next=greedy)
        for rid, toks, _ in entries:
            self.pos[rid] += len(toks)
        return lg, nxt


class Request:
    def __init__(self, rid, prompt, max_new, eos=None):
        self.id, self.prompt, self.max_new, self.eos = rid, [int(t) for t in prompt], int(max_new), eos
        self.fed, self.out = 0, []

    @property
    def need(self):                                     # cells the request can come to hold (its last token is never fed back)
        return len(self.prompt) + max(self.max_new - 1, 0)

    @property
    def done(self):
        return len(self.out) >= self.max_new or (self.eos is not None and self.out and self.out[-1] == self.eos)


class Scheduler:
    """Continuous batching with greedy sampling.  A request is admitted when the pool can hold all it may come to need."""

    def __init__(self, model, n_cells, max_live=16, budget=512):
        self.st = Stepper(model, n_cells, max_live)
        self.budget, self.max_live = int(budget), max_live
        self.waiting, self.running, self.finished = collections.deque(), [], {}

    def submit(self, rid, prompt, max_new, eos=None):
        r = Request(rid, prompt, max_new, eos)
        if not r.prompt or r.need > self.st.n_cells:
            raise ValueError("an empty prompt, or a request larger than the cache")
        self.waiting.append(r)

    def _admit(self):
        reserved = sum(r.need for r in self.running)
        while self.waiting and len(self.running) < self.max_live and reserved + self.waiting[0].need <= self.st.n_cells:
            r = self.waiting.popleft()
            reserved += r.need
            self.running.append(r)

    def step(self):
        """One batch; returns the tokens it sampled as (request id, token)."""
        self._admit()
        entries, sample, left = [], [], self.budget
        for r in self.running:                          # running requests first: one token each
            if r.fed >= len(r.prompt):
                entries.append((r.id, r.out[-1:], [0]))
                sample.append(r)
                left -= 1
        for r in self.running:
            if r.fed < len(r.prompt) and left > 0:
                part = r.prompt[r.fed:r.fed + left]
                last = r.fed + len(part) == len(r.prompt)
                entries.append((r.id, part, [len(part) - 1] if last else []))
                r.fed += len(part)
                left -= len(part)
                if last:
                    sample.append(r)
        if not entries:
            return []
        _, nxt = self.st.run(entries, logits=False, greedy=True)
        got = []
        for r, tok in zip(sample, nxt):
            r.out.append(int(tok))
            got.append((r.id, int(tok)))
        for r in [r for r in self.running if r.done]:
            self.running.remove(r)
            self.st.end(r.id)
            self.finished[r.id] = r.out
        return got

    def run(self):
        """Until every request has finished: request id -> generated tokens."""
        while self.waiting or self.running:
            self.step()
        return self.finished


def generate(model, prompts, max_new, n_cells=None, max_live=16, budget=512):
    """Greedy continuations of several prompts through the scheduler."""
    need = sum(len(p) + max_new for p in prompts)
    n_cells = n_cells or (need + 31) // 32 * 32
    s = Scheduler(model, n_cells, max_live, budget)
    for i, p in enumerate(prompts):
        s.submit(i, p, max_new)
    out = s.run()
    return [out[i] for i in range(len(prompts))]
