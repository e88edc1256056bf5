"""Scenarios that the tests of every mixer decoder run through the framework:
schedules of portions and single tokens, mixed batches, slots and pages used
again, generation, conversations.  A case brings a small model with random
weights and the plain oracle's logits (luzalorn_cases, lunulix_cases)."""

from __future__ import annotations

import random

import torch

from quickstart_streaming_agents_amd.models.serve import Engine, StepEntry

# largest error of a logit row (mean taken off, rms over the vocabulary,
# relative to the rms of the oracle's logits)
TOL = {torch.float32: 1e-4, torch.bfloat16: 5e-2}


class MixerCase:
    """raw: configuration as in config.json; cfg, weights, model from it;
    forward: the oracle's (raw, weights, tokens) -> (logits, trail)."""

    def __init__(self, raw, cfg, model_class, weights, forward, device,
                 dtype):
        self.raw, self.cfg, self.weights = raw, cfg, weights
        self.model = model_class(cfg, device=device, dtype=dtype,
                                 weights=weights)
        self.forward, self.device, self.dtype = forward, device, dtype
        self._oracle = {}

    def tokens(self, n, seed=0):
        r = random.Random(seed)
        return [r.randrange(self.cfg.vocab_size) for _ in range(n)]

    def oracle(self, tokens):
        key = tuple(tokens)
        if key not in self._oracle:
            self._oracle[key] = self.forward(self.raw, self.weights,
                                             tokens)[0]
        return self._oracle[key]

    def limits(self, want):
        """Largest error of every row of an oracle's logits."""
        return torch.full((len(want),), TOL[self.dtype], dtype=torch.float64)

    def engine(self, tokens=4096, **kw):
        kw.setdefault("max_batch", 4)
        return Engine(self.model, kv_pages=-(-tokens // 64),
                      max_seq_len=tokens, **kw)


def row_errors(got, want):
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    scale = want.pow(2).mean().sqrt()
    return d.pow(2).mean(-1).sqrt() / scale


def check(case, got, want, what=""):
    err, limit = row_errors(got, want), case.limits(want)
    worst = int((err / limit).argmax())
    assert float(err[worst]) <= float(limit[worst]), \
        f"{what}: row {worst} off by {float(err[worst]):.2e}"


def run_steps(case, requests, steps, pool=None, engine=None):
    """requests: id -> tokens; steps: lists of (id, count).  Every position's
    logits are asked for; requests leave when their tokens are used up.
    Returns id -> [T, vocab]."""
    total = sum(-(-len(t) // 64) * 64 for t in requests.values())
    eng = engine or case.engine(pool or total, state_slots=4)
    seq, at, out, free = {}, {}, {r: [] for r in requests}, 100
    for step in steps:
        entries = []
        for rid, n in step:
            if rid not in seq:
                seq[rid], at[rid] = free, 0
                free += 1
            toks = requests[rid][at[rid]:at[rid] + n]
            assert len(toks) == n
            entries.append(StepEntry(seq[rid], toks, at[rid],
                                     list(range(n))))
            at[rid] += n
        logits = eng.step_entries(entries).float().cpu()
        k = 0
        for rid, n in step:
            out[rid].append(logits[k:k + n])
            k += n
        for rid, _ in step:
            if at[rid] == len(requests[rid]):
                eng.kv.free(seq[rid])
    return {r: torch.cat(o) for r, o in out.items()}


def portions(n, sizes, tail=0):
    """Cut n tokens into portions cycling through sizes, the last `tail`
    one by one."""
    out, k = [], 0
    while sum(out) < n - tail:
        out.append(min(sizes[k % len(sizes)], n - tail - sum(out)))
        k += 1
    return out + [1] * (n - sum(out))


def alone(rid, cuts):
    return [[(rid, c)] for c in cuts]


# ---- scenarios --------------------------------------------------------------

CUTS = {
    "whole": lambda n: [n],
    "one by one": lambda n: [1] * n,
    "decoded tail": lambda n: [n - n // 3] + [1] * (n // 3),
    "twos and threes": lambda n: portions(n, [2, 3]),
    "odd sizes": lambda n: portions(n, [17, 2, 64, 16, 5, 65], tail=7),
    "page edges": lambda n: portions(n, [63, 2, 63, 128], tail=3),
}


def scenario_cuts(case, n, cuts):
    toks = case.tokens(n, seed=n)
    got = run_steps(case, {"a": toks}, alone("a", CUTS[cuts](n)))
    check(case, got["a"], case.oracle(toks), cuts)


def mixed_steps(lengths, seed):
    """Portions of some requests beside single tokens of others, pauses
    included; requests enter late and leave early."""
    r = random.Random(seed)
    left = dict(lengths)
    steps = []
    while left:
        live = list(left)[:4]
        step = []
        for rid in live:
            if r.random() < 0.2 and len(live) > 1:
                continue
            n = min(left[rid], r.choice([1, 1, 1, 2, 3, 16, 17, 40, 64, 90]))
            step.append((rid, n))
            left[rid] -= n
        left = {k: v for k, v in left.items() if v}
        if step:
            r.shuffle(step)
            steps.append(step)
    return steps


def scenario_mixed(case, seed=0):
    """Ten requests through four slots and a pool that holds four of them."""
    lengths = {f"r{i}": n for i, n in enumerate(
        [150, 1, 75, 33, 200, 64, 2, 129, 90, 20])}
    reqs = {r: case.tokens(n, seed=i)
            for i, (r, n) in enumerate(lengths.items())}
    got = run_steps(case, reqs, mixed_steps(lengths, seed), pool=4 * 256)
    for rid, toks in reqs.items():
        check(case, got[rid], case.oracle(toks), rid)


def scenario_reuse(case):
    """The same slot and pages again: nothing of the former owner shows."""
    eng = case.engine(256, state_slots=1)
    for i, n in enumerate((200, 3, 130, 1, 64)):
        toks = case.tokens(n, seed=50 + i)
        got = run_steps(case, {"a": toks}, alone("a", portions(n, [50, 2],
                                                               tail=1)),
                        engine=eng)
        check(case, got["a"], case.oracle(toks), f"owner {i}")
    assert eng.kv.free_pages == eng.kv.n_pages
    assert eng.kv.free_slots == eng.kv.n_slots


def greedy_check(case, prompt, out):
    """Every generated token is the oracle's best, up to rounding."""
    lg = case.oracle(prompt + out)[len(prompt) - 1:-1]
    best = lg.max(-1).values
    took = lg.gather(1, torch.tensor(out)[:, None])[:, 0]
    slack = 6 * TOL[case.dtype] * float(lg.pow(2).mean().sqrt())
    assert float((best - took).max()) <= slack


def scenario_generate(case, use_graph=None, chunk_tokens=None, new=40):
    prompts = [case.tokens(n, seed=n) for n in (5, 1, 90, 130, 17, 2)]
    news = [new, 7, new, 12, new, new]
    eng = case.engine(1024, max_batch=3, chunk_tokens=chunk_tokens)
    if use_graph is not None:
        eng.use_graph = use_graph
    for _ in range(2):                    # again: replays after the first
        outs = eng.generate_batch(prompts, news)
        assert [len(o) for o in outs] == news
        for p, o in zip(prompts, outs):
            greedy_check(case, p, o)
    assert eng.kv.free_pages == eng.kv.n_pages
    assert eng.kv.free_slots == eng.kv.n_slots
    return outs


def scenario_conversation(case):
    """Turns that extend each other build on the snapshot of the last one."""
    eng = case.engine(1024, max_batch=2)
    prompt, prev = case.tokens(70, seed=3), None
    for turn in range(3):
        seq = eng.submit(prompt, 9, continue_from=prev, keep_alive=True)
        assert seq.cached_len == (len(prev.prompt) if prev else 0)
        eng.run_to_completion()
        greedy_check(case, prompt, seq.out_tokens)
        prev = seq
        prompt = prompt + case.tokens(20 + 30 * turn, seed=90 + turn)
    # a prompt that branches off earlier starts afresh
    other = prompt[:50] + case.tokens(30, seed=77)
    seq = eng.submit(other, 5, continue_from=prev, keep_alive=True)
    assert seq.cached_len == 0
    eng.run_to_completion()
    greedy_check(case, other, seq.out_tokens)
    eng.release(seq)
    assert eng.kv.free_pages == eng.kv.n_pages
    assert eng.kv.free_slots == eng.kv.n_slots
