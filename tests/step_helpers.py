"""Helpers of the tests of models that run through a StepRunner."""

import numpy as np
import pytest
import torch

from fei_amd.engine.config import get_spec
from fei_amd.engine.step import StepEntry, StepRunner
from fei_amd.models import model_class

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F32_TOL = 3e-5


class Net:
    """A model with its oracle's weights. ``edit`` changes them first."""

    def __init__(self, tmp, oracle, cfg, seed=0, device="cpu",
                 dtype=torch.float32, edit=None, max_seq=512, **shape):
        self.cfg, self.oracle = cfg, oracle
        self.W = oracle.random_weights(cfg, seed, **shape)
        if edit:
            edit(self.W)
            self.W = {k: v.bfloat16().to(oracle.real)
                      for k, v in self.W.items()}
        self.path = str(tmp)
        oracle.save_model(self.path, cfg, self.W)
        spec = get_spec(self.path)
        self.model = model_class(spec)(spec, torch.device(device), dtype,
                                       max_seq_len=max_seq,
                                       weights=self.path)

    def runner(self, blocks=16, slots=4, block_size=64, poison=True):
        r = StepRunner(self.model, blocks, slots, block_size)
        if poison:        # whatever is read without having been written shows
            for t in r.cache.rows + r.cache.states:
                if t is not None:
                    t.fill_(float("nan"))
        return r

    def want(self, tokens):
        return self.oracle.forward(tokens, self.W, self.cfg)


def toks(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def row_errors(got, want):
    """Error of each row, relative to the row's size."""
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape
    return (got - want).norm(dim=-1) / want.norm(dim=-1)


def err(got, want):
    """Largest row error."""
    return float(row_errors(got, want).max())


def run(r, sid, tokens, sizes):
    """All logits of ``tokens`` run in portions of ``sizes`` (repeated)."""
    out, at, i = [], 0, 0
    while at < len(tokens):
        part = tokens[at:at + sizes[i % len(sizes)]]
        out.append(r.step([StepEntry(sid, part, range(len(part)))]))
        at += len(part)
        i += 1
    return torch.cat(out)


def run_mixed(r, reqs, seed=0):
    """All logits of each request, served together in random portions beside
    single tokens, with pauses; a request that ends makes room for another."""
    rng = np.random.default_rng(seed)
    at = {i: 0 for i in reqs}
    live, waiting = {}, list(reqs)
    got = {i: [] for i in reqs}
    while live or waiting:
        while waiting and r.cache.free_slots() and \
                len(reqs[waiting[0]]) + 64 <= r.cache.free_blocks() * 64:
            live[waiting[0]] = r.admit(len(reqs[waiting[0]]))
            waiting.pop(0)
        entries, who = [], []
        for i, sid in live.items():
            if len(live) > 1 and rng.random() < 0.2:
                continue
            n = int(rng.choice([1, 1, 2, 3, 17, 64, 70]))
            part = reqs[i][at[i]:at[i] + n]
            entries.append(StepEntry(sid, part, range(len(part))))
            who.append((i, len(part)))
        if not entries:
            continue
        logits = r.step(entries)
        row = 0
        for i, n in who:
            got[i].append(logits[row:row + n])
            row += n
            at[i] += n
            if at[i] == len(reqs[i]):
                r.release(live.pop(i))
    return {i: torch.cat(x) for i, x in got.items()}


def serve_sessions(mgr, prompts, max_new, steps=200):
    """Generated tokens of each prompt, opened as room allows."""
    todo, open_, got = list(range(len(prompts))), {}, {}
    for _ in range(steps):
        while todo:
            try:
                open_[todo[0]] = mgr.open(prompts[todo[0]],
                                          max_new_tokens=max_new)
                todo.pop(0)
            except MemoryError:
                break
        if mgr.step_chunk(3) == 0:
            break
        for i, sid in list(open_.items()):
            if mgr.result(sid)["done"]:
                got[i] = mgr.result(sid)["token_ids"]
                mgr.close(sid)
                del open_[i]
    return [got.get(i) for i in range(len(prompts))]
