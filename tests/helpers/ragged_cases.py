"""Schedules and comparisons for tests of ragged-step models: a trace of portions through ``RaggedEngine``, a mixer
alone over a used cache, and the error measure of logits against an oracle."""
import torch

from edgellm.engine.paged import PagedCache
from edgellm.engine.ragged import RaggedEngine
from edgellm.ops import seqmix


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def replay(model, schedule, reqs, max_tokens, slots=4, graphs=None):
    """``schedule``: steps of [(request name, token count)]; every row's logits are collected.
    A request ends (slot and pages given back) with its last token."""
    eng = RaggedEngine(model, max_tokens, slots=slots, use_graphs=graphs)
    at = {r: 0 for r in reqs}
    got = {r: [] for r in reqs}
    for step in schedule:
        entries = []
        for r, n in step:
            entries.append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
            at[r] += n
        logits = eng.step(entries).cpu()
        o = 0
        for r, n in step:
            got[r].append(logits[o:o + n])
            o += n
            if at[r] == len(reqs[r]):
                eng.close(r)
    assert all(at[r] == len(reqs[r]) for r in reqs)
    return {r: torch.cat(v) for r, v in got.items()}, eng


def row_err(got, want):
    """Root mean square over the vocabulary of the difference (its mean taken off), over the spread of ``want``."""
    d = got.double() - want
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std().item()


def close(got, want, tol):
    return row_err(got, want).max().item() < tol


def portions(total, first=2, mod=9):
    cuts, n = [], first
    while total:
        cuts.append(min(n, total))
        total -= cuts[-1]
        n = n % mod + 2
    return cuts


def step_meta(cache, slots, step, dev):
    """RaggedMeta of [(sequence, start, length)] with room made in the cache."""
    for s, st, n in step:
        cache.extend(slots[s], st + n)
    return seqmix.RaggedMeta.build([(slots[s], st, n) for s, st, n in step], cache.page_table, cache.page, dev)


def run_mixer(mod, spec, hs, cuts, dev, dtype=torch.float32):
    """Interleaved sequences ``hs`` (inputs [L, W]) through a mixer alone in portions from ``cuts``, over pages
    and state rows that held something else.  Returns (outputs per sequence, the run's cache)."""
    cache = PagedCache([spec], sum((h.shape[0] + 63) // 64 for h in hs) + 1, slots=len(hs) + 1, page=64, dtype=dtype, device=dev)
    run = cache.run(0)
    for t in (run.k, run.v, run.lat, run.ssm):
        if t is not None:
            t.normal_()
    slots = {s: cache.acquire() for s in range(len(hs))}
    at, got, step_i = [0] * len(hs), [[] for _ in hs], 0
    while any(at[s] < hs[s].shape[0] for s in range(len(hs))):
        step = [(s, at[s], min(cuts[(step_i + s) % len(cuts)], hs[s].shape[0] - at[s])) for s in range(len(hs)) if at[s] < hs[s].shape[0]]
        meta = step_meta(cache, slots, step, dev)
        with torch.no_grad():
            out = mod(torch.cat([hs[s][st:st + n] for s, st, n in step]).to(dev, dtype), meta, run).float().cpu()
        o = 0
        for s, st, n in step:
            got[s].append(out[o:o + n])
            o += n
            at[s] += n
        step_i += 1
    return [torch.cat(g) for g in got], run
