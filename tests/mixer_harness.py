"""What the tests of single mixer kernels share: the ragged layout of a step, keys and values in shuffled pages, inputs
in which single (query, key) pairs tower over the rest, and the ways a run of tokens is cut into a step."""
import random
from types import SimpleNamespace

import torch

DEV = "cuda:0"


def ragged(seqs, width=None):
    """seqs: [(ctx_len, new tokens, state slot, block table)] -> the step's ragged layout on the device."""
    q_start, token_seq = [0], []
    for i, (_, n, _, _) in enumerate(seqs):
        q_start.append(q_start[-1] + n)
        token_seq += [i] * n
    width = width or max(len(s[3]) for s in seqs) or 1
    tables = [list(s[3]) + [0] * (width - len(s[3])) for s in seqs]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)          # noqa: E731
    return SimpleNamespace(
        q_start=i32(q_start), ctx_len=i32([s[0] for s in seqs]), token_seq=i32(token_seq),
        state_slot=i32([s[2] for s in seqs]), block_tables=i32(tables).reshape(len(seqs), width), num_seqs=len(seqs),
        max_query_len=max(s[1] for s in seqs), max_pages_used=width,
        max_page_id=max([max(s[3]) for s in seqs if s[3]] or [0]), max_state_slot=max(s[2] for s in seqs))


def ops():
    from splitwise_amd import _C
    return _C.mixer_ops


def tol_of(dtype):
    return dict(atol=2e-5, rtol=2e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=2e-2)


def attention_case(H, G, d, dv, n, spikes, seed, big=6.0):
    """Random q, k, v with, for every (query position, key position, head) in ``spikes``, that query and key made
    long along a direction of their own, so that the pair's score towers over the query's other scores."""
    g = torch.Generator().manual_seed(seed)
    q = torch.randn(n, H, d, generator=g) * 0.5
    k = torch.randn(n, G, d, generator=g) * 0.5
    v = torch.randn(n, G, dv, generator=g)
    for num, (i, j, a) in enumerate(spikes):
        e = torch.zeros(d)
        e[num % d] = 1.0
        q[i, a] = big * e + 0.05 * q[i, a]
        k[j, a // (H // G)] = big * e + 0.05 * k[j, a // (H // G)]
    return q, k, v


def paged(rows_k, rows_v, page, dtype, seed):
    """Key / value rows in pages handed out in a shuffled order; unused pages hold NaN."""
    n = rows_k.shape[0]
    pages = -(-n // page)
    order = list(range(pages + 3))
    random.Random(seed).shuffle(order)
    table = order[:pages]
    kc = torch.full((pages + 3, page, rows_k.shape[1]), float("nan"), dtype=dtype)
    vc = None if rows_v is None else torch.full((pages + 3, page, rows_v.shape[1]), float("nan"), dtype=dtype)
    for t in range(n):
        kc[table[t // page], t % page] = rows_k[t].to(dtype)
        if vc is not None:
            vc[table[t // page], t % page] = rows_v[t].to(dtype)
    return kc.to(DEV), None if vc is None else vc.to(DEV), table


def steps_of(mode, n, table):
    """-> (the step's sequences, the positions they cover in order)."""
    if mode == "prompt":
        return [(0, n, 0, table)], list(range(n))
    if mode == "decode":
        rows = list(range(n - 45, n)) + [0, 1, 33]
        return [(t, 1, 0, table) for t in rows], rows
    if mode == "pairs":                                                  # steps of two tokens, and one of a single token
        firsts = list(range(n - 46, n, 2)) + [0, 32, 127]
        return [(t, 2, 0, table) for t in firsts] + [(n - 47, 1, 0, table)], \
            [t + i for t in firsts for i in range(2)] + [n - 47]
    cuts, at = [], 0
    for size in [3, 2, 27, 1, 31, 2, 64, 2, 33, 5, 32, 98]:
        cuts.append((at, size, 0, table))
        at += size
    assert at == n
    random.Random(3).shuffle(cuts)                                       # portions of "different sequences" in any order
    return cuts, [c[0] + i for c in cuts for i in range(c[1])]
