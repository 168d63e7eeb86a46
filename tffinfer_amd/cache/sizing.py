"""How many pages each group of layers gets.

A group that keeps every key needs pages for all the tokens the engine is to
hold.  A group with a window needs, per request, only the pages its window and
the step's new tokens touch, whatever the length of the request; giving it the
full pool would pay for the cache twice.  The reference has one geometry for
all layers and sizes its pool from the free device memory
(src/core/runtime/KVCache.h:267-281, src/core/runtime/InferRuntime.cu:123-136).
"""
from __future__ import annotations

import math

from ..parts.base import KVCacheSpec


def group_layers(requirements) -> dict[KVCacheSpec, int]:
    """Cache spec -> number of caches (layer calls that write one) of that spec, in the
    order the cache manager forms its groups."""
    spec_of = {}
    for cache_id, _writes, kv_spec, *_ in requirements:
        if kv_spec is not None:
            spec_of[cache_id] = kv_spec
    out: dict[KVCacheSpec, int] = {}
    for cache_id in sorted(spec_of):
        out[spec_of[cache_id]] = out.get(spec_of[cache_id], 0) + 1
    return out


def state_id(row) -> int:
    """The number of a layer call's state: the row's fifth element where it has one, else its cache's number."""
    return row[4] if len(row) > 4 else row[0]


def state_bytes(requirements, max_seqs: int) -> int:
    """Device bytes of the per-request state tensors (one row more than there are requests)."""
    seen, total = set(), 0
    for row in requirements:
        st, sid = row[3], state_id(row)
        if st is not None and sid not in seen:
            seen.add(sid)
            total += (max_seqs + 1) * math.prod(st.shape) * st.dtype.itemsize
    return total


def min_window_pages(window: int, page_size: int, keep_first: int = 0) -> int:
    """Pages a request must be able to hold in a group with a window to advance by one token:
    the window's tokens, wherever the window's start falls in its page, and the pages of the
    first tokens that the group keeps for good."""
    return -(-max(window - 1, 0) // page_size) + 1 + -(-keep_first // page_size)


def window_pool_pages(window: int, page_size: int, max_seqs: int, token_budget: int, keep_first: int = 0) -> int:
    """Pages with which a group with a window never runs short: a request that brings n tokens to
    a step touches the n + window - 1 tokens that end with them, at most ceil((n + window - 1) /
    page) + 1 pages, and a step's portions hold ``token_budget`` tokens between them; every
    request also keeps the pages of its first ``keep_first`` tokens."""
    return (max_seqs * (-(-max(window - 1, 0) // page_size) + 2 + -(-keep_first // page_size))
            + -(-token_budget // page_size))


def pool_pages(spec: KVCacheSpec, tokens: int, page_size: int) -> int:
    """Pages a request of ``tokens`` tokens holds for the whole blocks of all of the cache's block sizes."""
    return sum(-(-(tokens // p) // page_size) for p in spec.pools)


def request_pages(spec: KVCacheSpec, tokens: int, page_size: int) -> int:
    """Pages a request must be able to hold in this cache to reach ``tokens`` tokens one at a time."""
    n = -(-tokens // page_size)
    if spec.window > 0:
        n = min(n, min_window_pages(spec.reach, page_size, spec.keep_first))
    return n + pool_pages(spec, tokens, page_size)


def bytes_per_page(spec: KVCacheSpec, layers: int, page_size: int, elem_size: int) -> int:
    return 2 * layers * spec.num_kv_heads * spec.head_dim * page_size * elem_size


def plan_pages(requirements, page_size: int, elem_size: int, max_seqs: int, token_budget: int,
               tokens: int | None = None, kv_bytes: int | None = None,
               free_bytes: int | None = None) -> dict[KVCacheSpec, int]:
    """Pages per group.  ``tokens``: what the groups that keep every key shall hold (plus a page
    a request for the last, partly filled one); ``kv_bytes``: or the device bytes that all groups
    may take together; ``free_bytes``: a cap on those bytes (the state tensors come off it
    first).  Groups with a window get what :func:`window_pool_pages` says, never more than a
    group that keeps every key."""
    groups = group_layers(requirements)
    if not groups:
        return {}
    if any(s.pools for s in groups):
        return _plan_pages_with_blocks(requirements, groups, page_size, elem_size, max_seqs, token_budget, tokens,
                                       kv_bytes, free_bytes)
    full = [s for s in groups if s.window <= 0]
    want_full = None if tokens is None else -(-tokens // page_size) + max_seqs
    pages = {}
    for s in groups:
        if s.window > 0:
            n = window_pool_pages(s.window, page_size, max_seqs, token_budget, s.keep_first)
            pages[s] = n if want_full is None else min(n, want_full)
    budget = None
    if kv_bytes is not None:
        budget = int(kv_bytes)
    if free_bytes is not None:
        cap = max(0, int(free_bytes) - state_bytes(requirements, max_seqs))
        budget = cap if budget is None else min(budget, cap)

    def cost(spec, n):
        return n * bytes_per_page(spec, groups[spec], page_size, elem_size)

    if budget is None and want_full is None:
        raise ValueError("the cache needs a size: tokens, bytes or the free memory")
    if budget is not None:
        # the groups with a window first (they are small); if even they do not fit, they shrink alike
        win_cost = sum(cost(s, n) for s, n in pages.items())
        if win_cost > budget:
            pages = {s: int(n * budget / win_cost) for s, n in pages.items()}
            win_cost = sum(cost(s, n) for s, n in pages.items())
        per_full = sum(cost(s, 1) for s in full)
        fit = int((budget - win_cost) // per_full) if per_full else 0
        for s in full:
            pages[s] = fit if want_full is None else min(want_full, fit)
    else:
        for s in full:
            pages[s] = want_full
    bad = [s for s, n in pages.items() if n < 1]
    if bad:
        raise ValueError(f"the memory given to the cache holds no page of {page_size} tokens for {bad[0]}")
    return pages


def _plan_pages_with_blocks(requirements, groups, page_size, elem_size, max_seqs, token_budget, tokens, kv_bytes,
                            free_bytes) -> dict[KVCacheSpec, int]:
    """The same where some groups keep a key per block of tokens for good: those pages grow with the
    tokens held, so the most tokens that fit the bytes are found by bisection."""
    def pages_for(n: int) -> dict:
        full = -(-n // page_size) + max_seqs
        out = {}
        for s in groups:
            own = full
            if s.window > 0:
                own = min(full, window_pool_pages(s.reach, page_size, max_seqs, token_budget, s.keep_first))
            out[s] = own + sum(-(-(n // p) // page_size) + max_seqs for p in s.pools)
        return out

    budget = None if kv_bytes is None else int(kv_bytes)
    if free_bytes is not None:
        cap = max(0, int(free_bytes) - state_bytes(requirements, max_seqs))
        budget = cap if budget is None else min(budget, cap)
    if budget is None and tokens is None:
        raise ValueError("the cache needs a size: tokens, bytes or the free memory")

    def fits(n: int) -> bool:
        return budget is None or sum(k * bytes_per_page(s, groups[s], page_size, elem_size)
                                     for s, k in pages_for(n).items()) <= budget

    hi = int(tokens) if tokens is not None else 1 << 40
    if fits(hi):
        return pages_for(hi)
    lo = page_size
    if not fits(lo):
        raise ValueError(f"the memory given to the cache holds no page of {page_size} tokens a request")
    while hi - lo > 1:
        mid = (lo + hi) // 2
        lo, hi = (mid, hi) if fits(mid) else (lo, mid)
    return pages_for(lo)
