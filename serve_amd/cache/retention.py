"""How long a layer keeps a token's cache, as data.

A rule is None (for the whole context), an int W (a token sees the last W tokens, itself among them), or `Chunks(n)`
(the sequence is cut into runs of n positions, counted from its position 0; a token sees its own run up to itself).
Layers with equal rules share a group of pages; the manager gives a page back once no later token can see it.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Union


@dataclass(frozen=True)
class Chunks:
    size: int


Retention = Union[None, int, Chunks]


def check(rule: Retention) -> None:
    n = rule.size if isinstance(rule, Chunks) else rule
    if n is not None and n <= 0:
        raise ValueError("a window or a chunk must be positive")


def reach(rule: Retention) -> Optional[int]:
    """The most tokens that a token sees, itself among them (None: no bound)."""
    return rule.size if isinstance(rule, Chunks) else rule


def first_seen(rule: Retention, position: int) -> int:
    """The first position that a token at `position` sees (and so does every later token: none sees an earlier one)."""
    if rule is None:
        return 0
    if isinstance(rule, Chunks):
        return position - position % rule.size
    return max(0, position - rule + 1)


def mean_seen(rule: Retention, context: float) -> float:
    """How many tokens a token sees that is the last of a context of about `context` tokens, for accounts of bytes: a
    chunk is half full on the average."""
    if rule is None:
        return context
    if isinstance(rule, Chunks):
        return min(context, (rule.size + 1) / 2.0)
    return min(context, rule)


def sort_key(rule: Retention):
    """Full retention first, then windows and chunks by their length."""
    return (rule is not None, isinstance(rule, Chunks), reach(rule) or 0)
