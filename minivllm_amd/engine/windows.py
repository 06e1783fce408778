"""What an attention layer sees of a sequence, and how many places of a block table that takes.

A plain number is chunked attention: a token sees the earlier tokens of its own chunk of that size (0: all of the sequence).
``SlidingWindow`` is the ``size`` tokens up to a token's own (0: all); token ``p`` lies at place ``p mod places`` of the table,
a ring that is a little longer than the window: an entry of fewer than ``LONG_ROWS`` rows may be stored as a whole before its
first row reads the oldest token it sees."""
from __future__ import annotations

from dataclasses import dataclass

LONG_ROWS = 32                 # an entry of at least this many rows is long


@dataclass(frozen=True, order=True)
class SlidingWindow:
    size: int = 0

    @property
    def places(self) -> int:
        return self.size + LONG_ROWS - 2 if self.size else 0


def places(window) -> int:
    """Places of a table after which it starts anew; 0: never."""
    return window.places if isinstance(window, SlidingWindow) else window
