"""How far back the attention of a model reaches, for the scheduler: which cache blocks a sequence still needs."""
from __future__ import annotations

from dataclasses import dataclass

EVERYTHING = 1 << 30   # window of a layer that sees every earlier token


@dataclass(frozen=True)
class KeyReach:
    """windows: sizes of sliding windows; chunks: sizes of chunks (counted from position 0), of all layers that read the cache."""
    windows: tuple = ()
    chunks: tuple = ()

    def first_visible(self, pos: int) -> int:
        """The earliest position that a token at `pos` or any later one may see."""
        return max(0, min([pos] + [pos - w + 1 for w in self.windows] + [pos - pos % c for c in self.chunks]))

    @property
    def span(self) -> int:
        """Most positions that one token sees."""
        return max((0,) + tuple(self.windows) + tuple(self.chunks))
