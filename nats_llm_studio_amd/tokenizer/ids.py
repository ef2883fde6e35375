"""Tokenizer of checkpoints that come without one: text is token ids separated by white space. A word that is not an id
of the vocabulary becomes its UTF-8 bytes, folded into the vocabulary, so any chat text still makes a prompt."""
from __future__ import annotations

from typing import List, Optional, Sequence

TEMPLATE = "{% for m in messages %}{{ m['content'] }}\n{% endfor %}"


class IdTokenizer:
    def __init__(self, vocab_size: int):
        self.n = int(vocab_size)
        self.tokens: List[str] = []
        self.vocab: dict = {}
        self.bos_id: Optional[int] = None
        self.eos_id: Optional[int] = None

    def encode(self, text: str, add_bos: bool = False) -> List[int]:
        out: List[int] = []
        for w in text.split():
            if w.isascii() and w.isdigit() and int(w) < self.n:
                out.append(int(w))
            else:
                out += [b % self.n for b in w.encode("utf-8")]
        return out

    def decode(self, ids: Sequence[int]) -> str:
        return " ".join(str(int(i)) for i in ids)
