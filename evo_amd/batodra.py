"""Batodra: gated linear recurrences, differential attention over the whole sequence, and attention over a sliding window whose first tokens stay
visible, each with an ungated feed-forward (square of relu) or none.  The norm of a layer's sublayers sits behind the addition:

    x <- norm1(alpha x + mixer(x));   x <- norm2(alpha x + ff(x))          norm(t) = t / sqrt(mean(t^2) + eps) * w
"""
from __future__ import annotations

from functools import partial

from .decoder import LayeredDecoder
from .mixers import GatedRecurrence, HeadAttention, PlainFF


class Batodra(LayeredDecoder):
    MIXERS = {"rglru": GatedRecurrence, "attention": partial(HeadAttention, maps=2, qk_norm=True), "attention_2": partial(HeadAttention, unit_qk=True)}
    FEED_FORWARDS = {"dense": partial(PlainFF, act="relu2")}
    REQUIRED = LayeredDecoder.REQUIRED + ("postln_alpha",)

    def _read_config(self, c) -> None:
        self.alpha = float(c["postln_alpha"])
