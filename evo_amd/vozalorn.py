"""Vozalorn: latent attention over a sliding window or decayed linear attention, each with a gated feed-forward or none.  A norm sits on every
sublayer's OUTPUT, before it is added, with its weight stored as a difference from one:

    x <- x + norm1(mixer(x));   x <- x + norm2(ff(x))          norm(y) = y / sqrt(mean(y^2) + eps) * (1 + w)
"""
from __future__ import annotations

from .decoder import LayeredDecoder
from .mixers import GatedFF, LatentAttention, LightningMixer


class Vozalorn(LayeredDecoder):
    MIXERS = {"lightning": LightningMixer, "latent_attention": LatentAttention}
    FEED_FORWARDS = {"dense": GatedFF}
    REQUIRED = LayeredDecoder.REQUIRED + ("embedding",)
    NORM_OFFSET = 1.0

    def _read_config(self, c) -> None:
        self.embed_scale = float(c["embedding"]["scale"])
