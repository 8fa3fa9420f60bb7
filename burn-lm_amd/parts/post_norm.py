"""Layers with a norm before and behind each sublayer.

``x <- x + post1(mixer(norm1(x)))``; ``x <- x + post2(feed_forward(norm2(x)))``.  The norm behind a sublayer, the add into
the float32 residual and the norm in front of the next one are one kernel: a block hands on its feed-forward's result as
a ``Joining``, which the next norm takes.  A mixer may hand on several results (two mixers side by side), each with a
norm of its own in front of the sum; those are part of the same kernel."""
from __future__ import annotations

from .base import Block


class PostNormBlock(Block):
    roles = {"mixer_norm": "norm", "mixer": "mixer", "mixer_post": "norm", "ffn_norm": "norm",
             "feed_forward": "feed_forward", "ffn_post": "norm"}

    def forward(self, h, delta, step, view):
        x = self.mixer_norm.add_norm(h, delta)
        joined = self.mixer_post.post(self.mixer.forward_terms(x, step, view))
        x = self.ffn_norm.add_norm(h, joined)
        return self.ffn_post.post(self.feed_forward.forward_terms(x, step))


class PostNormMixerBlock(Block):
    """The same without a feed-forward."""
    roles = {"mixer_norm": "norm", "mixer": "mixer", "mixer_post": "norm"}

    def forward(self, h, delta, step, view):
        x = self.mixer_norm.add_norm(h, delta)
        return self.mixer_post.post(self.mixer.forward_terms(x, step, view))
