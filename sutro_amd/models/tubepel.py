"""Tubepel: a pre-norm layer-list decoder (models/prenorm.py) whose residual is a
bundle of streams (hyper-connections): every sublayer reads a weighted sum of
the streams and its result is added to all of them while they are mixed. A
layer's mixer is latent attention with a query latent and a rotated key part
shared by all heads (two kinds, which differ in the pairing of the rotated
dimensions: neighbours, or halves), or windowed grouped-query attention that
keeps the first tokens in view, with a learned sink per head in the softmax and
an elementwise sigmoid gate on its result. The feed-forward is an ungated
squared-ReLU unit or a mixture of SwiGLU experts whose sigmoid scores multiply
the experts' input, beside an ungated shared expert. A run of layers is passed
several times with the same weights, each pass with its own cache. Plain token
embedding, final norm over the sum of the streams, untied head.
"""

from __future__ import annotations

from .prenorm import PreNormModel


class TubepelModel(PreNormModel):
    """The pre-norm model under a spec of :func:`hybrid_spec.tubepel_spec`."""
