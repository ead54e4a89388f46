"""The parts a model is put together from.  Importing the package registers the built-in
kinds: mixers ``attention``, ``latent_attention``, ``time_mix``, ``gated_delta``,
``selective_scan``, ``decay_attention``, ``channel_delta``, ``rglru`` and ``parallel``; feed-forwards ``swiglu``, ``mlp``, ``gated_mlp``,
``clamped_glu``, ``token_side``, ``routed_swiglu`` and ``routed_mlp``; norms ``rmsnorm`` and ``layernorm``; position ``rope`` and ``none``; blocks
``prenorm``, ``postnorm``, ``sandwich``, ``hyper`` and ``parallel``; embedding ``token``; head
``linear``; junction ``embedding_rejoin``."""
from . import attention, block, embedding, junction, latent, mlp, norm, recurrent, rope  # noqa: F401  (registration)
from .base import (Block, BuildContext, CacheBinding, CacheRequest, Embedding, FeedForward,
                   Head, Junction, Mixer, Norm, NormedInput, Part, PartSpec, PositionEncoding,
                   ResidualStream, TensorSpec, create, lookup, normed, project, register,
                   tensor_specs)

__all__ = ["Block", "BuildContext", "CacheBinding", "CacheRequest", "Embedding", "FeedForward",
           "Head", "Junction", "Mixer", "Norm", "NormedInput", "Part", "PartSpec", "PositionEncoding",
           "ResidualStream", "TensorSpec", "create", "lookup", "normed", "project", "register",
           "tensor_specs"]
