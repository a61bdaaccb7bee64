"""The parts a model is put together from. Importing registers them."""

from .base import (AnySize, BiasedRows, CacheNeed, HyperAddend, NormSink, PagedTensor, Part, PartSpec, Precision, StreamAddend, TensorShape, UnscaledRows,
                   build_part)
from . import (attention, block, channel_delta, embedding, feed_forward, head, latent_attention, mamba2, mlstm,  # noqa: F401
               norm, parallel, pooled_window_attention, position, retention, rglru, routed_experts, sigmoid_attention,
               sink_attention, softcap_attention, span_attention)

__all__ = ["AnySize", "BiasedRows", "CacheNeed", "HyperAddend", "NormSink", "PagedTensor", "Part", "PartSpec", "Precision", "StreamAddend", "TensorShape", "UnscaledRows", "build_part"]
