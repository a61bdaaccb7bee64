"""Softmax attention over a sliding window of tokens and the means of the runs that have left it."""

import torch

from .. import ops
from ..config.registry import register_part
from .base import CacheNeed, PagedTensor, Part, TensorShape
from .linear import LinearWeight, joined_rows
from .position import scaled_rotation


@register_part("mixer", "pooled_window_attention")
class PooledWindowAttention(Part):
    """q = W_q h + b_q (heads x dim), k = W_k h + b_k (kv_heads x dim), v = W_v h + b_v (kv_heads x
    vdim); query head a reads key head a // (heads / kv_heads). q and k turn by the position over the
    first `rot_dims` numbers of every head, i and i + rot_dims / 2 together (`scaled_rotation`). The
    token at position i sees the keys at positions i - window < j <= i (`window` 0: all j <= i) and,
    beside them, one key and one value for every run of `pool` tokens that ends at i - window or
    before: the means of the run's keys and values as the cache holds them (`pool` 0: nothing behind
    the window). All of these share one softmax whose denominator holds exp(`sink`) more, a term
    without a key or a value, the same constant for every head. Head a's result is multiplied by
    sigmoid(W_g h)_a before the output product.

    The products are one and leave float32 rows; biases, angles, scores and the softmax are float32.
    The tokens' keys and values are paged as the matrix-core attention kernels read them, and given
    back as they leave the window and their run is complete; the means are paged per run of `pool`
    tokens (`CacheNeed.runs`) in the same layout and stay. bfloat16 with equal key and value sizes of
    64 or 128 runs on the matrix cores, everything else on a general kernel."""

    graph_safe = True
    feeds_sink = True

    def __init__(self, prefix, precision, device, hidden_size, heads, kv_heads, dim, vdim, scale, window=0, pool=0,
                 rot_dims=0, rot_base=1.0, rot_scaling=None, sink=0.0):
        super().__init__(prefix, precision, device)
        if heads % kv_heads:
            raise ValueError("heads (%d) must be a multiple of kv_heads (%d)" % (heads, kv_heads))
        if dim > 512 or vdim > 512 or rot_dims > dim or rot_dims % 2:
            raise ValueError("the attention kernels take keys and values of up to 512 numbers and an even rotation within "
                             "the keys, not %d, %d and %d" % (dim, vdim, rot_dims))
        if pool and not window:
            raise ValueError("runs are pooled behind a window: pool %d needs one" % pool)
        self.hidden_size, self.heads, self.kv_heads, self.dim, self.vdim = hidden_size, heads, kv_heads, dim, vdim
        self.scale, self.window, self.pool = float(scale), int(window), int(pool)
        self.rotation = (int(rot_dims), float(rot_base), rot_scaling)
        self.sink_value = float(sink)
        self.w_in = self.w_out = self.bias = self.inv_freq = self.sink = None
        self.rot_factor = 1.0

    def cache_need(self):
        def pair():
            return (PagedTensor("keys", (self.kv_heads, self.dim), token_axis=1),
                    PagedTensor("values", (self.kv_heads, self.vdim), token_axis=2))

        # a token stays until it is outside the window and its run's mean has been formed
        return CacheNeed(paged=pair(), window=max(self.window, self.pool), runs=pair() if self.pool else (),
                         run_length=self.pool)

    def tensors(self):
        H, G, d, dv, W = self.heads, self.kv_heads, self.dim, self.vdim, self.hidden_size
        return {self._name("q"): (H * d, W), self._name("k"): (G * d, W), self._name("v"): (G * dv, W),
                self._name("q.b"): TensorShape((H * d,), "bias"), self._name("k.b"): TensorShape((G * d,), "bias"),
                self._name("v.b"): TensorShape((G * dv,), "bias"), self._name("g"): (H, W), self._name("o"): (W, H * dv)}

    def load(self, fetch):
        act = self.precision.act
        joined = joined_rows([fetch(self._name(n), act, keep=False) for n in ("q", "k", "v", "g")])
        self.w_in = LinearWeight(joined, self.precision)
        self.w_out = LinearWeight(fetch(self._name("o"), act), self.precision)
        self.bias = torch.cat([fetch(self._name(n + ".b"), torch.float32) for n in ("q", "k", "v")]).contiguous()
        self.inv_freq, self.rot_factor = scaled_rotation(*self.rotation[:2], self.device, self.rotation[2])
        self.sink = torch.full((self.heads,), self.sink_value, dtype=torch.float32, device=self.device)

    @property
    def takes_unscaled(self):
        return self.w_in is not None and self.w_in.fuses

    def forward(self, x, batch, cache, sink=None):
        H, G, d, dv = self.heads, self.kv_heads, self.dim, self.vdim
        rows = self.w_in.forward(x, out_dtype=torch.float32)
        keys, values = cache.paged["keys"], cache.paged["values"]
        runs = (cache.runs["keys"], cache.runs["values"], cache.run_table, self.pool) if self.pool else None
        q = ops.turn_prepare(rows, self.bias, H, G, d, dv, self.inv_freq, self.rot_factor, batch.positions,
                             batch.seq_index, self.precision.act, block_table=cache.block_table, k_cache=keys,
                             v_cache=values, runs=runs, cu_seqlens_q=batch.cu_seqlens_q, kv_lens=batch.kv_lens,
                             max_q_len=batch.max_q_len)
        mixed = ops.softcap_attention(q, keys, values, cache.block_table, batch.cu_seqlens_q, batch.kv_lens,
                                      batch.seq_index, batch.positions, batch.max_q_len, batch.max_kv_len, self.scale,
                                      0.0, window=self.window, gate=rows[:, (H + G) * d + G * dv:(H + G) * d + G * dv + H],
                                      values_transposed=True, min_q_len=batch.min_q_len,
                                      max_kv_len_of_many=getattr(batch, "max_kv_len_portions", None), sink=self.sink,
                                      runs=runs)
        return self.w_out.forward(mixed) if sink is None else self.w_out.forward_into(mixed, sink)
