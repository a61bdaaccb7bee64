"""Attention whose keys count by the sigmoid of their scores and serve as values too."""

import torch

from .. import ops
from ..config.registry import register_part
from .base import CacheNeed, PagedTensor, Part, TensorShape
from .linear import LinearWeight, joined_rows
from .position import scaled_rotation


@register_part("mixer", "sigmoid_attention")
class SigmoidAttention(Part):
    """q = W_q h + b_q (heads x dim) and k = W_k h + b_k (kv_heads x dim) pass a causal convolution per
    channel (`conv` taps, the last tap the current token's, zeros before the start, no bias, no
    activation); query head a reads key head a // (heads / kv_heads). The values are k as it leaves
    the convolution; q and k then turn by the position over the first `rot_dims` numbers of every
    head, i and i + rot_dims / 2 together (`scaled_rotation`). The token at position i sees every key
    j <= i, which counts with sigmoid((q . k) scale + pb_a), pb_a a learned number per head, without any
    normalisation over the keys. The heads side by side are multiplied element by element with
    sigmoid(W_g h) before the output product.

    The products are one and leave float32 rows; convolutions, angles, scores and weights are float32.
    Keys (turned) and values (not) are paged as the matrix-core attention kernels read them; the
    convolutions' last taps - 1 inputs are the mixer's state. bfloat16 with heads of 64 or 128 numbers
    runs on the matrix cores, everything else on a general kernel."""

    graph_safe = True
    feeds_sink = True

    def __init__(self, prefix, precision, device, hidden_size, heads, kv_heads, dim, conv, scale, rot_dims=0, rot_base=1.0,
                 rot_scaling=None):
        super().__init__(prefix, precision, device)
        if heads % kv_heads:
            raise ValueError("heads (%d) must be a multiple of kv_heads (%d)" % (heads, kv_heads))
        if dim > 512 or rot_dims > dim or rot_dims % 2 or not 1 <= conv <= 8:
            raise ValueError("the kernels take keys of up to 512 numbers, an even rotation within them and 1 to 8 taps, "
                             "not %d, %d and %d" % (dim, rot_dims, conv))
        self.hidden_size, self.heads, self.kv_heads, self.dim = hidden_size, heads, kv_heads, dim
        self.taps, self.scale = int(conv), float(scale)
        self.rotation = (int(rot_dims), float(rot_base), rot_scaling)
        self.channels = (heads + kv_heads) * dim
        self.w_in = self.w_out = self.bias = self.conv = self.no_bias = self.score_bias = self.inv_freq = None
        self.rot_factor = 1.0

    def cache_need(self):
        tail = (self.taps - 1) * self.channels
        return CacheNeed(paged=(PagedTensor("keys", (self.kv_heads, self.dim), token_axis=1),
                                PagedTensor("values", (self.kv_heads, self.dim), token_axis=2)),
                         state_shape=(tail,) if tail else (), state_dtype=torch.float32)

    def tensors(self):
        H, G, d, W = self.heads, self.kv_heads, self.dim, self.hidden_size
        return {self._name("q"): (H * d, W), self._name("k"): (G * d, W),
                self._name("q.b"): TensorShape((H * d,), "bias"), self._name("k.b"): TensorShape((G * d,), "bias"),
                self._name("q.conv"): (H * d, self.taps), self._name("k.conv"): (G * d, self.taps),
                self._name("pb"): TensorShape((H,), "bias"), self._name("g"): (H * d, W), self._name("o"): (W, H * d)}

    def load(self, fetch):
        act = self.precision.act
        joined = joined_rows([fetch(self._name(n), act, keep=False) for n in ("q", "k", "g")])
        self.w_in = LinearWeight(joined, self.precision)
        self.w_out = LinearWeight(fetch(self._name("o"), act), self.precision)
        self.bias = torch.cat([fetch(self._name(n + ".b"), torch.float32) for n in ("q", "k")]).contiguous()
        self.conv = torch.cat([fetch(self._name(n + ".conv"), torch.float32) for n in ("q", "k")], dim=0).contiguous()
        self.no_bias = torch.zeros(self.channels, dtype=torch.float32, device=self.device)
        self.score_bias = fetch(self._name("pb"), torch.float32).contiguous()
        self.inv_freq, self.rot_factor = scaled_rotation(*self.rotation[:2], self.device, self.rotation[2])

    @property
    def takes_unscaled(self):
        return self.w_in is not None and self.w_in.fuses

    def forward(self, x, batch, cache, sink=None):
        H, G, d, C = self.heads, self.kv_heads, self.dim, self.channels
        rows = self.w_in.forward(x, out_dtype=torch.float32)
        state = cache.state
        if state is None:                      # one tap: nothing to carry, in as many slots as there may be
            state = torch.empty((1 << 20, 0), dtype=torch.float32, device=rows.device)
        qk = ops.causal_conv(rows[:, :C], self.conv, self.no_bias, state, batch.state_slots, batch.cu_seqlens_q,
                             batch.seq_index, out_dtype=torch.float32, in_bias=self.bias, max_q_len=batch.max_q_len)
        keys, values = cache.paged["keys"], cache.paged["values"]
        q = ops.turn_prepare(qk, None, H, G, d, d, self.inv_freq, self.rot_factor, batch.positions, batch.seq_index,
                             self.precision.act, block_table=cache.block_table, k_cache=keys, v_cache=values,
                             values_are_keys=True)
        mixed = ops.softcap_attention(q, keys, values, cache.block_table, batch.cu_seqlens_q, batch.kv_lens,
                                      batch.seq_index, batch.positions, batch.max_q_len, batch.max_kv_len, self.scale,
                                      0.0, gate=rows[:, C:C + H * d], values_transposed=True, min_q_len=batch.min_q_len,
                                      max_kv_len_of_many=getattr(batch, "max_kv_len_portions", None),
                                      sigmoid_bias=self.score_bias)
        return self.w_out.forward(mixed) if sink is None else self.w_out.forward_into(mixed, sink)
