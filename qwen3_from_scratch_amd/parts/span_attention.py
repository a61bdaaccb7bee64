"""Softmax attention over a span of the tokens before (a chunk of the sequence, or a sliding window and
the sequence's first tokens), with a norm per head on queries and keys and values that may mix with an
earlier layer's."""

import torch

from .. import ops
from ..config.registry import register_part
from .base import CacheNeed, PagedTensor, Part, TensorShape
from .linear import LinearWeight, joined_rows
from .position import rotation_frequencies

FIRST_VALUES = "first values"       # what the first of the layers that mix values leaves for the others in a step


@register_part("mixer", "span_attention")
class SpanAttention(Part):
    """q = W_q h (heads x dim), k = W_k h (kv_heads x dim), v = W_v h (kv_heads x vdim), no biases; query
    head a reads key head a // (heads / kv_heads). `qk_norm` "weighted": every head of q and of k is
    divided by its own root mean square (eps inside the root) and multiplied by a weight of dim numbers
    that the heads share (`q.norm`, `k.norm`), then both turn by the position over the first `rot_dims`
    numbers, i and i + rot_dims / 2 together, by position * rot_base^(-2i / rot_dims); "plain": they turn
    and are then divided by the root mean square, which a rotation leaves as it was, so that the kernel
    takes it before the turn in either case; None: no norm.

    The token at position i sees the keys at j <= i with i // chunk == j // chunk (`chunk` > 0), or with
    i - j < window or j < keep_first (`window` > 0), or all of them (neither). score = (q . k) scale,
    ordinary softmax. `values` "own": v as it is; "first": as it is, and left to the later layers of the
    step; "mixed": (1 - s) v + s v_first with the step's v_first and the layer's own share s (`vmix`); what
    is mixed is what is cached. `gated`: head a's result is multiplied by sigmoid(W_g h)_a (`g`) before
    the output product.

    The products are one and leave float32 rows; norms, angles, scores, softmax, mixing and gates are
    float32. Keys and values are paged as the matrix-core attention kernels read them; a page goes back when
    no later token sees any of its keys, a page of first tokens never while the request lives. bfloat16
    with the sizes of `ops.span_sizes` runs on the matrix cores, everything else on a general kernel."""

    graph_safe = True
    feeds_sink = True

    def __init__(self, prefix, precision, device, hidden_size, heads, kv_heads, dim, vdim, scale, eps, qk_norm=None, chunk=0,
                 window=0, keep_first=0, rot_dims=0, rot_base=1.0, values="own", gated=False):
        super().__init__(prefix, precision, device)
        if heads % kv_heads:
            raise ValueError("heads (%d) must be a multiple of kv_heads (%d)" % (heads, kv_heads))
        if dim > 512 or vdim > 512 or rot_dims > dim or rot_dims % 2:
            raise ValueError("the attention kernels take keys and values of up to 512 numbers and an even rotation within "
                             "the keys, not %d, %d and %d" % (dim, vdim, rot_dims))
        if qk_norm not in (None, "weighted", "plain") or values not in ("own", "first", "mixed"):
            raise ValueError("qk_norm is None, 'weighted' or 'plain', values 'own', 'first' or 'mixed'; not %r and %r"
                             % (qk_norm, values))
        self.need = CacheNeed(paged=(PagedTensor("keys", (kv_heads, dim), token_axis=1),
                                     PagedTensor("values", (kv_heads, vdim), token_axis=2)),
                              window=int(window), chunk=int(chunk), keep_first=int(keep_first))
        self.hidden_size, self.heads, self.kv_heads, self.dim, self.vdim = hidden_size, heads, kv_heads, dim, vdim
        self.scale, self.eps, self.qk_norm = float(scale), float(eps), qk_norm
        self.chunk, self.window, self.keep_first = int(chunk), int(window), int(keep_first)
        self.rot_dims, self.rot_base = int(rot_dims), float(rot_base)
        self.values, self.gated = values, bool(gated)
        self.w_in = self.w_out = self.q_norm = self.k_norm = self.share = self.inv_freq = None

    def cache_need(self):
        return self.need

    def tensors(self):
        H, G, d, dv, W = self.heads, self.kv_heads, self.dim, self.vdim, self.hidden_size
        names = {self._name("q"): (H * d, W), self._name("k"): (G * d, W), self._name("v"): (G * dv, W),
                 self._name("o"): (W, H * dv)}
        if self.qk_norm == "weighted":
            names.update({self._name("q.norm"): TensorShape((d,), "scale"), self._name("k.norm"): TensorShape((d,), "scale")})
        if self.values == "mixed":
            names[self._name("vmix")] = TensorShape((), "bias")
        if self.gated:
            names[self._name("g")] = (H, W)
        return names

    def load(self, fetch):
        act = self.precision.act
        joined = joined_rows([fetch(self._name(n), act, keep=False) for n in (("q", "k", "v", "g") if self.gated else "qkv")])
        self.w_in = LinearWeight(joined, self.precision)
        self.w_out = LinearWeight(fetch(self._name("o"), act), self.precision)
        if self.qk_norm == "weighted":
            self.q_norm = fetch(self._name("q.norm"), torch.float32)
            self.k_norm = fetch(self._name("k.norm"), torch.float32)
        if self.values == "mixed":
            self.share = fetch(self._name("vmix"), torch.float32).reshape(1)
        self.inv_freq = rotation_frequencies(self.rot_dims, self.rot_base, self.device)

    @property
    def takes_unscaled(self):
        return self.w_in is not None and self.w_in.fuses

    def forward(self, x, batch, cache, sink=None):
        H, G, d, dv = self.heads, self.kv_heads, self.dim, self.vdim
        at = (H + G) * d
        rows = self.w_in.forward(x, out_dtype=torch.float32)
        if self.values == "first":
            batch.carried[FIRST_VALUES] = rows[:, at:at + G * dv]
        mix = (batch.carried[FIRST_VALUES], self.share) if self.values == "mixed" else None
        keys, values = cache.paged["keys"], cache.paged["values"]
        q = ops.turn_prepare(rows, None, H, G, d, dv, self.inv_freq, 1.0, batch.positions, batch.seq_index,
                             self.precision.act, block_table=cache.block_table, k_cache=keys, v_cache=values,
                             norm_eps=self.eps if self.qk_norm else None, q_weight=self.q_norm, k_weight=self.k_norm, mix=mix)
        mixed = ops.softcap_attention(q, keys, values, cache.block_table, batch.cu_seqlens_q, batch.kv_lens,
                                      batch.seq_index, batch.positions, batch.max_q_len, batch.max_kv_len, self.scale, 0.0,
                                      window=self.window, gate=rows[:, at + G * dv:at + G * dv + H] if self.gated else None,
                                      values_transposed=True, min_q_len=batch.min_q_len,
                                      max_kv_len_of_many=getattr(batch, "max_kv_len_portions", None), chunk=self.chunk,
                                      keep_first=self.keep_first, span=True)
        return self.w_out.forward(mixed) if sink is None else self.w_out.forward_into(mixed, sink)
