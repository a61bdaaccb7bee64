"""The matrix memory of xLSTM (Beck et al., "xLSTM: Extended Long Short-Term Memory")."""

import torch

from .. import ops
from ..config.registry import register_part
from .base import CacheNeed, Part, TensorShape
from .linear import LinearWeight, joined_rows


@register_part("mixer", "mlstm")
class MatrixMemory(Part):
    """q = W_q h dim^(-1/2) and k = W_k h (heads x dim), v = W_v h (heads x vdim). Per head two gates'
    logarithms, i = cap tanh((W_i h + b_i) / cap) and f = logsigmoid(cap tanh((W_f h + b_f) / cap)),
    cap = `gate_cap`; with a running maximum m that starts at 0, a matrix S (dim x vdim) and a vector n
    (dim) that start at zero,

        m' = max(f + m, i);   S <- exp(f + m - m') S + exp(i - m') k v^T;   n <- the same with k alone;
        o = S^T q / (max(|n . q|, exp(-m')) + denominator_eps).

    Each head's o is divided by its root mean square (eps inside the root); the heads side by side are
    multiplied by `norm` and by sigmoid(W_g h) and go through the output product. The products are one
    and leave float32 rows; everything behind them is float32. Per request the mixer keeps S, n and m
    (see `ops.mlstm_state_numbers`)."""

    graph_safe = True
    feeds_sink = True

    def __init__(self, prefix, precision, device, hidden_size, heads, dim, vdim, gate_cap, eps, denominator_eps=1e-6):
        super().__init__(prefix, precision, device)
        if dim > 512:
            raise ValueError("the matrix memory's kernels take keys of up to 512 numbers, not %d" % dim)
        self.hidden_size, self.heads, self.dim, self.vdim = hidden_size, heads, dim, vdim
        self.gate_cap, self.eps, self.denominator_eps = float(gate_cap), float(eps), float(denominator_eps)
        self.w_in = self.w_out = self.i_bias = self.f_bias = self.norm = None

    def cache_need(self):
        return CacheNeed(state_shape=(ops.mlstm_state_numbers(self.heads, self.dim, self.vdim),),
                         state_dtype=torch.float32)

    def tensors(self):
        H, d, dv, W = self.heads, self.dim, self.vdim, self.hidden_size
        return {self._name("q"): (H * d, W), self._name("k"): (H * d, W), self._name("v"): (H * dv, W),
                self._name("g"): (H * dv, W), self._name("o"): (W, H * dv),
                self._name("norm"): TensorShape((H * dv,), "scale"),
                self._name("i"): (H, W), self._name("i.b"): TensorShape((H,), "bias"),
                self._name("f"): (H, W), self._name("f.b"): TensorShape((H,), "bias")}

    def load(self, fetch):
        act = self.precision.act
        joined = joined_rows([fetch(self._name(n), act, keep=False) for n in ("q", "k", "v", "g", "i", "f")])
        self.w_in = LinearWeight(joined, self.precision)
        self.w_out = LinearWeight(fetch(self._name("o"), act), self.precision)
        self.i_bias = fetch(self._name("i.b"), torch.float32).contiguous()
        self.f_bias = fetch(self._name("f.b"), torch.float32).contiguous()
        self.norm = fetch(self._name("norm"), torch.float32).contiguous()

    @property
    def takes_unscaled(self):
        return self.w_in is not None and self.w_in.fuses

    def forward(self, x, batch, cache, sink=None):
        mixed = ops.mlstm_scan(self.w_in.forward(x, out_dtype=torch.float32), self.heads, self.dim, self.vdim,
                               self.gate_cap, self.i_bias, self.f_bias, self.norm, self.eps, self.denominator_eps,
                               cache.state, batch.state_slots, batch.cu_seqlens_q, self.precision.act,
                               max_q_len=batch.max_q_len)
        return self.w_out.forward(mixed) if sink is None else self.w_out.forward_into(mixed, sink)
