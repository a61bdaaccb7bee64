"""The Zedotar decoder on one whole sequence with elementary tensor operations, one function per
mechanism, in the dtype of the weights it is given (float64 for a truth, float32 to see what
rounding does). It shares no code with the package: the tests compare the engine with this.

`config` is config.json as a dict, `w` maps tensor names to tensors.
"""

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x, weight, eps):
    """The stored weight is what the multiplier has beyond one."""
    return rms(x, eps) * (1.0 + weight)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def turning_frequencies(rot):
    """rot -> (list of dims / 2 frequencies, factor on cos and sin). Without `scaling` the plain
    geometric row; a scaling with `low` and `high` stretches slow turns and leaves fast ones; one
    with `fast` and `slow` goes by the pair's number and multiplies cos and sin too."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return f, 1.0
    factor, original = float(s["factor"]), float(s["original"])
    if "low" in s:
        low, high = float(s["low"]), float(s["high"])
        out = []
        for x in f:
            length = 2.0 * math.pi / x
            if length < original / high:
                out.append(x)
            elif length > original / low:
                out.append(x / factor)
            else:
                share = (original / length - low) / (high - low)
                out.append((1.0 - share) * x / factor + share * x)
        return out, 1.0

    def where(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(where(float(s["fast"]))), 0)
    hi = min(math.ceil(where(float(s["slow"]))), dims - 1)
    out = []
    for i, x in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / factor * ramp + x * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_half(x, positions, rot):
    """x (T, heads, n): of the first rot.dims numbers of every head, i and i + dims / 2 turn together."""
    freqs, factor = turning_frequencies(rot)
    dims = int(rot["dims"])
    f = torch.tensor(freqs, dtype=torch.float64).to(torch.float32)
    angle = (positions.to(torch.float32)[:, None] * f[None, :]).to(torch.float64)     # 32-bit angles, as the design forms them
    cos = (angle.cos() * factor).to(x.dtype)[:, None, :]
    sin = (angle.sin() * factor).to(x.dtype)[:, None, :]
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return torch.cat((u * cos - v * sin, v * cos + u * sin, x[..., dims:]), dim=-1)


def short_convolution(u, weight):
    """u (T, channels), weight (channels, taps): y_t = sum_j w_j u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], weight.shape[1]
    padded = torch.cat((torch.zeros((taps - 1, u.shape[1]), dtype=u.dtype), u), dim=0)
    return sum(padded[j:j + T] * weight[:, j] for j in range(taps))


def pooled_window_attention(q, k, v, scale, size, pool):
    """q (T, H, d), k (T, H, d), v (T, H, dv), per query head already. Position i sees the `size` last
    tokens and, as one key and value each (the means), every run of `pool` tokens that ends at
    i - size or before; one more 1 in the softmax's denominator. `size` 0: every token, no means."""
    T = q.shape[0]
    out = torch.zeros((T, q.shape[1], v.shape[2]), dtype=q.dtype)
    for i in range(T):
        lo = max(0, i - size + 1) if size else 0
        keys, values = k[lo:i + 1], v[lo:i + 1]
        runs = max(0, i - size + 1) // pool if size and pool else 0
        if runs:
            mk = k[:runs * pool].reshape((runs, pool) + k.shape[1:]).mean(dim=1)
            mv = v[:runs * pool].reshape((runs, pool) + v.shape[1:]).mean(dim=1)
            keys, values = torch.cat((mk, keys)), torch.cat((mv, values))
        s = torch.einsum("hd,shd->hs", q[i], keys) * scale
        top = torch.clamp(s.max(dim=-1, keepdim=True).values, min=0.0)
        e = torch.exp(s - top)
        p = e / (torch.exp(-top) + e.sum(dim=-1, keepdim=True))
        out[i] = torch.einsum("hs,shd->hd", p, values)
    return out


def attention(h, w, p, m):
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos = torch.arange(T)
    q = (h @ w[p + ".q"].T + w[p + ".q.b"]).view(T, H, d)
    k = (h @ w[p + ".k"].T + w[p + ".k.b"]).view(T, G, d)
    v = (h @ w[p + ".v"].T + w[p + ".v.b"]).view(T, G, dv)
    if m.get("rot"):
        q, k = rotate_half(q, pos, m["rot"]), rotate_half(k, pos, m["rot"])
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    mask = m.get("mask") or {}
    o = pooled_window_attention(q, k, v, float(m["scale"]), int(mask.get("size", 0)), int(mask.get("pool", 0)))
    o = o * torch.sigmoid(h @ w[p + ".g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w[p + ".o"].T


def sigmoid_attention(q, k, v, scale, pb):
    """Every visible key j <= i counts with sigmoid(score + pb_head); nothing is normalised."""
    T = q.shape[0]
    weight = torch.sigmoid(torch.einsum("thd,shd->hts", q, k) * scale + pb[:, None, None])
    weight = weight.masked_fill(torch.arange(T)[None, None, :] > torch.arange(T)[None, :, None], 0.0)
    return torch.einsum("hts,shd->thd", weight, v)


def attention_2(h, w, p, m):
    """The values are the keys before they turn."""
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    pos = torch.arange(T)
    q = short_convolution(h @ w[p + ".q"].T + w[p + ".q.b"], w[p + ".q.conv"]).view(T, H, d)
    k = short_convolution(h @ w[p + ".k"].T + w[p + ".k.b"], w[p + ".k.conv"]).view(T, G, d)
    v = k
    if m.get("rot"):
        q, k = rotate_half(q, pos, m["rot"]), rotate_half(k, pos, m["rot"])
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    o = sigmoid_attention(q, k, v, float(m["scale"]), w[p + ".pb"]).reshape(T, H * d)
    return (o * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def mlstm_recurrence(q, k, v, i_gate, f_gate):
    """q, k (T, H, d), v (T, H, dv), i_gate and f_gate (T, H), the gates' logarithms. Token by token:
    the maximum m starts at 0, the matrix and its normaliser at nothing."""
    T, H, d = q.shape
    S = torch.zeros((H, d, v.shape[2]), dtype=q.dtype)
    n = torch.zeros((H, d), dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for t in range(T):
        new = torch.maximum(f_gate[t] + m, i_gate[t])
        keep, enter = torch.exp(f_gate[t] + m - new), torch.exp(i_gate[t] - new)
        S = keep[:, None, None] * S + enter[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + enter[:, None] * k[t]
        m = new
        below = torch.maximum((n * q[t]).sum(dim=-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = torch.einsum("hdv,hd->hv", S, q[t]) / below[:, None]
    return out


def mlstm(h, w, p, m, eps):
    T = h.shape[0]
    H, d, dv, cap = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"])
    q = (h @ w[p + ".q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + ".k"].T).view(T, H, d)
    v = (h @ w[p + ".v"].T).view(T, H, dv)
    i_gate = cap * torch.tanh((h @ w[p + ".i"].T + w[p + ".i.b"]) / cap)
    f_gate = torch.nn.functional.logsigmoid(cap * torch.tanh((h @ w[p + ".f"].T + w[p + ".f.b"]) / cap))
    o = rms(mlstm_recurrence(q, k, v, i_gate, f_gate), eps).reshape(T, H * dv) * w[p + ".norm"]
    return (o * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def gated_unit(h, w, p):
    return (gelu_tanh(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def logits_of_sequence(config, w, tokens, layers_out=None):
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)]
    for i, layer in enumerate(config["layers"]):
        p = "l%d" % i
        h = norm(x, w[p + ".norm1"], eps)
        if layer["type"] == "attention":
            x = x + attention(h, w, p + ".mix", layer["mixer"])
        elif layer["type"] == "attention_2":
            x = x + attention_2(h, w, p + ".mix", layer["mixer"])
        else:
            assert layer["type"] == "mlstm"
            x = x + mlstm(h, w, p + ".mix", layer["mixer"], eps)
        if layer.get("mlp"):
            assert layer["mlp"]["kind"] == "dense"
            x = x + gated_unit(norm(x, w[p + ".norm2"], eps), w, p + ".mlp")
        if layers_out is not None:
            layers_out.append(x.clone())
    logits = norm(x, w["final.norm"], eps) @ w["head"].T
    cap = config.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits
