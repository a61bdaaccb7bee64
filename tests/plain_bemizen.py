"""The Bemizen decoder on one whole sequence with elementary tensor operations, one function per
mechanism, in the dtype of the weights it is given (float64 for a truth, float32 to see what
rounding does). It shares no code with the package: the tests compare the engine with this.

`config` is config.json as a dict, `w` maps tensor names to tensors.
"""

import torch


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def rotate_halves(x, positions, rot):
    """x (T, heads, n): the first rot.dims numbers of every head turn, i and i + dims / 2 together, by
    position * base^(-2i / dims); the rest pass."""
    dims, base = int(rot["dims"]), float(rot["base"])
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64).to(torch.float32)
    angle = positions.to(torch.float32)[:, None] * f[None, :]          # 32-bit angles, as the design forms them
    cos = angle.to(torch.float64).cos().to(x.dtype)[:, None, :]
    sin = angle.to(torch.float64).sin().to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat((u * cos - v * sin, v * cos + u * sin, x[..., dims:]), dim=-1)


def chunk_mask(T, size):
    """(T, T), true where row i sees column j: j <= i in the same chunk of `size` tokens from the sequence's first."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (torch.div(i, size, rounding_mode="floor") == torch.div(j, size, rounding_mode="floor"))


def window_mask(T, size, keep_first):
    """(T, T), true where row i sees column j: one of the last `size` tokens, or of the sequence's first `keep_first`."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def mixed_values(v, first, share):
    return (1.0 - share) * v + share * first


def softmax_attention(q, k, v, visible, scale):
    """q (T, H, d), k (T, G, d), v (T, G, dv), visible (T, T) -> (T, H, dv)."""
    shared = q.shape[1] // k.shape[1]
    k, v = k.repeat_interleave(shared, dim=1), v.repeat_interleave(shared, dim=1)
    scores = torch.einsum("thd,shd->hts", q, k) * scale
    return torch.einsum("hts,shd->thd", torch.softmax(scores.masked_fill(~visible[None], float("-inf")), dim=-1), v)


def attention(h, w, p, kind, m, eps, first_values):
    """Either attention; returns its result and its values before anything is mixed into them.
    `first_values`: those of the first layer that mixes, or None in that layer itself and in layers that
    do not mix."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos = torch.arange(T)
    q, k = (h @ w[p + ".q"].T).view(T, H, d), (h @ w[p + ".k"].T).view(T, G, d)
    own = v = (h @ w[p + ".v"].T).view(T, G, dv)
    if kind == "attention_2":                  # a weighted norm per head, before the turn
        q, k = unit_rms(q, eps) * w[p + ".q.norm"], unit_rms(k, eps) * w[p + ".k.norm"]
    if m.get("rot"):
        q, k = rotate_halves(q, pos, m["rot"]), rotate_halves(k, pos, m["rot"])
    if kind == "attention":                    # a plain one behind it
        q, k = unit_rms(q, eps), unit_rms(k, eps)
    if first_values is not None:
        v = mixed_values(v, first_values.view(T, G, dv), w[p + ".vmix"])
    mask = m.get("mask")
    if mask is None:
        visible = window_mask(T, T, 0)
    elif kind == "attention":
        visible = chunk_mask(T, int(mask["size"]))
    else:
        visible = window_mask(T, int(mask["size"]), int(mask.get("keep_first") or 0))
    o = softmax_attention(q, k, v, visible, float(m["scale"]))
    if kind == "attention_2":
        o = o * torch.sigmoid(h @ w[p + ".g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w[p + ".o"].T, own


def expert(h, w, p):
    return (silu(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def choose_experts(z, correction, top, groups, keep, scale):
    """z (T, E) router logits -> (chosen (T, top), their weights). The choice goes by softmax(z) +
    correction among the experts of the `keep` groups whose best such score is highest; the weights are
    softmax(z) of the chosen over their sum, times `scale`."""
    T, E = z.shape
    s = torch.softmax(z, dim=-1)
    grouped = (s + correction).view(T, groups, E // groups)
    kept = grouped.max(dim=-1).values.topk(keep, dim=-1).indices
    allowed = torch.zeros((T, groups), dtype=torch.bool)
    allowed[torch.arange(T)[:, None], kept] = True
    chosen = grouped.masked_fill(~allowed[:, :, None], float("-inf")).view(T, E).topk(top, dim=-1).indices
    share = s.gather(1, chosen)
    return chosen, share / (share.sum(dim=-1, keepdim=True) + 1e-20) * scale


def routed_feed_forward(h, w, p, f):
    r = f["router"]
    E, idle, top = int(r["experts"]), int(r.get("identity") or 0), int(r["top"])
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ w[p + ".router"].T
    chosen, share = choose_experts(z, w[p + ".correction"], top, int(groups["count"]), int(groups["keep"]),
                                   float(r.get("scale", 1.0)))
    out = torch.zeros_like(h)
    for e in range(E + idle):
        for k in range(top):
            rows = (chosen[:, k] == e).nonzero()[:, 0]
            if rows.numel():                   # from number E on an expert gives its input back
                out[rows] += share[rows, k, None] * (expert(h[rows], w, "%s.e%d" % (p, e)) if e < E else h[rows])
    return out


def logits_of_sequence(config, w, tokens, layers_out=None):
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)]
    first_values = None
    for i, layer in enumerate(config["layers"]):
        p, m = "l%d" % i, layer["mixer"]
        mixes = bool(m.get("v_mix"))
        h = unit_rms(x, eps) * w[p + ".norm1"]
        y, own = attention(h, w, p + ".mix", layer["type"], m, eps, first_values if mixes else None)
        if mixes and first_values is None:
            first_values = own
        x = x + y
        if layer.get("mlp"):
            h = unit_rms(x, eps) * w[p + ".norm2"]
            x = x + routed_feed_forward(h, w, p + ".mlp", layer["mlp"])
        if layers_out is not None:
            layers_out.append(x.clone())
    return (unit_rms(x, eps) * w["final.norm"]) @ w["head"].T
