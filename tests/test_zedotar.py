"""The Zedotar architecture through the engine against tests/plain_zedotar.py: each mechanism alone,
whole prompts against token-by-token decoding, portions down to two tokens, mixed batches with pages and
slots that are used again, keys and runs at the edges of windows and pages, the first tokens, long
decoding, and greedy generation through the engine. The configurations are made here; their sizes differ
from layer to layer and avoid values that hide a fault (equal key and value sizes, runs that divide a
page or the window, a rotation over the whole head, a head per key head); where a design's random weights
would forget or drown a far token, the weights are made so that it counts."""

import copy
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import load_file, save_file

import plain_zedotar as plain
from helpers import max_live_tokens, random_tokens, run_trace, trace_mixed, trace_portions, trace_tail_decoded, trace_whole
from qwen3_from_scratch_amd.cache import CacheManager, OutOfPages
from qwen3_from_scratch_amd.config import load_model_config
from qwen3_from_scratch_amd.config.model_config import ConfigError
from qwen3_from_scratch_amd.config.zedotar_config import ZedotarConfig
from qwen3_from_scratch_amd.engine import StepEntry, SyncEngine, load_runner
from qwen3_from_scratch_amd.parts import CacheNeed, PagedTensor
from qwen3_from_scratch_amd.weights import write_random_model

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _bands(factor=8.0, original=40, low=1.0, high=4.0):
    return {"factor": factor, "original": original, "low": low, "high": high}


def _ramp(factor=4.0, original=64, fast=8.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def _rot(dims, base=500.0, scaling=None):
    r = {"dims": dims, "base": base}
    if scaling:
        r["scaling"] = scaling
    return r


def _attention(heads, kv_heads, dim, vdim, size=0, pool=0, rot=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or 1.0 / math.sqrt(dim)}
    if size:
        m["mask"] = {"size": size, "pool": pool} if pool else {"size": size}
    if rot:
        m["rot"] = rot
    return {"type": "attention", "mixer": m}


def _sigmoid(heads, kv_heads, dim, conv, rot=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "conv": conv, "scale": scale or 1.0 / math.sqrt(dim)}
    if rot:
        m["rot"] = rot
    return {"type": "attention_2", "mixer": m}


def _mlstm(heads, dim, vdim, cap=15.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def _layer(mixer, ff):
    return dict(mixer, mlp={"kind": "dense", "ff": ff} if ff else None)


def _model(vocab, width, layers, eps=1e-5, cap=None):
    data = {"architecture": "Zedotar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if cap:
        data["logit_softcap"] = cap
    return data


# runs that divide neither the pages nor the window, a run longer than its window, both scalings on both mixers,
# a layer without a feed-forward
MIXED = _model(131, 48, [
    _layer(_attention(4, 2, 16, 24, size=20, pool=6, rot=_rot(8, scaling=_bands())), 56),
    _layer(_sigmoid(6, 2, 12, 3, rot=_rot(8, 300.0, _ramp())), 40),
    _layer(_mlstm(3, 8, 12, cap=5.0), None),
    _layer(_attention(6, 2, 8, 16, size=7, pool=12, rot=_rot(6, 2000.0, _ramp(original=32))), 24),
    _layer(_sigmoid(3, 3, 20, 2, rot=_rot(20, scaling=_bands(original=100))), None),
], cap=9.0)
# sizes that the matrix-core kernels take
CORES = _model(257, 128, [
    _layer(_sigmoid(8, 2, 64, 4, rot=_rot(32, 20000.0, _ramp(original=128))), 192),
    _layer(_attention(4, 1, 64, 64, size=50, pool=8, rot=_rot(64, 10000.0, _bands(original=256))), 160),
    _layer(_mlstm(2, 80, 144), 128),
    _layer(_attention(8, 4, 128, 128, size=40, pool=20, rot=_rot(32, 30000.0)), None),
    _layer(_sigmoid(2, 2, 128, 1), 64),
], eps=1e-6, cap=25.0)
# sizes that no vector access and no matrix instruction takes; one head, one tap, runs of one token, a window
# without runs, no window, no rotation, no cap on the logits
ODD = _model(53, 40, [
    _layer(_attention(3, 1, 10, 14, size=9, pool=1, rot=_rot(4)), 18),
    _layer(_mlstm(1, 5, 70, cap=2.0), 22),
    _layer(_sigmoid(1, 1, 6, 1), None),
    _layer(_attention(2, 2, 6, 10, size=5), 10),
    _layer(_attention(1, 1, 7, 3), 14),
    _layer(_mlstm(7, 3, 2, cap=30.0), None),
])
# the matrix memory alone, over several tiles of columns and slices of rows
MEMORY = _model(97, 64, [_layer(_mlstm(2, 130, 150, cap=8.0), 96), _layer(_mlstm(4, 16, 64), 48)], cap=12.0)
CONFIGS = {"mixed": MIXED, "cores": CORES, "odd": ODD, "memory": MEMORY}
# in bfloat16 heads of two or three numbers, whose root mean square is divided out, move by more than any bound
# on rounding; the same layers with more numbers in them
ROUNDED = {"odd": dict(ODD, layers=[
    _layer(_attention(3, 1, 10, 14, size=9, pool=1, rot=_rot(4)), 18), _layer(_mlstm(1, 13, 70, cap=2.0), 22),
    _layer(_sigmoid(1, 1, 26, 1), None), _layer(_attention(2, 2, 6, 30, size=5), 10), _layer(_attention(1, 1, 7, 23), 14)])}


def _write(folder, data, seed=5, std=0.2, keep=3.0, apart=2.0):
    """Random weights, with gates that keep the memory for some tens of tokens (`keep` on the forget gates'
    biases) and sigmoid weights that are small for most keys (`apart` off their biases)."""
    write_random_model(str(folder), ZedotarConfig.from_dict(data), seed=seed, std=std, norm_jitter=0.3)
    path = os.path.join(str(folder), "model.safetensors")
    tensors = load_file(path)
    for key in tensors:
        if key.endswith("mix.f.b"):
            tensors[key] = (tensors[key].float() + keep).to(tensors[key].dtype)
        if key.endswith("mix.pb"):
            tensors[key] = (tensors[key].float() - apart).to(tensors[key].dtype)
    save_file(tensors, path, metadata={"format": "pt"})
    return str(folder)


@pytest.fixture(scope="module", params=sorted(CONFIGS))
def folder(request, tmp_path_factory):
    return _write(tmp_path_factory.mktemp(request.param), CONFIGS[request.param])


@pytest.fixture(scope="module", params=sorted(CONFIGS))
def folders(request, tmp_path_factory):
    """{dtype: folder}: for bfloat16 smaller weights, and sigmoid weights that are small for all but a few keys (sums
    that hundreds of keys enter undivided make every later rounding count), so that rounding alone stays well
    inside the bound."""
    return {"float32": _write(tmp_path_factory.mktemp(request.param), CONFIGS[request.param]),
            "bfloat16": _write(tmp_path_factory.mktemp(request.param + "_bf16"), ROUNDED.get(request.param, CONFIGS[request.param]),
                               std=0.05, apart=4.0)}


def _truth(folder, requests, dtype=torch.float64):
    with open(os.path.join(folder, "config.json")) as fh:
        config = json.load(fh)
    w = {k: v.to(dtype) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return config, w, {rid: plain.logits_of_sequence(config, w, toks) for rid, toks in requests.items()}


def _requests(folder, lengths=(70, 9, 41, 130, 25, 2, 1)):
    vocab = load_model_config(folder).vocab
    return {"z%d" % i: random_tokens(n, vocab, 460 + i) for i, n in enumerate(lengths)}


def _off(got, want, dtype):
    """The worst row: its difference (mean taken off, root mean square) over the spread of the true
    row, in units of what the dtype may be off by."""
    worst = 0.0
    for rid, logits in want.items():
        for p in range(logits.shape[0]):
            d = got[(rid, p)].double() - logits[p].double()
            err = float((d - d.mean()).pow(2).mean().sqrt() / logits[p].double().std())
            worst = max(worst, err / (5e-5 if dtype == "float32" else 5e-2))
    return worst


# ---- configuration, weights, cache planes ----

def test_config_is_read_by_its_own_keys_and_written_back(folder):
    config = load_model_config(folder)
    assert isinstance(config, ZedotarConfig) and config.architecture == "Zedotar"
    with open(os.path.join(folder, "config.json")) as fh:
        raw = json.load(fh)
    assert config.to_dict() == raw and len(config.layers) == len(raw["layers"])
    assert config.logit_softcap == raw.get("logit_softcap", 0.0)
    names = set(load_file(os.path.join(folder, "model.safetensors")))
    assert {"embed", "head", "final.norm", "l0.norm1"} <= names
    for i, (layer, entry) in enumerate(zip(config.layers, raw["layers"])):
        p, m = "l%d." % i, entry["mixer"]
        assert layer.type == entry["type"] and (layer.ff == 0) == (entry["mlp"] is None)
        assert (p + "norm2" in names) == (entry["mlp"] is not None)
        if entry["type"] == "attention":
            assert {p + "mix.q.b", p + "mix.v.b", p + "mix.g", p + "mix.o"} <= names and p + "mix.q.norm" not in names
            assert (layer.mixer.window, layer.mixer.pool) == (m.get("mask", {}).get("size", 0), m.get("mask", {}).get("pool", 0))
        elif entry["type"] == "attention_2":
            assert {p + "mix.q.b", p + "mix.k.conv", p + "mix.pb", p + "mix.g"} <= names and p + "mix.v" not in names
        else:
            assert {p + "mix.i.b", p + "mix.f", p + "mix.norm"} <= names and p + "mix.q.b" not in names
        if entry["type"] != "mlstm" and m.get("rot", {}).get("scaling"):
            kind = "bands" if "low" in m["rot"]["scaling"] else "ramp"
            assert layer.mixer.rot.scaling[0] == kind


@pytest.mark.parametrize("change,word", [
    (lambda c: c["layers"][0].update(type="other"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_heads"), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "divide"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(pool=-1), "pool"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "head's size"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("low"), "low"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0.0), "positive"),
    (lambda c: c["layers"][1]["mixer"].pop("conv"), "conv"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=5), "vdim"),
    (lambda c: c["layers"][2]["mixer"].update(gate_cap=0.0), "gate_cap"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c.update(logit_softcap=-1.0), "logit_softcap"),
    (lambda c: c.pop("width"), "width"),
])
def test_config_errors_name_the_key(change, word):
    data = copy.deepcopy(MIXED)
    change(data)
    with pytest.raises(ConfigError, match=word):
        ZedotarConfig.from_dict(data)


def test_runs_are_paged_apart_from_tokens():
    """Tokens in windowed pages that go back, runs in pages of their own that stay, one table each."""
    pair = (PagedTensor("keys", (2, 4), 1), PagedTensor("values", (2, 6), 2))
    need = CacheNeed(paged=pair, window=6, runs=pair, run_length=6)
    m = CacheManager([need, CacheNeed(paged=pair), need], page_size=4, num_pages=30, max_requests=2)
    assert [(g.window, g.every, g.planes) for g in m.groups] == [(6, 1, [0, 2]), (0, 6, [0, 2]), (0, 1, [1])]
    assert m.groups[1].pool.num_pages == 5 + 2                     # ceil(30 / 6) and one more a request
    assert m.group_of_plane == [0, 2, 0] and m.run_group_of_plane == [1, -1, 1]
    m.admit("a")
    m.reserve("a", 23)
    assert len(m.block_table("a", 0)) == 6 and len(m.block_table("a", 1)) == 1        # three complete runs
    m.commit("a", 23)
    assert m.block_table("a", 0)[:5] == [-1] * 4 + [m.block_table("a", 0)[4]]        # token 18 starts the open run
    assert m.block_table("a", 0)[4] >= 0
    m.reserve("a", 1)
    m.commit("a", 1)
    assert len(m.block_table("a", 1)) == 1                          # a fourth run fills the page
    m.reserve("a", 6)
    assert len(m.block_table("a", 1)) == 2 and m.table_width(1, 30) == 2 and m.table_width(0, 30) == 8
    m.commit("a", 6)
    m.audit()
    assert m.capacity_tokens() == 30 * 4
    m.admit("b")
    with pytest.raises(OutOfPages):
        m.reserve("b", 120)
    m.release("a")
    m.reserve("b", 120)
    m.commit("b", 120)
    m.release("b")
    m.audit()
    assert all(g.pool.num_free == g.pool.num_pages for g in m.groups)
    assert not CacheManager([need], 4, 8, 1, prefix_cache=True).prefix_cache
    with pytest.raises(ValueError, match="run_length"):
        CacheNeed(runs=pair)
    assert need.bytes_per_token(torch.bfloat16) == 2 * (8 + 12) + math.ceil(2 * (8 + 12) / 6)


def test_cache_planes_of_the_model(cpu_ops, tmp_path):
    folder = _write(tmp_path / "m", MIXED)
    runner = load_runner(folder, dtype="float32", device="cpu", page_size=8, max_tokens=256, max_requests=4)
    groups = {(g.window, g.every, tuple(t.shape for t in g.tensors)) for g in runner.manager.groups}
    assert groups == {(20, 1, ((2, 16), (2, 24))), (0, 6, ((2, 16), (2, 24))), (0, 1, ((2, 12), (2, 12))),
                      (12, 1, ((2, 8), (2, 16))), (0, 12, ((2, 8), (2, 16))), (0, 1, ((3, 20), (3, 20)))}
    states = {g.shape for g in runner.manager.state_groups}
    assert states == {(2 * (6 + 2) * 12,), (3 * (8 * 12 + 8 + 1),), (1 * 6 * 20,)}


# ---- each mechanism alone, on the host twins and against the plain functions ----

@pytest.mark.parametrize("rot", [_rot(8), _rot(12, 700.0, _bands()), _rot(64, 10000.0, _bands(original=300)),
                                 _rot(16, 900.0, _ramp()), _rot(64, 200000.0, _ramp(original=3000, fast=24.0)),
                                 _rot(4, 50.0, _ramp(original=7, fast=2.0, slow=2.0))])
def test_scaled_frequencies(rot):
    from qwen3_from_scratch_amd.parts.position import scaled_rotation

    s = rot.get("scaling")
    kind = None if s is None else (("bands", s["factor"], s["original"], s["low"], s["high"]) if "low" in s
                                   else ("ramp", s["factor"], s["original"], s["fast"], s["slow"]))
    got, factor = scaled_rotation(rot["dims"], rot["base"], "cpu", kind)
    want, by = plain.turning_frequencies(rot)
    assert torch.allclose(got.double(), torch.tensor(want, dtype=torch.float64), rtol=1e-7) and abs(factor - by) < 1e-12
    if s is not None and "low" in s:                  # fast turns stay, slow ones are divided, some lie between
        plain_row, _ = plain.turning_frequencies(dict(rot, scaling=None))
        ratio = [a / b for a, b in zip(want, plain_row)]
        assert ratio[0] == 1.0 and abs(ratio[-1] - 1.0 / s["factor"]) < 1e-12


def test_norm_weight_is_stored_around_zero(cpu_ops):
    from qwen3_from_scratch_amd.parts.base import PartSpec, Precision, build_part

    norm = build_part(PartSpec.of("norm", "rms", size=6, eps=1e-5, leaf="", offset=1.0), "n", Precision.named("float32"), "cpu")
    stored = torch.tensor([0.004, -0.5, 0.25, 1.0, -1.0, 0.0]).to(torch.bfloat16)
    norm.load(lambda name, dtype=None, keep=True: stored if dtype is None else stored.to(dtype))
    assert norm.weight.dtype == torch.float32 and torch.equal(norm.weight, stored.float() + 1.0)
    x = torch.randn(4, 6, generator=torch.Generator().manual_seed(1))
    assert torch.allclose(norm.forward(x).double(), plain.norm(x.double(), stored.double(), 1e-5), atol=1e-6)


def test_plain_pooled_window_by_hand():
    """One head, values that name their token: which tokens and runs a position sees, one by one."""
    T, size, pool = 23, 5, 3
    k = torch.zeros((T, 1, 1), dtype=torch.float64)
    v = torch.eye(T, dtype=torch.float64)[:, None, :]
    o = plain.pooled_window_attention(k, k, v, 1.0, size, pool)[:, 0]
    for i in range(T):
        tokens = [j for j in range(T) if 0 <= i - j < size]
        runs = [b for b in range(T) if b * pool + pool - 1 <= i - size]
        share = 1.0 / (1 + len(tokens) + len(runs))                # every score is 0, as is the sink's
        want = torch.zeros(T, dtype=torch.float64)
        want[tokens] = share
        for b in runs:
            want[b * pool:(b + 1) * pool] += share / pool
        assert torch.allclose(o[i], want, atol=1e-12), i


def test_pooled_twin_against_plain(cpu_ops, tmp_path):
    """One layer through the engine's part: first a peaked query on a run far back, whose mean then carries
    the result, and a window's edge that moves by one token."""
    T, size, pool, page = 61, 11, 4, 8
    g = torch.Generator().manual_seed(3)
    k, v, q = (torch.randn((T, 2, n), generator=g) for n in (12, 20, 12))
    table = torch.randperm(8, generator=g).int()[None, :]
    runs_table = torch.randperm(3, generator=g).int()[None, :]
    kc, vc = torch.zeros((8, 2, page, 12)), torch.zeros((8, 2, 20, page))
    rk, rv = torch.full((3, 2, page, 12), float("nan")), torch.full((3, 2, 20, page), float("nan"))
    cu, kvl = torch.tensor([0, T], dtype=torch.int32), torch.tensor([T], dtype=torch.int32)
    pos, seq = torch.arange(T).int(), torch.zeros(T, dtype=torch.int32)
    rows = torch.cat((q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)), dim=1)
    runs = (rk, rv, runs_table, pool)
    got_q = cpu_ops.turn_prepare(rows, None, 2, 2, 12, 20, None, 1.0, pos, seq, torch.float32, table, kc, vc, runs=runs,
                                 cu_seqlens_q=cu, kv_lens=kvl, max_q_len=T)
    assert torch.equal(got_q, q)
    sink = torch.zeros(2)
    for scale in (0.3, 4.0):
        got = cpu_ops.softcap_attention(got_q, kc, vc, table, cu, kvl, seq, pos, T, T, scale, 0.0, window=size,
                                        values_transposed=True, sink=sink, runs=runs)
        want = plain.pooled_window_attention(q.double(), k.double(), v.double(), scale, size, pool)
        assert torch.allclose(got.view(T, 2, 20).double(), want, atol=1e-5)
    # moving the window's edge by one token, or the runs' by one, is far outside that bound
    for other in (dict(size=size + 1, pool=pool), dict(size=size - 1, pool=pool), dict(size=size, pool=pool + 1)):
        wrong = plain.pooled_window_attention(q.double(), k.double(), v.double(), 4.0, **other)
        assert float((wrong - want).abs().max()) > 0.05


def test_sigmoid_attention_and_convolution_by_hand():
    q = torch.tensor([[[1.0]], [[2.0]], [[-1.0]]], dtype=torch.float64)
    k = torch.tensor([[[0.5]], [[1.0]], [[3.0]]], dtype=torch.float64)
    v = torch.tensor([[[1.0]], [[10.0]], [[100.0]]], dtype=torch.float64)
    o = plain.sigmoid_attention(q, k, v, 2.0, torch.tensor([-0.5], dtype=torch.float64))[:, 0, 0]
    s = lambda x: 1.0 / (1.0 + math.exp(-x))                          # noqa: E731
    want = [s(0.5), s(1.5) + 10 * s(3.5), s(-1.5) + 10 * s(-2.5) + 100 * s(-6.5)]
    assert torch.allclose(o, torch.tensor(want, dtype=torch.float64))
    u = torch.tensor([[1.0], [2.0], [4.0], [8.0]], dtype=torch.float64)
    w = torch.tensor([[100.0, 10.0, 1.0]], dtype=torch.float64)
    assert plain.short_convolution(u, w)[:, 0].tolist() == [1.0, 12.0, 124.0, 248.0]


def _memory_inputs(T, H, d, dv, seed, f_shift=2.0, i_scale=3.0):
    g = torch.Generator().manual_seed(seed)
    rows = torch.randn((T, 2 * H * (d + dv) + 2 * H + 3), generator=g)
    base = 2 * H * (d + dv)
    rows[:, base:base + H] *= i_scale
    rows[:, base + H:base + 2 * H] = rows[:, base + H:base + 2 * H] * 2.0 + f_shift
    ib, fb = torch.randn(H, generator=g), torch.randn(H, generator=g)
    norm = torch.randn(H * dv, generator=g)
    return rows, ib, fb, norm


def _memory_plain(rows, H, d, dv, cap, ib, fb, norm, eps):
    z = rows.double().cpu()
    T = z.shape[0]
    base = 2 * H * (d + dv)
    q, k = z[:, :H * d].view(T, H, d) * d ** -0.5, z[:, H * d:2 * H * d].reshape(T, H, d)
    v = z[:, 2 * H * d:2 * H * d + H * dv].reshape(T, H, dv)
    i = cap * torch.tanh((z[:, base:base + H] + ib.double().cpu()) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((z[:, base + H:base + 2 * H] + fb.double().cpu()) / cap))
    o = plain.rms(plain.mlstm_recurrence(q, k, v, i, f), eps).reshape(T, H * dv) * norm.double().cpu()
    return o * torch.sigmoid(z[:, 2 * H * d + H * dv:base])


def test_memory_twin_against_plain(cpu_ops):
    """The gates' cap, a maximum that starts at nothing (not at minus infinity: closed input gates leave exp(-m)
    in the denominator), forgetting and keeping, over three cuts."""
    H, d, dv, cap = 3, 6, 70, 2.5
    for shift, i_scale in ((2.0, 3.0), (-4.0, 1.0), (9.0, 9.0)):
        rows, ib, fb, norm = _memory_inputs(40, H, d, dv, 7, shift, i_scale)
        want = _memory_plain(rows, H, d, dv, cap, ib, fb, norm, 1e-5)
        state = torch.zeros((2, cpu_ops.mlstm_state_numbers(H, d, dv)))
        slots, got, at = torch.tensor([1], dtype=torch.int32), [], 0
        for n in (17, 1, 22):
            cu = torch.tensor([0, n], dtype=torch.int32)
            got.append(cpu_ops.mlstm_scan(rows[at:at + n], H, d, dv, cap, ib, fb, norm, 1e-5, 1e-6, state, slots, cu,
                                          torch.float32))
            at += n
        assert torch.allclose(torch.cat(got).double(), want, atol=2e-4, rtol=2e-4)
    # a first token with a closed input gate: n . q is far below exp(-m) = 1, which then is the denominator
    one = torch.ones((1, 1, 1), dtype=torch.float64)
    o = plain.mlstm_recurrence(one, one, one, torch.tensor([[-6.0]], dtype=torch.float64), torch.tensor([[-0.1]], dtype=torch.float64))
    m = -0.1
    assert abs(float(o) - math.exp(-6.0 - m) / (math.exp(-m) + 1e-6)) < 1e-9


def test_logits_are_capped(cpu_ops):
    x = torch.tensor([[-50.0, -1.0, 0.0, 2.0, 400.0]])
    assert torch.allclose(cpu_ops.soft_cap(x.clone(), 5.0), 5.0 * torch.tanh(x / 5.0))


# ---- the model on the host ----

def test_logits_on_the_host_under_every_cutting(cpu_ops, folder):
    requests = _requests(folder)
    _, _, want = _truth(folder, requests)
    for make in (trace_whole, trace_tail_decoded, trace_portions, trace_mixed):
        steps = make(requests)
        runner = load_runner(folder, dtype="float32", device="cpu", page_size=8,
                             max_tokens=max_live_tokens(steps, page=8), max_requests=4)
        assert _off(run_trace(runner, steps), want, "float32") <= 1.0, make.__name__
        assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.groups)


def test_layer_streams_on_the_host(cpu_ops, tmp_path):
    folder = _write(tmp_path / "m", MIXED)
    tokens = random_tokens(57, MIXED["vocab"], 4)
    config, w, _ = _truth(folder, {})
    streams = []
    plain.logits_of_sequence(config, w, tokens, streams)
    runner = load_runner(folder, dtype="float32", device="cpu", page_size=8, max_tokens=64, max_requests=1)
    seen = []
    runner.model.observer = lambda i, x, pending: seen.append(x.double() + pending.double())
    runner.step([StepEntry("r", tokens, [])])
    assert len(seen) == len(streams) == len(MIXED["layers"])
    for got, want in zip(seen, streams):
        assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max())


def test_greedy_generation_through_the_engine_on_the_host(cpu_ops, folder):
    requests = _requests(folder)
    config, w, _ = _truth(folder, {})
    engine = SyncEngine(path=folder, dtype="float32", device="cpu", max_len=256, block_size=8, num_blocks=60,
                        max_num_seqs=3, max_num_tokens=24, chunked_prefill_size=16)
    prompts = [toks[:n] for toks, n in zip(requests.values(), (30, 9, 41, 2))]
    got = engine.generate_ids(prompts, max_new_tokens=5, temperature=0.0, ignore_eos=True)
    for prompt, new in zip(prompts, got):
        seq = list(prompt)
        for _ in range(5):
            seq.append(int(torch.argmax(plain.logits_of_sequence(config, w, seq)[-1])))
        assert new == seq[len(prompt):]
    manager = engine.runner.manager
    assert all(g.pool.num_free == g.pool.num_pages for g in manager.groups) and not manager.live()


def test_a_preempted_request_builds_its_means_and_states_again(cpu_ops, tmp_path):
    """Pages for one request and a half: one is preempted, its runs, tails and memories are made anew in other
    pages and another slot, and it generates what it would have alone."""
    folder = _write(tmp_path / "m", MIXED)
    config, w, _ = _truth(folder, {})
    engine = SyncEngine(path=folder, dtype="float32", device="cpu", max_len=64, block_size=8, num_blocks=9,
                        max_num_seqs=2, max_num_tokens=32, chunked_prefill_size=16)
    prompts = [random_tokens(n, MIXED["vocab"], 40 + n) for n in (26, 21)]
    params = engine.default_params(14, temperature=0.0, ignore_eos=True)
    requests = [engine.add_request(p, params) for p in prompts]
    while engine.scheduler.has_work():
        engine.step()
        engine.runner.manager.audit()
    assert sum(r.preemptions for r in requests) > 0
    for prompt, request in zip(prompts, requests):
        seq = list(prompt)
        for _ in range(14):
            seq.append(int(torch.argmax(plain.logits_of_sequence(config, w, seq)[-1])))
        assert list(request.generated) == seq[len(prompt):]


def test_command_line_writes_a_folder_from_the_nested_config(tmp_path):
    from qwen3_from_scratch_amd.engine.cli import main

    source = tmp_path / "config.json"
    source.write_text(json.dumps(MIXED))
    assert main(["--write_random", str(tmp_path / "m"), "--from_config", str(source), "--seed", "3"]) == 0
    assert load_model_config(str(tmp_path / "m")).to_dict() == MIXED
    tensors = load_file(str(tmp_path / "m" / "model.safetensors"))
    assert "l1.mix.k.conv" in tensors and "l2.mix.i.b" in tensors and "l2.norm2" not in tensors
    assert float(tensors["l0.norm1"].float().abs().mean()) < 0.1       # a norm's weight lacks its one


# ---- kernels against their twins ----

def _rand(shape, seed, dtype, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(dtype).cuda()


def _tables(kv, page, per, seed, spare=3):
    """Block tables of sequences of kv[b] tokens, `per` tokens an element, over shuffled pages; and the pages."""
    blocks = [-(-(n // per) // page) for n in kv]
    order = torch.randperm(sum(blocks) + spare, generator=torch.Generator().manual_seed(seed)).tolist()
    table = torch.full((len(kv), max(1, max(blocks))), -1, dtype=torch.int32)
    for b, n in enumerate(blocks):
        for j in range(n):
            table[b, j] = order.pop()
    return table.cuda(), sum(blocks) + spare


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,dv,half,page,pool", [(4, 2, 16, 24, 4, 8, 6), (16, 4, 64, 64, 32, 16, 8), (3, 1, 7, 5, 0, 16, 1),
                                                     (6, 3, 128, 128, 16, 16, 20), (2, 2, 300, 10, 129, 16, 33)])
def test_turn_prepare_kernel(dtype, H, G, d, dv, half, page, pool):
    """Portions of prompts beside single tokens, then single tokens alone (the means in the same kernel), then
    values that are keys; with runs, every one that ends in the step and no other."""
    import torch_ops
    from qwen3_from_scratch_amd import ops

    n = H * d + G * (d + dv)
    inv_freq = (torch.rand(half, generator=torch.Generator().manual_seed(4)) + 0.01).cuda() if half else None
    bias = _rand((n,), 2, torch.float32)
    for q_lens, kv in (([37, 1, 2, 5], [90, 41, 2, 66]), ([1, 1, 1, 1, 1], [pool, 2 * pool, 67, 1, 3 * pool - 1 or 1]),
                       ([300], [301])):
        T, B = sum(q_lens), len(kv)
        rows = _rand((T, n + 5), 1, torch.float32, 2.0)
        table, pages = _tables(kv, page, 1, 7)
        run_table, run_pages = _tables(kv, page, pool, 8)
        cu = torch.tensor([0] + list(np.cumsum(q_lens)), dtype=torch.int32).cuda()
        kvl = torch.tensor(kv, dtype=torch.int32).cuda()
        pos = torch.cat([torch.arange(L - m, L) for m, L in zip(q_lens, kv)]).int().cuda()
        seq = torch.cat([torch.full((m,), b) for b, m in enumerate(q_lens)]).int().cuda()
        out = []
        for impl in (ops, torch_ops):
            kc, vc = _rand((pages, G, page, d), 11, dtype), _rand((pages, G, dv, page), 12, dtype)
            rk, rv = _rand((run_pages, G, page, d), 13, dtype), _rand((run_pages, G, dv, page), 14, dtype)
            q = impl.turn_prepare(rows, bias, H, G, d, dv, inv_freq, 1.25, pos, seq, dtype, table, kc, vc,
                                  runs=(rk, rv, run_table, pool), cu_seqlens_q=cu, kv_lens=kvl, max_q_len=max(q_lens))
            out.append((q, kc, vc, rk, rv))
        tol = 3e-5 if dtype == torch.float32 else 6e-2
        for a, b in zip(*out):
            assert float((a.float() - b.float()).abs().max()) <= tol
        if dtype == torch.bfloat16 and max(q_lens) == 1:     # the means of both ways are the same numbers
            again = [t.clone() for t in out[0][1:]]
            ops.turn_prepare(rows, bias, H, G, d, dv, inv_freq, 1.25, pos, seq, dtype, table, again[0], again[1],
                             runs=(again[2], again[3], run_table, pool), cu_seqlens_q=cu, kv_lens=kvl, max_q_len=2)
            assert all(torch.equal(a, b) for a, b in zip(again, out[0][1:]))
        if d == dv:
            both = []
            for impl in (ops, torch_ops):
                kc, vc = _rand((pages, G, page, d), 11, dtype), _rand((pages, G, d, page), 12, dtype)
                q = impl.turn_prepare(rows[:, :(H + G) * d], None, H, G, d, d, inv_freq, 0.5, pos, seq, dtype, table, kc, vc,
                                      values_are_keys=True)
                both.append((q, kc, vc))
            for a, b in zip(*both):
                assert float((a.float() - b.float()).abs().max()) <= tol


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,dv,page,window,pool", [
    (4, 2, 16, 24, 8, 20, 6), (8, 2, 64, 64, 16, 50, 8), (10, 5, 128, 128, 16, 90, 10), (16, 4, 128, 128, 32, 256, 16),
    (3, 1, 64, 64, 16, 7, 12), (32, 1, 64, 64, 16, 33, 3), (5, 5, 10, 300, 16, 1, 1)])
def test_pooled_attention_kernels(dtype, H, G, d, dv, page, window, pool):
    """Portions, short portions and single tokens in one step, over scattered pages of which those behind the
    window are gone, against the twin; with a gate per head, per column and none."""
    import torch_ops
    from qwen3_from_scratch_amd import ops

    kv = [700, 333, 1, 257, 64, window + pool, 1500]
    q_lens = [150, 1, 1, 2, 64, 3, 9]
    T = sum(q_lens)
    table, pages = _tables(kv, page, 1, 17)
    run_table, run_pages = _tables(kv, page, pool, 18)
    kc, vc = _rand((pages, G, page, d), 21, dtype), _rand((pages, G, dv, page), 22, dtype)
    rk, rv = _rand((run_pages, G, page, d), 23, dtype), _rand((run_pages, G, dv, page), 24, dtype)
    for b, (n, L) in enumerate(zip(q_lens, kv)):              # what the manager would have taken back by now
        gone = max(0, L - n - max(window, pool) + 1) // page
        table[b, :gone] = -1
    cu = torch.tensor([0] + list(np.cumsum(q_lens)), dtype=torch.int32).cuda()
    kvl = torch.tensor(kv, dtype=torch.int32).cuda()
    pos = torch.cat([torch.arange(L - m, L) for m, L in zip(q_lens, kv)]).int().cuda()
    seq = torch.cat([torch.full((m,), b) for b, m in enumerate(q_lens)]).int().cuda()
    q = _rand((T, H, d), 3, dtype, 2.0)
    sink = torch.zeros(H).cuda()
    wide = _rand((T, H * dv + 7), 5, torch.float32, 2.0)
    tol = 2e-5 if dtype == torch.float32 else 2.5e-2
    for gate in (None, wide[:, 3:3 + H], wide[:, 3:3 + H * dv]):
        kw = dict(window=window, gate=gate, values_transposed=True, sink=sink, runs=(rk, rv, run_table, pool))
        a = ops.softcap_attention(q, kc, vc, table, cu, kvl, seq, pos, max(q_lens), max(kv), d ** -0.5, 0.0, min_q_len=1, **kw)
        b = torch_ops.softcap_attention(q, kc, vc, table, cu, kvl, seq, pos, max(q_lens), max(kv), d ** -0.5, 0.0, **kw)
        assert float((a.float() - b.float()).abs().max()) <= tol
    # single tokens alone: the decoding kernel with the keys shared out over blocks
    ones = torch.arange(len(kv) + 1, dtype=torch.int32).cuda()
    kw = dict(window=window, values_transposed=True, sink=sink, runs=(rk, rv, run_table, pool), gate=wide[:len(kv), :H])
    seq1, pos1 = torch.arange(len(kv)).int().cuda(), (kvl - 1).int()
    a = ops.softcap_attention(q[:len(kv)], kc, vc, table, ones, kvl, seq1, pos1, 1, max(kv), d ** -0.5, 0.0, **kw)
    b = torch_ops.softcap_attention(q[:len(kv)], kc, vc, table, ones, kvl, seq1, pos1, 1, max(kv), d ** -0.5, 0.0, **kw)
    assert float((a.float() - b.float()).abs().max()) <= tol


@pytest.mark.gpu
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_window_and_run_edges(dtype, decoded):
    """A query that stands on one key (or one run's mean) gets its value if it sees it and nothing of it if it does
    not: the first token of the window and the one before it, the last run behind the window and the one that
    still touches it, runs and tokens at page ends, hundreds of positions back; the sink takes what is left."""
    from qwen3_from_scratch_amd import ops

    H, G, d, page, window, pool, L = 4, 2, 64, 16, 100, 12, 900
    table, pages = _tables([L], page, 1, 31)
    run_table, run_pages = _tables([L], page, pool, 32)
    unit = lambda n, s: torch.nn.functional.normalize(_rand((n, G, d), s, torch.float32), dim=-1)     # noqa: E731
    keys, values = unit(L, 1), unit(L, 2)
    rkeys, rvalues = unit(L // pool, 3), unit(L // pool, 4)
    kc, vc = torch.zeros((pages, G, page, d), dtype=dtype).cuda(), torch.zeros((pages, G, d, page), dtype=dtype).cuda()
    rk, rv = torch.zeros((run_pages, G, page, d), dtype=dtype).cuda(), torch.zeros((run_pages, G, d, page), dtype=dtype).cuda()
    for src, k_to, v_to, tab in ((  (keys, values), kc, vc, table), ((rkeys, rvalues), rk, rv, run_table)):
        at = torch.arange(src[0].shape[0]).cuda()
        pg = tab[0, at // page].long()
        k_to[pg, :, at % page] = src[0].to(dtype)
        v_to[pg, :, :, at % page] = src[1].to(dtype)
    positions = [0, 99, 100, 111, 112, 113, 500, 527, 528, 623, 899]
    for i in positions:
        n = 1 if decoded else 9                                  # alone, or as the last row of a portion
        n = min(n, i + 1)
        cu, kvl = torch.tensor([0, n], dtype=torch.int32).cuda(), torch.tensor([i + 1], dtype=torch.int32).cuda()
        pos, seq = torch.arange(i + 1 - n, i + 1).int().cuda(), torch.zeros(n, dtype=torch.int32).cuda()
        seen_runs = max(0, i - window + 1) // pool
        cases = [("token", j, i - j < window) for j in {i, i - 1, i - window + 1, i - window, (i - 50) // page * page, 0} if 0 <= j <= i]
        cases += [("run", r, r < seen_runs) for r in {0, seen_runs - 1, seen_runs, 15, 16} if 0 <= r < (i + 1) // pool]
        for kind, at, seen in cases:
            k_of, v_of = (keys, values) if kind == "token" else (rkeys, rvalues)
            q = torch.zeros((n, H, d), dtype=dtype).cuda()
            q[-1] = (k_of[at] * 40.0).repeat_interleave(H // G, dim=0).to(dtype)
            got = ops.softcap_attention(q, kc, vc, table, cu, kvl, seq, pos, n, i + 1, 1.0, 0.0, window=window, min_q_len=n,
                                        values_transposed=True, sink=torch.zeros(H).cuda(), runs=(rk, rv, run_table, pool))
            share = (got[-1].view(H, d).float() * v_of[at].repeat_interleave(H // G, dim=0)).sum(dim=-1)
            if seen:
                assert float((share - 1.0).abs().max()) <= 2e-2, (i, kind, at)
            else:
                assert float(share.abs().max()) <= 0.75, (i, kind, at)
    # a sink of zero takes half of a single key whose score is zero
    got = ops.softcap_attention(torch.zeros((1, H, d), dtype=dtype).cuda(), kc, vc, table, torch.tensor([0, 1], dtype=torch.int32).cuda(),
                                torch.tensor([1], dtype=torch.int32).cuda(), torch.zeros(1, dtype=torch.int32).cuda(),
                                torch.zeros(1, dtype=torch.int32).cuda(), 1, 1, 1.0, 0.0, window=window, values_transposed=True,
                                sink=torch.zeros(H).cuda(), runs=(rk, rv, run_table, pool))
    assert torch.allclose(got.view(H, d).float(), 0.5 * values[0].to(dtype).float().repeat_interleave(H // G, dim=0), atol=2e-3)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,page", [(6, 2, 12, 8), (8, 2, 64, 16), (4, 4, 128, 32), (3, 1, 130, 16), (16, 1, 128, 16)])
def test_sigmoid_attention_kernels(dtype, H, G, d, page):
    import torch_ops
    from qwen3_from_scratch_amd import ops

    kv, q_lens = [700, 333, 1, 257, 64, 2600], [150, 1, 1, 2, 64, 5]
    T = sum(q_lens)
    table, pages = _tables(kv, page, 1, 17)
    kc, vc = _rand((pages, G, page, d), 21, dtype), _rand((pages, G, d, page), 22, dtype)
    bias = torch.linspace(-6.0, 1.0, H).cuda()
    wide = _rand((T, H * d + 3), 5, torch.float32, 2.0)
    q = _rand((T, H, d), 3, dtype, 2.0)
    kvl = torch.tensor(kv, dtype=torch.int32).cuda()
    for lens, rows in ((q_lens, T), ([1] * len(kv), len(kv))):
        cu = torch.tensor([0] + list(np.cumsum(lens)), dtype=torch.int32).cuda()
        pos = torch.cat([torch.arange(L - m, L) for m, L in zip(lens, kv)]).int().cuda()
        seq = torch.cat([torch.full((m,), b) for b, m in enumerate(lens)]).int().cuda()
        for gate in (None, wide[:rows, 2:2 + H * d]):
            kw = dict(values_transposed=True, sigmoid_bias=bias, gate=gate)
            a = ops.softcap_attention(q[:rows], kc, vc, table, cu, kvl, seq, pos, max(lens), max(kv), d ** -0.5, 0.0, **kw)
            b = torch_ops.softcap_attention(q[:rows], kc, vc, table, cu, kvl, seq, pos, max(lens), max(kv), d ** -0.5, 0.0, **kw)
            size = float(b.float().abs().max())                   # sums over keys that nothing divides
            assert float((a.float() - b.float()).abs().max()) <= (1e-5 if dtype == torch.float32 else 1e-2) * max(size, 1.0)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,d,dv,cap", [(3, 8, 12, 5.0), (2, 130, 150, 15.0), (5, 64, 64, 3.0), (1, 5, 70, 30.0), (2, 300, 33, 15.0)])
def test_memory_kernels_against_plain(dtype, H, d, dv, cap):
    """Cuts around the chunks' edges and down to single tokens, several sequences in one step, slots out of order,
    gates that keep for long, forget at once, or open wide: against the recurrence token by token."""
    from qwen3_from_scratch_amd import ops

    tol = 3e-4 if dtype == torch.float32 else 2e-2
    for shift, i_scale in ((3.0, 2.0), (-6.0, 2.0), (12.0, 9.0)):
        lengths = [200, 67, 130]
        data = [_memory_inputs(n, H, d, dv, 50 + n, shift, i_scale) for n in lengths]
        _, ib, fb, norm = [t.cuda() for t in data[0]]
        want = [_memory_plain(x[0], H, d, dv, cap, ib, fb, norm, 1e-5) for x in data]
        state = torch.zeros((5, ops.mlstm_state_numbers(H, d, dv)), dtype=torch.float32).cuda()
        slots = torch.tensor([3, 0, 4], dtype=torch.int32).cuda()
        at = [0, 0, 0]
        for cut in ([64, 9, 1], [1, 1, 1], [8, 2, 63], [63, 0, 65], [1, 1, 0], [60, 54, 0], [3, 0, 0]):
            rows = torch.cat([data[b][0][at[b]:at[b] + n] for b, n in enumerate(cut)]).cuda()
            cu = torch.tensor([0] + list(np.cumsum(cut)), dtype=torch.int32).cuda()
            got = ops.mlstm_scan(rows, H, d, dv, cap, ib, fb, norm, 1e-5, 1e-6, state, slots, cu, dtype, max_q_len=max(cut))
            first = 0
            for b, n in enumerate(cut):
                ref = want[b][at[b]:at[b] + n]
                if n:
                    off = (got[first:first + n].double().cpu() - ref).abs().max()
                    assert float(off) <= tol * max(1.0, float(ref.abs().max())), (shift, cut, b)
                first += n
                at[b] += n
        assert at == [200, 67, 130]
        assert float(state[1].abs().max()) == 0 and float(state[2].abs().max()) == 0       # others' slots


@pytest.mark.gpu
@pytest.mark.parametrize("M,I,K", [(1, 96, 64), (7, 200, 128), (16, 6144, 2048), (12, 6144, 2048), (48, 512, 256),
                                   (64, 6144, 2048), (90, 6144, 2048), (130, 256, 128), (5, 33, 40)])
def test_gelu_in_a_products_epilogue(M, I, K):
    """The same bits as the product followed by the activation's kernel, also for rows that still lack their
    norm's division; sizes of the few-row kernel (one slab and two a block), of the weight-streaming one, and
    of neither."""
    from qwen3_from_scratch_amd import ops

    x, w = _rand((M, K), 1, torch.bfloat16, 2.0), _rand((2 * I, K), 2, torch.bfloat16, K ** -0.5)
    tiled = ops.tile_weight(w)
    for unscaled in (None, (torch.full((1, ops.sums_stride(M)), 3.0 * K).cuda(), 1e-5, K)):
        if unscaled is not None and not (tiled is not None and (M <= ops.few_rows_limit(w) or ops.fused_rows_take(w, M))):
            continue
        for kind in ("gelu_tanh", "silu", "gelu_erf"):
            got = ops.linear_swiglu(x, w, tiled=tiled, unscaled=unscaled, kind=kind)
            want = ops.gated_act(ops.linear(x, w, tiled=tiled, unscaled=unscaled), kind)
            close = (got.float() - want.float()).abs().max() <= 2e-2 * max(1.0, float(want.float().abs().max()))
            # the kernels for a gated product and for a plain one may add up a row's terms in different orders
            assert bool(close) and float((got != want).float().mean()) < 0.2, kind


@pytest.mark.gpu
def test_soft_cap_kernel():
    from qwen3_from_scratch_amd import ops

    for shape in ((1, 5), (3, 1031), (7, 4096)):
        x = _rand(shape, 1, torch.float32, 40.0)
        want = 12.0 * torch.tanh(x.double() / 12.0)
        assert float((ops.soft_cap(x, 12.0).double() - want).abs().max()) <= 3e-6 * 12


# ---- the model on the GPU ----

@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_logits_under_every_cutting(folders, dtype):
    folder = folders[dtype]
    requests = _requests(folder, lengths=(70, 9, 141, 250, 25, 2, 1))
    _, _, want = _truth(folder, requests)
    for make in (trace_whole, trace_tail_decoded, trace_portions, trace_mixed):
        steps = make(requests)
        runner = load_runner(folder, dtype=dtype, device="cuda", page_size=16,
                             max_tokens=max_live_tokens(steps, page=16), max_requests=4)
        assert _off(run_trace(runner, steps), want, dtype) <= 1.0, make.__name__
        assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.groups)


@pytest.mark.gpu
def test_layer_streams(tmp_path):
    """The float32 engine's residual stream behind every layer against the plain one's."""
    folder = _write(tmp_path / "m", MIXED)
    tokens = random_tokens(75, MIXED["vocab"], 4)
    config, w, _ = _truth(folder, {})
    streams = []
    plain.logits_of_sequence(config, w, tokens, streams)
    runner = load_runner(folder, dtype="float32", device="cuda", page_size=16, max_tokens=80, max_requests=1)
    seen = []
    runner.model.observer = lambda i, x, pending: seen.append((x.double() + pending.double()).cpu())
    runner.step([StepEntry("r", tokens, [])])
    assert len(seen) == len(streams)
    for got, want in zip(seen, streams):
        assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max())


@pytest.mark.gpu
def test_long_decoding_and_first_tokens(folders):
    """A request decoded token by token from its second token on, through graph replays, page and run ends,
    beside a request that is decoded from its very first."""
    for dtype in ("float32", "bfloat16"):
        folder = folders[dtype]
        vocab = load_model_config(folder).vocab
        requests = {"long": random_tokens(200, vocab, 7), "short": random_tokens(3, vocab, 8)}
        _, _, want = _truth(folder, requests)
        runner = load_runner(folder, dtype=dtype, device="cuda", page_size=16, max_tokens=256, max_requests=2)
        steps = [([(rid, toks[:1], [0]) for rid, toks in requests.items()], [])]
        for i in range(1, 200):
            entries = [(rid, [toks[i]], [0]) for rid, toks in requests.items() if i < len(toks)]
            steps.append((entries, [rid for rid, toks in requests.items() if i == len(toks) - 1]))
        assert _off(run_trace(runner, steps), want, dtype) <= 1.0


def _far_model(folder, kind):
    """One layer of either attention. Queries are the keys' negatives, and the embedding of one token (`asks`) is
    another's (`holds`) negative: a query of the one stands on the keys of the other. Nothing turns. A prompt in
    which a whole run of the one that holds stands early and the one that asks near the end."""
    layer = (_attention(4, 2, 64, 64, size=40, pool=4, scale=0.25) if kind == "attention" else _sigmoid(4, 2, 64, 1, scale=0.25))
    data = _model(131, 128, [_layer(layer, 96)], cap=20.0)
    folder = _write(folder, data, std=0.1, apart=9.0)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    p = "l0.mix."
    k = tensors[p + "k"].view(2, 64, -1)
    tensors[p + "q"] = -k.repeat_interleave(2, dim=0).reshape(256, -1).contiguous()
    for name in ("q.b", "k.b"):
        tensors[p + name] = torch.zeros_like(tensors[p + name])
    if kind != "attention":
        for name in ("q.conv", "k.conv"):
            tensors[p + name] = torch.ones_like(tensors[p + name])
    asks, holds = data["vocab"] - 1, data["vocab"] - 2
    tensors["embed"][asks] = -tensors["embed"][holds]
    save_file(tensors, path, metadata={"format": "pt"})
    tokens = [min(t, holds - 1) for t in random_tokens(600, data["vocab"], 31)]
    tokens[36:40] = [holds] * 4
    tokens[-2] = asks
    return folder, tokens


@pytest.mark.parametrize("kind", ["attention", "attention_2"])
def test_the_far_model_leans_on_its_far_run(tmp_path, kind):
    """The truth of the test below: without the early run the row that asks is another one."""
    folder, tokens = _far_model(tmp_path / "m", kind)
    _, _, want = _truth(folder, {"far": tokens, "cut": tokens[:36] + [3, 5, 7, 11] + tokens[40:]})
    a, b = want["far"][-2], want["cut"][-2]
    assert float((a - b).pow(2).mean().sqrt()) > 0.3 * float(a.std())


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["attention", "attention_2"])
def test_a_far_run_carries_the_last_row(tmp_path, dtype, kind):
    """The row that asks leans on a run's mean (pooled attention) or on keys (sigmoid attention) hundreds of
    positions back, in a whole prompt, in portions, and decoded."""
    folder, tokens = _far_model(tmp_path / "m", kind)
    _, _, want = _truth(folder, {"far": tokens})
    for steps in (trace_whole({"far": tokens}), trace_tail_decoded({"far": tokens}, tail=4),
                  trace_portions({"far": tokens}, sizes=(130, 37, 2, 261, 64, 3))):
        runner = load_runner(folder, dtype=dtype, device="cuda", page_size=16, max_tokens=608, max_requests=1)
        got = run_trace(runner, steps)
        for p in range(590, 600):
            d = got[("far", p)].double() - want["far"][p]
            assert float((d - d.mean()).pow(2).mean().sqrt() / want["far"][p].std()) <= (5e-5 if dtype == "float32" else 5e-2)


@pytest.mark.gpu
def test_greedy_generation_through_the_engine(folders):
    for dtype in ("float32", "bfloat16"):
        folder = folders[dtype]
        requests = _requests(folder)
        config, w, _ = _truth(folder, {})
        engine = SyncEngine(path=folder, dtype=dtype, device="cuda", max_len=256, block_size=16, num_blocks=30,
                            max_num_seqs=3, max_num_tokens=48, chunked_prefill_size=32)
        prompts = [toks[:n] for toks, n in zip(requests.values(), (60, 9, 41, 2))]
        got = engine.generate_ids(prompts, max_new_tokens=8, temperature=0.0, ignore_eos=True)
        for prompt, new in zip(prompts, got):
            logits = plain.logits_of_sequence(config, w, prompt + new)
            for i, token in enumerate(new):
                row = logits[len(prompt) + i - 1]
                slack = 0.0 if dtype == "float32" else 0.02 * float(row.max() - row.min())
                assert float(row[token]) >= float(row.max()) - slack - 1e-9
        assert all(g.pool.num_free == g.pool.num_pages for g in engine.runner.manager.groups)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_replay_program(folders, tmp_path, dtype):
    folder = folders[dtype]
    requests = _requests(folder)
    _, _, want = _truth(folder, requests)
    steps = trace_mixed(requests, seed=3)
    lines = [json.dumps({"step": i, "entries": [{"id": r, "tokens": t, "want": ws} for r, t, ws in entries],
                         "end": ends}) for i, (entries, ends) in enumerate(steps)]
    out = str(tmp_path / dtype)
    proc = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", out,
         "--max-tokens", str(max_live_tokens(steps, page=64))],
        input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(len(steps))]
    got, lengths = {}, {}
    for i, (entries, _) in enumerate(steps):
        wanted = [(r, lengths.get(r, 0) + p) for r, t, ws in entries for p in ws]
        for r, t, _ in entries:
            lengths[r] = lengths.get(r, 0) + len(t)
        if wanted:
            rows = np.fromfile(os.path.join(out, "%d.f32" % i), dtype="<f4").reshape(len(wanted), -1)
            for key, row in zip(wanted, rows):
                got[key] = torch.from_numpy(row.copy())
    assert _off(got, want, dtype) <= 1.0


@pytest.mark.gpu
def test_command_line_generates(tmp_path):
    folder = _write(tmp_path / "m", CORES)
    config, w, _ = _truth(folder, {})
    prompt = random_tokens(70, CORES["vocab"], 12)
    proc = subprocess.run(
        [sys.executable, "-m", "qwen3_from_scratch_amd", "--path", folder, "--dtype", "float32", "--prompt_ids",
         ",".join(map(str, prompt)), "--max_new_tokens", "6", "--temperature", "0", "--ignore_eos", "--max_len", "128",
         "--block_size", "16", "--num_blocks", "16", "--max_num_seqs", "2"],
        capture_output=True, text=True, timeout=600, cwd=ROOT)
    assert proc.returncode == 0, proc.stderr[-2000:]
    got = [int(t) for t in proc.stdout.split()]
    seq = list(prompt)
    for _ in range(6):
        seq.append(int(torch.argmax(plain.logits_of_sequence(config, w, seq)[-1])))
    assert got == seq[len(prompt):]
