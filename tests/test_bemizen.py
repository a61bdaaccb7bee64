"""The Bemizen architecture through the engine against tests/plain_bemizen.py: each mechanism alone,
whole prompts against token-by-token decoding, portions down to two tokens, mixed batches with pages
that are used again, keys at the edges of windows, chunks, first tokens and pages, far keys, the first
tokens of a sequence, long decoding, and greedy generation through the engine. The configurations are
made here; their sizes differ from layer to layer and avoid values that hide a fault (equal key and
value sizes, one key head per query head, a rotation over the whole head, a router without identity
experts, groups that are all kept, a scale of one), beside one that has just these."""

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

import plain_bemizen as plain
from helpers import max_live_tokens, random_tokens, run_trace, trace_mixed, trace_portions, trace_tail_decoded, trace_whole
from qwen3_from_scratch_amd.cache.manager import CacheManager
from qwen3_from_scratch_amd.config import load_model_config
from qwen3_from_scratch_amd.config.bemizen_config import BemizenConfig
from qwen3_from_scratch_amd.config.model_config import ConfigError
from qwen3_from_scratch_amd.engine import StepEntry, SyncEngine, load_runner
from qwen3_from_scratch_amd.parts import CacheNeed, PagedTensor
from qwen3_from_scratch_amd.weights import write_random_model

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _mixer(heads, kv_heads, dim, vdim, mask, dims, base, scale, v_mix):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or 2.0 / math.sqrt(dim), "v_mix": v_mix}
    if mask:
        m["mask"] = mask
    if dims:
        m["rot"] = {"dims": dims, "base": base}
    return m


def _chunked(heads, kv_heads, dim, vdim, chunk, dims=None, base=500.0, scale=None, v_mix=True):
    return {"type": "attention", "mixer": _mixer(heads, kv_heads, dim, vdim, chunk and {"size": chunk}, dims, base, scale, v_mix)}


def _windowed(heads, kv_heads, dim, vdim, window, keep=0, dims=None, base=900.0, scale=None, v_mix=True):
    mask = {"size": window, "keep_first": keep} if window else None
    return {"type": "attention_2", "mixer": _mixer(heads, kv_heads, dim, vdim, mask, dims, base, scale, v_mix)}


def _moe(experts, identity, top, ff, groups=None, keep=None, scale=1.5):
    router = {"experts": experts, "identity": identity, "top": top, "scale": scale}
    if groups:
        router["groups"] = {"count": groups, "keep": keep}
    return {"kind": "moe", "router": router, "expert": {"ff": ff}}


def _layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def _model(vocab, width, layers, eps=1e-5):
    return {"architecture": "Bemizen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# both mixers, values mixed across layers whose key heads split the same numbers differently, a layer between
# them that does not mix, one without a feed-forward; windows and chunks that divide neither pages nor each other
MIXED = _model(131, 48, [
    _layer(_windowed(3, 1, 10, 14, 7, 3, dims=6, v_mix=False), _moe(5, 1, 2, 20, groups=3, keep=2)),
    _layer(_chunked(4, 2, 16, 24, 9, dims=8), _moe(6, 2, 2, 20, groups=4, keep=2)),
    _layer(_windowed(6, 3, 20, 16, 11, 5, dims=12), None),
    _layer(_chunked(8, 4, 12, 12, 21, dims=12), _moe(4, 4, 3, 12, groups=2, keep=1, scale=0.7)),
    _layer(_windowed(4, 1, 24, 48, 19, 26, dims=24), _moe(7, 3, 4, 16, groups=5, keep=3)),
])
# sizes that the matrix-core kernels take, keys and values of one size and of several; more first tokens than window
CORES = _model(257, 128, [
    _layer(_chunked(4, 2, 64, 64, 70, dims=32), _moe(6, 2, 2, 64, groups=4, keep=2)),
    _layer(_windowed(8, 2, 96, 64, 50, 21, dims=96), _moe(8, 1, 3, 64, groups=3, keep=2)),
    _layer(_windowed(4, 1, 192, 128, 33, 40, dims=64), _moe(3, 3, 2, 128, groups=2, keep=1)),
    _layer(_chunked(16, 1, 128, 128, 160, dims=128), _moe(4, 0, 2, 96, groups=2, keep=1)),
    _layer(_windowed(6, 2, 96, 96, 100, 0, dims=48, v_mix=False), _moe(4, 2, 3, 64)),
])
# sizes that no vector access and no matrix instruction takes; chunks and windows of one token, one expert, more
# identity experts than experts, groups of one, all experts a token
ODD = _model(53, 40, [
    _layer(_chunked(3, 1, 10, 14, 1, dims=4), _moe(1, 3, 2, 18, groups=4, keep=3)),
    _layer(_windowed(2, 2, 6, 7, 1, 1, dims=2), _moe(4, 0, 4, 9)),
    _layer(_windowed(1, 1, 7, 5, 6, 0, v_mix=False), _moe(3, 2, 1, 9)),
    _layer(_chunked(2, 1, 16, 14, 30), _moe(2, 1, 3, 10, groups=3, keep=3)),
])
# values that hide things in the others' place: equal sizes, one head, the whole head turned, a scale of one, no
# mask, no mixing
STRAIGHT = _model(97, 64, [
    _layer(_windowed(4, 4, 16, 16, 0, dims=16, v_mix=False), _moe(6, 0, 2, 32, groups=2, keep=2, scale=1.0)),
    _layer(_chunked(1, 1, 32, 32, 0, dims=32, v_mix=False), _moe(4, 0, 2, 32, scale=1.0)),
])
CONFIGS = {"mixed": MIXED, "cores": CORES, "odd": ODD, "straight": STRAIGHT}


def _write(folder, data, seed=5, std=0.2):
    """Random weights; shares of mixing between a third and four fifths, corrections of the size of the scores."""
    write_random_model(str(folder), BemizenConfig.from_dict(data), seed=seed, std=std, norm_jitter=0.3)
    path = os.path.join(str(folder), "model.safetensors")
    tensors = load_file(path)
    for i, layer in enumerate(data["layers"]):
        if layer["mixer"].get("v_mix"):       # the first that mixes has a share in the file too, which means nothing
            tensors["l%d.mix.vmix" % i] = torch.tensor(0.35 + 0.1 * i).to(torch.bfloat16)
        if layer["mlp"]:
            name = "l%d.mlp.correction" % i
            tensors[name] = (tensors[name].float() * 0.5).to(torch.bfloat16)
    save_file(tensors, path, metadata={"format": "pt"})
    return str(folder)


def _every_expert(data):
    """The configuration with every expert chosen for every token. In bfloat16 a router's score moves
    by a few thousandths, and with random weights some token in a hundred then changes an expert, which
    no bound on rounding covers; the choice itself is float32 in both precisions and is tested there and
    on the router kernel. With all experts chosen the weights still matter."""
    data = copy.deepcopy(data)
    for layer in data["layers"]:
        if layer["mlp"]:
            router = layer["mlp"]["router"]
            router["top"] = router["experts"] + router["identity"]
            if "groups" in router:
                router["groups"]["keep"] = router["groups"]["count"]
    return data


@pytest.fixture(scope="module", params=sorted(CONFIGS))
def folder(request, tmp_path_factory):
    return _write(tmp_path_factory.mktemp(request.param), CONFIGS[request.param])


@pytest.fixture(scope="module", params=sorted(CONFIGS))
def folders(request, tmp_path_factory):
    """{dtype: folder}: the configuration as it is for float32, with every expert chosen and smaller weights for bfloat16."""
    return {"float32": _write(tmp_path_factory.mktemp(request.param), CONFIGS[request.param]),
            "bfloat16": _write(tmp_path_factory.mktemp(request.param + "_all"), _every_expert(CONFIGS[request.param]), std=0.1)}


def _truth(folder, requests, dtype=torch.float64):
    with open(os.path.join(folder, "config.json")) as fh:
        config = json.load(fh)
    w = {k: v.to(dtype) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    return config, w, {rid: plain.logits_of_sequence(config, w, toks) for rid, toks in requests.items()}


def _requests(folder, lengths=(70, 9, 41, 130, 25, 2, 1)):
    vocab = load_model_config(folder).vocab
    return {"b%d" % i: random_tokens(n, vocab, 460 + i) for i, n in enumerate(lengths)}


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


# ---- configuration, weights, cache ----

def test_config_is_read_by_its_own_keys_and_written_back(folder):
    config = load_model_config(folder)
    assert isinstance(config, BemizenConfig) and config.architecture == "Bemizen"
    with open(os.path.join(folder, "config.json")) as fh:
        raw = json.load(fh)
    assert config.to_dict() == raw and len(config.layers) == len(raw["layers"])
    names = {k: tuple(v.shape) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}
    assert {"embed", "head", "final.norm", "l0.norm1"} <= set(names)
    for i, (layer, entry) in enumerate(zip(config.layers, raw["layers"])):
        p, m = "l%d." % i, entry["mixer"]
        mask = m.get("mask", {"size": 0})
        assert layer.type == entry["type"] and (layer.mlp is None) == (entry["mlp"] is None)
        assert layer.mixer.mixes_values == m["v_mix"] == (p + "mix.vmix" in names)
        if entry["type"] == "attention":
            assert (layer.mixer.chunk, layer.mixer.window, layer.mixer.keep_first) == (mask["size"], 0, 0)
            assert p + "mix.g" not in names and p + "mix.q.norm" not in names
        else:
            assert (layer.mixer.chunk, layer.mixer.window, layer.mixer.keep_first) == (0, mask["size"], mask.get("keep_first", 0))
            assert names[p + "mix.g"] == (m["heads"], raw["width"]) and names[p + "mix.k.norm"] == (m["dim"],)
        if entry["mlp"]:
            r = entry["mlp"]["router"]
            assert names[p + "mlp.router"] == (r["experts"] + r["identity"], raw["width"])
            assert names[p + "mlp.correction"] == (r["experts"] + r["identity"],)
            assert p + "mlp.e%d.down" % (r["experts"] - 1) in names and p + "mlp.e%d.down" % r["experts"] not in names


@pytest.mark.parametrize("change,word", [
    (lambda c: c["layers"][0].update(type="other"), "type"),
    (lambda c: c["layers"][1]["mixer"].pop("kv_heads"), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "divide"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][2]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18), "head's size"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(scaling={"low": 1.0, "high": 4.0, "factor": 2.0, "original": 9}), "scaling"),
    (lambda c: c["layers"][1]["mixer"].update(v_mix="yes"), "v_mix"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=15), "values"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=99), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "kept"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=2), "divide"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "identity"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=7), "keep"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "expert"),
    (lambda c: c.pop("width"), "width"),
])
def test_config_errors_name_the_key(change, word):
    data = copy.deepcopy(MIXED)
    change(data)
    with pytest.raises(ConfigError, match=word):
        BemizenConfig.from_dict(data)


def test_pages_of_chunks_and_of_first_tokens():
    """A chunk's pages go back when the next chunk begins, those behind a window as it moves on, those of
    first tokens that stay visible not before the request ends; layers with other spans have pools of their own."""
    pair = (PagedTensor("keys", (2, 4), 1), PagedTensor("values", (2, 6), 2))
    needs = [CacheNeed(paged=pair, chunk=10), CacheNeed(paged=pair, window=6, keep_first=5), CacheNeed(paged=pair, chunk=10),
             CacheNeed(paged=pair, window=6), CacheNeed(paged=pair)]
    m = CacheManager(needs, page_size=4, num_pages=20, max_requests=2)
    assert m.group_of_plane == [0, 1, 0, 2, 3] and [g.gives_back for g in m.groups] == [True, True, True, False]
    m.admit("a")
    held = lambda g: [b for b, page in enumerate(m.block_table("a", g)) if page >= 0]      # noqa: E731
    m.reserve("a", 9)
    m.commit("a", 9)
    assert held(0) == [0, 1, 2] and held(1) == [0, 1, 2] and held(2) == [1, 2]             # position 9 still sees 0 .. 9
    m.reserve("a", 1)
    m.commit("a", 1)
    assert held(0) == [2] and held(2) == [1, 2]                   # position 10 starts a chunk; page 2 holds 8 .. 11
    m.reserve("a", 21)
    m.commit("a", 21)                                             # the next stands at 31, in the chunk from 30 on
    assert held(0) == [7] and held(1) == [0, 1, 6, 7] and held(2) == [6, 7] and held(3) == list(range(8))
    m.audit()
    m.admit("b")
    m.reserve("b", 48)                                            # the pages that went back serve another request
    m.commit("b", 48)
    m.audit()
    m.release("a")
    m.release("b")
    m.audit()
    assert all(g.pool.num_free == g.pool.num_pages for g in m.groups)
    assert not CacheManager(needs[:1], 4, 8, 1, prefix_cache=True).prefix_cache
    with pytest.raises(ValueError, match="window or a chunk"):
        CacheNeed(paged=pair, window=3, chunk=4)


def test_cache_planes_and_roles_of_the_model(cpu_ops, tmp_path):
    runner = load_runner(_write(tmp_path / "m", MIXED), dtype="float32", device="cpu", page_size=8, max_tokens=64, max_requests=2)
    assert [(g.chunk, g.window, g.keep_first, g.planes) for g in runner.manager.groups] == [
        (0, 7, 3, [0]), (9, 0, 0, [1]), (0, 11, 5, [2]), (21, 0, 0, [3]), (0, 19, 26, [4])]
    mixers = [layer.mixer for layer in runner.model.layers]
    assert [m.values for m in mixers] == ["own", "first", "mixed", "mixed", "mixed"]
    assert [m.share is None for m in mixers] == [True, True, False, False, False]
    runner.step([StepEntry("r", [1, 2, 3], [])])
    straight = load_runner(_write(tmp_path / "s", STRAIGHT), dtype="float32", device="cpu", page_size=8, max_tokens=64, max_requests=2)
    assert {m.mixer.values for m in straight.model.layers} == {"own"} and not straight.manager.groups[0].gives_back


# ---- each mechanism alone, by hand and on the host twins ----

def test_masks_by_hand():
    seen = plain.window_mask(6, 2, 1).long().tolist()
    assert seen == [[1, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0], [1, 0, 1, 1, 0, 0], [1, 0, 0, 1, 1, 0],
                    [1, 0, 0, 0, 1, 1]]
    seen = plain.chunk_mask(5, 3).long().tolist()
    assert seen == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [1, 1, 1, 0, 0], [0, 0, 0, 1, 0], [0, 0, 0, 1, 1]]


def test_a_turn_leaves_the_root_mean_square():
    """What lets the kernel take a norm without weight before the turn: the two orders agree, also where
    only part of the head turns; with a weight they do not."""
    g = torch.Generator().manual_seed(2)
    x = torch.randn((9, 3, 20), generator=g, dtype=torch.float64)
    rot, pos = {"dims": 12, "base": 300.0}, torch.arange(9) * 7
    before = plain.rotate_halves(plain.unit_rms(x, 1e-5), pos, rot)
    assert torch.allclose(before, plain.unit_rms(plain.rotate_halves(x, pos, rot), 1e-5), atol=1e-12)
    w = torch.rand(20, generator=g, dtype=torch.float64) + 0.5
    assert not torch.allclose(plain.rotate_halves(plain.unit_rms(x, 1e-5) * w, pos, rot), before * w, atol=1e-2)
    pair = torch.tensor([[[1.0, 0.0, 5.0, 0.0, 2.0, 6.0]]], dtype=torch.float64)           # pairs (0, 2) and (1, 3)
    turned = plain.rotate_halves(pair, torch.tensor([1]), {"dims": 4, "base": 100.0})[0, 0]
    assert torch.allclose(turned[[0, 2]], torch.tensor([math.cos(1) - 5 * math.sin(1), 5 * math.cos(1) + math.sin(1)],
                                                       dtype=torch.float64), atol=1e-7)
    assert turned[[1, 3, 4, 5]].tolist() == [0.0, 0.0, 2.0, 6.0]


def _prepare_inputs(T, H, G, d, dv, half, seed=1, more=5, ahead=2):
    """Rows with `more` columns behind them, values to mix in with `ahead` columns before them."""
    g = torch.Generator().manual_seed(seed)
    rows = torch.randn((T, H * d + G * (d + dv) + more), generator=g) * 2.0
    first = torch.randn((T, G * dv + 2 * ahead), generator=g)[:, ahead:ahead + G * dv]
    qw, kw = torch.rand(d, generator=g) + 0.5, torch.rand(d, generator=g) + 0.5
    inv_freq = (torch.rand(half, generator=g) + 0.01) if half else None
    return rows, first, torch.tensor([0.37]), qw, kw, inv_freq


def test_prepare_twin_against_plain(cpu_ops):
    """Norms with and without a weight and mixed values of the preparation's twin, against the plain functions
    in the order that the design gives them."""
    T, H, G, d, dv, page, dims, base = 11, 4, 2, 14, 6, 4, 8, 70.0
    rows, first, share, qw, kw, _ = _prepare_inputs(T, H, G, d, dv, 0)
    inv_freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    pos, seq = torch.arange(5, 5 + T).int(), torch.zeros(T).int()
    table = torch.arange(4)[None].int()
    q0, k0 = rows[:, :H * d].double().view(T, H, d), rows[:, H * d:(H + G) * d].double().view(T, G, d)
    v0 = rows[:, (H + G) * d:(H + G) * d + G * dv].double()
    rot = {"dims": dims, "base": base}
    for weighted in (False, True):
        kc, vc = torch.zeros((4, G, page, d)), torch.zeros((4, G, dv, page))
        q = cpu_ops.turn_prepare(rows, None, H, G, d, dv, inv_freq, 1.0, pos, seq, torch.float32, table, kc, vc, norm_eps=1e-3,
                                 q_weight=qw if weighted else None, k_weight=kw if weighted else None, mix=(first, share))
        if weighted:
            want_q, want_k = (plain.rotate_halves(plain.unit_rms(x, 1e-3) * w.double(), pos, rot) for x, w in ((q0, qw), (k0, kw)))
        else:
            want_q, want_k = (plain.unit_rms(plain.rotate_halves(x, pos, rot), 1e-3) for x in (q0, k0))
        want_v = plain.mixed_values(v0, first.double(), share.double()).view(T, G, dv)
        at = pos.long()
        assert torch.allclose(q.double(), want_q, atol=1e-5)
        assert torch.allclose(kc[at // page, :, at % page].double(), want_k, atol=1e-5)
        assert torch.allclose(vc[at // page, :, :, at % page].double(), want_v, atol=1e-6)


def test_router_twin_and_plain_agree(cpu_ops):
    g = torch.Generator().manual_seed(1)
    for E, top, groups, keep in ((12, 3, 4, 2), (6, 2, 3, 2), (8, 8, 4, 4), (5, 1, 5, 1), (9, 2, 1, 1), (6, 4, 2, 2)):
        h, router = torch.randn(60, 24, generator=g), torch.randn(E, 24, generator=g) * 0.2
        correction = torch.randn(E, generator=g) * 0.1 - 0.1
        chosen, weights = cpu_ops.moe_route(h, router, top, scoring="softmax_groups", correction=correction,
                                            groups=groups, keep=keep, scale=1.7)
        at, share = plain.choose_experts(h.double() @ router.double().T, correction.double(), top, groups, keep, 1.7)
        assert torch.equal(chosen.long().sort(dim=-1).values, at.sort(dim=-1).values)
        assert torch.allclose(weights.double().sort(dim=-1).values, share.sort(dim=-1).values, atol=1e-6)


def test_choice_by_hand():
    """A group is judged by its best alone; the correction decides the choice and never a weight; what is
    left out counts as minus infinity when every corrected score is negative; weights sum to the scale."""
    z = torch.tensor([[0.5, 0.4, 0.6, -2.0, -1.0, -1.1]], dtype=torch.float64)             # groups (0,1) (2,3) (4,5)
    none = torch.zeros(6, dtype=torch.float64)
    at, share = plain.choose_experts(z, none, 2, 3, 1, 3.0)
    assert at[0].tolist() == [2, 3]              # group 0's two best sum higher, group 1 has the best one
    e = torch.exp(torch.tensor([0.6, -2.0], dtype=torch.float64))
    assert torch.allclose(share[0], 3.0 * e / e.sum())
    at, share = plain.choose_experts(z, torch.tensor([0.0, 0.0, 0.0, 0.0, 0.3, 0.3], dtype=torch.float64), 2, 3, 1, 1.0)
    assert sorted(at[0].tolist()) == [4, 5]
    e = torch.exp(torch.tensor([-1.0, -1.1], dtype=torch.float64))
    assert torch.allclose(share[0], e / e.sum())
    at, _ = plain.choose_experts(z, torch.full((6,), -5.0, dtype=torch.float64), 3, 3, 2, 1.0)
    assert sorted(at[0].tolist()) == [0, 1, 2]


def test_identity_experts_give_their_input_back(cpu_ops):
    g = torch.Generator().manual_seed(4)
    T, W, ff, E, back, top = 13, 10, 6, 2, 3, 3
    h = torch.randn((T, W), generator=g)
    gate_up, down = torch.randn((E, 2 * ff, W), generator=g), torch.randn((E, W, ff), generator=g)
    chosen = torch.stack([torch.randperm(E + back, generator=g)[:top] for _ in range(T)]).int()
    chosen[0] = torch.tensor([2, 3, 4])                             # nothing but identities
    weights = torch.rand((T, top), generator=g)
    w = {"x.e%d.%s" % (e, n): t for e in range(E)
         for n, t in (("gate", gate_up[e, 0::2]), ("up", gate_up[e, 1::2]), ("down", down[e]))}
    want = torch.zeros_like(h)
    for t in range(T):
        for k in range(top):
            e = int(chosen[t, k])
            want[t] += weights[t, k] * (plain.expert(h[t], w, "x.e%d" % e) if e < E else h[t])
    got = cpu_ops.moe_glu_experts(h, chosen, weights, gate_up, down, identity=back)
    assert torch.allclose(got, want, atol=1e-4) and torch.allclose(got[0], weights[0].sum() * h[0], atol=1e-5)


@pytest.mark.parametrize("change", [
    lambda c: [l["mixer"].pop("mask") for l in c["layers"]],
    lambda c: [l["mixer"]["mask"].update(size=l["mixer"]["mask"]["size"] + 1) for l in c["layers"]],
    lambda c: [l["mixer"]["mask"].update(keep_first=0) for l in c["layers"] if l["type"] == "attention_2"],
    lambda c: [l["mixer"].update(v_mix=False) for l in c["layers"]],
    lambda c: c["layers"][0]["mixer"].update(v_mix=True, vdim=48),
    lambda c: [l["mixer"].pop("rot") for l in c["layers"]],
    lambda c: [l["mlp"]["router"].update(groups={"count": 1, "keep": 1}) for l in c["layers"] if l["mlp"]],
    lambda c: [l["mlp"]["router"].update(scale=1.0) for l in c["layers"] if l["mlp"]],
])
def test_what_is_left_out_shows(tmp_path, change):
    """The truth itself: with these weights a mechanism left out, or an edge one token off, moves the logits far
    beyond what the comparisons below allow."""
    folder = _write(tmp_path / "m", MIXED)
    tokens = random_tokens(60, MIXED["vocab"], 9)
    config, w, want = _truth(folder, {"r": tokens})
    other = copy.deepcopy(config)
    change(other)
    if other["layers"][0]["mixer"]["vdim"] != config["layers"][0]["mixer"]["vdim"]:         # another first layer's values
        g = torch.Generator().manual_seed(3)
        w = dict(w, **{"l0.mix.v": torch.randn((48, 48), generator=g).double() * 0.2,
                       "l0.mix.o": torch.randn((48, 144), generator=g).double() * 0.2})
    got = plain.logits_of_sequence(other, w, tokens)
    d = got[-20:] - want["r"][-20:]
    assert float((d.pow(2).mean(dim=-1).sqrt() / want["r"][-20:].std(dim=-1)).max()) > 0.05


def test_logits_on_the_host_under_every_cutting(cpu_ops, folder):
    requests = _requests(folder)
    _, _, want = _truth(folder, requests)
    for make in (trace_whole, trace_tail_decoded, trace_portions, trace_mixed):
        steps = make(requests)
        runner = load_runner(folder, dtype="float32", device="cpu", page_size=8,
                             max_tokens=max_live_tokens(steps, page=8), max_requests=4)
        assert _off(run_trace(runner, steps), want, "float32") <= 1.0, make.__name__
        runner.manager.audit()
        assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.groups)


def test_layer_streams_on_the_host(cpu_ops, folder):
    config, w, _ = _truth(folder, {})
    tokens = random_tokens(37, config["vocab"], 4)
    streams, seen = [], []
    plain.logits_of_sequence(config, w, tokens, streams)
    runner = load_runner(folder, dtype="float32", device="cpu", page_size=8, max_tokens=64, max_requests=1)
    runner.model.observer = lambda i, x, pending: seen.append(x.double() + pending.double())
    runner.step([StepEntry("r", tokens, [])])
    assert len(seen) == len(streams) == len(config["layers"])
    for got, want in zip(seen, streams):
        assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max())


def test_values_do_not_leave_their_step(cpu_ops, tmp_path):
    """What the first mixing layer leaves for the others is gone behind the step, also where the same batch
    description runs twice."""
    folder = _write(tmp_path / "m", MIXED)
    runner = load_runner(folder, dtype="float32", device="cpu", page_size=8, max_tokens=64, max_requests=1)
    batches = []
    forward = runner.model.forward
    runner.model.forward = lambda batch, cache: (batches.append(batch), forward(batch, cache))[1]
    runner.step([StepEntry("r", [4, 8, 1], [2])])
    assert batches[0].carried == {}


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
    assert engine.runner.manager.num_free() == 60


def test_a_preempted_request_goes_on_where_it_was(cpu_ops, tmp_path):
    """Pages for one request and a half: one is preempted, its keys are made anew in other pages, and it
    generates what it would have alone."""
    folder = _write(tmp_path / "m", STRAIGHT)
    config, w, _ = _truth(folder, {})
    engine = SyncEngine(path=folder, dtype="float32", device="cpu", max_len=64, block_size=8, num_blocks=7,
                        max_num_seqs=2, max_num_tokens=32, chunked_prefill_size=16, enable_prefix_cache=False)
    prompts = [random_tokens(n, STRAIGHT["vocab"], 40 + n) for n in (26, 21)]
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
    names = load_file(str(tmp_path / "m" / "model.safetensors"))
    assert "l1.mix.vmix" not in names and tuple(names["l2.mix.vmix"].shape) == () and "l4.mlp.e6.down" in names


# ---- kernels against their twins ----

def _rand(shape, seed, dtype, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(dtype).cuda()


def _table(kv, page, seed, spare=3):
    """Block tables of sequences of kv[b] tokens over shuffled pages; and the number of pages."""
    blocks = [-(-n // page) for n in kv]
    order = torch.randperm(sum(blocks) + spare, generator=torch.Generator().manual_seed(seed)).tolist()
    table = torch.full((len(kv), max(blocks)), -1, dtype=torch.int32)
    for b, n in enumerate(blocks):
        for j in range(n):
            table[b, j] = order.pop()
    return table.cuda(), sum(blocks) + spare


def _packed(q_lens, kv):
    cu = torch.tensor([0] + list(np.cumsum(q_lens)), dtype=torch.int32).cuda()
    pos = torch.cat([torch.arange(L - m, L) for m, L in zip(q_lens, kv)]).int().cuda()
    seq = torch.cat([torch.full((m,), b) for b, m in enumerate(q_lens)]).int().cuda()
    return cu, torch.tensor(kv, dtype=torch.int32).cuda(), pos, seq


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,dv,half,page", [(4, 2, 16, 24, 4, 8), (16, 4, 64, 64, 32, 16), (3, 1, 7, 5, 0, 16), (2, 2, 1, 3, 0, 4),
                                                (6, 3, 128, 128, 16, 16), (2, 2, 300, 10, 129, 16), (8, 2, 96, 64, 48, 16),
                                                (4, 1, 192, 128, 96, 32), (5, 1, 130, 512, 65, 16), (3, 3, 512, 40, 256, 16),
                                                (12, 4, 256, 256, 128, 16), (9, 3, 128, 20, 4, 16)])
def test_prepare_kernel(dtype, H, G, d, dv, half, page):
    """Norms per head with a weight, without one and none, and values mixed or as they are: portions beside
    single tokens, single tokens alone, a long prompt, at positions beyond 100,000 too; rows that lie apart."""
    import torch_ops
    from qwen3_from_scratch_amd import ops

    cases = (([37, 1, 2, 5], [90, 41, 2, 66], 0), ([1, 1, 1, 1, 1], [9, 16, 67, 1, 33], 0), ([1100], [1101], 0), ([3], [9], 100000))
    # rows and values whose addresses allow 16-byte accesses (then sizes in steps of four take them), and others
    for (q_lens, kv, ahead), (more, before) in ((c, m) for c in cases for m in ((5, 2), (8, 4))):
        T = sum(q_lens)
        rows, first, share, qw, kw, inv_freq = (t if t is None else t.cuda()
                                                for t in _prepare_inputs(T, H, G, d, dv, half, more=more, ahead=before))
        if before == 4:                                  # a view again, as the product's rows give it
            first = torch.nn.functional.pad(first, (before, before))[:, before:-before]
        _, _, pos, seq = _packed(q_lens, kv)
        if ahead:
            table = torch.full((1, (ahead + 9) // page + 1), -1, dtype=torch.int32)
            table[0, ahead // page:] = torch.arange(table.shape[1] - ahead // page).int()
            table, pages, pos = table.cuda(), 8, pos + ahead
        else:
            table, pages = _table(kv, page, 7)
        for norm, mix in ((None, None), ("plain", (first, share)), ("weighted", (first, share)), ("weighted", None)):
            kw_args = dict(norm_eps=None if norm is None else 1e-3, mix=mix)
            if norm == "weighted":
                kw_args.update(q_weight=qw, k_weight=kw)
            out = []
            for impl in (ops, torch_ops):
                kc, vc = _rand((pages, G, page, d), 11, dtype), _rand((pages, G, dv, page), 12, dtype)
                q = impl.turn_prepare(rows, None, H, G, d, dv, inv_freq, 1.0, pos, seq, dtype, table, kc, vc, **kw_args)
                out.append((q, kc, vc))
            tol = (4e-5 if dtype == torch.float32 else 6e-2) * (4 if d == 1 else 1) + (2e-2 if ahead else 0.0)
            for a, b in zip(*out):
                assert float((a.float() - b.float()).abs().max()) <= tol, (norm, q_lens, more)


SPANS = [dict(chunk=9), dict(window=11, keep_first=5), dict(chunk=70), dict(window=50, keep_first=21), dict(window=1, keep_first=1),
         dict(chunk=1), dict(window=33, keep_first=140), dict(chunk=256), dict(window=300, keep_first=64), dict(window=20), dict()]


def _apart(a, b, dtype):
    """The largest difference in units of what rounding may leave: the softmax's weights and the result are rounded
    to bfloat16 there, so a number of size four is off by a thirty-second."""
    a, b = a.float(), b.float()
    bound = 2e-5 if dtype == torch.float32 else 2e-2 + 1e-2 * b.abs()
    return float(((a - b).abs() / bound).max())


def _give_back(table, kv, q_lens, page, chunk=0, window=0, keep_first=0):
    """The pages that the manager would have taken back by now."""
    for b, (n, L) in enumerate(zip(q_lens, kv)):
        first = L - n
        lo = first - first % chunk if chunk else max(0, first - window + 1) if window else 0
        table[b, -(-keep_first // page):max(lo // page, -(-keep_first // page))] = -1


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d,dv,page", [(4, 2, 16, 24, 8), (8, 2, 64, 64, 16), (6, 3, 96, 64, 16), (10, 5, 128, 128, 16),
                                           (8, 4, 192, 128, 32), (3, 1, 64, 128, 16), (32, 2, 128, 64, 64), (5, 5, 96, 96, 16),
                                           (5, 5, 10, 300, 16), (4, 4, 96, 64, 128), (2, 1, 192, 128, 16)])
def test_span_attention_kernels(dtype, H, G, d, dv, page):
    """Portions, short portions and single tokens in one step, over scattered pages of which those behind the
    span are gone, against the twin, with a gate per head and without; then single tokens alone; then portions of a
    long prompt, whose keys are shared out over blocks."""
    import torch_ops
    from qwen3_from_scratch_amd import ops

    q_lens, kv = [150, 1, 1, 2, 64, 3, 9, 1], [700, 333, 1, 257, 64, 12, 1500, 71]
    T = sum(q_lens)
    cu, kvl, pos, seq = _packed(q_lens, kv)
    q = _rand((T, H, d), 3, dtype, 2.0)
    wide = _rand((T, H + 7), 5, torch.float32, 2.0)
    for span in SPANS:
        table, pages = _table(kv, page, 17)
        kc, vc = _rand((pages, G, page, d), 21, dtype), _rand((pages, G, dv, page), 22, dtype)
        _give_back(table, kv, q_lens, page, **span)
        for gate in (None, wide[:, 3:3 + H]):
            args = (kc, vc, table, cu, kvl, seq, pos, max(q_lens), max(kv), d ** -0.5, 0.0)
            a = ops.softcap_attention(q, *args, gate=gate, values_transposed=True, span=True, **span)
            b = torch_ops.softcap_attention(q, *args, gate=gate, values_transposed=True, **span)
            assert _apart(a, b, dtype) <= 1.0, (span, gate is not None)
        # single tokens alone: the decoding kernel with the keys shared out over blocks
        table, _ = _table(kv, page, 17)
        _give_back(table, kv, [1] * len(kv), page, **span)
        n = len(kv)
        ones, _, pos1, seq1 = _packed([1] * n, kv)
        args = (kc, vc, table, ones, kvl, seq1, pos1, 1, max(kv), d ** -0.5, 0.0)
        a = ops.softcap_attention(q[:n], *args, gate=wide[:n, :H], values_transposed=True, span=True, **span)
        b = torch_ops.softcap_attention(q[:n], *args, gate=wide[:n, :H], values_transposed=True, **span)
        assert _apart(a, b, dtype) <= 1.0, span
    kv, q_lens = [5000], [300]
    cu, kvl, pos, seq = _packed(q_lens, kv)
    table, pages = _table(kv, page, 19)
    kc, vc, q = _rand((pages, G, page, d), 21, dtype), _rand((pages, G, dv, page), 22, dtype), _rand((300, H, d), 3, dtype, 2.0)
    for span in (dict(chunk=4800), dict(window=4000, keep_first=100), dict(window=3000, keep_first=2500), dict()):
        args = (kc, vc, table, cu, kvl, seq, pos, 300, 5000, d ** -0.5, 0.0)
        a = ops.softcap_attention(q, *args, gate=wide[:1, :H].expand(300, H).contiguous(), values_transposed=True, min_q_len=300,
                                  span=True, **span)
        b = torch_ops.softcap_attention(q, *args, gate=wide[:1, :H].expand(300, H), values_transposed=True, **span)
        assert _apart(a, b, dtype) <= 1.0, span


@pytest.mark.gpu
def test_spans_of_these_sizes_run_on_the_matrix_cores():
    from qwen3_from_scratch_amd import ops

    for d, dv in ((64, 64), (64, 128), (96, 64), (96, 96), (128, 64), (128, 128), (192, 128)):
        assert ops.span_sizes(8, 2, d, dv, 16, torch.bfloat16) and not ops.span_sizes(8, 2, d, dv, 16, torch.float32)
    for d, dv in ((192, 64), (80, 64), (64, 96), (256, 256)):
        assert not ops.span_sizes(8, 2, d, dv, 16, torch.bfloat16)
    assert not ops.span_sizes(34, 2, 64, 64, 16, torch.bfloat16) and not ops.span_sizes(8, 2, 64, 64, 24, torch.bfloat16)


@pytest.mark.gpu
@pytest.mark.parametrize("rows", [1, 2, 9, 40])
@pytest.mark.parametrize("dtype,d,dv", [(torch.float32, 64, 48), (torch.bfloat16, 64, 64), (torch.bfloat16, 96, 64), (torch.bfloat16, 192, 128)])
def test_span_edges(dtype, d, dv, rows):
    """A query that stands on one key gets its value if it sees it and nothing of it if it does not: the first
    token of a window and the one before it, the last of the first tokens and the one behind it, a chunk's first
    token and the one before it, page ends, hundreds of positions back; decoded alone or as a portion's last row."""
    from qwen3_from_scratch_amd import ops

    H, G, page, L = 4, 2, 16, 900
    table, pages = _table([L], page, 31)
    unit = lambda n, s: torch.nn.functional.normalize(_rand((L, G, n), s, torch.float32), dim=-1)     # noqa: E731
    keys, values = unit(d, 1), unit(dv, 2)
    kc, vc = torch.zeros((pages, G, page, d), dtype=dtype).cuda(), torch.zeros((pages, G, dv, page), dtype=dtype).cuda()
    at = torch.arange(L).cuda()
    pg = table[0, at // page].long()
    kc[pg, :, at % page] = keys.to(dtype)
    vc[pg, :, :, at % page] = values.to(dtype)
    for chunk, window, keep in ((0, 100, 20), (0, 33, 32), (0, 17, 70), (120, 0, 0), (64, 0, 0), (0, 200, 1)):
        size = chunk or window
        for i in {0, 1, keep - 1, keep, size - 1, size, size + keep, 2 * size - 1, 2 * size, 527, 528, 899} - {-1}:
            n = min(rows, i + 1)
            cu, kvl, pos, seq = _packed([n], [i + 1])
            lo = i - i % chunk if chunk else i - window + 1
            cases = {i, lo, lo - 1, keep - 1, keep, 0, i // page * page, i // page * page - 1, (keep + lo) // 2}
            for j in sorted(c for c in cases if 0 <= c <= i):
                seen = j >= lo or j < keep
                q = torch.zeros((n, H, d), dtype=dtype).cuda()
                q[-1] = (keys[j] * 60.0).repeat_interleave(H // G, dim=0).to(dtype)
                got = ops.softcap_attention(q, kc, vc, table, cu, kvl, seq, pos, n, i + 1, 1.0, 0.0, window=window, min_q_len=n,
                                            values_transposed=True, chunk=chunk, keep_first=keep, span=True)
                share = (got[-1].view(H, dv).float() * values[j].repeat_interleave(H // G, dim=0)).sum(dim=-1)
                if seen:
                    assert float((share - 1.0).abs().max()) <= 2e-2, (chunk, window, keep, i, j)
                else:
                    assert float(share.abs().max()) <= 0.75, (chunk, window, keep, i, j)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,width,E,top,groups,keep,more", [
    (1, 64, 12, 4, 4, 3, 1), (77, 48, 6, 2, 3, 2, 0), (300, 192, 72, 6, 8, 3, 0), (9, 33, 3, 1, 3, 1, 2),
    (50, 40, 8, 8, 4, 4, 1), (40, 32, 10, 3, 1, 1, 0), (33, 64, 130, 5, 65, 4, 1), (20, 32, 1, 1, 1, 1, 0)])
def test_grouped_softmax_router_kernel(dtype, T, width, E, top, groups, keep, more):
    """The choice against the plain function, from the logits the kernel's own product leaves; corrections of
    the size of the scores, so that many corrected scores are negative."""
    from qwen3_from_scratch_amd import ops

    h, router = _rand((T, width), 1, dtype), _rand((E + more, width), 2, dtype, 0.3)
    correction = _rand((E,), 3, torch.float32, 1.0 / E) - 1.0 / E
    chosen, weights, _ = ops.moe_route(h, router, top, scoring="softmax_groups", correction=correction, groups=groups,
                                       keep=keep, experts=E, scale=2.5)
    z = ops.linear(h, router, out_dtype=torch.float32).double().cpu()[:, :E]
    at, _ = plain.choose_experts(z, correction.double().cpu(), top, groups, keep, 2.5)
    s = torch.softmax(z, dim=-1)
    choice = s + correction.double().cpu()
    best_of_group = choice.view(T, groups, -1).max(dim=-1).values
    for t in range(T):
        got, want = sorted(chosen[t].tolist()), sorted(at[t].tolist())
        order = chosen[t].long().cpu()
        if got != want:                                  # only where two scores, or two groups, all but tie
            near = torch.cat((choice[t], best_of_group[t])).sort().values
            assert float((near[1:] - near[:-1]).min()) < 1e-6, t
        else:
            assert bool((choice[t, order][:-1] >= choice[t, order][1:] - 1e-7).all())       # in falling order
        share = s[t, order]
        assert torch.allclose(weights[t].double().cpu(), 2.5 * share / share.sum(), atol=1e-5)
    assert all(len(set(row)) == top for row in chosen.tolist())
    size = E // groups
    assert all(len({e // size for e in row}) <= keep for row in chosen.tolist())


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,width,ff,E,back,top", [(1, 64, 32, 7, 2, 3), (50, 48, 24, 5, 1, 2), (333, 128, 96, 6, 6, 3),
                                                   (17, 40, 20, 1, 3, 4), (700, 96, 160, 3, 2, 2), (900, 64, 64, 2, 1, 2),
                                                   (300, 64, 640, 100, 4, 3), (20, 64, 640, 100, 4, 3)])
def test_experts_with_identities(dtype, T, width, ff, E, back, top):
    import torch_ops
    from qwen3_from_scratch_amd import ops

    h = _rand((T, width), 1, dtype)
    gate_up, down = _rand((E, 2 * ff, width), 2, dtype, width ** -0.5), _rand((E, width, ff), 3, dtype, ff ** -0.5)
    chosen, weights = torch_ops.moe_route(h, _rand((E + back, width), 4, dtype), top, scoring="sigmoid")
    if back >= top:
        chosen[0] = torch.arange(E, E + top).int()      # a token without any expert
    a = ops.moe_glu_experts(h, chosen, weights, gate_up, down, identity=back)
    b = torch_ops.moe_glu_experts(h, chosen, weights, gate_up, down, identity=back)
    assert float((a.float() - b.float()).abs().max()) <= (3e-5 if dtype == torch.float32 else 5e-2)
    if back >= top:                                     # and a step of nothing but identities
        chosen[:] = torch.arange(E, E + top).int()
        a = ops.moe_glu_experts(h, chosen, weights, gate_up, down, identity=back)
        assert float((a.float() - h.float() * weights.sum(dim=-1, keepdim=True)).abs().max()) <= (1e-5 if dtype == torch.float32 else 4e-2)


# ---- the model on the GPU ----

@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_logits_under_every_cutting(folders, dtype):
    folder = folders[dtype]
    requests = _requests(folder, lengths=(70, 9, 141, 330, 25, 2, 1))
    _, _, want = _truth(folder, requests)
    for make in (trace_whole, trace_tail_decoded, trace_portions, trace_mixed):
        steps = make(requests)
        runner = load_runner(folder, dtype=dtype, device="cuda", page_size=16,
                             max_tokens=max_live_tokens(steps, page=16), max_requests=4)
        assert _off(run_trace(runner, steps), want, dtype) <= 1.0, make.__name__
        assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.groups)


@pytest.mark.gpu
def test_layer_streams(folder):
    """The float32 engine's residual stream behind every layer against the plain one's."""
    config, w, _ = _truth(folder, {})
    tokens = random_tokens(45, config["vocab"], 4)
    streams, seen = [], []
    plain.logits_of_sequence(config, w, tokens, streams)
    runner = load_runner(folder, dtype="float32", device="cuda", page_size=16, max_tokens=64, max_requests=1)
    runner.model.observer = lambda i, x, pending: seen.append((x.double() + pending.double()).cpu())
    runner.step([StepEntry("r", tokens, [])])
    assert len(seen) == len(streams)
    for got, want in zip(seen, streams):
        assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max())


@pytest.mark.gpu
def test_long_decoding_and_first_tokens(folders):
    """A request decoded token by token from its second token on, through graph replays, page ends, chunks and
    windows that move on, beside a request that joins late into pages that went back."""
    for dtype in ("float32", "bfloat16"):
        folder = folders[dtype]
        vocab = load_model_config(folder).vocab
        requests = {"long": random_tokens(300, vocab, 7), "short": random_tokens(40, vocab, 8)}
        _, _, want = _truth(folder, requests)
        runner = load_runner(folder, dtype=dtype, device="cuda", page_size=16, max_tokens=352, max_requests=2)
        steps = []
        for i in range(300):
            entries = [("long", [requests["long"][i]], [0])]
            if 200 <= i < 240:
                entries.append(("short", [requests["short"][i - 200]], [0]))
            steps.append((entries, ["short"] if i == 239 else ["long"] if i == 299 else []))
        assert _off(run_trace(runner, steps), want, dtype) <= 1.0


def _far_model(folder, kind):
    """One layer of either attention. Queries are the keys' negatives, and the embedding of one token (`asks`) is
    another's (`holds`) negative: a query of the one stands on the keys of the other. Nothing turns. The one that
    holds stands early, among the first tokens or early in a long chunk; the one that asks near the end, in
    that chunk's last place, and once more in the next chunk's first, where it finds nothing."""
    mixer = (_chunked(4, 2, 64, 64, 590, scale=0.25, v_mix=False) if kind == "attention"
             else _windowed(4, 2, 96, 64, 40, 38, scale=0.25, v_mix=False))
    data = _model(131, 128, [_layer(mixer, _moe(4, 2, 6, 64))])
    folder = _write(folder, data, std=0.1)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    d = mixer["mixer"]["dim"]
    tensors["l0.mix.q"] = -tensors["l0.mix.k"].view(2, d, -1).repeat_interleave(2, dim=0).reshape(4 * d, -1).contiguous()
    if kind == "attention_2":
        tensors["l0.mix.q.norm"] = tensors["l0.mix.k.norm"].clone()
    asks, holds = data["vocab"] - 1, data["vocab"] - 2
    tensors["embed"][asks] = -tensors["embed"][holds]
    save_file(tensors, path, metadata={"format": "pt"})
    tokens = [min(t, holds - 1) for t in random_tokens(600, data["vocab"], 31)]
    tokens[37] = holds
    tokens[589] = tokens[590] = asks
    return folder, tokens


@pytest.mark.parametrize("kind", ["attention", "attention_2"])
def test_the_far_model_leans_on_its_far_key(tmp_path, kind):
    """The truth of the test below: without the early key the row that asks is another one; across the chunk's
    end it is the same."""
    folder, tokens = _far_model(tmp_path / "m", kind)
    _, _, want = _truth(folder, {"far": tokens, "cut": tokens[:37] + [3] + tokens[38:]})
    moved = [float((want["far"][p] - want["cut"][p]).pow(2).mean().sqrt() / want["far"][p].std()) for p in (589, 590)]
    assert moved[0] > 0.3 and (moved[1] > 0.3 if kind == "attention_2" else moved[1] == 0.0)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["attention", "attention_2"])
def test_a_far_key_carries_the_asking_row(tmp_path, dtype, kind):
    folder, tokens = _far_model(tmp_path / "m", kind)
    _, _, want = _truth(folder, {"far": tokens})
    for steps in (trace_whole({"far": tokens}), trace_tail_decoded({"far": tokens}, tail=14),
                  trace_portions({"far": tokens}, sizes=(130, 37, 2, 261, 64, 3))):
        runner = load_runner(folder, dtype=dtype, device="cuda", page_size=16, max_tokens=608, max_requests=1)
        got = run_trace(runner, steps)
        for p in range(585, 600):
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
        assert engine.runner.manager.num_free() == 30


@pytest.mark.gpu
def test_logits_do_not_depend_on_pages_and_company(folders):
    """The same request alone and beside others, into a fresh cache and into pages that others have used: the same
    numbers to rounding, single tokens bit for bit where the same kernels with the same shares run."""
    folder = folders["bfloat16"]
    vocab = load_model_config(folder).vocab
    runner = load_runner(folder, dtype="bfloat16", device="cuda", page_size=16, max_tokens=640, max_requests=3)
    tokens = random_tokens(150, vocab, 3)
    rows = []
    for _ in range(2):
        rows.append(runner.step([StepEntry("a", tokens, [149])]).clone())
        runner.step([StepEntry("b", random_tokens(90, vocab, 4), [])])
        rows.append(runner.step([StepEntry("a", [5], [0])]).clone())
        runner.finish("a")
        runner.finish("b")
        runner.step([StepEntry("c", random_tokens(333, vocab, 6), [])])
        runner.finish("c")
    assert torch.equal(rows[0], rows[2]) and torch.equal(rows[1], rows[3])


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
            data = np.fromfile(os.path.join(out, "%d.f32" % i), dtype="<f4").reshape(len(wanted), -1)
            for key, row in zip(wanted, data):
                got[key] = torch.from_numpy(row.copy())
    assert _off(got, want, dtype) <= 1.0


@pytest.mark.gpu
def test_command_line_generates(tmp_path):
    folder = _write(tmp_path / "m", CORES)
    config, w, _ = _truth(folder, {})
    prompt = random_tokens(50, CORES["vocab"], 12)
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
