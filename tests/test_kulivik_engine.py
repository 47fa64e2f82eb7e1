"""Kulivik decoders through the engine (scheduler, paged cache, state slots, step function) against the plain
implementation in ``kulivik_oracle.py``. Small configurations with random weights made here; every test runs
on the CPU ops and, marked ``gpu``, on the HIP kernels."""
import copy
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import kulivik_oracle as oracle
from llm_consensus_amd._native import core
from llm_consensus_amd.engine.engine import Engine
from llm_consensus_amd.models.hybrid import HybridModel, config_from_dict, config_to_dict

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
BS = 16
ROOT = Path(__file__).resolve().parents[1]
DENSE = {"kind": "dense", "ff": 56, "limit": 0.7}


def moe(experts=5, top=2, ff=24):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def conv(heads=4, kv=2, dim=12, vdim=10, taps=3, scale=0.3, v_mix=True, mlp=DENSE):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "conv": taps,
                                           "v_mix": v_mix}, "mlp": mlp}


def win(heads=4, kv=2, dim=12, vdim=10, size=21, keep=3, rot=6, base=500.0, scale=0.3, cap=4.0, v_mix=True, mlp=DENSE):
    return {"type": "attention_2", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap,
                                             "mask": {"size": size, "keep_first": keep}, "rot": {"dims": rot, "base": base},
                                             "v_mix": v_mix}, "mlp": mlp}


def par(heads=4, kv=2, dim=10, vdim=8, scale=0.3, coef=0.6, every=8, rheads=3, rdim=6, rvdim=12, decay=None, ls=0.7, rs=1.3, mlp=DENSE):
    if decay is None:
        decay = [round(0.3 + 0.69 * (i + 1) / rheads, 3) for i in range(rheads)]
    return {"type": "parallel", "mixer": {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
                                                   "q_temp": {"coef": coef, "every": every}}, "left_scale": ls, "right_scale": rs,
                                          "right": {"heads": rheads, "dim": rdim, "vdim": rvdim, "decay": decay}}, "mlp": mlp}


def config(layers, width=40, vocab=67, eps=1e-5, logit_scale=1.7, cap=9.0):
    return {"architecture": "Kulivik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "logit_softcap": cap, "layers": layers}


MIXED = config([par(mlp=moe()), win(vdim=20, kv=1, v_mix=True), conv(), conv(heads=3, kv=1, vdim=20, taps=4, mlp=moe(7, 3)),
                win(heads=2, kv=2, size=9, keep=5, rot=12, v_mix=False, mlp=None), par(heads=2, kv=1, rheads=2, decay=[0.999, 0.2], mlp=None),
                win(size=40, keep=0, cap=30.0, mlp=moe(3, 1))])


def build(cfg, device, dtype=torch.float32, seed=0, blocks=24, slots=4, weights=None, **kw):
    W = weights if weights is not None else oracle.random_weights(cfg, seed)
    model = HybridModel(config_from_dict(cfg, "test", {k: tuple(v.shape) for k, v in W.items()}), device, dtype)
    model.set_weights(lambda n: W[n])
    eng = Engine(model, num_kv_blocks=blocks, block_size=BS, max_batch_seqs=kw.pop("max_batch_seqs", slots),
                 state_slots=slots, max_model_len=blocks * BS, enable_prefix_cache=False,
                 use_graphs=kw.pop("use_graphs", False), pipeline_decode=kw.pop("pipeline_decode", False), **kw)
    return eng, W


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def replay_alone(eng, toks, cuts):
    """One request fed in portions of the given sizes (the rest one token at a time); all logits."""
    rid, at, out = eng.replay_open(), 0, []
    sizes = list(cuts) + [1] * (len(toks) - sum(cuts))
    for n in sizes:
        out.append(eng.replay_step([(rid, toks[at:at + n], list(range(n)))]))
        at += n
    eng.replay_close(rid)
    return np.concatenate(out)


def row_errs(got, want):
    """Row errors: mean taken off, RMS over the vocabulary, against the mean RMS of the wanted rows."""
    want = want.numpy() if hasattr(want, "numpy") else want
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean(-1)).mean()


def rel_err(got, want):
    return float(row_errs(got, want).max())


def close(got, want, dtype):
    """32-bit: every row to rounding. bf16 (rounding errors of a percent or two, now and then a row whose gates and
    norms magnify them): the typical row close, no row far."""
    e = row_errs(got, want)
    return float(e.max()) < 2e-4 if dtype == torch.float32 else float(np.median(e)) < 4e-2 and float(e.max()) < 0.2


def steady(W):
    """Router biases far apart, so that 16-bit rounding never changes which experts are chosen."""
    for k in W:
        if k.endswith("router"):
            W[k] = (0.05 * W[k].float()).to(W[k].dtype)
        if k.endswith("router.b"):
            W[k] = torch.linspace(2.0, -2.0, W[k].numel())[torch.randperm(W[k].numel(), generator=torch.Generator().manual_seed(1))].to(W[k].dtype)
    return W


def _whole_prompt(cfg, device, dtype, name, cuts=None, seed=0, n=45):
    W = oracle.random_weights(cfg, seed)
    if dtype == torch.bfloat16:
        W = steady(W)
    eng, W = build(cfg, device, dtype, weights=W)
    toks = tokens(n if cuts is None else sum(cuts) + 3, cfg["vocab"], 3)
    got = replay_alone(eng, toks, cuts or [len(toks)])
    assert close(got, oracle.forward(cfg, W, toks), dtype), name


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,layers", [
    ("attention: grouped heads, values narrower than keys; values wider, two taps", [conv(), conv(heads=6, kv=3, dim=10, vdim=16, taps=2, v_mix=False)]),
    ("attention: one key head, four taps; as many key heads as heads, one tap", [conv(heads=4, kv=1, dim=16, vdim=16, taps=4, v_mix=False), conv(heads=3, kv=3, dim=8, vdim=4, taps=1, v_mix=False)]),
    ("attention: widths of the matrix-core kernel, six taps", [conv(heads=4, kv=2, dim=16, vdim=32, taps=6), conv(heads=8, kv=4, dim=32, vdim=16, taps=3)]),
    ("window attention: grouped heads, part of the head turns", [win(), win(heads=6, kv=3, dim=10, vdim=16, size=5, keep=2, rot=4, v_mix=False)]),
    ("window attention: one key head; nothing turns, no kept keys; the whole head turns", [win(heads=4, kv=1, dim=16, vdim=16, size=30, keep=1, rot=16, v_mix=False),
                                                                                          win(heads=3, kv=3, dim=7, vdim=4, size=19, keep=0, rot=0, v_mix=False),
                                                                                          win(heads=2, kv=2, dim=8, vdim=8, rot=8, v_mix=False)]),
    ("window attention: widths of the matrix-core kernel, more kept keys than a tile holds", [win(heads=4, kv=2, dim=16, vdim=32, size=7, keep=21, rot=8),
                                                                                             win(heads=8, kv=4, dim=32, vdim=16, size=18, keep=5, rot=32)]),
    ("window attention: a window of one, longer than the prompt, a cap that always binds, one that never does", [win(size=1, keep=4), win(size=500, keep=7, cap=0.3), win(cap=1e4)]),
    ("parallel: grouped heads; one key head, one decay", [par(), par(heads=3, kv=1, dim=8, vdim=16, rheads=1, rdim=5, rvdim=3)]),
    ("parallel: widths of the matrix-core kernel, six heads (slopes of no power of two), equal sizes on both sides", [par(heads=6, kv=3, dim=16, vdim=16, rheads=6, rdim=16, rvdim=16), par(heads=8, kv=8, dim=8, vdim=16)]),
    ("parallel: decays of zero and one, a key width past a wave, no temperature", [par(rheads=3, rdim=70, rvdim=66, decay=[0.0, 1.0, 0.95], coef=0.0)]),
    ("values mixed across both kinds, a layer between that does not mix, three and more mixing layers", [win(v_mix=False), par(), win(vdim=12, kv=2), conv(vdim=24, kv=1), conv(v_mix=False, vdim=6), win(vdim=8, kv=3, heads=3)]),
    ("one mixing layer only, which has nothing to mix in", [conv(v_mix=False), win()]),
    ("experts: one of many, all of few, many", [conv(mlp=moe(9, 1)), win(mlp=moe(3, 3)), par(mlp=moe(40, 5, 7))]),
    ("layers without a feed-forward", [par(mlp=None), conv(mlp=None), win(mlp=None)]),
    ("one layer", [win(mlp=moe())]),
])
def test_each_mechanism_whole_prompt(device, dtype, name, layers):
    _whole_prompt(config(layers), device, dtype, name)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_depths_the_mfma_products_take(device, dtype):
    """Widths of 64 / 128 with feed-forwards of 64 / 192 units and experts of 64: in bf16 on the GPU the projections go
    through the packed MFMA kernels (depths in multiples of 64, fp32 epilogues, biases), the experts through the grouped ones."""
    for width, ff in ((64, 64), (128, 192)):
        d = {"kind": "dense", "ff": ff, "limit": 1.1}
        cfg = config([win(heads=4, kv=2, dim=16, vdim=16, rot=8, mlp=d), conv(heads=4, kv=2, dim=16, vdim=16, mlp=moe(6, 2, 64)),
                      par(heads=4, kv=2, dim=16, vdim=16, rheads=4, rdim=16, rvdim=16, mlp=moe(33, 3, 64))], width=width, vocab=70)
        _whole_prompt(cfg, device, dtype, f"mfma depths {width}", cuts=[40, 2, 17])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_deep_products_and_a_long_portion(device, dtype):
    """Width 1024 (the bf16 products of a few rows split their depth over workgroups), fused projection widths that
    are no multiple of 32, a portion of a few hundred rows (scanned in segments), a short one, decoded tokens."""
    cfg = config([par(heads=3, kv=1, dim=16, vdim=16, rheads=2, rdim=24, rvdim=40, mlp={"kind": "dense", "ff": 72, "limit": 0.9}),
                  win(heads=2, kv=1, dim=24, vdim=16, size=100, keep=9, rot=8, mlp=moe(4, 2, 64)), conv(heads=2, kv=1, dim=24, vdim=16, mlp=None)],
                 width=1024, vocab=90)
    W = steady(oracle.random_weights(cfg, 0))
    eng, W = build(cfg, device, dtype, weights=W)
    toks = tokens(300, cfg["vocab"], 3)
    assert close(replay_alone(eng, toks, [270, 20]), oracle.forward(cfg, W, toks), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_widths_the_vector_accesses_do_not_take(device):
    """A width and channel counts that are multiples of nothing."""
    cfg = config([par(heads=3, kv=1, dim=5, vdim=3, rheads=1, rdim=3, rvdim=7, mlp=moe(3, 2, 5)), win(heads=1, kv=1, dim=7, vdim=5, rot=2),
                  conv(heads=1, kv=1, dim=3, vdim=5, mlp={"kind": "dense", "ff": 9, "limit": 0.5})], width=37, vocab=41)
    _whole_prompt(cfg, device, torch.float32, "odd widths", cuts=[13, 2, 9])


@pytest.mark.parametrize("device", DEVICES)
def test_constants_that_could_pass_for_one(device):
    """Scales, caps, limits and mixing shares of 1, then other constants with the SAME tensors; every constant on its
    own moves the logits of the oracle; a large eps."""
    layers = [win(scale=1.0, cap=1.0, mlp={"kind": "dense", "ff": 20, "limit": 1.0}), conv(scale=1.0, mlp=None),
              par(scale=1.0, coef=1.0, every=1, ls=1.0, rs=1.0, decay=[1.0, 1.0, 1.0])]
    cfg = config(layers, eps=1.0, logit_scale=1.0, cap=1.0)
    W = oracle.random_weights(cfg, 4)
    W["l1.mix.vmix"] = torch.tensor(1.0).to(torch.bfloat16)
    toks = tokens(30, cfg["vocab"], 9)
    base = oracle.forward(cfg, W, toks)
    eng, _ = build(cfg, device, weights=W)
    assert rel_err(replay_alone(eng, toks, [17]), base) < 2e-4

    def put(c, path, v):
        for k in path[:-1]:
            c = c[k]
        c[path[-1]] = v
    changes = [(("layers", 0, "mixer", "scale"), 0.4), (("layers", 0, "mixer", "softcap"), 2.5), (("layers", 0, "mlp", "limit"), 0.2),
               (("layers", 1, "mixer", "scale"), 0.3), (("layers", 2, "mixer", "left", "scale"), 0.4),
               (("layers", 2, "mixer", "left", "q_temp", "coef"), 0.2), (("layers", 2, "mixer", "left", "q_temp", "every"), 7),
               (("layers", 2, "mixer", "left_scale"), 0.5), (("layers", 2, "mixer", "right_scale"), 0.4),
               (("layers", 2, "mixer", "right", "decay"), [0.5, 0.9, 0.2]), (("logit_scale",), 2.0), (("logit_softcap",), 5.0),
               (("norm", "eps"), 1e-3)]
    for path, v in changes:
        other = copy.deepcopy(cfg)
        put(other, path, v)
        want = oracle.forward(other, W, toks)
        assert rel_err(want.numpy(), base) > 5e-3, path
        eng, _ = build(other, device, weights=W)
        assert rel_err(replay_alone(eng, toks, [17]), want) < 2e-4, path


@pytest.mark.parametrize("device", DEVICES)
def test_residual_stream_after_every_layer(device):
    eng, W = build(MIXED, device)
    toks = tokens(20, MIXED["vocab"], 5)
    taps, rid = [], eng.replay_open()
    eng.replay_step([(rid, toks, [])], taps=taps)
    _, want = oracle.forward(MIXED, W, toks, return_layers=True)
    assert len(taps) == len(want) == 7
    for i, t in enumerate(taps):
        torch.testing.assert_close(t.cpu().double(), want[i], atol=2e-4, rtol=2e-4, msg=f"layer {i}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[], [1], [40], [2, 2, 3, 2, 17, 2], [11, 1, 1, 12, 13], [5, 7, 12, 16, 1, 15, 2]])
def test_portions_and_token_by_token_decoding(device, dtype, cuts):
    """The same logits whether the prompt comes whole, in portions down to two tokens (cut inside pages of 16, inside
    windows and inside the reach of the convolutions), or one token at a time."""
    eng, W = build(MIXED, device, dtype, weights=steady(oracle.random_weights(MIXED, 0)))
    toks = tokens(70, MIXED["vocab"], 7)
    assert close(replay_alone(eng, toks, cuts), oracle.forward(MIXED, W, toks), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_past_pages_and_windows(device):
    eng, W = build(MIXED, device)
    toks = tokens(120, MIXED["vocab"], 11)
    assert rel_err(replay_alone(eng, toks, [3]), oracle.forward(MIXED, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_reused_pages_and_slots(device, dtype):
    """Up to four live requests, portions beside single tokens, in a pool too small for all of them at once: requests
    end, others take their pages and state slots (which are never cleared)."""
    eng, W = build(MIXED, device, dtype, blocks=12, slots=4, weights=steady(oracle.random_weights(MIXED, 0)))
    V = MIXED["vocab"]
    reqs = {n: tokens(L, V, 20 + i) for i, (n, L) in enumerate([("a", 50), ("b", 33), ("c", 1), ("d", 47), ("e", 40),
                                                                ("f", 18), ("g", 60)])}
    want = {n: oracle.forward(MIXED, W, t) for n, t in reqs.items()}
    sched = [[("a", 20), ("b", 2)], [("a", 1), ("b", 13), ("c", 1)], [("a", 1), ("b", 1), ("d", 30)],
             [("a", 28), ("d", 1)], [("b", 17), ("d", 16), ("e", 9)], [("e", 1)], [("e", 30), ("f", 18)],
             [("g", 33)], [("g", 1)], [("g", 26)]]
    at, rid, got = {n: 0 for n in reqs}, {}, {n: [] for n in reqs}
    free0 = eng.kvm.stats().blocks_free
    for step in sched:
        entries = []
        for n, k in step:
            if n not in rid:
                rid[n] = eng.replay_open()
            entries.append((rid[n], reqs[n][at[n]:at[n] + k], list(range(k))))
        lg = eng.replay_step(entries)
        o = 0
        for n, k in step:
            got[n].append(lg[o:o + k])
            o += k
            at[n] += k
            if at[n] == len(reqs[n]):
                eng.replay_close(rid[n])
    assert all(at[n] == len(reqs[n]) for n in reqs)
    assert eng.kvm.stats().blocks_free == free0
    for n in reqs:
        assert close(np.concatenate(got[n]), want[n], dtype), n


@pytest.mark.parametrize("device", DEVICES)
def test_previous_inputs_across_portions_single_tokens_and_reused_slots(device):
    """What a sequence keeps besides keys and values: the previous input row (shift weights of exactly one: the mixer
    reads ONLY the token before), the last inputs of a convolution of five taps whose OLDEST tap dominates, a memory
    that never decays. Portions shorter than the reach of the convolution, then single tokens; one state slot that
    three requests use one after another, so that anything left from the one before would show."""
    cfg = config([conv(taps=5, mlp=None), par(rheads=2, decay=[1.0, 1.0], mlp=None)])
    W = oracle.random_weights(cfg, 9)
    for i in (0, 1):
        W[f"l{i}.shift"] = torch.ones_like(W[f"l{i}.shift"])
    for n in ("q", "k", "v"):
        w = 0.1 * W[f"l0.mix.{n}.conv"].float()
        w[:, 0] = 1.5
        W[f"l0.mix.{n}.conv"] = w.to(torch.bfloat16)
    eng, _ = build(cfg, device, weights=W, slots=1, blocks=4)
    for seed, cuts in ((1, [2, 2, 3, 2, 2, 9]), (2, [1, 3, 2]), (3, [4, 4, 4, 11]), (4, [])):
        toks = tokens(30, cfg["vocab"], seed)
        assert rel_err(replay_alone(eng, toks, cuts), oracle.forward(cfg, W, toks)) < 2e-4, cuts


def _bare(layer, scale, **kw):
    layer = copy.deepcopy(layer)
    layer["mixer"].update(scale=scale, **kw)
    return layer


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size,keep", [(5, 0), (5, 3), (16, 1), (21, 18), (16, 16), (3, 40)])
@pytest.mark.parametrize("decode_from", [0, 3, 30])
def test_the_windows_edge_and_the_kept_first_keys_at_every_place_and_page_border(device, size, keep, decode_from):
    """ONE mixer, no token shift, no feed-forward (no other way for a token to reach a later row), a flat softmax: a
    changed token at place j moves the rows j .. j + size - 1 and no other; one of the first ``keep`` tokens moves
    every row from j on. As a prompt and decoded; pages of 16, whose borders the window's far edge crosses."""
    cfg = config([win(heads=2, kv=1, dim=8, vdim=16, size=size, keep=keep, rot=4, scale=0.05, mlp=None)], cap=50.0)
    W = oracle.random_weights(cfg, 0)
    W["l0.shift"] = torch.zeros_like(W["l0.shift"])
    eng, _ = build(cfg, device, weights=W)
    toks = tokens(60, cfg["vocab"], 31)
    cuts = [decode_from] if decode_from else [len(toks)]
    base = replay_alone(eng, toks, cuts)
    assert rel_err(base, oracle.forward(cfg, W, toks)) < 2e-4
    for j in (0, 1, keep - 1, keep, 10, 15, 16, 17, 31, 38, 59):
        if not 0 <= j < len(toks):
            continue
        alt = list(toks)
        alt[j] = (alt[j] + 1) % cfg["vocab"]
        moved = np.abs(replay_alone(eng, alt, cuts) - base).max(-1)
        inside = np.zeros(len(toks), dtype=bool)
        inside[j:len(toks) if j < keep else j + size] = True
        assert (moved[inside] > 2e-5).all() and (moved[~inside] < 5e-6).all(), (j, np.nonzero(moved > 5e-6)[0])


def _marked(cfg, place, n, seed=3):
    """Tokens of which the one at ``place`` is the marked one (the last of the vocabulary, nowhere else)."""
    V = cfg["vocab"]
    toks = tokens(n, V - 1, seed)
    toks[place] = V - 1
    return toks


def _mark_key(cfg, W, m, x, factor=3.0):
    """Makes every row's query meet the marked token's key: embedding coordinate 0 is large for it and zero for every
    other token, coordinate 1 the same for all; query coordinate 0 of each head reads coordinate 1, key coordinate 0
    of each key head reads coordinate 0. No shift, plain norms."""
    d, H, G, D = cfg["width"], m["heads"], m["kv_heads"], m["dim"]
    E = 0.3 * W["embed"].float()
    E[:, 0], E[:, 1] = 0.0, 2.0
    E[cfg["vocab"] - 1, 0] = 12.0
    q, k = torch.zeros(H, D, d), torch.zeros(G, D, d)
    q[:, 0, 1], k[:, 0, 0] = factor, factor
    q[:, 1:, 2:] = 0.05 * torch.randn(H, D - 1, d - 2, generator=torch.Generator().manual_seed(1))
    k[:, 1:, 2:] = 0.05 * torch.randn(G, D - 1, d - 2, generator=torch.Generator().manual_seed(2))
    W["embed"], W["l0.shift"], W["l0.norm1"] = E.to(torch.bfloat16), torch.zeros(d).bfloat16(), torch.zeros(d).bfloat16()
    W[x + "q"], W[x + "k"] = q.view(H * D, d).bfloat16(), k.view(G * D, d).bfloat16()
    Wd = {n: v.double() for n, v in W.items()}
    return Wd


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("place,keep", [(0, 0), (0, 1), (6, 7), (6, 6), (17, 4), (40, 40)])
def test_a_key_at_the_windows_edge_or_among_the_first_stands_out(device, place, keep):
    """The marked key holds most of the weight of every row that sees it: the rows inside the window after it, and, when
    it is among the kept first keys, all later ones; the first row that does not see it falls back to the others."""
    size = 23
    cfg = config([win(heads=2, kv=1, dim=8, vdim=16, size=size, keep=keep, rot=0, scale=2.0, cap=60.0, v_mix=False, mlp=None)], vocab=30)
    W = oracle.random_weights(cfg, 6)
    m, x = cfg["layers"][0]["mixer"], "l0.mix."
    for n in ("q.b", "k.b"):
        W[x + n] = torch.zeros_like(W[x + n])
    W[x + "q.norm"] = W[x + "k.norm"] = torch.ones(8).bfloat16()
    Wd = _mark_key(cfg, W, m, x)
    toks = _marked(cfg, place, 80)
    h = oracle.rms_norm(Wd["embed"][toks], 1 + Wd["l0.norm1"], 1e-5)
    _, wts = oracle.window_attention(h, Wd, x, m, 1e-5, {}, return_weights=True)
    seen = wts[0, :, place] > 0
    assert int(seen.sum()) == (80 - place if place < keep else size)
    assert float(wts[0, :, place][seen].min()) > 0.5
    for cuts in ([80], [place + size - 2, 4], [2]):
        eng, _ = build(cfg, device, weights=W)
        assert rel_err(replay_alone(eng, toks, cuts), oracle.forward(cfg, W, toks)) < 2e-4, cuts


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["attention", "parallel"])
def test_a_far_key_that_stands_out(device, kind):
    """One key far back among hundreds carries the answer (in the attention without positions, under a sink; in the
    attention with a distance bias, in the head whose slope is small, the bias takes part of its lead). The last rows
    are decoded, rows and key lie on either side of many page borders."""
    layer = conv(heads=2, kv=1, dim=8, vdim=16, taps=3, scale=2.5, v_mix=False, mlp=None) if kind == "attention" else \
        par(heads=4, kv=1, dim=8, vdim=16, scale=1.0, coef=0.3, every=64, rs=0.3, mlp=None)
    cfg = config([layer], vocab=50)
    W = oracle.random_weights(cfg, 8)
    m = layer["mixer"] if kind == "attention" else layer["mixer"]["left"]
    x = "l0.mix." if kind == "attention" else "l0.mix.left."
    if kind == "attention":
        W[x + "q.norm"], W[x + "k.norm"] = torch.ones(16).bfloat16(), torch.ones(8).bfloat16()
        for n in ("q", "k", "v"):
            w = torch.zeros_like(W[x + n + ".conv"].float())
            w[:, 1] = 1.0                              # every channel reads the token before
            W[x + n + ".conv"] = w.bfloat16()
    Wd = _mark_key(cfg, W, m, x, factor=3.0 if kind == "attention" else 0.8)
    toks = _marked(cfg, 33, 330)
    h = oracle.rms_norm(Wd["embed"][toks], 1 + Wd["l0.norm1"], 1e-5)
    if kind == "attention":
        _, wts = oracle.conv_attention(h, Wd, x, m, 1e-5, {}, return_weights=True)
        assert float(wts[0, 40:, 34].min()) > 0.5
    else:
        _, wts = oracle.distance_attention(h, Wd, x, m, return_weights=True)
        assert float(wts[3, 300:, 33].min()) > 0.3 and float(wts[0, 300:, 33].max()) < 1e-3
    eng, _ = build(cfg, device, weights=W, blocks=24)
    assert rel_err(replay_alone(eng, toks, [300]), oracle.forward(cfg, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_the_sink_takes_its_share_once_per_row(device):
    """Sinks above, near and far below the scores: they hold almost all, about half and nothing of a row's weight. They
    are neither scaled nor tied to a key: long rows of flat scores lose less to them than short ones."""
    cfg = config([conv(heads=3, kv=1, dim=8, vdim=16, scale=0.01, v_mix=False, mlp=None)])
    W = oracle.random_weights(cfg, 2)
    W["l0.mix.sink"] = torch.tensor([6.0, 2.5, -30.0]).bfloat16()
    toks = tokens(40, cfg["vocab"], 13)
    Wd = {k: v.double() for k, v in W.items()}
    h = oracle.token_shift(oracle.rms_norm(Wd["embed"][toks], 1 + Wd["l0.norm1"], 1e-5), Wd["l0.shift"])
    _, wts = oracle.conv_attention(h, Wd, "l0.mix.", cfg["layers"][0]["mixer"], 1e-5, {}, return_weights=True)
    sums = wts.sum(-1)
    assert float(sums[0].max()) < 0.2 and 0.4 < float(sums[1, 12]) < 0.7 and float(sums[2].min()) > 0.999
    assert float(sums[1, 1]) < 0.5 * float(sums[1, 39])
    for cuts in ([40], [25], [2, 2]):
        eng, _ = build(cfg, device, weights=W)
        assert rel_err(replay_alone(eng, toks, cuts), oracle.forward(cfg, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_the_query_temperature_steps_where_its_period_ends(device):
    """The factor changes at positions every - 1, 2 every - 1, ...: with a peaked softmax a factor that steps one
    position early or late shows in exactly those rows (the oracle with another period differs there)."""
    cfg = config([par(heads=2, kv=1, dim=8, vdim=16, scale=0.5, coef=3.0, every=7, rs=0.1, mlp=None)])
    eng, W = build(cfg, device)
    toks = tokens(50, cfg["vocab"], 5)
    want = oracle.forward(cfg, W, toks).numpy()
    late = copy.deepcopy(cfg)
    late["layers"][0]["mixer"]["left"]["q_temp"]["every"] = 8
    other = np.abs(oracle.forward(late, W, toks).numpy() - want).max(-1)
    assert other[:6].max() < 1e-12 and other[6] > 1e-2
    for cuts in ([50], [13, 2], []):
        assert rel_err(replay_alone(eng, toks, cuts), want) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_values_are_the_first_mixing_layers_own(device):
    """A later layer that takes ALL its values from the first mixing layer, which stands behind another layer that does
    not mix; the first one's own share is never used, whatever its tensor holds."""
    cfg = config([conv(v_mix=False), win(vdim=20, kv=1), conv(vdim=10, kv=2), win(vdim=5, kv=4)])
    W = oracle.random_weights(cfg, 3)
    for i in (2, 3):
        W[f"l{i}.mix.vmix"] = torch.tensor(1.0).bfloat16()
    toks = tokens(40, cfg["vocab"], 8)
    want = oracle.forward(cfg, W, toks)
    for own in (0.0, 5.0):
        W["l1.mix.vmix"] = torch.tensor(own).bfloat16()
        eng, _ = build(cfg, device, weights=W)
        assert rel_err(replay_alone(eng, toks, [21, 2]), want) < 2e-4
    W["l2.mix.v"] = torch.zeros_like(W["l2.mix.v"])        # (its own values play no part)
    eng, _ = build(cfg, device, weights=W)
    assert rel_err(replay_alone(eng, toks, [21, 2]), want) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_router_bias_chooses_and_only_the_chosen_share_the_weight(device):
    """A bias that lifts two experts far above the rest: the oracle with the softmax over ALL logits (another bias on the
    others) gives the same weights, so the others' logits must not matter; equal logits of the two give halves."""
    cfg = config([win(mlp=moe(6, 2))])
    W = oracle.random_weights(cfg, 5)
    toks = tokens(20, cfg["vocab"], 8)
    W["l0.mlp.router.b"] = torch.tensor([0.0, 9.0, 0.0, 0.0, 9.0, 0.0]).bfloat16()
    W["l0.mlp.router"] = (0.2 * W["l0.mlp.router"].float()).bfloat16()
    want = oracle.forward(cfg, W, toks)
    for rest in (0.0, 4.0, -9.0):
        W["l0.mlp.router.b"] = torch.tensor([rest, 9.0, rest, rest, 9.0, rest]).bfloat16()
        eng, _ = build(cfg, device, weights=W)
        assert rel_err(replay_alone(eng, toks, [12, 2]), want) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_and_single_token_requests(device):
    eng, W = build(MIXED, device)
    for toks in ([7], [7, 7], tokens(3, MIXED["vocab"], 2)):
        assert rel_err(replay_alone(eng, toks, [len(toks)]), oracle.forward(MIXED, W, toks)) < 2e-4
        assert rel_err(replay_alone(eng, toks, []), oracle.forward(MIXED, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_pool_or_slots_exhausted_is_an_error_and_leaves_the_engine_usable(device):
    cfg = config([conv(), par()])
    for blocks, slots in ((2, 4), (8, 2)):
        eng, W = build(cfg, device, blocks=blocks, slots=slots, max_batch_seqs=4)
        a, b, c = eng.replay_open(), eng.replay_open(), eng.replay_open()
        eng.replay_step([(a, [1, 2], []), (b, [3], [])])
        with pytest.raises(RuntimeError):
            eng.replay_step([(c, [4], [])])
        eng.replay_close(a)
        lg = eng.replay_step([(c, [4, 5], [1])])
        assert rel_err(lg, oracle.forward(cfg, W, [4, 5])[1:]) < 2e-4


def _greedy_oracle(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(oracle.forward(cfg, W, toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_submit_and_the_scheduler(device, graphs):
    """More requests than the batch holds, prompts cut by the scheduler's token budget, decoding chains riding
    in the steps that prefill later prompts; recorded decode steps on the GPU."""
    if graphs and device == "cpu":
        pytest.skip("decode graphs are a GPU feature")
    eng, W = build(MIXED, device, blocks=40, slots=3, max_batch_seqs=3, max_prefill_tokens=24, use_graphs=graphs,
                   pipeline_decode=graphs)
    p = core.SamplingParams()
    p.temperature, p.max_new_tokens, p.ignore_eos = 0.0, 9, True
    prompts = [tokens(n, MIXED["vocab"], 50 + n) for n in (30, 5, 41, 1, 17)]
    rids = [eng.submit(pr, params=p) for pr in prompts]
    eng.run_until_done()
    for rid, pr in zip(rids, prompts):
        out = eng.pop_result(rid)
        assert out.token_ids[0] == _greedy_oracle(MIXED, W, pr, 9)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_serving_steps_launch_only_the_kernel_library(dtype):
    """Prompt portions, mixed steps, decode steps and replayed steps: PyTorch launches no kernel of its own in
    any of them (allocations, views and buffer copies aside)."""
    from llm_consensus_amd.utils.audit import AtenAudit

    cfg = config([win(heads=4, kv=2, dim=16, vdim=16, rot=8, mlp={"kind": "dense", "ff": 64, "limit": 1.0}), conv(heads=4, kv=2, dim=16, vdim=16, mlp=moe(6, 2, 64)),
                  par(mlp=None), par(mlp=moe())], width=64, vocab=70)
    eng, _ = build(cfg, "cuda:0", dtype, blocks=40, slots=3, max_batch_seqs=3, max_prefill_tokens=24)
    p = core.SamplingParams()
    p.temperature, p.max_new_tokens, p.ignore_eos = 0.7, 5, True

    def work():
        rids = [eng.submit(tokens(n, cfg["vocab"], n), params=p) for n in (30, 5, 41)]
        eng.run_until_done()
        rid = eng.replay_open()
        eng.replay_step([(rid, tokens(20, cfg["vocab"], 1), [0, 19])])
        eng.replay_step([(rid, [3], [0])])
        eng.replay_close(rid)
        return [eng.pop_result(r) for r in rids]

    work()
    torch.cuda.synchronize()
    with AtenAudit() as audit:
        outs = work()
        torch.cuda.synchronize()
    assert all(len(o.token_ids[0]) == 5 for o in outs)
    assert audit.kernels == {}, audit.kernels


def test_checkpoint_directory_through_the_registry_the_trace_tool_and_the_command_line(tmp_path, capsys):
    """A Kulivik checkpoint directory is found by its config.json, loaded with the checkpoint's tensor names,
    replayed by ``bin/trace_run`` (two requests in one step, a request that ends and one that goes on) and
    answers a question through the command line."""
    from safetensors.torch import save_file

    from llm_consensus_amd import cli
    from llm_consensus_amd.models.loader import load_model
    from llm_consensus_amd.models.registry import resolve

    cfg = config([par(mlp=moe()), win(heads=2, kv=1, dim=8, vdim=8, size=6, rot=8), conv(vdim=4, v_mix=True, mlp=None)], width=32, vocab=300)
    W = oracle.random_weights(cfg, 3)
    ck = tmp_path / "kulivik"
    ck.mkdir()
    (ck / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in W.items()}, str(ck / "model.safetensors"))
    assert resolve(str(ck)).name == "hybrid"
    m = load_model(str(ck), "cpu", dtype=torch.float32)
    assert config_to_dict(m.cfg) == cfg
    a, b = tokens(21, 300, 1), tokens(9, 300, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}, {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[17:18], "want": [0]}, {"id": "b", "tokens": b[2:], "want": [6]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[18:], "want": [2]}], "end": ["a"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(ck), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128", "--device", "cpu"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = oracle.forward(cfg, W, a).numpy(), oracle.forward(cfg, W, b).numpy()
    got = [np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, 300) for i in range(3)]
    assert rel_err(got[0], la[[0, 16]]) < 2e-4
    assert rel_err(got[1], np.stack([la[17], lb[8]])) < 2e-4
    assert rel_err(got[2], la[[20]]) < 2e-4
    toml = tmp_path / "e.toml"
    toml.write_text(f"""strategy = "majority_vote"
decision_mode = "logprob"
choices = "ABCD"
[sampling]
temperature = 0.0
max_new_tokens = 4
[models.h]
path = "{ck}"
[[members]]
name = "hybrid"
model = "h"
""")
    q = tmp_path / "q.txt"
    q.write_text("Which? A. a B. b C. c D. d\n")
    assert cli.main(["--config", str(toml), "--questions", str(q), "--device", "cpu", "--no-warm-up"]) == 0
    assert capsys.readouterr().out.strip()[-1] in "ABCD"


def test_random_checkpoint_writer_and_random_init(tmp_path):
    """The family's checkpoint writer and ``random_init`` (benchmarks, stand-ins) know the design's tensors: what
    one writes the loader reads back, and both models answer the same."""
    from llm_consensus_amd.models.loader import load_model, write_random_hybrid_checkpoint

    cfg = config_from_dict(config([win(), conv(mlp=moe()), par(mlp=None)], width=24, vocab=80))
    ck = write_random_hybrid_checkpoint(cfg, str(tmp_path / "ck"), seed=7)
    assert json.loads((ck / "config.json").read_text())["architecture"] == "Kulivik"
    a = load_model(str(ck), "cpu", dtype=torch.float32)
    b = HybridModel.random_init(cfg, "cpu", seed=7, dtype=torch.float32)
    assert a.cfg.layers == b.cfg.layers and a.cfg.logit_softcap == b.cfg.logit_softcap == 9.0
    out = []
    for m in (a, b):
        eng = Engine(m, num_kv_blocks=8, block_size=BS, max_batch_seqs=2, state_slots=2, max_model_len=8 * BS,
                     enable_prefix_cache=False, use_graphs=False, pipeline_decode=False)
        out.append(replay_alone(eng, tokens(12, 80, 1), [7]))
    assert np.isfinite(out[0]).all() and np.abs(out[0]).max() > 0
    np.testing.assert_allclose(out[0], out[1], rtol=1e-6, atol=1e-6)


def test_a_configuration_without_the_optional_entries():
    """Absent mask, cap, rotation and temperature mean none; a layer that names no feed-forward has none; an absent
    ``v_mix`` needs no tensor."""
    c = config([win(v_mix=False), par(), conv(v_mix=False)])
    m = c["layers"][0]["mixer"]
    for k in ("mask", "softcap", "rot", "v_mix"):
        del m[k]
    del c["layers"][1]["mixer"]["left"]["q_temp"], c["layers"][1]["mlp"], c["layers"][2]["mixer"]["v_mix"], c["logit_softcap"]
    cfg = config_from_dict(c)
    a, p, v = cfg.layers
    assert (a.window, a.keep_first, a.softcap, a.rot_dims, a.v_mix) == (0, 0, 0.0, 0, False)
    assert p.q_temp[0] == 0.0 and not p.has_ff and cfg.logit_softcap == 0.0 and not v.v_mix
    full = config([win(v_mix=False, size=10 ** 6, keep=0, cap=1e9, rot=0), par(coef=0.0, mlp=None), conv(v_mix=False)], cap=1e9)
    W = oracle.random_weights(full, 1)
    eng, _ = build(c, "cpu", weights=W)
    toks = tokens(25, c["vocab"], 4)
    assert rel_err(replay_alone(eng, toks, [14]), oracle.forward(full, W, toks)) < 2e-4


def test_configurations_the_design_does_not_have_are_refused():
    with pytest.raises(ValueError):
        config_from_dict(config([par(rheads=3, decay=[0.5, 0.5])]))              # a decay per head
    with pytest.raises(ValueError):
        config_from_dict(config([win(vdim=8, kv=2), conv(vdim=8, kv=1)]))        # mixed values of another width
    with pytest.raises(ValueError):
        config_from_dict(config([win(heads=4, kv=3)]))
    with pytest.raises(ValueError):
        config_from_dict(config([win(rot=5)]))
    with pytest.raises(ValueError):
        config_from_dict(config([par(rdim=300)]))
    with pytest.raises(ValueError):
        config_from_dict(config([par(every=0)]))
    with pytest.raises(ValueError):
        config_from_dict(config([conv(mlp=moe(3, 4))]))                          # more choices than experts
    with pytest.raises(ValueError):
        config_from_dict(config([{"type": "mingru", "mixer": {"width": 8}, "mlp": None}]))
