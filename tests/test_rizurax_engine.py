"""Rizurax decoders through the engine (scheduler, paged cache, state slots, step function) against the plain
implementation in ``rizurax_oracle.py``. Small configurations with random weights made here; every test runs
on the CPU ops and, marked ``gpu``, on the HIP kernels."""
import copy
import json
import math
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import rizurax_oracle as oracle
from llm_consensus_amd._native import core
from llm_consensus_amd.engine.engine import Engine
from llm_consensus_amd.models.hybrid import HybridModel, config_from_dict, config_to_dict, rotary_frequencies

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
BS = 16
ROOT = Path(__file__).resolve().parents[1]
DENSE = {"kind": "dense", "ff": 56}


def delta(heads=4, kv=2, dim=12, vdim=10, conv=4, mlp=DENSE):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def attn(heads=4, kv=2, dim=12, vdim=10, scale=0.3, diff=0.4, rot=6, base=500.0, factor=3.0, original=64, fast=5.0, slow=0.5, mlp=DENSE):
    r = {"dims": rot, "base": base}
    if factor is not None:
        r["scaling"] = {"factor": factor, "original": original, "fast": fast, "slow": slow}
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff, "rot": r},
            "mlp": mlp}


def config(layers, width=40, vocab=67, eps=1e-5, loop=None, buckets=53, mul_prev=11, mul_cur=3):
    c = {"architecture": "Rizurax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if buckets:
        c["embedding"] = {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


MIXED = config([delta(), attn(vdim=20, kv=1), delta(heads=3, kv=3, dim=20, vdim=24, conv=3, mlp=None), attn(heads=2, kv=2, rot=12, factor=None),
                delta(heads=2, kv=1, conv=2), attn(heads=6, kv=3, dim=16, vdim=16, rot=0, mlp=None)], loop=(1, 4, 2))


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
    """32-bit: every row to rounding. bf16 (rounding errors of a percent or two, now and then a row whose norms magnify
    them): the typical row close, no row far."""
    e = row_errs(got, want)
    return float(e.max()) < 2e-4 if dtype == torch.float32 else float(np.median(e)) < 4e-2 and float(e.max()) < 0.2


def _whole_prompt(cfg, device, dtype, name, cuts=None, seed=0, n=45):
    eng, W = build(cfg, device, dtype, seed)
    toks = tokens(n if cuts is None else sum(cuts) + 3, cfg["vocab"], 3)
    got = replay_alone(eng, toks, cuts or [len(toks)])
    assert close(got, oracle.forward(cfg, W, toks), dtype), name


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,layers", [
    ("delta: grouped heads, values narrower than keys; values wider, two taps", [delta(), delta(heads=6, kv=3, dim=10, vdim=16, conv=2)]),
    ("delta: one key head, one tap; as many key heads as heads, six taps", [delta(heads=4, kv=1, dim=16, vdim=16, conv=1), delta(heads=3, kv=3, dim=8, vdim=4, conv=6)]),
    ("delta: widths of whole matrix tiles, a key width past a wave, one head", [delta(heads=4, kv=2, dim=32, vdim=64), delta(heads=2, kv=1, dim=70, vdim=66, conv=3), delta(heads=1, kv=1)]),
    ("attention: grouped heads, part of the map turns; values wider than keys", [attn(), attn(heads=6, kv=3, dim=10, vdim=24, rot=4)]),
    ("attention: one key head, the whole map turns; nothing turns, as many key heads as heads", [attn(heads=4, kv=1, dim=16, vdim=16, rot=16), attn(heads=3, kv=3, dim=7, vdim=4, rot=0)]),
    ("attention: widths of the matrix-core kernel", [attn(heads=4, kv=2, dim=16, vdim=32, rot=8), attn(heads=8, kv=4, dim=32, vdim=64, rot=32)]),
    ("attention: no frequency scaling, a ramp of no width, all pairs slowed down, none", [attn(factor=None), attn(fast=1.0, slow=1.0), attn(fast=1e3, slow=500.0, base=50.0), attn(fast=1e-2, slow=1e-3, rot=12)]),
    ("attention: nothing and all taken off, a factor below one", [attn(diff=0.0), attn(diff=0.95, factor=0.5)]),
    ("layers without a feed-forward", [delta(mlp=None), attn(mlp=None)]),
    ("one layer", [attn(mlp={"kind": "dense", "ff": 9})]),
])
def test_each_mechanism_whole_prompt(device, dtype, name, layers):
    _whole_prompt(config(layers), device, dtype, name)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("loop", [None, (0, 3, 1), (0, 3, 3), (1, 2, 4), (0, 1, 2), (2, 3, 2), (1, 1, 5)])
def test_loops_over_any_range(device, dtype, loop):
    """From the first layer, up to the last, over one layer, once, over nothing: every pass with a cache and a state of its
    own and nothing in between; as portions and decoded."""
    cfg = config([delta(mlp=None), attn(), delta(heads=2, kv=2, conv=3)], loop=loop)
    _whole_prompt(cfg, device, dtype, loop, cuts=[17, 2, 9])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_depths_the_mfma_products_take(device, dtype):
    """Widths of 64 / 128 with mixers and feed-forwards whose widths together are multiples of 64 though neither is: in bf16
    on the GPU all products go through the packed MFMA kernels."""
    for width, ff, vdim in ((64, 80, 12), (128, 192, 16)):
        d = {"kind": "dense", "ff": ff}
        cfg = config([attn(heads=4, kv=2, dim=16, vdim=vdim, rot=8, mlp=d), delta(heads=4, kv=2, dim=16, vdim=vdim, mlp=d)], width=width, vocab=70)
        _whole_prompt(cfg, device, dtype, f"mfma depths {width}", cuts=[40, 2, 17])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_deep_products_and_long_portions(device, dtype):
    """Width 1024 (the bf16 products of a few rows split their depth over workgroups), fused projection widths that are no
    multiple of 32, a portion of a few hundred rows (chunks side by side), one a row longer than a chunk, a short one."""
    cfg = config([delta(heads=3, kv=1, dim=24, vdim=40, mlp={"kind": "dense", "ff": 72}), attn(heads=2, kv=1, dim=24, vdim=48, rot=8, mlp=None),
                  delta(heads=2, kv=2, dim=36, vdim=20, mlp=None)], width=1024, vocab=90)
    eng, W = build(cfg, device, dtype, blocks=26)
    toks = tokens(360, cfg["vocab"], 3)
    assert close(replay_alone(eng, toks, [257, 65, 20]), oracle.forward(cfg, W, toks), dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_widths_the_vector_accesses_do_not_take(device):
    """A width and channel counts that are multiples of nothing."""
    cfg = config([delta(heads=3, kv=1, dim=5, vdim=3, conv=3, mlp={"kind": "dense", "ff": 9}), attn(heads=1, kv=1, dim=7, vdim=5, rot=2),
                  delta(heads=1, kv=1, dim=3, vdim=7, mlp={"kind": "dense", "ff": 11})], width=37, vocab=41)
    _whole_prompt(cfg, device, torch.float32, "odd widths", cuts=[93, 2, 9])


@pytest.mark.parametrize("device", DEVICES)
def test_constants_that_could_pass_for_one(device):
    """Scales, factors, multipliers and biases of 0 and 1, then other constants with the SAME tensors; every constant on its
    own moves the logits of the oracle; a large eps."""
    layers = [attn(heads=2, kv=2, scale=1.0, diff=0.0, factor=1.0, original=1, fast=1.0, slow=1.0, base=1.5, rot=8, mlp={"kind": "dense", "ff": 20}),
              delta(heads=2, kv=2, mlp=None)]
    cfg = config(layers, eps=1.0, buckets=53, mul_prev=1, mul_cur=1)
    W = oracle.random_weights(cfg, 4)
    for n in ("A_log", "dt_bias"):
        W["l1.mix." + n] = torch.zeros(2).bfloat16()
    W["l0.mix.lq1"] = W["l0.mix.lk1"] = torch.ones(12).bfloat16() * 0.3
    toks = tokens(30, cfg["vocab"], 9)
    base = oracle.forward(cfg, W, toks)
    eng, _ = build(cfg, device, weights=W)
    assert rel_err(replay_alone(eng, toks, [17]), base) < 2e-4

    def put(c, path, v):
        for k in path[:-1]:
            c = c[k]
        c[path[-1]] = v
    rot = ("layers", 0, "mixer", "rot")
    scaling = {"factor": 8.0, "original": 64, "fast": 20.0, "slow": 1.0}
    changes = [(("layers", 0, "mixer", "scale"), 0.4), (("layers", 0, "mixer", "diff"), 0.5), (rot + ("base",), 30.0), (rot + ("dims",), 6),
               (rot + ("scaling", "factor"), 2.5), (rot + ("scaling",), scaling), (("embedding", "bigram", "mul_prev"), 2),
               (("embedding", "bigram", "mul_cur"), 5), (("norm", "eps"), 1e-3), (("loop",), {"start": 0, "stop": 2, "times": 2})]
    for path, v in changes:
        other = copy.deepcopy(cfg)
        put(other, path, v)
        want = oracle.forward(other, W, toks)
        assert rel_err(want.numpy(), base) > 5e-3, path
        eng, _ = build(other, device, weights=W)
        assert rel_err(replay_alone(eng, toks, [17]), want) < 2e-4, path
    ramp = copy.deepcopy(cfg)
    put(ramp, rot + ("scaling",), scaling)
    put(ramp, rot + ("base",), 30.0)
    at = oracle.forward(ramp, W, toks)
    for k, v in (("original", 500), ("fast", 3.0), ("slow", 0.1)):
        other = copy.deepcopy(ramp)
        put(other, rot + ("scaling", k), v)
        want = oracle.forward(other, W, toks)
        assert rel_err(want.numpy(), at) > 5e-3, k
        eng, _ = build(other, device, weights=W)
        assert rel_err(replay_alone(eng, toks, [17]), want) < 2e-4, k


@pytest.mark.parametrize("device", DEVICES)
def test_residual_stream_after_every_layer_run(device):
    eng, W = build(MIXED, device)
    toks = tokens(20, MIXED["vocab"], 5)
    taps, rid = [], eng.replay_open()
    eng.replay_step([(rid, toks, [])], taps=taps)
    _, want = oracle.forward(MIXED, W, toks, return_layers=True)
    assert len(taps) == len(want) == 9
    for i, t in enumerate(taps):
        torch.testing.assert_close(t.cpu().double(), want[i], atol=2e-4, rtol=2e-4, msg=f"run {i}")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[], [1], [40], [2, 2, 3, 2, 17, 2], [11, 1, 1, 12, 13], [5, 7, 12, 16, 1, 15, 2]])
def test_portions_and_token_by_token_decoding(device, dtype, cuts):
    """The same logits whether the prompt comes whole, in portions down to two tokens (cut inside pages of 16 and inside the
    reach of the convolutions; row by row and in chunks), or one token at a time."""
    eng, W = build(MIXED, device, dtype)
    toks = tokens(70, MIXED["vocab"], 7)
    assert close(replay_alone(eng, toks, cuts), oracle.forward(MIXED, W, toks), dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[64], [63, 2], [65, 64], [128, 1, 17, 13], [150], [16, 17, 100]])
def test_chunk_borders_of_the_delta_rule(device, cuts):
    """Portions that end at, before and behind whole chunks of 64 rows, start anywhere inside the sequence, and the portion
    lengths at which the recurrence changes its form; memories that last for the whole sequence."""
    cfg = config([delta(heads=4, kv=2, dim=16, vdim=24, mlp=None)])
    W = oracle.random_weights(cfg, 2)
    W["l0.mix.dt_bias"] = torch.tensor([-9.0, -6.0, -3.0, 2.0]).bfloat16()
    eng, _ = build(cfg, device, weights=W)
    toks = tokens(160, cfg["vocab"], 12)
    assert rel_err(replay_alone(eng, toks, cuts), oracle.forward(cfg, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_past_pages_and_chunks(device):
    eng, W = build(MIXED, device)
    toks = tokens(140, MIXED["vocab"], 11)
    assert rel_err(replay_alone(eng, toks, [3]), oracle.forward(MIXED, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_reused_pages_and_slots(device, dtype):
    """Up to four live requests, portions beside single tokens, in a pool too small for all of them at once: requests
    end, others take their pages and state slots (which are never cleared)."""
    eng, W = build(MIXED, device, dtype, blocks=12, slots=4)
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
def test_previous_tokens_convolution_inputs_and_memories_across_portions_and_reused_slots(device):
    """What a sequence keeps besides keys and values: its last token (a model whose embedding is ALMOST only the pair table's,
    so that a wrong previous token is a wrong token), the last inputs of a convolution of five taps whose OLDEST tap
    dominates, a memory that hardly decays. Portions shorter than the reach of the convolution, then single tokens; one state
    slot that four requests use one after another, so that anything left from the one before would show."""
    cfg = config([delta(conv=5, mlp=None), delta(heads=2, kv=1, mlp=None)], loop=(0, 2, 2))
    W = oracle.random_weights(cfg, 9)
    W["embed"] = (0.01 * W["embed"].float()).bfloat16()
    for n in ("q", "k", "v"):
        w = 0.1 * W[f"l0.mix.{n}.conv"].float()
        w[:, 0] = 1.5
        W[f"l0.mix.{n}.conv"] = w.to(torch.bfloat16)
    W["l1.mix.dt_bias"] = torch.full((2,), -8.0).bfloat16()
    eng, _ = build(cfg, device, weights=W, slots=1, blocks=4)
    for seed, cuts in ((1, [2, 2, 3, 2, 2, 9]), (2, [1, 3, 2]), (3, [4, 4, 4, 11]), (4, []), (5, [40])):
        toks = tokens(45, cfg["vocab"], seed)
        assert rel_err(replay_alone(eng, toks, cuts), oracle.forward(cfg, W, toks)) < 2e-4, cuts


@pytest.mark.parametrize("device", DEVICES)
def test_token_pairs_name_their_row_and_the_first_token_the_last_row(device):
    """ONE layer that adds (almost) nothing, so that a row's logits depend on its token and the one before: equal pairs give
    equal logits wherever they stand (page and portion borders included), the same token first in a sequence another row;
    products past 32 bits; multipliers larger than the number of buckets."""
    for buckets, mp, mc in ((53, 11, 3), (1, 5, 7), (64, 2147483647, 2147483629), (97, 97, 1)):
        cfg = config([delta(mlp=None)], buckets=buckets, mul_prev=mp, mul_cur=mc, vocab=300)
        W = oracle.random_weights(cfg, 3)
        W["l0.mix.o"] = torch.zeros_like(W["l0.mix.o"])
        toks = [250, 250] + tokens(14, 300, 5) + [250, 250] + tokens(13, 300, 6) + [7, 250, 250, 7]
        want = oracle.forward(cfg, W, toks)
        assert buckets > 1 and float((want[1] - want[17]).abs().max()) < 1e-9 or buckets == 1
        assert float((want[0] - want[1]).abs().max()) > 1e-2
        for cuts in ([len(toks)], [1, 15, 1, 16], []):
            eng, _ = build(cfg, device, weights=W)
            assert rel_err(replay_alone(eng, toks, cuts), want) < 2e-4, (buckets, cuts)


@pytest.mark.parametrize("device", DEVICES)
def test_a_model_without_a_pair_table(device):
    cfg = config([attn(), attn(heads=2, kv=1)], buckets=0)
    eng, W = build(cfg, device)
    assert not eng.model.cfg.has_state
    toks = tokens(40, cfg["vocab"], 3)
    assert rel_err(replay_alone(eng, toks, [21, 2]), oracle.forward(cfg, W, toks)) < 2e-4


def _marked(cfg, place, n, seed=3):
    """Tokens of which the one at ``place`` is the marked one (the last of the vocabulary, nowhere else)."""
    V = cfg["vocab"]
    toks = tokens(n, V - 1, seed)
    toks[place] = V - 1
    return toks


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("which", [0, 1])
def test_a_far_key_that_stands_out_in_one_map(device, which):
    """One key far back among hundreds carries one map's answer while the other map stays flat: in the first map it is
    added, in the second taken off with the layer's weight. The last rows are decoded, rows and key lie on either side of
    many page borders; a pair table of zeros."""
    cfg = config([attn(heads=2, kv=1, dim=8, vdim=16, scale=1.0, rot=0, mlp=None)], vocab=50)
    W = oracle.random_weights(cfg, 8)
    d, x = cfg["width"], "l0.mix."
    W["bigram"] = torch.zeros_like(W["bigram"])
    E = 0.3 * W["embed"].float()
    E[:, 0], E[:, 1] = 0.0, 2.0
    E[-1, 0] = 12.0
    q, k = torch.zeros(2, 2, 8, d), torch.zeros(1, 2, 8, d)
    q[:, which, 0, 1], k[:, which, 0, 0] = 3.0, 3.0
    W["embed"], W["l0.norm1"] = E.bfloat16(), torch.zeros(d).bfloat16()
    W[x + "q"], W[x + "k"] = q.view(-1, d).bfloat16(), k.view(-1, d).bfloat16()
    toks = _marked(cfg, 33, 330)
    Wd = {n: v.double() for n, v in W.items()}
    h = oracle.rms_norm(Wd["embed"][toks], 1.0, 1e-5)
    _, wts = oracle.differential_attention(h, Wd, x, cfg["layers"][0]["mixer"], 1e-5, return_weights=True)
    assert float(wts[:, which, 300:, 33].min()) > 0.5 and float(wts[:, 1 - which, 300:, 33].max()) < 0.01
    eng, _ = build(cfg, device, weights=W, blocks=24)
    for cuts in ([300], [33, 1, 2, 250], [40, 40, 200]):
        assert rel_err(replay_alone(eng, toks, cuts), oracle.forward(cfg, W, toks)) < 2e-4, cuts


@pytest.mark.parametrize("device", DEVICES)
def test_the_two_maps_come_head_by_head_and_share_the_groups_values(device):
    """Swapping two heads' queries (both maps) and their columns of the output product changes nothing; swapping the two maps of
    ONE head does. Equal maps with a weight of one leave nothing (the norm then sees zeros)."""
    cfg = config([attn(heads=4, kv=2, dim=8, vdim=16, rot=4, mlp=None)])
    W = oracle.random_weights(cfg, 6)
    toks = tokens(40, cfg["vocab"], 2)
    base = oracle.forward(cfg, W, toks)

    def run(W, c=cfg):
        eng, _ = build(c, device, weights=W)
        return replay_alone(eng, toks, [25, 2])
    assert rel_err(run(W), base) < 2e-4
    V = dict(W)
    q = V["l0.mix.q"].view(4, 2, 8, 40).clone()
    o = V["l0.mix.o"].view(40, 4, 16).clone()
    V["l0.mix.q"], V["l0.mix.o"] = q[[1, 0, 2, 3]].reshape(-1, 40), o[:, [1, 0, 2, 3]].reshape(40, -1).contiguous()
    assert rel_err(run(V), base) < 2e-4
    q[0] = q[0].flip(0)
    V["l0.mix.q"], V["l0.mix.o"] = q.reshape(-1, 40), W["l0.mix.o"]
    want = oracle.forward(cfg, V, toks)
    assert rel_err(want.numpy(), base) > 2e-2 and rel_err(run(V), want) < 2e-4
    V = dict(W)
    for n, heads in (("q", 4), ("k", 2)):
        t = V["l0.mix." + n].view(heads, 2, 8, 40).clone()
        t[:, 1] = t[:, 0]
        V["l0.mix." + n] = t.reshape(-1, 40)
    for n in ("lq1", "lk1", "lq2", "lk2"):
        V["l0.mix." + n] = torch.zeros(8).bfloat16()
    one = copy.deepcopy(cfg)
    one["layers"][0]["mixer"]["diff"] = 0.5
    assert rel_err(run(V, one), oracle.forward(one, V, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_a_key_seen_again_far_back_is_corrected_not_added(device):
    """A memory with step sizes near one and no decay: a value written at a unit key is read back hundreds of rows later, and
    a second write at the same key replaces it. Keys come from single coordinates of the token's embedding."""
    cfg = config([delta(heads=1, kv=1, dim=16, vdim=16, conv=1, mlp=None)], width=40, vocab=20)
    W = oracle.random_weights(cfg, 5)
    d, x = 40, "l0.mix."
    E = torch.zeros(20, d)
    E[torch.arange(16), torch.arange(16)] = 6.0                # token j: key coordinate j
    E[:, 16:32] = torch.randn(20, 16, generator=torch.Generator().manual_seed(1))
    E[:, 39] = 1.0
    W["embed"], W["bigram"], W["l0.norm1"] = E.bfloat16(), 0.3 * W["bigram"], torch.zeros(d).bfloat16()
    W["bigram"][:, :16] = 0.0
    eye = torch.zeros(16, d)
    eye[:, :16] = 3.0 * torch.eye(16)
    W[x + "q"], W[x + "k"] = eye.bfloat16(), eye.bfloat16()
    for n in ("q", "k", "v"):
        W[x + n + ".conv"] = torch.ones(16, 1).bfloat16()
    W[x + "b"] = torch.zeros(1, d)
    W[x + "b"][0, 39] = 30.0
    W[x + "b"], W[x + "A_log"], W[x + "dt_bias"] = W[x + "b"].bfloat16(), torch.full((1,), -20.0).bfloat16(), torch.full((1,), -5.0).bfloat16()
    toks = [0, 0] + [1 + t % 15 for t in range(298)] + [0, 0, 3, 0]
    want = oracle.forward(cfg, W, toks)
    for cuts in ([len(toks)], [100, 200], [2, 150, 148]):
        eng, _ = build(cfg, device, weights=W)
        assert rel_err(replay_alone(eng, toks, cuts), want) < 2e-4, cuts


@pytest.mark.parametrize("device", DEVICES)
def test_steep_decays_beside_lasting_ones(device):
    """Decays that fall to nothing within a row (their logarithms add up to thousands inside a chunk) between rows that do
    not decay: ratios of cumulative decays keep their precision."""
    cfg = config([delta(heads=2, kv=1, dim=16, vdim=16, mlp=None)])
    W = oracle.random_weights(cfg, 7)
    W["l0.mix.A_log"] = torch.tensor([3.5, -2.0]).bfloat16()
    W["l0.mix.a"] = (8.0 * W["l0.mix.a"].float()).bfloat16()
    W["l0.mix.dt_bias"] = torch.tensor([-2.0, -2.0]).bfloat16()
    eng, _ = build(cfg, device, weights=W)
    toks = tokens(150, cfg["vocab"], 4)
    assert rel_err(replay_alone(eng, toks, [140]), oracle.forward(cfg, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_a_changed_token_moves_no_earlier_row(device):
    """As a prompt and decoded, at page borders: rows before the changed token stay as they are, the row itself moves and, by
    the pair table alone, so does the next one."""
    cfg = config([attn(heads=2, kv=1, dim=8, vdim=16, rot=4, mlp=None), delta(heads=2, kv=2, mlp=None)])
    eng, W = build(cfg, device)
    toks = tokens(60, cfg["vocab"], 31)
    for cuts in ([60], [30], [3]):
        base = replay_alone(eng, toks, cuts)
        for j in (0, 1, 15, 16, 17, 31, 32, 59):
            alt = list(toks)
            alt[j] = (alt[j] + 1) % cfg["vocab"]
            moved = np.abs(replay_alone(eng, alt, cuts) - base).max(-1)
            assert (moved[:j] < 5e-6).all() and (moved[j:j + 2] > 1e-3).all(), j


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_and_single_token_requests(device):
    eng, W = build(MIXED, device)
    for toks in ([7], [7, 7], tokens(3, MIXED["vocab"], 2)):
        assert rel_err(replay_alone(eng, toks, [len(toks)]), oracle.forward(MIXED, W, toks)) < 2e-4
        assert rel_err(replay_alone(eng, toks, []), oracle.forward(MIXED, W, toks)) < 2e-4


@pytest.mark.parametrize("device", DEVICES)
def test_pool_or_slots_exhausted_is_an_error_and_leaves_the_engine_usable(device):
    cfg = config([delta(), attn()])
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

    cfg = config([delta(heads=4, kv=2, dim=16, vdim=16, mlp={"kind": "dense", "ff": 64}), attn(heads=4, kv=2, dim=16, vdim=32, rot=8, mlp={"kind": "dense", "ff": 64}),
                  delta(mlp=None), attn()], width=64, vocab=70, loop=(1, 3, 2))
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
    """A Rizurax checkpoint directory is found by its config.json, loaded with the checkpoint's tensor names,
    replayed by ``bin/trace_run`` (two requests in one step, a request that ends and one that goes on) and
    answers a question through the command line."""
    from safetensors.torch import save_file

    from llm_consensus_amd import cli
    from llm_consensus_amd.models.loader import load_model
    from llm_consensus_amd.models.registry import resolve

    cfg = config([delta(), attn(heads=2, kv=1, dim=8, vdim=8, rot=8), delta(vdim=4, mlp=None)], width=32, vocab=300, loop=(0, 2, 2))
    W = oracle.random_weights(cfg, 3)
    ck = tmp_path / "rizurax"
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

    cfg = config_from_dict(config([delta(), attn(), attn(factor=None, mlp=None)], width=24, vocab=80))
    ck = write_random_hybrid_checkpoint(cfg, str(tmp_path / "ck"), seed=7)
    assert json.loads((ck / "config.json").read_text())["architecture"] == "Rizurax"
    a = load_model(str(ck), "cpu", dtype=torch.float32)
    b = HybridModel.random_init(cfg, "cpu", seed=7, dtype=torch.float32)
    assert a.cfg.layers == b.cfg.layers and a.cfg.pair == b.cfg.pair == (53, 11, 3)
    out = []
    for m in (a, b):
        eng = Engine(m, num_kv_blocks=8, block_size=BS, max_batch_seqs=2, state_slots=2, max_model_len=8 * BS,
                     enable_prefix_cache=False, use_graphs=False, pipeline_decode=False)
        out.append(replay_alone(eng, tokens(12, 80, 1), [7]))
    assert np.isfinite(out[0]).all() and np.abs(out[0]).max() > 0
    np.testing.assert_allclose(out[0], out[1], rtol=1e-6, atol=1e-6)


def test_rotary_frequencies_of_known_turn_counts():
    """Pairs that turn more than ``fast`` times over the original length keep their frequency, those that turn fewer than
    ``slow`` times are slowed down by the whole factor, and the frequencies fall with the pair everywhere."""
    base, dims, original, factor = 10000.0, 64, 4096, 8.0
    plain, one = rotary_frequencies(dims, base)
    f, mag = rotary_frequencies(dims, base, (factor, original, 32.0, 1.0))
    assert one == 1.0 and mag == pytest.approx(0.1 * math.log(8.0) + 1.0)
    for a, b in zip(plain, f):
        turns = original * a / (2 * math.pi)
        if turns > 50:
            assert b == pytest.approx(a, rel=1e-12)
        elif turns < 0.5:
            assert b == pytest.approx(a / factor, rel=1e-12)
        assert a / factor * (1 - 1e-12) <= b <= a * (1 + 1e-12)
    assert all(x > y for x, y in zip(f, f[1:]))


def test_a_configuration_without_the_optional_entries():
    """Absent rotation, frequency scaling, loop and pair table mean none; a layer that names no feed-forward has none; the
    score scale defaults to the inverse root of the map's width."""
    c = config([attn(factor=None), delta(), attn(rot=0)], buckets=0)
    del c["layers"][2]["mixer"]["rot"], c["layers"][0]["mixer"]["scale"], c["layers"][1]["mlp"]
    cfg = config_from_dict(c)
    a, dl, p = cfg.layers
    assert a.scale == 12 ** -0.5 and a.rot_scaling is None and p.rot_dims == 0 and not dl.has_ff and cfg.pair is None and not cfg.looped
    full = config([attn(factor=None, scale=12 ** -0.5), delta(mlp=None), attn(rot=0)], buckets=0)
    W = oracle.random_weights(full, 1)
    eng, _ = build(c, "cpu", weights=W)
    toks = tokens(25, c["vocab"], 4)
    assert rel_err(replay_alone(eng, toks, [14]), oracle.forward(full, W, toks)) < 2e-4


def test_configurations_the_design_does_not_have_are_refused():
    for bad in ([delta(heads=4, kv=3)], [delta(dim=300)], [delta(conv=0)], [attn(heads=4, kv=3)], [attn(rot=5)], [attn(rot=14)],
                [attn(slow=0.0)], [attn(vdim=600)], [{"type": "mingru", "mixer": {"width": 8}, "mlp": None}],
                [attn(mlp={"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 2, "top": 1}})]):
        with pytest.raises(ValueError):
            config_from_dict(config(bad))
    with pytest.raises(ValueError):
        config_from_dict(config([delta()], loop=(0, 2, 2)))
    with pytest.raises(ValueError):
        config_from_dict({**config([delta()]), "embedding": {"bigram": {"buckets": 0, "mul_prev": 1, "mul_cur": 1}}})
