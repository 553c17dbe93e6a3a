"""The Nosalorn design in the engine against the plain implementation (``plain_nosalorn.py``): each mechanism
alone through the step function (attention with biases, stretched frequencies, a window and kept first keys;
values mixed with the first layer's; linear attention with fixed decays; the state space behind its
convolution; routed experts with corrected choice, groups, clamped gates, identity experts and a gated shared
one), whole models of several shapes in every way of cutting and batching, models drawn at random, inputs made
so that a key at a window's edge, a kept first key, an old state or a lost convolution input shows, decays that
run far below a number's range inside one chunk, long decoding, pages and slots used again, and greedy
generation through the engine's entry point and scheduler.  Sizes differ from model to model in every number
and include values that make mechanisms degenerate: one query head per key head and all on one, nothing
rotated, frequencies unstretched, no window and a window of one key, no kept keys, one group, one norm group,
one tap, one head, layers without feed-forward, no identity experts, no shared expert, a decay of one, sizes
that fill no tile.
"""
import json
import os
import random

import pytest
import torch

import plain_nosalorn as plain
from helpers import (EngineDriver, assert_close_f32, mixed_schedule, peak_tokens, portions_schedule, random_tokens,
                     tail_decode_schedule, whole_schedule)
from test_gpu_vabuzen import assert_close, doubles, run_alone

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
STD = 0.08
SWISH = 1.702


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, identity=None, groups=None, scale=None, shared=None):
    """shared: (ff, limit)."""
    router = {"experts": experts, "top": top}
    if identity is not None:
        router["identity"] = identity
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    if scale is not None:
        router["scale"] = scale
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    if shared:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def rotation(rot):
    """rot: (base, dims, None or (factor, original, fast, slow))."""
    out = {"base": rot[0], "dims": rot[1]}
    if rot[2]:
        out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), rot[2]))
    return out


def attention(heads, kv_heads, dim, vdim, scale, rot, mask, v_mix, mlp):
    """mask: (size, keep_first)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot:
        m["rot"] = rotation(rot)
    if mask:
        m["mask"] = {"size": mask[0], "keep_first": mask[1]}
    if v_mix:
        m["v_mix"] = True
    return {"type": "attention", "mixer": m, "mlp": mlp}


def lightning(heads, dim, vdim, decay, mlp):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def mamba(heads, vdim, state, groups, conv, norm_groups, mlp):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}, "mlp": mlp}


YARN = (8.0, 64, 8.0, 0.5)
# sizes the matrix cores and the fused products take; the first layer that mixes values is not the first attention layer
N1 = {"architecture": "Nosalorn", "vocab": 310, "width": 128, "norm": {"eps": 1e-5}, "embedding": {"scale": 9.0}, "logit_scale": 1.5,
      "layers": [attention(4, 2, 32, 64, 0.2, (20000.0, 16, YARN), (24, 3), False, dense(192)),
                 mamba(4, 32, 32, 2, 4, 2, moe(7, 3, 32, 1.0, 1, (4, 2), 2.5, (64, 0.8))),
                 attention(8, 4, 32, 32, 0.2, (500.0, 32, (4.0, 100, 32.0, 1.0)), (33, 20), True, dense(96)),
                 lightning(2, 32, 64, [0.7, 0.995], moe(8, 2, 64, 2.0, 4, (3, 2), 1.5, (32, 1.5))), mamba(8, 16, 64, 1, 4, 4, None),
                 attention(4, 2, 32, 64, 0.2, (20000.0, 16, YARN), (24, 3), True, moe(12, 4, 32, 0.7, 0, None, 2.0, None))]}
# a width that is no multiple of 16, heads no matrix-core kernel takes, all query heads on one key head, nothing rotated, a
# window of one key, a head alone, one tap, one number of state, experts of which all are chosen
N2 = {"architecture": "Nosalorn", "vocab": 211, "width": 72, "norm": {"eps": 3e-6},
      "layers": [lightning(1, 20, 12, [1.0], dense(40)), attention(5, 1, 12, 20, 0.3, None, (1, 0), True, moe(3, 3, 24, 1.3)),
                 mamba(1, 12, 1, 1, 1, 1, dense(56)), attention(2, 2, 9, 10, 0.35, (300.0, 4, None), None, True, None),
                 mamba(6, 10, 20, 3, 2, 5, moe(4, 1, 20, 0.5, 2, (6, 1), 3.0, (12, 0.6))),
                 attention(4, 4, 10, 5, 0.3, (100.0, 10, (2.0, 30, 4.0, 1.0)), (7, 2), True, dense(24))]}
# wide heads: keys of 128 and 96, states whose sizes are no multiples of 16 and larger than 128, six taps
N3 = {"architecture": "Nosalorn", "vocab": 260, "width": 160, "norm": {"eps": 1e-4}, "embedding": {"scale": 3.0}, "logit_scale": 0.7,
      "layers": [mamba(2, 144, 72, 1, 6, 3, dense(96)), attention(2, 1, 128, 96, 0.1, (10000.0, 128, (16.0, 40, 2.0, 2.0)), (65, 70), True, dense(64)),
                 lightning(2, 136, 300, [0.9, 0.999], moe(33, 3, 40, 1.0, 3, (12, 5), 2.0, (48, 1.0))),
                 attention(4, 1, 80, 96, 0.1, (777.0, 40, YARN), None, True, None), mamba(3, 40, 136, 3, 3, 1, dense(96))]}
# sizes that are multiples of two only
N4 = {"architecture": "Nosalorn", "vocab": 333, "width": 100, "norm": {"eps": 1e-6}, "embedding": {"scale": 2.0},
      "layers": [attention(3, 3, 18, 22, 0.22, (777.0, 14, YARN), (40, 1), True, moe(5, 2, 18, 0.9, 1, (2, 1), 1.0, (14, 1.1))),
                 lightning(3, 10, 14, [0.5, 0.97, 1.0], dense(34)), mamba(5, 14, 6, 5, 5, 7, moe(6, 2, 22, 1.0, 4, (5, 3), 0.5, None)),
                 attention(6, 3, 14, 22, 0.25, None, None, True, None), lightning(5, 6, 30, [0.9] * 5, None)]}
MODELS = {"N1": (N1, 61), "N2": (N2, 62), "N3": (N3, 63), "N4": (N4, 64)}
LENGTHS = {"N1": [40, 57, 90, 150, 65, 33], "N2": [45, 130, 64, 100, 17, 33], "N3": [31, 32, 150, 64, 49, 80], "N4": [70, 19, 101, 64, 13, 50]}
SCHEDULES = {"whole": whole_schedule, "tail12": lambda reqs: tail_decode_schedule(reqs, tail=12),
             "portions": portions_schedule, "mixed": mixed_schedule}


def write_model(folder, cfg, seed, storage=torch.float32, std=STD, change=None):
    """A model folder of random tensors for ``cfg``; ``change``: name -> function of the drawn tensor."""
    from celeg_amd import native
    from celeg_amd.weights import random_tensors
    from celeg_amd.weights.safetensors_io import write_safetensors
    expected = native.describe_config(cfg)["expected_tensors"]
    tensors = random_tensors(expected, seed, std, torch.float32)
    for name in tensors:
        unit = tensors[name] / std
        if name.endswith(".vmix"):
            tensors[name] = 0.45 + 0.2 * unit
        elif name.endswith((".q.b", ".k.b", ".v.b")):
            tensors[name] = 0.4 * unit
        elif name.endswith(".A_log"):
            tensors[name] = 0.8 * unit - 1.0
        elif name.endswith(".dt_bias"):
            tensors[name] = unit - 1.5              # steps on both sides of one, states that last
        elif name.endswith(".D"):
            tensors[name] = 1.0 + 0.3 * unit
        elif name.endswith(".conv"):
            tensors[name] = 0.5 * unit
        elif name.endswith(".conv.b"):
            tensors[name] = 0.3 * unit
        elif name.endswith(".correction"):
            tensors[name] = 0.1 * unit - 0.1        # choice scores on both sides of zero
        elif name.endswith(".router"):
            tensors[name] = 2.0 * tensors[name]
        elif name == "embed":
            tensors[name] = 3.0 * tensors[name]
    # a state read with a query at right angles to its keys is a small number that the norm behind it makes large,
    # sign and all: keys that lean towards the queries keep rounding from deciding such rows
    for i, layer in enumerate(cfg["layers"]):
        if layer["type"] == "lightning":
            p = f"l{i}.mix."
            tensors[p + "k"] = 0.5 * tensors[p + "k"] + 0.9 * tensors[p + "q"]
    for name, fn in (change or {}).items():
        tensors[name] = fn(tensors[name])
    tensors = {k: v.to(storage).contiguous() for k, v in tensors.items()}
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    write_safetensors(os.path.join(folder, "model.safetensors"), tensors)
    return str(folder)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            cfg, seed = MODELS[name]
            storage = torch.float32 if dtype == "float32" else torch.bfloat16
            made[(name, dtype)] = write_model(tmp_path_factory.mktemp(f"{name}_{dtype}"), cfg, seed, storage)
        return made[(name, dtype)]
    return get


_plain = {}


def requests_of(name):
    cfg, seed = MODELS[name]
    return {f"r{i}": random_tokens(cfg["vocab"], n, seed=100 * seed + i) for i, n in enumerate(LENGTHS[name])}


def plain_logits(folder, key, requests):
    if key not in _plain:
        cfg, W = plain.load_model_folder(folder)
        _plain[key] = {rid: plain.model_logits(cfg, W, toks) for rid, toks in requests.items()}
    return _plain[key]


def load(folder, dtype, steps, max_requests=4, **kw):
    from celeg_amd.engine import load_model
    max_tokens = peak_tokens(steps)
    lm = load_model(folder, dtype=dtype, device=DEV, page_tokens=16, n_pages=max_tokens // 16, max_requests=max_requests,
                    max_context=max_tokens, max_batched_tokens=max(max_tokens, 64), **kw)
    return lm, max_tokens


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("mode", list(SCHEDULES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MODELS))
def test_engine_matches_plain(folders, name, dtype, mode):
    """Whole prompts; prefill then 12 tokens one by one; portions down to two tokens (and single
    ones) that cross page borders; four live requests with pages and slots used again."""
    folder = folders(name, dtype)
    reqs = requests_of(name)
    steps = SCHEDULES[mode](reqs)
    lm, max_tokens = load(folder, dtype, steps)
    got = EngineDriver(lm).run(steps)
    ref = plain_logits(folder, (name, dtype), reqs)
    for rid in reqs:
        assert_close(got[rid], ref[rid], dtype, f"{name}/{dtype}/{mode}/{rid}")
    lm.cache.check()
    assert lm.cache.n_free_slots == 4 and lm.cache.free_pages() == [max_tokens // 16] * len(lm.cache.free_pages())
    paths = lm.paths()
    assert paths["attention_biased"] > 0 and paths["decay_scan"] > 0 and paths["routed_experts"] > 0
    if mode != "whole":
        assert paths["decay_scan_step"] > 0
    if mode != "tail12":
        assert paths["decay_scan_rows"] > 0
    if dtype == "bfloat16" and name in ("N1", "N3"):
        assert paths["attention_biased_rows"] + paths["attention_biased_decode"] > 0     # the matrix cores took these heads


@pytest.mark.parametrize("name", ["N1", "N2", "N4"])
def test_residual_stream_after_every_layer(folders, tmp_path, monkeypatch, name):
    """32-bit: the stream behind each layer as CELEG_DUMP_HIDDEN writes it, for a prompt's portion and two
    single tokens, against the plain layers: the first that differs is where a fault lies."""
    import numpy as np
    from celeg_amd.engine import StepEntry, load_model
    cfg, _ = MODELS[name]
    folder = folders(name, "float32")
    _, W = plain.load_model_folder(folder)
    toks = random_tokens(cfg["vocab"], 23, seed=2)
    after = plain.model_hidden(cfg, W, toks)
    dump = str(tmp_path / "hidden")
    monkeypatch.setenv("CELEG_DUMP_HIDDEN", dump)
    lm = load_model(folder, dtype="float32", page_tokens=16, n_pages=8, max_requests=2, max_batched_tokens=64)
    monkeypatch.delenv("CELEG_DUMP_HIDDEN")
    slot = lm.cache.open()
    assert lm.cache.prepare(slot, 0, 23)
    for k, (start, n) in enumerate([(0, 21), (21, 1), (22, 1)]):
        lm.runner.step([StepEntry(slot, start, toks[start:start + n], [n - 1])])
        for i in range(len(after)):
            rows = np.fromfile(os.path.join(dump, f"step{k}_layer{i}.f32"), dtype="<f4").reshape(n, cfg["width"])
            assert_close_f32(torch.from_numpy(rows), after[i][start:start + n], f"step {k}, layer {i}")
    lm.close()


@pytest.mark.parametrize("name", ["N1", "N3"])
def test_batches_of_unequal_requests_equal_each_alone(folders, name):
    """In 32-bit a row's logits depend on the cut of its prompt and on the batch by no more than the
    rounding of sums taken in another order (the states' chunks of 64 rows begin where a portion begins)."""
    folder = folders(name, "float32")
    reqs = requests_of(name)
    alone_steps, mixed_steps, cut_steps = whole_schedule(reqs), mixed_schedule(reqs, seed=3), portions_schedule(reqs)
    lm, _ = load(folder, "float32", alone_steps)
    alone = EngineDriver(lm).run(alone_steps)
    for steps in (mixed_steps, cut_steps):
        lm2, _ = load(folder, "float32", steps)
        other = EngineDriver(lm2).run(steps)
        for rid in reqs:
            assert float((alone[rid] - other[rid]).abs().max()) <= 5e-5 * float(alone[rid].abs().max()), rid


def test_the_fused_products_and_the_plain_ones_agree(folders):
    """bfloat16: steps whose products take norms and sums along against the same steps with separate kernels;
    the first form runs (its paths count) and both are within rounding of each other."""
    folder = folders("N1", "bfloat16")
    reqs = requests_of("N1")
    steps = mixed_schedule(reqs, seed=6)
    got = {}
    for fused in (1, 0):
        lm, _ = load(folder, "bfloat16", steps)
        lm.set_knob("use_fused", fused)
        got[fused] = EngineDriver(lm).run(steps)
        taken = sum(lm.paths()[p] for p in ("fused_sliced", "fused_rows", "tiled"))
        assert (taken > 0) == bool(fused)
        lm.close()
    for rid in reqs:
        assert_close(got[1][rid], got[0][rid], "bfloat16", rid)


def drawn_model(rng):
    """A configuration drawn at random: widths, head counts and sizes (those the matrix cores take, and
    others), order and number of layers, windows, kept keys, rotations, decays, taps, groups and routers."""
    cfg = {"architecture": "Nosalorn", "vocab": rng.randint(100, 700), "width": rng.choice([64, 96, 160, 192, 200, 320]),
           "norm": {"eps": rng.choice([1e-6, 1e-5])}, "embedding": {"scale": round(rng.uniform(0.5, 8.0), 3)},
           "logit_scale": round(rng.uniform(0.3, 2.0), 3)}
    mixed = rng.choice([(1, 64), (2, 32), (4, 16), (2, 48), (3, 20)])          # key heads and value size of the layers that mix
    layers = []
    for _ in range(rng.randint(3, 6)):
        kind = rng.random()
        if kind < 0.15:
            mlp = None
        elif kind < 0.4:
            mlp = dense(rng.choice([64, 128, 200, 256]))
        else:
            count, per = rng.choice([(1, 9), (2, 7), (4, 3), (3, 8), (6, 2)])
            keep = rng.randint(1, count)
            total = count * per
            identity = rng.choice([0, 1, 2, total // 3])
            mlp = moe(total - identity, rng.randint(1, min(4, keep * per)), rng.choice([32, 64, 96, 40]), round(rng.uniform(0.4, 3.0), 2), identity,
                      (count, keep) if count > 1 else None, round(rng.uniform(0.5, 3.0), 2),
                      (rng.choice([32, 64, 72]), round(rng.uniform(0.4, 3.0), 2)) if rng.random() < 0.7 else None)
        kind = rng.choice(["a", "a", "l", "m"])
        if kind == "a":
            v_mix = rng.random() < 0.7
            kv, vdim = mixed if v_mix else (rng.choice([1, 2, 3]), rng.choice([16, 32, 48, 64, 96]))
            dim = rng.choice([16, 32, 40, 64, 80, 128])
            rot = None if rng.random() < 0.15 else (rng.choice([1000.0, 50000.0]), rng.choice([dim, dim // 2, 8]),
                                                    (round(rng.uniform(1.5, 16.0), 2), rng.choice([32, 100, 1024]), rng.choice([8.0, 32.0]),
                                                     rng.choice([0.5, 1.0])) if rng.random() < 0.8 else None)
            mask = (rng.choice([1, 5, 16, 31, 64, 65, 100]), rng.choice([0, 1, 4, 17])) if rng.random() < 0.8 else None
            layers.append(attention(kv * rng.choice([1, 2, 4]), kv, dim, vdim, round(dim ** -0.5 * rng.uniform(0.7, 1.5), 4), rot, mask, v_mix, mlp))
        elif kind == "l":
            heads = rng.choice([1, 2, 3, 4, 8])
            layers.append(lightning(heads, rng.choice([8, 16, 24, 32, 48, 64, 96]), rng.choice([16, 32, 40, 64, 128]),
                                    [round(1.0 - 0.5 ** rng.uniform(0.5, 10.0), 6) for _ in range(heads)], mlp))
        else:
            groups = rng.choice([1, 2, 4])
            heads = groups * rng.choice([1, 2, 3])
            vdim = rng.choice([8, 16, 32, 40, 64])
            layers.append(mamba(heads, vdim, rng.choice([8, 16, 40, 48, 64, 128]), groups, rng.choice([2, 3, 4, 5]),
                                rng.choice([1, groups, heads, 4 if vdim % 4 == 0 else 1]), mlp))
    cfg["layers"] = layers
    return cfg


@pytest.mark.parametrize("seed", range(8))
def test_models_drawn_at_random(tmp_path, seed):
    """Eight models drawn at random, weights stored in bfloat16, four requests of 20 to 200 tokens,
    in a mixed schedule and in long and short portions, in 32-bit and in bfloat16.  For bfloat16 the corrections lie
    further apart than scores can, so that no choice of experts hangs on the rounding of a row (a changed choice moves the row
    and, through states and keys, all later ones); the choices themselves are what the 32-bit runs hold."""
    rng = random.Random(4000 + seed)
    cfg = drawn_model(rng)
    reqs = {f"r{i}": random_tokens(cfg["vocab"], rng.randint(20, 200), seed=seed * 10 + i) for i in range(4)}
    tail = rng.randint(3, 20)
    for dtype in ("float32", "bfloat16"):
        decided = {f"l{i}.mlp.correction": lambda w: 1.5 * w.argsort().argsort().float() for i, layer in enumerate(cfg["layers"])
                   if layer["mlp"] and layer["mlp"]["kind"] == "moe" and dtype == "bfloat16"}
        folder = write_model(tmp_path / dtype, cfg, seed, torch.bfloat16, std=0.06, change=decided)
        c, W = plain.load_model_folder(folder)
        ref = {rid: plain.model_logits(c, W, toks) for rid, toks in reqs.items()}
        for steps in (mixed_schedule(reqs, seed=seed, decode_tail=tail), portions_schedule(reqs, sizes=(70, 2, 33, 1, 130, 16, 5))):
            lm, _ = load(folder, dtype, steps)
            got = EngineDriver(lm).run(steps)
            for rid in reqs:
                assert_close(got[rid], ref[rid], dtype, f"drawn model {seed}/{dtype}/{rid}: {json.dumps(cfg)}")
            lm.close()


# ------------------------------------------------------------------ long decoding, pages and slots
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_while_the_windows_pass(folders, dtype):
    """A short prompt, then 200 tokens one by one (steps replayed from a recorded graph): the windows of 24 and
    33 keys pass wholly over decoded tokens while the kept first keys stay, pages go back to the pool, and the
    states live in their slots alone."""
    folder = folders("N1", dtype)
    toks = random_tokens(N1["vocab"], 215, seed=77)
    steps = tail_decode_schedule({"long": toks}, tail=200)
    lm, _ = load(folder, dtype, steps)
    got = EngineDriver(lm).run(steps)["long"]
    c, W = plain.load_model_folder(folder)
    assert_close(got, plain.model_logits(c, W, toks), dtype, "long decoding")
    assert lm.runner.counters()["graph_replays"] > 100


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_replayed_from_a_recorded_graph(folders, dtype):
    """Portions of 70 tokens of three requests, one after the other and with single tokens of another request
    between them: from the second on they are replayed from a recorded graph (a chunk of the states and six rows
    of a second one), and every portion's last logits are the plain ones."""
    from celeg_amd.engine import StepEntry, load_model
    folder = folders("N1", dtype)
    c, W = plain.load_model_folder(folder)
    lm = load_model(folder, dtype=dtype, device=DEV, page_tokens=16, n_pages=64, max_requests=3, max_context=256, max_batched_tokens=128)
    other = random_tokens(N1["vocab"], 9, seed=90)
    other_slot, at = lm.cache.open(), 0
    other_ref = plain.model_logits(c, W, other)
    got_rows, ref_rows = [], []
    for r in range(3):
        toks = random_tokens(N1["vocab"], 210, seed=91 + r)
        ref = plain.model_logits(c, W, toks)
        slot = lm.cache.open()
        for start in (0, 70, 140):
            assert lm.cache.prepare(slot, start, 70)
            got = lm.runner.step([StepEntry(slot, start, toks[start:start + 70], [69])]).detach().cpu()
            got_rows.append(got[0].clone())
            ref_rows.append(ref[start + 69])
            assert lm.cache.prepare(other_slot, at, 1)
            single = lm.runner.step([StepEntry(other_slot, at, other[at:at + 1], [0])]).detach().cpu()
            got_rows.append(single[0].clone())
            ref_rows.append(other_ref[at])
            at += 1
        lm.cache.close(slot)
    assert_close(torch.stack(got_rows), torch.stack(ref_rows), dtype, "portions and single tokens in turn")
    assert lm.runner.counters()["graph_replays"] >= 16
    lm.close()


def test_pages_of_passed_windows_return_and_kept_ones_stay(folders):
    """While a request grows, its window groups hold the pages of the window and of the kept first keys only."""
    from celeg_amd.engine import StepEntry, load_model
    folder = folders("N1", "float32")
    toks = random_tokens(N1["vocab"], 200, seed=5)
    lm = load_model(folder, dtype="float32", device=DEV, page_tokens=16, n_pages=16, max_requests=2, max_context=256, max_batched_tokens=256)
    slot = lm.cache.open()
    assert lm.cache.prepare(slot, 0, 150)
    lm.runner.step([StepEntry(slot, 0, toks[:150], [149])])
    assert lm.cache.prepare(slot, 150, 50)
    logits = lm.runner.step([StepEntry(slot, 150, toks[150:], list(range(50)))]).detach().cpu()
    # windows of 24 and 33 from position 150 on: pages 7 to 12 of 13 (positions 127 and 118 lie in page 7), plus page 0
    # for three kept keys, and pages 0 and 1 for twenty
    assert sorted(len(p) for p in lm.cache.pages_held(slot)) == [7, 8]
    c, W = plain.load_model_folder(folder)
    assert_close_f32(logits, plain.model_logits(c, W, toks)[150:], "after the windows passed")
    lm.cache.close(slot)
    lm.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_pages_and_slots_used_again(folders, dtype):
    """Ten requests through two slots and a pool of six pages: every page and state slot serves several
    requests (a state or a convolution's saved input that outlives its request would show at the next one's
    first tokens)."""
    from celeg_amd.engine import load_model
    folder = folders("N1", dtype)
    reqs = {f"q{i}": random_tokens(N1["vocab"], n, seed=500 + i) for i, n in enumerate([30, 18, 33, 16, 5, 47, 31, 1, 40, 17])}
    steps = mixed_schedule(reqs, max_live=2, seed=4, decode_tail=6)
    lm = load_model(folder, dtype=dtype, device=DEV, page_tokens=16, n_pages=6, max_requests=2, max_context=64, max_batched_tokens=128)
    got = EngineDriver(lm).run(steps)
    c, W = plain.load_model_folder(folder)
    for rid, toks in reqs.items():
        assert_close(got[rid], plain.model_logits(c, W, toks), dtype, rid)
    assert all(n == 6 for n in lm.cache.free_pages())


# ------------------------------------------------------------------ generation through the entry point
@pytest.mark.parametrize("name", ["N1", "N2"])
def test_greedy_generation_through_the_entry_point(folders, name):
    """More requests than places, prompts cut by a token budget, steps launched before the last token is on
    the host."""
    from celeg_amd.engine import Engine
    from celeg_amd.sampling import GenerationConfig
    folder = folders(name, "float32")
    cfg, W = plain.load_model_folder(folder)
    prompts = [random_tokens(cfg["vocab"], n, seed=40 + n) for n in (5, 23, 1, 37, 12)]
    engine = Engine.from_folder(folder, dtype="float32", device=DEV, max_active_requests=3, max_batched_tokens=64,
                                prefill_chunk_tokens=16, context=128, n_pages=24)
    greedy = GenerationConfig(temperature=0.0, repetition_penalty=1.0)
    outs = engine.generate(prompts, max_new_tokens=14, generation=greedy, eos_token_ids=[])
    for prompt, out in zip(prompts, outs):
        assert out == plain.greedy(cfg, W, prompt, 14)
    engine.close()


def test_command_line(folders, tmp_path):
    """``bin/celeg-run`` on a model folder of the design: greedy tokens and the prompt's last logits."""
    import subprocess
    import sys
    import numpy as np
    folder = folders("N4", "float32")
    cfg, W = plain.load_model_folder(folder)
    prompt = random_tokens(cfg["vocab"], 19, seed=5)
    dump = str(tmp_path / "logits.f32")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "celeg-run"), "--model", folder, "--dtype", "float32", "--prompt",
                           ",".join(map(str, prompt)), "--max-new-tokens", "8", "--repetition-penalty", "1.0", "--context", "128",
                           "--runtime-tokens", "--dump-logits", dump], capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr
    line = [l for l in proc.stdout.splitlines() if l.startswith("CELEG_GENERATED_TOKEN_IDS=")][0]
    assert json.loads(line.split("=", 1)[1]) == plain.greedy(cfg, W, prompt, 8)
    logits = np.fromfile(dump, dtype="<f4")
    assert_close_f32(torch.from_numpy(logits.copy()), plain.model_logits(cfg, W, prompt)[-1], "command line")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_program(folders, tmp_path, dtype):
    """``bin/trace_run`` in a process of its own: four schedules one after the other, a pool sized for
    the live requests only, logits read from the files it writes."""
    from helpers import TraceClient
    folder = folders("N1", dtype)
    reqs = requests_of("N1")
    ref = plain_logits(folder, ("N1", dtype), reqs)
    all_steps = []
    for tag, make in (("w", whole_schedule), ("t", tail_decode_schedule), ("p", portions_schedule), ("m", mixed_schedule)):
        for s in make({f"{tag}{rid}": toks for rid, toks in reqs.items()}):
            all_steps.append(dict(s, step=len(all_steps)))
    client = TraceClient(folder, dtype, str(tmp_path), peak_tokens(all_steps))
    got = {}
    for s in all_steps:
        logits = client.step(s["step"], s["entries"], s["end"])
        row = 0
        for e in s["entries"]:
            for _ in e["want"]:
                got.setdefault(e["id"], []).append(torch.as_tensor(logits[row]))
                row += 1
    assert client.close() == 0
    for rid_tagged, rows in got.items():
        assert_close(torch.stack(rows), ref[rid_tagged[1:]], dtype, f"trace/{dtype}/{rid_tagged}")


# ------------------------------------------------------------------ each mechanism alone
EPS = 1e-5
LONG_CUT = (130, 2, 97, 31, 16, 1, 7) + (1,) * 16


def attention_case(T, W_, H, G, D, V, scale, rot=None, mask=None, seed=1, x_std=1.0, bias_std=0.7):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    t = {"table": r(T, W_) * x_std, "q": r(H * D, W_) * 0.3, "k": r(G * D, W_) * 0.3, "v": r(G * V, W_) * 0.3, "o": r(W_, H * V) * 0.3,
         "q.b": r(H * D) * bias_std, "k.b": r(G * D) * bias_std, "v.b": r(G * V) * bias_std}
    params = {"width": W_, "heads": H, "kv_heads": G, "head_dim": D, "v_dim": V, "scale": scale, "bias": True}
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": scale}
    if rot:
        m["rot"] = rotation(rot)
        rope = {"theta": rot[0], "rotary_dim": rot[1], "head_dim": D, "pairing": "halves"}
        if rot[2]:
            rope["scaling"] = dict(m["rot"]["scaling"], rule="yarn")
        params["position"] = {"kind": "rope", "params": rope}
    if mask:
        m["mask"] = {"size": mask[0], "keep_first": mask[1]}
        params["window"], params["keep_first"] = mask
    names = {c: c for c in ("q", "k", "v", "o")}
    return t, m, {"kind": "biased_attention", "params": params, "tensors": dict(names, q_bias="q.b", k_bias="k.b", v_bias="v.b")}


@pytest.mark.parametrize("G,D,V,rot,mask", [(3, 12, 20, (100.0, 12, (4.0, 20, 4.0, 0.5)), (9, 2)), (1, 8, 8, None, None),
                                            (6, 32, 16, (10000.0, 4, (32.0, 64, 32.0, 1.0)), (16, 0)), (2, 7, 9, (50.0, 6, (1.0, 40, 2.0, 1.0)), (1, 3)),
                                            (2, 16, 64, (1000.0, 2, None), (17, 20)), (3, 64, 32, (10000.0, 64, (8.0, 30, 3.0, 3.0)), None)])
def test_attention_with_biases_and_stretched_rotation_alone(tmp_path, G, D, V, rot, mask):
    T, W_ = 45, 40
    t, m, part = attention_case(T, W_, 6, G, D, V, 0.4, rot, mask)
    got, _ = run_alone(tmp_path, {"width": W_, "rows": T, "mixer": part}, t)
    Wd = doubles(t)
    assert_close_f32(got, Wd["table"] + plain.window_attention(Wd["table"], Wd, "", m, EPS, {}), "attention alone")


@pytest.mark.parametrize("D,V", [(32, 32), (64, 64), (64, 128), (96, 60), (104, 12), (128, 96)])
def test_matrix_core_attention_equals_the_general_kernel(tmp_path, D, V):
    """bfloat16: the kernels on the matrix cores against the kernel that scores key by key, on the same pages,
    with windows and kept first keys at the borders of pages and blocks, in whole prompts, portions and single
    tokens.  The two differ in the rounding of the weights to bfloat16 numbers only."""
    T, W_ = 300, 64
    for mask in ((7, 3), (64, 64), (65, 1), (40, 4), None):
        t, m, part = attention_case(T, W_, 4, 2, D, V, D ** -0.5, (10000.0, D // 2, (4.0, 64, 8.0, 1.0)), mask, seed=D + V, x_std=1.5)
        got = {}
        long_cut = (15, 2, 17, 1, 130, 3, 16, 64)
        for form, cut in (("general", long_cut), (-1, long_cut), (-1, (300,)), (-1, (270,) + (1,) * 30)):
            knobs = {"use_biased_mfma": 0} if form == "general" else {"biased_rows_form": form}
            out, lm = run_alone(tmp_path / f"{mask}_{form}_{len(cut)}", {"width": W_, "rows": T, "mixer": part}, t, cut=cut, dtype="bfloat16",
                                knobs=knobs, n_pages=20)
            took = lm.paths()["attention_biased_rows"] + lm.paths()["attention_biased_decode"]
            assert (took > 0) == (form != "general")
            got[(form, len(cut))] = out
        ref = got[("general", 8)]
        for key, out in got.items():
            rel = float((out - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt())
            assert rel <= 1e-2, f"heads of {D} and {V}, mask {mask}, {key}: rel rms {rel:.3e}"


def edge_case(size, keep, rot=None):
    """Rows whose weight sits on one key: the last key inside the window and the first one outside, the last kept
    first key hundreds of positions back and the first one not kept, for rows inside a prompt's portion and rows
    decoded alone.  Queries and keys are the same map of the input's first half, in which the marked rows point one
    way and are long; the marked rows differ in the second half, which only the values read.  With rot, the first
    half of a head turns and the maps feed the other half only."""
    T, W_, H, D = 300, 32, 2, 32
    t, m, part = attention_case(T, W_, H, H, D, D, 0.25, rot, (size, keep), seed=5, x_std=0.3, bias_std=0.1)
    t["q"][:, W_ // 2:] = 0.0
    if rot:
        t["q"] *= 1.4
        t["q"].view(H, D, W_)[:, :rot[1]] = 0.0
    t["k"] = t["q"].clone()
    g = torch.Generator().manual_seed(9)
    direction = torch.randn(W_, generator=g)
    direction[W_ // 2:] = 0.0
    direction = direction / direction.norm()
    queries = (200, 290)
    for row in (keep - 1, keep) + tuple(q - size + 1 for q in queries) + tuple(q - size for q in queries):
        own = torch.randn(W_, generator=g)
        own[:W_ // 2] = 0.0
        t["table"][row] = 8.0 * direction + 6.0 * own / own.norm()
    for row in queries:
        t["table"][row] = 2.0 * direction
    return t, m, part, queries


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size,keep,rot", [(40, 5, None), (64, 4, (10000.0, 16, (4.0, 32, 8.0, 1.0))), (33, 17, None)])
def test_keys_at_the_windows_edge_and_kept_first_keys(tmp_path, dtype, size, keep, rot):
    """The plain result with a window or a number of kept keys that is one off differs in the marked rows by more
    than a tenth."""
    t, m, part, queries = edge_case(size, keep, rot)
    Wd = doubles(t)
    want = Wd["table"] + plain.window_attention(Wd["table"], Wd, "", m, EPS, {})
    for other in ((size + 1, keep), (size - 1, keep), (size, keep + 1), (size, keep - 1)):
        off = Wd["table"] + plain.window_attention(Wd["table"], Wd, "", dict(m, mask={"size": other[0], "keep_first": other[1]}), EPS, {})
        for row in queries:
            assert float((want[row] - off[row]).abs().max()) > 0.1 * float(want[row].abs().max()), (other, row)
    got, lm = run_alone(tmp_path, {"width": 32, "rows": 300, "mixer": part}, t, cut=LONG_CUT, dtype=dtype, n_pages=20)
    if dtype == "float32":
        assert_close_f32(got, want, "keys at the edges")
    else:
        Wb = {k_: v.bfloat16().double() for k_, v in Wd.items()}
        ref = Wb["table"] + plain.window_attention(Wb["table"], Wb, "", m, EPS, {})
        for row in queries + (120, 299):
            assert float((got[row] - ref[row]).abs().max()) <= 0.04 * float(ref[row].abs().max()), row
        assert lm.paths()["attention_biased_rows"] > 0 and lm.paths()["attention_biased_decode"] > 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_values_mixed_with_the_first_layers(tmp_path, dtype):
    """Four attention layers, of which the second keeps its values and the third and fourth mix (numbers of
    0.9 and -0.7, so that kept values of another token, another request or another step give other logits),
    with the same values in other head shapes; the kept values' own number is stored and not used."""
    cfg = {"architecture": "Nosalorn", "vocab": 140, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 4.0},
           "layers": [attention(2, 2, 16, 24, 0.25, None, None, False, None), attention(4, 2, 16, 16, 0.25, (100.0, 8, YARN), (30, 2), True, dense(32)),
                      attention(4, 1, 32, 32, 0.2, None, (9, 1), True, None), attention(4, 4, 16, 8, 0.2, None, None, True, None)]}
    storage = torch.float32 if dtype == "float32" else torch.bfloat16
    put = lambda x: lambda w: torch.full_like(w, x)
    folder = write_model(tmp_path / "mix", cfg, 7, storage, std=0.1,
                         change={"l1.mix.vmix": put(100.0), "l2.mix.vmix": put(0.9), "l3.mix.vmix": put(-0.7)})
    c, W = plain.load_model_folder(folder)
    reqs = {"a": random_tokens(cfg["vocab"], 120, seed=3), "b": random_tokens(cfg["vocab"], 90, seed=4), "c": random_tokens(cfg["vocab"], 31, seed=5)}
    ref = {rid: plain.model_logits(c, W, toks) for rid, toks in reqs.items()}
    for name in ("l2.mix.vmix", "l3.mix.vmix"):
        off = plain.model_logits(c, dict(W, **{name: torch.zeros_like(W[name])}), reqs["a"])
        assert float((off - ref["a"]).abs().max()) > 0.05 * float(ref["a"].abs().max()), name
    for steps in (tail_decode_schedule(reqs, tail=30), portions_schedule(reqs, sizes=(37, 2, 3, 1, 4, 5, 2, 16, 1, 31)),
                  mixed_schedule(reqs, seed=5, decode_tail=10)):
        lm, _ = load(folder, dtype, steps)
        got = EngineDriver(lm).run(steps)
        for rid in reqs:
            assert_close(got[rid], ref[rid], dtype, f"mixed values/{dtype}/{rid}")
        lm.close()


def decay_case(T, W_, H, D, V, decay, seed=4, x_std=1.0):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    t = {"table": r(T, W_) * x_std, "q": r(H * D, W_) * 0.3, "v": r(H * V, W_) * 0.3, "g": r(H * V, W_) * 0.3, "norm": 1 + 0.3 * r(H * V),
         "o": r(W_, H * V) * 0.3}
    t["k"] = 0.6 * t["q"] + 0.2 * r(H * D, W_)
    m = {"heads": H, "dim": D, "vdim": V, "decay": decay}
    params = {"width": W_, "heads": H, "dim": D, "vdim": V, "decay": decay, "eps": EPS}
    return t, m, {"kind": "fixed_decay_attention", "params": params, "tensors": {c: c for c in ("q", "k", "v", "g", "norm", "o")}}


@pytest.mark.parametrize("H,D,V,decay", [(3, 12, 20, [0.5, 0.9, 0.99]), (1, 16, 16, [1.0]), (2, 32, 64, [1e-6, 0.999]), (4, 7, 5, [0.8] * 4),
                                         (1, 256, 40, [0.95]), (1, 40, 1100, [0.97]), (2, 130, 258, [0.6, 0.98]), (2, 1, 1, [0.9, 0.3])])
def test_linear_attention_with_fixed_decays_alone(tmp_path, H, D, V, decay):
    """Portions of 5, 2, 9, 1, ... rows, then whole chunks, a chunk and a row, a chunk less a row; a decay of one
    (nothing is forgotten) and decays so small that their power over a chunk is no 32-bit number."""
    T, W_ = 150, 40
    t, m, part = decay_case(T, W_, H, D, V, decay)
    Wd = doubles(t)
    want = Wd["table"] + plain.fixed_decay_attention(Wd["table"], Wd, "", m, EPS, {})
    for cut in ((5, 2, 9, 1, 3, 17), (150,), (64, 65, 21), (63, 1, 64, 1, 21)):
        got, lm = run_alone(tmp_path / str(len(cut)), {"width": W_, "rows": T, "mixer": part}, t, cut=cut, n_pages=12)
        assert_close_f32(got, want, f"fixed decays alone, portions {cut}")
        assert lm.paths()["decay_scan_rows"] > 0


def space_case(T, W_, H, V, N, G, taps, parts, seed=6, x_std=1.0, a_log=-1.0, dt=-1.0):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    inner, channels = H * V, H * V + 2 * G * N
    t = {"table": r(T, W_) * x_std, "in": r(inner + channels + H, W_) * 0.3, "conv": r(channels, taps) * 0.6, "conv.b": r(channels) * 0.4,
         "dt_bias": r(H) + dt, "A_log": r(H) * 0.7 + a_log, "D": 1 + 0.4 * r(H), "norm": 1 + 0.3 * r(inner), "o": r(W_, inner) * 0.3}
    m = {"heads": H, "vdim": V, "state": N, "groups": G, "conv": taps, "norm_groups": parts}
    params = {"width": W_, "heads": H, "vdim": V, "state": N, "groups": G, "taps": taps, "norm_groups": parts, "eps": EPS}
    names = {c: c for c in ("in", "conv", "dt_bias", "A_log", "D", "norm", "o")}
    return t, m, {"kind": "state_space", "params": params, "tensors": dict(names, conv_bias="conv.b")}


@pytest.mark.parametrize("H,V,N,G,taps,parts", [(6, 10, 12, 3, 4, 5), (1, 16, 16, 1, 1, 1), (4, 32, 64, 2, 4, 2), (4, 7, 5, 4, 2, 4), (2, 40, 256, 1, 3, 1),
                                                (1, 1100, 24, 1, 6, 11), (2, 258, 130, 2, 4, 1), (8, 4, 1, 2, 9, 8)])
def test_state_space_alone(tmp_path, H, V, N, G, taps, parts):
    """Taps of one to nine (longer than some portions), one group and a group per head, one norm for all and one
    per head, states of one number and of more than a tile's."""
    T, W_ = 150, 40
    t, m, part = space_case(T, W_, H, V, N, G, taps, parts)
    Wd = doubles(t)
    want = Wd["table"] + plain.state_space(Wd["table"], Wd, "", m, EPS, {})
    for cut in ((5, 2, 9, 1, 3, 17), (150,), (64, 65, 21), (63, 1, 64, 1, 21)):
        got, lm = run_alone(tmp_path / str(len(cut)), {"width": W_, "rows": T, "mixer": part}, t, cut=cut, n_pages=12)
        assert_close_f32(got, want, f"state space alone, portions {cut}")
        assert lm.paths()["decay_scan_rows"] > 0


@pytest.mark.parametrize("a_log,dt", [(2.5, 1.0), (-6.0, 3.0), (0.0, -12.0)])
def test_decays_from_the_input_keep_their_precision(tmp_path, a_log, dt):
    """Log decays of twenty a token (their sum over a chunk runs to -1000 while neighbouring tokens' weights hang on
    differences of a few units), states that hardly forget and steps close to zero."""
    T, W_ = 140, 24
    t, m, part = space_case(T, W_, 4, 16, 16, 2, 4, 2, seed=8, a_log=a_log, dt=dt)
    Wd = doubles(t)
    want = Wd["table"] + plain.state_space(Wd["table"], Wd, "", m, EPS, {})
    for cut in ((140,), (40, 1, 1, 98)):
        got, _ = run_alone(tmp_path / str(len(cut)), {"width": W_, "rows": T, "mixer": part}, t, cut=cut, n_pages=12)
        assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max())


def old_state_case(kind):
    """Row 3 is written strongly and hardly forgotten; rows 250 (inside a portion) and 299 (decoded alone) ask for its
    key.  Returns tensors, sizes, part, the plain function."""
    T, W_, half = 300, 32, 16
    g = torch.Generator().manual_seed(3)
    direction = torch.randn(half, generator=g)
    direction = direction / direction.norm()
    own = torch.randn(half, generator=g)
    if kind == "fixed":
        t, m, part = decay_case(T, W_, 2, 32, 32, [0.9999, 1.0], seed=6, x_std=0.1)
        t["q"][:, half:] = 0.0
        t["q"] *= 3.0
        t["k"] = t["q"].clone()
        plain_fn = plain.fixed_decay_attention
    else:
        t, m, part = space_case(T, W_, 2, 32, 32, 1, 2, 1, seed=6, x_std=0.1, a_log=-9.0, dt=-3.0)
        t["conv"][:, 0] = 0.0
        t["conv"][:, 1] = 1.0
        t["conv.b"] *= 0.0
        t["D"] *= 0.1
        rows = t["in"][128:192]                   # B and C: the same map of the input's first half
        rows[:, half:] = 0.0
        rows *= 3.0
        t["in"][160:192] = t["in"][128:160]
        plain_fn = plain.state_space
    t["table"][3] = torch.cat([3.0 * direction, 3.0 * own])
    for row in (250, 299):
        t["table"][row] = torch.cat([3.0 * direction, 0.2 * torch.randn(half, generator=g)])
    return t, m, part, plain_fn


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["fixed", "input"])
def test_a_state_hundreds_of_tokens_old(tmp_path, kind, dtype):
    """With the row lost, or the state zeroed somewhere between, the asking rows' outputs are others; the row lies
    four chunks, several portions and dozens of single steps back."""
    t, m, part, fn = old_state_case(kind)
    Wd = doubles(t)
    want = Wd["table"] + fn(Wd["table"], Wd, "", m, EPS, {})
    without = Wd["table"].clone()
    without[3] = Wd["table"][4]
    lost = without + fn(without, Wd, "", m, EPS, {})
    late = fn(Wd["table"][200:], Wd, "", m, EPS, {})          # the state zeroed in front of row 200
    for row in (250, 299):
        assert float((want[row] - lost[row]).abs().max()) > 0.1 * float(want[row].abs().max())
        assert float((want[row] - Wd["table"][row] - late[row - 200]).abs().max()) > 0.1 * float(want[row].abs().max())
    got, _ = run_alone(tmp_path, {"width": 32, "rows": 300, "mixer": part}, t, cut=LONG_CUT, dtype=dtype, n_pages=20)
    if dtype == "float32":
        assert_close_f32(got, want, "an old state")
    else:
        Wb = {k_: v.bfloat16().double() for k_, v in Wd.items()}
        ref = Wb["table"] + fn(Wb["table"], Wb, "", m, EPS, {})
        for row in (250, 299):
            assert float((got[row] - ref[row]).abs().max()) <= 0.06 * float(ref[row].abs().max()), row


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("taps", [2, 4, 6])
def test_saved_inputs_of_the_convolution_between_steps(tmp_path, taps, dtype):
    """Weights that put most on the oldest inputs: a token's x, B and C hang on the tokens before it, which lie in
    an earlier step for the first rows of every portion (and for every single token), in portions shorter than the
    taps too; requests run side by side."""
    cfg = {"architecture": "Nosalorn", "vocab": 140, "width": 64, "norm": {"eps": 1e-5}, "embedding": {"scale": 4.0},
           "layers": [mamba(4, 16, 16, 2, taps, 2, dense(32)), mamba(3, 10, 12, 1, taps, 3, None)]}
    weights = torch.tensor([3.0, 2.0, 1.0, 0.3, 0.2, 0.1][:taps])
    storage = torch.float32 if dtype == "float32" else torch.bfloat16
    folder = write_model(tmp_path / "conv", cfg, 7, storage, std=0.1, change={f"l{i}.mix.conv": lambda w: w * weights for i in (0, 1)})
    c, W = plain.load_model_folder(folder)
    reqs = {"a": random_tokens(cfg["vocab"], 120, seed=3), "b": random_tokens(cfg["vocab"], 90, seed=4), "c": random_tokens(cfg["vocab"], 33, seed=6)}
    ref = {rid: plain.model_logits(c, W, toks) for rid, toks in reqs.items()}
    last = torch.zeros(taps, dtype=torch.float64)
    last[-1] = 1.0
    newest = {k: (v * last if k.endswith(".conv") else v) for k, v in W.items()}
    assert float((plain.model_logits(c, newest, reqs["a"]) - ref["a"]).abs().max()) > 0.1 * float(ref["a"].abs().max())
    for steps in (tail_decode_schedule(reqs, tail=30), portions_schedule(reqs, sizes=(37, 2, 3, 1, 4, 5, 2, 16, 1, 31)),
                  mixed_schedule(reqs, seed=5, decode_tail=10)):
        lm, _ = load(folder, dtype, steps)
        got = EngineDriver(lm).run(steps)
        for rid in reqs:
            assert_close(got[rid], ref[rid], dtype, f"saved inputs/{dtype}/{rid}")
        lm.close()


def experts_case(T, W_, ff, limit, experts, top, identity, groups, scale, shared, seed=5, correction=(0.1, -0.1)):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    outputs = experts + identity
    t = {"table": r(T, W_), "router": r(outputs, W_) * 0.4, "correction": correction[0] * r(outputs) + correction[1]}
    names = {"router": "router", "correction": "correction"}
    for e in range(experts):
        for what, shape in (("gate", (ff, W_)), ("up", (ff, W_)), ("down", (W_, ff))):
            t[f"e{e}.{what}"] = r(*shape) * 0.3
            names[f"{what}.{e}"] = f"e{e}.{what}"
    params = {"width": W_, "ff": ff, "experts": experts, "identity": identity, "top": top, "score": "softmax", "renormalize": False,
              "route_scale": scale, "group_score": "best", "correction": True, "weight_on": "output", "activation": "clamped", "limit": limit,
              "alpha": SWISH}
    f = {"router": {"experts": experts, "top": top, "scale": scale, "identity": identity}, "expert": {"ff": ff, "limit": limit}}
    if groups:
        f["router"]["groups"] = params["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        for what, shape in (("gate", (shared[0], W_)), ("up", (shared[0], W_)), ("down", (W_, shared[0])), ("sg", (1, W_))):
            t[f"shared.{what}"] = r(*shape) * 0.3
            names["shared_gate" if what == "sg" else f"shared.{what}"] = f"shared.{what}"
        params["shared"] = {"kind": "swiglu", "params": {"width": W_, "ff": shared[0], "activation": "clamped", "limit": shared[1], "alpha": SWISH}}
        params["shared_gate"] = True
        f["shared"] = {"ff": shared[0], "limit": shared[1]}
    return t, f, {"kind": "routed_experts", "params": params, "tensors": names}


EXPERTS = [(12, 3, 4, (4, 2), 2.0, (40, 0.5)), (5, 2, 0, None, 1.0, None), (5, 1, 3, (8, 3), 0.5, (16, 2.0)), (2, 6, 4, (2, 2), 1.5, (24, 1.0)),
           (9, 2, 0, (3, 1), 3.0, None), (68, 4, 2, (7, 2), 1.0, (8, 0.3)), (1, 1, 1, None, 2.0, None), (3, 2, 9, (2, 1), 4.0, None)]


@pytest.mark.parametrize("router_kernel", [1, 0])
@pytest.mark.parametrize("experts,top,identity,groups,scale,shared", EXPERTS)
def test_routed_experts_alone(tmp_path, experts, top, identity, groups, scale, shared, router_kernel):
    """Groups that hold experts with weights and identity experts, identity experts alone; choice scores below
    zero in every group (a group left out must lose to them); both forms of the router."""
    T, W_, ff = 33, 40, 24
    t, f, part = experts_case(T, W_, ff, 0.8, experts, top, identity, groups, scale, shared, correction=(0.15, -0.6))
    got, lm = run_alone(tmp_path, {"width": W_, "rows": T, "ffn": part}, t, knobs={"use_router_kernel": router_kernel})
    Wd = doubles(t)
    assert_close_f32(got, Wd["table"] + plain.routed_ff(Wd["table"], Wd, "", f), "routed experts alone")
    assert lm.paths()["routed_experts"] > 0


@pytest.mark.parametrize("shift", [(0.0, 5.0), (5.0, 0.0)])
def test_rows_that_choose_only_identity_experts_or_none(tmp_path, shift):
    """A correction that sends every row to the identity experts (no expert has a row), or to none of them."""
    T, W_ = 33, 40
    t, f, part = experts_case(T, W_, 24, 0.8, 6, 2, 3, None, 2.0, (16, 1.0))
    t["correction"][:6] += shift[0]
    t["correction"][6:] += shift[1]
    got, _ = run_alone(tmp_path, {"width": W_, "rows": T, "ffn": part}, t)
    Wd = doubles(t)
    assert_close_f32(got, Wd["table"] + plain.routed_ff(Wd["table"], Wd, "", f), "one kind of expert only")


@pytest.mark.parametrize("W_,ff,shared", [(64, 32, (64, 0.7)), (128, 96, (32, 1.0)), (72, 24, (40, 1.0))])
def test_routed_experts_alone_in_bfloat16(tmp_path, W_, ff, shared):
    """Sizes the matrix cores take and sizes they do not, in one long portion, in portions and in single tokens; a row
    whose choice hangs on rounding may differ, the others are within bfloat16's rounding of the plain result."""
    T = 150
    t, f, part = experts_case(T, W_, ff, 0.8, 10, 3, 2, (4, 2), 2.0, shared)
    t = {k: v * (0.5 if k != "table" and k != "correction" else 1.0) for k, v in t.items()}
    Wb = {k: v.bfloat16().double() for k, v in t.items()}
    want = Wb["table"] + plain.routed_ff(Wb["table"], Wb, "", f)
    for cut in ((150,), (5, 2, 9, 1, 70, 17), (130,) + (1,) * 20):
        got, _ = run_alone(tmp_path / str(len(cut)), {"width": W_, "rows": T, "ffn": part}, t, cut=cut, dtype="bfloat16", n_pages=12)
        assert_close(got, want, "bfloat16", f"routed experts, cut {cut}")
