"""The Minilorn design in the engine against the plain implementation (``plain_minilorn.py``): each
mechanism alone through the step function (attention with a learned sink, bent scores, a factor per query
position and values of unit root mean square; attention over compressed rows inside a window, its queries
through a compressed row of their own; the matrix memory with exponential gates; the feed-forward's
activation; the embedding of token pairs), whole models of several shapes in every way of cutting and
batching, models drawn at random, inputs made so that a key at a window's edge, a far key, a sink or a lost
memory shows, long decoding, pages and slots used again, and greedy generation through the engine's entry
point and scheduler.  Sizes differ from model to model in every number and include values that make
mechanisms degenerate: one query head per key head and all on one, no factor, no bend, no window and a
window of one key, nothing rotated, one head, layers without feed-forward, an embedding without pairs, a
table of pairs of one row, keys and values of sizes that fill no tile.
"""
import json
import os
import random

import pytest
import torch

import plain_minilorn as plain
from helpers import (EngineDriver, assert_close, assert_close_f32, mixed_schedule, peak_tokens, portions_schedule, random_tokens,
                     tail_decode_schedule, whole_schedule)
from test_gpu_vabuzen import doubles, run_alone

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
STD = 0.08


def dense(ff):
    return {"kind": "dense", "ff": ff}


def attention(heads, kv_heads, dim, vdim, scale, q_temp, softcap, mlp):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if q_temp:
        m["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    if softcap:
        m["softcap"] = softcap
    return {"type": "attention", "mixer": m, "mlp": mlp}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base, window, mlp):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}
    if rot_dim:
        m["rot"] = {"base": base, "dims": rot_dim}
    if window:
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def mlstm(heads, dim, vdim, cap, mlp):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def pairs(buckets, mul_prev, mul_cur):
    return {"bigram": {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}}


# sizes the matrix cores and the fused products take
M1 = {"architecture": "Minilorn", "vocab": 310, "width": 128, "norm": {"eps": 1e-5}, "embedding": pairs(101, 31, 7),
      "layers": [latent(4, 16, 16, 32, 64, 48, 0.2, 20000.0, 24, dense(192)), mlstm(2, 32, 64, 9.0, dense(128)),
                 attention(4, 2, 32, 64, 0.2, (0.4, 16), 12.0, dense(192)), mlstm(4, 16, 32, 20.0, None),
                 latent(3, 24, 8, 16, 32, 32, 0.2, 500.0, None, dense(64)), latent(4, 16, 16, 32, 64, 48, 0.2, 20000.0, 24, None)]}
# a width that is no multiple of 16, heads no matrix-core kernel takes, all query heads on one key head, no factor, no
# bend, nothing rotated, a window of one key, one head, an embedding without pairs
M2 = {"architecture": "Minilorn", "vocab": 211, "width": 72, "norm": {"eps": 3e-6},
      "layers": [attention(5, 1, 12, 20, 0.3, None, None, dense(40)), mlstm(1, 20, 12, 5.0, dense(56)),
                 latent(2, 12, 0, 20, 24, 24, 0.3, 0.0, 1, dense(40)), attention(2, 2, 9, 7, 0.35, (1.0, 1), None, None),
                 latent(6, 10, 4, 14, 10, 20, 0.3, 300.0, 7, dense(24))]}
# wide heads: keys of 128 and 96, memories whose sizes are no multiples of 16 and larger than 128, a bend that bites
M3 = {"architecture": "Minilorn", "vocab": 260, "width": 160, "norm": {"eps": 1e-4}, "embedding": pairs(997, 1000003, 77),
      "layers": [mlstm(2, 72, 144, 15.0, dense(96)), attention(2, 1, 128, 96, 0.3, (0.2, 50), 2.0, dense(64)),
                 latent(8, 32, 32, 32, 48, 64, 0.125, 10000.0, 65, dense(64)), mlstm(1, 136, 300, 3.0, None),
                 attention(4, 2, 80, 128, 0.1, (0.5, 7), 30.0, dense(96))]}
# sizes that are multiples of two only, a table of pairs of one row besides the first token's
M4 = {"architecture": "Minilorn", "vocab": 333, "width": 100, "norm": {"eps": 1e-6}, "embedding": pairs(1, 3, 5),
      "layers": [latent(3, 10, 6, 14, 22, 18, 0.25, 777.0, 33, dense(50)), mlstm(3, 10, 14, 12.0, dense(34)),
                 attention(3, 3, 18, 22, 0.22, (0.3, 10), 5.0, dense(50)), mlstm(5, 6, 30, 7.5, None)]}
MODELS = {"M1": (M1, 51), "M2": (M2, 52), "M3": (M3, 53), "M4": (M4, 54)}
LENGTHS = {"M1": [40, 57, 90, 150, 65, 33], "M2": [45, 130, 64, 100, 17, 33], "M3": [31, 32, 150, 64, 49, 80], "M4": [70, 19, 101, 64, 13, 50]}
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
        if name.endswith(".i.b"):
            tensors[name] = 1.5 * unit - 1.0        # log input gates on both sides of zero
        elif name.endswith(".f.b"):
            tensors[name] = unit + 2.0              # memories that last
        elif name.endswith(".sink") or name.endswith(".act"):
            tensors[name] = 1.2 * unit
        elif name in ("embed", "bigram"):
            tensors[name] = 3.0 * tensors[name]
    # a memory read with a query at right angles to its keys is a small number that the norm behind it makes large,
    # sign and all: keys that lean towards the queries keep rounding from deciding such rows
    for name in [n for n in tensors if n.endswith(".mix.i")]:
        p = name[:-1]
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
    assert paths["attention_biased"] > 0 and paths["attention_latent"] > 0 and paths["matrix_memory"] > 0
    if mode != "whole":
        assert paths["matrix_memory_step"] > 0
    if dtype == "bfloat16" and name in ("M1", "M3"):
        assert paths["attention_biased_rows"] + paths["attention_biased_decode"] > 0     # the matrix cores took these heads


@pytest.mark.parametrize("name", ["M1", "M2", "M4"])
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


@pytest.mark.parametrize("name", ["M1", "M3"])
def test_batches_of_unequal_requests_equal_each_alone(folders, name):
    """In 32-bit a row's logits depend on the cut of its prompt and on the batch by no more than the
    rounding of sums taken in another order (the memory's chunks of 64 rows begin where a portion begins)."""
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
    folder = folders("M1", "bfloat16")
    reqs = requests_of("M1")
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
    others), order and number of layers, windows, factors, bends, caps and the table of pairs."""
    cfg = {"architecture": "Minilorn", "vocab": rng.randint(100, 700), "width": rng.choice([64, 96, 160, 192, 200, 320]),
           "norm": {"eps": rng.choice([1e-6, 1e-5])}}
    if rng.random() < 0.85:
        cfg["embedding"] = pairs(rng.choice([1, 7, 256, 1021]), rng.randint(0, 5000), rng.randint(0, 5000))
    layers = []
    for _ in range(rng.randint(2, 5)):
        mlp = None if rng.random() < 0.2 else dense(rng.choice([64, 128, 200, 256]))
        kind = rng.choice(["a", "l", "l", "m", "m"])
        if kind == "a":
            kv, dim = rng.choice([1, 2, 3, 4]), rng.choice([16, 32, 40, 64, 80, 128])
            layers.append(attention(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([16, 32, 48, 64, 96, 128]),
                                    round(dim ** -0.5 * rng.uniform(0.7, 1.5), 4),
                                    (round(rng.uniform(0.05, 0.6), 3), rng.choice([1, 13, 64, 100])) if rng.random() < 0.8 else None,
                                    round(rng.uniform(1.0, 50.0), 2) if rng.random() < 0.8 else None, mlp))
        elif kind == "l":
            dim, rot_dim = rng.choice([16, 32, 48, 64]), rng.choice([0, 8, 16, 32, 64])
            layers.append(latent(rng.choice([1, 2, 3, 8, 17]), dim, rot_dim, rng.choice([16, 32, 64]), rng.choice([24, 32, 64, 96]),
                                 rng.choice([16, 32, 64, 96, 40]), round((dim + rot_dim) ** -0.5 * rng.uniform(0.7, 1.5), 4),
                                 rng.choice([1000.0, 50000.0]), rng.choice([None, 1, 5, 16, 31, 64, 65, 100]), mlp))
        else:
            layers.append(mlstm(rng.choice([1, 2, 3, 4, 8]), rng.choice([8, 16, 24, 32, 48, 64, 96]), rng.choice([16, 32, 40, 64, 128]),
                                round(rng.uniform(3.0, 30.0), 2), mlp))
    cfg["layers"] = layers
    return cfg


@pytest.mark.parametrize("seed", range(8))
def test_models_drawn_at_random(tmp_path, seed):
    """Eight models drawn at random, weights stored in bfloat16, four requests of 20 to 300 tokens,
    in a mixed schedule and in long and short portions, in 32-bit and in bfloat16."""
    rng = random.Random(3000 + seed)
    cfg = drawn_model(rng)
    folder = write_model(tmp_path / "drawn", cfg, seed, torch.bfloat16, std=0.06)
    c, W = plain.load_model_folder(folder)
    reqs = {f"r{i}": random_tokens(cfg["vocab"], rng.randint(20, 300), seed=seed * 10 + i) for i in range(4)}
    ref = {rid: plain.model_logits(c, W, toks) for rid, toks in reqs.items()}
    for dtype in ("float32", "bfloat16"):
        for steps in (mixed_schedule(reqs, seed=seed, decode_tail=rng.randint(3, 20)), portions_schedule(reqs, sizes=(70, 2, 33, 1, 130, 16, 5))):
            lm, _ = load(folder, dtype, steps)
            got = EngineDriver(lm).run(steps)
            for rid in reqs:
                assert_close(got[rid], ref[rid], dtype, f"drawn model {seed}/{dtype}/{rid}: {json.dumps(cfg)}")
            lm.close()


# ------------------------------------------------------------------ long decoding, pages and slots
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_while_the_window_passes(folders, dtype):
    """A short prompt, then 200 tokens one by one (steps replayed from a recorded graph): the window of 24
    keys passes wholly over decoded tokens, its pages go back to the pool, and the memories and the pair's
    previous token live in their slots alone."""
    folder = folders("M1", dtype)
    toks = random_tokens(M1["vocab"], 215, seed=77)
    steps = tail_decode_schedule({"long": toks}, tail=200)
    lm, _ = load(folder, dtype, steps)
    got = EngineDriver(lm).run(steps)["long"]
    c, W = plain.load_model_folder(folder)
    assert_close(got, plain.model_logits(c, W, toks), dtype, "long decoding")
    assert lm.runner.counters()["graph_replays"] > 100


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_replayed_from_a_recorded_graph(folders, dtype):
    """Portions of 70 tokens of three requests, one after the other and with single tokens of another request
    between them: from the second on they are replayed from a recorded graph (a chunk of the memory and six rows
    of a second one), and every portion's last logits are the plain ones."""
    from celeg_amd.engine import StepEntry, load_model
    folder = folders("M1", dtype)
    c, W = plain.load_model_folder(folder)
    lm = load_model(folder, dtype=dtype, device=DEV, page_tokens=16, n_pages=64, max_requests=3, max_context=256, max_batched_tokens=128)
    other = random_tokens(M1["vocab"], 9, seed=90)
    other_slot, at = lm.cache.open(), 0
    other_ref = plain.model_logits(c, W, other)
    for r in range(3):
        toks = random_tokens(M1["vocab"], 210, seed=91 + r)
        ref = plain.model_logits(c, W, toks)
        slot = lm.cache.open()
        for start in (0, 70, 140):
            assert lm.cache.prepare(slot, start, 70)
            got = lm.runner.step([StepEntry(slot, start, toks[start:start + 70], [69])]).detach().cpu()
            assert_close(got[0], ref[start + 69], dtype, f"request {r}, portion from {start}")
            assert lm.cache.prepare(other_slot, at, 1)
            single = lm.runner.step([StepEntry(other_slot, at, other[at:at + 1], [0])]).detach().cpu()
            assert_close(single[0], other_ref[at], dtype, f"single token {at}")
            at += 1
        lm.cache.close(slot)
    assert lm.runner.counters()["graph_replays"] >= 16
    lm.close()


def test_pages_of_the_passed_window_return(folders):
    """While a request grows, the group of the windowed compressed rows holds the pages of the window only;
    the other groups hold all."""
    from celeg_amd.engine import StepEntry, load_model
    folder = folders("M1", "float32")
    toks = random_tokens(M1["vocab"], 200, seed=5)
    lm = load_model(folder, dtype="float32", device=DEV, page_tokens=16, n_pages=16, max_requests=2, max_context=256, max_batched_tokens=256)
    slot = lm.cache.open()
    assert lm.cache.prepare(slot, 0, 150)
    lm.runner.step([StepEntry(slot, 0, toks[:150], [149])])
    assert lm.cache.prepare(slot, 150, 50)
    logits = lm.runner.step([StepEntry(slot, 150, toks[150:], list(range(50)))]).detach().cpu()
    # position 150 sees keys from 127 on (page 7): pages 7 to 12 of 13
    assert sorted(len(p) for p in lm.cache.pages_held(slot)) == [6, 13, 13]
    c, W = plain.load_model_folder(folder)
    assert_close_f32(logits, plain.model_logits(c, W, toks)[150:], "after the window passed")
    lm.cache.close(slot)
    lm.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_pages_and_slots_used_again(folders, dtype):
    """Ten requests through two slots and a pool of six pages: every page and state slot serves several
    requests (a memory, a running maximum or a previous token that outlives its request would show at the
    next one's first tokens)."""
    from celeg_amd.engine import load_model
    folder = folders("M1", dtype)
    reqs = {f"q{i}": random_tokens(M1["vocab"], n, seed=500 + i) for i, n in enumerate([30, 18, 33, 16, 5, 47, 31, 1, 40, 17])}
    steps = mixed_schedule(reqs, max_live=2, seed=4, decode_tail=6)
    lm = load_model(folder, dtype=dtype, device=DEV, page_tokens=16, n_pages=6, max_requests=2, max_context=64, max_batched_tokens=128)
    got = EngineDriver(lm).run(steps)
    c, W = plain.load_model_folder(folder)
    for rid, toks in reqs.items():
        assert_close(got[rid], plain.model_logits(c, W, toks), dtype, rid)
    assert all(n == 6 for n in lm.cache.free_pages())


# ------------------------------------------------------------------ generation through the entry point
@pytest.mark.parametrize("name", ["M1", "M2"])
def test_greedy_generation_through_the_entry_point(folders, name):
    """More requests than places, prompts cut by a token budget, steps launched before the last token is on
    the host (the pair's tokens then come from the device)."""
    from celeg_amd.engine import Engine
    from celeg_amd.sampling import GenerationConfig
    folder = folders(name, "float32")
    cfg, W = plain.load_model_folder(folder)
    prompts = [random_tokens(cfg["vocab"], n, seed=40 + n) for n in (5, 23, 1, 37, 12)]
    engine = Engine.from_folder(folder, dtype="float32", device=DEV, max_active_requests=3, max_batched_tokens=64,
                                prefill_chunk_tokens=16, context=128, n_pages=24)
    greedy = GenerationConfig(temperature=0.0, repetition_penalty=1.0)
    outs = engine.generate(prompts, max_new_tokens=20, generation=greedy, eos_token_ids=[])
    for prompt, out in zip(prompts, outs):
        assert out == plain.greedy(cfg, W, prompt, 20)
    engine.close()


def test_command_line(folders, tmp_path):
    """``bin/celeg-run`` on a model folder of the design: greedy tokens and the prompt's last logits."""
    import subprocess
    import sys
    import numpy as np
    folder = folders("M4", "float32")
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
    folder = folders("M1", dtype)
    reqs = requests_of("M1")
    ref = plain_logits(folder, ("M1", dtype), reqs)
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


def attention_case(T, W_, H, G, D, V, scale, q_temp=None, softcap=None, seed=1, x_std=1.0, sink_std=1.5):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    t = {"table": r(T, W_) * x_std, "q": r(H * D, W_) * 0.3, "k": r(G * D, W_) * 0.3, "v": r(G * V, W_) * 0.3, "o": r(W_, H * V) * 0.3,
         "sink": r(H) * sink_std}
    params = {"width": W_, "heads": H, "kv_heads": G, "head_dim": D, "v_dim": V, "scale": scale, "sink": True, "value_norm": True, "eps": EPS}
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": scale}
    if q_temp:
        m["q_temp"] = params["query_temperature"] = {"coef": q_temp[0], "every": q_temp[1]}
    if softcap:
        m["softcap"] = params["softcap"] = softcap
    return t, m, {"kind": "biased_attention", "params": params, "tensors": {c: c for c in ("q", "k", "v", "o", "sink")}}


@pytest.mark.parametrize("G,D,V,q_temp,softcap", [(3, 12, 20, (0.7, 5), 3.0), (1, 8, 8, None, None), (6, 32, 16, (0.2, 1), 1.0), (2, 7, 9, None, 10.0),
                                                  (2, 16, 64, (1.5, 20), None)])
def test_sink_attention_alone(tmp_path, G, D, V, q_temp, softcap):
    T, W_ = 45, 40
    t, m, part = attention_case(T, W_, 6, G, D, V, 0.4, q_temp, softcap)
    got, _ = run_alone(tmp_path, {"width": W_, "rows": T, "mixer": part}, t)
    Wd = doubles(t)
    assert_close_f32(got, Wd["table"] + plain.sink_attention(Wd["table"], Wd, "", m, EPS), "attention with a sink alone")


@pytest.mark.parametrize("D,V", [(32, 32), (48, 80), (64, 128), (96, 60), (104, 12), (128, 96)])
def test_matrix_core_attention_equals_the_general_kernel(tmp_path, D, V):
    """bfloat16: the kernels on the matrix cores (heads that fill their tiles and heads that do not) against the
    kernel that scores key by key, on the same pages, in whole prompts, portions and single tokens.  The two
    differ in the rounding of the weights to two bfloat16 numbers only."""
    T, W_ = 200, 64
    for q_temp, softcap in (((0.3, 30), 4.0), (None, None), (None, 40.0)):
        t, m, part = attention_case(T, W_, 4, 2, D, V, D ** -0.5, q_temp, softcap, seed=D + V, x_std=1.5)
        got = {}
        long_cut = (15, 2, 17, 1, 80, 3, 16, 64)
        for form, cut in (("general", long_cut), (-1, long_cut), (0, long_cut), (1, long_cut), (-1, (200,)), (-1, (170,) + (1,) * 30)):
            knobs = {"use_biased_mfma": 0} if form == "general" else {"biased_rows_form": form}
            out, lm = run_alone(tmp_path / f"{softcap}_{form}_{len(cut)}", {"width": W_, "rows": T, "mixer": part}, t, cut=cut, dtype="bfloat16",
                                knobs=knobs, n_pages=16)
            took = lm.paths()["attention_biased_rows"] + lm.paths()["attention_biased_decode"]
            assert (took > 0) == (form != "general")
            got[(form, len(cut))] = out
        ref = got[("general", 8)]
        for key, out in got.items():
            rel = float((out - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt())
            assert rel <= 1e-2, f"heads of {D} and {V}, softcap {softcap}, form {key}: rel rms {rel:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_far_key_and_the_sink_show(tmp_path, dtype):
    """Rows 250 (inside a prompt's portion) and 299 (decoded alone) whose weight is shared between one key some
    hundred positions back, among many that score far lower, and the sink, which is about as large as that
    key's score: with the key or the sink left out, or with the factor of the query's position wrong, the
    rows' outputs are others."""
    T, W_, H, D = 300, 32, 2, 32
    t, m, part = attention_case(T, W_, H, H, D, D, 0.25, (0.5, 40), 60.0, seed=5, x_std=0.3)
    t["q"][:, W_ // 2:] = 0.0
    t["k"] = t["q"].clone()
    g = torch.Generator().manual_seed(9)
    direction = torch.randn(W_, generator=g)
    direction[W_ // 2:] = 0.0
    direction = direction / direction.norm()
    own = torch.randn(W_, generator=g)
    own[:W_ // 2] = 0.0
    t["table"][3] = 5.0 * direction + 6.0 * own / own.norm()
    for row in (250, 299):
        t["table"][row] = 1.5 * direction
    Wd = doubles(t)
    for h in range(H):       # the sink at the bent score of row 250 against key 3
        q, k = (Wd["table"][row] @ Wd["q"].view(H, D, W_)[h].T for row in (250, 3))
        s = float(q @ k) * 0.25 * plain.query_factor(250, m["q_temp"])
        t["sink"][h] = float(60.0 * torch.tanh(torch.tensor(s / 60.0)))
    Wd = doubles(t)
    want = Wd["table"] + plain.sink_attention(Wd["table"], Wd, "", m, EPS)
    moved = lambda out, row: float((want[row] - out[row]).abs().max()) / float(want[row].abs().max())
    without = Wd["table"].clone()
    without[3] = Wd["table"][4]
    for change in (dict(Wd, sink=Wd["sink"] - 50.0), None):
        out = (Wd["table"] + plain.sink_attention(Wd["table"], change, "", m, EPS) if change else
               without + plain.sink_attention(without, Wd, "", m, EPS))
        assert moved(out, 250) > 0.1 and moved(out, 299) > 0.1
    cut = (130, 2, 97, 31, 16, 1, 7) + (1,) * 16
    got, lm = run_alone(tmp_path, {"width": W_, "rows": T, "mixer": part}, t, cut=cut, dtype=dtype, n_pages=20)
    if dtype == "float32":
        assert_close_f32(got, want, "a far key and the sink")
    else:
        Wb = {k_: v.bfloat16().double() for k_, v in Wd.items()}
        ref = Wb["table"] + plain.sink_attention(Wb["table"], Wb, "", m, EPS)
        for row in (250, 299, 120):
            assert float((got[row] - ref[row]).abs().max()) <= 0.06 * float(ref[row].abs().max()), row
        assert lm.paths()["attention_biased_rows"] > 0 and lm.paths()["attention_biased_decode"] > 0


def latent_case(T, W_, H, D, R, V, q_rank, rank, scale, base, window, seed=3, x_std=1.0):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    t = {"table": r(T, W_) * x_std, "dq": r(q_rank, W_) * 0.3, "dq.norm": 1 + 0.3 * r(q_rank), "uq": r(H * (D + R), q_rank) * 0.4,
         "dkv": r(rank + R, W_) * 0.3, "dkv.norm": 1 + 0.3 * r(rank), "uk": r(H * D, rank) * 0.4, "uv": r(H * V, rank) * 0.4,
         "o": r(W_, H * V) * 0.3}
    params = {"width": W_, "heads": H, "dim": D, "rot_dim": R, "vdim": V, "q_rank": q_rank, "kv_rank": rank, "scale": scale, "eps": EPS,
              "sink": False, "gate": False}
    m = {"heads": H, "dim": D, "rot_dim": R, "vdim": V, "q_rank": q_rank, "kv_rank": rank, "scale": scale}
    if R:
        m["rot"] = {"base": base, "dims": R}
        params["position"] = {"kind": "rope", "params": {"theta": base, "rotary_dim": R, "head_dim": R, "pairing": "neighbours"}}
    if window:
        m["mask"] = {"size": window}
        params["window"] = window
    names = {c: c for c in ("dq", "uq", "dkv", "uk", "uv", "o")}
    return t, m, {"kind": "latent_attention", "params": params, "tensors": dict(names, dq_norm="dq.norm", dkv_norm="dkv.norm")}


@pytest.mark.parametrize("H,D,R,V,q_rank,rank,window", [(5, 12, 8, 14, 11, 20, 9), (2, 8, 0, 8, 40, 12, 1), (16, 32, 16, 32, 24, 64, 17),
                                                        (1, 16, 32, 24, 1, 48, None), (3, 16, 4, 8, 16, 16, 16)])
def test_windowed_latent_attention_alone(tmp_path, H, D, R, V, q_rank, rank, window):
    T, W_ = 45, 40
    t, m, part = latent_case(T, W_, H, D, R, V, q_rank, rank, (D + R) ** -0.5, 300.0, window)
    Wd = doubles(t)
    want = Wd["table"] + plain.compressed_attention(Wd["table"], Wd, "", m, EPS)
    got, lm = run_alone(tmp_path, {"width": W_, "rows": T, "mixer": part}, t)
    assert_close_f32(got, want, "latent attention alone")
    assert lm.paths()["attention_latent"] > 0


@pytest.mark.parametrize("H,D,R,V,rank", [(16, 32, 16, 32, 64), (3, 16, 8, 16, 32), (20, 64, 32, 32, 256), (4, 16, 64, 64, 512)])
def test_matrix_core_latent_attention_equals_the_general_kernel(tmp_path, H, D, R, V, rank):
    """bfloat16: the kernel that brings blocks of 64 compressed rows to the matrix cores against the one that
    scores key by key, with windows that begin at, before and behind the borders of pages, blocks and tiles of
    64 rows, and with none, in whole prompts, portions and single tokens (whose keys are cut into shares)."""
    T, W_ = 300, 64
    for window in (1, 5, 63, 64, 65, 130, None):
        t, m, part = latent_case(T, W_, H, D, R, V, 32, rank, (D + R) ** -0.5, 10000.0, window, seed=rank, x_std=1.5)
        got = {}
        long_cut = (15, 2, 17, 1, 130, 3, 16, 64)
        for form, cut in (("general", long_cut), ("cores", long_cut), ("cores", (300,)), ("cores", (270,) + (1,) * 30)):
            out, lm = run_alone(tmp_path / f"{window}_{form}_{len(cut)}", {"width": W_, "rows": T, "mixer": part}, t, cut=cut, dtype="bfloat16",
                                knobs={"use_latent_mfma": 0} if form == "general" else None, n_pages=20)
            took = lm.paths()["attention_latent_rows"] + lm.paths()["attention_latent_decode"]
            assert (took > 0) == (form != "general")
            got[(form, len(cut))] = out
        ref = got[("general", 8)]
        for key, out in got.items():
            rel = float((out - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt())
            assert rel <= 1e-2, f"rows of {rank} + {R}, window {window}, {key}: rel rms {rel:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("size", [40, 64, 129])
def test_keys_at_the_windows_edge(tmp_path, dtype, size):
    """Rows whose weight sits on one key: the last one inside the window and the first one outside, for rows
    inside a prompt's portion and rows decoded alone.  Queries and keys read the input's first half alone, in
    which the marked rows point one way; compressed rows and queries are normed, so the scale makes the score
    stand out.  The marked rows differ in the second half, which only the values read.  A window that is one
    off gives these rows other results by more than a tenth."""
    T, W_, H, D, V = 300, 32, 16, 16, 32
    half = W_ // 2
    t, m, part = latent_case(T, W_, H, D, 16, V, half, W_, 2.0, 1e4, size, seed=5, x_std=0.3)
    g = torch.Generator().manual_seed(9)
    t["dq.norm"], t["dkv.norm"] = torch.ones(half), torch.ones(W_)
    t["dq"] = torch.eye(half, W_)
    t["dkv"] = torch.cat([torch.eye(W_), torch.zeros(16, W_)])
    for h in range(H):
        turned = torch.linalg.qr(torch.randn(D, D, generator=g))[0]
        t["uq"][h * 32:(h + 1) * 32] = torch.cat([turned, torch.zeros(16, half)])
        t["uk"][h * D:(h + 1) * D] = torch.cat([turned, torch.zeros(D, half)], 1)
    direction = torch.randn(half, generator=g)
    direction = direction / direction.norm()
    queries = (200, 290)
    for row in tuple(q - size + 1 for q in queries) + tuple(q - size for q in queries):
        own = torch.randn(half, generator=g)
        t["table"][row] = torch.cat([8.0 * direction, 6.0 * own / own.norm()])
    for row in queries:
        t["table"][row] = torch.cat([2.0 * direction, 2.0 * torch.randn(half, generator=g)])
    Wd = doubles(t)
    want = Wd["table"] + plain.compressed_attention(Wd["table"], Wd, "", m, EPS)
    for other in (size - 1, size + 1):
        off = Wd["table"] + plain.compressed_attention(Wd["table"], Wd, "", dict(m, mask={"size": other}), EPS)
        for row in queries:
            assert float((want[row] - off[row]).abs().max()) > 0.1 * float(want[row].abs().max()), (other, row)
    cut = (130, 2, 97, 31, 16, 1, 7) + (1,) * 16
    got, lm = run_alone(tmp_path, {"width": W_, "rows": T, "mixer": part}, t, cut=cut, dtype=dtype, n_pages=20)
    if dtype == "float32":
        assert_close_f32(got, want, "keys at the edges")
    else:
        Wb = {k_: v.bfloat16().double() for k_, v in Wd.items()}
        ref = Wb["table"] + plain.compressed_attention(Wb["table"], Wb, "", m, EPS)
        for row in queries + (120, 299):
            assert float((got[row] - ref[row]).abs().max()) <= 0.05 * float(ref[row].abs().max()), row
        assert lm.paths()["attention_latent_rows"] > 0 and lm.paths()["attention_latent_decode"] > 0


def memory_case(T, W_, H, D, V, cap, seed=4, x_std=1.0, keep=2.0, write=0.0):
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g)
    t = {"table": r(T, W_) * x_std, "q": r(H * D, W_) * 0.3, "k": r(H * D, W_) * 0.3, "v": r(H * V, W_) * 0.3, "g": r(H * V, W_) * 0.3,
         "i": r(H, W_) * 0.3, "i.b": r(H) + write, "f": r(H, W_) * 0.3, "f.b": r(H) + keep, "norm": 1 + 0.3 * r(H * V), "o": r(W_, H * V) * 0.3}
    m = {"heads": H, "dim": D, "vdim": V, "gate_cap": cap}
    params = {"width": W_, "heads": H, "dim": D, "vdim": V, "gate_cap": cap, "eps": EPS}
    names = {c: c for c in ("q", "k", "v", "g", "i", "f", "norm", "o")}
    return t, m, {"kind": "matrix_memory", "params": params, "tensors": dict(names, i_bias="i.b", f_bias="f.b")}


@pytest.mark.parametrize("H,D,V,cap,write", [(3, 12, 20, 5.0, 0.0), (1, 16, 16, 15.0, -4.0), (2, 32, 64, 30.0, 4.0), (4, 7, 5, 2.0, 0.0),
                                             (1, 256, 40, 15.0, 0.0), (1, 40, 512, 15.0, 0.0), (2, 130, 258, 8.0, -2.0)])
def test_matrix_memory_alone(tmp_path, H, D, V, cap, write):
    """Portions of 5, 2, 9, 1, ... rows, then whole chunks, a chunk and a row, a chunk less a row; gates that
    open wide and gates so low that the running maximum stays with its start and the floor of the
    denominator counts."""
    T, W_ = 150, 40
    t, m, part = memory_case(T, W_, H, D, V, cap, write=write)
    Wd = doubles(t)
    want = Wd["table"] + plain.matrix_memory(Wd["table"], Wd, "", m, EPS)
    for cut in ((5, 2, 9, 1, 3, 17), (150,), (64, 65, 21), (63, 1, 64, 1, 21)):
        got, lm = run_alone(tmp_path / str(len(cut)), {"width": W_, "rows": T, "mixer": part}, t, cut=cut, n_pages=12)
        assert_close_f32(got, want, f"matrix memory alone, portions {cut}")
        assert lm.paths()["matrix_memory_rows"] > 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_memory_hundreds_of_tokens_old(tmp_path, dtype):
    """Row 3 is written through a wide open gate and hardly forgotten; rows 250 (inside a portion) and 299
    (decoded alone) ask for its key.  With the row lost, or the state zeroed somewhere between, the rows'
    outputs are others; the row lies four chunks, several portions and dozens of single steps back."""
    T, W_, H, D, V = 300, 32, 2, 32, 32
    t, m, part = memory_case(T, W_, H, D, V, 15.0, seed=6, x_std=0.2, keep=8.0, write=-6.0)
    g = torch.Generator().manual_seed(3)
    half = W_ // 2
    t["q"][:, half:] = 0.0
    t["k"] = t["q"].clone()
    direction = torch.randn(half, generator=g)
    direction = direction / direction.norm()
    own = torch.randn(half, generator=g)
    t["table"][3] = torch.cat([3.0 * direction, 3.0 * own])
    t["i"][:] = 0.0
    t["i"][:, half:] = 8.0 * own / (own @ own)
    for row in (250, 299):
        t["table"][row] = torch.cat([3.0 * direction, 0.2 * torch.randn(half, generator=g)])
    Wd = doubles(t)
    want = Wd["table"] + plain.matrix_memory(Wd["table"], Wd, "", m, EPS)
    without = Wd["table"].clone()
    without[3] = Wd["table"][4]
    lost = without + plain.matrix_memory(without, Wd, "", m, EPS)
    late = plain.matrix_memory(Wd["table"][200:], Wd, "", m, EPS)          # the state zeroed in front of row 200
    for row in (250, 299):
        assert float((want[row] - lost[row]).abs().max()) > 0.1 * float(want[row].abs().max())
        assert float((want[row] - Wd["table"][row] - late[row - 200]).abs().max()) > 0.1 * float(want[row].abs().max())
    cut = (130, 2, 97, 31, 16, 1, 7) + (1,) * 16
    got, _ = run_alone(tmp_path, {"width": W_, "rows": T, "mixer": part}, t, cut=cut, dtype=dtype, n_pages=20)
    if dtype == "float32":
        assert_close_f32(got, want, "an old memory")
    else:
        Wb = {k_: v.bfloat16().double() for k_, v in Wd.items()}
        ref = Wb["table"] + plain.matrix_memory(Wb["table"], Wb, "", m, EPS)
        for row in (250, 299, 120):
            assert float((got[row] - ref[row]).abs().max()) <= 0.06 * float(ref[row].abs().max()), row


def test_gates_that_shut_for_long_keep_their_precision(tmp_path):
    """Log forget gates near -13 a token and log input gates near zero: the sum of the log gates over a chunk
    runs to -800 while neighbouring tokens' weights hang on differences of a few units."""
    T, W_ = 130, 24
    t, m, part = memory_case(T, W_, 2, 16, 16, 15.0, seed=8, keep=-18.0)
    Wd = doubles(t)
    want = Wd["table"] + plain.matrix_memory(Wd["table"], Wd, "", m, EPS)
    for cut in ((130,), (40, 1, 1, 88)):
        got, _ = run_alone(tmp_path / str(len(cut)), {"width": W_, "rows": T, "mixer": part}, t, cut=cut, n_pages=12)
        assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max())


@pytest.mark.parametrize("act", [(0.7, -0.4), (-3.0, 2.5), (0.0, 0.0)])
def test_feed_forward_alone(tmp_path, act):
    torch.manual_seed(4)
    T, W_, ff = 29, 36, 50
    t = {"table": torch.randn(T, W_) * 2, "up": torch.randn(ff, W_) * 0.3, "down": torch.randn(W_, ff) * 0.3, "act": torch.tensor(act)}
    part = {"kind": "mlp", "params": {"width": W_, "ff": ff, "activation": "xielu", "bias": False}, "tensors": {c: c for c in ("up", "down", "act")}}
    got, _ = run_alone(tmp_path, {"width": W_, "rows": T, "ffn": part}, t)
    Wd = doubles(t)
    assert_close_f32(got, Wd["table"] + plain.dense_ff(Wd["table"], Wd, ""), "feed-forward alone")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rule", [(13, 5, 7), (1, 1, 1), (1021, 1000003, 999983), (64, 0, 1), (64, 1, 0)])
def test_embedding_of_pairs_alone(tmp_path, rule, dtype):
    """A model whose one mixer adds nothing (a zero output matrix): the logits show the embedding's rows.
    Portions of every size, so that the previous token lies in the same portion, in an earlier step's
    portion, or was decoded alone; two requests side by side, slots used again."""
    cfg = {"architecture": "Minilorn", "vocab": 97, "width": 64, "norm": {"eps": 1e-5}, "embedding": pairs(*rule),
           "layers": [attention(2, 1, 8, 8, 0.3, None, None, None)]}
    storage = torch.float32 if dtype == "float32" else torch.bfloat16
    folder = write_model(tmp_path / "pairs", cfg, 3, storage, change={"l0.mix.o": lambda w: 0.0 * w})
    c, W = plain.load_model_folder(folder)
    reqs = {f"r{i}": random_tokens(cfg["vocab"], n, seed=20 + i) for i, n in enumerate((33, 1, 20, 70, 2))}
    ref = {rid: plain.model_logits(c, W, toks) for rid, toks in reqs.items()}
    for steps in (whole_schedule(reqs), portions_schedule(reqs, sizes=(1, 2, 1, 1, 5, 3)), mixed_schedule(reqs, max_live=2, decode_tail=5)):
        lm, _ = load(folder, dtype, steps, max_requests=2)
        got = EngineDriver(lm).run(steps)
        for rid in reqs:
            assert_close(got[rid], ref[rid], dtype, f"pairs {rule}/{dtype}/{rid}")
        lm.close()
