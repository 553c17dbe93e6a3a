"""The plain Minilorn implementation by itself: what distinguishes the design's mechanisms moves its results by
far more than any tolerance the engine is held to (the sink, the bend, the query's factor, the value norm, the
pairing of the rotation, the norms of the compressed rows, a window that is one off, where the running maximum
starts, the floor of the denominator, the first token's row of the table of pairs), and a row never depends on
later tokens.  No GPU."""
import torch

import plain_minilorn as plain
from helpers import random_tokens
from test_gpu_minilorn import EPS, M1, attention_case, doubles, latent_case, memory_case, write_model


def moved(out, right):
    return float((out - right).abs().max()) / float(right.abs().max())


def test_the_attentions_options_show():
    t, m, _ = attention_case(60, 24, 2, 1, 16, 16, 0.5, (0.5, 10), 2.0)
    Wd = doubles(t)
    right = plain.sink_attention(Wd["table"], Wd, "", m, EPS)
    for other in (dict(m, softcap=None), dict(m, q_temp=None), dict(m, q_temp={"coef": 0.5, "every": 11}), dict(m, scale=0.55)):
        assert moved(plain.sink_attention(Wd["table"], Wd, "", other, EPS), right) > 0.01, other
    for sink in (Wd["sink"] * 0.5, Wd["sink"] - 30.0):
        assert moved(plain.sink_attention(Wd["table"], dict(Wd, sink=sink), "", m, EPS), right) > 0.05
    assert moved(plain.sink_attention(Wd["table"], dict(Wd, v=2.0 * Wd["v"]), "", m, EPS), right) < 1e-3       # values of unit size
    assert plain.query_factor(8, m["q_temp"]) == 1.0 and plain.query_factor(9, m["q_temp"]) > 1.3


def test_the_compressed_rows_and_the_window_show():
    t, m, _ = latent_case(60, 24, 2, 16, 8, 16, 12, 20, 0.5, 100.0, 9)
    Wd = doubles(t)
    right = plain.compressed_attention(Wd["table"], Wd, "", m, EPS)
    for size in (8, 10):
        assert moved(plain.compressed_attention(Wd["table"], Wd, "", dict(m, mask={"size": size}), EPS), right) > 0.02, size
    for name in ("dq.norm", "dkv.norm"):
        assert moved(plain.compressed_attention(Wd["table"], dict(Wd, **{name: torch.ones_like(Wd[name])}), "", m, EPS), right) > 0.05
    assert moved(plain.compressed_attention(Wd["table"], dict(Wd, dq=3.0 * Wd["dq"]), "", m, EPS), right) < 1e-3     # queries of unit size
    x = torch.randn(5, 1, 8, dtype=torch.float64)
    halves = x.clone()
    for i in range(4):
        a = torch.arange(5, dtype=torch.float64)[:, None] * 100.0 ** (-2.0 * i / 8)
        halves[..., i], halves[..., i + 4] = x[..., i] * a.cos() - x[..., i + 4] * a.sin(), x[..., i + 4] * a.cos() + x[..., i] * a.sin()
    assert moved(plain.turn_neighbours(x, 100.0, 8), halves) > 0.1


def memory_by_hand(h, W, m, start=0.0, floor=True):
    """One head's read-outs before the norm, straight from the recurrence."""
    D, cap = m["dim"], m["gate_cap"]
    q, k, v = (h @ W["q"].T)[:, :D] * D ** -0.5, (h @ W["k"].T)[:, :D], (h @ W["v"].T)[:, :m["vdim"]]
    S, n, top, out = torch.zeros(D, m["vdim"], dtype=torch.float64), torch.zeros(D, dtype=torch.float64), start, []
    for t in range(h.shape[0]):
        i = float(cap * torch.tanh((h[t] @ W["i"][0] + W["i.b"][0]) / cap))
        f = float(torch.nn.functional.logsigmoid(cap * torch.tanh((h[t] @ W["f"][0] + W["f.b"][0]) / cap)))
        new = max(f + top, i)
        a, b = (torch.exp(torch.tensor(x - new, dtype=torch.float64)) for x in (f + top, i))
        S, n, top = a * S + b * torch.outer(k[t], v[t]), a * n + b * k[t], new
        low = torch.exp(torch.tensor(-new, dtype=torch.float64)) if floor else 0.0
        out.append((S.T @ q[t]) / (max(abs(float(n @ q[t])), float(low)) + 1e-6))
    return torch.stack(out)


def test_the_memorys_start_and_floor_show():
    """Low input gates: the running maximum starts at 0 and sinks with the forget gate, and the floor of the
    denominator is what counts for many tokens."""
    t, m, _ = memory_case(40, 24, 1, 8, 8, 15.0, write=-3.0, keep=3.0)
    Wd = doubles(t)
    h = Wd["table"]
    read = memory_by_hand(h, Wd, m)
    full = (plain.unit_rms(read, EPS) * Wd["norm"] * torch.sigmoid(h @ Wd["g"].T)) @ Wd["o"].T
    assert moved(plain.matrix_memory(h, Wd, "", m, EPS), full) < 1e-12
    assert moved(memory_by_hand(h, Wd, m, floor=False), read) > 0.1
    t2, m2, _ = memory_case(40, 24, 1, 8, 8, 4.0, write=-2.0, keep=1.0)
    W2 = doubles(t2)
    assert moved(memory_by_hand(W2["table"], W2, m2, start=-1e30), memory_by_hand(W2["table"], W2, m2)) < 1e-3     # the same in another scaling ..
    right = plain.matrix_memory(W2["table"], W2, "", m2, EPS)
    for other in (dict(m2, gate_cap=5.0), dict(m2, gate_cap=15.0)):
        assert moved(plain.matrix_memory(W2["table"], W2, "", other, EPS), right) > 0.002


def test_the_table_of_pairs_shows():
    table = {"buckets": 11, "mul_prev": 3, "mul_cur": 5}
    tokens = [4, 9, 9, 0]
    assert [plain.pair_row(tokens, i, table) for i in range(4)] == [11, (12 + 45) % 11, (27 + 45) % 11, 27 % 11]


def test_a_row_does_not_depend_on_later_tokens(tmp_path):
    """Whole model, random weights: the logits of a prompt's first rows are those of the shorter prompt."""
    folder = write_model(tmp_path / "m", M1, 3)
    cfg, W = plain.load_model_folder(folder)
    toks = random_tokens(M1["vocab"], 50, seed=1)
    whole, part = plain.model_logits(cfg, W, toks), plain.model_logits(cfg, W, toks[:31])
    assert float((whole[:31] - part).abs().max()) <= 1e-6 * float(whole.abs().max())
    assert plain.greedy(cfg, W, toks[:5], 3) == plain.greedy(cfg, W, toks[:5], 4)[:3]
