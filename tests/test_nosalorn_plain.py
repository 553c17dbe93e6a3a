"""The plain Nosalorn implementation by itself: what distinguishes the design's mechanisms moves its results by far
more than any tolerance the engine is held to (biases, the pairing and the stretching of the rotation, its factor on
cosine and sine, the window, the kept first keys, the values' mixing, the decays, the order of gate and norm, the
convolution's bias, the step's softplus, where a correction counts, what a left-out group scores, the clamps, the
identity experts, the shared expert's gate), and a row never depends on later tokens.  No GPU."""
import math

import pytest
import torch

import plain_nosalorn as plain
from helpers import random_tokens
from test_gpu_nosalorn import EPS, N1, attention_case, decay_case, doubles, edge_case, experts_case, old_state_case, space_case, write_model


def moved(out, right):
    return float((out - right).abs().max()) / float(right.abs().max())


def test_the_attentions_options_show():
    t, m, _ = attention_case(60, 24, 4, 2, 16, 12, 0.5, (100.0, 12, (4.0, 30, 4.0, 0.5)), (9, 2))
    Wd = doubles(t)
    run = lambda W, m: plain.window_attention(Wd["table"], W, "", m, EPS, {})
    right = run(Wd, m)
    for name in ("q.b", "k.b", "v.b"):
        assert moved(run(dict(Wd, **{name: 0 * Wd[name]}), m), right) > 0.02, name
    scaling = m["rot"]["scaling"]
    for rot in (None, dict(m["rot"], scaling=None), dict(m["rot"], scaling=dict(scaling, factor=5.0)), dict(m["rot"], dims=10)):
        assert moved(run(Wd, dict(m, rot=rot)), right) > 0.02, rot
    for mask in ({"size": 8, "keep_first": 2}, {"size": 10, "keep_first": 2}, {"size": 9, "keep_first": 1}, {"size": 9, "keep_first": 3}):
        assert moved(run(Wd, dict(m, mask=mask)), right) > 0.02, mask
    # the first caller keeps, the second mixes
    carry = {}
    assert torch.equal(plain.window_attention(Wd["table"], Wd, "", dict(m, v_mix=True), EPS, carry), right)
    again = plain.window_attention(Wd["table"] + 1.0, dict(Wd, vmix=torch.tensor(1.0, dtype=torch.float64)), "", dict(m, v_mix=True), EPS, carry)
    assert moved(again, plain.window_attention(Wd["table"] + 1.0, Wd, "", m, EPS, {})) > 0.05


def test_stretched_frequencies_by_hand():
    """Fast pairs keep their frequency, slow ones have it divided, a line between; the pairs' borders are those whose
    wavelength fits `fast` and `slow` times into the original length."""
    base, dims, sc = 1000.0, 16, {"factor": 8.0, "original": 500, "fast": 20.0, "slow": 2.0}
    freq, factor = plain.stretched_frequencies(base, dims, sc)
    assert factor == pytest.approx(1.0 + 0.1 * math.log(8.0))
    turns = [500 / (2 * math.pi * base ** (2 * i / dims)) for i in range(8)]
    lo = max(i for i in range(8) if turns[i] >= 20.0)
    hi = min(i for i in range(8) if turns[i] <= 2.0)
    for i in range(8):
        f = base ** (-2 * i / dims)
        share = 0.0 if i <= lo else 1.0 if i >= hi else (i - lo) / (hi - lo)
        assert freq[i] == pytest.approx(f * (1 - share) + f / 8.0 * share)
    assert plain.stretched_frequencies(base, dims, None) == ([base ** (-2.0 * i / dims) for i in range(8)], 1.0)
    x = torch.randn(5, 1, 4, dtype=torch.float64)
    turned = plain.rotate_halves(x, {"base": 100.0, "dims": 4})
    p = 3
    assert float(turned[p, 0, 0]) == pytest.approx(float(x[p, 0, 0] * math.cos(p) - x[p, 0, 2] * math.sin(p)))
    assert float(turned[p, 0, 2]) == pytest.approx(float(x[p, 0, 2] * math.cos(p) + x[p, 0, 0] * math.sin(p)))


def test_the_linear_attentions_pieces_show():
    t, m, _ = decay_case(40, 24, 2, 8, 12, [0.8, 0.99])
    Wd = doubles(t)
    run = lambda W, m: plain.fixed_decay_attention(Wd["table"], W, "", m, EPS, {})
    right = run(Wd, m)
    for decay in ([0.82, 0.99], [0.8, 0.98], [0.99, 0.8]):
        assert moved(run(Wd, dict(m, decay=decay)), right) > 0.01, decay
    assert moved(run(dict(Wd, g=2.0 * Wd["g"]), m), right) > 0.05
    # one head by hand, straight from the sum over earlier tokens
    one, m1, _ = decay_case(12, 24, 1, 8, 12, [0.7])
    W1 = doubles(one)
    h = W1["table"]
    q, k, v = (plain.silu(h @ W1[c].T) for c in "qkv")
    o = torch.stack([sum(0.7 ** (i - j) * (q[i] @ k[j]) * v[j] for j in range(i + 1)) for i in range(12)])
    want = (o / (o.pow(2).mean(-1, keepdim=True) + EPS).sqrt() * W1["norm"] * torch.sigmoid(h @ W1["g"].T)) @ W1["o"].T
    assert moved(plain.fixed_decay_attention(h, W1, "", m1, EPS, {}), want) < 1e-12


def test_the_state_spaces_pieces_show():
    t, m, _ = space_case(40, 24, 4, 6, 5, 2, 3, 2)
    Wd = doubles(t)
    run = lambda W, m: plain.state_space(Wd["table"], W, "", m, EPS, {})
    right = run(Wd, m)
    for name in ("conv.b", "dt_bias", "A_log", "D"):
        assert moved(run(dict(Wd, **{name: Wd[name] + 0.5}), m), right) > 0.01, name
    for parts in (1, 4):
        assert moved(run(Wd, dict(m, norm_groups=parts)), right) > 0.02
    # one head by hand: sums over earlier tokens, the gate in front of the norm
    one, m1, _ = space_case(12, 24, 1, 6, 5, 1, 3, 1)
    W1 = doubles(one)
    z, xbc, dt = (W1["table"] @ W1["in"].T).split([6, 16, 1], 1)
    padded = torch.cat([torch.zeros(2, 16, dtype=torch.float64), xbc])
    xbc = plain.silu(sum(padded[j:j + 12] * W1["conv"][:, j] for j in range(3)) + W1["conv.b"])
    x, B, C = xbc.split([6, 5, 5], 1)
    w = torch.log1p(torch.exp(dt[:, 0] + W1["dt_bias"]))
    F = torch.cumsum(-torch.exp(W1["A_log"]) * w, 0)
    y = torch.stack([sum(torch.exp(F[i] - F[j]) * w[j] * (B[j] @ C[i]) * x[j] for j in range(i + 1)) + W1["D"] * x[i] for i in range(12)])
    y = y * plain.silu(z)
    want = (y / (y.pow(2).mean(-1, keepdim=True) + EPS).sqrt() * W1["norm"]) @ W1["o"].T
    assert moved(plain.state_space(W1["table"], W1, "", m1, EPS, {}), want) < 1e-10


def test_the_routers_choice_by_hand():
    z = torch.tensor([2.0, 1.0, 0.0, -1.0, 0.5, 0.4], dtype=torch.float64)
    s = torch.softmax(z, 0)
    none = torch.zeros(6, dtype=torch.float64)
    rule = {"experts": 5, "identity": 1, "top": 2, "scale": 3.0, "groups": {"count": 3, "keep": 1}}
    chosen, weights = plain.choose_experts(z, none, rule)
    assert chosen == [0, 1] and float(weights[1]) == pytest.approx(3.0 * float(s[1]))
    # a correction moves the choice and not the weights; choice scores below zero still beat left-out groups
    low = torch.tensor([-3.0, -3.0, -2.0, -5.0, -4.0, -4.0], dtype=torch.float64)
    chosen, weights = plain.choose_experts(z, low, rule)
    assert chosen == [2, 3] and float(weights[1]) == pytest.approx(3.0 * float(s[3]))
    # the group of the largest score, not of the largest sum
    chosen, _ = plain.choose_experts(torch.tensor([0.0, 1.5, 1.4, 1.4, 0.0, 0.0], dtype=torch.float64), none, rule)
    assert chosen == [1, 0]


def test_the_experts_pieces_show():
    t, f, _ = experts_case(20, 24, 12, 0.8, 6, 2, 2, (4, 2), 2.0, (16, 0.5))
    Wd = doubles(t)
    run = lambda W, f: plain.routed_ff(Wd["table"], W, "", f)
    right = run(Wd, f)
    assert moved(run(Wd, dict(f, expert={"ff": 12, "limit": 1.0})), right) > 0.01
    assert moved(run(Wd, dict(f, shared={"ff": 16, "limit": 0.7})), right) > 0.01
    assert moved(run(dict(Wd, correction=0 * Wd["correction"]), f), right) > 0.05
    assert moved(run(dict(Wd, **{"shared.sg": 0 * Wd["shared.sg"]}), f), right) > 0.05
    x = torch.randn(24, dtype=torch.float64) * 5
    g = (Wd["e0.gate"] @ x).clamp(max=0.8)
    u = (Wd["e0.up"] @ x).clamp(-0.8, 0.8)
    assert moved(plain.clamped_expert(x, Wd, "e0.", 0.8), Wd["e0.down"] @ ((u + 1) * g / (1 + torch.exp(-1.702 * g)))) < 1e-12


@pytest.mark.parametrize("size,keep,rot", [(40, 5, None), (64, 4, (10000.0, 16, (4.0, 32, 8.0, 1.0))), (33, 17, None)])
def test_inputs_made_for_the_windows_edges_show_them(size, keep, rot):
    t, m, _, queries = edge_case(size, keep, rot)
    Wd = doubles(t)
    run = lambda m: Wd["table"] + plain.window_attention(Wd["table"], Wd, "", m, EPS, {})
    want = run(m)
    for other in ((size + 1, keep), (size - 1, keep), (size, keep + 1), (size, keep - 1)):
        off = run(dict(m, mask={"size": other[0], "keep_first": other[1]}))
        for row in queries:
            assert float((want[row] - off[row]).abs().max()) > 0.1 * float(want[row].abs().max()), (other, row)


@pytest.mark.parametrize("kind", ["fixed", "input"])
def test_inputs_made_for_old_states_show_them(kind):
    t, m, _, fn = old_state_case(kind)
    Wd = doubles(t)
    want = Wd["table"] + fn(Wd["table"], Wd, "", m, EPS, {})
    without = Wd["table"].clone()
    without[3] = Wd["table"][4]
    lost = without + fn(without, Wd, "", m, EPS, {})
    late = fn(Wd["table"][200:], Wd, "", m, EPS, {})
    for row in (250, 299):
        assert float((want[row] - lost[row]).abs().max()) > 0.1 * float(want[row].abs().max())
        assert float((want[row] - Wd["table"][row] - late[row - 200]).abs().max()) > 0.1 * float(want[row].abs().max())


def test_a_row_does_not_depend_on_later_tokens(tmp_path):
    """Whole model, random weights: the logits of a prompt's first rows are those of the shorter prompt."""
    folder = write_model(tmp_path / "m", N1, 3)
    cfg, W = plain.load_model_folder(folder)
    toks = random_tokens(N1["vocab"], 40, seed=1)
    whole, part = plain.model_logits(cfg, W, toks), plain.model_logits(cfg, W, toks[:31])
    assert float((whole[:31] - part).abs().max()) <= 1e-6 * float(whole.abs().max())
    assert plain.greedy(cfg, W, toks[:5], 3) == plain.greedy(cfg, W, toks[:5], 4)[:3]
