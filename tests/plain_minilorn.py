"""Minilorn in plain float64 PyTorch, one function per mechanism, whole sequences at a time.

Nothing here is shared with the library: the functions take the dictionary of config.json and
a dictionary of tensors by checkpoint name, and run one request's tokens from position 0.
Slow on purpose: loops over tokens and heads where the definition has them.

The model: token embedding plus a row of a second table chosen by the pair (previous token,
token); pre-norm layers `x += mixer(n1(x))`, `x += ff(n2(x))` with RMS norms; final RMS norm and a
head matrix of its own.  Mixers: grouped-query attention without rotation (a factor per query
position, bent scores, values of unit root mean square, a learned sink per head in the softmax's
denominator); attention over a compressed row per token inside a sliding window, its queries made
through a compressed row of their own; a matrix memory per head with exponential input gates
(mLSTM).  Feed-forward: one matrix up, a piecewise activation with two learned numbers, one down.
"""
import json
import math
import os

import torch
from safetensors.torch import load_file

F64 = torch.float64


def load_model_folder(folder):
    with open(os.path.join(folder, "config.json")) as fh:
        cfg = json.load(fh)
    return cfg, {k: v.to(F64) for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}


# ------------------------------------------------------------------ small pieces
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def turn_neighbours(x, base, dims):
    """x [n, heads, size], row = position: values 2i and 2i + 1 turn by position * base^(-2i / dims)."""
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=F64)[:, None]
    for i in range(dims // 2):
        a = pos * float(base) ** (-2.0 * i / dims)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return out


# ------------------------------------------------------------------ embedding
def pair_row(tokens, i, table):
    """Which row of the second table position i reads: the last one for the first token."""
    if i == 0:
        return table["buckets"]
    return (tokens[i - 1] * table["mul_prev"] + tokens[i] * table["mul_cur"]) % table["buckets"]


def embed(cfg, W, tokens):
    x = W["embed"][torch.tensor(tokens)].clone()
    table = (cfg.get("embedding") or {}).get("bigram")
    if table:
        for i in range(len(tokens)):
            x[i] += W["bigram"][pair_row(tokens, i, table)]
    return x


# ------------------------------------------------------------------ mixers
def query_factor(position, q_temp):
    return 1.0 + q_temp["coef"] * math.log((position + 1) // q_temp["every"] + 1) if q_temp else 1.0


def sink_attention(h, W, p, m, eps):
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = (h @ W[p + "q"].T).view(n, H, D), (h @ W[p + "k"].T).view(n, G, D)
    v = unit_rms((h @ W[p + "v"].T).view(n, G, V), eps)
    out = torch.zeros(n, H, V, dtype=F64)
    cap = m.get("softcap")
    for i in range(n):
        for a in range(H):
            g = a // (H // G)
            s = (k[: i + 1, g] @ (q[i, a] * query_factor(i, m.get("q_temp")))) * m["scale"]
            if cap:
                s = cap * torch.tanh(s / cap)
            sink = W[p + "sink"][a] if p + "sink" in W else torch.tensor(-math.inf, dtype=F64)
            top = torch.maximum(s.max(), sink)
            e = torch.exp(s - top)
            out[i, a] = (e / (torch.exp(sink - top) + e.sum())) @ v[: i + 1, g]
    return out.reshape(n, H * V) @ W[p + "o"].T


def compressed_attention(h, W, p, m, eps):
    n = h.shape[0]
    H, D, R, V, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    c_q = unit_rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
    q = (c_q @ W[p + "uq"].T).view(n, H, D + R)
    down = h @ W[p + "dkv"].T
    c = unit_rms(down[:, :rank], eps) * W[p + "dkv.norm"]
    q_turn, k_turn = q[..., D:], down[:, None, rank:]
    if R:
        q_turn, k_turn = turn_neighbours(q_turn, m["rot"]["base"], R), turn_neighbours(k_turn, m["rot"]["base"], R)
    k_turn = k_turn[:, 0]
    k_plain, v = (c @ W[p + "uk"].T).view(n, H, D), (c @ W[p + "uv"].T).view(n, H, V)
    size = (m.get("mask") or {}).get("size")
    out = torch.zeros(n, H, V, dtype=F64)
    for i in range(n):
        lo = 0 if size is None else max(0, i - size + 1)
        for a in range(H):
            s = (k_plain[lo: i + 1, a] @ q[i, a, :D] + k_turn[lo: i + 1] @ q_turn[i, a]) * m["scale"]
            out[i, a] = torch.softmax(s, 0) @ v[lo: i + 1, a]
    return out.reshape(n, H * V) @ W[p + "o"].T


def matrix_memory(h, W, p, m, eps):
    n = h.shape[0]
    H, D, V, cap = m["heads"], m["dim"], m["vdim"], float(m["gate_cap"])
    q = (h @ W[p + "q"].T).view(n, H, D) * D ** -0.5
    k, v = (h @ W[p + "k"].T).view(n, H, D), (h @ W[p + "v"].T).view(n, H, V)
    log_in = cap * torch.tanh((h @ W[p + "i"].T + W[p + "i.b"]) / cap)
    log_keep = -softplus(-cap * torch.tanh((h @ W[p + "f"].T + W[p + "f.b"]) / cap))
    out = torch.zeros(n, H, V, dtype=F64)
    for a in range(H):
        S, norm, top = torch.zeros(D, V, dtype=F64), torch.zeros(D, dtype=F64), torch.zeros((), dtype=F64)
        for t in range(n):
            new_top = torch.maximum(log_keep[t, a] + top, log_in[t, a])
            keep, write = torch.exp(log_keep[t, a] + top - new_top), torch.exp(log_in[t, a] - new_top)
            S = keep * S + write * torch.outer(k[t, a], v[t, a])
            norm = keep * norm + write * k[t, a]
            top = new_top
            out[t, a] = (S.T @ q[t, a]) / (torch.maximum((norm @ q[t, a]).abs(), torch.exp(-top)) + 1e-6)
    out = unit_rms(out, eps).reshape(n, H * V) * W[p + "norm"] * torch.sigmoid(h @ W[p + "g"].T)
    return out @ W[p + "o"].T


MIXERS = {"attention": sink_attention, "latent_attention": compressed_attention, "mlstm": matrix_memory}


# ------------------------------------------------------------------ feed-forward
def bent_activation(z, act):
    right, left = softplus(act[0]), 0.5 + softplus(act[1])
    return torch.where(z > 0, right * z * z, left * (torch.expm1(torch.clamp(z, max=0.0)) - torch.clamp(z, max=0.0))) + 0.5 * z


def dense_ff(h, W, p):
    return bent_activation(h @ W[p + "up"].T, W[p + "act"]) @ W[p + "down"].T


# ------------------------------------------------------------------ the model
def model_hidden(cfg, W, tokens):
    """The residual stream after every layer: list of [n, width]."""
    eps = cfg["norm"]["eps"]
    x, after = embed(cfg, W, tokens), []
    for L, layer in enumerate(cfg["layers"]):
        p = f"l{L}."
        x = x + MIXERS[layer["type"]](unit_rms(x, eps) * W[p + "norm1"], W, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            x = x + dense_ff(unit_rms(x, eps) * W[p + "norm2"], W, p + "mlp.")
        after.append(x)
    return after


def model_logits(cfg, W, tokens):
    x = model_hidden(cfg, W, tokens)[-1]
    return (unit_rms(x, cfg["norm"]["eps"]) * W["final.norm"] @ W["head"].T).to(torch.float32)


def greedy(cfg, W, prompt, n_new):
    tokens = list(prompt)
    for _ in range(n_new):
        tokens.append(int(model_logits(cfg, W, tokens)[-1].argmax()))
    return tokens[len(prompt):]
