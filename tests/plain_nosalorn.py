"""Nosalorn in plain float64 PyTorch, one function per mechanism, whole sequences at a time.

Nothing here is shared with the library: the functions take the dictionary of config.json and
a dictionary of tensors by checkpoint name, and run one request's tokens from position 0.
Slow on purpose: loops over tokens, heads and keys where the definition has them.

The model: scaled token embedding; pre-norm layers `x += mixer(n1(x))`, `x += ff(n2(x))` with RMS
norms; final RMS norm, head, logits times a constant.  Mixers: grouped-query attention with biases,
frequencies stretched by wavelength ("YaRN"), a sliding window that also keeps the sequence's first
keys, and values mixed with those of the first attention layer that mixes; linear attention with a
fixed decay per head; a state space with input-dependent decays behind a short convolution
(Mamba-2).  Feed-forward: dense SwiGLU, or routed experts with clamped gates, some of which are
the identity, chosen by corrected scores inside the best groups, plus a gated shared expert.
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


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def causal_taps(u, w, bias):
    """u [n, channels], w [channels, taps]: y_t = bias + sum_j w[:, j] u_(t - taps + 1 + j), zeros before 0."""
    n, taps = u.shape[0], w.shape[1]
    y = bias.expand(n, -1).clone()
    for t in range(n):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def stretched_frequencies(base, dims, scaling):
    """([dims / 2] angles per position, the factor on cosine and sine)."""
    freq = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freq, 1.0
    def dim_of(turns):      # the (fractional) pair number whose wavelength fits `turns` times into the original length
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(dim_of(scaling["fast"])), 0)
    hi = min(math.ceil(dim_of(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / scaling["factor"] * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_halves(x, rot):
    """x [n, heads, size], row = position: values i and i + dims/2 form pair i; the rest passes."""
    dims = rot["dims"]
    freq, factor = stretched_frequencies(rot["base"], dims, rot.get("scaling"))
    out, half = x.clone(), dims // 2
    pos = torch.arange(x.shape[0], dtype=F64)[:, None]
    for i, f in enumerate(freq):
        c, s = torch.cos(pos * f) * factor, torch.sin(pos * f) * factor
        u, v = x[..., i], x[..., i + half]
        out[..., i], out[..., i + half] = u * c - v * s, v * c + u * s
    return out


# ------------------------------------------------------------------ mixers
def window_attention(h, W, p, m, eps, carry):
    """carry: a dictionary that lives for one pass over the layers and holds the first mixed values."""
    n = h.shape[0]
    H, G, D, V = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
    q = (h @ W[p + "q"].T + W[p + "q.b"]).view(n, H, D)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).view(n, G, D)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(n, G, V)
    rot = m.get("rot")
    if rot and rot["dims"]:
        q, k = rotate_halves(q, rot), rotate_halves(k, rot)
    if m.get("v_mix"):
        if "v" in carry:
            lam = W[p + "vmix"]
            v = (1.0 - lam) * v + lam * carry["v"].view(n, G, V)
        else:
            carry["v"] = v
    mask = m.get("mask") or {}
    size, keep = mask.get("size"), mask.get("keep_first", 0)
    out = torch.zeros(n, H, V, dtype=F64)
    for i in range(n):
        seen = [j for j in range(i + 1) if size is None or i - j < size or j < keep]
        for a in range(H):
            g = a // (H // G)
            out[i, a] = torch.softmax((k[seen, g] @ q[i, a]) * m["scale"], 0) @ v[seen, g]
    return out.reshape(n, H * V) @ W[p + "o"].T


def fixed_decay_attention(h, W, p, m, eps, carry):
    n = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ W[p + "q"].T).view(n, H, D), silu(h @ W[p + "k"].T).view(n, H, D)
    v = silu(h @ W[p + "v"].T).view(n, H, V)
    out = torch.zeros(n, H, V, dtype=F64)
    for a in range(H):
        S = torch.zeros(D, V, dtype=F64)
        for t in range(n):
            S = m["decay"][a] * S + torch.outer(k[t, a], v[t, a])
            out[t, a] = S.T @ q[t, a]
    y = unit_rms(out.reshape(n, H * V), eps) * W[p + "norm"] * torch.sigmoid(h @ W[p + "g"].T)
    return y @ W[p + "o"].T


def state_space(h, W, p, m, eps, carry):
    n = h.shape[0]
    H, V, N, G, parts = m["heads"], m["vdim"], m["state"], m["groups"], m["norm_groups"]
    inner = H * V
    z, xbc, dt = (h @ W[p + "in"].T).split([inner, inner + 2 * G * N, H], 1)
    x, B, C = silu(causal_taps(xbc, W[p + "conv"], W[p + "conv.b"])).split([inner, G * N, G * N], 1)
    x, B, C = x.view(n, H, V), B.view(n, G, N), C.view(n, G, N)
    dt = softplus(dt + W[p + "dt_bias"])
    out = torch.zeros(n, H, V, dtype=F64)
    for a in range(H):
        S, g = torch.zeros(N, V, dtype=F64), a // (H // G)
        for t in range(n):
            S = torch.exp(-torch.exp(W[p + "A_log"][a]) * dt[t, a]) * S + dt[t, a] * torch.outer(B[t, g], x[t, a])
            out[t, a] = S.T @ C[t, g] + W[p + "D"][a] * x[t, a]
    y = (out.reshape(n, inner) * silu(z)).view(n, parts, inner // parts)
    return (unit_rms(y, eps).reshape(n, inner) * W[p + "norm"]) @ W[p + "o"].T


MIXERS = {"attention": window_attention, "lightning": fixed_decay_attention, "mamba2": state_space}


# ------------------------------------------------------------------ feed-forwards
def dense_ff(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def clamped_expert(x, W, p, limit):
    g = torch.clamp(W[p + "gate"] @ x, max=limit)
    u = torch.clamp(W[p + "up"] @ x, min=-limit, max=limit)
    return W[p + "down"] @ (g * torch.sigmoid(1.702 * g) * (u + 1.0))


def choose_experts(z, correction, r):
    """z [experts + identity] logits -> (chosen, their weights).  A group of neighbours counts by its
    largest corrected score; the weights are the scores without the correction."""
    s = torch.softmax(z, 0)
    choice = s + correction
    groups = r.get("groups") or {"count": 1, "keep": 1}
    total = r["experts"] + r.get("identity", 0)
    per = total // groups["count"]
    best = sorted(range(groups["count"]), key=lambda g: (-float(choice[g * per:(g + 1) * per].max()), g))[: groups["keep"]]
    allowed = [e for e in range(total) if e // per in best]
    chosen = sorted(allowed, key=lambda e: (-float(choice[e]), e))[: r["top"]]
    return chosen, [s[e] * r.get("scale", 1.0) for e in chosen]


def routed_ff(h, W, p, f):
    r = f["router"]
    z = h @ W[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen, weights = choose_experts(z[t], W[p + "correction"], r)
        for e, w in zip(chosen, weights):
            out[t] += w * (clamped_expert(h[t], W, f"{p}e{e}.", f["expert"]["limit"]) if e < r["experts"] else h[t])
        if f.get("shared"):
            gate = torch.sigmoid(W[p + "shared.sg"] @ h[t])
            out[t] += gate * clamped_expert(h[t], W, p + "shared.", f["shared"]["limit"])
    return out


# ------------------------------------------------------------------ the model
def model_hidden(cfg, W, tokens):
    """The residual stream after every layer: list of [n, width]."""
    eps = cfg["norm"]["eps"]
    x, after, carry = W["embed"][torch.tensor(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0), [], {}
    for L, layer in enumerate(cfg["layers"]):
        p = f"l{L}."
        x = x + MIXERS[layer["type"]](unit_rms(x, eps) * W[p + "norm1"], W, p + "mix.", layer["mixer"], eps, carry)
        f = layer.get("mlp")
        if f:
            h = unit_rms(x, eps) * W[p + "norm2"]
            x = x + (dense_ff(h, W, p + "mlp.") if f["kind"] == "dense" else routed_ff(h, W, p + "mlp.", f))
        after.append(x)
    return after


def model_logits(cfg, W, tokens):
    x = model_hidden(cfg, W, tokens)[-1]
    return (unit_rms(x, cfg["norm"]["eps"]) * W["final.norm"] @ W["head"].T * cfg.get("logit_scale", 1.0)).to(torch.float32)


def greedy(cfg, W, prompt, n_new):
    tokens = list(prompt)
    for _ in range(n_new):
        tokens.append(int(model_logits(cfg, W, tokens)[-1].argmax()))
    return tokens[len(prompt):]
