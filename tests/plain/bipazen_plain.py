"""Bipazen, whole sequences, no cache, float64 numpy: one function per mechanism. It shares no code with the product
path.

A Bipazen layer norms what a sublayer reads and scales what it puts out, channel by channel: ``x += s1 * mixer(N1(x))``,
then ``x += s2 * ff(N2(x))``, with ``N(y) = w y / rms(y)``. Three mixers:

* ``mamba2``: one projection makes a gate, values, keys and queries (the latter two shared by the heads of a group) and a
  step size per head; values, keys and queries pass a short causal convolution and a SiLU; per head a matrix state that
  forgets by ``exp(-exp(A) d_t)`` and takes in ``d_t k_t v_t^T``; the read-out and a share of the value, times the gate's
  SiLU, normed in equal parts, projected.
* ``rglru``: two branches, one of which passes a short causal convolution and then a gated linear recurrence per channel
  whose two gates are block-diagonal products of the convolved branch; the other, through a GELU, multiplies the result.
* ``latent_attention``: keys and values of every head made from one normed latent vector per token, beside one rotated key
  part that all heads share; causal softmax; a sigmoid gate on every element of the heads' outputs.

Feed-forward: a mixture of gated SiLU experts; the router's sigmoid scores choose, and a chosen expert reads its input
times its score. The head is the embedding table.

Notation: T tokens, W width, H heads, N state size, E value size, G groups, C latent size, R rotated elements.
"""

from __future__ import annotations

import math

import numpy as np


# ---------------------------------------------------------------- rounding, for error estimates


def no_rounding(a):
    return a


def to_bfloat16(a):
    """``a`` rounded to the nearest bfloat16 (ties to even), as float64: what a 16-bit product is fed."""
    bits = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    bits = ((bits + 0x7FFF + ((bits >> 16) & 1)) >> 16) << 16
    return bits.astype(np.uint32).view(np.float32).astype(np.float64).reshape(np.shape(a))


# What the inputs of the matrix products go through. ``forward(..., rounding=to_bfloat16)`` rounds them as a 16-bit
# engine must (norm outputs, what the cache holds, what the output and down projections read), and nothing else: the
# difference to the exact result is a sample of the error that rounding alone causes at each position.
_round = no_rounding


# ---------------------------------------------------------------- norms and activations


def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def weighted_norm(x, w, eps):
    return unit_rms(x, eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z**3)))


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


# ---------------------------------------------------------------- over time


def causal_conv(u, w, b):
    """``y_t[c] = b[c] + sum_j w[c, j] u_(t - taps + 1 + j)[c]``; before the start there are zeros."""
    T, taps = u.shape[0], w.shape[1]
    y = np.zeros_like(u) + b
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[: T - back]
    return y


def scalar_decay_recurrence(q, k, v, log_decay, step, skip):
    """Per head ``S_t = exp(log_decay_t) S_(t-1) + step_t k_t v_t^T``, ``o_t = S_t^T q_t + skip v_t``; ``q, k [T, H, N]``,
    ``v [T, H, E]``, ``log_decay, step [T, H]``, ``skip [H]``. Returns the outputs and the last state ``[H, N, E]``."""
    T, H, N = q.shape
    out, S = np.zeros_like(v), np.zeros((H, N, v.shape[2]))
    for t in range(T):
        S = np.exp(log_decay[t])[:, None, None] * S + step[t][:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hne,hn->he", S, q[t]) + skip[:, None] * v[t]
    return out, S


def channel_recurrence(log_a, x):
    """``S_t = a_t S_(t-1) + sqrt(1 - a_t^2) x_t`` per channel from zero, with ``a = exp(log_a)``; ``[T, width]``."""
    S, out = np.zeros(x.shape[1]), np.zeros_like(x)
    for t in range(x.shape[0]):
        S = np.exp(log_a[t]) * S + np.sqrt(-np.expm1(2.0 * log_a[t])) * x[t]
        out[t] = S
    return out


# ---------------------------------------------------------------- mixers


def mamba2(h, w, m, eps):
    T = h.shape[0]
    H, E, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * E
    z, xbc, dt = np.split(h @ w["in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    of_head = np.arange(H) // (H // G)
    k = B.reshape(T, G, N)[:, of_head]
    q = C.reshape(T, G, N)[:, of_head]
    step = softplus(dt + w["dt_bias"])
    y, _ = scalar_decay_recurrence(q, k, x.reshape(T, H, E), -np.exp(w["A_log"]) * step, step, w["D"])
    y = y.reshape(T, inner) * silu(z)
    y = unit_rms(y.reshape(T, m["norm_groups"], -1), eps).reshape(T, inner) * w["norm"]
    return _round(y) @ w["o"].T


def rglru(h, w, m):
    T = h.shape[0]
    n = m["blocks"]
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = causal_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    parts = u.reshape(T, n, -1)
    r, i = (np.concatenate([sigmoid(parts[:, b] @ w[g][b].T + w[g + ".b"][b]) for b in range(n)], axis=1) for g in ("ra", "ri"))
    S = channel_recurrence(-8.0 * r * softplus(w["lam"]), i * u)
    return _round(S * y) @ w["o"].T


def rotate_halves(x, positions, rot):
    """Turns the pairs (i, i + R/2), i < R/2, of the first R elements of the last axis of ``x [T, heads, >= R]`` by
    ``position * base^(-2i/R)``; what lies behind R passes."""
    R = rot["dims"]
    ang = positions[:, None] * float(rot["base"]) ** (-2.0 * np.arange(R // 2) / R)
    cos, sin = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.copy()
    a, b = x[..., : R // 2], x[..., R // 2 : R]
    out[..., : R // 2] = a * cos - b * sin
    out[..., R // 2 : R] = b * cos + a * sin
    return out


def causal_softmax(scores):
    T = scores.shape[-1]
    s = np.where(np.tril(np.ones((T, T), dtype=bool)), scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def latent_attention(h, w, m, eps, positions):
    T = h.shape[0]
    H, D, R, E, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w["q"].T).reshape(T, H, D + R)
    down = h @ w["dkv"].T
    c = _round(weighted_norm(down[:, :C], w["dkv.norm"], eps))
    shared = _round(rotate_halves(down[:, None, C:], positions, m["rot"]))[:, 0]
    plain_q, turned_q = _round(q[..., :D]), _round(rotate_halves(q[..., D:], positions, m["rot"]))
    k = (c @ w["uk"].T).reshape(T, H, D)
    v = (c @ w["uv"].T).reshape(T, H, E)
    out = np.zeros((T, H, E))
    for a in range(H):
        p = causal_softmax((plain_q[:, a] @ k[:, a].T + turned_q[:, a] @ shared.T) * m["scale"])
        out[:, a] = p @ v[:, a]
    return _round(out.reshape(T, H * E) * sigmoid(h @ w["g"].T)) @ w["o"].T


# ---------------------------------------------------------------- feed-forward


def route(h, router_weights, top):
    """Per token the chosen experts, largest score first (ties: the lower number), and their scores."""
    s = sigmoid(h @ router_weights.T)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=-1)


def expert(h, gate, up, down):
    return _round(silu(h @ gate.T) * (h @ up.T)) @ down.T


def mixture_ff(h, w, mlp):
    chosen, score = route(h, w["router"], mlp["router"]["top"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(chosen[t], score[t]):
            out[t] += expert(s * h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"])
    return out


# ---------------------------------------------------------------- the model


def weights_layer(cfg, i):
    """The layer whose tensors layer ``i`` runs: itself, or the end of its chain of ``weights_of``."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def _sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, return_layers=False, watch=None, rounding=None):
    """Logits ``[T, vocab]`` of one sequence (and, asked for, the stream after every layer ``[layers, T, W]``).
    ``watch(i, x)`` is shown the stream that layer ``i``'s feed-forward norm reads. ``rounding``: see ``_round``."""
    global _round
    before, _round = _round, rounding or no_rounding
    try:
        return _forward(cfg, weights, tokens, return_layers, watch)
    finally:
        _round = before


def _forward(cfg, weights, tokens, return_layers, watch):
    eps = cfg["norm"]["eps"]
    tokens = np.asarray(tokens)
    positions = np.arange(len(tokens), dtype=np.float64)
    x = weights["embed"][tokens].astype(np.float64)
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{weights_layer(cfg, i)}."
        w, m = _sub(weights, p + "mix."), layer["mixer"]
        h = _round(weighted_norm(x, weights[p + "norm1"], eps))
        if layer["type"] == "mamba2":
            y = mamba2(h, w, m, eps)
        elif layer["type"] == "rglru":
            y = rglru(h, w, m)
        elif layer["type"] == "latent_attention":
            y = latent_attention(h, w, m, eps, positions)
        else:
            raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
        x = x + weights[p + "ls1"] * y
        if layer.get("mlp"):
            if watch is not None:
                watch(i, x)
            h = _round(weighted_norm(x, weights[p + "norm2"], eps))
            x = x + weights[p + "ls2"] * mixture_ff(h, _sub(weights, p + "mlp."), layer["mlp"])
        after.append(x.copy())
    logits = _round(weighted_norm(x, weights["final.norm"], eps)) @ weights["embed"].T
    return (logits, np.stack(after)) if return_layers else logits


def greedy(cfg, weights, prompt, new_tokens):
    """The ``new_tokens`` tokens that greedy decoding appends to ``prompt`` (the whole sequence is run again each time)."""
    toks = list(prompt)
    for _ in range(new_tokens):
        toks.append(int(np.argmax(forward(cfg, weights, toks)[-1])))
    return toks[len(prompt):]
