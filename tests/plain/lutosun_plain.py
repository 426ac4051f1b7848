"""Lutosun, whole sequences, no cache, float64 numpy: one function per mechanism. It shares no code with the product
path.

A Lutosun layer norms what a sublayer reads (a layer norm with weight and bias) and adds what it puts out times one constant
``m`` of the model: ``x += m mixer(N1(x))``, then ``x += m ff(N2(x))``. The stream starts as the token's scaled embedding plus a
row that the token and the one before it choose together (``bigram_rows``). A run of layers may be run several times in a row
with the same weights, every pass over keys of its own; in front of a pass a vector that belongs to the pass joins the stream,
and, in front of every pass but the first, what the embedding put out as well (``run_plan``).

* ``latent_attention``: queries made from one normed latent of the token, keys and values of every head from another, beside one
  rotated key part that all heads share; causal softmax.
* ``mixture_ff``: experts with bounded gate and up values, chosen by the softmax over all experts plus a correction that the
  weights do not see; the chosen ones' softmax values are brought to the sum one and scaled; a shared expert of the same form
  runs for every token, times a sigmoid read off the token.

The logits are bounded by a tanh.

Notation: T tokens, W width, H heads, D plain and R rotated elements of a head, E value size, Q and C latent sizes.
"""

from __future__ import annotations

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
# engine must (norm outputs, both latents, the turned parts, what the output and down projections read), and nothing else:
# the difference to the exact result is a sample of the error that rounding alone causes at each position.
_round = no_rounding


# ---------------------------------------------------------------- embedding


def bigram_rows(tokens, bigram):
    """The row of the pair table that every token adds: ``(previous * a + token * b) mod n``, and row ``n`` for the first."""
    n = bigram["buckets"]
    t = [int(x) for x in tokens]
    return np.array([n] + [(t[i - 1] * bigram["mul_prev"] + t[i] * bigram["mul_cur"]) % n for i in range(1, len(t))], dtype=np.int64)


def embed(tokens, weights, e):
    x = weights["embed"][np.asarray(tokens)] * e["scale"]
    if e.get("bigram"):
        x = x + weights["bigram"][bigram_rows(tokens, e["bigram"])]
    return x


# ---------------------------------------------------------------- norms


def layer_norm(x, w, b, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + eps) * w + b


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


# ---------------------------------------------------------------- mixer


def rotate_neighbours(x, positions, rot):
    """Turns the pairs (2i, 2i + 1), i < n/2, of the first n elements of the last axis of ``x [T, heads, >= n]`` by
    ``position * base^(-2i/n)``; what lies behind n passes."""
    n = rot["dims"]
    ang = positions[:, None] * float(rot["base"]) ** (-np.arange(0, n, 2) / n)
    cos, sin = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * cos - v * sin
    out[..., 1:n:2] = v * cos + u * sin
    return out


def causal_softmax(scores):
    T = scores.shape[-1]
    s = np.where(np.tril(np.ones((T, T), dtype=bool)), scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def latent_queries(h, w, m, eps):
    """``[T, H, D + R]`` from the token's normed query latent."""
    c = _round(rms_norm(h @ w["dq"].T, w["dq.norm"], eps))
    return (c @ w["uq"].T).reshape(len(h), m["heads"], m["dim"] + m["rot_dim"])


def latent_attention(h, w, m, eps, positions):
    T = h.shape[0]
    H, D, R, E, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = latent_queries(h, w, m, eps)
    down = h @ w["dkv"].T
    c = _round(rms_norm(down[:, :C], w["dkv.norm"], eps))
    shared = _round(rotate_neighbours(down[:, None, C:], positions, m["rot"]))[:, 0]
    plain_q, turned_q = _round(q[..., :D]), _round(rotate_neighbours(q[..., D:], positions, m["rot"]))
    k = (c @ w["uk"].T).reshape(T, H, D)
    v = (c @ w["uv"].T).reshape(T, H, E)
    out = np.zeros((T, H, E))
    for a in range(H):
        p = causal_softmax((plain_q[:, a] @ k[:, a].T + turned_q[:, a] @ shared.T) * m["scale"])
        out[:, a] = p @ v[:, a]
    return _round(out.reshape(T, H * E)) @ w["o"].T


# ---------------------------------------------------------------- feed-forward


def route(h, router_weights, correction, router):
    """Per token the chosen experts, largest corrected score first (ties: the lower number), and their weights."""
    z = h @ router_weights.T
    s = np.exp(z - z.max(axis=-1, keepdims=True))
    s = s / s.sum(axis=-1, keepdims=True)
    chosen = np.argsort(-(s + correction), axis=-1, kind="stable")[:, : router["top"]]
    picked = np.take_along_axis(s, chosen, axis=-1)
    return chosen, picked / (picked.sum(axis=-1, keepdims=True) + 1e-20) * router["scale"]


def bounded_swiglu(gate, up, limit):
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(h, gate, up, down, limit, factor=1.0):
    """``factor`` multiplies the result; where a 16-bit engine applies it, between activation and ``down``, is where the
    rounding is."""
    return _round(bounded_swiglu(h @ gate.T, h @ up.T, limit) * factor) @ down.T


def mixture_ff(h, w, mlp):
    chosen, weight = route(h, w["router"], w["correction"], mlp["router"])
    out = np.zeros_like(h)
    limit = mlp["expert"]["limit"]
    for t in range(h.shape[0]):
        for e, p in zip(chosen[t], weight[t]):
            out[t] += p * expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], limit)
    if mlp.get("shared"):
        out += expert(h, w["shared.gate"], w["shared.up"], w["shared.down"], mlp["shared"]["limit"], sigmoid(h @ w["shared.sg"].T))
    return out


# ---------------------------------------------------------------- the model


def run_plan(cfg):
    """The layer runs in order: ``(layer, pass)``, ``pass`` the number of the pass that begins with this run, else None."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    looped = [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)]
    return [(i, None) for i in range(a)] + looped + [(i, None) for i in range(b, n)]


def begin_pass(x, start, steps, t):
    """What joins the stream ``x`` ahead of pass ``t``: its own vector, and from the second pass on the embedding's output."""
    return x + steps[t] + (start if t > 0 else 0.0)


def bound_logits(z, cap):
    return cap * np.tanh(z / cap) if cap else z


def _sub(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, return_layers=False, watch=None, rounding=None):
    """Logits ``[T, vocab]`` of one sequence (and, asked for, the stream after every layer run ``[runs, T, W]``).
    ``watch(run, layer, x)`` is shown the stream that a run's feed-forward norm reads. ``rounding``: see ``_round``."""
    global _round
    before, _round = _round, rounding or no_rounding
    try:
        return _forward(cfg, weights, tokens, return_layers, watch)
    finally:
        _round = before


def _forward(cfg, weights, tokens, return_layers, watch):
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    positions = np.arange(len(tokens), dtype=np.float64)
    start = embed(tokens, weights, cfg["embedding"])
    x = start.copy()
    after = []
    for run, (i, t) in enumerate(run_plan(cfg)):
        layer, p = cfg["layers"][i], f"l{i}."
        if t is not None:
            x = begin_pass(x, start, weights["loop.step"], t)
        if layer["type"] != "latent_attention":
            raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
        h = _round(layer_norm(x, weights[p + "norm1"], weights[p + "norm1.b"], eps))
        x = x + m * latent_attention(h, _sub(weights, p + "mix."), layer["mixer"], eps, positions)
        if layer.get("mlp"):
            if watch is not None:
                watch(run, i, x)
            h = _round(layer_norm(x, weights[p + "norm2"], weights[p + "norm2.b"], eps))
            x = x + m * mixture_ff(h, _sub(weights, p + "mlp."), layer["mlp"])
        after.append(x.copy())
    h = _round(layer_norm(x, weights["final.norm"], weights["final.norm.b"], eps))
    logits = bound_logits(h @ weights["head"].T, cfg["logit_softcap"])
    return (logits, np.stack(after)) if return_layers else logits


def greedy(cfg, weights, prompt, new_tokens):
    """The ``new_tokens`` tokens that greedy decoding appends to ``prompt`` (the whole sequence is run again each time)."""
    toks = list(prompt)
    for _ in range(new_tokens):
        toks.append(int(np.argmax(forward(cfg, weights, toks)[-1])))
    return toks[len(prompt):]
