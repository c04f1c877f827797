"""Plain numpy statement of a decoder stack whose layers mix tokens by differential attention or by lightning attention
(a linear recurrence with a fixed decay per head) and end in a dense or a routed feed-forward.  One function per
mechanism, written token by token and head by head from the equations; slow, and nothing here is used by the product.

Arrays are float64 unless a caller passes something else; weights are [out, in] and applied as W x."""
from __future__ import annotations

import numpy as np


# ---- elementwise and norms ---------------------------------------------------------------------------------------------
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return np.maximum(z, 0.0) ** 2


def unit_rms(x, eps):
    """x over the root of (its mean square + eps), along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


# ---- mixers ------------------------------------------------------------------------------------------------------------
def lightning_recurrence(q, k, v, decay, state=None):
    """q, k [T, H, d], v [T, H, e], decay [H].  Returns (o [T, H, e], final state [H, d, e])."""
    T, H, d = q.shape
    e = v.shape[2]
    S = np.zeros((H, d, e), q.dtype) if state is None else state.copy()
    out = np.zeros((T, H, e), q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out, S


def lightning_mixer(h, w, heads, dim, vdim, decay, eps, state=None):
    """h [T, width] (already normed) -> (mixer output [T, width], final state)."""
    T = h.shape[0]
    q = silu(h @ w["q"].T).reshape(T, heads, dim)
    k = silu(h @ w["k"].T).reshape(T, heads, dim)
    v = silu(h @ w["v"].T).reshape(T, heads, vdim)
    o, state = lightning_recurrence(q, k, v, np.asarray(decay, h.dtype), state)
    o = unit_rms(o.reshape(T, heads * vdim), eps) * w["norm"]
    return (o * sigmoid(h @ w["g"].T)) @ w["o"].T, state


def diff_lambda(w, diff):
    return np.exp(np.sum(w["lq1"] * w["lk1"])) - np.exp(np.sum(w["lq2"] * w["lk2"])) + diff


def causal_softmax_attention(q, k, v, scale, start):
    """One head: q [n, d] at positions start .. start + n, k [L, d] and v [L, e] from position 0."""
    out = np.zeros((q.shape[0], v.shape[1]), q.dtype)
    for i in range(q.shape[0]):
        s = (k[:start + i + 1] @ q[i]) * scale
        p = np.exp(s - s.max())
        out[i] = (p / p.sum()) @ v[:start + i + 1]
    return out


def differential_combine(a1, a2, lam, diff, eps):
    """Two maps' outputs of one head -> the head's output."""
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def differential_mixer(h, w, heads, kv_heads, dim, vdim, scale, diff, eps, past=None):
    """h [T, width]; `past` = (k, v) rows of the tokens before.  Returns (output [T, width], (k, v) of all tokens)."""
    T = h.shape[0]
    q = (h @ w["q"].T + w["q.b"]).reshape(T, heads, 2, dim)
    k = (h @ w["k"].T + w["k.b"]).reshape(T, kv_heads, 2, dim)
    v = (h @ w["v"].T + w["v.b"]).reshape(T, kv_heads, vdim)
    start = 0
    if past is not None:
        start = past[0].shape[0]
        k, v = np.concatenate([past[0], k]), np.concatenate([past[1], v])
    lam = diff_lambda(w, diff)
    o = np.zeros((T, heads, vdim), h.dtype)
    for hd in range(heads):
        g = hd // (heads // kv_heads)
        a1 = causal_softmax_attention(q[:, hd, 0], k[:, g, 0], v[:, g], scale, start)
        a2 = causal_softmax_attention(q[:, hd, 1], k[:, g, 1], v[:, g], scale, start)
        o[:, hd] = differential_combine(a1, a2, lam, diff, eps)
    return o.reshape(T, heads * vdim) @ w["o"].T, (k, v)


# ---- feed-forwards -----------------------------------------------------------------------------------------------------
def dense_ff(h, up, down):
    return gelu_tanh(h @ up.T) @ down.T


def route(h, router, top):
    """Per token the chosen experts (best first) and their weights."""
    s = sigmoid(h @ router.T)
    ids = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return ids, np.take_along_axis(s, ids, axis=1)


def moe_ff(h, router, ups, downs, top):
    ids, weights = route(h, router, top)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t], weights[t]):
            out[t] += downs[e] @ relu_squared(ups[e] @ (wt * h[t]))
    return out


# ---- the stack ---------------------------------------------------------------------------------------------------------
def layer_runs(n_layers, loop):
    """[(layer, pass of the loop or 0)] in running order."""
    if not loop:
        return [(i, 0) for i in range(n_layers)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    return ([(i, 0) for i in range(a)] + [(i, p) for p in range(times) for i in range(a, b)]
            + [(i, 0) for i in range(b, n_layers)])


def _sub(tensors, prefix):
    return {n[len(prefix):]: t for n, t in tensors.items() if n.startswith(prefix)}


def run_layer(cfg, i, tensors, x, memory):
    """One run of layer i; `memory` is what this run carried over from earlier tokens (None at first)."""
    spec, eps = cfg["layers"][i], cfg["norm"]["eps"]
    mix, w = spec["mixer"], _sub(tensors, f"l{i}.mix.")
    h = unit_rms(x, eps) * tensors[f"l{i}.norm1"]
    if spec["type"] == "lightning":
        y, memory = lightning_mixer(h, w, mix["heads"], mix["dim"], mix["vdim"], mix["decay"], eps, memory)
    else:
        y, memory = differential_mixer(h, w, mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"], mix["scale"], mix["diff"], eps, memory)
    x = x + y
    ff = spec.get("mlp")
    if ff is not None:
        h = unit_rms(x, eps) * tensors[f"l{i}.norm2"]
        m = _sub(tensors, f"l{i}.mlp.")
        if ff["kind"] == "dense":
            x = x + dense_ff(h, m["up"], m["down"])
        else:
            n = ff["router"]["experts"]
            x = x + moe_ff(h, m["router"], [m[f"e{e}.up"] for e in range(n)], [m[f"e{e}.down"] for e in range(n)], ff["router"]["top"])
    return x, memory


def forward(cfg, tensors, tokens, memory=None, residuals=None):
    """Logits [T, vocab] of `tokens`, which follow the tokens that `memory` (a dict, updated) has seen."""
    memory = {} if memory is None else memory
    x0 = tensors["embed"][np.asarray(tokens)]
    x = x0
    loop = cfg.get("loop")
    for i, p in layer_runs(len(cfg["layers"]), loop):
        if p > 0 and i == loop["start"]:
            x = x + x0
        x, memory[i, p] = run_layer(cfg, i, tensors, x, memory.get((i, p)))
        if residuals is not None:
            residuals.append(x)
    return (unit_rms(x, cfg["norm"]["eps"]) * tensors["final.norm"]) @ tensors["head"].T
