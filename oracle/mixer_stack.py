"""Plain numpy statement of decoder stacks.  Komirax: layers that mix tokens by differential attention or by lightning
attention (a linear recurrence with a fixed decay per head) and end in a dense or a routed feed-forward, norms in front of
the branches.  Vifivik: latent attention, retention and Mamba-2 layers with gated feed-forwards, norms behind the branches,
capped logits.  One function per mechanism, written token by token and head by head from the equations; slow, and nothing
here is used by the product.

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


# ---- mixers of Vifivik -------------------------------------------------------------------------------------------------
def rotate_pairs(x, positions, base):
    """Rotary positions on all of the last axis: entries (2i, 2i + 1) turn by position * base^(-2i / size)."""
    n = x.shape[-1]
    out = x.copy()
    for t, p in enumerate(positions):
        for i in range(n // 2):
            a = p * base ** (-2.0 * i / n)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i], out[t, ..., 2 * i + 1] = u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)
    return out


def sink_softmax_attention(q, k, v, scale, sink, start):
    """One head: as causal_softmax_attention, with exp(sink) as one more term of every denominator."""
    out = np.zeros((q.shape[0], v.shape[1]), q.dtype)
    for i in range(q.shape[0]):
        s = (k[:start + i + 1] @ q[i]) * scale
        m = max(s.max(), sink)
        p = np.exp(s - m)
        out[i] = (p / (p.sum() + np.exp(sink - m))) @ v[:start + i + 1]
    return out


def latent_rows(h, w, kv_rank, base, eps, start):
    """What a latent-attention layer caches per token: (latent [T, kv_rank], rotated shared key part [T, rot_dim])."""
    d = h @ w["dkv"].T
    return unit_rms(d[:, :kv_rank], eps) * w["dkv.norm"], rotate_pairs(d[:, kv_rank:], range(start, start + h.shape[0]), base)


def latent_mixer(h, w, heads, dim, rot_dim, vdim, base, scale, latent, rotated, start):
    """h [T, width] at positions start ..; `latent` and `rotated` are the cached rows of all tokens up to the last of h."""
    T = h.shape[0]
    q = (h @ w["q"].T).reshape(T, heads, dim + rot_dim)
    qr = rotate_pairs(q[:, :, dim:], range(start, start + T), base)
    k, v = (latent @ w["uk"].T).reshape(-1, heads, dim), (latent @ w["uv"].T).reshape(-1, heads, vdim)
    gate = sigmoid(h @ w["g"].T)
    o = np.zeros((T, heads, vdim), h.dtype)
    for i in range(heads):
        qi, ki = np.concatenate([q[:, i, :dim], qr[:, i]], axis=1), np.concatenate([k[:, i], rotated], axis=1)
        o[:, i] = gate[:, i:i + 1] * sink_softmax_attention(qi, ki, v[:, i], scale, w["sink"][i], start)
    return o.reshape(T, heads * vdim) @ w["o"].T


def retention_mixer(h, w, heads, dim, vdim, decay, eps, state=None):
    """Linear attention with a fixed decay, unit norm per head, SiLU gate -> (output, final state)."""
    T = h.shape[0]
    q, k = (h @ w["q"].T).reshape(T, heads, dim), (h @ w["k"].T).reshape(T, heads, dim) * dim ** -0.5
    o, state = lightning_recurrence(q, k, (h @ w["v"].T).reshape(T, heads, vdim), np.asarray(decay, h.dtype), state)
    o = unit_rms(o, eps).reshape(T, heads * vdim)
    return (o * silu(h @ w["g"].T)) @ w["o"].T, state


def softplus(z):
    return np.logaddexp(0.0, z)


def causal_conv(x, past, taps, bias):
    """x [T, channels] after the rows `past` [K - 1, channels]; taps [channels, K], the last for the current row.
    Returns (output, the last K - 1 rows)."""
    K = taps.shape[1]
    rows = np.concatenate([past, x])
    out = np.stack([bias + sum(taps[:, j] * rows[t + j] for j in range(K)) for t in range(x.shape[0])])
    return out, rows[rows.shape[0] - (K - 1):]


def selective_recurrence(x, B, C, dt, a_log, D, state=None):
    """x [T, H, e], B and C [T, G, N], dt [T, H].  Returns (y [T, H, e], state [H, N, e])."""
    T, H, e = x.shape
    per = H // B.shape[1]
    S = np.zeros((H, B.shape[2], e), x.dtype) if state is None else state.copy()
    y = np.zeros((T, H, e), x.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = np.exp(-np.exp(a_log[h]) * dt[t, h]) * S[h] + dt[t, h] * np.outer(B[t, h // per], x[t, h])
            y[t, h] = S[h].T @ C[t, h // per] + D[h] * x[t, h]
    return y, S


def gated_group_norm(y, z, weight, groups, eps):
    """RMS norm of y * silu(z) in `groups` equal parts, times the weight."""
    u = (y * silu(z)).reshape(y.shape[0], groups, -1)
    return unit_rms(u, eps).reshape(y.shape) * weight


def mamba2_mixer(h, w, heads, vdim, state, groups, conv, norm_groups, eps, memory=None):
    """Returns (output [T, width], (convolution inputs still needed, recurrent state))."""
    T, inner, n = h.shape[0], heads * vdim, groups * state
    p = h @ w["in"].T
    z, u, dt = p[:, :inner], p[:, inner:2 * inner + 2 * n], p[:, 2 * inner + 2 * n:]
    past, S = (np.zeros((conv - 1, u.shape[1]), h.dtype), None) if memory is None else memory
    c, past = causal_conv(u, past, w["conv"], w["conv.b"])
    c = silu(c)
    x, B, C = c[:, :inner].reshape(T, heads, vdim), c[:, inner:inner + n].reshape(T, groups, state), c[:, inner + n:].reshape(T, groups, state)
    y, S = selective_recurrence(x, B, C, softplus(dt + w["dt_bias"]), w["A_log"], w["D"], S)
    return gated_group_norm(y.reshape(T, inner), z, w["norm"], norm_groups, eps) @ w["o"].T, (past, S)


# ---- feed-forwards -----------------------------------------------------------------------------------------------------
def dense_ff(h, up, down):
    return gelu_tanh(h @ up.T) @ down.T


def gated_ff(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


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


def softcap(z, cap):
    return cap * np.tanh(z / cap)


def run_output_norm_layer(cfg, i, tensors, x, memory, start):
    """One layer whose norms follow its branches; `memory` (a dict by layer, updated) holds caches and states."""
    spec, eps = cfg["layers"][i], cfg["norm"]["eps"]
    m, w = spec["mixer"], _sub(tensors, f"l{i}.mix.")
    if spec["type"] == "latent_attention":
        base, source = m["rot"]["base"], m.get("kv_from", i)
        if source == i:
            rows = latent_rows(x, w, m["kv_rank"], base, eps, start)
            memory[i] = rows if i not in memory else tuple(np.concatenate(r) for r in zip(memory[i], rows))
        y = latent_mixer(x, w, m["heads"], m["dim"], m["rot_dim"], m["vdim"], base, m["scale"], *memory[source], start)
    elif spec["type"] == "retention":
        y, memory[i] = retention_mixer(x, w, m["heads"], m["dim"], m["vdim"], m["decay"], eps, memory.get(i))
    else:
        y, memory[i] = mamba2_mixer(x, w, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"], eps, memory.get(i))
    x = x + unit_rms(y, eps) * tensors[f"l{i}.norm1"]
    if spec.get("mlp") is not None:
        f = _sub(tensors, f"l{i}.mlp.")
        x = x + unit_rms(gated_ff(x, f["gate"], f["up"], f["down"]), eps) * tensors[f"l{i}.norm2"]
    return x


def forward_output_norm(cfg, tensors, tokens, memory=None, residuals=None):
    """`forward` of a stack whose norms follow the branches."""
    memory = {} if memory is None else memory
    start = memory.get("tokens", 0)
    x = tensors["embed"][np.asarray(tokens)]
    for i in range(len(cfg["layers"])):
        x = run_output_norm_layer(cfg, i, tensors, x, memory, start)
        if residuals is not None:
            residuals.append(x)
    memory["tokens"] = start + len(tokens)
    logits = (unit_rms(x, cfg["norm"]["eps"]) * tensors["final.norm"]) @ tensors["head"].T
    return softcap(logits, cfg["logit_softcap"]) if cfg.get("logit_softcap") else logits


def forward(cfg, tensors, tokens, memory=None, residuals=None):
    """Logits [T, vocab] of `tokens`, which follow the tokens that `memory` (a dict, updated) has seen."""
    if cfg["architecture"] == "Vifivik":
        return forward_output_norm(cfg, tensors, tokens, memory, residuals)
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
