"""Plain float64 restatement of a layered decoder whose mixers are two mixers side by side (sliding-window
attention with normalised, rotated queries and keys; the gated delta rule), whose norms sit on the
sublayers' outputs and whose feed-forwards clamp both halves.  One function per mechanism (test
infrastructure only; shares no code with the product).

Everything works on one sequence of `t` tokens at once, from position 0, with explicit loops where a
loop is the definition.  `config` is the parsed config.json, `weights` maps tensor names to arrays.
"""
from __future__ import annotations

import numpy as np

from .hybrid_model import f64, rms_unit, sigmoid, silu, softplus


def offset_rms_norm(x, w, eps):
    """The norm whose weight is stored around zero."""
    return rms_unit(x, eps) * (1.0 + w)


def frequencies(dims, base, factor):
    """One per rotated pair, all divided by the scaling factor."""
    return np.array([base ** (-2.0 * i / dims) / factor for i in range(dims // 2)])


def rotate(x, dims, base, factor):
    """x [t, heads, d]: component i < dims / 2 with component i + dims / 2, by position times frequency."""
    out = x.copy()
    half = dims // 2
    f = frequencies(dims, base, factor)
    for p in range(x.shape[0]):
        c, s = np.cos(p * f), np.sin(p * f)
        u, v = x[p, :, :half], x[p, :, half:dims]
        out[p, :, :half] = u * c - v * s
        out[p, :, half:dims] = v * c + u * s
    return out


def in_window(i, j, size):
    """True when position i sees position j: itself and the size - 1 positions before it."""
    return 0 <= i - j and (size is None or i - j < size)


def window_attention(q, k, v, scale, size):
    """q [t, H, d], k [t, G, d], v [t, G, e] -> [t, H, e]."""
    t, heads, _ = q.shape
    per = heads // k.shape[1]
    out = np.zeros((t, heads, v.shape[2]))
    for i in range(t):
        seen = [j for j in range(t) if in_window(i, j, size)]
        for h in range(heads):
            s = (k[seen, h // per] @ q[i, h]) * scale
            e = np.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[seen, h // per]
    return out


def attention_mixer(h, m, w, eps):
    t, heads, kv, dim = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    rot, mask = m.get("rot") or {"dims": 0, "base": 1.0}, m.get("mask")
    turn = (rot["dims"], rot["base"], rot["scaling"]["factor"] if rot.get("scaling") else 1.0)
    q = rms_unit((h @ w("q").T).reshape(t, heads, dim), eps) * w("q.norm")
    k = rms_unit((h @ w("k").T).reshape(t, kv, dim), eps) * w("k.norm")
    v = (h @ w("v").T).reshape(t, kv, m["vdim"])
    out = window_attention(rotate(q, *turn), rotate(k, *turn), v, m["scale"],
                           mask["size"] if mask else None)
    return out.reshape(t, -1) @ w("o").T


def short_conv(x, w):
    """Per channel over time: x [t, c], w [c, taps] (last column: the current token), zeros before the start."""
    out = np.zeros_like(x)
    taps = w.shape[1]
    for i in range(x.shape[0]):
        for back in range(min(taps, i + 1)):
            out[i] += w[:, taps - 1 - back] * x[i - back]
    return out


def unit(x):
    """Every head's vector to length one."""
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_scan(q, k, v, decay, beta):
    """q, k [t, G, d], v [t, H, e], decay [t, H, d], beta [t, H] -> [t, H, e].  Token by token:
    S <- diag(decay) S; u = beta (v - S^T k); S <- S + k u^T; out = S^T q."""
    t, heads, e = v.shape
    per = heads // k.shape[1]
    state = np.zeros((heads, k.shape[2], e))
    out = np.zeros_like(v)
    for i in range(t):
        for h in range(heads):
            s, key = decay[i, h][:, None] * state[h], k[i, h // per]
            u = beta[i, h] * (v[i, h] - s.T @ key)
            state[h] = s + np.outer(key, u)
            out[i, h] = state[h].T @ q[i, h // per]
    return out


def channel_decay(h, w, heads, dim):
    """One factor per head and key channel."""
    step = softplus((h @ w("a1").T) @ w("a2").T + w("dt_bias")).reshape(-1, heads, dim)
    return np.exp(-np.exp(w("A_log"))[None, :, None] * step)


def delta_mixer(h, m, w, eps):
    t, heads, kv, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda name: silu(short_conv(h @ w(name).T, w(name + ".conv")))
    q = unit(conv("q").reshape(t, kv, dim)) / np.sqrt(dim)
    k = unit(conv("k").reshape(t, kv, dim))
    v = conv("v").reshape(t, heads, vdim)
    o = delta_scan(q, k, v, channel_decay(h, w, heads, dim), sigmoid(h @ w("b").T))
    gate = sigmoid((h @ w("g1").T) @ w("g2").T).reshape(t, heads, vdim)
    return (rms_unit(o, eps) * w("norm") * gate).reshape(t, -1) @ w("o").T


def parallel_mixer(h, m, w, eps):
    left = attention_mixer(h, m["left"], lambda name: w("left." + name), eps)
    right = delta_mixer(h, m["right"], lambda name: w("right." + name), eps)
    return m["left_scale"] * left + m["right_scale"] * right


def clamped_ffn(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def forward(config, weights, tokens):
    """Logits [t, vocab] and the residual stream after every layer [layers, t, width]."""
    eps, m = config["norm"]["eps"], config["residual_mult"]
    get = lambda name: f64(weights[name])
    x, streams = get("embed")[np.asarray(tokens)], []
    for index, layer in enumerate(config["layers"]):
        prefix = "l%d." % index
        y = parallel_mixer(x, layer["mixer"], lambda name: get(prefix + "mix." + name), eps)
        x = x + m * offset_rms_norm(y, get(prefix + "norm1"), eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            y = clamped_ffn(x, *(get(prefix + "mlp." + name) for name in ("gate", "up", "down")), mlp["limit"])
            x = x + m * offset_rms_norm(y, get(prefix + "norm2"), eps)
        streams.append(x)
    cap = config["logit_softcap"]
    logits = offset_rms_norm(x, get("final.norm"), eps) @ get("embed").T
    return cap * np.tanh(logits / cap), np.stack(streams)
