"""Plain float64 restatement of the layered decoder (attention / Mamba-2 mixers, dense and routed
feed-forwards), one function per mechanism (test infrastructure only; shares no code with the product).

Everything works on one sequence of `t` tokens at once, from position 0, with explicit loops where a
loop is the definition.  `config` is the parsed config.json, `weights` maps tensor names to arrays.
"""
from __future__ import annotations

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


def silu(z):
    return z / (1.0 + np.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_unit(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def grouped_rms_norm(x, w, eps, groups):
    """Every one of `groups` equal parts of the last axis by its own root mean square."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms_unit(parts, eps).reshape(x.shape) * w


def visible(i, j, chunk):
    """True when position i sees position j: not later, and in the same chunk (chunk None: no chunks)."""
    return j <= i and (chunk is None or i // chunk == j // chunk)


def chunk_attention(q, k, v, scale, softcap, sink, chunk):
    """q [t, H, d], k [t, G, d], v [t, G, e], sink [H] -> [t, H, e].  Scores scaled, then capped; the sink adds to
    the denominator only."""
    t, heads, _ = q.shape
    group = heads // k.shape[1]
    out = np.zeros((t, heads, v.shape[2]))
    for i in range(t):
        seen = [j for j in range(t) if visible(i, j, chunk)]
        for h in range(heads):
            s = (k[seen, h // group] @ q[i, h]) * scale
            if softcap is not None:
                s = softcap * np.tanh(s / softcap)
            top = max(s.max(), sink[h]) if sink is not None else s.max()
            e = np.exp(s - top)
            denominator = e.sum() + (np.exp(sink[h] - top) if sink is not None else 0.0)
            out[i, h] = (e / denominator) @ v[seen, h // group]
    return out


def causal_conv(x, w, b):
    """Per channel over time: x [t, c], w [c, taps] (last column: the current token), zeros before the start."""
    t, taps = x.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    out = np.zeros_like(x)
    for i in range(t):
        out[i] = np.sum(padded[i:i + taps] * w.T, axis=0) + b
    return out


def ssm_scan(x, b, c, dt, a, d):
    """x [t, heads, v], b, c [t, groups, n], dt [t, heads] (after softplus), a [heads] (positive), d [heads]:
    S <- exp(-a dt) S + dt b x^T, y = S^T c + d x, token by token."""
    t, heads, vdim = x.shape
    per = heads // b.shape[1]
    y = np.zeros_like(x)
    state = np.zeros((heads, b.shape[2], vdim))
    for i in range(t):
        for h in range(heads):
            g = h // per
            state[h] = np.exp(-a[h] * dt[i, h]) * state[h] + dt[i, h] * np.outer(b[i, g], x[i, h])
            y[i, h] = state[h].T @ c[i, g] + d[h] * x[i, h]
    return y


def attention_mixer(h, m, w, v_first):
    """Returns (output, the layer's own values) - the latter are what later layers mix in."""
    t = h.shape[0]
    heads, kv = m["heads"], m["kv_heads"]
    q = (h @ w("q").T).reshape(t, heads, m["dim"])
    k = (h @ w("k").T).reshape(t, kv, m["dim"])
    own = (h @ w("v").T).reshape(t, kv, m["vdim"])
    v = own
    if m.get("v_mix") and v_first is not None:
        mix = float(w("vmix"))
        v = (1.0 - mix) * own + mix * v_first
    mask = m.get("mask")
    out = chunk_attention(q, k, v, m["scale"], m.get("softcap"), w("sink"), None if mask is None else mask["size"])
    return out.reshape(t, -1) @ w("o").T, own


def mamba2_mixer(h, m, w, eps):
    t = h.shape[0]
    heads, vdim, n, groups = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = heads * vdim
    p = h @ w("in").T
    z, xbc, dt = p[:, :inner], p[:, inner:2 * inner + 2 * groups * n], p[:, 2 * inner + 2 * groups * n:]
    xbc = silu(causal_conv(xbc, w("conv"), w("conv.b")))
    x = xbc[:, :inner].reshape(t, heads, vdim)
    b = xbc[:, inner:inner + groups * n].reshape(t, groups, n)
    c = xbc[:, inner + groups * n:].reshape(t, groups, n)
    y = ssm_scan(x, b, c, softplus(dt + w("dt_bias")), np.exp(w("A_log")), w("D")).reshape(t, inner)
    return grouped_rms_norm(y * silu(z), w("norm"), eps, m["norm_groups"]) @ w("o").T


def gated_ffn(h, gate, up, down, act):
    return (act(h @ gate.T) * (h @ up.T)) @ down.T


def route(z, top):
    """The `top` largest logits of one token and the softmax over them alone."""
    chosen = np.argsort(-z, kind="stable")[:top]
    e = np.exp(z[chosen] - z[chosen].max())
    return chosen, e / e.sum()


def moe_ffn(h, m, w):
    logits = h @ w("router").T
    out = np.zeros((h.shape[0], w("e0.down").shape[0]))
    for i in range(h.shape[0]):
        for expert, weight in zip(*route(logits[i], m["router"]["top"])):
            name = "e%d." % expert
            out[i] += weight * gated_ffn(h[i], w(name + "gate"), w(name + "up"), w(name + "down"), silu)
    if m.get("shared") is not None:
        shared = gated_ffn(h, w("shared.gate"), w("shared.up"), w("shared.down"), silu)
        out += sigmoid(h @ w("shared.sg").T) * shared
    return out


def forward(config, weights, tokens):
    """Logits [t, vocab] and the residual stream after every layer [layers, t, width]."""
    eps = config["norm"]["eps"]
    get = lambda name: f64(weights[name])
    x = get("embed")[np.asarray(tokens)] * config["embedding"]["scale"]
    v_first, streams = None, []
    for index, layer in enumerate(config["layers"]):
        prefix = "l%d." % index
        h = rms_norm(x, get(prefix + "norm1"), eps)
        w = lambda name: get(prefix + "mix." + name)
        if layer["type"] == "attention":
            y, own = attention_mixer(h, layer["mixer"], w, v_first)
            if layer["mixer"].get("v_mix") and v_first is None:
                v_first = own
        elif layer["type"] == "mamba2":
            y = mamba2_mixer(h, layer["mixer"], w, eps)
        else:
            raise ValueError(layer["type"])
        x = x + y
        mlp = layer.get("mlp")
        if mlp is not None:
            h = rms_norm(x, get(prefix + "norm2"), eps)
            w = lambda name: get(prefix + "mlp." + name)
            x = x + (gated_ffn(h, w("gate"), w("up"), w("down"), gelu_tanh) if mlp["kind"] == "dense" else
                     moe_ffn(h, mlp, w))
        streams.append(x)
    return rms_norm(x, get("final.norm"), eps) @ get("head").T, np.stack(streams)
