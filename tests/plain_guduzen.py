"""Plain, slow Guduzen forward pass: whole sequences, no cache, float64 NumPy.

One function per mechanism, written from the design's equations; nothing here
is shared with the engine (it reads a model folder with `json` and the
`safetensors` library and never touches a GPU).  Every engine path of the design
is compared with `forward()`.

Notation: X is the residual [streams, T, width]; a linear weight W is stored
[out, in] and applied as x W^T; positions count from 0.
"""
import json
import math
from pathlib import Path

import numpy as np


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis (eps inside the root)."""
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rmsnorm(x, weight, eps):
    return rms(x, eps) * np.asarray(weight, np.float64)


def rmsnorm_around_zero(x, weight, eps):
    """The RMS norm with weight 1 + w."""
    return rms(x, eps) * (1.0 + np.asarray(weight, np.float64))


def linear(x, w, b=None):
    y = np.asarray(x, np.float64) @ np.asarray(w, np.float64).T
    return y if b is None else y + np.asarray(b, np.float64)


def sigmoid(z):
    z = np.asarray(z, np.float64)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softmax(scores, visible):
    s = np.where(visible, scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


# -- the residual as several streams ------------------------------------------------------------------------------

def spread(x, streams):
    """Every stream starts as the embedding's rows."""
    return np.stack([np.asarray(x, np.float64)] * streams)


def read_streams(X, w_in):
    """u = sum_s in[s] X_s: what a sublayer's norm sees."""
    return np.tensordot(np.asarray(w_in, np.float64), X, axes=(0, 0))


def write_streams(X, mix, w_out, y):
    """X_t <- sum_s mix[s, t] X_s + out[t] y, with the X_s as they were (row s of mix: where X_s goes)."""
    mix, w_out = np.asarray(mix, np.float64), np.asarray(w_out, np.float64)
    return np.stack([sum(mix[s, t] * X[s] for s in range(X.shape[0])) + w_out[t] * y for t in range(X.shape[0])])


# -- attention ----------------------------------------------------------------------------------------------------

def window_visible(T, size):
    """visible[i, j]: 0 <= i - j < size (j <= i without a size)."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = j <= i
    return seen if size is None else seen & (i - j < size)


def attention_kv(h, w, p, m, eps):
    """Keys (normed per head, no weight) and values of an attention layer, [T, kv_heads, dim] and [T, kv_heads, vdim]."""
    T = h.shape[0]
    k = linear(h, w[p + ".k"], w[p + ".k.b"]).reshape(T, m["kv_heads"], m["dim"])
    v = linear(h, w[p + ".v"], w[p + ".v.b"]).reshape(T, m["kv_heads"], m["vdim"])
    return rms(k, eps), v


def attention(h, w, p, m, eps, kv):
    """Grouped-query softmax attention over a sliding window; queries normed per head without a weight; no rotation."""
    T = h.shape[0]
    H, G = m["heads"], m["kv_heads"]
    q = rms(linear(h, w[p + ".q"], w[p + ".q.b"]).reshape(T, H, m["dim"]), eps)
    k, v = kv
    visible = window_visible(T, (m.get("mask") or {}).get("size"))
    out = np.stack([softmax((q[:, a] @ k[:, a // (H // G)].T) * m["scale"], visible) @ v[:, a // (H // G)] for a in range(H)], axis=1)
    return linear(out.reshape(T, H * m["vdim"]), w[p + ".o"])


def latent_attention(h, w, p, m, eps):
    """Softmax attention over every earlier token; keys and values are made from one normed latent a token, queries
    from a normed latent of their own; no positions."""
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = linear(rmsnorm(linear(h, w[p + ".dq"]), w[p + ".dq.norm"], eps), w[p + ".uq"]).reshape(T, H, D)
    c = rmsnorm(linear(h, w[p + ".dkv"]), w[p + ".dkv.norm"], eps)
    k = linear(c, w[p + ".uk"]).reshape(T, H, D)
    v = linear(c, w[p + ".uv"]).reshape(T, H, V)
    visible = window_visible(T, None)
    out = np.stack([softmax((q[:, a] @ k[:, a].T) * m["scale"], visible) @ v[:, a] for a in range(H)], axis=1)
    return linear(out.reshape(T, H * V), w[p + ".o"])


# -- the delta rule with a decay a key channel --------------------------------------------------------------------

def short_conv(x, taps):
    """y[t, c] = silu(sum_j taps[c, j] x[t - (n - 1) + j, c]), x zero at negative times."""
    taps = np.asarray(taps, np.float64)
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
    return silu(sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n)))


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def channel_decay(h, w, p, heads, dim):
    """g [T, heads, dim] = exp(-exp(A_log) softplus(Wa2 Wa1 h + dt_bias))."""
    z = linear(linear(h, w[p + ".a1"]), w[p + ".a2"]) + np.asarray(w[p + ".dt_bias"], np.float64)
    return np.exp(-np.exp(np.asarray(w[p + ".A_log"], np.float64))[None, :, None] * softplus(z.reshape(-1, heads, dim)))


def delta_scan(q, k, v, g, beta):
    """One head: S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  q, k, g [T, dim], v [T, vdim], beta [T]."""
    S = np.zeros((k.shape[1], v.shape[1]))
    out = np.zeros(v.shape)
    for t in range(k.shape[0]):
        S = g[t][:, None] * S
        S = S + np.outer(k[t], beta[t] * (v[t] - k[t] @ S))
        out[t] = q[t] @ S
    return out


def channel_delta(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit(short_conv(linear(h, w[p + ".q"]), w[p + ".q.conv"]).reshape(T, G, D)) * D ** -0.5
    k = unit(short_conv(linear(h, w[p + ".k"]), w[p + ".k.conv"]).reshape(T, G, D))
    v = short_conv(linear(h, w[p + ".v"]), w[p + ".v.conv"]).reshape(T, H, V)
    beta = sigmoid(linear(h, w[p + ".b"]))
    g = channel_decay(h, w, p, H, D)
    out = np.stack([delta_scan(q[:, a // (H // G)], k[:, a // (H // G)], v[:, a], g[:, a], beta[:, a]) for a in range(H)], axis=1)
    gate = sigmoid(linear(linear(h, w[p + ".g1"]), w[p + ".g2"])).reshape(T, H, V)
    return linear((rmsnorm(out, w[p + ".norm"], eps) * gate).reshape(T, H * V), w[p + ".o"])


# -- feed-forward and head ----------------------------------------------------------------------------------------

def gated_ff(h, w, p):
    return linear(gelu_tanh(linear(h, w[p + ".gate"])) * linear(h, w[p + ".up"]), w[p + ".down"])


def capped(logits, cap):
    return cap * np.tanh(logits / cap)


# -- the model ----------------------------------------------------------------------------------------------------

def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of a whole sequence.  `layers_out`: a list that receives the sum of the streams after every layer."""
    eps = cfg["norm"]["eps"]
    X = spread(np.asarray(w["embed"], np.float64)[np.asarray(tokens)], cfg["streams"])
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        h = rmsnorm_around_zero(read_streams(X, w[p + ".hc1.in"]), w[p + ".norm1"], eps)
        if layer["type"] == "attention":
            source = m.get("kv_from")
            if source is None:
                kept[i] = attention_kv(h, w, p + ".mix", m, eps)
            y = attention(h, w, p + ".mix", m, eps, kept[i if source is None else source])
        elif layer["type"] == "latent_attention":
            y = latent_attention(h, w, p + ".mix", m, eps)
        elif layer["type"] == "channel_delta":
            y = channel_delta(h, w, p + ".mix", m, eps)
        else:
            raise ValueError(f"layer type {layer['type']!r}")
        X = write_streams(X, w[p + ".hc1.mix"], w[p + ".hc1.out"], y)
        if layer.get("mlp") is not None:
            h = rmsnorm_around_zero(read_streams(X, w[p + ".hc2.in"]), w[p + ".norm2"], eps)
            X = write_streams(X, w[p + ".hc2.mix"], w[p + ".hc2.out"], gated_ff(h, w, p + ".mlp"))
        if layers_out is not None:
            layers_out.append(X.sum(axis=0))
    x = rmsnorm_around_zero(X.sum(axis=0), w["final.norm"], eps)
    return capped(linear(x, w["embed"]), cfg["logit_softcap"])


def read_folder(folder):
    """(config.json as a dict, {name: float64 array}) of a model folder, read with the safetensors library."""
    import torch
    from safetensors.torch import load_file
    folder = Path(folder)
    cfg = json.loads((folder / "config.json").read_text())
    weights = {k: v.to(torch.float64).numpy() for k, v in load_file(str(folder / "model.safetensors")).items()}
    return cfg, weights


def greedy(cfg, w, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(np.argmax(forward(cfg, w, tokens)[-1])))
    return tokens[len(prompt):]
