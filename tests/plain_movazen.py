"""Plain, slow Movazen forward pass: whole sequences, no cache, float64 NumPy.

One function per mechanism, written from the design's equations; nothing here
is shared with the engine (it reads a model folder with `json` and the
`safetensors` library and never touches a GPU).  Every engine path of the design
is compared with `forward()`.

Notation: x is the residual stream [T, width]; a linear weight W is stored
[out, in] and applied as x W^T; positions count from 0.
"""
import json
import math
from pathlib import Path

import numpy as np

SLOPE, SHIFT = 1.702, 1.0        # of the experts' gate


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis (eps inside the root)."""
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def linear(x, w, b=None):
    y = np.asarray(x, np.float64) @ np.asarray(w, np.float64).T
    return y if b is None else y + np.asarray(b, np.float64)


def sigmoid(z):
    z = np.asarray(z, np.float64)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    z = np.asarray(z, np.float64)
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# -- embedding ----------------------------------------------------------------------------------------------------

def sinusoids(positions, width, base=10000.0):
    """[T, width]: columns 2i and 2i + 1 are sine and cosine of position * base^(-2i / width)."""
    out = np.zeros((len(positions), width))
    for d in range(width):
        angle = np.asarray(positions, np.float64) * base ** (-2.0 * (d // 2) / width)
        out[:, d] = np.cos(angle) if d % 2 else np.sin(angle)
    return out


# -- attention ----------------------------------------------------------------------------------------------------

def visible(T, size=None, keep=0):
    """seen[i, j]: j <= i and (fewer than `size` behind, or one of the first `keep`); all j <= i without a size."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = j <= i
    return seen if size is None else seen & ((i - j < size) | (j < keep))


def head_slopes(heads):
    return 2.0 ** (-8.0 * (np.arange(heads) + 1) / heads)


def temperature(positions, coef, every):
    """What the query at a position is multiplied by."""
    return 1.0 + coef * np.log(np.floor((np.asarray(positions, np.float64) + 1.0) / every) + 1.0)


def softmax_heads(q, k, v, scale, seen, slopes=None, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V].  `slopes` [H]: slope * (i - j) is taken off a score; `sink`: a
    score that joins every denominator and has no value."""
    T, H, _ = q.shape
    G = k.shape[1]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = q[:, h] @ k[:, g].T * scale
        if slopes is not None:
            s = s - slopes[h] * (i - j)
        s = np.where(seen, s, -np.inf)
        top = s.max(axis=1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink)
        e = np.exp(s - top)
        den = e.sum(axis=1, keepdims=True) + (0.0 if sink is None else np.exp(sink - top))
        out[:, h] = (e / den) @ v[:, g]
    return out


def window_attention(h, w, p, m, eps):
    """Queries and keys normed per head, scores that fall with the distance, a window with kept first tokens, and a gate
    element by element."""
    T, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms(linear(h, w[p + ".q"]).reshape(T, H, D), eps) * w[p + ".q.norm"]
    k = rms(linear(h, w[p + ".k"]).reshape(T, G, D), eps) * w[p + ".k.norm"]
    v = linear(h, w[p + ".v"]).reshape(T, G, V)
    mask = m.get("mask") or {}
    seen = visible(T, mask.get("size"), mask.get("keep_first", 0))
    out = softmax_heads(q, k, v, m["scale"], seen, slopes=head_slopes(H)).reshape(T, H * V)
    return linear(out * sigmoid(linear(h, w[p + ".g"])), w[p + ".o"])


def sink_attention(h, w, p, m):
    """Biased projections, a query temperature that grows with the position, every earlier key, one in the denominator."""
    T, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(h, w[p + ".q"], w[p + ".q.b"]).reshape(T, H, D)
    k = linear(h, w[p + ".k"], w[p + ".k.b"]).reshape(T, G, D)
    v = linear(h, w[p + ".v"], w[p + ".v.b"]).reshape(T, G, V)
    if m.get("q_temp"):
        q = q * temperature(np.arange(T), m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    return linear(softmax_heads(q, k, v, m["scale"], visible(T), sink=0.0).reshape(T, H * V), w[p + ".o"])


# -- lightning attention ------------------------------------------------------------------------------------------

def decayed_memory(q, k, v, decay, state=None):
    """S <- decay S + k v^T; o = S^T q, one head: q, k [T, D], v [T, V].  Returns (o [T, V], S)."""
    S = np.zeros((k.shape[1], v.shape[1])) if state is None else np.array(state, np.float64)
    out = np.zeros((len(q), v.shape[1]))
    for t in range(len(q)):
        S = decay * S + np.outer(k[t], v[t])
        out[t] = q[t] @ S
    return out, S


def lightning_attention(h, w, p, m, eps):
    T, H, D, V = len(h), m["heads"], m["dim"], m["vdim"]
    q, k = (silu(linear(h, w[f"{p}.{n}"])).reshape(T, H, D) for n in ("q", "k"))
    v = silu(linear(h, w[p + ".v"])).reshape(T, H, V)
    o = np.stack([decayed_memory(q[:, i], k[:, i], v[:, i], m["decay"][i])[0] for i in range(H)], axis=1).reshape(T, H * V)
    o = rms(o, eps) * w[p + ".norm"]
    return linear(o * sigmoid(linear(h, w[p + ".g"])), w[p + ".o"])


def mixer(h, w, p, layer, eps):
    m = layer["mixer"]
    if layer["type"] == "attention":
        return window_attention(h, w, p, m, eps)
    return (m["left_scale"] * sink_attention(h, w, p + ".left", m["left"])
            + m["right_scale"] * lightning_attention(h, w, p + ".right", m["right"], eps))


# -- feed-forward -------------------------------------------------------------------------------------------------

def clamped_expert(h, w, p, limit):
    g = np.minimum(linear(h, w[p + ".gate"]), limit)
    u = np.clip(linear(h, w[p + ".up"]), -limit, limit)
    return linear(g * sigmoid(SLOPE * g) * (u + SHIFT), w[p + ".down"])


def route(z, correction, top, groups=None):
    """Router logits [T, E] -> (chosen [T, top], weights [T, top], margin [T]: how far the nearest decision is from turning
    round, in scores)."""
    s = sigmoid(z)
    c = s + np.asarray(correction, np.float64)
    T, E = z.shape
    chosen, weights, margin = np.zeros((T, top), int), np.zeros((T, top)), np.full(T, np.inf)
    for t in range(T):
        scores = c[t].copy()
        if groups is not None:
            count, keep = groups["count"], groups["keep"]
            best = np.array([np.sort(part)[::-1][:2].sum() for part in scores.reshape(count, E // count)])
            order = np.argsort(-best, kind="stable")
            if keep < count:
                margin[t] = min(margin[t], best[order[keep - 1]] - best[order[keep]])
            for g in order[keep:]:
                scores[g * (E // count):(g + 1) * (E // count)] = -np.inf
        order = np.argsort(-scores, kind="stable")
        chosen[t] = order[:top]
        if top < E:
            margin[t] = min(margin[t], scores[order[top - 1]] - scores[order[top]])
        weights[t] = s[t, chosen[t]] / (s[t, chosen[t]].sum() + 1e-20)
    return chosen, weights, margin


def mixture(h, w, p, m, margins=None):
    r = m["router"]
    chosen, weights, margin = route(linear(h, w[p + ".router"]), w[p + ".correction"], r["top"], r.get("groups"))
    if margins is not None:
        margins.append(margin)
    out = np.zeros_like(np.asarray(h, np.float64))
    for e in range(r["experts"]):
        rows, place = np.nonzero(chosen == e)
        if len(rows):
            out[rows] += weights[rows, place][:, None] * clamped_expert(h[rows], w, f"{p}.e{e}", m["expert"]["limit"])
    if m.get("shared"):
        q = p + ".shared"
        out = out + sigmoid(linear(h, w[q + ".sg"])) * clamped_expert(h, w, q, m["shared"]["limit"])
    return out


# -- the whole ----------------------------------------------------------------------------------------------------

def token_side(x, tokens, w, p, i, dim, eps, margins=None):
    """The part of a token's row that belongs to layer i, gated by the stream, projected, normed.  `margins` (a list)
    receives how small the gate leaves a row, times 0.4: what is nearly gated away and then normed is mostly rounding."""
    e = np.asarray(w["side.embed"], np.float64)[tokens, i * dim:(i + 1) * dim]
    z = linear(x, w[p + ".side.gate"])
    if margins is not None:
        size = lambda a: np.sqrt(np.mean(a * a, axis=-1))
        margins.append(0.4 * size(gelu_tanh(z) * e) / np.maximum(size(z * e), 1e-300))
    y = linear(gelu_tanh(z) * e, w[p + ".side.proj"])
    return rms(y, eps) * w[p + ".side.norm"]


def read_folder(folder):
    """(config, {tensor name: float64 array}) of a model folder."""
    from safetensors.torch import load_file
    import torch
    config = json.loads((Path(folder) / "config.json").read_text())
    return config, {k: t.to(torch.float64).numpy() for k, t in load_file(str(Path(folder) / "model.safetensors")).items()}


def forward(config, w, tokens, layers_out=None, margins=None):
    """Logits [T, vocab] of one sequence; `layers_out` (a list) receives the residual stream after every layer, `margins`
    (a list) how far every router's decisions are from turning round and how much of a row its side gates leave."""
    tokens = np.asarray(tokens, int)
    eps = config["norm"]["eps"]
    x = np.asarray(w["embed"], np.float64)[tokens] * config["embedding"]["scale"] + sinusoids(np.arange(len(tokens)), config["width"])
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}"
        x = x + mixer(rms(x, eps) * (1.0 + w[p + ".norm1"]), w, p + ".mix", layer, eps)
        if layer.get("mlp"):
            x = x + mixture(rms(x, eps) * (1.0 + w[p + ".norm2"]), w, p + ".mlp", layer["mlp"], margins)
        x = x + token_side(x, tokens, w, p, i, config["token_side"]["dim"], eps, margins)
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(rms(x, eps) * (1.0 + w["final.norm"]), w["head"])


def greedy(config, w, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(np.argmax(forward(config, w, tokens)[-1])))
    return tokens[len(prompt):]
