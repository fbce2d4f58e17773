"""Tiny Guduzen configurations with weights of the tests' own making, written with the `safetensors` library (not the
engine's writer), and the plain implementation's logits for them.

The configurations differ from each other in every size and constant, and inside each the sizes that could be confused
are unequal: key and value sizes of a head, query and key/value heads, ranks, windows of a layer and of the layers that
read its keys (looking further back and less far than it does itself), the mixers' own head counts.  One has a single
stream, a width that is no multiple of 4, one head, a window of one key, one tap and latents that are no multiple of 8; one is
drawn sharp (scores with a spread of several units, decays close to one); one has twenty heads over four, a latent too
large for the matrix-core kernels and heads of 128 rows of state; one has no window, five streams and several layers
that read one layer's keys.
"""
import json
from pathlib import Path

import numpy as np


def attention(heads, kv_heads, dim, vdim, scale, window=None, kv_from=None, ff=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window is not None:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return layer("attention", m, ff)


def latent(heads, dim, vdim, kv_rank, q_rank, scale, ff=None):
    return layer("latent_attention", {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale}, ff)


def delta(heads, kv_heads, dim, vdim, conv, ff=None):
    return layer("channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, ff)


def layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(vocab, width, streams, cap, eps, layers):
    return {"architecture": "Guduzen", "vocab": vocab, "width": width, "streams": streams, "logit_softcap": cap, "norm": {"eps": eps},
            "layers": layers}


CONFIGS = {
    # a layer's keys read by one that looks back further than it does itself; a delta layer without a feed-forward
    "a": config(131, 64, 2, 8.0, 1e-5, [
        attention(4, 2, 24, 16, 0.3, 20, ff=72), delta(4, 2, 16, 12, 3), attention(4, 2, 24, 16, 0.25, 37, kv_from=0, ff=40),
        latent(3, 20, 24, 40, 28, 0.3, ff=56)]),
    # one stream, a width that is no multiple of 4, one head, one visible key, one tap, latents that are no multiple of 8
    "b": config(77, 50, 1, 5.0, 1e-6, [
        delta(1, 1, 5, 7, 1, ff=20), attention(1, 1, 10, 24, 0.5, 1), latent(1, 6, 10, 13, 9, 0.5, ff=12),
        attention(1, 1, 10, 24, 0.5, 7)]),
    # sharp (the weights' maker reads "sharp"): a window of 48 keys, its keys read over 31, all keys through a latent
    "s": config(97, 48, 3, 10.0, 1e-5, [
        attention(4, 1, 32, 16, 0.4, 48, ff=64), delta(2, 1, 24, 32, 4, ff=40), attention(4, 1, 32, 16, 0.35, 31, kv_from=0),
        latent(2, 16, 24, 48, 32, 0.4, ff=72)]),
    # twenty heads over four, a latent of 288, states of 128 rows, five heads of queries a key head of the rule
    "w": config(211, 96, 4, 30.0, 1e-5, [
        latent(7, 64, 32, 288, 72, 0.125, ff=136), attention(20, 4, 64, 64, 0.125, 100, ff=88), delta(10, 2, 128, 40, 4, ff=64)]),
    # no window, values larger than keys, five streams, one layer's keys read by two others (one of them with a window)
    "n": config(53, 40, 5, 4.0, 1e-5, [
        delta(3, 3, 12, 20, 2), attention(3, 3, 16, 40, 0.25, None, ff=36), attention(6, 3, 16, 40, 0.2, 30, kv_from=1),
        attention(3, 3, 16, 40, 0.3, None, kv_from=1, ff=28)]),
}
SEEDS = {"a": 51, "b": 52, "s": 53, "w": 54, "n": 55}
RANKS = {"a": (10, 6), "b": (3, 5), "s": (8, 12), "w": (40, 136), "n": (16, 7)}      # inner sizes of the decays' and the gates' projections


def tensor_shapes(c, ranks=(16, 24)):
    H, V, S = c["width"], c["vocab"], c["streams"]
    shapes = {"embed": (V, H), "final.norm": (H,)}
    for i, lay in enumerate(c["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        shapes.update({p + "norm1": (H,), p + "hc1.in": (S,), p + "hc1.out": (S,), p + "hc1.mix": (S, S)})
        q, nh, D, Vd = p + "mix.", m["heads"], m["dim"], m["vdim"]
        shapes[q + "o"] = (H, nh * Vd)
        if lay["type"] == "attention":
            shapes.update({q + "q": (nh * D, H), q + "q.b": (nh * D,)})
            if "kv_from" not in m:
                G = m["kv_heads"]
                shapes.update({q + "k": (G * D, H), q + "k.b": (G * D,), q + "v": (G * Vd, H), q + "v.b": (G * Vd,)})
        elif lay["type"] == "latent_attention":
            r, rq = m["kv_rank"], m["q_rank"]
            shapes.update({q + "dq": (rq, H), q + "dq.norm": (rq,), q + "uq": (nh * D, rq), q + "dkv": (r, H), q + "dkv.norm": (r,),
                           q + "uk": (nh * D, r), q + "uv": (nh * Vd, r)})
        else:
            G, K = m["kv_heads"], m["conv"]
            shapes.update({q + "q": (G * D, H), q + "k": (G * D, H), q + "v": (nh * Vd, H), q + "q.conv": (G * D, K), q + "k.conv": (G * D, K),
                           q + "v.conv": (nh * Vd, K), q + "b": (nh, H), q + "a1": (ranks[0], H), q + "a2": (nh * D, ranks[0]),
                           q + "dt_bias": (nh * D,), q + "A_log": (nh,), q + "g1": (ranks[1], H), q + "g2": (nh * Vd, ranks[1]), q + "norm": (Vd,)})
        if lay["mlp"] is not None:
            F = lay["mlp"]["ff"]
            shapes.update({p + "norm2": (H,), p + "hc2.in": (S,), p + "hc2.out": (S,), p + "hc2.mix": (S, S),
                           p + "mlp.gate": (F, H), p + "mlp.up": (F, H), p + "mlp.down": (H, F)})
    return shapes


def make_weights(c, seed, sharp=False, ranks=(16, 24)):
    """Matrices N(0, 1/in), biases N(0, 0.3), norms that add one to their weight N(0, 0.2), the other norms 1 + N(0, 0.1), streams read
    with 1/s + N(0, 0.2), written with 1 + N(0, 0.2) and mixed with 0.8 I + N(0, 0.09/s), convolutions N(0, 1/taps), A_log N(-1, 1), dt_bias
    N(-1, 1), embedding rows N(0, 16/width).  `sharp`: the query latents' norms times 2.5 (a query's result hangs on single keys),
    A_log N(-5, 0.5) (the state keeps the first tokens)."""
    import torch
    rng = np.random.default_rng(seed)
    out, S = {}, c["streams"]
    for name, shape in sorted(tensor_shapes(c, ranks).items()):
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            w = 0.2 * rng.standard_normal(shape)
        elif last == "norm":
            w = 1.0 + 0.1 * rng.standard_normal(shape)
            if sharp and name.endswith("dq.norm"):
                w = 2.5 * w
        elif last == "in":
            w = 1.0 / S + 0.2 * rng.standard_normal(shape)
        elif last == "out":
            w = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "mix":
            w = 0.8 * np.eye(S) + 0.3 * rng.standard_normal(shape) / np.sqrt(S)
        elif last == "b" and len(shape) == 1:
            w = 0.3 * rng.standard_normal(shape)
        elif last == "A_log":
            w = (-5.0 if sharp else -1.0) + (0.5 if sharp else 1.0) * rng.standard_normal(shape)
        elif last == "dt_bias":
            w = -1.0 + rng.standard_normal(shape)
        elif name == "embed":
            w = 4.0 * rng.standard_normal(shape) / np.sqrt(shape[-1])
        else:
            w = rng.standard_normal(shape) / np.sqrt(shape[-1])
        out[name] = torch.from_numpy(np.asarray(w, np.float32)).to(torch.bfloat16)
    return out


def write_folder(folder, c, seed, sharp=False, ranks=(16, 24)):
    from safetensors.torch import save_file
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(c))
    save_file(make_weights(c, seed, sharp, ranks), str(folder / "model.safetensors"))
    return folder


_PLAIN = {}


def plain_logits(folder, tokens):
    """float64 logits [T, V] of the plain implementation, cached per (folder, tokens)."""
    import plain_guduzen
    key = (str(folder), tuple(tokens))
    if key not in _PLAIN:
        cfg, w = _PLAIN.setdefault(("folder", str(folder)), plain_guduzen.read_folder(folder))
        _PLAIN[key] = plain_guduzen.forward(cfg, w, list(tokens))
    return _PLAIN[key]
