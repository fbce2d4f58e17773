"""Tiny Movazen configurations with weights of the tests' own making, written with the `safetensors` library (not the
engine's writer), and the plain implementation's logits for them.

The configurations differ from each other in every size and constant, and inside each the sizes that could be confused
are unequal: key and value sizes of a head, query and key/value heads, heads of the two mixers of a layer, windows and
kept keys of neighbouring layers, experts, chosen experts and groups, an expert's and the shared expert's size and limit.
One has a width that is no multiple of 4 and odd sizes, one head, a window of one key, no kept keys, one group, every
expert chosen and no shared expert; one is drawn sharp (scores with a spread of several units, a decay close to one); one
has twenty heads over four and sixteen experts in four groups; one has no window at all, no query temperature, as many
key/value heads as query heads, groups of one expert, and layers without a feed-forward.
"""
import json
from pathlib import Path

import numpy as np


def attention(heads, kv_heads, dim, vdim, scale, mask=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if mask is not None:
        m["mask"] = {"size": mask[0], "keep_first": mask[1]}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def parallel(left, right, left_scale, right_scale, mlp=None):
    """left = (heads, kv_heads, dim, vdim, scale, (coef, every) or None), right = (heads, dim, vdim, decays)."""
    l = dict(zip(("heads", "kv_heads", "dim", "vdim", "scale"), left))
    if left[5] is not None:
        l["q_temp"] = {"coef": left[5][0], "every": left[5][1]}
    r = dict(zip(("heads", "dim", "vdim"), right)) | {"decay": list(right[3])}
    return {"type": "parallel", "mixer": {"left": l, "right": r, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def moe(ff, limit, experts, top, groups=None, shared=None):
    router = {"experts": experts, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def config(vocab, width, scale, eps, side, layers):
    return {"architecture": "Movazen", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
            "token_side": {"dim": side}, "layers": layers}


CONFIGS = {
    # two windows with different numbers of kept keys (two groups of pages beside the one that keeps everything)
    "a": config(131, 64, 0.7, 1e-5, 12, [
        attention(4, 2, 24, 16, 0.3, (21, 6), moe(24, 1.5, 6, 3, (3, 2), (40, 0.8))),
        parallel((4, 1, 16, 24, 0.3, (0.4, 16)), (2, 12, 20, (0.9, 0.99)), 1.1, 0.7, moe(20, 2.5, 8, 2, (2, 1), (12, 3.0))),
        attention(4, 2, 24, 16, 0.25, (37, 17)),
        parallel((2, 2, 8, 32, 0.4, (0.1, 50)), (3, 16, 8, (0.5, 0.95, 0.999)), 0.6, 1.3)]),
    # odd sizes and ones
    "b": config(77, 90, 1.0, 1e-6, 5, [
        attention(1, 1, 10, 23, 0.5, (1, 0), moe(11, 1.0, 3, 3)),
        parallel((1, 1, 9, 14, 0.5, (0.3, 1)), (1, 5, 7, (0.8,)), 0.5, 2.0, moe(13, 0.7, 2, 1, (1, 1), (9, 1.1))),
        attention(1, 1, 13, 7, 0.4, (1, 3), moe(8, 2.0, 2, 2, None, (17, 0.5)))]),
    # sharp: a window and kept keys around the page size, far keys, old state
    "s": config(97, 48, 0.6, 1e-5, 8, [
        attention(4, 1, 32, 16, 0.35, (48, 18), moe(32, 3.0, 4, 2, (2, 1), (16, 2.0))),
        parallel((2, 1, 16, 16, 0.4, (0.5, 32)), (2, 16, 16, (0.97, 0.9995)), 1.2, 0.5, moe(24, 2.0, 6, 2, (3, 2), (32, 1.5)))]),
    # twenty heads over four, heads of one size, sixteen experts in four groups
    "w": config(211, 96, 0.9, 1e-5, 32, [
        parallel((20, 4, 64, 64, 0.125, (0.2, 40)), (8, 32, 32, [1.0 - 2.0 ** -(i + 1) for i in range(8)]), 1.0, 1.0, moe(48, 4.0, 16, 4, (4, 2), (40, 5.0))),
        attention(20, 4, 64, 64, 0.125, (100, 33), moe(40, 4.0, 16, 5, (4, 3), (48, 2.0)))]),
    # no window, no temperature, groups of one expert, layers without a feed-forward, values larger than keys
    "n": config(53, 40, 1.3, 1e-5, 10, [
        attention(3, 3, 16, 40, 0.25), parallel((3, 3, 12, 20, 0.3, None), (2, 12, 20, (0.7, 0.98)), 0.8, 1.2, moe(16, 1.2, 4, 2, (4, 3), None)),
        attention(6, 3, 16, 40, 0.2, (30, 0)), attention(3, 3, 16, 40, 0.3, None, moe(28, 9.0, 5, 1, None, (20, 0.9)))]),
}
SEEDS = {"a": 61, "b": 62, "s": 63, "w": 64, "n": 65}


def tensor_shapes(c):
    H, V, side = c["width"], c["vocab"], c["token_side"]["dim"]
    shapes = {"embed": (V, H), "head": (V, H), "final.norm": (H,), "side.embed": (V, side * len(c["layers"]))}
    for i, lay in enumerate(c["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        shapes.update({p + "norm1": (H,), p + "side.gate": (side, H), p + "side.proj": (H, side), p + "side.norm": (H,)})
        q = p + "mix."
        if lay["type"] == "attention":
            nh, G, D, Vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            shapes.update({q + "q": (nh * D, H), q + "k": (G * D, H), q + "v": (G * Vd, H), q + "q.norm": (D,), q + "k.norm": (D,),
                           q + "g": (nh * Vd, H), q + "o": (H, nh * Vd)})
        else:
            l, r = m["left"], m["right"]
            nh, G, D, Vd = l["heads"], l["kv_heads"], l["dim"], l["vdim"]
            shapes.update({q + "left.q": (nh * D, H), q + "left.q.b": (nh * D,), q + "left.k": (G * D, H), q + "left.k.b": (G * D,),
                           q + "left.v": (G * Vd, H), q + "left.v.b": (G * Vd,), q + "left.o": (H, nh * Vd)})
            K, W = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            shapes.update({q + "right.q": (K, H), q + "right.k": (K, H), q + "right.v": (W, H), q + "right.g": (W, H), q + "right.o": (H, W),
                           q + "right.norm": (W,)})
        if lay["mlp"] is None:
            continue
        e, r = lay["mlp"]["expert"], lay["mlp"]["router"]
        q = p + "mlp."
        shapes.update({p + "norm2": (H,), q + "router": (r["experts"], H), q + "correction": (r["experts"],)})
        for j in range(r["experts"]):
            shapes.update({f"{q}e{j}.gate": (e["ff"], H), f"{q}e{j}.up": (e["ff"], H), f"{q}e{j}.down": (H, e["ff"])})
        if "shared" in lay["mlp"]:
            F = lay["mlp"]["shared"]["ff"]
            shapes.update({q + "shared.gate": (F, H), q + "shared.up": (F, H), q + "shared.down": (H, F), q + "shared.sg": (1, H)})
    return shapes


def make_weights(c, seed, sharp=False):
    """Matrices N(0, 1/in), norms that add one to their weight N(0, 0.2), the other norms 1 + N(0, 0.1), biases N(0, 0.3),
    routers N(0, 4/in), corrections N(0, 0.1), both tables of the tokens N(0, 1), lightning keys N(0, 4/in).
    `sharp`: the query norms' weights times 4 and the left queries times 3 (scores with a spread of several units: a
    query's result hangs on single keys)."""
    import torch
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in sorted(tensor_shapes(c).items()):
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            w = 0.2 * rng.standard_normal(shape)
        elif last == "norm":
            w = 1.0 + 0.1 * rng.standard_normal(shape)
            if sharp and name.endswith("q.norm"):
                w = 4.0 * w
        elif last == "b":
            w = 0.3 * rng.standard_normal(shape)
        elif last == "correction":
            w = 0.1 * rng.standard_normal(shape)
        elif name in ("embed", "side.embed"):
            w = rng.standard_normal(shape)
        else:
            w = rng.standard_normal(shape) / np.sqrt(shape[-1])
            if last == "router" or name.endswith("right.k"):
                w = 2.0 * w
            if sharp and name.endswith("left.q"):
                w = 3.0 * w
        out[name] = torch.from_numpy(np.asarray(w, np.float32)).to(torch.bfloat16)
    return out


def write_folder(folder, c, seed, sharp=False):
    from safetensors.torch import save_file
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(c))
    save_file(make_weights(c, seed, sharp), str(folder / "model.safetensors"))
    return folder


_PLAIN = {}
CLOSE_CALL = 0.02     # a router's margin (in scores) that bfloat16 rounding may turn round


def _plain(folder, tokens):
    import plain_movazen
    key = (str(folder), tuple(tokens))
    if key not in _PLAIN:
        cfg, w = _PLAIN.setdefault(("folder", str(folder)), plain_movazen.read_folder(folder))
        margins = []
        logits = plain_movazen.forward(cfg, w, list(tokens), margins=margins)
        _PLAIN[key] = (logits, np.min(margins, axis=0) if margins else np.full(len(tokens), np.inf))
    return _PLAIN[key]


def plain_logits(folder, tokens):
    """float64 logits [T, V] of the plain implementation, cached per (folder, tokens)."""
    return _plain(folder, tokens)[0]


def decided_rows(folder, tokens):
    """Which positions of a sequence have no close call of their own: True where every router's margin is at least
    CLOSE_CALL and no side's gate leaves next to nothing of a row (which the norm behind it would blow up, rounding and
    all).  In bfloat16 a narrower margin may choose another expert than the float64 implementation does, which is no
    fault; such a position is compared in float32 only."""
    return _plain(folder, tokens)[1] >= CLOSE_CALL


def decisive_tokens(folder, seed, n, vocab, margin=2 * CLOSE_CALL, tries=200):
    """`n` token ids drawn from `seed` at none of whose positions the plain model's margins are under `margin`: positions at
    which they are get other tokens until none is left."""
    kept = _PLAIN.get(("tokens", str(folder), seed, n, margin))
    if kept is not None:
        return list(kept)
    rng = np.random.default_rng(seed)
    tokens = [int(t) for t in rng.integers(0, vocab, n)]
    for _ in range(tries):
        close = np.nonzero(_plain(folder, tokens)[1] < margin)[0]
        if not len(close):
            _PLAIN[("tokens", str(folder), seed, n, margin)] = list(tokens)
            return tokens
        _PLAIN.pop((str(folder), tuple(tokens)), None)
        for at in close:
            tokens[int(at)] = int(rng.integers(0, vocab))
    raise AssertionError(f"no sequence of {n} tokens without a close call after {tries} tries")
