"""The Movazen decoder as a list of parts chosen by MovazenConfig, layer by layer: an embedding that is scaled and has a
sinusoidal vector of the position added; layers that norm before their sublayers (weights stored around zero) and add the
results as they are, then a third sublayer that reads a table by the token and whose result is normed; an "attention" layer
mixes with softmax attention over a window that keeps the first keys, its scores falling with the distance (queries and
keys normed per head, a gate an element); a "parallel" layer with a_left left + a_right right: softmax attention over every
earlier key with one in the denominator and a query temperature beside lightning attention; feed-forwards are mixtures of
clamped gated experts routed by sigmoid scores.  Tensor names: `embed`, `side.embed`, `l<i>.norm1|norm2`, `l<i>.mix.*`,
`l<i>.mix.left.*`, `l<i>.mix.right.*`, `l<i>.mlp.router|correction|e<j>.gate|up|down|shared.gate|up|down|sg`,
`l<i>.side.gate|proj|norm`, `final.norm`, `head`.
"""
from ..config.base import register_architecture
from ..config.movazen import MovazenConfig
from ..parts import make_part, distance_slopes, LMHead, SinusoidEmbedding
from .model import Model

SINK = 0.0               # the score that joins the denominator on the left of a parallel layer: one is added to it
WEIGHT_FLOOR = 1e-20     # added to the sum of the chosen scores before they are divided by it
SLOPE, SHIFT = 1.702, 1.0        # of the experts' gate


def build_movazen(config):
    c = config
    H, eps = c.width, c.norm_eps

    def norm(tensor):
        return make_part("norm", "rmsnorm", name=tensor, dim=H, eps=eps, tensor=tensor, around_zero=True)

    embedding = SinusoidEmbedding("embed", c.vocab, H, scale=c.embedding_scale, tensor="embed", side=("side.embed", len(c.layers) * c.side_dim))
    layers = []
    for i, spec in enumerate(c.layers):
        p = f"l{i}"
        if spec.type == "attention":
            a = spec.mixer
            mixer = make_part("mixer", "normed_gated_attention", name=p + ".mix", hidden=H, heads=a.heads, kv_heads=a.kv_heads, dim=a.dim,
                              vdim=a.vdim, scale=a.scale, eps=eps, head_gate="element", window=a.window, float_rows=True,
                              slopes=distance_slopes(a.heads), keep_first=a.keep_first)
        else:
            a, r = spec.mixer.left, spec.mixer.right
            left = make_part("mixer", "normed_gated_attention", name=p + ".mix.left", hidden=H, heads=a.heads, kv_heads=a.kv_heads, dim=a.dim,
                             vdim=a.vdim, scale=a.scale, eps=eps, qk_norm=False, head_gate=False, bias=True, sink=[SINK] * a.heads,
                             q_temp=a.q_temp)
            right = make_part("mixer", "lightning_attention", name=p + ".mix.right", hidden=H, heads=r.heads, dim=r.dim, vdim=r.vdim,
                              decay=r.decay, eps=eps)
            mixer = make_part("mixer", "side_by_side", name=p + ".mix", hidden=H, first=left, second=right, eps=eps,
                              scales=(spec.mixer.left_scale, spec.mixer.right_scale))
        ffn = {}
        m = spec.mlp
        if m is not None:
            shared = None
            if m.shared is not None:
                shared = make_part("ffn", "clamped_glu", name=p + ".mlp.shared", hidden=H, intermediate=m.shared[0], limit=m.shared[1],
                                   slope=SLOPE, shift=SHIFT)
            ffn = dict(ffn_norm=norm(p + ".norm2"),
                       ffn=make_part("ffn", "scored_experts", name=p + ".mlp", hidden=H, intermediate=m.ff, experts=m.experts, top=m.top,
                                     groups=m.groups, shared=shared, scores="sigmoid", group_pairs=True, floor=WEIGHT_FLOOR,
                                     law=(m.limit, SLOPE, SHIFT), shared_gate=None if shared is None else "shared.sg"))
        side = make_part("ffn", "token_side", name=p + ".side", hidden=H, width=c.side_dim, first=i * c.side_dim, source=embedding)
        side_post = make_part("norm", "rmsnorm", name=p + ".side.norm", dim=H, eps=eps, tensor=p + ".side.norm")
        layers.append(make_part("block", "sandwich", mixer_norm=norm(p + ".norm1"), mixer=mixer, mixer_post=None, side=side,
                                side_post=side_post, **ffn))
    head = LMHead("head", c.vocab, H, tensor="head")
    return Model(c, embedding, layers, norm("final.norm"), head, max_positions=c.max_positions, vocab_size=c.vocab)


register_architecture(["Movazen", "movazen"], MovazenConfig, build_movazen)
