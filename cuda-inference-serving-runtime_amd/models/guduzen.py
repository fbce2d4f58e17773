"""The Guduzen decoder as a list of parts chosen by GuduzenConfig, layer by layer: a residual of several streams with
weights that read, mix and write them around every sublayer (hyper-connections); RMS norms whose weights are stored
around zero; a mixer that is softmax attention over a sliding window without positions (queries and keys normed per head
without a weight, biases; optionally reading the keys and values of an earlier layer), latent attention without
positions over every earlier token, or the gated delta rule with a decay a key channel; feed-forwards gated by the tanh
form of gelu; the logits are the embedding table times the normed sum of the streams, capped.  Tensor names: `embed`,
`l<i>.norm1|norm2`, `l<i>.hc1|hc2.in|out|mix`, `l<i>.mix.*`, `l<i>.mlp.gate|up|down`, `final.norm`.
"""
from ..config.base import register_architecture
from ..config.guduzen import GuduzenConfig
from ..parts import make_part, LMHead, StreamsEmbedding
from .model import Model, ScheduleEntry


def build_guduzen(config):
    c = config
    H, S, eps = c.width, c.streams, c.norm_eps

    def norm(tensor, reads=None):
        return make_part("norm", "streams_norm", name=tensor, dim=H, eps=eps, streams=S, reads=reads, tensor=tensor, around_zero=True)

    # a layer whose keys others read keeps as many as the one of them that looks back furthest
    windows = {}
    for i, spec in enumerate(c.layers):
        if spec.attention is not None:
            a = spec.attention
            windows.setdefault(i if a.kv_from is None else a.kv_from, []).append(a.window)
    keep = {i: None if None in seen else max(seen) for i, seen in windows.items()}

    layers, schedule = [], []
    for i, spec in enumerate(c.layers):
        p, m, reads = f"l{i}", spec.mixer, None
        common = dict(name=p + ".mix", hidden=H, heads=m.heads, dim=m.dim, vdim=m.vdim, eps=eps)
        if spec.type == "attention":
            reads, own = m.kv_from, m.kv_from is None
            mixer = make_part("mixer", "normed_gated_attention", kv_heads=m.kv_heads, scale=m.scale, qk_norm="plain", head_gate=False,
                              window=m.window, bias=True, own_kv=own, keep=keep[i] if own else "own", **common)
        elif spec.type == "latent_attention":
            from ..weights.loader import AnySize
            mixer = make_part("mixer", "latent_attention", rot_dim=0, kv_rank=m.kv_rank, scale=m.scale, position=None, head_gate=False,
                              q_rank=m.q_rank if m.q_rank is not None else AnySize(max(8, H // 2)), **common)
        else:
            mixer = make_part("mixer", "channel_delta_rule", kv_heads=m.kv_heads, taps=m.conv, **common)
        ffn = {}
        if spec.ff is not None:
            ffn = dict(ffn_norm=norm(p + ".norm2", p + ".hc2.in"),
                       ffn=make_part("ffn", "gated_mlp", name=p + ".mlp", hidden=H, intermediate=spec.ff, activation="gelu_tanh",
                                     names=("gate", "up", "down")))
        layers.append(make_part("block", "hyper_connected", name=p, streams=S, mixer_norm=norm(p + ".norm1", p + ".hc1.in"), mixer=mixer, **ffn))
        schedule.append(ScheduleEntry(i, reads=reads))
    embedding = StreamsEmbedding("embed", c.vocab, H, S, tensor="embed")
    head = LMHead("head", c.vocab, H, tied_to=embedding, softcap=c.logit_softcap)
    return Model(c, embedding, layers, norm("final.norm"), head, schedule=schedule, max_positions=c.max_positions, vocab_size=c.vocab)


register_architecture(["Guduzen", "guduzen"], GuduzenConfig, build_guduzen)
