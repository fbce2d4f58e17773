"""Token embedding and output head.

x0[r] = E[token_r] with no scaling (reference: runtime/model.py:105), or with PairHashEmbedding
E[token_r] * scale + B[hash(token before, token_r)], with SinusoidEmbedding E[token_r] * scale + a vector of the position; logits =
h . W^T with W the head's own matrix or, when tied, the embedding matrix
(reference: runtime/checkpoint.py:38-39).  Logits are always float.
"""
import math

import torch

from ..kernels import ops
from .base import Part, TensorSpec, matrix_operand


class TokenEmbedding(Part):
    def __init__(self, name, vocab, hidden, tensor=None):
        """`tensor`: the table's full name where it is not `<name>.weight`."""
        self.name, self.vocab, self.hidden = name, vocab, hidden
        self.tensor = tensor if tensor is not None else name + ".weight"
        self.weight = None

    def tensor_specs(self):
        return [TensorSpec(self.tensor, (self.vocab, self.hidden))]

    def bind(self, tensors, dtype):
        self.weight = matrix_operand(tensors[self.tensor], dtype)

    def forward(self, ctx):
        out = ctx.buffer("residual", (ctx.tokens.shape[0], self.hidden), torch.float32)
        return ops.embedding(ctx.tokens, self.weight, out)


class StreamsEmbedding(TokenEmbedding):
    """The embedding of a model whose residual is `streams` streams: every stream of a row starts as the token's row, and
    the first sublayer's read of them (a norm that says `reads_streams`) is made on the way."""

    def __init__(self, name, vocab, hidden, streams, tensor=None):
        super().__init__(name, vocab, hidden, tensor=tensor)
        self.streams = int(streams)

    def forward(self, ctx):
        T = ctx.tokens.shape[0]
        x = ctx.buffer("residual", (T, self.streams * self.hidden), torch.float32)
        reader = ctx.next_norm
        read = reader.read_args(T, ctx) if getattr(reader, "reads_streams", None) == self.streams else None
        ops.streams_embed(ctx.tokens, self.weight, x, self.streams, read=read)
        if read is not None:
            ctx.leave_normed(reader, x, read[3])
        return x


class SinusoidEmbedding(TokenEmbedding):
    """x[r] = E[token_r] * scale + a vector of the position, sines in its even columns and cosines in its odd ones: entries
    2i and 2i + 1 turn by base^(-2i / hidden) a position.  The norm that reads the rows first is made by the same kernel.
    `side` = (tensor name, columns): a second table of the tokens, in the activations' type, that layers read (TokenSide);
    it is this part's tensor and is found as `side_table`."""

    def __init__(self, name, vocab, hidden, scale=1.0, base=10000.0, tensor=None, side=None):
        super().__init__(name, vocab, hidden, tensor=tensor)
        self.scale, self.base, self.side, self.side_table = float(scale), float(base), side, None

    def tensor_specs(self):
        return super().tensor_specs() + ([] if self.side is None else [TensorSpec(self.side[0], (self.vocab, self.side[1]))])

    def bind(self, tensors, dtype):
        super().bind(tensors, dtype)
        if self.side is not None:
            self.side_table = matrix_operand(tensors[self.side[0]], dtype)

    def prepare(self, device, dtype):
        pairs = torch.arange((self.hidden + 1) // 2, dtype=torch.float64)
        self.turns = (self.base ** (-2.0 * pairs / self.hidden) / (2.0 * math.pi)).to(device)

    def forward(self, ctx):
        T = ctx.tokens.shape[0]
        out = ctx.buffer("residual", (T, self.hidden), torch.float32)
        norm, reader = None, ctx.next_norm
        if getattr(reader, "fusable_as", None) == "rms":
            norm = (reader.weight, reader.eps, ctx.buffer("residual.normed", (T, self.hidden), ctx.dtype))
        ops.embedding_sinusoid(ctx.tokens, ctx.positions, self.weight, self.turns, out, scale=self.scale, norm=norm)
        if norm is not None:
            ctx.leave_normed(reader, out, norm[2])
        return out


STATE_SITE = "embedding"      # the key of the embedding's state among the cache manager's state sites


class PairHashEmbedding(TokenEmbedding):
    """x[r] = E[token_r] * scale + B[(token before * mul_prev + token_r * mul_cur) mod buckets], B a second table of
    `buckets` + 1 rows whose last row serves a sequence's first token (`buckets` None: no second table, only the scale).
    The token before a portion's first one is the last token of the request's step before: part of the request's state,
    one int32 in its state slot, written on the device (so a token that was picked on the device and has not reached
    the host yet serves as well).  The rows are also left in the activations' type for a layer whose sublayers read
    the stream itself (parts.base.CAST)."""

    def __init__(self, name, vocab, hidden, scale=1.0, buckets=None, mul_prev=0, mul_cur=0, tensor=None, pairs_tensor=None):
        super().__init__(name, vocab, hidden, tensor=tensor)
        if buckets is not None and (buckets <= 0 or mul_prev < 0 or mul_cur < 0):
            raise ValueError("a table of token pairs needs a positive number of buckets and multipliers >= 0")
        self.scale, self.buckets, self.mul_prev, self.mul_cur = float(scale), buckets, int(mul_prev), int(mul_cur)
        self.pairs_tensor = pairs_tensor if pairs_tensor is not None else name + ".pairs"
        self.pairs = None

    def tensor_specs(self):
        specs = super().tensor_specs()
        if self.buckets is not None:
            specs.append(TensorSpec(self.pairs_tensor, (self.buckets + 1, self.hidden)))
        return specs

    def bind(self, tensors, dtype):
        super().bind(tensors, dtype)
        if self.buckets is not None:
            self.pairs = matrix_operand(tensors[self.pairs_tensor], dtype)

    def state_need(self):
        from ..cache.pages import StateNeed
        return StateNeed((1,), "int32") if self.buckets is not None else None

    def forward(self, ctx):
        from .base import CAST
        T = ctx.tokens.shape[0]
        out = ctx.buffer("residual", (T, self.hidden), torch.float32)
        cast = ctx.buffer("residual.cast", (T, self.hidden), ctx.dtype) if ctx.dtype != torch.float32 else None
        kept = ctx.cache.state_storage[STATE_SITE].view(-1) if self.buckets is not None else None
        ops.embedding_pairs(ctx.tokens, ctx.positions, ctx.seg_of_row, ctx.seg_start, ctx.state_slots, self.weight, out,
                            scale=self.scale, pairs=self.pairs, last_token=kept, buckets=self.buckets or 0,
                            mul_prev=self.mul_prev, mul_cur=self.mul_cur, cast=cast, single_rows=ctx.decode_only)
        ctx.leave_normed(CAST, out, out if cast is None else cast)
        return out


class LMHead(Part):
    def __init__(self, name, vocab, hidden, tied_to=None, tensor=None, softcap=None):
        """`softcap`: the logits become cap tanh(logits / cap)."""
        if softcap is not None and not softcap > 0:
            raise ValueError("the logits' cap must be positive")
        self.name, self.vocab, self.hidden, self.tied_to, self.softcap = name, vocab, hidden, tied_to, softcap
        self.tensor = tensor if tensor is not None else name + ".weight"
        self.weight = None

    def tensor_specs(self):
        return [] if self.tied_to is not None else [TensorSpec(self.tensor, (self.vocab, self.hidden))]

    def bind(self, tensors, dtype):
        self.weight = self.tied_to.weight if self.tied_to is not None else matrix_operand(tensors[self.tensor], dtype)

    def fuses_norm(self, norm, residual, rows):
        return getattr(norm, "fusable_as", None) == "rms" and ops.fused_norm_ok(residual, self.weight, rows.shape[0])

    def forward(self, h, ctx, norm=None, residual=None):
        """Logits of the normed rows h; or, with `norm`, of RMSNorm(residual[ctx.logit_rows]) in one kernel."""
        n = ctx.logit_rows.shape[0] if norm is not None else h.shape[0]
        logits = ctx.buffer("logits", (n, self.vocab), torch.float32)
        if norm is not None:
            ops.gemm_normed(residual, (norm.weight, norm.eps, ctx.logit_rows), self.weight, logits)
        else:
            ops.gemm(h, self.weight, logits, after_norm=True, scratch=ctx.scratch)
        return logits if self.softcap is None else ops.softcap(logits, self.softcap)
