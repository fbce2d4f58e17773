"""Gated feed-forward (SwiGLU): x + (silu(h Wg^T) * (h Wu^T)) Wd^T
(reference: runtime/model.py:116-119).  Gate and up run as one product against
the concatenated weight [gate; up].  With `bias` every projection adds `<name>.*_proj.bias`:
the products run as they are and a small kernel adds the bias (no fused activation then)."""
import torch

from ..kernels import ops
from .base import FeedForward, TensorSpec, matrix_operand, register_part


class GatedMLP(FeedForward):
    LAWS = {"silu": None, "gelu_tanh": ops.GELU_TANH_LAW}      # what the kernels take as the gate's law (None: silu)

    def __init__(self, name, hidden, intermediate, activation="silu", bias=False, names=None):
        """`names` = (gate, up, down): the matrices' full names under `name` where they are not `<x>_proj.weight`
        (no biases then).  `activation`: "silu", or "gelu_tanh" (the gelu's tanh form)."""
        if activation not in self.LAWS:
            raise ValueError(f"activation {activation!r}: one of {sorted(self.LAWS)}")
        if activation != "silu" and bias:
            raise ValueError("biases come with silu")
        self.law = self.LAWS[activation]
        if names is not None and bias:
            raise ValueError("biases come with the default tensor names")
        self.name, self.hidden, self.intermediate = name, hidden, intermediate
        self.bias = bool(bias)
        self.names = tuple(names) if names is not None else ("gate_proj.weight", "up_proj.weight", "down_proj.weight")
        self.w_gate_up = self.w_down = self.b_gate_up = self.b_down = None

    def tensor_specs(self):
        n, H, I = self.name, self.hidden, self.intermediate
        specs = [TensorSpec(f"{n}.{self.names[0]}", (I, H)), TensorSpec(f"{n}.{self.names[1]}", (I, H)),
                 TensorSpec(f"{n}.{self.names[2]}", (H, I))]
        if self.bias:
            specs += [TensorSpec(f"{n}.gate_proj.bias", (I,)), TensorSpec(f"{n}.up_proj.bias", (I,)), TensorSpec(f"{n}.down_proj.bias", (H,))]
        return specs

    def bind(self, tensors, dtype):
        gate = matrix_operand(tensors[f"{self.name}.{self.names[0]}"], dtype)
        up = matrix_operand(tensors[f"{self.name}.{self.names[1]}"], dtype)
        self.w_gate_up = torch.cat([gate, up], dim=0).contiguous()
        self.w_down = matrix_operand(tensors[f"{self.name}.{self.names[2]}"], dtype)
        if self.bias:   # (a bias keeps the type it is stored in; it is added in float)
            self.b_gate_up = torch.cat([tensors[f"{self.name}.gate_proj.bias"], tensors[f"{self.name}.up_proj.bias"]], dim=0).contiguous()
            self.b_down = tensors[f"{self.name}.down_proj.bias"].contiguous()

    def fuses_norm(self, norm, residual, ctx):
        return not self.bias and self.law is None and getattr(norm, "fusable_as", None) == "rms" and ops.fused_norm_ok(residual, self.w_gate_up, residual.shape[0])

    def forward(self, h, residual, ctx, norm=None):
        T = residual.shape[0]
        act = ctx.buffer("ffn.act", (T, self.intermediate), ctx.dtype)
        if self.bias:
            gate_up = ops.gemm(h, self.w_gate_up, ctx.buffer("ffn.gate_up", (T, 2 * self.intermediate), ctx.dtype), scratch=ctx.scratch)
            ops.swiglu(ops.bias_add(gate_up, self.b_gate_up), act)
            return ops.bias_add(ctx.add_product(act, self.w_down, residual), self.b_down)
        if norm is not None:
            ops.gemm_swiglu(residual, self.w_gate_up, act, norm=(norm.weight, norm.eps, None), scratch=ctx.scratch)
        elif ops.swiglu_fused_ok(h, self.w_gate_up):
            ops.gemm_swiglu(h, self.w_gate_up, act, scratch=ctx.scratch, law=self.law)   # one kernel: product and activation
        else:
            ops.gemm_swiglu(h, self.w_gate_up, act, gate_up=ctx.buffer("ffn.gate_up", (T, 2 * self.intermediate), ctx.dtype),
                            scratch=ctx.scratch, law=self.law)
        return ctx.add_product(act, self.w_down, residual)

    def output(self, h, ctx, tag="ffn", unfinished=False):
        """The feed-forward's result, float [T, hidden], without the residual sum (no biases); `unfinished`: it may be
        left as partial sums (ops.Partials) for a reader that adds them."""
        if self.bias:
            raise NotImplementedError("the result without the residual sum is made for the form without biases")
        T = h.shape[0]
        act = ctx.buffer(tag + ".act", (T, self.intermediate), ctx.dtype)
        if ops.swiglu_fused_ok(h, self.w_gate_up):
            ops.gemm_swiglu(h, self.w_gate_up, act, scratch=ctx.scratch, law=self.law)
        else:
            ops.gemm_swiglu(h, self.w_gate_up, act, gate_up=ctx.buffer(tag + ".gate_up", (T, 2 * self.intermediate), ctx.dtype),
                            scratch=ctx.scratch, law=self.law)
        if unfinished:
            return ctx.product_for_norm(act, self.w_down, tag + ".out")
        return ops.gemm(act, self.w_down, ctx.buffer(tag + ".out", (T, self.hidden), torch.float32), scratch=ctx.scratch)


class ClampedGLU(FeedForward):
    """y = (g sigmoid(slope g) (u + shift)) Wd^T with g = min(h Wg^T, limit), u = clamp(h Wu^T, -limit, limit).
    Gate and up run as one product against [gate; up]; `names` = (gate, up, down), the tensors' names under `name`."""

    def __init__(self, name, hidden, intermediate, limit, slope=1.702, shift=1.0, names=("gate", "up", "down")):
        if not limit > 0:
            raise ValueError("the clamp's limit must be positive")
        self.name, self.hidden, self.intermediate = name, hidden, intermediate
        self.limit, self.slope, self.shift, self.names = float(limit), float(slope), float(shift), tuple(names)
        self.w_gate_up = self.w_down = None

    def _tensor(self, which):
        return f"{self.name}.{self.names[which]}"

    def tensor_specs(self):
        H, I = self.hidden, self.intermediate
        return [TensorSpec(self._tensor(0), (I, H)), TensorSpec(self._tensor(1), (I, H)), TensorSpec(self._tensor(2), (H, I))]

    def bind(self, tensors, dtype):
        gate, up = (matrix_operand(tensors[self._tensor(i)], dtype) for i in (0, 1))
        self.w_gate_up = torch.cat([gate, up], dim=0).contiguous()
        self.w_down = matrix_operand(tensors[self._tensor(2)], dtype)

    def output(self, h, ctx, tag="ffn", unfinished=True):
        """The feed-forward's result, float [T, hidden], without the residual sum; `unfinished`: it may be left as partial
        sums (ops.Partials) for a reader that adds them."""
        T = h.shape[0]
        law = (self.limit, self.slope, self.shift)
        act = ctx.buffer(tag + ".act", (T, self.intermediate), ctx.dtype)
        if ops.swiglu_fused_ok(h, self.w_gate_up):
            ops.gemm_swiglu(h, self.w_gate_up, act, scratch=ctx.scratch, law=law)      # the product and the activation are one kernel
        else:
            ops.gemm_swiglu(h, self.w_gate_up, act, gate_up=ctx.buffer(tag + ".gate_up", (T, 2 * self.intermediate), ctx.dtype),
                            scratch=ctx.scratch, law=law)
        if unfinished:
            return ctx.product_for_norm(act, self.w_down, tag + ".out")
        return ops.gemm(act, self.w_down, ctx.buffer(tag + ".out", (T, self.hidden), torch.float32), scratch=ctx.scratch)

    def forward(self, h, residual, ctx, norm=None):
        from .block import add_sublayer
        return add_sublayer(residual, self.output(h, ctx), None, 1.0)


class DenseMLP(FeedForward):
    """y = act(h Wu^T) Wd^T, one matrix up and one down, no gate.  `activation`: "gelu" (the exact form, with the error
    function), "gelu_tanh" or "relu2" (the square of relu).  `names` = (up, down), the tensors' names under `name`.
    `bias`: both products add `<tensor>.b` (the up product's activation is then a kernel after the bias, not its epilogue)."""

    def __init__(self, name, hidden, intermediate, activation="gelu", names=("up", "down"), bias=False):
        if activation not in ops.GELU_KINDS:
            raise ValueError(f"activation {activation!r}: one of {sorted(ops.GELU_KINDS)}")
        self.name, self.hidden, self.intermediate, self.activation = name, hidden, intermediate, activation
        self.names, self.bias = tuple(names), bool(bias)
        self.w_up = self.w_down = self.b_up = self.b_down = None

    def _tensor(self, which):
        return f"{self.name}.{self.names[which]}"

    def tensor_specs(self):
        specs = [TensorSpec(self._tensor(0), (self.intermediate, self.hidden)), TensorSpec(self._tensor(1), (self.hidden, self.intermediate))]
        if self.bias:
            specs += [TensorSpec(self._tensor(0) + ".b", (self.intermediate,)), TensorSpec(self._tensor(1) + ".b", (self.hidden,))]
        return specs

    def bind(self, tensors, dtype):
        self.w_up, self.w_down = (matrix_operand(tensors[self._tensor(i)], dtype) for i in (0, 1))
        if self.bias:
            self.b_up, self.b_down = (tensors[self._tensor(i) + ".b"].to(torch.float32).contiguous() for i in (0, 1))

    def _activations(self, h, ctx):
        T = h.shape[0]
        if self.bias:
            up = ops.gemm(h, self.w_up, ctx.buffer("ffn.up", (T, self.intermediate), ctx.dtype), scratch=ctx.scratch)
            return ops.bias_act(up, self.b_up, ctx.buffer("ffn.act", (T, self.intermediate), ctx.dtype), self.activation)
        # the activation is the epilogue of the product where a kernel of this repository runs it
        return ops.gemm_gelu(h, self.w_up, ctx.buffer("ffn.act", (T, self.intermediate), ctx.dtype), self.activation, scratch=ctx.scratch,
                             product=ctx.buffer("ffn.up", (T, self.intermediate), ctx.dtype))

    def output(self, h, ctx):
        """The feed-forward's result, float [T, hidden], without the residual sum."""
        if self.bias:
            y = ops.gemm(self._activations(h, ctx), self.w_down, ctx.buffer("ffn.out", (h.shape[0], self.hidden), torch.float32), scratch=ctx.scratch)
            return ops.Biased(y, self.b_down)          # (the kernel that adds the result adds the bias)
        return ctx.product_for_norm(self._activations(h, ctx), self.w_down, "ffn.out")

    def forward(self, h, residual, ctx, norm=None):
        if self.bias:
            from .block import add_sublayer
            return add_sublayer(residual, self.output(h, ctx), None, 1.0)
        return ctx.add_product(self._activations(h, ctx), self.w_down, residual)


class RoutedExperts(FeedForward):
    """A mixture of `experts` small feed-forwards of which every row uses `top`: router logits W_r h + b in float, the
    `top` largest chosen (the lowest index wins a tie), their weights the softmax over the chosen logits only; an
    expert is W_down relu(W_up h)^2 without biases, and the result is the weighted sum of the chosen experts'.

    The rows of a step are ordered by expert on the device (ops.experts_route) and each expert's matrix meets only its
    own rows, in tiles (ops.experts_gemm); the down products are left as `top` rows a step row for the kernel that
    adds the sublayer's result (ops.WeightedRows).  `ride(weight)`: further rows for the router's product, whose
    float results are then `rider`.  `names`: (router, expert prefix, up, down), the tensors' names under `name`;
    expert j's matrices are `<name>.<prefix>j.<up|down>`."""

    def __init__(self, name, hidden, intermediate, experts, top, names=("router", "e", "up", "down")):
        if not 0 < top <= min(experts, 16):
            raise ValueError(f"{top} of {experts} experts: between 1 and min(experts, 16)")
        self.name, self.hidden, self.intermediate, self.experts, self.top = name, hidden, intermediate, int(experts), int(top)
        self.names = tuple(names)
        self.rider, self.rider_rows = None, 0

    def _expert(self, j, which):
        return f"{self.name}.{self.names[1]}{j}.{self.names[2 + which]}"

    def tensor_specs(self):
        H, I, router = self.hidden, self.intermediate, f"{self.name}.{self.names[0]}"
        specs = [TensorSpec(router, (self.experts, H)), TensorSpec(router + ".b", (self.experts,))]
        for j in range(self.experts):
            specs += [TensorSpec(self._expert(j, 0), (I, H)), TensorSpec(self._expert(j, 1), (H, I))]
        return specs

    def _join(self, extra=None):
        parts = [self.w_router] + ([] if extra is None else [extra])
        rows = sum(p.shape[0] for p in parts)
        if rows % 8:
            parts.append(torch.zeros(8 - rows % 8, self.hidden, dtype=parts[0].dtype, device=parts[0].device))
        self.w_in = torch.cat(parts, dim=0).contiguous()

    def bind(self, tensors, dtype):
        router = f"{self.name}.{self.names[0]}"
        self.w_router = matrix_operand(tensors[router], dtype)
        self.router_bias = tensors[router + ".b"].to(torch.float32).contiguous()
        self._join()
        self.w_up = torch.stack([matrix_operand(tensors[self._expert(j, 0)], dtype) for j in range(self.experts)]).contiguous()
        self.w_down = torch.stack([matrix_operand(tensors[self._expert(j, 1)], dtype) for j in range(self.experts)]).contiguous()

    def ride(self, weight):
        self.rider_rows = weight.shape[0]
        self._join(weight)

    def output(self, h, ctx):
        """The feed-forward's result as ops.WeightedRows (float [T * top, hidden] and the weights [T, top])."""
        T, E, top = h.shape[0], self.experts, self.top
        logits = ops.gemm(h, self.w_in, ctx.buffer("moe.logits", (T, self.w_in.shape[0]), torch.float32), scratch=ctx.scratch)
        self.rider = logits[:, E:E + self.rider_rows] if self.rider_rows else None
        chosen, weights = ctx.buffer("moe.chosen", (T, top), torch.int32), ctx.buffer("moe.weights", (T, top), torch.float32)
        down = ctx.buffer("moe.down", (T * top, self.hidden), torch.float32)
        if ops.experts_rows_ok(h, self.w_up, T * top) and ops.experts_rows_ok(h, self.w_down, T * top):
            # few rows (decoding): every (row, choice) pair streams its expert's two matrices
            ops.experts_route(logits[:, :E], self.router_bias, top, chosen, weights)
            up = ops.experts_rows(h, self.w_up, chosen, ctx.buffer("moe.up", (T * top, self.intermediate), ctx.dtype), top=top, act=True)
            ops.experts_rows(up, self.w_down, chosen, down)
            return ops.WeightedRows(down, weights, top)
        tiles = ops.expert_tiles(T, top, E)
        places, tile_expert = ctx.buffer("moe.places", (tiles * ops.EXPERT_TILE,), torch.int32), ctx.buffer("moe.tiles", (tiles,), torch.int32)
        ops.experts_route(logits[:, :E], self.router_bias, top, chosen, weights, places, tile_expert)
        up = ops.experts_gemm(h, self.w_up, places, tile_expert, ctx.buffer("moe.up", (tiles * ops.EXPERT_TILE, self.intermediate), ctx.dtype),
                              top=top, act=True)
        ops.experts_gemm(up, self.w_down, places, tile_expert, down, scatter=True)
        return ops.WeightedRows(down, weights, top)

    def forward(self, h, residual, ctx, norm=None):
        return _add_weighted(residual, self.output(h, ctx))


class ScoredExperts(FeedForward):
    """A mixture of experts routed by scores: s = softmax(W_r h) over all router outputs, in float (`scores` "sigmoid": the
    sigmoid of each); the choice goes by s + `correction` (a tensor; the weights use s without it), optionally held to the
    best `groups[1]` of `groups[0]` equal groups of neighbouring outputs (a group's score is its largest choice score, with
    `group_pairs` the sum of its two largest; the others count as minus infinity); the `top` largest are chosen and weigh s
    itself, or with `floor` s divided by the sum of the chosen s plus that number.  The first `experts` outputs are gated
    feed-forwards without biases, W_down (silu(W_gate h) * (W_up h)), or with `law` = (limit, slope, shift) the clamped form of
    ClampedGLU; the last `identity` outputs have no tensors: their result is the input itself.  `shared`: a feed-forward
    part (with `output`) that every row goes through, added, with `shared_gate` (a tensor's name under `name`, [1, hidden])
    times sigmoid of that row's product with h.

    The rows of a step are ordered by expert on the device and each expert's matrices meet only their own rows
    (ops.experts_gemm; steps of few rows stream each pair's matrices, ops.experts_rows); gate and up are one product over
    [gate; up] a expert with the activation as its epilogue (float32: a kernel after it).  `names`: (router, correction, expert
    prefix, gate, up, down)."""
    leaves_rows = True       # `output` takes `unsummed`

    def __init__(self, name, hidden, intermediate, experts, top, identity=0, groups=None, shared=None, correction=True,
                 names=("router", "correction", "e", "gate", "up", "down"), scores="softmax", group_pairs=False, floor=None, law=None,
                 shared_gate=None):
        outputs = experts + identity
        if not 0 < top <= min(outputs, 16) or experts <= 0 or identity < 0:
            raise ValueError(f"{top} of {experts} + {identity} router outputs: between 1 and min(outputs, 16)")
        if groups is not None:
            count, keep = groups
            if count <= 0 or count > 64 or outputs % count or not 0 < keep <= count or keep * (outputs // count) < top:
                raise ValueError(f"{outputs} router outputs in {count} groups of which {keep} are kept, for {top} choices")
        if shared is not None and not hasattr(shared, "output"):
            raise ValueError("the shared feed-forward must give its result without the residual sum (output)")
        if scores not in ("softmax", "sigmoid"):
            raise ValueError(f"scores {scores!r} are neither softmax nor sigmoid")
        if law is not None and not law[0] > 0:
            raise ValueError("the clamp's limit must be positive")
        if shared_gate is not None and (shared is None or identity):
            raise ValueError("a gate of the shared feed-forward comes with one, and without identity outputs")
        self.name, self.hidden, self.intermediate = name, hidden, intermediate
        self.experts, self.identity, self.outputs, self.top = int(experts), int(identity), outputs, int(top)
        self.groups, self.shared, self.has_correction, self.names = groups, shared, bool(correction), tuple(names)
        self.route = dict(sigmoid=scores == "sigmoid", group_pairs=bool(group_pairs), floor=floor)
        self.law = None if law is None else tuple(float(v) for v in law)
        self.shared_gate = None if shared_gate is None else f"{name}.{shared_gate}"

    def _expert(self, j, which):
        return f"{self.name}.{self.names[2]}{j}.{self.names[3 + which]}"

    def tensor_specs(self):
        H, I = self.hidden, self.intermediate
        specs = [TensorSpec(f"{self.name}.{self.names[0]}", (self.outputs, H))]
        if self.has_correction:
            specs.append(TensorSpec(f"{self.name}.{self.names[1]}", (self.outputs,)))
        for j in range(self.experts):
            specs += [TensorSpec(self._expert(j, 0), (I, H)), TensorSpec(self._expert(j, 1), (I, H)), TensorSpec(self._expert(j, 2), (H, I))]
        if self.shared_gate is not None:
            specs.append(TensorSpec(self.shared_gate, (1, H)))
        return specs + ([] if self.shared is None else self.shared.tensor_specs())

    def bind(self, tensors, dtype):
        # (the shared part's gate is one more row of the router's product)
        rows = [matrix_operand(tensors[f"{self.name}.{self.names[0]}"], dtype)]
        if self.shared_gate is not None:
            rows.append(matrix_operand(tensors[self.shared_gate], dtype))
        n = sum(r.shape[0] for r in rows)
        if n % 8:      # rows of the router's product are a multiple of 8: zero rows at the end
            rows.append(torch.zeros(8 - n % 8, self.hidden, dtype=rows[0].dtype, device=rows[0].device))
        self.w_router = torch.cat(rows, dim=0).contiguous()
        self.correction = tensors[f"{self.name}.{self.names[1]}"].to(torch.float32).contiguous() if self.has_correction else None
        self.w_gate_up = torch.stack([torch.cat([matrix_operand(tensors[self._expert(j, 0)], dtype), matrix_operand(tensors[self._expert(j, 1)], dtype)])
                                      for j in range(self.experts)]).contiguous()
        self.w_down = torch.stack([matrix_operand(tensors[self._expert(j, 2)], dtype) for j in range(self.experts)]).contiguous()
        if self.shared is not None:
            self.shared.bind(tensors, dtype)

    def prepare(self, device, dtype):
        if self.shared is not None:
            self.shared.prepare(device, dtype)

    def _activation(self, gate_up, act):
        return ops.swiglu(gate_up, act) if self.law is None else ops.glu_clamped(gate_up, act, *self.law)

    def rows(self, h, ctx):
        """The feed-forward's result as an ops.ExpertSum: the chosen experts' rows and their weights, and the shared part's
        rows, for a kernel that adds them all (no identity outputs)."""
        T, E, top, I = h.shape[0], self.experts, self.top, self.intermediate
        chosen, weights = ctx.buffer("moe.chosen", (T, top), torch.int32), ctx.buffer("moe.weights", (T, top), torch.float32)
        down = ctx.buffer("moe.down", (T * top, self.hidden), torch.float32)
        gate = None
        if ops.experts_route_product_ok(h, self.w_router, self.outputs + (self.shared_gate is not None)):
            gate = None if self.shared_gate is None else ctx.buffer("moe.gate", (T, 1), torch.float32)      # the product and the choice in one kernel

            def route(*layout):
                ops.experts_route_product(h, self.w_router, self.correction, top, chosen, weights, self.outputs, E, self.groups, *layout, gate=gate, **self.route)
        else:
            logits = ops.gemm(h, self.w_router, ctx.buffer("moe.logits", (T, self.w_router.shape[0]), torch.float32), scratch=ctx.scratch)
            gate = None if self.shared_gate is None else logits[:, self.outputs:self.outputs + 1]

            def route(*layout):
                ops.experts_route_scored(logits[:, :self.outputs], self.correction, top, chosen, weights, E, self.groups, *layout, **self.route)
        if ops.experts_rows_ok(h, self.w_gate_up, T * top) and ops.experts_rows_ok(h, self.w_down, T * top):
            # few rows (decoding): every (row, choice) pair streams its expert's matrices
            route()
            act = ops.experts_rows_gated(h, self.w_gate_up, chosen, ctx.buffer("moe.act", (T * top, I), ctx.dtype), self.law or (0.0, 0.0, 0.0), top=top)
            ops.experts_rows(act, self.w_down, chosen, down)
        else:
            tiles = ops.expert_tiles(T, top, E)
            places, tile_expert = ctx.buffer("moe.places", (tiles * ops.EXPERT_TILE,), torch.int32), ctx.buffer("moe.tiles", (tiles,), torch.int32)
            route(places, tile_expert)
            act = ctx.buffer("moe.act", (tiles * ops.EXPERT_TILE, I), ctx.dtype)
            if ops.experts_gemm_gated_ok(h, self.w_gate_up):
                ops.experts_gemm_gated(h, self.w_gate_up, places, tile_expert, act, self.law or (0.0, 0.0, 0.0), top=top)
            else:
                gate_up = ops.experts_gemm(h, self.w_gate_up, places, tile_expert, ctx.buffer("moe.gate_up", (tiles * ops.EXPERT_TILE, 2 * I), ctx.dtype), top=top)
                self._activation(gate_up, act)
            ops.experts_gemm(act, self.w_down, places, tile_expert, down, scatter=True)
        also = None if self.shared is None else self.shared.output(h, ctx, tag="moe.shared", unfinished=False)
        return ops.ExpertSum(down, weights, chosen, E, shared=also, gate=gate)

    def output(self, h, ctx, unsummed=False):
        """The feed-forward's result, float [T, hidden], without the residual sum; `unsummed`: it may be left as an
        ops.ExpertSum for a reader that adds the rows to the residual stream itself."""
        parts = self.rows(h, ctx)
        if unsummed and self.identity == 0 and self.hidden <= ops.EXPERTS_ADD_MAX_COLS:
            return parts
        y = ctx.buffer("moe.y", (h.shape[0], self.hidden), torch.float32)
        if parts.gate is not None:
            y.zero_()
            return ops.experts_add(y, parts)
        return ops.experts_combine(parts.down, parts.weights, parts.chosen, h, y, self.experts, shared=parts.shared)

    def forward(self, h, residual, ctx, norm=None):
        from .block import add_sublayer
        return add_sublayer(residual, self.output(h, ctx, unsummed=True), None, 1.0)


class TokenSide(FeedForward):
    """A sublayer that reads a table by the token: y = Wp (gelu_tanh(Wg h) * e), e the columns [first, first + width) of the
    token's row in `source.side_table` (a part that owns the table of all layers).  `names`: (gate, projection)."""

    def __init__(self, name, hidden, width, first, source, names=("gate", "proj")):
        self.name, self.hidden, self.width, self.first, self.source, self.names = name, hidden, int(width), int(first), source, tuple(names)
        self.padded = -(-self.width // 8) * 8
        self.w_gate = self.w_proj = None

    def tensor_specs(self):
        return [TensorSpec(f"{self.name}.{self.names[0]}", (self.width, self.hidden)), TensorSpec(f"{self.name}.{self.names[1]}", (self.hidden, self.width))]

    def bind(self, tensors, dtype):
        gate, proj = (matrix_operand(tensors[f"{self.name}.{n}"], dtype) for n in self.names)
        extra = self.padded - self.width          # (zero rows and columns: operands in whole 16-byte words)
        if extra:
            gate = torch.cat([gate, torch.zeros(extra, self.hidden, dtype=gate.dtype, device=gate.device)])
            proj = torch.cat([proj, torch.zeros(self.hidden, extra, dtype=proj.dtype, device=proj.device)], dim=1)
        self.w_gate, self.w_proj = gate.contiguous(), proj.contiguous()

    def output(self, h, ctx, unfinished=True):
        """The sublayer's result, float [T, hidden], without the residual sum."""
        T = h.shape[0]
        act, table = ctx.buffer("side.act", (T, self.padded), ctx.dtype), self.source.side_table
        if ops.side_rows_ok(h, self.w_gate):
            ops.side_rows(h, self.w_gate, ctx.tokens, table, self.first, self.width, act)        # few rows: the gate's product as well
        else:
            z = ops.gemm(h, self.w_gate, ctx.buffer("side.z", (T, self.padded), torch.float32), scratch=ctx.scratch)
            ops.side_gate(z, ctx.tokens, table, self.first, self.width, act)
        return ctx.product_for_norm(act, self.w_proj, "side.y")

    def forward(self, h, residual, ctx, norm=None):
        from .block import add_sublayer
        return add_sublayer(residual, self.output(h, ctx), None, 1.0)


def _add_weighted(residual, y):
    """residual += sum_k weights[:, k] * rows[k]: for an arrangement that adds a feed-forward's result itself (torch's own
    kernels: no arrangement of this package takes this way)."""
    rows, dim = residual.shape
    residual += (y.rows.view(rows, y.top, dim) * y.weights.unsqueeze(-1)).sum(dim=1)
    return residual


register_part("ffn", "routed_experts", RoutedExperts)
register_part("ffn", "scored_experts", ScoredExperts)
register_part("ffn", "token_side", TokenSide)
register_part("ffn", "gated_mlp", GatedMLP)
register_part("ffn", "dense_mlp", DenseMLP)
register_part("ffn", "clamped_glu", ClampedGLU)
