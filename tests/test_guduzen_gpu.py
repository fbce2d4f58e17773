"""The Guduzen design on the GPU: every new kernel alone against plain float arithmetic of the same operands, then
whole models against the plain implementation (tests/plain_guduzen.py): layer by layer, prompt against token-by-token
decoding, portions down to two tokens, mixed batches with pages and state slots used again, batches against each
request alone, far keys, a window's edge and old state in a model drawn sharp, the first tokens, long decoding, eager
and captured, generation through the scheduler, the command line, the replay program."""
import json

import numpy as np
import pytest
import torch

import plain_guduzen as P
import conftest
from conftest import assert_close, random_tokens
from guduzen_models import CONFIGS, RANKS, SEEDS, plain_logits, write_folder
from trace_tools import Trace

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("guduzen")
    return {name: write_folder(base / name, CONFIGS[name], SEEDS[name], sharp=name == "s", ranks=RANKS[name]) for name in CONFIGS}


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.asarray(a), dtype=dtype).cuda().contiguous()


def ints(a):
    return torch.as_tensor(np.asarray(a, dtype=np.int32)).cuda()


def close(got, want, tol=2e-5):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape
    assert np.isfinite(got).all()
    err = np.abs(got - want).max() / max(np.abs(want).max(), 1e-30)
    assert err < tol, f"differs by {err:.3e} (bound {tol})"


def rounded(a, dtype="float32"):
    """The values a tensor of `dtype` holds of the array, as float64."""
    return torch.as_tensor(np.asarray(a), dtype=torch.float32).to(TORCH[dtype]).to(torch.float64).numpy()


# -- kernels alone ----------------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams, dim", [(1, 40), (2, 62), (3, 256), (4, 500), (5, 1500), (6, 4096), (7, 7), (8, 3000), (3, 5000), (2, 9001)])
def test_streams_filled_read_mixed_and_written(dtype, streams, dim):
    """The embedding into the streams with the first read, a read of gathered rows, a write with the read that follows, a
    write alone, a write of a product left as partial sums."""
    from runtime.kernels import ops
    rng = np.random.default_rng(dim)
    rows, vocab, eps, td = 6, 11, 1e-4, TORCH[dtype]
    tol = 2e-5 if dtype == "float32" else 6e-3
    table, tokens = rng.standard_normal((vocab, dim)), rng.integers(0, vocab, rows)
    w_in, w_out, mix = rng.standard_normal(streams), rng.standard_normal(streams), rng.standard_normal((streams, streams))
    weight = 1 + 0.2 * rng.standard_normal(dim)
    x = torch.full((rows, streams * dim), float("nan"), device="cuda")
    h = torch.full((rows, dim), float("nan"), dtype=td, device="cuda")
    read = lambda: (dev(w_in), dev(weight), eps, h)
    ops.streams_embed(ints(tokens), dev(table, td), x, streams, read=read())
    X = P.spread(rounded(table, dtype)[tokens], streams)
    at = lambda: x.cpu().numpy().reshape(rows, streams, dim).transpose(1, 0, 2)
    close(at(), X, 1e-7)
    fr = lambda X: P.rms(P.read_streams(X, rounded(w_in)), eps) * rounded(weight)
    close(h.float().cpu().numpy(), fr(X), tol)
    # streams that differ
    start = rng.standard_normal((rows, streams * dim))
    X = rounded(start).reshape(rows, streams, dim).transpose(1, 0, 2)
    x = dev(start)
    some = [4, 0, 5, 4]
    out = torch.full((4, dim), float("nan"), dtype=td, device="cuda")
    ops.streams_read(x, streams, dev(w_in), dev(weight), eps, out, rows=ints(some))
    close(out.float().cpu().numpy(), fr(X)[some], tol)
    y = rng.standard_normal((rows, dim))
    h.fill_(float("nan"))
    ops.streams_step(x, streams, dev(y), dev(mix), dev(w_out), read=read())
    X = P.write_streams(X, rounded(mix), rounded(w_out), rounded(y))
    close(at(), X, 1e-5)
    close(h.float().cpu().numpy(), fr(X), tol)
    ops.streams_step(x, streams, dev(y), dev(mix), dev(w_out))
    X = P.write_streams(X, rounded(mix), rounded(w_out), rounded(y))
    close(at(), X, 1e-5)
    parts = rng.standard_normal((3, rows, dim))
    ops.streams_step(x, streams, ops.Partials(dev(parts.reshape(-1)), 3, rows, dim), dev(mix), dev(w_out), read=read())
    X = P.write_streams(X, rounded(mix), rounded(w_out), rounded(parts).sum(axis=0))
    close(at(), X, 1e-5)
    close(h.float().cpu().numpy(), fr(X), tol)


@pytest.mark.parametrize("rows, cols", [(1, 1), (3, 77), (5, 1024), (64, 4099)])
def test_capped_logits(rows, cols):
    from runtime.kernels import ops
    x = 40.0 * np.random.default_rng(rows).standard_normal((rows, cols))
    got = ops.softcap(dev(x), 15.0).cpu().numpy()
    close(got, P.capped(rounded(x), 15.0), 1e-6)
    with pytest.raises(ops.KernelError):
        ops.softcap(dev(x), 0.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m, n, k", [(1, 72, 64), (1, 3000, 2048), (3, 40, 96), (8, 128, 512), (11, 2600, 1024), (40, 4096, 4096), (64, 136, 96), (100, 72, 64),
                                     (257, 136, 104), (300, 2304, 1024), (5, 20, 50), (16, 8192, 4096), (30, 2000, 2048)])
def test_the_gate_is_the_tanh_form_of_gelu(dtype, m, n, k):
    """In every kernel that takes the product of gate and up: few rows and many, small weights and large."""
    from runtime.kernels import ops
    if dtype == "float32" and n * k > 4 << 20:
        pytest.skip("the float kernel has one form; small weights show it")
    gen = torch.Generator(device="cuda").manual_seed(m + n)
    td = TORCH[dtype]
    a = torch.randn(m, k, generator=gen, device="cuda").to(td)
    w = (torch.randn(2 * n, k, generator=gen, device="cuda") * (3.0 / k ** 0.5)).to(td)
    out = torch.full((m, n), float("nan"), dtype=td, device="cuda")
    ops.gemm_swiglu(a, w, out, gate_up=torch.empty(m, 2 * n, dtype=td, device="cuda"), law=ops.GELU_TANH_LAW)
    gu = (a.float() @ w.float().t()).double()
    want = torch.nn.functional.gelu(gu[:, :n], approximate="tanh") * gu[:, n:]
    close(out.double().cpu().numpy(), want.cpu().numpy(), 1e-5 if dtype == "float32" else 1.2e-2)


@pytest.mark.parametrize("dtype, float_rows", [("float32", True), ("bfloat16", True), ("bfloat16", False)])
@pytest.mark.parametrize("heads, kv_heads, dim, vdim", [(4, 2, 24, 16), (1, 1, 10, 24), (20, 4, 64, 64), (3, 3, 16, 40), (5, 1, 200, 256)])
def test_biases_and_norms_without_a_weight_land_in_the_pages(dtype, float_rows, heads, kv_heads, dim, vdim):
    from runtime.kernels import ops
    rng = np.random.default_rng(dim)
    rows, page_size, pages, eps, td = 37, 8, 7, 1e-3, TORCH[dtype]
    pad = -(-max(dim, vdim) // 8) * 8
    nq, nk, nv = heads * dim, kv_heads * dim, kv_heads * vdim
    proj, bias = rng.standard_normal((rows, nq + nk + nv + 5)), rng.standard_normal(nq + nk + nv)
    slots = rng.permutation(pages * page_size)[:rows]
    slots[3] = -1                                                       # a padding row: its queries only
    q_out = torch.full((rows, heads * pad), float("nan"), dtype=td, device="cuda")
    kc = torch.full((pages, kv_heads, page_size, pad), 7.0, dtype=td, device="cuda")
    vc = torch.full((pages, kv_heads, pad, page_size), 7.0, dtype=td, device="cuda")
    src = dev(proj, torch.float32 if float_rows else td)
    ops.qk_norm_scatter(src, None, None, q_out, kc, vc, ints(slots), heads, kv_heads, dim, vdim, pad, page_size, eps, bias=dev(bias), plain_norm=True)
    pr = src.double().cpu().numpy()[:, :nq + nk + nv] + rounded(bias)
    q, k = P.rms(pr[:, :nq].reshape(rows, heads, dim), eps), P.rms(pr[:, nq:nq + nk].reshape(rows, kv_heads, dim), eps)
    v = pr[:, nq + nk:].reshape(rows, kv_heads, vdim)
    tol = 1e-5 if dtype == "float32" else 5e-3
    got = q_out.float().cpu().numpy().reshape(rows, heads, pad)
    close(got[:, :, :dim], q, tol)
    assert not got[:, :, dim:].any()
    kk, vv = kc.float().cpu().numpy(), vc.float().cpu().numpy()
    for i, slot in enumerate(slots):
        if slot < 0:
            continue
        a, b = slot // page_size, slot % page_size
        close(kk[a, :, b, :dim], k[i], tol)
        close(vv[a, :, :vdim, b], v[i], tol)
        assert not kk[a, :, b, dim:].any() and not vv[a, :, vdim:, b].any()
    free = sorted(set(range(pages * page_size)) - set(slots.tolist()))
    assert all((kk[s // page_size, :, s % page_size] == 7.0).all() and (vv[s // page_size, :, :, s % page_size] == 7.0).all() for s in free)
    # a layer that reads another's keys: queries only
    alone = torch.full((rows, heads * pad), float("nan"), dtype=td, device="cuda")
    ops.qk_norm_scatter(src[:, :nq].contiguous(), None, None, alone, None, None, None, heads, kv_heads, dim, vdim, pad, page_size, eps,
                        bias=dev(bias[:nq]), plain_norm=True)
    assert torch.equal(alone, q_out)


@pytest.mark.parametrize("m, n, heads, dim, splits", [(1, 96, 4, 64, 8), (3, 200, 2, 128, 4), (8, 192, 6, 64, 8), (14, 64, 3, 32, 4), (1, 4096, 16, 128, 8)])
def test_a_product_that_merges_split_attention_without_a_residual(m, n, heads, dim, splits):
    from runtime.kernels import ops
    gen = torch.Generator(device="cuda").manual_seed(m * n)
    k = heads * dim
    w = (torch.randn(n, k, generator=gen, device="cuda") / k ** 0.5).to(torch.bfloat16)
    assert ops.gemm_merged_ok(m, w, heads, dim, splits)
    part = torch.randn(m, heads, splits, dim, generator=gen, device="cuda").to(torch.bfloat16)
    ml = torch.stack([torch.randn(m, heads, splits, generator=gen, device="cuda"), 0.5 + torch.rand(m, heads, splits, generator=gen, device="cuda")], dim=-1).contiguous()
    out = torch.full((m, n), float("nan"), device="cuda")
    ops.gemm_merged((part, ml, splits), heads, dim, w, out)
    share = torch.exp2((ml[..., 0] - ml[..., 0].amax(dim=-1, keepdim=True)).double()) * ml[..., 1].double()
    share = share / share.sum(dim=-1, keepdim=True)
    want = (share[..., None] * part.double()).sum(dim=2).reshape(m, k).cpu() @ w.double().cpu().t()
    close(out.cpu().numpy(), want.numpy(), 1e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank", [13, 40, 96, 300])
def test_latents_without_a_turning_part_land_in_the_pages(dtype, rank):
    from runtime.kernels import ops
    rng = np.random.default_rng(rank)
    rows, page_size, pages, eps, heads, dim, td = 9, 4, 5, 1e-5, 3, 12, TORCH[dtype]
    pad = -(-rank // 8) * 8
    down, weight = rng.standard_normal((rows, rank + 6)), 1 + 0.1 * rng.standard_normal(rank)
    slots = rng.permutation(pages * page_size)[:rows]
    kc = torch.full((pages, 1, page_size, pad), 7.0, dtype=td, device="cuda")
    vc = torch.full((pages, 1, pad, page_size), 7.0, dtype=td, device="cuda")
    q_out = torch.full((rows, heads * pad), 7.0, dtype=td, device="cuda")
    ops.latent_keys(dev(down)[:, 2:2 + rank], dev(weight), dev(rng.standard_normal((rows, heads * dim)), td), q_out, kc, vc, ints(np.zeros(rows)),
                    ints(slots), None, None, heads, dim, 0, rank, pad, page_size, eps)
    c = P.rmsnorm(rounded(down)[:, 2:2 + rank], rounded(weight), eps)
    kk, vv = kc.float().cpu().numpy(), vc.float().cpu().numpy()
    for i, slot in enumerate(slots):
        a, b = slot // page_size, slot % page_size
        for got in (kk[a, 0, b], vv[a, 0, :, b]):
            close(got[:rank], c[i], 1e-5 if dtype == "float32" else 5e-3)
            assert not got[rank:].any()
    q = q_out.float().cpu().numpy().reshape(rows, heads, pad)
    assert (q[:, :, :rank] == 7.0).all() and not q[:, :, rank:].any()        # the latent's coordinates are the caller's


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, taps, ranks, columns", [
    (4, 2, 16, 12, 3, (10, 6), None), (1, 1, 5, 7, 1, (3, 5), 4), (10, 2, 128, 40, 4, (40, 136), 32), (3, 3, 200, 24, 2, (16, 33), 8),
    (2, 1, 256, 16, 4, (64, 130), 16), (4, 4, 48, 300, 16, (24, 72), None), (2, 1, 32, 64, 4, (128, 32), 16), (2, 2, 20, 33, 4, (8, 8), 32),
    (3, 1, 100, 10, 5, (7, 200), 4), (2, 2, 64, 96, 3, (32, 64), 8)])
def test_delta_rule_with_a_decay_a_channel_over_segments_with_states_carried_and_slots_used_again(dtype, heads, kv_heads, dim, vdim, taps, ranks, columns):
    """Three steps over four state slots: portions and single rows of several requests in one step, portions shorter than
    the convolution, a step of single rows, padding rows, a slot zeroed and used again; the operands, the scan and the
    gated norm against the recurrence written out."""
    from runtime.kernels import ops
    rng = np.random.default_rng(heads + dim)
    td, eps, share = TORCH[dtype], 1e-5, heads // kv_heads
    qk, inner = kv_heads * dim, heads * vdim
    ch, (ra, rg) = 2 * qk + inner, ranks
    up4 = lambda n: -(-n // 4) * 4
    at_b, at_a = ch, up4(ch + heads)
    at_g = up4(at_a + ra)
    width = up4(at_g + rg)
    taps_w, up_a, up_g = rng.standard_normal((ch, taps)), rng.standard_normal((heads * dim, ra)) / ra ** 0.5, rng.standard_normal((inner, rg)) / rg ** 0.5
    dt_bias, a_log, weight = rng.standard_normal(heads * dim) - 1, rng.standard_normal(heads) - 1, 1 + 0.1 * rng.standard_normal(vdim)
    dt_bias[0] = 30.0                                            # softplus far from zero: a decay that is nothing
    size = heads * dim * vdim
    state = torch.zeros(4, size + (taps - 1) * ch, device="cuda")
    fresh = lambda: (np.zeros((heads, dim, vdim)), np.zeros((taps - 1, ch)))
    kept = {s: fresh() for s in range(4)}
    ua, ug = ops.low_rank_rows(dev(up_a, td)), ops.low_rank_rows(dev(up_g, td))
    chunk_state, step_state = state.clone(), state.clone()
    eqv = ops.channel_step_ok(step_state, dim, vdim)
    steps = [([7, 1, 300, 2], [2, 0, 3, 1]), ([1, 1, 1, 1], [3, 1, 0, 2]), ([1, 2, 33], [1, 2, 0]), ([1, 1], [3, 0])]
    for n, (counts, slots) in enumerate(steps):
        if n == 2:
            for st in (state, chunk_state, step_state):
                st[1].zero_()
            kept[1] = fresh()
        single = all(c == 1 for c in counts)
        T = sum(counts) + 2                                      # two padding rows, which belong to no segment
        proj = rng.standard_normal((T, width))
        start = np.concatenate(([0], np.cumsum(counts)))
        seg_of_row = np.concatenate([np.repeat(np.arange(len(counts)), counts), [-1, -1]])
        dp = dev(proj)
        qkv, decay, gate, o = (torch.full((T, c), float("nan"), device="cuda") for c in (ch, heads * dim, inner, inner))
        args = (ints(start), ints(slots))
        ops.channel_delta_inputs(dp, dev(taps_w.T), state[:, size:], qkv, ints(seg_of_row), *args, kv_heads, dim, heads, vdim, at_a, ua,
                                 dev(dt_bias), dev(a_log), decay, at_g, ug, gate, single_rows=single)
        operands = (qkv[:, :qk], qkv[:, qk:2 * qk], qkv[:, 2 * qk:], decay, dp[:, at_b:at_b + heads])
        law = dict(share=share, q_scale=dim ** -0.5)
        ops.channel_delta_scan(*operands, o, state, *args, heads, dim, vdim, columns=columns, **law)
        # the same chunk by chunk, a few chunks a launch
        chunked = torch.full((T, inner), float("nan"), device="cuda")
        work = torch.full((ops.channel_chunk_work(T, len(counts), heads, dim, vdim, slab=7),), float("nan"), device="cuda")
        ops.channel_delta_chunks(*operands, chunked, chunk_state, *args, heads, dim, vdim, work, slab=7, **law)
        if eqv:       # single rows with norm and gate in the kernel; the other steps move its state on row by row
            stepped = torch.full((T, inner), float("nan"), dtype=td, device="cuda")
            if single:
                ops.channel_delta_step(*operands, gate, dev(weight), stepped, step_state, *args, heads, dim, vdim, eps, **law)
            else:
                ops.channel_delta_scan(*operands, o.clone(), step_state, *args, heads, dim, vdim, **law)
        out = torch.full((T, inner), float("nan"), device="cuda")
        ops.group_norm_gate(o, gate, dev(weight), out, heads, eps, gate_first=False, shared_weight=True, sigmoid=True)
        pr = rounded(proj)
        z = pr[:, at_a:at_a + ra] @ rounded(up_a, dtype).T + rounded(dt_bias)
        g = np.exp(-np.exp(rounded(a_log))[:, None] * P.softplus(z).reshape(T, heads, dim))
        gz = pr[:, at_g:at_g + rg] @ rounded(up_g, dtype).T
        beta = P.sigmoid(pr[:, at_b:at_b + heads])
        rows = slice(0, sum(counts))
        close(decay.cpu().numpy()[rows], g.reshape(T, -1)[rows], 2e-5 if dtype == "float32" else 4e-5)
        g = decay.double().cpu().numpy().reshape(T, heads, dim)              # (the recurrence from the decays as they came out)
        close(gate.cpu().numpy()[rows], gz[rows], 2e-5 if dtype == "float32" else 4e-5)
        for s, slot in enumerate(slots):
            S, past = kept[slot]
            own = pr[start[s]:start[s + 1]]
            x = np.concatenate([past, own[:, :ch]])
            y = P.silu(sum(x[j:j + len(own)] * rounded(taps_w)[:, j] for j in range(taps)))
            q = P.unit(y[:, :qk].reshape(-1, kv_heads, dim))
            k = P.unit(y[:, qk:2 * qk].reshape(-1, kv_heads, dim))
            v = y[:, 2 * qk:].reshape(-1, heads, vdim)
            close(qkv.cpu().numpy()[start[s]:start[s + 1]], np.concatenate([q.reshape(-1, qk), k.reshape(-1, qk), v.reshape(-1, inner)], axis=1))
            want = np.zeros((len(own), heads, vdim))
            for i in range(len(own)):
                t = start[s] + i
                for h in range(heads):
                    S[h] = g[t, h][:, None] * S[h]
                    S[h] = S[h] + np.outer(k[i, h // share], beta[t, h] * (v[i, h] - k[i, h // share] @ S[h]))
                    want[i, h] = q[i, h // share] @ S[h] * dim ** -0.5
            close(o.cpu().numpy()[start[s]:start[s + 1]], want.reshape(-1, inner), 3e-5)
            close(chunked.cpu().numpy()[start[s]:start[s + 1]], want.reshape(-1, inner), 3e-5)
            want = P.rms(want, eps) * rounded(weight) * P.sigmoid(gate.double().cpu().numpy()[start[s]:start[s + 1]].reshape(-1, heads, vdim))
            close(out.cpu().numpy()[start[s]:start[s + 1]], want.reshape(-1, inner), 1e-4)
            if eqv and single:
                close(stepped.float().cpu().numpy()[start[s]:start[s + 1]], want.reshape(-1, inner), 1e-4 if dtype == "float32" else 6e-3)
            kept[slot] = (S, x[len(x) - (taps - 1):] if taps > 1 else past)
        for slot in range(4):
            have = state[slot].cpu().numpy()
            for st in (state, chunk_state, step_state) if eqv else (state, chunk_state):
                close(st[slot, :size].cpu().numpy().reshape(heads, dim, vdim) + 1.0, kept[slot][0] + 1.0, 2e-5)
            if taps > 1:
                close(have[size:].reshape(taps - 1, ch) + 1.0, kept[slot][1] + 1.0, 1e-6)


# -- whole models -----------------------------------------------------------------------------------------------------

def make_runner(folder, dtype, pages=40, page_size=16, max_requests=4, execution="eager"):
    from runtime.engine import load_model, ModelRunner
    return ModelRunner(load_model(folder, dtype=dtype), n_pages=pages, page_size=page_size, max_requests=max_requests, execution=execution)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_layers_one_by_one_and_a_whole_prompt(folders, name, dtype):
    from runtime.engine import StepEntry
    cfg, w = P.read_folder(folders[name])
    tokens = random_tokens(3, 45, cfg["vocab"])
    layers = []
    want = P.forward(cfg, w, tokens, layers)
    runner = make_runner(folders[name], dtype)
    seen = {}
    runner.layer_tap = lambda i, x: seen.__setitem__(i, x.float().cpu().numpy().reshape(len(tokens), cfg["streams"], -1).sum(axis=1))
    runner.create("r")
    got = runner.step([StepEntry("r", tokens, list(range(len(tokens))))]).cpu().numpy()
    for i, x in enumerate(layers):
        assert_close(seen[i], x, dtype, f"the sum of the streams after layer {i}")
    assert_close(got, want, dtype, "whole prompt")


@pytest.mark.parametrize("execution", ["eager", "graph"])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_then_tokens_one_by_one_and_portions_down_to_two_tokens(folders, name, dtype, execution):
    from runtime.engine import StepEntry
    V = CONFIGS[name]["vocab"]
    tokens = random_tokens(4, 150, V)
    want = plain_logits(folders[name], tokens)
    runner = make_runner(folders[name], dtype, execution=execution)
    runner.create("d")
    got = [runner.step([StepEntry("d", tokens[:97], list(range(97)))]).cpu().numpy()]
    got += [runner.step([StepEntry("d", [t], [0])]).cpu().numpy() for t in tokens[97:]]      # a long run of single tokens
    assert_close(np.concatenate(got), want, dtype, "prompt, then decoded")
    runner.release("d")
    runner.create("c")                                     # the same slot and pages once more, now in portions
    at, got = 0, []
    for n in [2, 3, 1, 2, 17, 2, 16, 31, 1, 5, 2, 33, 2, 100]:
        n = min(n, len(tokens) - at)
        got.append(runner.step([StepEntry("c", tokens[at:at + n], list(range(n)))]).cpu().numpy())
        at += n
    assert at == len(tokens)
    assert_close(np.concatenate(got), want, dtype, "portions")
    runner.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_portion_beside_another_request(folders, dtype):
    from runtime.engine import StepEntry
    name = "a"
    V = CONFIGS[name]["vocab"]
    long, other = random_tokens(31, 700, V), random_tokens(32, 300, V)
    runner = make_runner(folders[name], dtype, pages=70)
    runner.create("l"); runner.create("o")
    got = [runner.step([StepEntry("l", long[:100], list(range(100)))]).cpu().numpy()]
    out = runner.step([StepEntry("l", long[100:], list(range(600))), StepEntry("o", other, list(range(300)))]).cpu().numpy()
    assert_close(np.concatenate([got[0], out[:600]]), plain_logits(folders[name], long), dtype, "the long one")
    assert_close(out[600:], plain_logits(folders[name], other), dtype, "the second request")


@pytest.mark.parametrize("name, dtype, execution", [("b", "float32", "graph"), ("a", "bfloat16", "graph"), ("s", "float32", "eager"), ("n", "float32", "graph")])
def test_long_decoding_from_the_first_token(folders, name, dtype, execution):
    """A request decoded one token at a time from its very first token, over a dozen pages, beside a second request that
    joins late and leaves early (its slot and pages go back while the first goes on)."""
    from runtime.engine import StepEntry
    V = CONFIGS[name]["vocab"]
    first, second = random_tokens(61, 200, V), random_tokens(62, 40, V)
    runner = make_runner(folders[name], dtype, pages=24, execution=execution)
    runner.create("x")
    got, got2 = [], []
    for i, t in enumerate(first):
        entries = [StepEntry("x", [t], [0])]
        j = i - 50
        if j == 0:
            runner.create("y")
        if 0 <= j < len(second):
            entries.append(StepEntry("y", [second[j]], [0]))
        out = runner.step(entries).cpu().numpy()
        got.append(out[:1])
        if len(entries) == 2:
            got2.append(out[1:])
        if j == len(second) - 1:
            runner.release("y")
    assert_close(np.concatenate(got), plain_logits(folders[name], first), dtype, "decoded from the first token")
    assert_close(np.concatenate(got2), plain_logits(folders[name], second), dtype, "the late one")
    runner.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_prompt_of_thousands_of_tokens_then_single_tokens(tmp_path, dtype, no_gemv):
    """Long enough that the rule's chunks take several launches (one call's operands wait in a bounded memory), that the
    attention of a decoded token is split along its keys and merged by the output projection, and that a window of a
    thousand keys has passed; with the first tokens still in the state."""
    from guduzen_models import attention, config, delta, latent
    from runtime.engine import StepEntry
    from runtime.kernels import ops
    cfg = config(150, 192, 2, 12.0, 1e-5, [attention(6, 3, 64, 64, 0.125, 1000, ff=160), delta(3, 1, 64, 48, 4), latent(3, 32, 24, 96, 64, 0.2, ff=96),
                                           attention(6, 3, 64, 64, 0.125, None, kv_from=0)])
    cfg["layers"][3]["mixer"]["mask"] = {"size": 1400}
    folder = write_folder(tmp_path / "m", cfg, 91, sharp=True, ranks=(20, 24))
    n = ops.CHANNEL_SLAB * 16 + 140
    tokens = random_tokens(17, n + 8, cfg["vocab"])
    want = plain_logits(folder, tokens)
    merged = []
    plain_merge = ops.gemm_merged
    runner = make_runner(folder, dtype, pages=-(-len(tokens) // 16) + 2)
    runner.create("r")
    places = list(range(5)) + list(range(990, 1010)) + list(range(1390, 1410)) + list(range(n - 40, n))
    got = [runner.step([StepEntry("r", tokens[:n], places)]).cpu().numpy()]
    try:
        ops.gemm_merged = lambda *a, **k: (merged.append(1), plain_merge(*a, **k))[1]
        got += [runner.step([StepEntry("r", [t], [0])]).cpu().numpy() for t in tokens[n:]]
    finally:
        ops.gemm_merged = plain_merge
    assert dtype == "float32" or merged, "no output projection merged the split keys: the test does not test it"
    assert_close(np.concatenate(got), want[places + list(range(n, n + 8))], dtype, "a long prompt and what follows")


def mixed(V, seed, lengths=(70, 33, 120, 9, 64, 97, 40, 130), live_at_once=4):
    """Up to `live_at_once` live requests: portions of some beside single tokens of others; requests end and new ones
    start on the pages and state slots they gave back; one request sits out some steps."""
    rng = np.random.default_rng(seed)
    seqs = {f"m{i}": random_tokens(seed * 100 + i, n, V) for i, n in enumerate(lengths)}
    waiting, live, fed, trace, step = list(seqs), [], {}, Trace(), 0
    while waiting or live:
        while waiting and len(live) < live_at_once:
            rid = waiting.pop(0); live.append(rid); fed[rid] = 0
        entries, ending = [], []
        for rid in list(live):
            remaining = len(seqs[rid]) - fed[rid]
            if rid == live[0] and step % 5 == 3 and len(live) > 1:
                continue
            if remaining > 12:
                n = max(1, min(int(rng.choice([2, 3, 7, 16, 21, 40])), remaining - 8))
                want = [n - 1] if rng.random() < 0.5 else list(range(n))
            else:
                n, want = 1, [0]
            entries.append((rid, seqs[rid][fed[rid]:fed[rid] + n], want))
            fed[rid] += n
            if fed[rid] == len(seqs[rid]):
                ending.append(rid); live.remove(rid)
        if entries:
            trace.add(entries, end=ending)
        step += 1
    return trace, seqs


@pytest.mark.parametrize("execution", ["eager", "graph"])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mixed_batches_through_the_replay_program_with_pages_and_slots_used_again(folders, tmp_path, name, dtype, execution):
    from runtime.engine.replay import replay, MAX_LIVE
    V = CONFIGS[name]["vocab"]
    trace, seqs = mixed(V, seed=5)
    assert any(len(s["entries"]) == 4 for s in trace.steps)
    done = []
    runner = replay(folders[name], dtype, tmp_path, trace.peak, trace.lines(), echo=done.append, execution=execution)
    assert done == [f"done {i}" for i in range(len(trace.steps))]
    assert runner.cache.slots.n_slots == MAX_LIVE < len(seqs), "state slots must be used again"
    assert all(sum(-(-len(s) // 16) for s in seqs.values()) > g.pool.n_pages for g in runner.cache.groups), "pages must be used again"
    runner.cache.check()
    trace.check(folders[name], tmp_path, dtype, V, seqs, plain=plain_logits)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_batch_of_unequal_requests_gives_what_each_gives_alone(folders, dtype):
    from runtime.engine import StepEntry
    name = "w"
    V = CONFIGS[name]["vocab"]
    seqs = {k: random_tokens(50 + i, n, V) for i, (k, n) in enumerate({"a": 61, "b": 5, "c": 1, "d": 30}.items())}
    alone = {}
    for k, toks in seqs.items():
        runner = make_runner(folders[name], dtype)
        runner.create(k)
        alone[k] = runner.step([StepEntry(k, toks, list(range(len(toks))))]).cpu().numpy()
    runner = make_runner(folders[name], dtype, max_requests=4)
    for k in seqs:
        runner.create(k)
    got = runner.step([StepEntry(k, toks, list(range(len(toks)))) for k, toks in seqs.items()]).cpu().numpy()
    at = 0
    for k, toks in seqs.items():
        piece = got[at:at + len(toks)]
        at += len(toks)
        err = np.abs(piece - alone[k]).max() / np.abs(alone[k]).max()
        assert err < (1e-5 if dtype == "float32" else 2e-2), f"request {k} differs from itself alone by {err:.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys_a_window_s_edge_and_old_state_in_a_model_drawn_sharp(folders, dtype):
    """In the sharp model a query's result hangs on single keys and the rule's state keeps the first tokens.  The test first
    shows that a window one key longer or shorter (of the layer with the keys and of the one that reads them), the far keys
    of the latent layer, and a state that started late would each move the logits by many times the bound; then a prompt of
    many pages cut in the middle of a page and of a window, and tokens one by one over their borders, hold the bound."""
    from runtime.engine import StepEntry
    name = "s"
    cfg, w = P.read_folder(folders[name])
    tokens = random_tokens(9, 410, cfg["vocab"])
    want = plain_logits(folders[name], tokens)
    scale = np.abs(want).max()
    for i, delta in [(0, -1), (0, 1), (2, -1), (2, 1)]:
        off = json.loads(json.dumps(cfg))
        off["layers"][i]["mixer"]["mask"]["size"] += delta
        assert np.abs(P.forward(off, w, tokens)[60:] - want[60:]).max() > 1e-2 * scale, "a window one key off does not show"
    late = P.forward(cfg, w, tokens[150:])                       # without the first 150 tokens: far keys and old state are missing
    assert np.abs(late[-40:] - want[-40:]).max() > 0.05 * scale, "the first 150 tokens do not reach the last 40"
    only_state = dict(w, **{f"l{i}.mix.o": np.zeros_like(w[f"l{i}.mix.o"]) for i in (3,)})
    a, b = P.forward(cfg, only_state, tokens), P.forward(cfg, only_state, tokens[150:])
    assert np.abs(a[-40:] - b[-40:]).max() > 1e-3 * scale, "the state does not keep the first tokens"
    runner = make_runner(folders[name], dtype, pages=60)
    runner.create("f")
    got = [runner.step([StepEntry("f", tokens[:201], list(range(201)))]).cpu().numpy(),
           runner.step([StepEntry("f", tokens[201:340], list(range(139)))]).cpu().numpy()]
    got += [runner.step([StepEntry("f", [t], [0])]).cpu().numpy() for t in tokens[340:]]
    got = np.concatenate(got)
    assert_close(got, want, dtype, "far keys")
    assert_close(got[:3], want[:3], dtype, "the first tokens")
    assert_close(got[28:52], want[28:52], dtype, "where the windows fill up")


def test_a_window_gives_its_pages_back_and_its_readers_still_see_their_own(folders):
    """Model a: the layer with the keys looks back over 20, its reader over 37: the group keeps 37, whatever the owner's own
    window; a request far longer than the pool, in portions and single tokens."""
    from runtime.engine import StepEntry
    cfg = json.loads(json.dumps(CONFIGS["a"]))
    cfg["layers"] = cfg["layers"][:3]                            # (without the latent layer, which keeps every key)
    import tempfile, pathlib
    with tempfile.TemporaryDirectory() as tmp:
        folder = write_folder(pathlib.Path(tmp) / "m", cfg, 77, ranks=(10, 6))
        tokens = random_tokens(13, 330, cfg["vocab"])
        want = plain_logits(folder, tokens)
        runner = make_runner(folder, "float32", pages=8, page_size=16)       # 128 slots for 330 tokens
        assert len(runner.cache.groups) == 1
        runner.create("w")
        got, at = [], 0
        for n in [40, 33, 1, 1, 50, 2, 64, 1, 1, 1, 30, 60, 44, 1, 1]:
            got.append(runner.step([StepEntry("w", tokens[at:at + n], list(range(n)))]).cpu().numpy())
            at += n
        assert at == len(tokens)
        assert_close(np.concatenate(got), want, "float32", "windows that give pages back")
        assert runner.cache.groups[0].pool.used <= 4, "pages behind the longest window are given back"
        runner.cache.check()


@pytest.mark.parametrize("name, dtype, execution, overlap", [("a", "float32", "graph", True), ("a", "float32", "eager", False),
                                                             ("w", "bfloat16", "graph", True), ("n", "float32", "graph", True)])
def test_greedy_generation_through_the_scheduler(folders, name, dtype, execution, overlap):
    from runtime.engine.scheduler import Engine
    cfg, w = P.read_folder(folders[name])
    prompts = [random_tokens(70 + i, n, cfg["vocab"]) for i, n in enumerate([11, 3, 26, 1, 40])]
    engine = Engine.from_folder(folders[name], dtype=dtype, pages=24, page_size=16, execution=execution,
                                max_active=3, token_budget=24, prefill_chunk=9, overlap=overlap)
    got = engine.generate(prompts, max_new_tokens=10)
    for prompt, new in zip(prompts, got):
        assert len(new) == 10
        logits = P.forward(cfg, w, prompt + new)[len(prompt) - 1:-1]
        for row, token in zip(logits, new):       # every picked token is the plain model's best or within rounding of it, given the same past
            assert row.max() - row[token] < (1e-4 if dtype == "float32" else 0.05) * (row.max() - row.min())
    engine.runner.cache.check()
    assert not engine.runner.cache.lengths, "every request gave back what it held"


def test_fork_shares_pages_and_copies_state(folders):
    from runtime.engine import StepEntry
    name = "a"
    V = CONFIGS[name]["vocab"]
    base, one, two = random_tokens(1, 45, V), random_tokens(2, 12, V), random_tokens(3, 9, V)
    runner = make_runner(folders[name], "float32")
    runner.create("x")
    runner.step([StepEntry("x", base, [])])
    runner.fork("x", "y")
    got = runner.step([StepEntry("x", one, list(range(12))), StepEntry("y", two, list(range(9)))]).cpu().numpy()
    assert_close(got[:12], plain_logits(folders[name], base + one)[45:], "float32", "the source goes on")
    assert_close(got[12:], plain_logits(folders[name], base + two)[45:], "float32", "the fork goes its own way")


def test_command_line_serves_the_design(folders, tmp_path):
    """`python -m runtime` chooses the design by config.json: requests of a file against a folder, in float32, give the
    plain model's greedy tokens; the named configuration with random weights generates and reports its state slots."""
    import os, subprocess, sys
    from conftest import ROOT
    cfg, w = P.read_folder(folders["n"])
    requests = [{"key": "x", "prompt": [1, 2, 3, 4, 5, 6, 7], "max_new_tokens": 5}, {"key": "y", "prompt": [9], "max_new_tokens": 4}]
    (tmp_path / "requests.json").write_text(json.dumps(requests))
    env = dict(os.environ, PYTHONPATH=str(ROOT))
    proc = subprocess.run([sys.executable, "-m", "runtime", "--checkpoint", str(folders["n"]), "--dtype", "float32",
                           "--requests", str(tmp_path / "requests.json"), "--policy", "chunked", "--pages", "16",
                           "--token-budget", "6", "--prefill-chunk", "3"], capture_output=True, text=True, timeout=300, env=env, cwd=str(tmp_path))
    assert proc.returncode == 0, proc.stderr[-2000:]
    by_key = {r["key"]: r for r in json.loads(proc.stdout)["requests"]}
    assert by_key["x"]["generated"] == P.greedy(cfg, w, [1, 2, 3, 4, 5, 6, 7], 5)
    assert by_key["y"]["generated"] == P.greedy(cfg, w, [9], 4)
    proc = subprocess.run([sys.executable, "-m", "runtime", "--model", "guduzen-tiny", "--tokens", "5,6,7", "--max-new-tokens", "3",
                           "--overlap", "--report"], capture_output=True, text=True, timeout=300, env=env, cwd=str(tmp_path))
    assert proc.returncode == 0, proc.stderr[-2000:]
    out = json.loads(proc.stdout)
    assert out["weights"] == "random-guduzen-tiny" and len(out["requests"][0]["generated"]) == 3
    assert out["runner"]["replays"] >= 1 and out["runner"]["cache"][0]["resident_pages"] == 0


# -- configurations drawn at random -----------------------------------------------------------------------------------

def random_config(seed):
    """A configuration drawn at random: sizes, head counts, windows, whose keys a layer reads, streams, constants, the kinds
    of layers in an order of their own.  Every second draw has sizes of the order of a small real model."""
    from guduzen_models import attention, config, delta, latent
    rng = np.random.default_rng(1000 + seed)
    pick = lambda *values: values[int(rng.integers(len(values)))]
    big = seed % 2 == 1
    width = pick(192, 264, 384) if big else pick(40, 58, 72, 100)
    layers, owners = [], []
    for i in range(int(rng.integers(2, 7))):
        ff = pick(None, 256, 520) if big else pick(None, 24, 60, 100)
        kind = rng.random()
        if kind < 0.45:
            window = pick(None, 1, 2, 15, 16, 17, 33, 64, 90)
            scale = float(rng.uniform(0.05, 0.4))
            if owners and rng.random() < 0.5:
                j = pick(*owners)
                o = layers[j]["mixer"]
                layers.append(attention(o["kv_heads"] * pick(1, 2, 3), o["kv_heads"], o["dim"], o["vdim"], scale, window, kv_from=j, ff=ff))
            else:
                kv_heads, dim = pick(1, 2, 3), pick(64, 96, 128) if big else pick(6, 16, 24, 40)
                layers.append(attention(kv_heads * pick(1, 2, 4), kv_heads, dim, pick(dim, 32, 80) if big else pick(dim, 8, 12, 48), scale, window, ff=ff))
                owners.append(i)
        elif kind < 0.7:
            layers.append(latent(pick(1, 2, 5), pick(48, 64, 128) if big else pick(6, 12, 20), pick(32, 64, 96) if big else pick(5, 8, 24),
                                 pick(96, 160, 256, 264) if big else pick(9, 16, 40), pick(64, 100, 192) if big else pick(7, 16, 24), float(rng.uniform(0.1, 0.4)), ff=ff))
        else:
            kv_heads = pick(1, 2, 3)
            layers.append(delta(kv_heads * pick(1, 2, 3), kv_heads, pick(64, 96, 128) if big else pick(4, 10, 16, 33), pick(48, 64, 100) if big else pick(5, 8, 24),
                                pick(1, 2, 4, 7), ff=ff))
    ranks = (pick(16, 48, 96), pick(24, 64)) if big else (pick(3, 8, 17), pick(4, 9))
    return config(int(rng.integers(40, 700)), width, int(rng.integers(1, 7)), float(rng.uniform(6.0, 40.0)), pick(1e-5, 1e-6), layers), ranks


_DRAWN = {}


@pytest.fixture(scope="module")
def drawn(tmp_path_factory):
    """seed -> (configuration, folder, trace, sequences), made once for both dtypes."""
    def make(seed):
        if seed not in _DRAWN:
            cfg, ranks = random_config(seed)
            folder = write_folder(tmp_path_factory.mktemp(f"drawn{seed}") / "model", cfg, 300 + seed, sharp=seed % 3 == 0, ranks=ranks)
            trace, seqs = mixed(cfg["vocab"], seed=40 + seed, lengths=(70, 33, 90, 9, 48) if seed % 2 else (70, 33, 120, 9, 64, 97))
            _DRAWN[seed] = (cfg, folder, trace, seqs)
        return _DRAWN[seed]
    return make


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random_in_mixed_batches(drawn, tmp_path, seed, dtype):
    from runtime.engine.replay import replay
    cfg, folder, trace, seqs = drawn(seed)
    done = []
    runner = replay(folder, dtype, tmp_path / "out", trace.peak, trace.lines(), echo=done.append, execution="graph" if seed % 2 else "eager")
    assert done == [f"done {i}" for i in range(len(trace.steps))]
    runner.cache.check()
    trace.check(folder, tmp_path / "out", dtype, cfg["vocab"], seqs, plain=plain_logits)
