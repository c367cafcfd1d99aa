"""The Mapedra decoder on the GPU against the plain implementation (tests/plain_mapedra.py): every mechanism alone through
its kernels, then the engine whole, token by token, in portions down to two tokens, in mixed batches on reused pages and
slots, long decoding, and greedy generation through the scheduler. The configurations are made here
(tests/mapedra_tiny.py) and differ from each other in every size."""
import io
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_mapedra as plain
from mapedra_tiny import CONFIGS, STDS, make_mapedra_folder
from replay_tools import collect, mixed, portions, prefill_then_decode, round_up, to_lines, whole

pytestmark = pytest.mark.gpu

F32_BOUND = 2e-5        # of the logits' scale: float32 against float64, sums in other orders
BF16_BOUND = 0.06       # of the logits' scale: what the format costs on these models; a fault costs far more
F = torch.float64
_models = {}


def model_for(tmp_path_factory, which):
    if which not in _models:
        folder = make_mapedra_folder(tmp_path_factory.mktemp(f"mapedra_{which}"), which)
        _models[which] = (folder, plain.read_config(folder), plain.read_tensors(folder))
    return _models[which]


def tokens_for(seed, count, vocab):
    return np.random.default_rng(seed).integers(0, vocab, size=count).tolist()


def row_errors(got, want):
    difference = got - want
    difference = difference - difference.mean(-1, keepdims=True)
    return np.sqrt((difference ** 2).mean(-1)) / np.sqrt(((want - want.mean(-1, keepdims=True)) ** 2).mean())


def run_trace(folder, dtype, steps, out_dir, max_tokens, max_requests=4, **options):
    from microllm_rocm_amd.engine import Engine
    from microllm_rocm_amd.engine.replay import replay
    engine = Engine.from_folder(folder, dtype=dtype, max_tokens=max_tokens, max_requests=max_requests, **options)
    report = io.StringIO()
    replay(engine, io.StringIO(to_lines(steps)), str(out_dir), report)
    assert report.getvalue().split() == [word for step in steps for word in ("done", str(step["step"]))]
    engine.cache.check()
    assert not engine.cache.requests and all(free == group.pool.num_pages for free, group in zip(engine.cache.free_pages(), engine.cache.groups))
    return engine


_plain_runs = {}


def plain_run(config, weights, tokens):
    """Logits, the residual stream after every layer, and every position's sensitivity: how far the plain implementation
    itself, run in 32-bit, lies from its 64-bit run there, over twice its median (at least 1). A sublayer's result is
    divided by its root mean square, part by part, before it joins the stream; where a part nearly cancels, any format's
    error is divided by the same small number, in the plain run as in the engine."""
    key = (id(weights), tuple(tokens))
    if key not in _plain_runs:
        streams = []
        logits = plain.forward(config, weights, tokens, layers_out=streams).numpy()
        plain.F = torch.float32
        try:
            single = row_errors(plain.forward(config, weights, tokens).double().numpy(), logits)
        finally:
            plain.F = torch.float64
        sensitivity = np.maximum(1.0, single / (2.0 * np.median(single)))
        _plain_runs[key] = (logits, torch.stack(streams).numpy(), sensitivity)
    return _plain_runs[key]


def within_bound(errors, dtype):
    return errors.max() < (F32_BOUND if dtype == "float32" else BF16_BOUND)


def check_against_plain(steps, out_dir, requests, config, weights, dtype):
    got = collect(steps, str(out_dir), config["vocab"])
    for rid, tokens in requests.items():
        want, _, sensitivity = plain_run(config, weights, tokens)
        places = sorted(place for (request, place) in got if request == rid)
        assert places, f"no logits came back for {rid}"
        errors = row_errors(np.stack([got[(rid, place)] for place in places]), want[places]) / sensitivity[places]
        assert within_bound(errors, dtype), f"{rid}: position {places[int(errors.argmax())]} is off by {errors.max():.3g} of the scale"


def device(array, dtype=torch.float32):
    return torch.as_tensor(np.asarray(array), dtype=dtype).cuda().contiguous()


def as_bf16(array):
    return torch.as_tensor(np.asarray(array), dtype=torch.float32).to(torch.bfloat16).to(torch.float64).numpy()


def t64(array):
    return torch.as_tensor(np.asarray(array), dtype=F)


# ---- mechanisms alone -------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width,groups", [(64, 4), (50, 1), (96, 16), (21, 3), (2048, 2), (5120, 4), (30, 30), (8, 8), (4352, 17)])
def test_norm_in_groups_of_what_joins_the_stream(width, groups):
    """``h + mult * N(delta) * w`` and the norm in groups of the sum, the sum as it is, or no output, in one kernel; partial
    sums; chosen rows; one part far larger than the others, which must not touch them."""
    from microllm_rocm_amd.ops import kernels
    rng = np.random.default_rng(width)
    h, delta = rng.normal(size=(6, width)) * 3, rng.normal(size=(6, width)) * 5
    delta[:, :width // groups] *= 1e4
    after, weight = rng.normal(size=width) + 1, rng.normal(size=width) + 1
    joined = t64(h) + 0.7 * plain.grouped_rms(t64(delta), groups, 1e-5) * t64(after)
    want = (plain.grouped_rms(joined, groups, 1e-4) * t64(weight)).numpy()
    for parts in (delta, np.stack([delta * 0.25, delta * 0.75])):
        stream = device(h)
        got = kernels.rms_norm_after(stream, device(parts), device(after), 1e-5, 0.7, device(weight), 1e-4, torch.float32, write_h=True, groups=groups)
        assert np.abs(got.cpu().numpy() - want).max() < 3e-5 * np.abs(want).max() and np.abs(stream.cpu().numpy() - joined.numpy()).max() < 3e-5
    stream = device(h)
    got = kernels.rms_norm_after(stream, device(delta), device(after), 1e-5, 0.7, None, 1.0, torch.bfloat16, write_h=True, groups=groups, raw=True)
    assert torch.equal(got, stream.to(torch.bfloat16)) and np.abs(stream.cpu().numpy() - joined.numpy()).max() < 3e-5
    stream = device(h)
    assert kernels.rms_norm_after(stream, device(delta), device(after), 1e-5, 0.7, None, 1.0, torch.float32, write_h=True, groups=groups) is None
    assert np.abs(stream.cpu().numpy() - joined.numpy()).max() < 3e-5
    chosen = device([4, 1], torch.int32)
    got = kernels.rms_norm_after(device(h), device(delta), device(after), 1e-5, 0.7, None, 1.0, torch.float32, rows=chosen, groups=groups, raw=True)
    assert np.abs(got.cpu().numpy() - joined.numpy()[[4, 1]]).max() < 3e-5
    got = kernels.rms_norm_after(device(h), None, None, 0.0, 1.0, device(weight), 1e-4, torch.float32, rows=chosen, groups=groups)
    assert np.abs(got.cpu().numpy() - (plain.grouped_rms(t64(h), groups, 1e-4) * t64(weight)).numpy()[[4, 1]]).max() < 3e-5 * np.abs(want).max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_norm_parts_whatever_delta_they_are_given(dtype):
    """The norm part with groups and the part that norms nothing, given no delta, a plain one, partial sums, or one that is
    still to be normed in the same parts or in others; all rows (the sum then stays in the stream) or some."""
    from microllm_rocm_amd.parts import PartSpec, Runtime, build_part
    rng = np.random.default_rng(5)
    width, eps = 48, 1e-5
    runtime = Runtime(dtype, torch.device("cuda:0"))
    norm = build_part("norm", PartSpec("rms_norm", {"size": width, "eps": eps, "groups": 4}, {"weight": "w"}), runtime)
    whole_norm = build_part("norm", PartSpec("rms_norm", {"size": width, "eps": eps}, {"weight": "w"}), runtime)
    nothing = build_part("norm", PartSpec("unnormed"), runtime)
    h, delta, w, v = rng.normal(size=(5, width)) * 2, rng.normal(size=(5, width)) * 3, rng.normal(size=width) + 1, rng.normal(size=width) + 1
    norm.bind({"w": device(w)})
    whole_norm.bind({"w": device(v)})
    assert norm.weight_then_factor() is None and whole_norm.weight_then_factor() is not None
    deltas = {
        "none": (None, t64(h)), "plain": (device(delta), t64(h) + t64(delta)),
        "parts": (device(np.stack([delta * 0.5, delta * 0.5])), t64(h) + t64(delta)),
        "groups": (norm.delayed(device(delta), 1.5), t64(h) + 1.5 * plain.grouped_rms(t64(delta), 4, eps) * t64(w)),
        "whole": (whole_norm.delayed(device(delta), 1.0), t64(h) + plain.rms(t64(delta), eps) * t64(v)),
    }
    bound = 2e-5 if dtype == torch.float32 else 0.01
    for name, (given, joined) in deltas.items():
        for part, want in ((norm, plain.grouped_rms(joined, 4, eps) * t64(w)), (whole_norm, plain.rms(joined, eps) * t64(v)), (nothing, joined)):
            stream = device(h)
            got = part.forward(stream, delta=given, write_h=True)
            assert got.dtype == dtype and np.abs(got.float().cpu().numpy() - want.numpy()).max() < bound * np.abs(want.numpy()).max(), name
            assert np.abs(stream.cpu().numpy() - joined.numpy()).max() < 2e-5, name
            stream = device(h)
            got = part.forward(stream, delta=given, write_h=False, rows=device([3, 0], torch.int32))
            assert np.abs(got.float().cpu().numpy() - want.numpy()[[3, 0]]).max() < bound * np.abs(want.numpy()).max(), name
            assert torch.equal(stream, device(h)), name


@pytest.mark.parametrize("rows,width,ff", [(1, 64, 40), (5, 96, 128), (16, 256, 48), (23, 96, 128), (64, 64, 40), (200, 96, 128), (300, 256, 512), (9, 50, 33)])
def test_feed_forward_gated_by_the_tanh_gelu(rows, width, ff):
    """Through every product a step may take: a few rows, up to 64, many, with both copies of the weights or the packed one
    alone, and float32."""
    from microllm_rocm_amd.parts import PartSpec, Runtime, build_part
    rng = np.random.default_rng(rows + ff)
    x = as_bf16(rng.normal(size=(rows, width)))
    names = {f"{role}_proj.weight": role for role in ("gate", "up", "down")}
    tensors = {"gate": as_bf16(rng.normal(size=(ff, width)) * 0.3), "up": as_bf16(rng.normal(size=(ff, width)) * 0.2), "down": as_bf16(rng.normal(size=(width, ff)) * 0.2)}
    want = plain.gated_gelu(t64(x), {f"m.{name}": t64(value) for name, value in tensors.items()}, "m").numpy()
    for dtype, keep, bound in ((torch.float32, True, 1e-5), (torch.bfloat16, True, 0.01), (torch.bfloat16, False, 0.01)):
        if not keep and (width % 8 or ff % 8):
            continue
        part = build_part("ffn", PartSpec("swiglu", {"hidden_size": width, "intermediate_size": ff, "activation": "gelu_tanh"}, names),
                          Runtime(dtype, torch.device("cuda:0"), keep_plain_weights=keep))
        part.bind({name: device(value, dtype) for name, value in tensors.items()})
        got = part.forward(device(x, dtype), None)
        got = (got.sum(0) if got.dim() == 3 else got).float().cpu().numpy()
        assert np.abs(got - want).max() < bound * np.abs(want).max(), (dtype, keep)


@pytest.mark.parametrize("dim,width,layers,layer", [(8, 64, 4, 3), (7, 50, 3, 0), (96, 96, 2, 1), (33, 128, 5, 2)])
@pytest.mark.parametrize("rows", [1, 11, 16, 40, 130])
def test_side_vector_of_a_token(dim, width, layers, layer, rows):
    from microllm_rocm_amd.parts import PartSpec, Runtime, build_part
    rng = np.random.default_rng(dim + rows)
    vocab = 29
    x, ids = as_bf16(rng.normal(size=(rows, width))), rng.integers(0, vocab, size=rows)
    tensors = {"side.embed": as_bf16(rng.normal(size=(vocab, layers * dim))), f"l{layer}.side.gate": as_bf16(rng.normal(size=(dim, width)) * 0.3),
               f"l{layer}.side.proj": as_bf16(rng.normal(size=(width, dim)))}
    want = plain.token_side_input(t64(x), {name: t64(value) for name, value in tensors.items()}, layer, dim, torch.as_tensor(ids)).numpy()
    names = {"table": "side.embed", "gate": f"l{layer}.side.gate", "proj": f"l{layer}.side.proj"}
    for dtype, bound in ((torch.float32, 1e-5), (torch.bfloat16, 0.01)):
        part = build_part("ffn", PartSpec("token_side_input", {"hidden_size": width, "vocab_size": vocab, "dim": dim, "table_columns": layers * dim,
                                                               "column_at": layer * dim}, names), Runtime(dtype, torch.device("cuda:0")))
        part.bind({name: device(value, dtype) for name, value in tensors.items()})
        got = part.forward(device(x, dtype), SimpleNamespace(tokens=device(ids, torch.int32)))
        got = (got.sum(0) if got.dim() == 3 else got).cpu().numpy()
        assert np.abs(got - want).max() < bound * np.abs(want).max(), dtype


def test_side_gate_of_an_id_outside_the_table():
    from microllm_rocm_amd.ops import kernels
    z, table = device(np.ones((4, 6))), device(np.ones((3, 12)))
    got = kernels.token_side_gate(z, table, 6, device([2, 3, -1, 0], torch.int32), torch.float32)
    assert torch.isnan(got[1:3]).all() and torch.isfinite(got[[0, 3]]).all()
    weight = kernels.pack_weight(device(np.ones((6, 16)), torch.bfloat16))
    got = kernels.gemm_skinny_side(device(np.ones((4, 16)), torch.bfloat16), weight, 6, table, 6, device([2, 3, -1, 0], torch.int32))
    assert torch.isnan(got[1:3]).all() and torch.isfinite(got[[0, 3]]).all()


def capped(q, k, v, gate, scale, cap, portions_of, mfma, norm_weights=None, inv_freq=None, eps=1e-5, value_norm=True, page_size=16, window=0):
    """The engine's kernels on one request: the norms of queries, keys and values, their rotation, keys and values into
    pages that are scattered and out of order, and the attention with capped scores and a gate a channel, in the given
    portions: plain pages and the kernel that takes a wave a token and head (float32), or the tiled pages and the MFMA
    kernels (bfloat16)."""
    from microllm_rocm_amd.cache.layout import key_page_shape, value_page_shape
    from microllm_rocm_amd.ops import kernels
    from microllm_rocm_amd.parts.attention import QueryTilePlanner
    n, heads, dim = q.shape
    kv_heads, vdim = k.shape[1], v.shape[2]
    dtype = torch.bfloat16 if mfma else torch.float32
    blocks = -(-n // page_size)
    pages = [2 + 3 * block for block in reversed(range(blocks))]
    count = 3 * blocks + 2
    table = device([pages], torch.int32)
    q_weight = k_weight = None
    if norm_weights is not None:
        q_weight, k_weight = device(norm_weights[0]), device(norm_weights[1])
    rates = device(inv_freq, torch.float64) if inv_freq is not None else None
    if mfma:
        k_pages = torch.zeros(key_page_shape(count, kv_heads, page_size, dim), dtype=dtype, device="cuda")
        v_pages = torch.zeros(value_page_shape(count, kv_heads, page_size, dim), dtype=dtype, device="cuda")
        planner = QueryTilePlanner(bool(window))
    else:
        k_pages = torch.full((count, page_size, kv_heads, dim), 1e4, dtype=dtype, device="cuda")      # what is not this request's must not count
        v_pages = torch.full((count, page_size, kv_heads, vdim), 1e4, dtype=dtype, device="cuda")
    out, first = [], 0
    for portion in portions_of:
        portion = min(portion, n - first)
        if portion <= 0:
            break
        rows = slice(first, first + portion)
        parts = [q[rows].reshape(portion, -1), k[rows].reshape(portion, -1), v[rows].reshape(portion, -1), gate[rows].reshape(portion, -1)]
        positions = np.arange(first, first + portion)
        slots = [pages[p // page_size] * page_size + p % page_size for p in positions]
        pos, seq_of_token = device(positions, torch.int32), device(np.zeros(portion), torch.int32)
        proj = device(np.concatenate(parts, axis=1))
        queries = kernels.qk_norm_store(proj, q_weight, k_weight, eps, pos, device(slots, torch.int32), 0.0, 1, k_pages, v_pages, heads,
                                        kv_heads, dim, vdim, dtype, tiled_page_size=page_size if mfma else 0, normed=norm_weights is not None,
                                        cos_sin=kernels.rope_table(pos, rates) if rates is not None else None,
                                        further_columns=heads * vdim, values_normed=value_norm)
        gates = proj[:, proj.shape[1] - heads * vdim:]
        if mfma:
            host = SimpleNamespace(counts=[portion], cu=np.array([0, portion]), starts=[first], totals=[first + portion],
                                   single_tokens_only=portion == 1, n_tokens=portion, n_seqs=1, page_size=page_size)
            ctx = SimpleNamespace(max_count=portion, planned_total=first + portion, max_total=first + portion, n_tokens=portion,
                                  seq_of_token=seq_of_token, positions=pos, fixed=False, host=host, tokens=pos, planned={})
            arrays, values = planner.plan(host)
            plan = SimpleNamespace(**values, **{name: device(array, torch.int32) for name, array in arrays.items()})
            ctx.plan_of = lambda _planner: plan
            view = SimpleNamespace(block_table=table, page_size=page_size)
            found = torch.empty((portion, heads * dim), dtype=dtype, device="cuda")
            extras = kernels.AttentionExtras(None, None, 1.0, gate=gates, softcap=cap or 0.0)
            kernels.paged_attention(queries, k_pages, v_pages, view, ctx, scale, window, heads, kv_heads, dim, planner=planner, extras=extras, out=found)
        else:
            found = kernels.bias_attention(queries, k_pages, v_pages, table, seq_of_token, pos, None, None, scale, 1.0, heads, kv_heads, dim,
                                           vdim, gate=gates, softcap=cap or 0.0, window=window)
        out.append(found.float().cpu().numpy().reshape(portion, heads, vdim))
        first += portion
    return np.concatenate(out)


def plain_capped(q, k, v, gate, scale, cap, norm_weights=None, turn=None, eps=1e-5, value_norm=True):
    q, k, v = t64(q), t64(k), t64(v)
    if norm_weights is not None:
        q, k = plain.rms(q, eps) * t64(norm_weights[0]), plain.rms(k, eps) * t64(norm_weights[1])
    if turn is not None:
        q, k = turn(q), turn(k)
    if value_norm:
        v = plain.rms(v, eps)
    return (plain.attend_capped(q, k, v, scale, cap) * torch.sigmoid(t64(gate))).numpy()


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,cap,rot,n,mfma", [
    (4, 2, 24, 16, 3.0, 8, 70, False), (3, 1, 10, 6, 50.0, 10, 33, False), (5, 5, 6, 11, None, 0, 130, False),
    (1, 1, 128, 200, 7.0, 64, 150, False), (6, 2, 16, 16, 3.0, 8, 150, True), (8, 2, 32, 32, 50.0, 32, 300, True),
    (2, 1, 48, 48, 2.0, 16, 270, True), (4, 4, 96, 96, 10.0, 64, 300, True), (1, 1, 128, 128, None, 128, 70, True),
    (20, 1, 64, 64, 5.0, 32, 280, True), (2, 2, 160, 160, 4.0, 96, 200, True), (2, 1, 256, 256, 30.0, 0, 150, True)])
def test_attention_with_capped_scores_and_a_gate_a_channel(heads, kv_heads, dim, vdim, cap, rot, n, mfma):
    """Random queries, keys, values and gates; whole, decoded, in portions of two and of sizes that cut pages anywhere. The
    queries are large, so that scores reach far into the cap."""
    rng = np.random.default_rng(dim + n)
    q, k, v = (as_bf16(rng.normal(size=shape)) for shape in ((n, heads, dim), (n, kv_heads, dim), (n, kv_heads, vdim)))
    gate = rng.normal(size=(n, heads, vdim)) * 2
    weights = ((rng.normal(size=dim) + 1) * 2, rng.normal(size=dim) + 1)
    base, positions = 1000.0, torch.arange(n)
    bands = {"factor": 3.0, "low": 1.0, "high": 6.0, "original": 50.0}
    # the kernels turn channel i with i + rot / 2: handed channels that are already in that order
    order = np.concatenate([np.arange(0, rot, 2), np.arange(1, rot, 2), np.arange(rot, dim)]).astype(int)
    turn = (lambda a: plain.turn_neighbours(a, positions, base, rot, bands)) if rot else None
    want = plain_capped(q, k, v, gate, 0.3, cap, weights, turn)
    inv_freq = plain.rates(base, rot, bands) if rot else None
    bound = 0.03 * np.abs(want).max() if mfma else 3e-5
    mine = (q[..., order], k[..., order], v, gate, 0.3, cap)
    weights = (weights[0][order], weights[1][order])
    got = capped(*mine, [n], mfma, weights, inv_freq)
    assert np.abs(got - want).max() < bound
    for portions_of in ([max(n - 40, 2)] + [1] * 40, [2] * (n // 2 + 1), [1] * 5 + [3, 16, 1, 2, 31, 129, 1, 1, 500]):
        again = capped(*mine, portions_of, mfma, weights, inv_freq)
        assert np.abs(again - want).max() < bound, portions_of
        if not mfma:
            assert np.array_equal(again, got), portions_of      # a row does not depend on how the request was cut


@pytest.mark.parametrize("mfma", [False, True])
def test_long_contexts_split_over_workgroups(mfma):
    """Decoding with so many keys that the decode kernel splits them and joins the splits: caps and gates a channel survive
    the join; the first token of all and a key at a split's edge stand out in turn."""
    rng = np.random.default_rng(8)
    n, heads, dim = 2100, 2, 16
    q, k = as_bf16(rng.normal(size=(n, heads, dim)) * 0.1), as_bf16(rng.normal(size=(n, 1, dim)) * 0.1)
    v, gate = as_bf16(rng.normal(size=(n, 1, dim))), rng.normal(size=(n, heads, dim)) * 2
    k[:, 0, 3] = 0.0
    for key in (0, 511, 512, 1055, n - 1):
        sharp_q, sharp_k = q.copy(), k.copy()
        sharp_q[n - 1, 0] = 0.0
        sharp_q[n - 1, 0, 3] = 5.0
        sharp_k[key, 0, 3] = 5.0
        scores = t64(sharp_k[:, 0]) @ t64(sharp_q[n - 1]).T * 2.0
        weights = torch.softmax(20.0 * torch.tanh(scores / 20.0), dim=0)
        want = (weights.T @ plain.rms(t64(v[:, 0]), 1e-5) * torch.sigmoid(t64(gate[n - 1]))).numpy()
        got = capped(sharp_q, sharp_k, v, gate, 2.0, 20.0, [n - 1, 1], mfma)
        assert np.abs(got[n - 1] - want).max() < (0.03 if mfma else 1e-4), key


@pytest.mark.parametrize("mfma", [False, True])
def test_the_cap_bounds_a_score_that_stands_out(mfma):
    """A key whose score would be 400 gets the cap: among ``m`` keys of score 0 it weighs ``e^c / (e^c + m - 1)``, and the one
    of -400 ``e^-c / (e^c + ...)``; without a cap it takes everything. Wherever the key lies: the first token, at page
    borders, far away, the query itself; in a prompt, decoded, and in portions of two."""
    rng = np.random.default_rng(1)
    n, heads, dim, cap = 300, 2, 16, 3.0
    v = as_bf16(rng.normal(size=(n, 1, dim)))
    gate = np.full((n, heads, dim), 30.0)
    bound = 0.03 if mfma else 1e-4
    for query in (n - 1, 200, 128, 64, 17):
        for key, sign in ((0, 1), (15, -1), (16, 1), (query, 1), (query - 1, -1)):
            q, k = np.zeros((n, heads, dim)), np.zeros((n, 1, dim))
            q[query, :, 3], k[key, 0, 3] = 20.0, 20.0 * sign
            values = plain.rms(t64(v[:query + 1, 0]), 1e-5)
            weights = torch.ones(query + 1, dtype=F)
            weights[key] = np.exp(sign * cap)
            want = ((weights / weights.sum())[:, None] * values).sum(0).numpy()
            pairs = min(70 if query == 128 else 8, (query + 1) // 2)
            in_twos = ([query + 1 - 2 * pairs] if query + 1 > 2 * pairs else []) + [2] * pairs
            for portions_of in ([query + 1], [query, 1], in_twos):
                got = capped(q[:query + 1], k[:query + 1], v[:query + 1], gate[:query + 1], 1.0, cap, portions_of, mfma)
                assert np.abs(got[query, 0] - want).max() < bound, (query, key, portions_of)
        q, k = np.zeros((n, heads, dim)), np.zeros((n, 1, dim))
        q[query, :, 3], k[5, 0, 3] = 20.0, 20.0
        got = capped(q[:query + 1], k[:query + 1], v[:query + 1], gate[:query + 1], 1.0, None, [query, 1], mfma)
        assert np.abs(got[query, 0] - plain.rms(t64(v[5, 0]), 1e-5).numpy()).max() < bound


@pytest.mark.parametrize("mfma", [False, True])
def test_a_cap_beside_a_window(mfma):
    """The cap is a parameter of the attention, not of this design: under a window of 20 the standing-out key counts just
    inside the edge and not just outside it."""
    rng = np.random.default_rng(2)
    n, heads, dim, cap, window = 150, 2, 32, 8.0, 20
    v, gate = as_bf16(rng.normal(size=(n, 1, dim))), np.full((n, heads, dim), 30.0)
    for query in (149, 90, 33):
        for key in (query - window + 1, query - window):
            q, k = np.zeros((n, heads, dim)), np.zeros((n, 1, dim))
            q[query, :, 3], k[key, 0, 3] = 10.0, 10.0
            first = query - window + 1
            weights = torch.ones(window, dtype=F)
            if key >= first:
                weights[key - first] = np.exp(cap * np.tanh(100.0 / cap))
            want = ((weights / weights.sum())[:, None] * plain.rms(t64(v[first:query + 1, 0]), 1e-5)).sum(0).numpy()
            for portions_of in ([query + 1], [query, 1]):
                got = capped(q[:query + 1], k[:query + 1], v[:query + 1], gate[:query + 1], 1.0, cap, portions_of, mfma, window=window)
                assert np.abs(got[query, 0] - want).max() < (0.03 if mfma else 1e-4), (query, key)


def lightened(q, k, v, gate, weight, decay, portions_of, eps=1e-5, dtype=torch.float32, chunks_from=1 << 30):
    """Lightning attention's kernels on one request in the given portions: SiLU, the walk with one decay a head (from
    ``chunks_from`` tokens on the recurrence in chunks), one norm over all heads and the sigmoid gate; the state carried in
    a slot."""
    from microllm_rocm_amd.ops import kernels
    n, heads, dim = q.shape
    vdim = v.shape[2]
    keys, values = heads * dim, heads * vdim
    state = torch.zeros((3, heads, dim, vdim), device="cuda")
    state[0] = state[2] = 1e4       # other requests' slots
    decay_row = device(np.repeat(np.asarray(decay, dtype=np.float64), dim))
    out, first = [], 0
    for portion in portions_of:
        portion = min(portion, n - first)
        if portion <= 0:
            break
        rows = slice(first, first + portion)
        proj = device(np.concatenate([a[rows].reshape(portion, -1) for a in (q, k, v, gate)], axis=1))
        cu, slots = device([0, portion], torch.int32), device([1], torch.int32)
        if portion >= chunks_from:
            walked = kernels.gla_chunks(proj, 0, keys, 2 * keys, device(decay), state, cu, slots, 1, heads, dim, vdim, 1.0, silu_inputs=True)
        else:
            long_portions = portion >= 8
            if long_portions:
                kernels.gla_silu(proj, 0, 2 * keys + values)
            walked = kernels.gla_scan(proj, 0, keys, 2 * keys, decay_row, state, cu, slots, 1, heads, dim, vdim, 1.0, long_portions=long_portions,
                                      silu_inputs=not long_portions)
        found = kernels.gla_gate(walked, proj, 2 * keys + values, device(weight), eps, heads, vdim, 1.0, dtype, heads_together=True)
        out.append(found.float().cpu().numpy())
        first += portion
    assert float(state[0].min()) == 1e4 and float(state[2].max()) == 1e4
    return np.concatenate(out)


@pytest.mark.parametrize("heads,dim,vdim,n", [(3, 12, 10, 70), (1, 9, 14, 40), (4, 8, 8, 90), (2, 40, 7, 50), (1, 128, 12, 35), (6, 32, 32, 300), (2, 300, 20, 30)])
def test_lightning_attention(heads, dim, vdim, n):
    rng = np.random.default_rng(heads * dim)
    q, k, v, gate = (rng.normal(size=shape) for shape in ((n, heads, dim), (n, heads, dim), (n, heads, vdim), (n, heads, vdim)))
    v[:, 0] *= 30.0         # one head much larger than the others: the norm is over all of them together
    weight = rng.normal(size=heads * vdim) + 1
    decay = [1.0, 0.0, 0.7, 0.97, 0.998046875, 0.5][:heads]
    walked = plain.retain(plain.silu(t64(q)), plain.silu(t64(k)), plain.silu(t64(v)), decay).reshape(n, -1)
    want = (plain.rms(walked, 1e-5) * t64(weight) * torch.sigmoid(t64(gate).reshape(n, -1))).numpy()
    got = lightened(q, k, v, gate, weight, decay, [n])
    assert np.abs(got - want).max() < 3e-5 * np.abs(want).max()
    for portions_of in ([max(n - 30, 2)] + [1] * 30, [2] * (n // 2 + 1), [1] * 5 + [3, 16, 1, 2, 31, 129, 1, 1, 500]):
        again = lightened(q, k, v, gate, weight, decay, portions_of)
        assert np.abs(again - want).max() < 3e-5 * np.abs(want).max(), portions_of
        if dim <= 128:
            chunked = lightened(q, k, v, gate, weight, decay, portions_of, chunks_from=2)
            assert np.abs(chunked - want).max() < 3e-5 * np.abs(want).max(), portions_of
    rounded = lightened(q, k, v, gate, weight, decay, [n], dtype=torch.bfloat16)
    assert np.abs(rounded - want).max() < 0.01 * np.abs(want).max()


def test_a_far_token_stays_in_the_state():
    """A decay of one forgets nothing: the first token's value, written along one key channel that later keys hardly touch
    (SiLU of a very negative number), is read back by the last query 400 tokens on; with a decay of 1/2 nothing of it is
    left."""
    n, dim, vdim = 401, 16, 8
    rng = np.random.default_rng(5)
    q, k = np.full((n, 2, dim), -40.0), rng.normal(size=(n, 2, dim))
    v, gate = rng.normal(size=(n, 2, vdim)), np.full((n, 2, vdim), 30.0)
    k[:, :, 3] = -60.0
    k[0, :, 3] = 4.0
    q[n - 1, :, 3] = 1.0
    first = plain.silu(t64(v[0, 0])) * float(plain.silu(t64(4.0)) * plain.silu(t64(1.0)))
    together = torch.cat([first, torch.zeros(vdim, dtype=F)])
    want = plain.rms(together, 1e-5).numpy()
    for portions_of in ([n], [n - 1, 1], [100, 2, 2, 297]):
        for chunks_from in (1 << 30, 2):
            got = lightened(q, k, v, gate, np.ones(2 * vdim), [1.0, 0.5], portions_of, chunks_from=chunks_from)
            assert np.abs(got[n - 1] - want).max() < 1e-4, portions_of


@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 128), (3, 20, 70), (1, 128, 16), (4, 100, 33)])
def test_chunks_of_several_requests(heads, dim, vdim):
    """Requests of unequal lengths in one step (one without tokens, ends on a chunk's edge, one before and one past it), each
    from a state of its own, against each request's tokens one after the other; no SiLU and a factor on the read-out."""
    from microllm_rocm_amd.ops import kernels
    rng = np.random.default_rng(dim)
    lengths, slots = [130, 1, 0, 64, 63, 65, 200], [3, 0, 7, 5, 1, 2, 6]
    cu = np.concatenate([[0], np.cumsum(lengths)])
    n, keys, values = cu[-1], heads * dim, heads * vdim
    q, k, v = (rng.normal(size=(n, heads, size)) for size in (dim, dim, vdim))
    decay = [0.99, 0.0, 1.0, 0.6][:heads]
    before = rng.normal(size=(8, heads, dim, vdim))
    proj = device(np.concatenate([a.reshape(n, -1) for a in (q, k, v)], axis=1))
    state = device(before)
    got = kernels.gla_chunks(proj, 0, keys, 2 * keys, device(decay), state, device(cu, torch.int32), device(slots, torch.int32), len(lengths),
                             heads, dim, vdim, 0.5).cpu().numpy().reshape(n, heads, vdim)
    walked = device(before)
    kernels.gla_scan(proj, 0, keys, 2 * keys, device(np.repeat(decay, dim)), walked, device(cu, torch.int32), device(slots, torch.int32),
                     len(lengths), heads, dim, vdim, 0.5, long_portions=True)
    assert (state - walked).abs().max() < 2e-5 * walked.abs().max() and torch.equal(state[4], device(before)[4])
    assert torch.equal(state[7], device(before)[7])        # the request that brought nothing
    for index, slot in enumerate(slots):
        rows = slice(cu[index], cu[index + 1])
        want = 0.5 * plain.retain(t64(q[rows]), t64(k[rows]), t64(v[rows]), decay, t64(before[slot])).numpy()
        if lengths[index]:
            assert np.abs(got[rows] - want).max() < 2e-5 * np.abs(want).max(), index


# ---- the engine ---------------------------------------------------------------------------------------------------
def single_layer_folder(tmp_path, layer_of, which, with_mlp):
    """A model of one layer: the mixer ``layer_of`` of configuration ``which``, with its own feed-forward or none."""
    import dataclasses
    from microllm_rocm_amd.weights import write_model_folder
    source = CONFIGS[which]
    layer = source.layers[layer_of]
    if not with_mlp:
        layer = dataclasses.replace(layer, mlp=None)
    config = dataclasses.replace(source, layers=(layer,))
    folder = os.path.join(str(tmp_path), f"one_{which}_{layer_of}")
    write_model_folder(folder, config, 50 + layer_of, dtype=torch.bfloat16, stds=STDS)
    return folder


@pytest.mark.parametrize("which,layer_of,with_mlp", [("A", 0, False), ("A", 1, True), ("A", 2, False), ("A", 3, True), ("B", 0, False),
                                                     ("B", 1, True), ("B", 2, False), ("B", 3, True), ("C", 0, True), ("C", 1, False),
                                                     ("C", 2, True), ("C", 3, False)])
def test_every_mixer_as_a_model_of_one_layer(tmp_path, which, layer_of, with_mlp):
    tokens = tokens_for(layer_of, 90, CONFIGS[which].vocab)
    folder = single_layer_folder(tmp_path, layer_of, which, with_mlp)
    config, weights = plain.read_config(folder), plain.read_tensors(folder)
    for dtype in ("float32", "bfloat16"):
        for name, steps in (("whole", whole({"r": tokens})), ("decode", prefill_then_decode("r", tokens, tail=40)),
                            ("portions", portions("r", tokens, [2, 5, 1, 17]))):
            run_trace(folder, dtype, steps, tmp_path / f"{dtype}_{name}", max_tokens=128)
            check_against_plain(steps, tmp_path / f"{dtype}_{name}", {"r": tokens}, config, weights, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_whole_decode_and_portions(tmp_path_factory, tmp_path, which, dtype):
    folder, config, weights = model_for(tmp_path_factory, which)
    requests = {"long": tokens_for(1, 150, config["vocab"]), "short": tokens_for(2, 37, config["vocab"]), "one": tokens_for(3, 1, config["vocab"])}
    run_trace(folder, dtype, whole(requests), tmp_path / "whole", max_tokens=256)
    check_against_plain(whole(requests), tmp_path / "whole", requests, config, weights, dtype)
    for rid, tail in (("long", 70), ("short", 34)):      # the decoded tokens cross pages' edges
        steps = prefill_then_decode(rid, requests[rid], tail=tail)
        run_trace(folder, dtype, steps, tmp_path / f"decode_{rid}", max_tokens=round_up(len(requests[rid]), 64))
        check_against_plain(steps, tmp_path / f"decode_{rid}", {rid: requests[rid]}, config, weights, dtype)
    for sizes in ([2], [3, 16, 1, 2, 31], [64, 2, 17], [131, 2, 7]):
        steps = portions("long", requests["long"], sizes)
        run_trace(folder, dtype, steps, tmp_path / f"portions_{sizes[0]}", max_tokens=192)
        check_against_plain(steps, tmp_path / f"portions_{sizes[0]}", {"long": requests["long"]}, config, weights, dtype)
    steps = portions("short", requests["short"], [1])       # from its first token on, one token a step
    run_trace(folder, dtype, steps, tmp_path / "one_by_one", max_tokens=64)
    check_against_plain(steps, tmp_path / "one_by_one", {"short": requests["short"]}, config, weights, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_mixed_batches_on_reused_pages_and_slots(tmp_path_factory, tmp_path, which, dtype):
    folder, config, weights = model_for(tmp_path_factory, which)
    lengths = [90, 41, 130, 2, 67, 25, 110, 58]
    requests = {f"r{index}": tokens_for(10 + index, length, config["vocab"]) for index, length in enumerate(lengths)}
    steps, peak = mixed(requests, seed=4, max_live=3, decode_tail=12, max_portion=23)
    engine = run_trace(folder, dtype, steps, tmp_path / "mixed", max_tokens=peak, max_requests=3)
    assert all(group.pool.total_taken > group.pool.num_pages for group in engine.cache.groups)      # pages were used again
    assert engine.cache.slots.total_taken > 3                                                        # and so were slots
    check_against_plain(steps, tmp_path / "mixed", requests, config, weights, dtype)


def test_a_row_does_not_depend_on_the_batch(tmp_path_factory):
    """Float32: a request's logits are the same bits alone and beside others."""
    from microllm_rocm_amd.engine import Engine, StepEntry
    folder, config, _ = model_for(tmp_path_factory, "A")
    engine = Engine.from_folder(folder, dtype="float32", max_tokens=512, max_requests=4)
    a, b, c = (tokens_for(seed, length, config["vocab"]) for seed, length in ((1, 45), (2, 20), (3, 33)))
    engine.open("alone")
    alone = [engine.step([StepEntry("alone", a[:30], list(range(30)))]).clone(), engine.step([StepEntry("alone", a[30:44], list(range(14)))]).clone(),
             engine.step([StepEntry("alone", a[44:], [0])]).clone()]
    engine.close("alone")
    for name in "abc":
        engine.open(name)
    first = engine.step([StepEntry("b", b[:7], []), StepEntry("a", a[:30], list(range(30))), StepEntry("c", c[:2], [])])
    second = engine.step([StepEntry("a", a[30:44], list(range(14))), StepEntry("c", c[2:], []), StepEntry("b", b[7:8], [])])
    third = engine.step([StepEntry("b", b[8:9], [0]), StepEntry("a", a[44:], [0])])
    assert torch.equal(torch.cat(alone), torch.cat([first, second, third[1:]]))


@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_long_decoding_through_graphs(tmp_path_factory, which):
    """A short prompt, then 140 tokens one by one (steps replayed from captured graphs, state carried in slots, cached
    rows crossing many pages), two requests at once with unequal lengths."""
    from microllm_rocm_amd.engine import Engine, StepEntry
    folder, config, weights = model_for(tmp_path_factory, which)
    sequences = {"x": tokens_for(7, 150, config["vocab"]), "y": tokens_for(8, 160, config["vocab"])}
    starts = {"x": 10, "y": 3}
    for dtype in ("float32", "bfloat16"):
        engine = Engine.from_folder(folder, dtype=dtype, max_tokens=512, max_requests=2)
        assert engine.use_graphs
        rows = {name: [] for name in sequences}
        for name in sequences:
            engine.open(name)
        logits = engine.step([StepEntry(name, sequences[name][:starts[name]], [starts[name] - 1]) for name in sequences])
        for index, name in enumerate(sequences):
            rows[name].append(logits[index].cpu().numpy())
        for offset in range(140):
            entries = [StepEntry(name, [sequences[name][starts[name] + offset]], [0]) for name in sequences]
            logits = engine.step(entries)
            for index, name in enumerate(sequences):
                rows[name].append(logits[index].cpu().numpy())
        assert engine.graph_replays >= 139
        for name, tokens in sequences.items():
            want, _, sensitivity = plain_run(config, weights, tokens[:starts[name] + 140])
            want, sensitivity = want[starts[name] - 1:], sensitivity[starts[name] - 1:]
            assert within_bound(row_errors(np.stack(rows[name]), want) / sensitivity, dtype), (dtype, name)


@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_greedy_generation_through_the_scheduler(tmp_path_factory, which):
    from microllm_rocm_amd import Engine, GenerationConfig, generate, generate_serial
    folder, config, weights = model_for(tmp_path_factory, which)
    prompts = [tokens_for(20 + index, length, config["vocab"]) for index, length in enumerate((5, 31, 12))]
    expected = [prompt + plain.generate_greedy(config, weights, prompt, 10) for prompt in prompts]
    engine = Engine.from_folder(folder, dtype="float32", max_tokens=512, max_requests=4)
    got = generate(engine, prompts, GenerationConfig(max_new_tokens=10, temperature=0.0), prefill_chunk=7, max_batched_tokens=16)
    assert got == expected
    assert generate_serial(engine, prompts[0], GenerationConfig(max_new_tokens=10, temperature=0.0)) == expected[0]
    bf16 = Engine.from_folder(folder, dtype="bfloat16", max_tokens=512, max_requests=4)
    close = generate(bf16, prompts, GenerationConfig(max_new_tokens=10, temperature=0.0), prefill_chunk=7)
    assert [len(tokens) for tokens in close] == [len(tokens) for tokens in expected]
    assert all(tokens[:len(prompt)] == prompt for tokens, prompt in zip(close, prompts))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_residual_stream_after_every_layer(tmp_path_factory, tmp_path, which, dtype):
    folder, config, weights = model_for(tmp_path_factory, which)
    tokens = tokens_for(5, 19, config["vocab"])
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": tokens, "want": list(range(19))}], "end": ["q"]}]
    from microllm_rocm_amd.engine import Engine
    from microllm_rocm_amd.engine.replay import replay
    engine = Engine.from_folder(folder, dtype=dtype, max_tokens=64, max_requests=1)
    replay(engine, io.StringIO(to_lines(steps)), str(tmp_path), io.StringIO(), dump_layers=True)
    streams = plain_run(config, weights, tokens)[1]
    got = np.fromfile(os.path.join(str(tmp_path), "0.layers.f32"), dtype="<f4").reshape(len(config["layers"]), 19, config["width"])
    for layer in range(len(config["layers"])):
        bound = 1e-4 if dtype == "float32" else 0.1
        assert np.abs(got[layer] - streams[layer]).max() < bound * np.abs(streams[layer]).max(), layer


def test_one_copy_of_the_weights(tmp_path_factory, tmp_path):
    """The packed copy alone: every product through this package's own kernels, the gated gelu in the tiled one's epilogue."""
    folder, config, weights = model_for(tmp_path_factory, "C")
    tokens = tokens_for(9, 180, config["vocab"])
    steps = portions("p", tokens, [120, 30, 17, 1])
    run_trace(folder, "bfloat16", steps, tmp_path, max_tokens=192, weight_copies="packed")
    check_against_plain(steps, tmp_path, {"p": tokens}, config, weights, "bfloat16")


def test_command_line_and_trace_runner_as_programs(tmp_path_factory, tmp_path, capsys):
    import json
    import subprocess
    import sys
    from microllm_rocm_amd.cli import hf_infer
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder, config, weights = model_for(tmp_path_factory, "A")
    prompt = tokens_for(31, 13, config["vocab"])
    expected = plain.generate_greedy(config, weights, prompt, 6)
    base = ["--model", folder, "--tokens", ",".join(map(str, prompt)), "--new-tokens", "6", "--dtype", "float32"]

    def run(*more):
        capsys.readouterr()
        assert hf_infer.main(base + list(more)) == 0
        return json.loads(capsys.readouterr().out.strip().splitlines()[-1])

    report = run()
    assert report["architecture"] == "Mapedra" and report["generated_tokens"] == expected
    for more in (["--use-cache", "false"], ["--cache-prefill-mode", "token"], ["--batch", "2", "--batch-argmax-mode", "host"]):
        assert run(*more)["generated_tokens"] == expected, more
    sampled = [run("--temperature", "0.9", "--sample-top-k", "5", "--seed", "7")["generated_tokens"] for _ in range(2)]
    assert sampled[0] == sampled[1] and len(sampled[0]) == 6
    steps = portions("p", prompt + expected, [5, 2, 1])
    result = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out",
                             str(tmp_path / "trace"), "--max-tokens", "64"], input=to_lines(steps), capture_output=True, text=True, timeout=300)
    assert result.returncode == 0, result.stderr
    assert [line for line in result.stdout.splitlines() if line.startswith("done")] == [f"done {step['step']}" for step in steps]
    check_against_plain(steps, tmp_path / "trace", {"p": prompt + expected}, config, weights, "float32")
