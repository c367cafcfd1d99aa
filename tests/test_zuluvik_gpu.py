"""The Zuluvik decoder on the GPU against the plain implementation (tests/plain_zuluvik.py): every mechanism alone
through its kernels, then the engine whole, token by token, in portions down to two tokens, in mixed batches on reused
pages and slots, long decoding, and greedy generation through the scheduler. The configurations are made here
(tests/zuluvik_tiny.py) and differ from each other in every size."""
import io
import math
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_zuluvik as plain
from replay_tools import collect, mixed, portions, prefill_then_decode, round_up, to_lines, whole
from zuluvik_tiny import CONFIGS, STDS, make_zuluvik_folder, without_choice

pytestmark = pytest.mark.gpu

F32_BOUND = 2e-5        # of the logits' scale: float32 against float64, sums in other orders
BF16_BOUND = 0.06       # of the logits' scale: what the format costs on these models; a fault costs far more
F = torch.float64
_models = {}


def model_for(tmp_path_factory, which, dtype="float32"):
    """The model ``which``; for a bfloat16 engine the same model with every token sent to all places
    (``zuluvik_tiny.without_choice`` says why)."""
    choice = dtype == "float32"
    if (which, choice) not in _models:
        folder = make_zuluvik_folder(tmp_path_factory.mktemp(f"zuluvik_{which}"), which, choice)
        _models[(which, choice)] = (folder, plain.read_config(folder), plain.read_tensors(folder))
    return _models[(which, choice)]


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
    itself, run in 32-bit, lies from its 64-bit run there, over twice its median (at least 1). The difference of a head's two
    maps is divided by its own root mean square; where it nearly cancels, any format's error is divided by the same small
    number, in the plain run as in the engine."""
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


def check_rows(got, want, sensitivity, dtype, what):
    errors = row_errors(got, want) / sensitivity
    bound = F32_BOUND if dtype == "float32" else BF16_BOUND
    assert errors.max() < bound, f"{what}: row {int(errors.argmax())} is off by {errors.max():.3g} of the scale"


def check_against_plain(steps, out_dir, requests, config, weights, dtype):
    got = collect(steps, str(out_dir), config["vocab"])
    for rid, tokens in requests.items():
        want, _, sensitivity = plain_run(config, weights, tokens)
        places = sorted(place for (request, place) in got if request == rid)
        assert places, f"no logits came back for {rid}"
        check_rows(np.stack([got[(rid, place)] for place in places]), want[places], sensitivity[places], dtype, rid)


def device(array, dtype=torch.float32):
    return torch.as_tensor(np.asarray(array), dtype=dtype).cuda().contiguous()


def as_bf16(array):
    return torch.as_tensor(np.asarray(array), dtype=torch.float32).to(torch.bfloat16).to(torch.float64).numpy()


def t64(array):
    return torch.as_tensor(np.asarray(array), dtype=F)


# ---- mechanisms alone -------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width", [64, 50, 7, 1000, 5000])
@pytest.mark.parametrize("shapes", [(0,), (3,), (0, 2), (5, 9, 0), (1, 0, 12, 2)])
def test_norm_of_the_stream_and_several_sources(width, shapes):
    """The stream plus tensors in places of their own (0: one tensor, n: n parts of it), normed: what the layer before left
    when both of its sublayers read one norm."""
    from microllm_rocm_amd.ops import kernels
    rng = np.random.default_rng(width + len(shapes))
    h, weight = rng.normal(size=(6, width)) * 3, rng.normal(size=width) + 1
    sources = [rng.normal(size=(6, width) if parts == 0 else (parts, 6, width)) for parts in shapes]
    joined = t64(h) + sum(t64(source) if source.ndim == 2 else t64(source).sum(0) for source in sources)
    want = (plain.rms(joined, 1e-5) * t64(weight)).numpy()
    for dtype, bound in ((torch.float32, 3e-5), (torch.bfloat16, 0.005 * np.abs(want).max())):
        stream = device(h)
        got = kernels.rms_norm_sum(stream, device(weight), 1e-5, dtype, [device(source) for source in sources], write_h=True)
        assert np.abs(got.float().cpu().numpy() - want).max() < bound and np.abs(stream.cpu().numpy() - joined.numpy()).max() < 3e-5
        stream = device(h)
        got = kernels.rms_norm_sum(stream, device(weight), 1e-5, dtype, [device(source) for source in sources], rows=device([4, 1], torch.int32))
        assert np.abs(got.float().cpu().numpy() - want[[4, 1]]).max() < bound
        assert np.array_equal(stream.cpu().numpy(), device(h).cpu().numpy())


def test_several_sources_before_any_norm():
    """A summed delta before what takes no several sources: a norm in groups, no norm, more sources than the kernel takes, and
    rows that join the stream between layers."""
    from microllm_rocm_amd.parts import PartSpec, Runtime, build_part
    from microllm_rocm_amd.parts.model import Model
    from microllm_rocm_amd.parts.norm import SummedDelta
    rng = np.random.default_rng(3)
    h, weight = rng.normal(size=(5, 24)), rng.normal(size=24) + 1
    arrays = [rng.normal(size=(5, 24)), rng.normal(size=(3, 5, 24))]
    joined = t64(h) + t64(arrays[0]) + t64(arrays[1]).sum(0)
    runtime = Runtime(torch.float32, torch.device("cuda:0"))

    def norm(kind, **params):
        part = build_part("norm", PartSpec(kind, {"size": 24, "eps": 1e-5, **params}, {"weight": "w"}), runtime)
        if kind != "unnormed":
            part.bind({"w": device(weight)})
        return part

    delta = SummedDelta([device(array) for array in arrays])
    assert np.abs(delta.resolved().cpu().numpy() - (joined - t64(h)).numpy()).max() < 1e-5
    whole_norm, runs = plain.rms(joined, 1e-5) * t64(weight), plain.rms(joined.view(5, 4, 6), 1e-5).view(5, 24) * t64(weight)
    for kind, params, want in (("rms_norm", {}, whole_norm), ("rms_norm", {"groups": 4}, runs), ("unnormed", {}, joined)):
        stream = device(h)
        got = norm(kind, **params).forward(stream, delta=delta, write_h=True)
        assert np.abs(got.cpu().numpy() - want.numpy()).max() < 2e-5 and np.abs(stream.cpu().numpy() - joined.numpy()).max() < 1e-5, kind
    stream = device(h)
    taken = Model._add_to_stream(stream, delta, device(arrays[0]))
    assert len(taken.sources) == 3 and len(delta.sources) == 2
    many = taken
    for _ in range(3):
        many = many.with_extra(device(arrays[0]))
    want = plain.rms(joined + 4 * t64(arrays[0]), 1e-5) * t64(weight)
    assert np.abs(norm("rms_norm").forward(stream, delta=many, write_h=False).cpu().numpy() - want.numpy()).max() < 2e-5


class Pages:
    """One request's keys and values in scattered pages that are out of order and hold other requests' data, as plain pages
    (float32, or bfloat16 without the MFMA kernels) or as the MFMA kernels' tiles."""

    def __init__(self, n, kv_heads, key_dim, value_dim, mfma, dtype, page_size=16):
        from microllm_rocm_amd.cache.layout import key_page_shape, value_page_shape
        from microllm_rocm_amd.parts.attention import QueryTilePlanner
        blocks = -(-n // page_size)
        self.pages = [2 + 3 * block for block in reversed(range(blocks))]
        count = 3 * blocks + 2
        self.page_size, self.mfma, self.dtype = page_size, mfma, dtype
        self.table = device([self.pages], torch.int32)
        self.planner = QueryTilePlanner(False)
        if mfma:
            self.k = torch.full(key_page_shape(count, kv_heads, page_size, key_dim), 99.0, dtype=dtype, device="cuda")
            self.v = torch.full(value_page_shape(count, kv_heads, page_size, value_dim), 99.0, dtype=dtype, device="cuda")
        else:
            self.k = torch.full((count, page_size, kv_heads, key_dim), 1e4, dtype=dtype, device="cuda")
            self.v = torch.full((count, page_size, kv_heads, value_dim), 1e4, dtype=dtype, device="cuda")

    def step(self, first, portion):
        """The step's metadata for ``portion`` tokens from position ``first`` on."""
        positions = np.arange(first, first + portion)
        slots = [self.pages[p // self.page_size] * self.page_size + p % self.page_size for p in positions]
        pos = device(positions, torch.int32)
        host = SimpleNamespace(counts=[portion], cu=np.array([0, portion]), starts=[first], totals=[first + portion],
                               single_tokens_only=portion == 1, n_tokens=portion, n_seqs=1, page_size=self.page_size)
        arrays, values = self.planner.plan(host)
        plan = SimpleNamespace(**values, **{name: device(array, torch.int32) for name, array in arrays.items()})
        ctx = SimpleNamespace(max_count=portion, planned_total=first + portion, max_total=first + portion, n_tokens=portion, n_seqs=1,
                              seq_of_token=device(np.zeros(portion), torch.int32), positions=pos, fixed=False, tokens=pos,
                              cu_tokens=device([0, portion], torch.int32), slots=device([1], torch.int32), plan_of=lambda _planner: plan)
        return ctx, SimpleNamespace(block_table=self.table, page_size=self.page_size), device(slots, torch.int32)


def in_portions(n, portions_of):
    first = 0
    for portion in portions_of:
        portion = min(portion, n - first)
        if portion <= 0:
            return
        yield first, portion
        first += portion


def differenced(q, k, v, taps, scale, factor, diff, portions_of, mfma, eps=1e-5, dtype=None):
    """The differential attention's kernels on one request in the given portions: the convolution over time continued from
    a slot, queries and keys of both maps and values into their pages, the maps' attention, their difference with its norm.
    ``q`` ``[n, H, 2, d]``, ``k`` ``[n, G, 2, d]``, ``v`` ``[n, G, dv]``; ``taps`` ``[columns, t]``."""
    from microllm_rocm_amd.ops import kernels
    n, heads, _, dim = q.shape
    kv_heads, vdim = v.shape[1], v.shape[2]
    dtype = dtype or (torch.bfloat16 if mfma else torch.float32)
    kept_dim = round_up(max(2 * dim, vdim), 16) if mfma else 0
    store = Pages(n, kv_heads, kept_dim or 2 * dim, kept_dim or vdim, mfma, dtype)
    columns, n_taps = taps.shape
    kept = torch.zeros((3, n_taps - 1, columns), device="cuda") if n_taps > 1 else None
    if kept is not None:
        kept[0] = kept[2] = 1e4       # other requests' slots
    out = []
    for first, portion in in_portions(n, portions_of):
        rows = slice(first, first + portion)
        proj = device(np.concatenate([part[rows].reshape(portion, -1) for part in (q, k, v)], axis=1))
        ctx, view, slots = store.step(first, portion)
        convolution = kernels.Convolution(device(taps), kept, ctx.seq_of_token, ctx.cu_tokens, ctx.slots)
        queries = kernels.qk_norm_store(proj, None, None, eps, ctx.positions, slots, 0.0, 1, store.k, store.v, 2 * heads, kv_heads, 2 * dim,
                                        vdim, dtype, tiled_page_size=16 if mfma else 0, normed=False, stored_dim=kept_dim, maps=2,
                                        convolution=convolution)
        if kept is not None:
            kernels.conv_keep(proj, 0, kept, ctx.cu_tokens, ctx.slots, 1)
        if mfma:
            combined = kernels.HeadDifference(vdim, factor, eps, 1.0 - diff)
            found = kernels.paged_attention(queries, store.k, store.v, view, ctx, scale, 0, 2 * heads, kv_heads, kept_dim, planner=store.planner,
                                            extras=kernels.AttentionExtras(difference=combined))
        else:
            maps = torch.empty((portion, 2 * heads * vdim), dtype=torch.float32, device="cuda")
            kernels.bias_attention(queries, store.k, store.v, view.block_table, ctx.seq_of_token, ctx.positions, None, None, scale, 1.0,
                                   2 * heads, kv_heads, 2 * dim, vdim, out=maps)
            found = kernels.attention_difference(maps, heads, vdim, factor, eps, 1.0 - diff, dtype)
        out.append(found.float().cpu().numpy().reshape(portion, heads, vdim))
    if kept is not None:
        assert float(kept[0].min()) == 1e4 and float(kept[2].max()) == 1e4
    return np.concatenate(out)


def plain_differenced(q, k, v, taps, scale, factor, diff, eps=1e-5):
    n, heads, _, dim = q.shape
    kv_heads, vdim = v.shape[1], v.shape[2]
    flat = plain.convolve(torch.cat([t64(part).reshape(n, -1) for part in (q, k, v)], dim=1), t64(taps))
    q = flat[:, :2 * heads * dim].view(n, heads, 2, dim)
    k = flat[:, 2 * heads * dim:2 * (heads + kv_heads) * dim].view(n, kv_heads, 2, dim)
    v = flat[:, 2 * (heads + kv_heads) * dim:].view(n, kv_heads, vdim)
    first, second = (plain.attend(q[:, :, m], k[:, :, m], v, scale) for m in (0, 1))
    return (plain.rms(first - factor * second, eps) * (1.0 - diff)).numpy()


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,n_taps,n,mfma", [
    (4, 2, 8, 16, 3, 70, False), (3, 1, 5, 6, 1, 33, False), (5, 5, 6, 11, 7, 90, False), (1, 1, 64, 200, 2, 150, False),
    (4, 2, 8, 16, 4, 150, True), (8, 2, 16, 32, 3, 300, True), (3, 3, 6, 10, 2, 140, True), (2, 1, 16, 40, 5, 270, True),
    (6, 2, 40, 24, 1, 200, True), (20, 1, 32, 64, 3, 280, True), (1, 1, 128, 256, 3, 150, True)])
def test_differential_attention(heads, kv_heads, dim, vdim, n_taps, n, mfma):
    """Random projections; whole, decoded, in portions of two and of sizes that cut pages and the convolution's reach
    anywhere."""
    rng = np.random.default_rng(dim + vdim)
    q, k, v = (as_bf16(rng.normal(size=shape)) for shape in ((n, heads, 2, dim), (n, kv_heads, 2, dim), (n, kv_heads, vdim)))
    taps = rng.normal(size=(2 * (heads + kv_heads) * dim + kv_heads * vdim, n_taps)) * 0.5
    taps[:, -1] += 1.0
    want = plain_differenced(q, k, v, taps, dim ** -0.5, 0.3, 0.6)
    bound = 0.06 * np.abs(want).max() if mfma else 5e-5
    got = differenced(q, k, v, taps, dim ** -0.5, 0.3, 0.6, [n], mfma)
    assert np.abs(got - want).max() < bound
    for portions_of in ([max(n - 40, 2)] + [1] * 40, [2] * (n // 2 + 1), [1] * 5 + [3, 16, 1, 2, 31, 129, 1, 1, 500]):
        again = differenced(q, k, v, taps, dim ** -0.5, 0.3, 0.6, portions_of, mfma)
        assert np.abs(again - want).max() < bound, portions_of
        if not mfma:
            assert np.array_equal(again, got), portions_of      # a row does not depend on how the request was cut


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,n", [(2, 1, 16, 32, 1100), (3, 1, 24, 20, 5200)])
def test_difference_where_the_splits_meet(heads, kv_heads, dim, vdim, n):
    """Decoding over so many keys that they go to several workgroups, whose results meet in the kernel that combines the maps
    (two splits, and more than eight of them)."""
    from microllm_rocm_amd.ops import kernels
    assert kernels.decode_splits(1, kv_heads, n) == (2 if n == 1100 else 10)
    rng = np.random.default_rng(n)
    q, k, v = (as_bf16(rng.normal(size=shape)) for shape in ((n, heads, 2, dim), (n, kv_heads, 2, dim), (n, kv_heads, vdim)))
    q[n - 3:] *= 4.0        # the last queries single out a few keys
    taps = np.ones((2 * (heads + kv_heads) * dim + kv_heads * vdim, 1))
    got = differenced(q, k, v, taps, dim ** -0.5, 0.4, 0.6, [n - 3, 1, 1, 1], True)[n - 3:]
    for back, query in enumerate(range(n - 3, n)):
        maps = []
        for m in (0, 1):
            s = torch.einsum("hd,jhd->hj", t64(q[query, :, m]), t64(k[:query + 1, :, m]).repeat_interleave(heads // kv_heads, 1)) * dim ** -0.5
            maps.append(torch.einsum("hj,jhd->hd", torch.softmax(s, -1), t64(v[:query + 1]).repeat_interleave(heads // kv_heads, 1)))
        want = (plain.rms(maps[0] - 0.4 * maps[1], 1e-5) * 0.4).numpy()
        assert np.abs(got[back] - want).max() < 0.03 * np.abs(want).max(), query


def test_differential_attention_on_plain_pages_in_bfloat16():
    """The kernel for plain pages leaves float32 results of bfloat16 keys and values too."""
    rng = np.random.default_rng(8)
    n, heads, kv_heads, dim, vdim = 60, 4, 2, 8, 12
    q, k, v = (as_bf16(rng.normal(size=shape)) for shape in ((n, heads, 2, dim), (n, kv_heads, 2, dim), (n, kv_heads, vdim)))
    taps = np.concatenate([np.zeros((2 * (heads + kv_heads) * dim + kv_heads * vdim, 1)), np.ones((2 * (heads + kv_heads) * dim + kv_heads * vdim, 1))], 1)
    want = plain_differenced(q, k, v, taps, 0.3, 0.9, 0.6)
    got = differenced(q, k, v, taps, 0.3, 0.9, 0.6, [40, 1, 2, 17], False, dtype=torch.bfloat16)
    assert np.abs(got - want).max() < 0.01 * np.abs(want).max()      # nothing is rounded between the maps and their difference's norm


@pytest.mark.parametrize("mfma", [False, True])
def test_far_keys_of_one_map(mfma):
    """One map of a head looks at one key alone (their score stands out), the other map is even over all keys it sees: the
    head gives that key's value minus the mean's share, or with the maps exchanged the reverse, wherever the key lies (the
    first token, the edges of pages and of the kernel's tiles of keys, the query itself), in a prompt, decoded, and in
    portions of two."""
    rng = np.random.default_rng(4)
    n, heads, dim, vdim = 300, 2, 8, 16
    columns = 2 * (heads + 1) * dim + vdim
    taps = np.ones((columns, 1))
    v = as_bf16(rng.normal(size=(n, 1, vdim)))
    for query in (299, 160, 128, 64, 17):
        for key in sorted({0, 1, 15, 16, 63, 64, 127, query - 1, query}):
            if key > query:
                continue
            for sharp_map in (0, 1):
                q, k = np.zeros((n, heads, 2, dim)), np.zeros((n, 1, 2, dim))
                q[query, 0, sharp_map, 3] = 6.0
                k[key, 0, sharp_map, 3] = 6.0
                k[:, 0, 1 - sharp_map, 3] = 6.0         # what the other map would make of it: a map that reads its neighbour's keys shows
                q[query, 0, 1 - sharp_map, 3] = 0.0
                mean = v[:query + 1, 0].mean(0)
                other = v[key, 0]
                raw = (other - 0.5 * mean) if sharp_map == 0 else (mean - 0.5 * other)
                want = raw / math.sqrt((raw ** 2).mean() + 1e-5) * 0.25
                assert np.abs(plain_differenced(q[:query + 1], k[:query + 1], v[:query + 1], taps, 2.0, 0.5, 0.75)[query, 0] - want).max() < 1e-6
                pairs = min(8, (query + 1) // 2)
                in_twos = ([query + 1 - 2 * pairs] if query + 1 > 2 * pairs else []) + [2] * pairs
                for portions_of in ([query + 1], [query, 1], in_twos):
                    got = differenced(q[:query + 1], k[:query + 1], v[:query + 1], taps, 2.0, 0.5, 0.75, portions_of, mfma)
                    assert np.abs(got[query, 0] - want).max() < (0.02 if mfma else 1e-4), (query, key, sharp_map, portions_of)


@pytest.mark.parametrize("n_taps", [1, 2, 3, 6])
def test_the_convolution_across_cuts(n_taps):
    """A single token with everything zero before and after: what it leaves in the next ``taps - 1`` tokens, and in none
    after, however the request is cut (portions shorter than the taps included), and zeros before the first token."""
    from microllm_rocm_amd.ops import kernels
    n, at = 24, 9
    rng = np.random.default_rng(n_taps)
    dim, vdim = 4, 6
    columns = 2 * 2 * dim + vdim         # one head, one key/value head, two maps
    taps = rng.normal(size=(columns, n_taps))
    for impulse_at in (0, at, n - 1):
        u = np.zeros((n, columns))
        u[impulse_at] = rng.normal(size=columns)
        want = plain.convolve(t64(u), t64(taps)).numpy()
        for portions_of in ([n], [1] * n, [2] * n, [impulse_at + 1, 1, 1, 1, 30], [3, 1, 2, 5, 1, 1, 30]):
            store = Pages(n, 1, 2 * dim, vdim, False, torch.float32)
            kept = torch.zeros((2, n_taps - 1, columns), device="cuda") if n_taps > 1 else None
            queries = []
            for first, portion in in_portions(n, portions_of):
                proj = device(u[first:first + portion])
                ctx, _, slots = store.step(first, portion)
                queries.append(kernels.qk_norm_store(proj, None, None, 1e-5, ctx.positions, slots, 0.0, 1, store.k, store.v, 2, 1, 2 * dim, vdim,
                                                     torch.float32, normed=False, maps=2,
                                                     convolution=kernels.Convolution(device(taps), kept, ctx.seq_of_token, ctx.cu_tokens, ctx.slots)))
                if kept is not None:
                    kernels.conv_keep(proj, 0, kept, ctx.cu_tokens, ctx.slots, 1)
            q = torch.cat(queries).cpu().numpy().reshape(n, 2, 2 * dim)
            assert np.abs(q[:, 0, :dim] - want[:, :dim]).max() < 1e-6 and np.abs(q[:, 1, dim:] - want[:, dim:2 * dim]).max() < 1e-6, portions_of
            assert not q[:, 0, dim:].any() and not q[:, 1, :dim].any()       # a query meets its own map's keys alone
            place = [store.pages[p // 16] * 16 + p % 16 for p in range(n)]
            assert np.abs(store.k.cpu().numpy().reshape(-1, 2 * dim)[place] - want[:, 2 * dim:4 * dim]).max() < 1e-6
            assert np.abs(store.v.cpu().numpy().reshape(-1, vdim)[place] - want[:, 4 * dim:]).max() < 1e-6


def turned_and_normed(q, k, v, bias, rot, scale, portions_of, mfma, eps, normed=True):
    """The rotary attention's kernels on one request in the given portions: biases, the rotation, the norm of the turned
    queries and keys, padding to one width, the attention. ``rot`` as in a configuration (neighbours are paired: the channels
    of queries, keys and their biases come reordered, as the part reorders its weights' rows)."""
    from microllm_rocm_amd.ops import kernels
    n, heads, dim = q.shape
    kv_heads, vdim = v.shape[1], v.shape[2]
    dtype = torch.bfloat16 if mfma else torch.float32
    kept_dim = round_up(max(dim, vdim), 16) if mfma else 0
    store = Pages(n, kv_heads, kept_dim or dim, kept_dim or vdim, mfma, dtype)
    dims = rot["dims"]
    order = list(range(0, dims, 2)) + list(range(1, dims, 2)) + list(range(dims, dim))
    rates, magnitude = plain.yarn(rot["base"], dims, rot.get("scaling"))
    inv_freq = device(rates, torch.float64)
    q_bias, k_bias, v_bias = bias
    all_bias = device(np.concatenate([q_bias.reshape(heads, dim)[:, order].ravel(), k_bias.reshape(kv_heads, dim)[:, order].ravel(), v_bias]))
    out = []
    for first, portion in in_portions(n, portions_of):
        rows = slice(first, first + portion)
        proj = device(np.concatenate([q[rows][:, :, order].reshape(portion, -1), k[rows][:, :, order].reshape(portion, -1),
                                      v[rows].reshape(portion, -1)], axis=1))
        ctx, view, slots = store.step(first, portion)
        queries = kernels.qk_norm_store(proj, None, None, eps, ctx.positions, slots, 0.0, 1, store.k, store.v, heads, kv_heads, dim, vdim, dtype,
                                        tiled_page_size=16 if mfma else 0, bias=all_bias, normed=normed,
                                        cos_sin=kernels.rope_table(ctx.positions, inv_freq, magnitude), stored_dim=kept_dim, norm_turned=normed)
        if mfma:
            found = torch.empty((portion, heads * kept_dim), dtype=dtype, device="cuda")
            kernels.paged_attention(queries, store.k, store.v, view, ctx, scale, 0, heads, kv_heads, kept_dim, planner=store.planner,
                                    extras=kernels.AttentionExtras(), out=found)
            found = found.view(portion, heads, kept_dim)
            assert not found[:, :, vdim:].any()
            found = found[:, :, :vdim]
        else:
            found = kernels.bias_attention(queries, store.k, store.v, view.block_table, ctx.seq_of_token, ctx.positions, None, None, scale, 1.0,
                                           heads, kv_heads, dim, vdim).view(portion, heads, vdim)
        out.append(found.float().cpu().numpy())
    return np.concatenate(out)


def plain_turned(q, k, v, bias, rot, scale, eps):
    n, heads, dim = q.shape
    kv_heads, vdim = v.shape[1], v.shape[2]
    positions = torch.arange(n)
    q = plain.rms(plain.turn_neighbours(t64(q) + t64(bias[0]).view(heads, dim), positions, rot), eps)
    k = plain.rms(plain.turn_neighbours(t64(k) + t64(bias[1]).view(kv_heads, dim), positions, rot), eps)
    return plain.attend(q, k, t64(v) + t64(bias[2]).view(kv_heads, vdim), scale).numpy()


RAMP = dict(factor=8.0, original=64.0, fast=8.0, slow=0.5)


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot,n,mfma", [
    (4, 2, 24, 16, dict(base=100.0, dims=8, scaling=RAMP), 70, False), (3, 1, 10, 6, dict(base=77.0, dims=10), 33, False),
    (5, 5, 6, 11, dict(base=1e4, dims=2, scaling=RAMP), 130, False), (1, 1, 128, 200, dict(base=1e4, dims=64, scaling=RAMP), 150, False),
    (6, 2, 16, 16, dict(base=100.0, dims=8, scaling=RAMP), 150, True), (8, 2, 32, 24, dict(base=5e5, dims=32, scaling=RAMP), 300, True),
    (2, 1, 20, 48, dict(base=1e4, dims=16), 270, True), (4, 4, 96, 96, dict(base=1e4, dims=40, scaling=RAMP), 300, True),
    (1, 1, 128, 128, dict(base=1e4, dims=128, scaling=RAMP), 70, True), (32, 2, 64, 64, dict(base=1e6, dims=32, scaling=RAMP), 280, True)])
def test_norm_after_the_turn(heads, kv_heads, dim, vdim, rot, n, mfma):
    """Biases on queries, keys and values, a rotation whose magnitude is not one on part of the head, and then the norm over
    the whole head: taken before the turn, or of the turned part alone, the scores would be others. A large eps makes the
    order count also where the whole head turns."""
    rng = np.random.default_rng(dim + n)
    q, k, v = (as_bf16(rng.normal(size=shape)) for shape in ((n, heads, dim), (n, kv_heads, dim), (n, kv_heads, vdim)))
    bias = tuple(rng.normal(size=size) for size in (heads * dim, kv_heads * dim, kv_heads * vdim))
    for eps in (1e-5, 0.5):
        want = plain_turned(q, k, v, bias, rot, 0.5, eps)
        bound = 0.04 * np.abs(want).max() if mfma else 3e-5
        got = turned_and_normed(q, k, v, bias, rot, 0.5, [n], mfma, eps)
        assert np.abs(got - want).max() < bound
        for portions_of in ([max(n - 40, 2)] + [1] * 40, [2] * (n // 2 + 1), [1] * 5 + [3, 16, 1, 2, 31, 129, 1, 1, 500]):
            again = turned_and_normed(q, k, v, bias, rot, 0.5, portions_of, mfma, eps)
            assert np.abs(again - want).max() < bound, portions_of
            if not mfma:
                assert np.array_equal(again, got), portions_of


@pytest.mark.parametrize("mfma", [False, True])
def test_far_keys_of_the_rotary_attention(mfma):
    """The query and one key alone have what their scores are made of in channels that do not turn; that key takes all the
    weight wherever it lies, in a prompt, decoded and in portions of two."""
    rng = np.random.default_rng(6)
    n, heads, dim = 300, 2, 16
    rot = dict(base=1e4, dims=8, scaling=RAMP)
    v = as_bf16(rng.normal(size=(n, 1, dim)))
    bias = tuple(np.zeros(size) for size in (heads * dim, dim, dim))
    for query in (299, 200, 128, 64, 16):
        for key in sorted({0, 1, 15, 16, 63, 64, query - 1, query}):
            if key > query:
                continue
            q, k = as_bf16(rng.normal(size=(n, heads, dim)) * 0.1), as_bf16(rng.normal(size=(n, 1, dim)) * 0.1)
            k[:, 0, 12] = 0.0
            q[query, 0] = 0.0
            q[query, 0, 12] = 5.0
            k[key, 0] = 0.0
            k[key, 0, 12] = 5.0            # normed: 4 each; no other key has anything there
            want = plain_turned(q, k, v, bias, rot, 3.0, 1e-5)
            assert np.abs(want[query, 0] - v[key, 0]).max() < 1e-6
            pairs = min(8, (query + 1) // 2)
            in_twos = ([query + 1 - 2 * pairs] if query + 1 > 2 * pairs else []) + [2] * pairs
            for portions_of in ([query + 1], [query, 1], in_twos):
                got = turned_and_normed(q[:query + 1], k[:query + 1], v[:query + 1], bias, rot, 3.0, portions_of, mfma, 1e-5)
                assert np.abs(got[query, 0] - v[key, 0]).max() < (0.02 if mfma else 1e-4), (query, key, portions_of)


def test_table_with_a_magnitude():
    from microllm_rocm_amd.ops import kernels
    positions = np.array([0, 1, 7, 300, 100000])
    for scaling in (RAMP, None):
        rates, magnitude = plain.yarn(1e4, 16, scaling)
        got = kernels.rope_table(device(positions, torch.int32), device(rates, torch.float64), magnitude).cpu().numpy()
        angle = positions[:, None] * np.asarray(rates)[None, :]
        assert np.abs(got - np.stack([np.cos(angle), np.sin(angle)], -1) * magnitude).max() < 2e-7


@pytest.mark.parametrize("places,top,groups,keep", [(8, 3, 4, 2), (16, 4, 4, 3), (5, 1, 1, 1), (20, 6, 5, 3), (12, 12, 1, 1), (6, 4, 3, 2),
                                                    (64, 6, 8, 3), (100, 6, 10, 4), (250, 9, 25, 7), (300, 8, 6, 2)])
@pytest.mark.parametrize("shift", [0.0, -3.0])
def test_choice_with_a_correction(places, top, groups, keep, shift):
    """Corrections as large as the scores (and with ``shift`` all choice scores negative): the choice follows the corrected
    scores, over groups and places, the weights the scores."""
    from microllm_rocm_amd.ops import kernels
    rng = np.random.default_rng(places + top)
    z = rng.normal(size=(200, places)) * 2
    correction = rng.normal(size=places) * 0.1 + shift
    router = {"groups": {"count": groups, "keep": keep}, "top": top}
    ids, weights, _ = kernels.moe_route(device(z), places, top, softmax_scores=True, renormalize=True, groups=groups if groups > 1 else 0,
                                        keep=keep if groups > 1 else 0, correction=device(correction), weight_eps=1e-20, weight_scale=2.5)
    scores = torch.softmax(t64(device(z).cpu()), dim=-1)
    exact = t64(device(correction).cpu())
    same = 0
    for token in range(z.shape[0]):
        want, gap = plain.route(scores[token], exact, router)
        if gap < 1e-6:
            continue
        same += 1
        assert ids[token].tolist() == want, token
        chosen = scores[token, want]
        assert np.abs(weights[token].cpu().numpy() - (chosen / (chosen.sum() + 1e-20) * 2.5).numpy()).max() < 1e-5
    assert same > 190


def test_choice_of_ties_and_of_what_is_no_number():
    from microllm_rocm_amd.ops import kernels
    for places in (8, 300):
        z = np.zeros((3, places))
        z[1] = np.nan
        z[2, 5] = np.inf
        correction = np.zeros(places)
        ids, _, _ = kernels.moe_route(device(z), places, 4, softmax_scores=True, renormalize=True, correction=device(correction))
        ids = ids.cpu().numpy()
        assert ids[0].tolist() == [0, 1, 2, 3]                        # ties go to the lower place
        assert all(len(set(row)) == 4 and row.min() >= 0 and row.max() < places for row in ids)      # whatever the row holds, four places


@pytest.mark.parametrize("dtype,grouped", [(torch.float32, False), (torch.bfloat16, False), (torch.bfloat16, True)])
@pytest.mark.parametrize("width,ff,experts,identity,top,n", [(64, 24, 6, 2, 3, 50), (50, 20, 5, 0, 1, 9), (96, 64, 16, 4, 6, 200), (40, 7, 3, 3, 3, 5),
                                                             (1000, 48, 4, 1, 2, 8), (64, 40, 2, 9, 5, 30)])
def test_clamped_experts_and_places_that_return_their_input(dtype, grouped, width, ff, experts, identity, top, n):
    from microllm_rocm_amd.ops import kernels
    if grouped and (width % 8 or ff % 8):
        pytest.skip("the tiled products take widths in steps of 8")
    rng = np.random.default_rng(width + ff)
    x, down = as_bf16(rng.normal(size=(n, width))), as_bf16(rng.normal(size=(experts, width, ff)) * 0.2)
    gate_up = as_bf16(rng.normal(size=(experts, 2 * ff, width)) * (3.0 / math.sqrt(width)))      # as often beyond the limit as within
    ids = np.stack([rng.permutation(experts + identity)[:top] for _ in range(n)])
    weights = rng.uniform(0.05, 1.6, size=(n, top))
    limit = 1.25
    got = kernels.moe_experts(device(x, dtype), device(ids, torch.int32), device(weights), device(gate_up, dtype), device(down, dtype), False,
                              grouped=grouped, activation="clamped_glu", limit=limit, slope=1.702, identity=identity).cpu().numpy()
    want = np.zeros((top, n, width))
    for token in range(n):
        for choice in range(top):
            e = ids[token, choice]
            if e >= experts:
                want[choice, token] = weights[token, choice] * x[token]
                continue
            inner = t64(gate_up[e]) @ t64(x[token])
            g, u = torch.clamp(inner[:ff], max=limit), torch.clamp(inner[ff:], min=-limit, max=limit)
            inner = g * torch.sigmoid(1.702 * g) * (u + 1.0)
            if dtype == torch.bfloat16:
                inner = t64(as_bf16(inner.numpy()))
            want[choice, token] = weights[token, choice] * (t64(down[e]) @ inner).numpy()
    assert np.abs(got - want).max() < (3e-5 if dtype == torch.float32 else 4e-3) * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("keep_plain", [True, False])
@pytest.mark.parametrize("width,ff", [(64, 40), (96, 64), (256, 24)])
def test_clamped_gate_after_a_product_of_any_number_of_rows(width, ff, keep_plain):
    """In the product's epilogue, or after products whose columns come in the weight's order or by turns."""
    from microllm_rocm_amd.parts.linear import Weight, linear_clamped_glu
    rng = np.random.default_rng(ff)
    weight = as_bf16(rng.normal(size=(2 * ff, width)) * (2.0 / math.sqrt(width)))
    held = Weight(device(weight, torch.bfloat16), gated=True, keep_plain=keep_plain)
    for rows in (1, 3, 16, 17, 40, 64, 65, 300):
        x = as_bf16(rng.normal(size=(rows, width)))
        inner = t64(x) @ t64(weight).T
        g, u = torch.clamp(inner[:, :ff], max=1.1), torch.clamp(inner[:, ff:], min=-1.1, max=1.1)
        want = (g * torch.sigmoid(1.702 * g) * (u + 1.0)).numpy()
        got = linear_clamped_glu(device(x, torch.bfloat16), held, 1.1, 1.702).float().cpu().numpy()
        assert np.abs(got - want).max() < 0.006 * np.abs(want).max(), rows
    exact = Weight(device(weight), gated=True)
    got = linear_clamped_glu(device(x), exact, 1.1, 1.702).cpu().numpy()
    assert np.abs(got - want).max() < 2e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top,groups,keep,shared", [(8, 3, 4, 2, False), (20, 6, 5, 3, True), (64, 8, 0, 0, True), (64, 5, 8, 2, False),
                                                            (3, 3, 0, 0, True), (70, 4, 7, 3, True)])
def test_router_and_choice_in_one_kernel(dtype, experts, top, groups, keep, shared):
    """The same places and weights as the two kernels give one after the other, with and without a correction."""
    from microllm_rocm_amd.ops import kernels
    rng = np.random.default_rng(experts)
    x = device(rng.normal(size=(77, 144)), dtype)
    weight = device(rng.normal(size=(experts + int(shared), 144)) * 0.2)
    for softmax_scores in (True, False):
        for correction in (None, device(rng.normal(size=experts) * 0.05)):
            options = dict(softmax_scores=softmax_scores, renormalize=True, shared_at=experts if shared else -1, groups=groups, keep=keep,
                           correction=correction, weight_eps=1e-20, weight_scale=1.5)
            ids, weights, gate = kernels.moe_choose(x, weight, experts, top, **options)
            z = kernels.router_logits(x, weight)
            want_ids, want_weights, want_gate = kernels.moe_route(z, experts, top, **options)
            assert torch.equal(ids, want_ids) and torch.equal(weights, want_weights)
            assert (gate is None) == (not shared) and (not shared or torch.equal(gate, want_gate))
            scores = torch.softmax(z[:, :experts].double(), -1) if softmax_scores else torch.sigmoid(z[:, :experts].double())
            decides = scores if correction is None else scores + correction.double()
            if not groups:
                best = torch.topk(decides, top, dim=-1).indices
                assert (ids.long().sort(-1).values == best.sort(-1).values).all()
            chosen = torch.gather(scores, 1, ids.long())
            assert torch.allclose(weights.double(), chosen / chosen.sum(-1, keepdim=True) * 1.5, atol=1e-6)


@pytest.mark.parametrize("width,ff,experts,identity,top,n", [(256, 288, 4, 1, 3, 9), (512, 256, 9, 3, 5, 21), (1024, 320, 3, 0, 2, 20), (4096, 1280, 5, 2, 4, 8),
                                                             (320, 256, 2, 2, 2, 31), (256, 64, 6, 0, 2, 40)])
@pytest.mark.parametrize("form", ["clamped_glu", "silu", "plain"])
@pytest.mark.parametrize("on_input", [False, True])
def test_few_pairs_on_the_matrix_units(width, ff, experts, identity, top, n, form, on_input):
    """Reductions of a multiple of 32 from 256 on: an expert with no pair, with one, with more than the 16 columns of a product;
    the last wave's steps overlap another's where the reduction is no multiple of 256."""
    from microllm_rocm_amd.ops import kernels
    rng = np.random.default_rng(width + n)
    gated = form != "plain"
    x, down = as_bf16(rng.normal(size=(n, width))), as_bf16(rng.normal(size=(experts, width, ff)) / math.sqrt(ff))
    inner_weight = as_bf16(rng.normal(size=(experts, (2 if gated else 1) * ff, width)) * (2.0 / math.sqrt(width)))
    places = rng.permutation(experts + identity)[:max(top, experts + identity - 1)]        # one place no token takes
    ids = np.stack([rng.permutation(places)[:top] for _ in range(n)])
    weights = rng.uniform(0.2, 1.6, size=(n, top))
    options = dict(gated=gated, activation={"clamped_glu": "clamped_glu", "silu": "silu", "plain": "gelu_erf"}[form], identity=identity,
                   **(dict(limit=1.25, slope=1.702) if form == "clamped_glu" else {}))
    got = kernels.moe_experts(device(x, torch.bfloat16), device(ids, torch.int32), device(weights), device(inner_weight, torch.bfloat16),
                              device(down, torch.bfloat16), on_input, grouped=False, **options).cpu().numpy()
    for token in range(n):
        for choice in range(top):
            e, w = ids[token, choice], float(np.float32(weights[token, choice]))
            if e >= experts:
                assert np.abs(got[choice, token] - w * x[token]).max() < 1e-5
                continue
            inner = t64(inner_weight[e]) @ t64(as_bf16(x[token] * w) if on_input else x[token])
            if form == "clamped_glu":
                g, u = torch.clamp(inner[:ff], max=1.25), torch.clamp(inner[ff:], min=-1.25, max=1.25)
                inner = g * torch.sigmoid(1.702 * g) * (u + 1.0)
            elif form == "silu":
                inner = inner[:ff] * torch.sigmoid(inner[:ff]) * inner[ff:]
            else:
                inner = 0.5 * inner * (1.0 + torch.erf(inner / math.sqrt(2.0)))
            want = ((1.0 if on_input else w) * (t64(down[e]) @ inner)).numpy()
            assert np.abs(got[choice, token] - want).max() < 0.015 * np.abs(want).max(), (token, choice)


# ---- the engine ---------------------------------------------------------------------------------------------------
def single_layer_folder(tmp_path, layer_of, which, with_mlp, choice=True, twice=False):
    """A model of one layer: the mixer ``layer_of`` of configuration ``which``, with its own feed-forward or none; with ``twice``
    run a second time with the same tensors."""
    import dataclasses
    from microllm_rocm_amd.weights import write_model_folder
    source = CONFIGS[which] if choice else without_choice(CONFIGS[which])
    layer = dataclasses.replace(source.layers[layer_of], weights_of=None)
    if not with_mlp:
        layer = dataclasses.replace(layer, mlp=None)
    config = dataclasses.replace(source, layers=(layer, dataclasses.replace(layer, weights_of=0)) if twice else (layer,))
    folder = os.path.join(str(tmp_path), f"one_{which}_{layer_of}_{int(choice)}")
    write_model_folder(folder, config, 50 + layer_of, dtype=torch.bfloat16, stds=STDS)
    return folder


@pytest.mark.parametrize("which,layer_of,with_mlp,twice", [
    ("A", 0, False, False), ("A", 0, True, True), ("A", 1, False, False), ("A", 1, True, False), ("A", 2, False, True),
    ("B", 0, True, False), ("B", 1, False, True), ("B", 2, True, False), ("C", 0, True, False), ("C", 1, False, True),
    ("C", 2, True, False), ("C", 3, True, False)])
def test_every_mixer_as_a_model_of_one_layer(tmp_path, which, layer_of, with_mlp, twice):
    tokens = tokens_for(layer_of, 90, CONFIGS[which].vocab)
    for dtype in ("float32", "bfloat16"):
        folder = single_layer_folder(tmp_path, layer_of, which, with_mlp, choice=dtype == "float32", twice=twice)
        config, weights = plain.read_config(folder), plain.read_tensors(folder)
        for name, steps in (("whole", whole({"r": tokens})), ("decode", prefill_then_decode("r", tokens, tail=40)),
                            ("portions", portions("r", tokens, [2, 5, 1, 17]))):
            run_trace(folder, dtype, steps, tmp_path / f"{dtype}_{name}", max_tokens=128)
            check_against_plain(steps, tmp_path / f"{dtype}_{name}", {"r": tokens}, config, weights, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_whole_decode_and_portions(tmp_path_factory, tmp_path, which, dtype):
    folder, config, weights = model_for(tmp_path_factory, which, dtype)
    requests = {"long": tokens_for(1, 150, config["vocab"]), "short": tokens_for(2, 37, config["vocab"]), "one": tokens_for(3, 1, config["vocab"])}
    run_trace(folder, dtype, whole(requests), tmp_path / "whole", max_tokens=256)
    check_against_plain(whole(requests), tmp_path / "whole", requests, config, weights, dtype)
    for rid, tail in (("long", 70), ("short", 34)):      # the decoded tokens cross pages' edges
        steps = prefill_then_decode(rid, requests[rid], tail=tail)
        run_trace(folder, dtype, steps, tmp_path / f"decode_{rid}", max_tokens=round_up(len(requests[rid]), 64))
        check_against_plain(steps, tmp_path / f"decode_{rid}", {rid: requests[rid]}, config, weights, dtype)
    for sizes in ([2], [3, 16, 1, 2, 31], [64, 2, 17]):
        steps = portions("long", requests["long"], sizes)
        run_trace(folder, dtype, steps, tmp_path / f"portions_{sizes[0]}", max_tokens=192)
        check_against_plain(steps, tmp_path / f"portions_{sizes[0]}", {"long": requests["long"]}, config, weights, dtype)
    steps = portions("short", requests["short"], [1])       # from its first token on, one token a step
    run_trace(folder, dtype, steps, tmp_path / "one_by_one", max_tokens=64)
    check_against_plain(steps, tmp_path / "one_by_one", {"short": requests["short"]}, config, weights, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_mixed_batches_on_reused_pages_and_slots(tmp_path_factory, tmp_path, which, dtype):
    folder, config, weights = model_for(tmp_path_factory, which, dtype)
    lengths = [90, 41, 130, 2, 67, 25, 110, 58]
    requests = {f"r{index}": tokens_for(10 + index, length, config["vocab"]) for index, length in enumerate(lengths)}
    steps, peak = mixed(requests, seed=4, max_live=3, decode_tail=12, max_portion=23)
    engine = run_trace(folder, dtype, steps, tmp_path / "mixed", max_tokens=peak, max_requests=3)
    assert all(group.pool.total_taken > group.pool.num_pages for group in engine.cache.groups)      # pages were used again
    assert engine.cache.slots.total_taken > 3                                                        # and so were slots
    check_against_plain(steps, tmp_path / "mixed", requests, config, weights, dtype)


def test_a_row_does_not_depend_on_the_batch(tmp_path_factory):
    """Float32: a request's logits are the same bits alone and beside others, whole and in portions."""
    from microllm_rocm_amd.engine import Engine, StepEntry
    folder, config, _ = model_for(tmp_path_factory, "A")
    engine = Engine.from_folder(folder, dtype="float32", max_tokens=512, max_requests=4)
    a, b, c = (tokens_for(seed, length, config["vocab"]) for seed, length in ((1, 45), (2, 20), (3, 33)))
    engine.open("alone")
    alone = engine.step([StepEntry("alone", a, list(range(len(a))))]).clone()
    engine.close("alone")
    for name in "abc":
        engine.open(name)
    first = engine.step([StepEntry("b", b[:7], []), StepEntry("a", a[:30], list(range(30))), StepEntry("c", c[:2], [])])
    second = engine.step([StepEntry("a", a[30:44], list(range(14))), StepEntry("c", c[2:], []), StepEntry("b", b[7:8], [])])
    third = engine.step([StepEntry("b", b[8:9], [0]), StepEntry("a", a[44:], [0])])
    together = torch.cat([first, second, third[1:]])
    assert torch.equal(alone, together)


@pytest.mark.parametrize("which", ["A", "B"])
def test_long_decoding_through_graphs(tmp_path_factory, which):
    """A short prompt, then 140 tokens one by one (steps replayed from captured graphs, state carried in slots, cached
    rows crossing many pages), two requests at once with unequal lengths."""
    from microllm_rocm_amd.engine import Engine, StepEntry
    folder, config, weights = model_for(tmp_path_factory, which)
    engine = Engine.from_folder(folder, dtype="float32", max_tokens=512, max_requests=2)
    assert engine.use_graphs
    sequences = {"x": tokens_for(7, 150, config["vocab"]), "y": tokens_for(8, 160, config["vocab"])}
    starts = {"x": 10, "y": 3}
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
        check_rows(np.stack(rows[name]), want[starts[name] - 1:], sensitivity[starts[name] - 1:], "float32", name)


@pytest.mark.parametrize("which", ["A", "C"])
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


@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_residual_stream_after_every_layer(tmp_path_factory, tmp_path, which):
    """A layer that runs with another's tensors counts as its own."""
    folder, config, weights = model_for(tmp_path_factory, which)
    tokens = tokens_for(5, 19, config["vocab"])
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": tokens, "want": list(range(19))}], "end": ["q"]}]
    from microllm_rocm_amd.engine import Engine
    from microllm_rocm_amd.engine.replay import replay
    engine = Engine.from_folder(folder, dtype="float32", max_tokens=64, max_requests=1)
    replay(engine, io.StringIO(to_lines(steps)), str(tmp_path), io.StringIO(), dump_layers=True)
    streams = plain_run(config, weights, tokens)[1]
    runs = len(config["layers"])
    assert streams.shape[0] == runs
    got = np.fromfile(os.path.join(str(tmp_path), "0.layers.f32"), dtype="<f4").reshape(runs, 19, config["width"])
    for run in range(runs):
        assert np.abs(got[run] - streams[run]).max() < 1e-4 * np.abs(streams[run]).max(), run


def test_one_copy_of_the_weights(tmp_path_factory, tmp_path):
    """A bfloat16 engine that keeps the packed weights alone (prompts on the tiled products) gives the same model."""
    folder, config, weights = model_for(tmp_path_factory, "C", "bfloat16")
    requests = {"long": tokens_for(1, 150, config["vocab"]), "short": tokens_for(2, 37, config["vocab"])}
    run_trace(folder, "bfloat16", whole(requests), tmp_path / "whole", max_tokens=256, weight_copies="packed")
    check_against_plain(whole(requests), tmp_path / "whole", requests, config, weights, "bfloat16")
    steps = prefill_then_decode("long", requests["long"], tail=30)
    run_trace(folder, "bfloat16", steps, tmp_path / "decode", max_tokens=192, weight_copies="packed")
    check_against_plain(steps, tmp_path / "decode", requests={"long": requests["long"]}, config=config, weights=weights, dtype="bfloat16")


def test_plain_pages_in_bfloat16(tmp_path_factory):
    """A bfloat16 engine whose attention layers are told not to take the MFMA kernels runs the same model on plain
    pages; it stays within the format's cost of the plain run."""
    import dataclasses
    from microllm_rocm_amd.config.registry import load_config
    from microllm_rocm_amd.engine import Engine, StepEntry
    from microllm_rocm_amd.parts import Model, PartSpec, Runtime
    from microllm_rocm_amd.weights import load_folder
    folder, config, weights = model_for(tmp_path_factory, "C", "bfloat16")
    architecture, typed = load_config(folder)
    built = architecture.build_spec(typed)
    spec = dataclasses.replace(built, layers=tuple(dataclasses.replace(layer, mixer=PartSpec(layer.mixer.kind, {**layer.mixer.params, "mfma": False}, layer.mixer.names))
                                                   for layer in built.layers))
    probe = Model(spec, Runtime(torch.bfloat16, torch.device("cpu")))
    assert not any(getattr(part, "tiled", False) for part in probe.parts())
    tiled = Model(built, Runtime(torch.bfloat16, torch.device("cpu")))
    assert sum(bool(getattr(part, "tiled", False)) for part in tiled.parts()) == 4      # as built, every mixer takes the MFMA kernels
    tensors = load_folder(folder, probe.tensors(), torch.bfloat16, torch.device("cuda:0"))
    engine = Engine(spec, tensors, dtype="bfloat16", max_tokens=256, max_requests=2, tensors_placed=True)
    tokens = tokens_for(9, 120, config["vocab"])
    engine.open("p")
    first = engine.step([StepEntry("p", tokens[:40], list(range(40)))]).cpu().numpy()
    rest = [engine.step([StepEntry("p", [token], [0])]).cpu().numpy() for token in tokens[40:]]
    want, _, sensitivity = plain_run(config, weights, tokens)
    check_rows(np.concatenate([first] + rest), want, sensitivity, "bfloat16", "p")


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
    assert report["architecture"] == "Zuluvik" and report["generated_tokens"] == expected
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
