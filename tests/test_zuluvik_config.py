"""Host logic of the Zuluvik decoder: its configuration (keys, what may be absent, refusals), layers that run with another's
tensors, the model it is built into and the cache needs of its mixers, the rates stretched along a ramp, and the plain
implementation's own pieces against values worked out by hand."""
import copy
import json
import math
import os

import pytest
import torch

import plain_zuluvik as plain
from zuluvik_tiny import CONFIGS, make_zuluvik_folder
from microllm_rocm_amd.cache import CompositeNeed, PagedKVNeed, PagedLatentNeed, StateNeed
from microllm_rocm_amd.config import ConfigError, load_config
from microllm_rocm_amd.config.zuluvik import ZuluvikConfig
from microllm_rocm_amd.parts import Model, PartSpec, Runtime, build_part
from microllm_rocm_amd.parts.base import PagedKeyValueNeed

F = torch.float64


def round_up(value, multiple):
    return -(-value // multiple) * multiple


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("which", ["A", "B", "C"])
def test_folder_round_trip(tmp_path, which, dtype):
    folder = make_zuluvik_folder(tmp_path, which)
    written = json.load(open(os.path.join(folder, "config.json")))
    assert written["architecture"] == "Zuluvik"
    architecture, config = load_config(folder)
    assert architecture.name == "Zuluvik" and config == CONFIGS[which]
    spec = architecture.build_spec(config)
    model = Model(spec, Runtime(dtype, torch.device("cpu")))
    tensors = plain.read_tensors(folder)
    assert set(model.tensors()) == set(tensors)
    assert all(tuple(tensors[name].shape) == tuple(decl.shape) for name, decl in model.tensors().items())
    needs = model.cache_needs()
    assert len(needs) == len(spec.order) == len(written["layers"])
    for need, layer in zip(needs, written["layers"]):
        mixer = layer["mixer"]
        if layer["type"] == "latent_attention":
            row = mixer["kv_rank"] + mixer["rot_dim"]
            assert need == (PagedKVNeed(1, row, None) if dtype == torch.bfloat16 and row % 16 == 0 else PagedLatentNeed(row, None))
            continue
        keys = mixer["dim"] * (2 if layer["type"] == "attention" else 1)
        pages = (PagedKVNeed(mixer["kv_heads"], round_up(max(keys, mixer["vdim"]), 16), None) if dtype == torch.bfloat16
                 else PagedKeyValueNeed(mixer["kv_heads"], keys, mixer["vdim"], None))
        if layer["type"] == "attention" and mixer["conv"] > 1:
            columns = mixer["heads"] * keys + mixer["kv_heads"] * (keys + mixer["vdim"])
            assert need == CompositeNeed((pages, StateNeed((mixer["conv"] - 1, columns), torch.float32)))
        else:
            assert need == pages


def test_layers_that_run_with_anothers_tensors():
    """One more run entry of the owner's layer, with a cache of its own; a chain leads to its end; an entry may name a
    later layer."""
    from microllm_rocm_amd.architectures.zuluvik import build_spec
    spec = build_spec(CONFIGS["B"])
    assert [entry.layer for entry in spec.order] == [0, 1, 2, 1, 1, 0]
    assert all(entry.reads_cache_of is None for entry in spec.order) and len(spec.layers) == 3
    assert [entry.layer for entry in build_spec(CONFIGS["A"]).order] == [0, 1, 2, 0, 2]
    source = CONFIGS["A"].to_dict()
    source["layers"][0], source["layers"][3] = source["layers"][3], source["layers"][0]
    source["layers"][0]["weights_of"] = 3
    config = ZuluvikConfig.from_dict(source)
    spec = build_spec(config)
    assert [entry.layer for entry in spec.order] == [2, 0, 1, 2, 1]
    assert spec.layers[2].mixer_norm.names["weight"] == "l3.norm1"
    assert plain.owner(source, 0) == 3


def test_what_a_file_may_leave_out():
    source = CONFIGS["B"].to_dict()
    del source["embedding"]
    del source["layers"][0]["mlp"]["router"]["groups"], source["layers"][0]["mlp"]["router"]["identity"], source["layers"][0]["mlp"]["router"]["scale"]
    assert "shared" not in source["layers"][0]["mlp"] and "scaling" not in source["layers"][1]["mixer"]["rot"]
    source["layers"][5]["mlp"] = copy.deepcopy(source["layers"][0]["mlp"])
    config = ZuluvikConfig.from_dict(source)
    assert config == CONFIGS["B"]
    assert config.layers[0].mlp.identity == 0 and config.layers[0].mlp.shared is None and config.layers[1].mlp is None


@pytest.mark.parametrize("change,text", [
    (lambda c: c["layers"][0].__setitem__("type", "window"), "unknown layer type"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "dense"), "unknown feed-forward kind"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 18), "at most mixer.dim"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 7), "must be even"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].__setitem__("factor", 0.0), "must be positive"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].__delitem__("slow"), "missing slow"),
    (lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("base", 1), "must not be 1"),
    (lambda c: c["layers"][2]["mixer"]["rot"].__setitem__("dims", 6), "rot.dims must equal"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 3), "must divide"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("conv", 0), "must be positive"),
    (lambda c: c["layers"][0]["mixer"].__delitem__("diff"), "missing diff"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 9), "cannot exceed"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("identity", 3), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("keep", 1), "fewer places"),
    (lambda c: c["layers"][0]["mlp"]["expert"].__delitem__("limit"), "missing limit"),
    (lambda c: c["layers"][3].__setitem__("weights_of", 9), "names no layer"),
    (lambda c: c["layers"][0].__setitem__("weights_of", 3), "leads to no layer"),
    (lambda c: c["layers"][3].__setitem__("weights_of", 1), "differs from the layer"),
    (lambda c: c["layers"][3]["mlp"]["router"].__setitem__("scale", 3.5), "differs from the layer"),
    (lambda c: c.__setitem__("vocab", 3.5), "must be an integer"),
])
def test_refusals(change, text):
    source = copy.deepcopy(CONFIGS["A"].to_dict())
    change(source)
    with pytest.raises(ConfigError, match=text):
        ZuluvikConfig.from_dict(source)


@pytest.mark.parametrize("base,n,scaling", [
    (1e3, 8, dict(factor=4.0, original=64.0, fast=8.0, slow=0.5)), (1e6, 64, dict(factor=12.0, original=8192.0, fast=30.0, slow=1.5)),
    (300.0, 6, dict(factor=16.0, original=40.0, fast=2.0, slow=0.1)), (1e4, 2, dict(factor=2.0, original=100.0, fast=24.0, slow=1.5)),
    (50.0, 10, dict(factor=3.0, original=4.0, fast=32.0, slow=30.0)),        # both ends of the ramp below the first pair
    (1e4, 32, dict(factor=5.0, original=1e9, fast=1.0, slow=0.001)),         # both beyond the last
    (1e4, 32, dict(factor=1.0, original=500.0, fast=24.0, slow=1.5)), (500.0, 20, None)])
def test_rates_stretched_along_a_ramp(base, n, scaling):
    params = {"theta": base, "head_dim": n, "rotary_dim": n}
    if scaling is not None:
        params["scaling_ramp"] = {**scaling, "magnitude_slope": 0.1}
    position = build_part("position", PartSpec("rope_neighbours", params), Runtime(torch.float32, torch.device("cpu")))
    rates, magnitude = plain.yarn(base, n, scaling)
    assert torch.allclose(position.inv_freq, torch.tensor(rates, dtype=F), rtol=1e-13, atol=0.0)
    assert abs(position.magnitude - magnitude) < 1e-15


def test_the_ramp_by_hand():
    """Base 10 and 8 dimensions: pair i has the rate 10^(-i/4). Over 2 pi * 10^(3/4) positions pair 3 turns once, so with slow
    1 the ramp ends there; with fast 10^(3/4) it begins at pair 0; between, a third more of the stretched rate a pair."""
    original = 2.0 * math.pi * 10.0 ** 0.75
    rates, magnitude = plain.yarn(10.0, 8, dict(factor=4.0, original=original * (1 + 1e-12), fast=10.0 ** 0.75, slow=1.0 + 1e-9))
    for i in range(4):
        plain_rate = 10.0 ** (-i / 4.0)
        share = i / 3.0
        assert abs(rates[i] - plain_rate * (share / 4.0 + 1.0 - share)) < 1e-12, i
    assert abs(magnitude - (1.0 + 0.1 * math.log(4.0))) < 1e-15
    assert plain.yarn(10.0, 8)[1] == 1.0


def test_convolution_by_hand():
    u = torch.tensor([[1.0, 1.0], [2.0, 0.0], [3.0, 0.0], [4.0, 5.0]], dtype=F)
    taps = torch.tensor([[0.5, 0.0, 1.0], [1.0, 10.0, 100.0]], dtype=F)      # the last tap is the token's own
    assert torch.equal(plain.convolve(u, taps), torch.tensor([[1.0, 100.0], [2.0, 10.0], [3.5, 1.0], [5.0, 500.0]], dtype=F))


def test_choice_among_places_with_a_correction():
    router = {"groups": {"count": 2, "keep": 1}, "top": 2}
    scores = torch.tensor([0.30, 0.05, 0.20, 0.15, 0.18, 0.12], dtype=F)
    assert plain.route(scores, torch.zeros(6, dtype=F), router)[0] == [0, 2]
    correction = torch.tensor([-1.0, -1.0, -1.0, -0.9, -0.5, -0.5], dtype=F)       # every choice score is negative
    assert plain.route(scores, correction, router)[0] == [4, 5]
    router = {"groups": {"count": 3, "keep": 2}, "top": 3}
    chosen, gap = plain.route(scores, torch.tensor([0.0, 0.0, 0.5, 0.0, 0.0, 0.0], dtype=F), router)
    assert chosen == [2, 0, 3]      # groups (2,3) and (0,1); 4 scores more than 3, but its group lost
    assert abs(gap - 0.10) < 1e-12  # 3 against 1; the groups 0.30 against 0.18


def test_clamped_expert_and_shared_weights_by_hand():
    one = torch.ones(1, 1, dtype=F)
    tensors = {"e.gate": 3.0 * one, "e.up": -5.0 * one, "e.down": 2.0 * one}
    got = float(plain.clamped_expert(one, tensors, "e", 2.0))
    assert abs(got - 2.0 * (2.0 / (1.0 + math.exp(-3.404)) * (-2.0 + 1.0))) < 1e-12
    tensors["e.gate"] = -30.0 * one          # the gate has no lower limit
    assert abs(float(plain.clamped_expert(one, tensors, "e", 2.0)) - 2.0 * (-30.0 / (1.0 + math.exp(51.06)) * -1.0)) < 1e-12
