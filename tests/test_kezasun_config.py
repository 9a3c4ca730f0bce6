"""Kezasun without a GPU: its configuration keys and their errors, the ModelSpec they become (run order, needs, tensor names), steps and generation
of a model in host memory on the null device, and the plain implementation pinned by closed forms."""
import copy
import math

import pytest
import torch

import kezasun_common as C
import plain_kezasun as plain
from tq_kv_amd import Engine, GenerationParams, Model, generate
from tq_kv_amd.cache import PAGE
from tq_kv_amd.config import ConfigError, config_from_dict, known_architectures
from tq_kv_amd.config.registry import spec_from_dict
from tq_kv_amd.parts.spec import ModelSpec


def test_the_architecture_is_known_by_its_name():
    assert "Kezasun" in known_architectures()
    for make in (C.config_mixed, C.config_ones, C.config_odd):
        name, typed = config_from_dict(make())
        assert name == "Kezasun"
        assert config_from_dict(typed.to_dict())[1] == typed            # round trip through config.json
    name, typed = config_from_dict(C.config_mixed())
    assert (typed.vocab, typed.width, typed.norm_eps, typed.residual_mult) == (331, 96, 3e-6, 0.55)
    assert typed.layers[0].mixer["window"] == 37 and typed.layers[2].mixer["kv_from"] == 0 and typed.layers[3].mlp is None
    assert typed.layers[0].mlp == {"kind": "moe", "ff": 40, "experts": 9, "top": 3, "identity": 3, "groups": 4, "keep": 2}
    # what a router may leave out: experts that give back their input, and groups
    raw = C.config_mixed()
    del raw["layers"][0]["mlp"]["router"]["groups"], raw["layers"][0]["mlp"]["router"]["identity"]
    mlp = config_from_dict(raw)[1].layers[0].mlp
    assert (mlp["identity"], mlp["groups"], mlp["keep"]) == (0, 1, 1)


def test_the_spec_names_tensors_parts_and_needs():
    cfg = C.config_mixed()
    spec = spec_from_dict(cfg)
    assert ModelSpec.from_json(spec.to_json()) == spec
    assert spec.embedding_name == "embed" and spec.head_name == "head" and spec.final_norm_prefix == "final.norm" and spec.final_norm.kind == "rms_norm"
    assert [r.layer for r in spec.order] == list(range(8)) and [r.cache_of for r in spec.order] == [None, None, 0, None, None, 0, None, 4]
    assert all(l.block.kind == "joint" and l.block.params["scale"] == 0.55 and l.block.params["norm"].params["unit_offset"] for l in spec.layers)
    assert [l.block.params["mixer"].kind for l in spec.layers] == ["attention", "time_mixing", "attention", "time_mixing", "attention", "attention", "time_mixing", "attention"]
    att = spec.layers[2].block.params["mixer"].params
    assert (att["own_kv"], att["window"], att["cache_window"], att["sink_score"], att["gate"], att["qk_norm_over"]) == (False, 70, 70, 0.0, "head", "projection")
    assert att["position"].params["scaling"] == {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64.0}
    assert "scaling" not in spec.layers[4].block.params["mixer"].params["position"].params
    model = Model(spec, dtype="float32", device="cpu")
    specs = model.tensor_specs()
    w = C.weights(cfg, 1)
    assert set(specs) == set(w)
    for name, t in w.items():
        # (the decay's rank is the checkpoint's to say)
        assert name.split(".")[-1] in ("w1", "w2") or list(t.shape) == list(specs[name].shape), name
    # what the cache keeps: the largest window of those that read it
    needs = model.needs
    assert [needs[i].window for i in (0, 2, 4, 5, 7)] == [70, 70, 64, 70, 64]
    assert needs[1].shape == (3 * 20 * 20 + 96,) and needs[6].shape == (8 * 8 + 96,)


@pytest.mark.parametrize("path,value,word", [
    (("width",), None, "width"), (("vocab",), "many", "vocab"), (("norm",), None, "norm"), (("norm", "eps"), None, "eps"), (("layers",), [], "layers"),
    (("residual_mult",), None, "residual_mult"), (("layers", 0, "type"), "convolution", "convolution"), (("layers", 0, "mixer"), None, "mixer"),
    (("layers", 1, "mixer", "heads"), 0, "heads"), (("layers", 1, "mixer", "dim"), 600, "key channels"), (("layers", 0, "mixer", "kv_heads"), 4, "kv_heads"),
    (("layers", 0, "mixer", "mask"), None, "mask"), (("layers", 0, "mixer", "mask", "size"), 0, "size"), (("layers", 0, "mixer", "rot", "dims"), 7, "dims"),
    (("layers", 0, "mixer", "rot", "dims"), 26, "dims"), (("layers", 0, "mixer", "rot", "scaling", "factor"), None, "factor"),
    (("layers", 0, "mixer", "rot", "scaling", "high"), 1.0, "high"), (("layers", 4, "mixer", "dim"), 300, "dim"), (("layers", 4, "mixer", "scale"), None, "scale"),
    (("layers", 2, "mixer", "kv_from"), 1, "kv_from"), (("layers", 2, "mixer", "kv_from"), 2, "kv_from"), (("layers", 5, "mixer", "kv_from"), 2, "of its own"),
    (("layers", 2, "mixer", "vdim"), 48, "vdim"), (("layers", 7, "mixer", "kv_heads"), 2, "kv_heads"),
    (("layers", 0, "mlp", "kind"), "sparse", "sparse"), (("layers", 0, "mlp", "expert"), None, "expert"), (("layers", 0, "mlp", "router", "top"), 7, "top"),
    (("layers", 0, "mlp", "router", "groups", "count"), 5, "count"), (("layers", 0, "mlp", "router", "groups", "keep"), 5, "keep"),
    (("layers", 0, "mlp", "router", "experts"), 601, "experts")])
def test_what_is_missing_or_wrong_is_named(path, value, word):
    raw = copy.deepcopy(C.config_mixed())
    at = raw
    for key in path[:-1]:
        at = at[key]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    with pytest.raises(ConfigError, match=word):
        spec = spec_from_dict(raw)
        Model(spec, dtype="float32", device="cpu")          # what a part refuses is refused when the model is put together


def test_more_windows_than_the_cache_has_groups():
    """Seventeen different windows: layers of equal pages keep the largest of them and share a group."""
    layers = [(C.attention(2, 1, 8, 8, 5 + n, 4), None) for n in range(17)] + [(C.attention(2, 1, 8, 8, 90, 4, kv_from=3), None), (C.attention(2, 2, 8, 8, 7, 4), None)]
    model = Model(spec_from_dict(C.config(40, 32, layers)), dtype="float32", device="cpu")
    assert {n.window for n in model.needs[:18]} == {90} and model.needs[18].window == 7
    few = Model(spec_from_dict(C.config(40, 32, layers[:3])), dtype="float32", device="cpu")
    assert [n.window for n in few.needs] == [5, 6, 7]


@pytest.mark.parametrize("make", [C.config_mixed, C.config_ones, C.config_odd])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_steps_and_generation_on_the_null_device(make, dtype):
    cfg = make()
    model = Model.random(cfg, seed=3, dtype=dtype, device="cpu")
    assert not model.on_gpu and model.graph_safe
    engine = Engine(model, max_tokens=6 * PAGE, max_slots=4)
    free0 = [g.pool.n_free for g in engine.cache.kv_groups]
    assert len(engine.cache.kv_groups) >= 1 and all(g.state.dtype == torch.float32 for g in engine.cache.state_groups)
    a, b = engine.open(), engine.open()
    out = engine.step([(a, C.tokens(150, cfg["vocab"], 1), [0, 149]), (b, C.tokens(3, cfg["vocab"], 2), [2])])
    assert tuple(out.shape) == (3, cfg["vocab"])
    for step in range(3):
        engine.step([(a, [step], [0]), (b, [step], [0])])
    assert (engine.length(a), engine.length(b)) == (153, 6)
    engine.close(a), engine.close(b)
    assert [g.pool.n_free for g in engine.cache.kv_groups] == free0
    engine.cache.check()
    got = generate(engine, [C.tokens(n, cfg["vocab"], 10 + n) for n in (5, 1, 17, 70)], GenerationParams(max_tokens=4, temperature=0.0, repeat_penalty=1.0),
                   eos_ids=(), max_batch=3)
    assert got == [[0] * 4] * 4
    assert [g.pool.n_free for g in engine.cache.kv_groups] == free0


# ---- the plain implementation, pinned by closed forms ----------------------------------------------------
def test_plain_time_mixing_as_one_sum():
    """o_t = sum_(s<t) (product of the decays of s+1 .. t-1, times k_s . r_t channel by channel) v_s + (u k_t . r_t) v_t"""
    g = torch.Generator().manual_seed(3)
    T, H, d = 9, 2, 3
    r, k, v = (torch.randn(T, H, d, generator=g, dtype=torch.float64) for _ in range(3))
    a, u = torch.rand(T, H, d, generator=g, dtype=torch.float64), torch.randn(H, d, generator=g, dtype=torch.float64)
    out, S = plain.time_mixing(r, k, v, a, u)
    for h in range(H):
        for t in range(T):
            want = (u[h] * k[t, h] * r[t, h]).sum() * v[t, h]
            for s in range(t):
                want = want + (a[s + 1:t, h].prod(0) * k[s, h] * r[t, h]).sum() * v[s, h]
            assert torch.allclose(out[t, h], want)
    first, state = plain.time_mixing(r[:4], k[:4], v[:4], a[:4], u)
    second, last = plain.time_mixing(r[4:], k[4:], v[4:], a[4:], u, state)
    assert torch.allclose(torch.cat([first, second]), out) and torch.allclose(last, S)


def test_plain_mechanisms_in_closed_form():
    assert torch.allclose(plain.decay(torch.tensor([0.0, -100.0, 100.0])), torch.tensor([math.exp(-1.0), 1.0, 0.0]))
    h = torch.tensor([[1.0, 2.0], [3.0, 5.0]])
    assert plain.shifted(h).tolist() == [[0.0, 0.0], [1.0, 2.0]]
    assert plain.mixed(h, plain.shifted(h), torch.tensor([0.0, 1.0])).tolist() == [[1.0, 0.0], [3.0, 2.0]]
    # three scores of zero share the denominator with the one; it counts once however many keys there are
    assert torch.allclose(plain.softmax_with_one(torch.zeros(3)), torch.full((3,), 0.25))
    assert torch.allclose(plain.softmax_with_one(torch.tensor([-200.0])), torch.tensor([0.0])) and torch.allclose(plain.softmax_with_one(torch.tensor([200.0])), torch.tensor([1.0]))
    assert [plain.first_visible(i, 3) for i in range(5)] == [0, 0, 0, 1, 2]
    assert torch.allclose(plain.offset_norm(torch.tensor([[3.0, -3.0]]), torch.tensor([0.0, 1.0]), 0.0), torch.tensor([[1.0, -2.0]]))
    v = torch.tensor([[[1.0, 0.0, 0.0, 2.0, 5.0]]]).expand(3, 1, 5)
    ang = torch.arange(3.0)[:, None] * plain.frequencies({"base": 16.0, "dims": 4})          # angles: position, position / 4
    turned = plain.turn_halves(v, ang.float())[2, 0]
    assert torch.allclose(turned, torch.tensor([math.cos(2.0), -2.0 * math.sin(0.5), math.sin(2.0), 2.0 * math.cos(0.5), 5.0]), atol=1e-6)


def test_plain_frequencies_below_between_and_above():
    rot = {"base": 10000.0, "dims": 8}
    f = plain.frequencies(rot)
    scaled = plain.frequencies(dict(rot, scaling=C.scaled(4.0, 1.0, 4.0, 200)))
    length = 2 * math.pi / f
    assert length[0] < 50 < length[1] < 200 < length[2]
    assert scaled[0] == f[0] and torch.allclose(scaled[2:], f[2:] / 4)
    s = (200 / length[1] - 1) / 3
    assert torch.allclose(scaled[1], (1 - s) * f[1] / 4 + s * f[1]) and f[1] / 4 < scaled[1] < f[1]


def test_plain_routing():
    router = {"experts": 5, "top": 2, "identity": 1, "groups": {"count": 3, "keep": 2}}
    z = torch.tensor([0.0, 1.0, 2.0, 3.0, 4.0, 5.0])
    s = torch.softmax(z, 0)
    chosen, weight = plain.route(z, torch.zeros(6), router)
    assert chosen.tolist() == [5, 4] and torch.allclose(weight, s[[5, 4]] / s[[5, 4]].sum())
    # corrections decide the groups and the choice, not the weights; choice scores below zero still beat a closed group's
    chosen, weight = plain.route(z, torch.tensor([0.9, -2.0, -1.0, -3.0, -2.0, -2.0]), dict(router, groups={"count": 3, "keep": 1}))
    assert chosen.tolist() == [0, 1] and torch.allclose(weight, s[[0, 1]] / s[[0, 1]].sum())
