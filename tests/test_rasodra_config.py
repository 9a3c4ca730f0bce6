"""Rasodra without a GPU: its configuration keys and their errors, the ModelSpec they become (run order, needs, tensor names), the cache's
chunks, steps and generation of a model in host memory on the null device, and the plain implementation pinned by closed forms."""
import copy
import math

import pytest
import torch

import plain_rasodra as plain
import rasodra_common as C
from tq_kv_amd import Engine, GenerationParams, Model, generate
from tq_kv_amd.cache import PAGE, Cache
from tq_kv_amd.config import ConfigError, config_from_dict, known_architectures
from tq_kv_amd.config.registry import spec_from_dict
from tq_kv_amd.parts.spec import KVNeed, ModelSpec, need_from_json


def test_the_architecture_is_known_by_its_name():
    assert "Rasodra" in known_architectures()
    name, typed = config_from_dict(C.config_mixed())
    assert name == "Rasodra"
    assert config_from_dict(typed.to_dict())[1] == typed                # round trip through config.json
    assert (typed.vocab, typed.width, typed.norm_eps) == (331, 96, 3e-6)
    assert [l.source for l in typed.layers] == [0, 1, 2, 1, 4, 0, 6, 7, 2, 0, 1] == [plain.source_of(C.config_mixed()["layers"], i) for i in range(11)]
    assert typed.layers[2].mixer["chunk"] == 37 and typed.layers[0].mixer["gate_cap"] == 6.0 and typed.layers[7].mlp is None


def test_the_spec_names_tensors_parts_and_needs():
    cfg = C.config_mixed()
    spec = spec_from_dict(cfg)
    assert ModelSpec.from_json(spec.to_json()) == spec
    assert spec.embedding_name == "embed" and spec.head_name == "head" and spec.final_norm_prefix == "final.norm" and spec.final_norm.kind == "layer_norm"
    assert [l.prefix for l in spec.layers] == ["l0.", "l1.", "l2.", "l4.", "l6.", "l7."]
    assert [r.layer for r in spec.order] == [0, 1, 2, 1, 3, 0, 4, 5, 2, 0, 1] and all(r.cache_of is None for r in spec.order)
    assert all(l.block.kind == "pre_norm" and l.block.params["post_mixer_norm"].params["bias"] is False for l in spec.layers)
    assert [l.block.params["mixer"].kind for l in spec.layers] == ["mlstm", "latent_attention", "attention", "attention", "mlstm", "latent_attention"]
    lat = spec.layers[1].block.params["mixer"].params
    assert (lat["q_rank"], lat["gate_per"], lat["sink"], lat["position"].params["style"], lat["position"].params["rot_dim"]) == (None, "element", True, "pairs", 8)
    att = spec.layers[2].block.params["mixer"].params
    assert (att["values_are_keys"], att["qkv_bias"], att["qk_norm"], att["chunk"], att["position"].params["rot_dim"]) == (True, True, True, 37, 16)
    model = Model(spec, dtype="float32", device="cpu")
    specs = model.tensor_specs()
    w = C.weights(cfg, 1)
    assert set(specs) == set(w)
    for name, t in w.items():
        assert list(t.shape) == list(specs[name].shape), name
    # the cache: every run has an entry of its own, whoever's tensors it uses
    needs = model.needs
    assert len(needs) == 11
    assert needs[0].shape == ((3 * (24 * 40 + 24) + 3 + 3) // 4 * 4,) and needs[1].key_page == (PAGE, 64) and needs[1].value_page == (56, PAGE)
    assert needs[2] == KVNeed(3, 24, None, None, chunk=37) and needs[8] == needs[2] and needs[4].chunk == 70
    assert need_from_json(needs[2].to_json()) == needs[2]


@pytest.mark.parametrize("path,value,word", [
    (("width",), None, "width"), (("vocab",), "many", "vocab"), (("norm",), None, "norm"), (("norm", "eps"), None, "eps"), (("layers",), [], "layers"),
    (("layers", 0, "type"), "convolution", "convolution"), (("layers", 0, "mixer"), None, "mixer"), (("layers", 0, "mixer", "gate_cap"), 0, "gate_cap"),
    (("layers", 6, "mixer", "dim"), 600, "key channels"), (("layers", 7, "mixer", "kv_rank"), 600, "latent"), (("layers", 1, "mixer", "kv_rank"), None, "kv_rank"),
    (("layers", 1, "mixer", "rot", "dims"), 10, "rot_dim"), (("layers", 2, "mixer", "kv_heads"), 4, "kv_heads"), (("layers", 2, "mixer", "vdim"), 32, "vdim"),
    (("layers", 2, "mixer", "mask"), None, "mask"), (("layers", 2, "mixer", "mask", "size"), 0, "size"), (("layers", 2, "mixer", "rot", "dims"), 7, "dims"),
    (("layers", 4, "mixer", "dim"), 300, "dim"), (("layers", 0, "mlp", "kind"), "sparse", "sparse"), (("layers", 0, "mlp", "ff"), None, "ff"),
    (("layers", 1, "weights_of"), 3, "weights_of"), (("layers", 3, "weights_of"), 11, "weights_of"), (("layers", 3, "weights_of"), 2, "type"), (("layers", 3, "mixer", "vdim"), 48, "mixer"), (("layers", 3, "mlp"), None, "mlp")])
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


def test_more_kinds_of_chunks_than_the_cache_has_groups():
    """Chunks of seventeen different sizes beside a latent: the chunked layers keep every page and share one group."""
    layers = [(C.chunked(2, 1, 8, 5 + n, 4), None) for n in range(17)] + [(C.latent(2, 8, 4, 8, 12), None)]
    model = Model(spec_from_dict(C.config(40, 32, layers)), dtype="float32", device="cpu")
    assert all(n.chunk == 0 for n in model.needs) and len({(n.key_page, n.n_kv_heads) for n in model.needs}) == 2
    few = Model(spec_from_dict(C.config(40, 32, layers[:3])), dtype="float32", device="cpu")
    assert [n.chunk for n in few.needs] == [5, 6, 7]


def test_a_group_of_chunks_gives_pages_back():
    full, chunk = KVNeed(2, 16, None), KVNeed(2, 16, None, chunk=150)
    c = Cache([full, chunk, KVNeed(2, 16, 100, chunk=150)], [None] * 3, PAGE * 8, 4, torch.float32, "cpu")
    assert len(c.kv_groups) == 3
    all_, own, both = c.kv_groups
    s = c.acquire()
    for length, first in ((149, 0), (150, 150), (151, 150), (299, 150), (300, 300), (310, 300)):
        c.reserve([(s, length - c.length(s))])
        assert own.pool.n_held <= (length + PAGE - 1) // PAGE
        c.commit([(s, length - c.length(s))])
        held = [k for k, p in enumerate(own.pages[s]) if p >= 0]
        assert held == list(range(first // PAGE, (length + PAGE - 1) // PAGE)), length
        assert own.first_needed(length) == first and both.first_needed(length) == max(first, length - 99)
        held = [k for k, p in enumerate(both.pages[s]) if p >= 0]
        assert held == list(range(max(first, length - 99) // PAGE, (length + PAGE - 1) // PAGE)), length
        c.check()
    assert all_.pool.n_held == 5
    c.release(s)
    assert own.pool.n_held == 0 and both.pool.n_held == 0


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
def test_plain_matrix_memory_without_its_maximum():
    """The running maximum only keeps the numbers small: without it, S~_t = sum_s exp(a_s + f_(s+1) + ... + f_t) k_s v_s^T, and the output
    is S~^T q over max(|n~ . q|, 1) but for the 1e-6."""
    g = torch.Generator().manual_seed(3)
    T, H, d, dv = 12, 2, 3, 4
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=torch.float64) for n in (d, d, dv))
    a = 3.0 * torch.randn(T, H, generator=g, dtype=torch.float64)
    f = -torch.rand(T, H, generator=g, dtype=torch.float64)
    out, (S, n, m) = plain.matrix_memory(q, k, v, a, f)
    for h in range(H):
        for t in range(T):
            w = torch.stack([torch.exp(a[s, h] + f[s + 1:t + 1, h].sum()) for s in range(t + 1)])
            dots = w * (k[:t + 1, h] @ q[t, h])
            want = (dots[:, None] * v[:t + 1, h]).sum(0) / max(abs(float(dots.sum())), 1.0)
            assert torch.allclose(out[t, h], want, rtol=1e-4, atol=1e-5)
    assert (m >= 0).any() or (m > -20).all()
    # the state carries over: in two pieces as in one
    first, state = plain.matrix_memory(q[:5], k[:5], v[:5], a[:5], f[:5])
    second, _ = plain.matrix_memory(q[5:], k[5:], v[5:], a[5:], f[5:], *state)
    assert torch.allclose(torch.cat([first, second]), out)


def test_plain_gates_sink_chunks_and_norm_in_closed_form():
    a, f = plain.gate_logarithms(torch.tensor([0.0, 100.0]), torch.tensor([0.0, -100.0]), 4.0)
    assert torch.allclose(a, torch.tensor([0.0, 4.0])) and torch.allclose(f, torch.tensor([-math.log(2.0), -4.0 - math.log1p(math.exp(-4.0))]))
    # a sink as large as the one score halves its weight; it counts once however many keys there are
    assert torch.allclose(plain.softmax_of(torch.tensor([2.0]), torch.tensor(2.0)), torch.tensor([0.5]))
    assert torch.allclose(plain.softmax_of(torch.zeros(3), torch.tensor(0.0)), torch.full((3,), 0.25))
    assert [plain.visible(i, 37) for i in (0, 36, 37, 73, 74)] == [0, 0, 37, 37, 74]
    assert torch.allclose(plain.layer_norm(torch.tensor([[1.0, 3.0]]), torch.tensor([2.0, 2.0]), 0.0), torch.tensor([[-2.0, 2.0]]))
    v = torch.tensor([[[1.0, 0.0, 0.0, 2.0, 5.0, 7.0]]]).expand(3, 1, 6)
    pairs = plain.turn_pairs(v, plain.angles(torch.arange(3), 16.0, 4))[2, 0]         # angles: position, position / 4
    assert torch.allclose(pairs, torch.tensor([math.cos(2.0), math.sin(2.0), -2.0 * math.sin(0.5), 2.0 * math.cos(0.5), 5.0, 7.0]), atol=1e-6)
