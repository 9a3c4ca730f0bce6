"""The Kezasun decoder through the library against the plain implementation (plain_kezasun.py): each mechanism alone through its part,
then whole models through Engine.step and generate() with every way of cutting and batching, on configurations made here."""
import pytest
import torch

import kezasun_common as C
import plain_kezasun as plain
from tq_kv_amd import Engine, GenerationParams, Model, generate
from tq_kv_amd.cache import Cache
from tq_kv_amd.engine.context import StepContext
from tq_kv_amd.parts import BuildEnv, PartSpec

pytestmark = pytest.mark.gpu
DEV = torch.device("cuda")
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
DTYPES = ["float32", "bfloat16"]
MAXPOS = 1024


@pytest.fixture(autouse=True)
def _seeded():
    torch.manual_seed(1234)


def position(rot):
    if rot["dims"] == 0:
        return PartSpec("none", {"max_positions": MAXPOS})
    p = {"theta": rot["base"], "rot_dim": rot["dims"], "max_positions": MAXPOS, "style": "halves"}
    if "scaling" in rot:
        p["scaling"] = rot["scaling"]
    return PartSpec("rotary", p)


def mixer_spec(kind, m, hidden, eps, own_kv=True, cache_window=None):
    if kind == "wkv":
        return PartSpec("time_mixing", {"hidden": hidden, "heads": m["heads"], "head_dim": m["dim"], "eps": eps})
    return PartSpec("attention", {"hidden": hidden, "n_heads": m["heads"], "n_kv_heads": m["kv_heads"], "head_dim": m["dim"], "value_dim": m["vdim"], "scale": m["scale"],
                                  "qkv_bias": True, "qk_norm": True, "qk_norm_over": "projection", "eps": eps, "window": m["mask"]["size"],
                                  "cache_window": cache_window or m["mask"]["size"], "sink_score": 0.0, "gate": "head", "own_kv": own_kv, "position": position(m["rot"]),
                                  "names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "gate": "g", "q_bias": "q.b", "k_bias": "k.b",
                                            "v_bias": "v.b"}})


SC = C.scaled(8.0, 1.0, 4.0, 64)
MIXERS = [C.wkv(3, 20), C.wkv(1, 1), C.wkv(2, 2), C.wkv(3, 10), C.wkv(5, 64), C.wkv(2, 128), C.wkv(1, 200), C.wkv(2, 68), C.wkv(5, 7), C.wkv(1, 300), C.wkv(6, 32),
          C.attention(6, 3, 24, 40, 37, 16, base=300.0, scale=0.35, scaling=SC), C.attention(1, 1, 2, 1, 1, 0), C.attention(3, 3, 10, 14, 9, 6, scaling=SC),
          C.attention(8, 2, 64, 64, 64, 64, scaling=C.scaled(4.0, 0.5, 8.0, 200)), C.attention(16, 2, 128, 128, 100, 32), C.attention(2, 1, 160, 200, 200, 40, scale=0.05),
          C.attention(5, 5, 32, 32, 130, 2), C.attention(6, 2, 96, 64, 1000, 96, scale=0.2), C.attention(40, 2, 32, 48, 63, 32), C.attention(6, 2, 64, 64, 129, 20),
          C.attention(4, 1, 16, 24, 65, 16, scale=-0.3)]


def step_ctx(cache, items):
    sizes = [(s, len(t)) for s, t in items]
    cache.reserve(sizes)
    return StepContext([(s, cache.length(s), t) for s, t in items], [[] for _ in items], cache, DEV), sizes


def mixer_ids(m):
    return m[0] + "-" + "x".join(str(v) for v in m[1].values() if isinstance(v, int)) + ("-%d" % m[1]["mask"]["size"] if "mask" in m[1] else "")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mix", MIXERS, ids=mixer_ids)
def test_a_mixer_alone(dtype, mix):
    """Two sequences in shared steps: one in portions of 230, 26, 2 and 2 tokens and then token by token, across pages' and chunks' borders; the
    other whole beside the first portion.  Then the slots are given back and taken again: nothing of the first use may be left."""
    kind, m = mix
    hidden, eps = 88, 1e-5
    cfg = C.config(50, hidden, [(mix, None)])
    w = {k[len("l0.mix."):]: v for k, v in C.weights(cfg, 3, codes=False).items() if k.startswith("l0.mix.")}
    part = BuildEnv(DEV, DT[dtype]).build("mixer", mixer_spec(kind, m, hidden, eps))
    assert part.graph_safe and sorted(part.tensors()) == sorted(w)
    part.load({k: v.to(DT[dtype]).to(DEV) for k, v in w.items()})
    need = part.cache_need()
    cache = Cache([need], [None], 64 * 8, 2, DT[dtype], DEV)
    assert len(cache.state_groups) == (kind == "wkv") and len(cache.kv_groups) == (kind == "attention")
    xs = [torch.randn(n, hidden).to(DT[dtype]) for n in (300, 40)]
    f = C.as_float(w)
    want = [plain.wkv(x.float(), f, "", m, eps, DT[dtype]) if kind == "wkv" else plain.attention(x.float(), f, "", m, eps, DT[dtype])[0] for x in xs]
    # (the first step is long enough for the recurrences to run in chunks, beside a sequence shorter than a chunk; the second is not)
    plan = [[(0, 0, 230), (1, 0, 40)], [(0, 230, 256)], [(0, 256, 258)], [(0, 258, 260)]] + [[(0, t, t + 1)] for t in range(260, 300)]
    for use in range(2):
        slots = [cache.acquire(), cache.acquire()]
        got = [[], []]
        for step in plan:
            ctx, sizes = step_ctx(cache, [(slots[i], [0] * (b - a)) for i, a, b in step])
            y = part.forward(torch.cat([xs[i][a:b] for i, a, b in step]).to(DEV), ctx, cache.entry(0))
            cache.commit(sizes)
            off = 0
            for i, a, b in step:
                got[i].append(y[off:off + b - a])
                off += b - a
        for i in range(2):
            e = C.row_errors(torch.cat(got[i]), want[i])
            # (where heads have one or two values, a row may come out next to zero, and its error is told by its own magnitude)
            limit = (5e-5 if dtype == "float32" else 0.06 if kind == "wkv" else 0.03) * (8.0 if m.get("vdim", m["dim"]) <= 2 else 1.0)
            assert e.max().item() < limit, "use %d, sequence %d: %.3g at row %d" % (use, i, e.max().item(), int(e.argmax()))
        for s in slots:
            cache.release(s)


@pytest.mark.parametrize("mix", [m for m in MIXERS if m[0] == "wkv"], ids=mixer_ids)
def test_time_mixing_is_as_exact_in_chunks_as_token_by_token(mix):
    """Inputs and weights of small whole numbers, so that the products come out as numbers that bfloat16 holds exactly: then the long step's kernels
    must leave the state that the token-by-token kernel leaves, far closer than bfloat16's rounding, and the outputs with it.  Decays from
    next to one down to nothing within a few tokens."""
    kind, m = mix
    hidden, eps = 88, 1e-5
    g = torch.Generator().manual_seed(5)
    w = {k[len("l0.mix."):]: v for k, v in C.weights(C.config(50, hidden, [(mix, None)]), 3, codes=False).items() if k.startswith("l0.mix.")}

    def ternary(shape, density):
        return (torch.randint(0, 2, shape, generator=g) * 2 - 1).float() * (torch.rand(shape, generator=g) < density).float()

    for k in ("r", "k", "v"):
        w[k] = ternary(w[k].shape, 0.15).to(torch.bfloat16)
    for s in "rkvgw":
        w["mu." + s] = torch.full((hidden,), 0.5 if s in "rv" else 0.0).to(torch.bfloat16)
    w["w0"] = torch.linspace(-8.0, 3.0, w["w0"].shape[0]).to(torch.bfloat16)
    part = BuildEnv(DEV, torch.bfloat16).build("mixer", mixer_spec(kind, m, hidden, eps))
    part.load({k: v.to(DEV) for k, v in w.items()})
    x = (2.0 * ternary((300, hidden), 0.6)).to(torch.bfloat16).to(DEV)
    states, outputs = [], []
    for cuts in ([300], [167, 300], list(range(1, 301))):
        cache = Cache([part.cache_need()], [None], 64 * 8, 2, torch.bfloat16, DEV)
        slot, a, out = cache.acquire(), 0, []
        for b in cuts:
            ctx, sizes = step_ctx(cache, [(slot, [0] * (b - a))])
            out.append(part.forward(x[a:b], ctx, cache.entry(0)))
            cache.commit(sizes)
            a = b
        states.append(cache.state_groups[0].state[0, slot].float().cpu().clone())
        outputs.append(torch.cat(out))
    for s, o in zip(states[:2], outputs[:2]):
        assert torch.isfinite(s).all()
        d = ((s - states[2]).norm() / states[2].norm().clamp_min(1e-6)).item()
        assert d < 5e-5, d
        e = C.row_errors(o, outputs[2])
        assert e.median().item() < 0.006 and e.max().item() < 0.1, (e.median().item(), e.max().item())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("z", [-30.0, -6.0, 0.0, 2.0, 6.0])
def test_decays_at_their_ends(z, dtype):
    """States that lose nothing for hundreds of tokens, that halve, and that are gone at once (a decay that underflows to zero)."""
    hidden, eps, mix = 40, 1e-5, C.wkv(2, 16)[1]
    w = {k[len("l0.mix."):]: v for k, v in C.weights(C.config(50, hidden, [(C.wkv(2, 16), None)]), 3, codes=False).items() if k.startswith("l0.mix.")}
    w["w0"] = torch.full_like(w["w0"], z)
    part = BuildEnv(DEV, DT[dtype]).build("mixer", mixer_spec("wkv", mix, hidden, eps))
    part.load({k: v.to(DT[dtype]).to(DEV) for k, v in w.items()})
    x = torch.randn(260, hidden).to(DT[dtype])
    want = plain.wkv(x.float(), C.as_float(w), "", mix, eps, DT[dtype])
    for cuts in ([260], [200, 260], [130, 131, 132, 260]):
        cache = Cache([part.cache_need()], [None], 64 * 8, 1, DT[dtype], DEV)
        slot, a, out = cache.acquire(), 0, []
        for b in cuts:
            ctx, sizes = step_ctx(cache, [(slot, [0] * (b - a))])
            out.append(part.forward(x[a:b].to(DEV), ctx, cache.entry(0)))
            cache.commit(sizes)
            a = b
        e = C.row_errors(torch.cat(out), want)
        assert torch.isfinite(e).all() and e.max().item() < (5e-5 if dtype == "float32" else 0.06), "cuts %s: %.3g at row %d" % (cuts, e.max().item(), int(e.argmax()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,borrowed", [(37, 37), (37, 90), (90, 20), (64, 1)])
def test_attention_on_another_runs_keys_and_values(window, borrowed, dtype):
    """Two runs on one cache: the first writes it, the second has queries, a window, a gate and an output of its own."""
    hidden, eps = 72, 1e-5
    lender = C.attention(6, 3, 24, 40, window, 16, base=300.0, scale=0.35, scaling=SC)[1]
    reader = dict(C.attention(6, 3, 24, 40, borrowed, 16, base=300.0, scale=0.5, scaling=SC)[1], kv_from=0)
    w = C.weights(C.config(50, hidden, [(("attention", lender), None), (("attention", reader), None)]), 3, codes=False)
    wa, wb = ({k[7:]: v for k, v in w.items() if k.startswith(p)} for p in ("l0.mix.", "l1.mix."))
    env = BuildEnv(DEV, DT[dtype])
    keep = max(window, borrowed)
    a = env.build("mixer", mixer_spec("attention", lender, hidden, eps, cache_window=keep))
    b = env.build("mixer", mixer_spec("attention", reader, hidden, eps, own_kv=False, cache_window=keep))
    assert sorted(b.tensors()) == sorted(wb) == sorted(["q", "q.b", "q.norm", "g", "o"]) and a.cache_need() == b.cache_need() and a.cache_need().window == keep
    a.load({k: v.to(DT[dtype]).to(DEV) for k, v in wa.items()})
    b.load({k: v.to(DT[dtype]).to(DEV) for k, v in wb.items()})
    cache = Cache([a.cache_need(), b.cache_need()], [None, 0], 64 * 8, 2, DT[dtype], DEV)
    x, y = torch.randn(260, hidden).to(DT[dtype]), torch.randn(260, hidden).to(DT[dtype])
    want_a, kv = plain.attention(x.float(), C.as_float(wa), "", lender, eps, DT[dtype])
    want_b, _ = plain.attention(y.float(), C.as_float(wb), "", reader, eps, DT[dtype], lent=kv)
    slot, at, got_a, got_b = cache.acquire(), 0, [], []
    for end in [150, 152, 220] + list(range(221, 261)):
        ctx, sizes = step_ctx(cache, [(slot, [0] * (end - at))])
        got_a.append(a.forward(x[at:end].to(DEV), ctx, cache.entry(0)))
        got_b.append(b.forward(y[at:end].to(DEV), ctx, cache.entry(1)))
        cache.commit(sizes)
        at = end
    limit = 5e-5 if dtype == "float32" else 0.03
    for got, want in ((got_a, want_a), (got_b, want_b)):
        e = C.row_errors(torch.cat(got), want)
        assert e.max().item() < limit, "%.3g at row %d" % (e.max().item(), int(e.argmax()))


ROUTERS = [C.moe(40, 9, 3, 3, 4, 2), C.moe(8, 1, 1), C.moe(8, 1, 2, 1), C.moe(22, 3, 2, 2, 5, 3), C.moe(16, 6, 6, 2, 1, 1), C.moe(32, 60, 4, 4, 16, 3), C.moe(16, 2, 1, 6, 4, 1),
           C.moe(64, 100, 8, 28, 128, 100), C.moe(24, 130, 5, 6, 2, 1), C.moe(64, 16, 4), C.moe(192, 5, 3, 3, 4, 2), C.moe(64, 2, 2)]


def router_ids(m):
    r = m["router"]
    return "%d+%d-top%d-%d-of-%d" % (r["experts"], r["identity"], r["top"], r["groups"]["keep"], r["groups"]["count"])


def experts_spec(mlp, hidden):
    r = mlp["router"]
    return PartSpec("routed_experts", {"hidden": hidden, "inter": mlp["expert"]["ff"], "n_experts": r["experts"], "top": r["top"], "router_scale": 1.0, "gate": "silu",
                                       "normalize": "chosen", "identity": r["identity"], "correction": "correction", "n_groups": r["groups"]["count"],
                                       "keep_groups": r["groups"]["keep"], "weight_floor": 1e-20, "shared": None})


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [64, 50])
@pytest.mark.parametrize("mlp", ROUTERS, ids=router_ids)
def test_experts_alone(mlp, hidden, dtype):
    """Corrections as large as the scores (of both signs: choice scores below zero among them), groups, experts that give back their input."""
    w = {k[len("l0.mlp."):]: v for k, v in C.weights(C.config(50, hidden, [(C.wkv(1, 4), mlp)]), 3, codes=False).items() if k.startswith("l0.mlp.")}
    w["correction"] = (w["correction"].float() * 4.0 - 0.3).to(torch.bfloat16)
    ff = BuildEnv(DEV, DT[dtype]).build("feed_forward", experts_spec(mlp, hidden))
    assert ff.graph_safe and sorted(ff.tensors()) == sorted(w)
    ff.load({k: v.to(DT[dtype]).to(DEV) for k, v in w.items()})
    cache = Cache([], [], 64, 1, DT[dtype], DEV)
    f = C.as_float(w)
    for rows in (1, 5, 130) + ((700,) if mlp["expert"]["ff"] >= 64 else ()):          # (up to experts of several tiles of every size)
        x = torch.randn(rows, hidden).to(DT[dtype])
        ctx = StepContext([(0, 0, [0] * rows)], [[]], cache, DEV)
        got = ff.forward(x.to(DEV), ctx)
        e = C.row_errors(got, plain.experts(x.float(), f, "", mlp, DT[dtype]))
        assert e.max().item() < (2e-5 if dtype == "float32" else 0.03), "%d rows: %.3g at row %d" % (rows, e.max().item(), int(e.argmax()))


def test_a_group_is_kept_for_its_best_choice_score_and_choices_stay_inside():
    """Two groups: the corrections lift one group's best above the other's although the other holds the larger scores; every choice score is
    negative; the second choice is the kept group's, however small."""
    hidden, mlp = 32, C.moe(8, 5, 2, 1, 2, 1)
    ff = BuildEnv(DEV, torch.float32).build("feed_forward", experts_spec(mlp, hidden))
    w = {k[len("l0.mlp."):]: v.float() for k, v in C.weights(C.config(50, hidden, [(C.wkv(1, 4), mlp)]), 9, codes=False).items() if k.startswith("l0.mlp.")}
    w["router"] = torch.zeros(6, hidden)
    w["router"][:, 0] = torch.tensor([3.0, 2.0, 1.0, 0.5, 0.0, 0.2])
    w["correction"] = torch.tensor([-3.0, -3.0, -3.0, -1.0, -9.0, -5.0])
    ff.load({k: v.to(DEV) for k, v in w.items()})
    x = torch.randn(3, hidden)
    x[:, 0] = 1.0
    s = torch.softmax(w["router"][:, 0], 0)
    chosen, weight = plain.route(w["router"][:, 0], w["correction"], mlp["router"])
    assert chosen.tolist() == [3, 5] and torch.allclose(weight, s[[3, 5]] / (s[3] + s[5]))
    want = torch.stack([weight[0] * plain.expert(x[t:t + 1], w, "e3.", torch.float32)[0] + weight[1] * x[t] for t in range(3)])
    got = ff.forward(x.to(DEV), StepContext([(0, 0, [0] * 3)], [[]], Cache([], [], 64, 1, torch.float32, DEV), DEV)).cpu()
    assert torch.allclose(got, want, atol=1e-5)


# ---- whole models ----------------------------------------------------------------------------------------
_MODELS = {}
MAKERS = {"mixed": C.config_mixed, "ones": C.config_ones, "odd": C.config_odd, "wkv": lambda: C.config_single("wkv"), "slow": lambda: C.config_single("wkv"),
          "attention": lambda: C.config_single("attention"),
          "wide1030": lambda: C.config(61, 1030, [(C.attention(2, 1, 16, 16, 40, 8), C.moe(24, 3, 2, 1)), (C.wkv(2, 8), C.moe(16, 2, 1))]),
          "wide4160": lambda: C.config(61, 4160, [(C.wkv(2, 16), C.moe(32, 3, 2, 1)), (C.attention(2, 1, 16, 16, 40, 8), None), (C.wkv(2, 16), C.moe(32, 2, 2))]),
          "wide9000": lambda: C.config(61, 9000, [(C.wkv(2, 16), C.moe(32, 2, 1)), (C.attention(2, 2, 32, 32, 50, 32), C.moe(16, 2, 1, 1))])}


def model(name, tmp_path_factory):
    if name not in _MODELS:
        cfg = MAKERS[name]()
        w = C.weights(cfg, seed=11 + len(name))
        if name == "slow":              # decays next to one: the state reaches back hundreds of tokens
            w["l0.mix.w0"] = torch.full_like(w["l0.mix.w0"], -8.0)
        _MODELS[name] = (cfg, w, C.write_folder(str(tmp_path_factory.mktemp("kezasun_%s" % name)), cfg, w), {})
    return _MODELS[name]


def engine(name, dtype, tmp_path_factory, max_tokens=4096, slots=8):
    cfg, w, folder, engines = model(name, tmp_path_factory)
    if dtype not in engines:
        engines[dtype] = Engine(Model.from_dir(folder, dtype=dtype), max_tokens=max_tokens, max_slots=slots)
    return cfg, w, engines[dtype]


def run_cut(eng, toks, cuts):
    """One request alone, its tokens in portions that end at `cuts`; the logits of every position."""
    s = eng.open()
    out, a = [], 0
    for b in list(cuts) + [len(toks)]:
        b = min(b, len(toks))
        if b > a:
            out.append(eng.step([(s, toks[a:b], list(range(b - a)))]))
            a = b
    eng.close(s)
    return torch.cat(out)


def spread(got, want):
    """Per row: the root mean square of the difference (its mean taken off) over the spread of all that is wanted."""
    d = got.float().cpu() - want.float().cpu()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.float().std().clamp_min(1e-6)


class Wanted:
    """The plain logits of a sequence, and what rounding alone does to them: the plain computation with its products rounded to bfloat16.
    A norm of a head's output makes small outputs as large as any, and with them their rounding, so the size of that is the sequence's own."""

    def __init__(self, cfg, w, toks):
        f = C.as_float(w)
        self.rows = plain.forward(cfg, f, toks)
        self.rounding = spread(plain.forward(cfg, f, toks, low=torch.bfloat16), self.rows).max().item()


def close(got, want, dtype, what="", rows=None):
    """got: logits of the rows (a slice or list; all unless given) of want."""
    wanted = want.rows if rows is None else want.rows[rows]
    assert got.shape == wanted.shape, "%s: shapes %s and %s" % (what, tuple(got.shape), tuple(wanted.shape))
    d = got.float().cpu() - wanted
    d = d - d.mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / want.rows.std().clamp_min(1e-6)
    assert torch.isfinite(e).all(), "%s: logits are not finite" % what
    limit = 1e-4 if dtype == "float32" else max(0.06, 2.5 * want.rounding)
    assert e.max().item() <= limit, "%s: row error %.3g at row %d (limit %.3g)" % (what, e.max().item(), int(e.argmax()), limit)


_WANTED = {}


def wanted(name, cfg, w, toks):
    key = (name, tuple(toks))
    if key not in _WANTED:
        _WANTED[key] = Wanted(cfg, w, toks)
    return _WANTED[key]


def plain_logits(cfg, w, toks):
    return plain.forward(cfg, C.as_float(w), toks)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "ones", "odd"])
def test_whole_prompts_and_every_cut(name, dtype, tmp_path_factory):
    cfg, w, eng = engine(name, dtype, tmp_path_factory)
    assert eng.model.spec.architecture == "Kezasun" and eng.model.graph_safe and len(eng.model.spec.order) == len(cfg["layers"])
    toks = C.tokens(200, cfg["vocab"], 5)
    want = wanted(name, cfg, w, toks)
    whole = run_cut(eng, toks, [])
    close(whole, want, dtype, "whole")
    for cuts in ([64], [63, 65], [1, 3, 128, 130], [37, 74], [150, 152, 154] + list(range(155, 200)), list(range(2, 200, 2)), list(range(1, 200))):
        got = run_cut(eng, toks, cuts)
        close(got, want, dtype, "cuts %s" % cuts[:4])
        if dtype == "float32":          # no sum depends on the cut: states are carried exactly
            assert torch.equal(got, whole), "float32 logits depend on the cut %s" % cuts[:4]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["wide1030", "wide4160", "wide9000"])
def test_streams_of_other_widths(name, dtype, tmp_path_factory):
    """Widths that take the kernels between the layers in all their shapes (experts' sum, stream and next norm in one pass of one or two pieces a
    thread, or in two kernels), in prompts and in steps of few and of many sequences."""
    cfg, w, eng = engine(name, dtype, tmp_path_factory, slots=24)
    toks = C.tokens(60, cfg["vocab"], 5)
    want = wanted(name, cfg, w, toks)
    for cuts in ([], [40], list(range(50, 60))):
        close(run_cut(eng, toks, cuts), want, dtype, "cuts %s" % cuts[:3])
    reqs = [C.tokens(2 + i % 3, cfg["vocab"], 300 + i) for i in range(20)]
    slots = [eng.open() for _ in reqs]
    eng.step([(s, r[:-1], []) for s, r in zip(slots, reqs)])
    got = eng.step([(s, r[-1:], [0]) for s, r in zip(slots, reqs)])
    for i in (0, 1, 2, 19):
        close(got[i:i + 1], wanted(name, cfg, w, reqs[i]), dtype, "sequence %d" % i, [len(reqs[i]) - 1])
    for s in slots:
        eng.close(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_prompt_of_which_one_row_is_wanted(dtype, tmp_path_factory):
    """Steps that want their last row alone (the last layer goes on with the wanted rows; once with a feed-forward, once without)."""
    for name in ("mixed", "odd", "attention", "wkv"):
        cfg, w, eng = engine(name, dtype, tmp_path_factory)
        toks = C.tokens(150, cfg["vocab"], 6)
        want = wanted(name, cfg, w, toks)
        s, t = eng.open(), eng.open()
        got = eng.step([(s, toks, [149]), (t, toks[:70], [3, 69])])
        close(got, want, dtype, name, [149, 3, 69])
        assert eng.step([(t, toks[70:140], [])]).shape[0] == 0
        close(eng.step([(t, toks[140:], [9])]), want, dtype, name, [149])
        eng.close(s), eng.close(t)


def poison(eng):
    """NaN into every page that no sequence holds and into the state rows of every slot that is free: nothing may read them
    (a slot's state is cleared when the slot is taken)."""
    for g in eng.cache.kv_groups:
        held = {p for pages in g.pages.values() for p in pages if p >= 0}
        free = [p for p in range(g.pool.n) if p not in held]
        if free:
            g.keys[:, torch.tensor(free, device=g.keys.device)] = float("nan")
            g.values[:, torch.tensor(free, device=g.keys.device)] = float("nan")
    free = [s for s in range(eng.cache.max_slots) if not eng.cache.slots.is_held(s)]
    for g in eng.cache.state_groups:
        if free:
            g.state[:, torch.tensor(free, device=g.state.device)] = float("nan")


@pytest.mark.parametrize("dtype", DTYPES)
def test_batches_of_unequal_requests_and_reused_slots(dtype, tmp_path_factory):
    cfg, w, _ = engine("mixed", dtype, tmp_path_factory)
    eng = Engine(Model.from_dir(model("mixed", tmp_path_factory)[2], dtype=dtype), max_tokens=64 * 8, max_slots=4)
    reqs = [C.tokens(n, cfg["vocab"], 30 + n) for n in (130, 7, 66, 1, 95, 64, 20)]
    want = [wanted("mixed", cfg, w, t) for t in reqs]
    alone = [run_cut(eng, t, []) for t in reqs]
    # three batches one after the other in a cache that only holds them because ended requests give pages and slots back;
    # what they leave behind is overwritten with NaN as soon as nobody holds it
    for batch in ([0, 1, 2, 3], [4, 5, 6, 1], [2, 0, 4]):
        heads = {i: max(1, len(reqs[i]) - 3 - 5 * k) for k, i in enumerate(batch)}
        slots = {i: eng.open() for i in batch}
        poison(eng)
        got = eng.step([(slots[i], reqs[i][:heads[i]], list(range(heads[i]))) for i in batch])
        off = 0
        for i in batch:
            close(got[off:off + heads[i]], want[i], dtype, "prompt of %d in a batch" % i, slice(heads[i]))
            if dtype == "float32":
                assert torch.equal(got[off:off + heads[i]], alone[i][:heads[i]])
            off += heads[i]
        pos, live = dict(heads), [i for i in batch if heads[i] < len(reqs[i])]
        for i in batch:
            if i not in live:
                eng.close(slots[i])
        while live:
            poison(eng)
            got = eng.step([(slots[i], [reqs[i][pos[i]]], [0]) for i in live])
            for k, i in enumerate(live):
                close(got[k:k + 1], want[i], dtype, "request %d decoded at %d" % (i, pos[i]), [pos[i]])
                if dtype == "float32":
                    assert torch.equal(got[k], alone[i][pos[i]])
                pos[i] += 1
            for i in live:
                if pos[i] == len(reqs[i]):
                    eng.close(slots[i])
            live = [i for i in live if pos[i] < len(reqs[i])]
    eng.cache.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [20, 40, 130])
def test_steps_of_many_sequences(dtype, rows, tmp_path_factory):
    """One token each of more sequences than the few-row products take, and of more than the mid-sized ones take: beside each alone."""
    cfg, w, folder, _ = model("mixed", tmp_path_factory)
    eng = Engine(Model.from_dir(folder, dtype=dtype), max_tokens=64 * rows, max_slots=rows)
    reqs = [C.tokens(3 + i % 5, cfg["vocab"], 200 + i) for i in range(rows)]
    slots = [eng.open() for _ in reqs]
    eng.step([(s, r[:-1], []) for s, r in zip(slots, reqs)])
    got = eng.step([(s, r[-1:], [0]) for s, r in zip(slots, reqs)])
    for i in (0, 1, 2, 3, 4, rows // 2, rows - 1):
        close(got[i:i + 1], wanted("mixed", cfg, w, reqs[i]), dtype, "sequence %d of %d" % (i, rows), [len(reqs[i]) - 1])


def window_only(tmp_path_factory, window, borrowed=None):
    key = "edges_%d_%s" % (window, borrowed)
    if key not in _MODELS:
        a = dict(heads=4, kv_heads=2, dim=16, vdim=24, rot_dims=8, base=100.0, scale=0.5)
        layers = [(C.attention(window=window, **a), None)]
        if borrowed is not None:
            layers.append((C.attention(window=borrowed, kv_from=0, **a), None))
        cfg = C.config(60, 48, layers)
        w = C.weights(cfg, 21)
        _MODELS[key] = (cfg, w, C.write_folder(str(tmp_path_factory.mktemp("kezasun_" + key)), cfg, w), {})
    return key


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,borrowed", [(1, None), (37, None), (64, None), (65, None), (128, None), (150, None), (500, None), (20, 90), (90, 20)])
def test_what_a_position_sees_of_its_window(window, borrowed, dtype, tmp_path_factory):
    """Changing the token at j changes the logits at i if and only if 0 <= i - j < window (the larger of the two where a second layer reads the
    first one's keys and values): keys just inside and just outside, at the sequence's start and at pages' borders; queries in a prompt, in a
    later portion, and decoded one by one."""
    cfg, w, eng = engine(window_only(tmp_path_factory, window, borrowed), dtype, tmp_path_factory)
    n, reach = 200, max(window, borrowed or 0)
    toks = C.tokens(n, cfg["vocab"], 8)

    def logits_of(seq, how):
        return run_cut(eng, seq, {"prompt": [], "portions": [61, 63, 130], "decoded": [120] + list(range(121, n))}[how])

    for how in ("prompt", "portions", "decoded"):
        base = logits_of(toks, how)
        close(base, wanted("window%d_%s" % (window, borrowed), cfg, w, toks), dtype, how)
        for i in (130, 149, 150, 192, 199):
            lo = i - reach + 1
            for j in sorted({0, 1, 63, 64, 65, 127, 128, lo - 2, lo - 1, lo, lo + 1, i - 1, i, i + 1}):
                if j < 0 or j >= n:
                    continue
                changed = list(toks)
                changed[j] = (toks[j] + 1 + j) % cfg["vocab"]
                moved = (logits_of(changed, how)[i] - base[i]).abs().max().item()
                if lo <= j <= i:
                    assert moved > 0.0 or dtype == "bfloat16", "%s: query %d does not see the token at %d" % (how, i, j)
                else:
                    assert moved == 0.0, "%s: query %d sees the token at %d" % (how, i, j)


def one_key(tmp_path_factory, borrowed):
    """A model in which two tokens have an element of the embedding to themselves; the keys of the one and the queries of the other read it with
    one and the same long vector, so that this one key stands far above everything else the query sees.  borrowed: in a second layer that
    reads the first one's keys and values through a larger window."""
    a = dict(heads=2, kv_heads=1, dim=64, vdim=40, rot_dims=0, scale=0.5)
    layers = [(C.attention(window=250, **a), None)]
    if borrowed:
        layers = [(C.attention(window=30, **a), None), (C.attention(window=250, kv_from=0, **a), None)]
    cfg = C.config(60, 32, layers)
    special, asker = 7, 11
    f = C.as_float(C.weights(cfg, 4, codes=False))
    f["embed"][:, :2] = 0.0
    f["embed"][special, 0] = f["embed"][asker, 1] = 3.0
    direction = torch.randn(64)
    for k in list(f):
        if k.endswith("q.norm") or k.endswith("k.norm"):
            f[k].fill_(1.0)
        if k.endswith("norm1"):
            f[k].zero_()
        if k.endswith("mix.o"):
            f[k][:2] = 0.0                     # (the two elements stay what the embedding made them)
        if k.endswith("mix.q"):
            f[k][:, 1] = 6.0 * direction.repeat(2)
    f["l0.mix.k"][:, 0] = 6.0 * direction
    w = {k: v.to(torch.bfloat16) for k, v in f.items()}
    return cfg, w, C.write_folder(str(tmp_path_factory.mktemp("kezasun_far")), cfg, w), special, asker


@pytest.mark.parametrize("borrowed", [False, True])
def test_one_key_far_away_carries_the_output(borrowed, tmp_path_factory):
    """The output at the query is the one key's value, wherever its token stands (at a page's border, at the window's first place, just before
    the query), however the query comes (in the prompt or decoded); and with the key in front of the window, it is not."""
    cfg, w, folder, special, asker = one_key(tmp_path_factory, borrowed)
    n = 330
    toks = [t if t not in (special, asker) else 20 for t in C.tokens(n, cfg["vocab"], 2)]
    for dtype in DTYPES:
        eng = Engine(Model.from_dir(folder, dtype=dtype), max_tokens=1024, max_slots=2)
        for place in (0, 63, 78, 79, 80, 81, 127, 128, 251, 320, n - 2):
            seq = list(toks)
            seq[place], seq[n - 1] = special, asker
            want = wanted("far%s" % borrowed, cfg, w, seq)
            other = list(seq)
            other[place] = 21
            difference = C.row_errors(wanted("far%s" % borrowed, cfg, w, other).rows[-1:], want.rows[-1:]).item()
            assert (difference > 0.1) if place >= 80 else difference == 0.0, (place, difference)          # the one key matters
            close(run_cut(eng, seq, [])[-1:], want, dtype, "prompt, key at %d" % place, [n - 1])
            close(run_cut(eng, seq, [300] + list(range(301, n)))[-1:], want, dtype, "decoded, key at %d" % place, [n - 1])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("length", [1, 2, 5, 64, 65, 200])
def test_the_one_in_the_denominator(length, dtype, tmp_path_factory):
    """Scores far below zero (the denominator is nearly the one alone), around it and far above, in prompts (tiles), in decoding (one part or
    several, merged) and for the first tokens, where it weighs most."""
    for scale in (0.02, 2.0, -0.5):
        key = "sink_%g" % scale
        if key not in _MODELS:
            cfg = C.config(60, 48, [(C.attention(6, 2, 16, 24, 1000, 8, base=100.0, scale=scale), None)])
            w = C.weights(cfg, 22)
            _MODELS[key] = (cfg, w, C.write_folder(str(tmp_path_factory.mktemp("kezasun_" + key)), cfg, w), {})
        cfg, w, eng = engine(key, dtype, tmp_path_factory)
        toks = C.tokens(length, cfg["vocab"], length)
        want = wanted(key, cfg, w, toks)
        close(run_cut(eng, toks, []), want, dtype, "prompt")
        close(run_cut(eng, toks, list(range(1, length))), want, dtype, "one by one")


def test_plain_scores_below_zero_show_the_one(tmp_path_factory):
    """(What the test above rests on: without the one, the logits would be others.)"""
    cfg = C.config(60, 48, [(C.attention(6, 2, 16, 24, 1000, 8, base=100.0, scale=0.02), None)])
    w = C.as_float(C.weights(cfg, 22))
    toks = C.tokens(5, 60, 5)
    want = plain.forward(cfg, w, toks)
    kept = plain.softmax_with_one
    try:
        plain.softmax_with_one = lambda s: torch.softmax(s, -1)
        assert C.row_errors(plain.forward(cfg, w, toks), want).min().item() > 0.02
    finally:
        plain.softmax_with_one = kept


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[1], [2], [64], [65, 66], [100, 102]])
def test_the_previous_token_at_the_start_of_a_portion(cuts, dtype, tmp_path_factory):
    """A portion's first token mixes with the last one of the portion before, a sequence's first with nothing: a model whose mixes are the previous
    token alone, and whose state is gone at once, so that nothing else of the past is left."""
    key = "shift"
    if key not in _MODELS:
        cfg = C.config(60, 40, [(C.wkv(2, 16), None)])
        w = C.weights(cfg, 23)
        for s in "rkvgw":
            w["l0.mix.mu." + s] = torch.ones_like(w["l0.mix.mu." + s])
        w["l0.mix.w0"] = torch.full_like(w["l0.mix.w0"], 8.0)
        _MODELS[key] = (cfg, w, C.write_folder(str(tmp_path_factory.mktemp("kezasun_shift")), cfg, w), {})
    cfg, w, eng = engine(key, dtype, tmp_path_factory)
    toks = C.tokens(110, cfg["vocab"], 4)
    want = wanted(key, cfg, w, toks)
    close(run_cut(eng, toks, cuts), want, dtype, "cuts %s" % cuts)
    for c in cuts:
        other = list(toks)
        other[c - 1] = (toks[c - 1] + 1) % cfg["vocab"]
        assert C.row_errors(plain_logits(cfg, w, other)[c:c + 1], want.rows[c:c + 1]).item() > 0.02
        assert torch.equal(plain_logits(cfg, w, other)[c + 2:], want.rows[c + 2:])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["slow"])
def test_the_first_token_reaches_the_last(name, dtype, tmp_path_factory):
    """Hundreds of tokens: the first one still moves the last logits, and the library agrees with the plain implementation there, in a prompt
    and after two hundred decoded tokens."""
    cfg, w, eng = engine(name, dtype, tmp_path_factory)
    n = 500
    toks = C.tokens(n, cfg["vocab"], 17)
    want = wanted(name, cfg, w, toks)
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    assert (plain_logits(cfg, w, other)[-1] - want.rows[-1]).abs().max().item() > 1e-4
    close(run_cut(eng, toks, []), want, dtype, "prompt")
    close(run_cut(eng, toks, [300] + list(range(301, n))), want, dtype, "decoded")


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_loop(dtype, tmp_path_factory):
    cfg, w, eng = engine("mixed", dtype, tmp_path_factory)
    prompts = [C.tokens(n, cfg["vocab"], 50 + n) for n in (1, 9, 70, 33, 128)]
    params = GenerationParams(max_tokens=12, temperature=0.0, repeat_penalty=1.0)
    out = generate(eng, prompts, params, eos_ids=(), max_batch=3)
    for p, o in zip(prompts, out):
        assert len(o) == 12
        z = plain_logits(cfg, w, list(p) + o)
        for k, t in enumerate(o):
            row = z[len(p) - 1 + k]
            # a step whose two best logits are closer than rounding may go either way
            assert int(row.argmax()) == t or (dtype == "bfloat16" and (row.max() - row[t]).item() < 0.15 * row.std().item()), "token %d of a prompt of %d" % (k, len(p))
    again = generate(eng, prompts[::-1], params, eos_ids=(), max_batch=2)
    assert again[::-1] == out or dtype == "bfloat16"


@pytest.mark.parametrize("dtype", DTYPES)
def test_replay_of_steps_and_the_command_line(dtype, tmp_path_factory):
    """bin/trace_run fed steps on standard input (a request whole, then its last tokens one by one beside a second request), and bin/tq
    generate on the same folder: logits and greedy tokens of the plain implementation."""
    import json
    import os
    import subprocess
    import sys
    from test_gpu_trace_run import Replay
    root = os.path.join(os.path.dirname(os.path.abspath(__file__)), "..")
    cfg = C.config_odd()
    w = C.weights(cfg, seed=77)
    folder = C.write_folder(str(tmp_path_factory.mktemp("kezasun_replay")), cfg, w)
    a, b = C.tokens(150, cfg["vocab"], 1), C.tokens(9, cfg["vocab"], 2)
    want_a, want_b = wanted("replay", cfg, w, a), wanted("replay", cfg, w, b)
    r = Replay(folder, dtype, str(tmp_path_factory.mktemp("out")), max_tokens=64 * 6)
    got = r.step([("x", a, list(range(150)))], end=["x"])
    close(got.view(-1, cfg["vocab"]), want_a, dtype, "whole")
    assert r.step([("y", a[:140], []), ("z", b[:5], [])]) is None
    for t in range(10):
        live = [("y", [a[140 + t]], [0])] + ([("z", [b[5 + t]], [0])] if t < 4 else [])
        got = r.step(live, end=(["y"] if t == 9 else []) + (["z"] if t == 3 else [])).view(-1, cfg["vocab"])
        close(got[0:1], want_a, dtype, "one by one at %d" % t, [140 + t])
        if t < 4:
            close(got[1:2], want_b, dtype, "the second request at %d" % t, [5 + t])
    r.finish()
    if dtype != "float32":
        return
    cmd = [sys.executable, os.path.join(root, "bin", "tq"), "--fp32", "generate", folder, "--prompt-ids", ",".join(str(t) for t in b), "-n", "5", "-t", "0",
           "--repeat-penalty", "1.0", "--json"]
    out = subprocess.run(cmd, capture_output=True, text=True)
    assert out.returncode == 0, out.stderr
    tokens = json.loads(out.stdout.strip().splitlines()[-1])["outputs"][0]
    seq = list(b)
    for t in tokens:
        assert int(plain_logits(cfg, w, seq)[-1].argmax()) == t
        seq.append(t)
