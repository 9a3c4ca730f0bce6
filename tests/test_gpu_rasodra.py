"""The Rasodra decoder through the library against the plain implementation (plain_rasodra.py): each mechanism alone through its part,
then whole models through Engine.step and generate() with every way of cutting and batching, on configurations made here."""
import pytest
import torch

import plain_rasodra as plain
import rasodra_common as C
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
    return PartSpec("rotary", {"theta": rot["base"], "rot_dim": rot["dims"], "max_positions": MAXPOS, "style": "pairs"})


def mixer_spec(kind, m, hidden, eps):
    if kind == "mlstm":
        return PartSpec("mlstm", {"hidden": hidden, "heads": m["heads"], "head_dim": m["dim"], "value_dim": m["vdim"], "gate_cap": m["gate_cap"], "eps": eps,
                                  "names": {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm", "i": "i", "i_bias": "i.b", "f": "f", "f_bias": "f.b"}})
    if kind == "latent_attention":
        return PartSpec("latent_attention", {"hidden": hidden, "n_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"], "value_dim": m["vdim"], "q_rank": None,
                                             "kv_rank": m["kv_rank"], "scale": m["scale"], "eps": eps, "own_kv": True, "gate_per": "element", "sink": True,
                                             "position": position(m["rot"])})
    return PartSpec("attention", {"hidden": hidden, "n_heads": m["heads"], "n_kv_heads": m["kv_heads"], "head_dim": m["dim"], "values_are_keys": True, "scale": m["scale"],
                                  "qkv_bias": True, "qk_norm": True, "eps": eps, "chunk": m["mask"]["size"], "position": position(m["rot"]),
                                  "names": {"q": "q", "k": "k", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "q_bias": "q.b", "k_bias": "k.b"}})


MIXERS = [C.mlstm(3, 24, 40, cap=6.0), C.mlstm(1, 1, 1, cap=1.0), C.mlstm(2, 10, 14, cap=3.0), C.mlstm(4, 64, 64), C.mlstm(2, 128, 256, cap=15.0), C.mlstm(1, 200, 136),
          C.mlstm(2, 68, 300, cap=2.0), C.mlstm(2, 16, 132), C.mlstm(3, 300, 20, cap=4.0),
          C.latent(6, 24, 8, 40, 56, base=40.0, scale=0.3), C.latent(1, 1, 0, 1, 1), C.latent(3, 10, 6, 14, 22), C.latent(20, 32, 16, 24, 128), C.latent(4, 64, 32, 64, 256),
          C.latent(2, 16, 64, 32, 512, scale=0.1), C.latent(17, 8, 8, 16, 40),
          C.chunked(6, 3, 24, 37, 16, base=300.0, scale=0.35), C.chunked(1, 1, 2, 1, 0), C.chunked(3, 3, 10, 9, 6), C.chunked(8, 2, 64, 64, 64), C.chunked(16, 2, 128, 100, 32),
          C.chunked(2, 1, 160, 200, 40, scale=0.05), C.chunked(5, 5, 32, 130, 2), C.chunked(6, 2, 96, 1000, 96, scale=0.2), C.chunked(40, 2, 32, 63, 32)]


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
    w = {k[len("l0.mix."):]: v for k, v in C.weights(cfg, 3).items() if k.startswith("l0.mix.")}
    part = BuildEnv(DEV, DT[dtype]).build("mixer", mixer_spec(kind, m, hidden, eps))
    assert part.graph_safe and sorted(part.tensors()) == sorted(w)
    part.load({k: v.to(DT[dtype]).to(DEV) for k, v in w.items()})
    need = part.cache_need()
    cache = Cache([need], [None], 64 * 8, 2, DT[dtype], DEV)
    assert len(cache.state_groups) == (kind == "mlstm") and len(cache.kv_groups) == (kind != "mlstm")
    xs = [torch.randn(n, hidden).to(DT[dtype]) for n in (300, 40)]
    want = [plain.MIXERS[kind](x.float(), C.as_float(w), "", m, eps, torch.arange(x.shape[0]), DT[dtype]) for x in xs]
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
            # (a head of one value is divided by its own magnitude: next to zero, rounding decides how much of the sign is left)
            # (and the short steps keep q, k and v of a memory in float32, where the plain computation rounds them)
            limit = (5e-5 if dtype == "float32" else 0.06 if kind == "mlstm" else 0.03) * (6.0 if kind == "mlstm" and m["vdim"] == 1 else 1.0)
            assert e.max().item() < limit, "use %d, sequence %d: %.3g at row %d" % (use, i, e.max().item(), int(e.argmax()))
        for s in slots:
            cache.release(s)


@pytest.mark.parametrize("mix", [m for m in MIXERS if m[0] == "mlstm"], ids=mixer_ids)
def test_the_matrix_memory_is_as_exact_in_chunks_as_token_by_token(mix):
    """Inputs and weights of small whole numbers, so that the products come out as numbers that bfloat16 holds exactly: then the long step's
    kernels (which take bfloat16 operands and split every float32 number into two of them) must leave the state that the token-by-token kernels
    leave, far closer than bfloat16's rounding, and the outputs with it."""
    kind, m = mix
    hidden, eps = 88, 1e-5
    g = torch.Generator().manual_seed(5)
    w = {k[len("l0.mix."):]: v for k, v in C.weights(C.config(50, hidden, [(mix, None)]), 3).items() if k.startswith("l0.mix.")}

    def ternary(shape, density):
        return (torch.randint(0, 2, shape, generator=g) * 2 - 1).float() * (torch.rand(shape, generator=g) < density).float()

    for k in ("q", "k", "v"):
        w[k] = ternary(w[k].shape, 0.15).to(torch.bfloat16)
    part = BuildEnv(DEV, torch.bfloat16).build("mixer", mixer_spec(kind, m, hidden, eps))
    part.load({k: v.to(DEV) for k, v in w.items()})
    x = ternary((200, hidden), 0.6).to(torch.bfloat16).to(DEV)
    states, outputs = [], []
    for cuts in ([200], [67, 200], list(range(1, 201))):
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
        assert e.median().item() < 0.006 and e.max().item() < 0.06, (e.median().item(), e.max().item())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size", [1, 50, 52, 192, 1000, 2048, 4096, 5120, 8192])
def test_layer_norm_without_a_bias(dtype, size):
    env = BuildEnv(DEV, DT[dtype])
    part = env.build("norm", PartSpec("layer_norm", {"size": size, "eps": 1e-5, "tensor": "", "bias": False}))
    assert sorted(part.tensors()) == [""]
    w = (1.0 + 0.3 * torch.randn(size)).to(DT[dtype])
    part.load({"": w.to(DEV)})
    x = (3.0 + 2.0 * torch.randn(9, size)).to(DT[dtype])
    got = part.forward(x.to(DEV)).float().cpu()
    want = plain.layer_norm(x.float(), w.float(), 1e-5)
    assert (got - want).abs().max().item() < (1e-4 if dtype == "float32" else 0.06)


# ---- whole models ----------------------------------------------------------------------------------------
_MODELS = {}
MAKERS = {"wide1028": lambda: C.config(61, 1028, [(C.chunked(2, 1, 16, 40, 8), 24), (C.mlstm(2, 8, 12), None)]),
          "wide1030": lambda: C.config(61, 1030, [(C.chunked(2, 1, 16, 40, 8), 24), (C.latent(2, 8, 4, 12, 20), 16)]),
          "wide4160": lambda: C.config(61, 4160, [(C.latent(2, 16, 8, 16, 24), 32), (C.chunked(2, 1, 16, 40, 8), None)]),
          "wide9000": lambda: C.config(61, 9000, [(C.mlstm(2, 8, 16), 32)]),
          "slow": lambda: C.config_single("mlstm"), "mixed": C.config_mixed, "ones": C.config_ones, "odd": C.config_odd, "mlstm": lambda: C.config_single("mlstm"), "latent": lambda: C.config_single("latent"),
          "chunked": lambda: C.config_single("chunked")}


def model(name, tmp_path_factory):
    if name not in _MODELS:
        cfg = MAKERS[name]()
        w = C.weights(cfg, seed=11 + len(name))
        if name == "slow":              # a forget gate next to one: the memory reaches back hundreds of tokens
            w["l0.mix.f.b"] = torch.full_like(w["l0.mix.f.b"], 9.0)
        _MODELS[name] = (cfg, w, C.write_folder(str(tmp_path_factory.mktemp("rasodra_%s" % name)), cfg, w), {})
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
    A norm on a part's output makes small outputs as large as any, and with them their rounding, so the size of that is the sequence's own."""

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
    assert eng.model.spec.architecture == "Rasodra" and eng.model.graph_safe and len(eng.model.spec.order) == len(cfg["layers"])
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
@pytest.mark.parametrize("name", ["wide1028", "wide1030", "wide4160", "wide9000"])
def test_norms_over_wide_rows(name, dtype, tmp_path_factory):
    """Streams of widths that take the norms' kernels in all their shapes (a row in one, two or three pieces a thread, or element by element),
    in prompts and in steps of few and of many sequences."""
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
    for name in ("mixed", "odd", "chunked", "latent", "mlstm"):
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


def chunked_only(tmp_path_factory, chunk, heads=4, kv=2):
    key = "edges_%d_%d" % (chunk, heads)
    if key not in _MODELS:
        cfg = C.config(60, 48, [(C.chunked(heads, kv, 16, chunk, 8, base=100.0, scale=0.5), 32)])
        w = C.weights(cfg, 21)
        _MODELS[key] = (cfg, w, C.write_folder(str(tmp_path_factory.mktemp("rasodra_" + key)), cfg, w), {})
    return key


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [1, 37, 64, 96, 150, 500])
def test_what_a_position_sees_of_its_chunk(chunk, dtype, tmp_path_factory):
    """Changing the token at j changes the logits at i if and only if j <= i lies in i's chunk: keys at the chunk's first place and at the last
    of the one before, at the sequence's start and at pages' borders; queries in a prompt, in a later portion, and decoded one by one."""
    cfg, w, eng = engine(chunked_only(tmp_path_factory, chunk), dtype, tmp_path_factory)
    n = 200
    toks = C.tokens(n, cfg["vocab"], 8)

    def logits_of(seq, how):
        return run_cut(eng, seq, {"prompt": [], "portions": [61, 63, 130], "decoded": [120] + list(range(121, n))}[how])

    for how in ("prompt", "portions", "decoded"):
        base = logits_of(toks, how)
        close(base, wanted("chunk%d" % chunk, cfg, w, toks), dtype, how)
        for i in (130, 149, 150, 192, 199):
            lo = i // chunk * chunk
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


def one_key(tmp_path_factory, kind, sink):
    """A model of one layer in which two tokens have an element of the embedding to themselves; the keys of the one and the queries of the
    other read it with one and the same long vector, so that this one key stands far above everything else the query sees."""
    cfg = C.config(60, 32, [(C.latent(2, 64, 0, 24, 48, scale=0.5) if kind == "latent" else C.chunked(2, 1, 64, 250, 0, scale=0.5), None)])
    special, asker = 7, 11
    f = C.as_float(C.weights(cfg, 4))
    # the two elements are zero for every other token, and stay zero through the layer norm because a row's other elements add up to nothing
    f["embed"][:, :2] = 0.0
    f["embed"][:, 2:] -= f["embed"][:, 2:].mean(1, keepdim=True)
    f["embed"][special, 0] = f["embed"][asker, 1] = 3.0
    f["l0.norm1"].fill_(1.0)
    direction = torch.randn(64)
    if kind == "latent":
        # a latent's first element is the special token's alone, and a key reads it
        f["l0.mix.dkv"][0] = 0.0
        f["l0.mix.dkv"][0, 0] = 12.0
        f["l0.mix.uk"] *= 0.1
        f["l0.mix.uk"][:, 0] = 0.7 * direction.repeat(2)
        f["l0.mix.sink"].fill_(sink)
        f["l0.mix.q"] *= 0.1
    else:
        for k in ("q.norm", "k.norm"):
            f["l0.mix." + k].fill_(1.0)
        f["l0.mix.k"][:, 0] = 6.0 * direction
    f["l0.mix.q"][:, 1] = 6.0 * direction.repeat(2)
    w = {k: v.to(torch.bfloat16) for k, v in f.items()}
    return cfg, w, C.write_folder(str(tmp_path_factory.mktemp("rasodra_far")), cfg, w), special, asker


@pytest.mark.parametrize("kind,sink", [("latent", -5.0), ("chunked", 0.0)])
def test_one_key_far_away_carries_the_output(kind, sink, tmp_path_factory):
    """The output at the query is the one key's value, wherever its token stands (at the start, at a page's border, at the chunk's first place,
    just before the query), however the query comes (in the prompt or decoded); and with the key in the chunk before, it is not."""
    cfg, w, folder, special, asker = one_key(tmp_path_factory, kind, sink)
    n = 330
    toks = [t if t not in (special, asker) else 20 for t in C.tokens(n, cfg["vocab"], 2)]
    for dtype in DTYPES:
        eng = Engine(Model.from_dir(folder, dtype=dtype), max_tokens=1024, max_slots=2)
        for place in (0, 1, 63, 64, 128, 249, 250, 251, 320, n - 2):
            seq = list(toks)
            seq[place], seq[n - 1] = special, asker
            want = wanted(kind, cfg, w, seq)
            other = list(seq)
            other[place] = 21
            difference = C.row_errors(wanted(kind, cfg, w, other).rows[-1:], want.rows[-1:]).item()
            assert difference > 0.2 if (kind == "latent" or place >= 250) else difference == 0.0          # the one key matters
            close(run_cut(eng, seq, [])[-1:], want, dtype, "prompt, key at %d" % place, [n - 1])
            close(run_cut(eng, seq, [300] + list(range(301, n)))[-1:], want, dtype, "decoded, key at %d" % place, [n - 1])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("length", [1, 2, 5, 64, 65, 200])
def test_a_sink_that_outweighs_the_keys(length, dtype, tmp_path_factory):
    """Sinks far above, among and far below the scores, in prompts (tiles), in decoding (one part or several, merged) and for the first
    tokens, where the sink is nearly all there is."""
    key = "sinks"
    if key not in _MODELS:
        cfg = C.config(60, 48, [(C.latent(5, 16, 8, 24, 40, base=100.0), None)])
        w = C.weights(cfg, 22)
        w["l0.mix.sink"] = torch.tensor([6.0, 2.0, 0.0, -3.0, -30.0]).to(torch.bfloat16)
        _MODELS[key] = (cfg, w, C.write_folder(str(tmp_path_factory.mktemp("rasodra_sinks")), cfg, w), {})
    cfg, w, eng = engine(key, dtype, tmp_path_factory)
    toks = C.tokens(length, cfg["vocab"], length)
    want = wanted(key, cfg, w, toks)
    without = dict(w)
    without["l0.mix.sink"] = torch.full((5,), -100.0).to(torch.bfloat16)
    assert C.row_errors(plain_logits(cfg, without, toks)[-1:], want.rows[-1:]).item() > 0.02
    close(run_cut(eng, toks, []), want, dtype, "prompt")
    close(run_cut(eng, toks, list(range(1, length))), want, dtype, "one by one")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["slow", "latent"])
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
@pytest.mark.parametrize("forget,inp", [(20.0, 0.0), (-20.0, 0.0), (3.0, 20.0), (3.0, -20.0), (0.0, 0.0)])
def test_gates_at_their_ends(forget, inp, dtype, tmp_path_factory):
    """Gates at either end of their cap: a memory that forgets nothing for hundreds of tokens, one that forgets everything at once, inputs far
    above what is kept and inputs far below e^(-m) (where the denominator is its floor)."""
    cfg = C.config(60, 40, [(C.mlstm(2, 16, 24, cap=9.0), None), (C.mlstm(1, 20, 8, cap=9.0), 24)])
    w = C.weights(cfg, 31)
    for p in ("l0.mix.", "l1.mix."):
        w[p + "f.b"] = torch.full_like(w[p + "f.b"], forget)
        w[p + "i.b"] = torch.full_like(w[p + "i.b"], inp)
    eng = Engine(Model.from_dir(C.write_folder(str(tmp_path_factory.mktemp("rasodra_gates")), cfg, w), dtype=dtype), max_tokens=1024, max_slots=2)
    toks = C.tokens(280, cfg["vocab"], 3)
    want = plain_logits(cfg, w, toks)
    # what rounding the products alone does to the plain computation is the yardstick where little is left to divide by
    rounding = C.row_errors(plain.forward(cfg, C.as_float(w), toks, low=torch.bfloat16), want).max().item() if dtype == "bfloat16" else 0.0
    for cuts in ([], [200, 202] + list(range(203, 280)), [30, 60, 250]):
        got = run_cut(eng, toks, cuts)
        assert torch.isfinite(got).all()
        e = C.row_errors(got, want).max().item()
        assert e <= (2e-4 if dtype == "float32" else max(0.06, 3.0 * rounding)), "cuts %s: %.3g (rounding alone %.3g)" % (cuts[:3], e, rounding)


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
    folder = C.write_folder(str(tmp_path_factory.mktemp("rasodra_replay")), cfg, w)
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
