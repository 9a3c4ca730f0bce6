"""Kezasun configurations drawn from a seed (layers of both mixers in any order, with and without experts, layers that read others' keys and
values, windows of any size) through Engine.step against the plain implementation: whole prompts, a cut into portions and single tokens,
and a batch of two unequal requests."""
import random

import pytest
import torch

import kezasun_common as C
import plain_kezasun as plain
from tq_kv_amd import Engine, Model

pytestmark = pytest.mark.gpu


def draw(seed):
    r = random.Random(seed)
    width = r.choice([48, 64, 96, 100, 160, 192, 256])
    layers = []
    for i in range(r.randint(1, 6)):
        lenders = [k for k, ((t, m), _) in enumerate(layers) if t == "attention" and "kv_from" not in m]
        window = r.choice([1, 3, 16, 40, 64, 100, 128, 139, 200, 1000])
        if r.random() < 0.4:
            mix = C.wkv(r.choice([1, 2, 3, 6]), r.choice([3, 4, 8, 12, 32, 48, 64, 96, 128]))
        elif lenders and r.random() < 0.5:
            j = r.choice(lenders)
            m = layers[j][0][1]
            mix = ("attention", dict(m, kv_from=j, mask={"size": window}, scale=r.uniform(0.5, 1.5) / m["dim"] ** 0.5))
        else:
            kv, dim = r.choice([1, 2, 3, 4]), r.choice([8, 12, 16, 24, 32, 48, 64, 96, 128])
            scaling = r.choice([None, C.scaled(r.choice([2.0, 8.0]), r.choice([0.5, 1.0]), r.choice([2.0, 4.0]), r.choice([32, 100, 500]))])
            mix = C.attention(kv * r.choice([1, 1, 2, 3, 4, 8]), kv, dim, r.choice([dim, 8, 20, 32, 64, 128]), window, r.choice([0, 2, dim // 4 * 2, dim]),
                              base=r.choice([10.0, 500.0, 1e6]), scale=r.uniform(0.5, 1.5) / dim ** 0.5, scaling=scaling)
        mlp = None
        if r.random() < 0.7:
            experts, identity = r.choice([1, 2, 4, 7, 12, 30]), r.choice([0, 0, 1, 2, 5])
            n = experts + identity
            count = r.choice([c for c in range(1, n + 1) if n % c == 0])
            keep = r.randint(1, count)
            mlp = C.moe(r.choice([8, 24, 64, 100]), experts, r.randint(1, min(4, keep * (n // count))), identity, count, keep)
        layers.append((mix, mlp))
    return C.config(r.choice([50, 131, 300]), width, layers, eps=r.choice([1e-6, 1e-5, 1e-4]), mult=r.choice([0.3, 0.7, 1.0, 1.3]))


def errors(got, want):
    got, want = got.float().cpu(), want.float().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std().clamp_min(1e-6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(20))
def test_random_configuration(seed, dtype, tmp_path):
    cfg = draw(seed)
    w = C.weights(cfg, seed=100 + seed)
    eng = Engine(Model.from_dir(C.write_folder(str(tmp_path), cfg, w), dtype=dtype), max_tokens=2048, max_slots=4)
    a, b = C.tokens(290, cfg["vocab"], seed), C.tokens(37, cfg["vocab"], seed + 1)
    want_a, want_b = plain.forward(cfg, C.as_float(w), a), plain.forward(cfg, C.as_float(w), b)

    def check(got, want, toks, what):
        e = errors(got, want)
        assert torch.isfinite(e).all(), what
        if dtype == "float32":
            assert e.max().item() <= 2e-4, "%s: row error %.3g at row %d" % (what, e.max().item(), int(e.argmax()))
            return
        # What rounding alone does is the yardstick: the plain implementation with its products rounded to bfloat16.  Where a head of a few
        # values comes out next to nothing and is then divided by its own magnitude, rounding decides much of that row; such rows are few,
        # and float32 (which runs the same indexing) is held to every row.
        r = errors(plain.forward(cfg, C.as_float(w), toks, low=torch.bfloat16), want)
        limit = max(0.08, 2.5 * r.max().item())
        over = int((e > limit).sum())
        assert e.median().item() <= 1.5 * r.median().item() + 0.005 and over <= max(1, e.numel() // 50) and e.max().item() <= 1.0, \
            "%s: median row error %.3g (rounding alone: %.3g), %d rows of %d over %.3g, the worst %.3g" % (
                what, e.median().item(), r.median().item(), over, e.numel(), limit, e.max().item())

    s = eng.open()
    whole = eng.step([(s, a, list(range(len(a))))])
    eng.close(s)
    check(whole, want_a, a, "whole")
    # portions beside a second request, then single tokens of both
    s, t = eng.open(), eng.open()
    out = [eng.step([(s, a[:200], list(range(200))), (t, b[:30], list(range(30)))])]
    got_a, got_b = [out[0][:200]], [out[0][200:]]
    got_a.append(eng.step([(s, a[200:270], list(range(70)))]))
    for k in range(20):
        items = [(s, [a[270 + k]], [0])] + ([(t, [b[30 + k]], [0])] if k < 7 else [])
        o = eng.step(items)
        got_a.append(o[0:1])
        if k < 7:
            got_b.append(o[1:2])
        if k == 6:
            eng.close(t)
    eng.close(s)
    check(torch.cat(got_a), want_a, a, "portions and single tokens")
    check(torch.cat(got_b), want_b, b, "the second request")
    if dtype == "float32":
        assert torch.equal(torch.cat(got_a), whole), "float32 logits depend on the cut or the batch"
    eng.cache.check()
