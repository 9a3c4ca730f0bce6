"""Shared by the Kezasun tests: small configurations made here, random weights of a sensible size, model folders written with the
safetensors package, and how logits are compared."""
import json
import math
import os

import torch
from safetensors.torch import save_file

CODES = 6           # channels that tell a router which token it is (see weights)


def wkv(heads, dim):
    return ("wkv", {"heads": heads, "dim": dim})


def scaled(factor, low, high, original):
    return {"factor": factor, "low": low, "high": high, "original": original}


def attention(heads, kv_heads, dim, vdim, window, rot_dims, base=10000.0, scale=None, scaling=None, kv_from=None):
    rot = {"base": base, "dims": rot_dims}
    if scaling is not None:
        rot["scaling"] = scaling
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "rot": rot,
         "scale": scale if scale is not None else 1.0 / math.sqrt(dim)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return ("attention", m)


def moe(ff, experts, top, identity=0, count=1, keep=1):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "identity": identity, "groups": {"count": count, "keep": keep}}}


def config(vocab, width, layers, eps=1e-5, mult=0.7):
    """layers: (type, mixer), mlp each."""
    return {"architecture": "Kezasun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "layers": [{"type": t, "mixer": json.loads(json.dumps(m)), "mlp": json.loads(json.dumps(f))} for (t, m), f in layers]}


# Sizes chosen away from each other: values larger and smaller than keys, part of a head turned (with and without scaled frequencies), heads in
# groups, windows that are no multiples of the page, borrowed keys and values seen through larger, smaller and equal windows, layers without
# experts of every kind, groups of experts that end inside the ones without weights.
def config_mixed():
    sc = scaled(8.0, 1.0, 4.0, 64)
    a = dict(heads=6, kv_heads=3, dim=24, vdim=40, rot_dims=16, base=300.0, scale=0.35, scaling=sc)
    b = dict(heads=4, kv_heads=1, dim=40, vdim=12, rot_dims=40, base=777.0)
    return config(331, 96, [(attention(window=37, **a), moe(40, 9, 3, 3, 4, 2)), (wkv(3, 20), moe(24, 5, 2, 1, 2, 1)), (attention(window=70, kv_from=0, **a), moe(16, 4, 1)),
                            (wkv(2, 40), None), (attention(window=64, **b), None), (attention(window=5, kv_from=0, **a), None), (wkv(1, 8), moe(8, 1, 1, 1)),
                            (attention(window=64, kv_from=4, **b), moe(32, 6, 6, 2, 1, 1))], eps=3e-6, mult=0.55)


# The smallest of everything: one head, one group, one element a value, a window of one position, nothing turned, one expert.
def config_ones():
    return config(67, 32, [(attention(1, 1, 2, 1, 1, 0), moe(8, 1, 1)), (wkv(1, 2), None), (attention(2, 2, 2, 2, 2, 2, base=2.0), moe(8, 1, 2, 1)), (wkv(1, 4), moe(8, 2, 1, 2, 4, 1))],
                  eps=1e-4, mult=1.0)


# Sizes that are no multiples of 8, or of 4.
def config_odd():
    sc = scaled(2.5, 0.5, 2.0, 100)
    return config(101, 52, [(wkv(3, 10), moe(22, 3, 2, 2, 5, 3)), (attention(3, 3, 10, 14, 9, 6, base=55.0, scaling=sc), None), (wkv(5, 7), None),
                            (attention(5, 1, 14, 10, 100, 14), moe(30, 7, 3)), (attention(5, 1, 14, 10, 33, 14, kv_from=3), None)], eps=2e-5, mult=-0.8)


def config_single(kind, width=64):
    mix = {"wkv": wkv(3, 12), "attention": attention(4, 2, 16, 24, 24, 8, base=50.0, scale=0.4)}[kind]
    return config(97, width, [(mix, moe(24, 6, 2, 2, 4, 2))])


def weights(cfg, seed, store=torch.bfloat16, codes=True):
    """name -> tensor of the store dtype.  Products keep the size of what they read (std 1/sqrt(inputs)); decays lie around a slow one, so that a
    state reaches far back.

    codes: the routers read CODES channels of the stream that hold one of two equal and opposite values per token and that no layer writes to.  A
    rounding of the stream then scales a token's router logits all alike, and never turns a choice between experts around."""
    g = torch.Generator().manual_seed(seed)

    def lin(o, i, gain=1.0):
        return torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def vec(n, around=0.0, spread=0.1):
        return around + spread * torch.randn(n, generator=g)

    D = cfg["width"]
    w = {"embed": lin(cfg["vocab"], D, math.sqrt(D)), "head": lin(cfg["vocab"], D, 3.0), "final.norm": vec(D)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        x = p + "mix."
        w[p + "norm1"] = vec(D)
        H, d = m["heads"], m["dim"]
        if layer["type"] == "wkv":
            rank = 4 + 3 * i
            w.update({x + "mu." + s: vec(D, 0.5, 0.3) for s in "rkvgw"})
            w.update({x + s: lin(H * d, D) for s in "rkvg"})
            w.update({x + "w1": lin(rank, D), x + "w2": lin(H * d, rank, 1.5), x + "w0": vec(H * d, -3.0, 1.5), x + "u": vec(H * d, 0.5, 0.5).view(H, d),
                      x + "norm": vec(H * d, 1.0, 0.2), x + "o": lin(D, H * d)})
        else:
            G, dv = m["kv_heads"], m["vdim"]
            w.update({x + "q": lin(H * d, D), x + "q.b": vec(H * d, 0.0, 0.3), x + "q.norm": vec(H * d, 1.0, 0.3), x + "g": lin(H, D, 2.0), x + "o": lin(D, H * dv)})
            if m.get("kv_from") is None:
                w.update({x + "k": lin(G * d, D), x + "k.b": vec(G * d, 0.0, 0.3), x + "k.norm": vec(G * d, 1.0, 0.3), x + "v": lin(G * dv, D), x + "v.b": vec(G * dv, 0.0, 0.3)})
        if layer["mlp"] is not None:
            r, ff = layer["mlp"]["router"], layer["mlp"]["expert"]["ff"]
            n = r["experts"] + r["identity"]
            w.update({p + "mlp.router": lin(n, D, 2.0), p + "mlp.correction": vec(n, 0.0, 0.15)})
            for e in range(r["experts"]):
                q = p + "mlp.e%d." % e
                w.update({q + "gate": lin(ff, D), q + "up": lin(ff, D), q + "down": lin(D, ff, 1.5)})
    if codes:
        k = min(CODES, D // 4)
        bits = torch.randint(0, 2, (cfg["vocab"], k), generator=g) * 2 - 1
        w["embed"][:, :k] = 1.5 * bits
        for name, t in w.items():
            if name.endswith(".norm1"):
                t[:k] = 0.0
            elif name.endswith(".mix.o") or name.endswith(".down"):
                t[:k] = 0.0
            elif name.endswith(".router"):
                t[:, k:] = 0.0
                t[:, :k] = torch.randn(t.shape[0], k, generator=g)
    return {name: t.to(store) for name, t in w.items()}


def write_folder(path, cfg, w):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return str(path)


def as_float(w):
    return {k: v.to(torch.float32) for k, v in w.items()}


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def row_errors(got, want):
    """Per row: the root mean square of the difference over that of the wanted row."""
    got, want = got.detach().float().cpu(), want.detach().float().cpu()
    return torch.sqrt(((got - want) ** 2).mean(-1)) / torch.sqrt((want ** 2).mean(-1) + 1e-12)
