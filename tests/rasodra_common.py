"""Shared by the Rasodra tests: small configurations made here, random weights of a sensible size, model folders written with the
safetensors package, and how logits are compared."""
import json
import math
import os

import torch
from safetensors.torch import save_file


def mlstm(heads, dim, vdim, cap=8.0):
    return ("mlstm", {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap})


def latent(heads, dim, rot_dim, vdim, kv_rank, base=10000.0, scale=None):
    return ("latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                                 "scale": scale if scale is not None else 1.0 / math.sqrt(dim + rot_dim), "rot": {"base": base, "dims": rot_dim}})


def chunked(heads, kv_heads, dim, chunk, rot_dims, base=10000.0, scale=None):
    return ("attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "mask": {"size": chunk}, "rot": {"base": base, "dims": rot_dims},
                          "scale": scale if scale is not None else 1.0 / math.sqrt(dim)})


def config(vocab, width, layers, eps=1e-5):
    """layers: (type, mixer), ff or None [, the number of the layer whose tensors it uses] each."""
    out = []
    for l in layers:
        (t, m), ff = l[0], l[1]
        d = {"type": t, "mixer": json.loads(json.dumps(m)), "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
        if len(l) > 2:
            d["weights_of"] = l[2]
        out.append(d)
    return {"architecture": "Rasodra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": out}


# Sizes chosen away from each other: values larger and smaller than keys, part of a head turned, heads in groups, chunks that are no multiples of
# the page or of each other, layers that use the tensors of earlier ones (one of them through another such layer) in another order, a layer
# without a feed-forward of every kind.
def config_mixed():
    a = mlstm(3, 24, 40, cap=6.0)
    b = latent(6, 24, 8, 40, 56, base=5000.0, scale=0.3)
    c = chunked(6, 3, 24, 37, 16, base=300.0, scale=0.35)
    d = chunked(4, 1, 40, 70, 40, base=777.0)
    e = mlstm(2, 40, 12, cap=15.0)
    return config(331, 96, [(a, 72), (b, 100), (c, None), (b, 100, 1), (d, 56), (a, 72, 0), (e, None), (latent(3, 16, 4, 8, 24, base=50.0), None), (c, None, 2), (a, 72, 5),
                            (b, 100, 3)], eps=3e-6)


# The smallest of everything: one head, one group, one element a value, chunks of one position, a latent of one element, nothing turned.
def config_ones():
    return config(67, 32, [(mlstm(1, 1, 1, cap=1.0), 8), (latent(1, 1, 0, 1, 1), None), (chunked(1, 1, 2, 1, 0), 16), (chunked(2, 2, 2, 1, 2, base=2.0), None),
                           (mlstm(1, 2, 1), None, ) ], eps=1e-4)


# Sizes that are no multiples of 8, or of 4.
def config_odd():
    return config(101, 52, [(mlstm(3, 10, 14, cap=3.0), 44), (latent(3, 10, 6, 14, 22, base=77.0), 30), (chunked(3, 3, 10, 9, 6), None), (chunked(5, 1, 14, 100, 14), 20)])


def config_single(kind, width=64):
    mix = {"mlstm": mlstm(3, 12, 20, cap=5.0), "latent": latent(4, 16, 8, 24, 40, base=50.0, scale=0.4), "chunked": chunked(4, 2, 16, 24, 8, base=50.0, scale=0.4)}[kind]
    return config(97, width, [(mix, 48)])


def weights(cfg, seed, store=torch.bfloat16):
    """name -> tensor of the store dtype.  Products keep the size of what they read (std 1/sqrt(inputs)); forget gates lie around a slow
    decay, so that a state reaches far back."""
    g = torch.Generator().manual_seed(seed)

    def lin(o, i, gain=1.0):
        return (torch.randn(o, i, generator=g) * gain / math.sqrt(i)).to(store)

    def vec(n, around=0.0, spread=0.1):
        return (around + spread * torch.randn(n, generator=g)).to(store)

    D = cfg["width"]
    w = {"embed": lin(cfg["vocab"], D, math.sqrt(D)), "head": lin(cfg["vocab"], D, 3.0), "final.norm": vec(D, 1.0)}
    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = "l%d." % i, layer["mixer"]
        x = p + "mix."
        w.update({p + "norm1": vec(D, 1.0), p + "norm1b": vec(D, 1.0, 0.3)})
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        w[x + "o"] = lin(D, H * dv)
        if layer["type"] == "mlstm":
            w.update({x + "q": lin(H * d, D), x + "k": lin(H * d, D), x + "v": lin(H * dv, D), x + "g": lin(H * dv, D), x + "norm": vec(H * dv, 1.0, 0.2),
                      x + "i": lin(H, D, 2.0), x + "i.b": vec(H, 0.0, 1.0), x + "f": lin(H, D, 2.0), x + "f.b": vec(H, 3.0, 1.0)})
        elif layer["type"] == "latent_attention":
            rk, dr = m["kv_rank"], m["rot_dim"]
            w.update({x + "q": lin(H * (d + dr), D), x + "dkv": lin(rk + dr, D), x + "dkv.norm": vec(rk, 1.0, 0.2), x + "uk": lin(H * d, rk), x + "uv": lin(H * dv, rk),
                      x + "sink": vec(H, 0.0, 1.0), x + "g": lin(H * dv, D)})
        else:
            G = m["kv_heads"]
            w.update({x + "q": lin(H * d, D), x + "q.b": vec(H * d, 0.0, 0.3), x + "k": lin(G * d, D), x + "k.b": vec(G * d, 0.0, 0.3), x + "q.norm": vec(d, 1.0, 0.2),
                      x + "k.norm": vec(d, 1.0, 0.2)})
        if layer["mlp"] is not None:
            w.update({p + "norm2": vec(D, 1.0), p + "norm2b": vec(D, 1.0, 0.3), p + "mlp.up": lin(layer["mlp"]["ff"], D), p + "mlp.down": lin(D, layer["mlp"]["ff"])})
    return w


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
