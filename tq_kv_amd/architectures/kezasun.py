"""Kezasun: a decoder whose configuration lists its layers one by one.  A layer is one RMS norm (its weight stored around zero) that a mixer and a
feed-forward both read, x + m (mixer(h) + ff(h)).  Mixers: "wkv" (time mixing: a matrix state per head that decays per key channel and token,
inputs mixed with the previous token's, a bonus for the current token) and "attention" (biases, q and k normed over the whole projection, a
sliding window, a sink of score 0, a gate per head; some layers read an earlier layer's keys and values).  The feed-forwards are routed experts
chosen by corrected scores within the best groups, some of which give back their input; or absent.

Which config.json keys the architecture reads and how they become a ModelSpec is csrc/engine/kezasun.cpp's; this is the typed
configuration as Python sees it.
"""
from dataclasses import dataclass
from typing import Optional, Tuple

from ..config.registry import config_class, spec_from_dict


@dataclass(frozen=True)
class KezasunLayer:
    type: str                   # "wkv" or "attention"
    mixer: dict                 # heads, dim and, for attention, kv_heads, vdim, scale, window, rot_base, rot_dims, rot_scaling, kv_from
    mlp: Optional[dict]         # None or {"kind": "moe", "ff", "experts", "top", "identity", "groups", "keep"}

    def mixer_dict(self):
        """The mixer as config.json writes it."""
        if self.type == "wkv":
            return dict(self.mixer)
        m = dict(self.mixer)
        m["mask"] = {"size": m.pop("window")}
        m["rot"] = {"base": m.pop("rot_base"), "dims": m.pop("rot_dims")}
        scaling = m.pop("rot_scaling")
        if scaling is not None:
            m["rot"]["scaling"] = dict(scaling)
        if m["kv_from"] is None:
            del m["kv_from"]
        return m

    def mlp_dict(self):
        m = self.mlp
        if m is None:
            return None
        return {"kind": m["kind"], "expert": {"ff": m["ff"]},
                "router": {"experts": m["experts"], "top": m["top"], "identity": m["identity"], "groups": {"count": m["groups"], "keep": m["keep"]}}}

    def __hash__(self):
        return hash((self.type, repr(sorted(self.mixer.items())), repr(self.mlp)))


@config_class("Kezasun")
@dataclass(frozen=True)
class KezasunConfig:
    vocab: int
    width: int
    norm_eps: float
    residual_mult: float
    max_positions: int
    layers: Tuple[KezasunLayer, ...]

    @classmethod
    def from_typed(cls, typed):
        """From what the engine library made of a config.json (every key, defaults filled in)."""
        layers = tuple(KezasunLayer(l["type"], dict(l["mixer"]), l["mlp"]) for l in typed["layers"])
        return cls(typed["vocab"], typed["width"], typed["norm_eps"], typed["residual_mult"], typed["max_positions"], layers)

    @classmethod
    def from_dict(cls, raw, where="config.json"):
        from ..config.registry import config_from_dict
        return config_from_dict(dict(raw, architecture="Kezasun"), where)[1]

    def to_dict(self):
        """The config.json that reads back as this configuration."""
        return {"architecture": "Kezasun", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult,
                "max_positions": self.max_positions, "layers": [{"type": l.type, "mixer": l.mixer_dict(), "mlp": l.mlp_dict()} for l in self.layers]}


def build_spec(cfg: KezasunConfig):
    return spec_from_dict(cfg.to_dict())
