"""Rasodra: a decoder whose configuration lists its layers one by one.  A sublayer has a layer norm (a weight, no bias) in front of the
part and another on its output; a layer is a mixer and an optional feed-forward of one product and its activation.  Mixers: "mlstm" (a
matrix memory with gates kept as logarithms against a running maximum), "latent_attention" (one cached latent and one rotated key part per
position, a sink, an output gate for every element) and "attention" (biases, values that are the keys as projected, heads normed in front of
the rotation, positions in chunks that see nothing of an earlier one).  A layer may use an earlier layer's tensors, with a cache or state
of its own.

Which config.json keys the architecture reads and how they become a ModelSpec is csrc/engine/rasodra.cpp's; this is the typed
configuration as Python sees it.
"""
from dataclasses import dataclass
from typing import Optional, Tuple

from ..config.registry import config_class, spec_from_dict


@dataclass(frozen=True)
class RasodraLayer:
    type: str                   # "mlstm", "latent_attention" or "attention"
    mixer: dict                 # heads, dim, vdim and: mlstm gate_cap; latent_attention rot_dim, kv_rank, scale, rot_base, rot_dims;
                                # attention kv_heads, chunk, scale, rot_base, rot_dims
    mlp: Optional[dict]         # None or {"kind": "dense", "ff"}
    source: int                 # the layer whose tensors this one uses (its own number unless it names another)

    def mixer_dict(self):
        """The mixer as config.json writes it."""
        m = dict(self.mixer)
        if "rot_base" in m:
            m["rot"] = {"base": m.pop("rot_base"), "dims": m.pop("rot_dims")}
        if "chunk" in m:
            m["mask"] = {"size": m.pop("chunk")}
        return m

    def __hash__(self):
        return hash((self.type, tuple(sorted(self.mixer.items())), None if self.mlp is None else tuple(sorted(self.mlp.items())), self.source))


@config_class("Rasodra")
@dataclass(frozen=True)
class RasodraConfig:
    vocab: int
    width: int
    norm_eps: float
    max_positions: int
    layers: Tuple[RasodraLayer, ...]

    @classmethod
    def from_typed(cls, typed):
        """From what the engine library made of a config.json (every key, defaults filled in)."""
        layers = tuple(RasodraLayer(l["type"], dict(l["mixer"]), l["mlp"], l["source"]) for l in typed["layers"])
        return cls(typed["vocab"], typed["width"], typed["norm_eps"], typed["max_positions"], layers)

    @classmethod
    def from_dict(cls, raw, where="config.json"):
        from ..config.registry import config_from_dict
        return config_from_dict(dict(raw, architecture="Rasodra"), where)[1]

    def to_dict(self):
        """The config.json that reads back as this configuration."""
        layers = []
        for i, l in enumerate(self.layers):
            d = {"type": l.type, "mixer": l.mixer_dict(), "mlp": l.mlp}
            if l.source != i:
                d["weights_of"] = l.source
            layers.append(d)
        return {"architecture": "Rasodra", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps}, "max_positions": self.max_positions,
                "layers": layers}


def build_spec(cfg: RasodraConfig):
    return spec_from_dict(cfg.to_dict())
