"""Sizizen: a decoder-only stack whose layers are listed one by one in config.json.

  layer         x += n1(mixer(x)), then x += n2(ff(x)): a layer norm (weight, no bias) on every sublayer's output and none in
                front of it
  mixer         'parallel': two mixers read the same x; half the sum of their outputs, each divided by its root mean square
                and weighted
                  left    grouped-query softmax attention within chunks of mask.size positions (counted from position 0):
                          biases on q, k and v, an RMS norm per head of q and k, rotation of halves over the first
                          rot.dims dimensions
                  right   gated linear attention: a [dim, vdim] memory per head whose rows decay by sigmoid(z)^(1 / tau), z
                          out of a low-rank map with a bias; an RMS norm and a SiLU gate per head on the output
  feed-forward  dense with a SiLU gate; or a mixture of squared-ReLU experts routed by sigmoid scores plus a correction
                within the best groups of neighbouring experts, beside an optional shared expert; or none
  output        the model's layer norm and a table of its own
The residual stream is fp32.

This module holds the configuration (every size and constant is read from config.json), the tensor names and a
random-weight builder for tests and benchmarks.  The compute path is core/layer/ragged_runner.py.
"""
import math
from dataclasses import dataclass, field
from typing import Dict, List

import torch

from .pagazen import PagazenModel

MIXERS = ("parallel",)
FEED_FORWARDS = ("dense", "moe")
BRANCH_SCALE = 0.5          # what the two branches' normed outputs are summed with


def expert_groups(router: dict):
    """(number of groups, groups whose experts can be chosen); without groups every expert is in one."""
    g = router.get("groups") or {}
    return int(g.get("count", 1)), int(g.get("keep", 1))


def _check_mlp(i: int, mlp: dict):
    if mlp.get("kind") not in FEED_FORWARDS:
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
    if mlp["kind"] == "moe":
        E, top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
        count, keep = expert_groups(mlp["router"])
        if count < 1 or E % count or not 1 <= keep <= count or not 1 <= top <= keep * (E // count):
            raise ValueError(f"layer {i}: {top} of {E} experts in {keep} of {count} groups")


@dataclass
class SizizenConfig:
    vocab_size: int
    width: int
    layers: List[dict]
    eps: float = 1e-5
    name: str = "sizizen"
    architecture: str = "Sizizen"
    family: str = "ragged"
    raw: dict = field(default_factory=dict, repr=False)

    @property
    def hidden_size(self):
        return self.width

    @property
    def num_hidden_layers(self):
        return len(self.layers)

    @property
    def max_position_embeddings(self):
        return 1 << 20

    def layer_runs(self):
        """[(index of the layer whose tensors the run uses, its description)] in running order."""
        return list(enumerate(self.layers))

    @classmethod
    def from_json(cls, d: dict, name: str = "sizizen") -> "SizizenConfig":
        layers = d["layers"]
        for i, layer in enumerate(layers):
            if layer["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {layer['type']!r}")
            left, right = layer["mixer"]["left"], layer["mixer"]["right"]
            H, G = int(left["heads"]), int(left["kv_heads"])
            if G <= 0 or H % G:
                raise ValueError(f"layer {i}: {H} heads do not divide over {G} key/value heads")
            rot = int(left["rot"]["dims"])
            if rot % 2 or not 0 <= rot <= int(left["dim"]):
                raise ValueError(f"layer {i}: rotation over {rot} of {left['dim']} dimensions")
            if int(left["mask"]["size"]) < 1:
                raise ValueError(f"layer {i}: mask {left['mask']!r}")
            if not float(right["tau"]) > 0.0:
                raise ValueError(f"layer {i}: tau {right['tau']!r}")
            if layer.get("mlp") is not None:
                _check_mlp(i, layer["mlp"])
        return cls(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=layers, eps=float(d["norm"]["eps"]), name=name,
                   raw=d)

    def to_json(self) -> dict:
        return {"architecture": self.architecture, "layers": self.layers, "norm": {"eps": self.eps},
                "vocab": self.vocab_size, "width": self.width}


# The low-rank map of the right mixer's decays has an inner width of its own; no key of config.json gives it, the tensors'
# shapes do.
DEFAULT_RANK = 16


def tensor_shapes(cfg: SizizenConfig, rank: int = DEFAULT_RANK) -> Dict[str, tuple]:
    """Name -> shape of every tensor a checkpoint of this configuration holds (`rank`: inner width of the low-rank map,
    which a checkpoint chooses by the shapes of its tensors)."""
    W = cfg.width
    out = {"embed": (cfg.vocab_size, W), "final.norm": (W,), "head": (cfg.vocab_size, W)}
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer["mixer"]
        L, R = m["left"], m["right"]
        H, G, d, dv = int(L["heads"]), int(L["kv_heads"]), int(L["dim"]), int(L["vdim"])
        a = p + "mix.left."
        out.update({p + "norm1": (W,), a + "q": (H * d, W), a + "q.b": (H * d,), a + "k": (G * d, W), a + "k.b": (G * d,),
                    a + "v": (G * dv, W), a + "v.b": (G * dv,), a + "q.norm": (d,), a + "k.norm": (d,), a + "o": (W, H * dv),
                    a + "out": (W,)})
        H, n, dv = int(R["heads"]), int(R["dim"]), int(R["vdim"])
        a = p + "mix.right."
        out.update({a + "q": (H * n, W), a + "k": (H * n, W), a + "v": (H * dv, W), a + "g": (H * dv, W), a + "o": (W, H * dv),
                    a + "norm": (dv,), a + "a1": (rank, W), a + "a2": (H * n, rank), a + "a2.b": (H * n,), a + "out": (W,)})
        mlp = layer.get("mlp")
        if mlp is None:
            continue
        out[p + "norm2"] = (W,)
        if mlp["kind"] == "dense":
            ff = int(mlp["ff"])
            out.update({p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
            continue
        E, ff = int(mlp["router"]["experts"]), int(mlp["expert"]["ff"])
        out.update({p + "mlp.router": (E, W), p + "mlp.correction": (E,)})
        for e in range(E):
            out.update({p + f"mlp.e{e}.up": (ff, W), p + f"mlp.e{e}.down": (W, ff)})
        if mlp.get("shared"):
            sf = int(mlp["shared"]["ff"])
            out.update({p + "mlp.shared.up": (sf, W), p + "mlp.shared.down": (W, sf)})
    return out


class SizizenModel(PagazenModel):
    """Configuration plus a name -> tensor source (`get(name)`): a checkpoint's files or a dict."""


def random_weights(cfg: SizizenConfig, seed: int = 0, dtype=torch.bfloat16, rank: int = DEFAULT_RANK) -> Dict[str, torch.Tensor]:
    """Random tensors of the right shapes and sensible ranges (projections ~ 1/sqrt(fan-in), norm weights near one, decay
    biases so that the gates spread over (0, 1), corrections of either sign)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, rank).items():
        if name == "embed":
            t = torch.randn(shape, generator=g)
        elif len(shape) == 2:
            t = torch.randn(shape, generator=g) / math.sqrt(shape[1])
        elif name.endswith("a2.b"):
            t = torch.rand(shape, generator=g) * 8.0 - 4.0
        elif name.endswith("correction"):
            t = torch.randn(shape, generator=g) * 0.5 - 0.3
        elif name.endswith(".b"):
            t = torch.randn(shape, generator=g) * 0.3
        else:
            t = 1.0 + torch.randn(shape, generator=g) * 0.1
        out[name] = t.to(dtype)
    return out


def build_random_model(cfg: SizizenConfig, seed: int = 0, rank: int = DEFAULT_RANK) -> SizizenModel:
    return SizizenModel(cfg, random_weights(cfg, seed, rank=rank))


def bench_config(width: int, n_layers: int, vocab: int = 32000, ff_mult: int = 4, chunk: int = 1024, moe_every: int = 0,
                 right_vdim: int = 128) -> SizizenConfig:
    """A configuration with the proportions of a served model: 128-wide heads, one key/value head per four query heads on
    the left, width / 256 memories on the right; every `moe_every`-th feed-forward routed (16 experts in four groups, two
    of them kept, four experts used, beside a shared one; 0: dense ones only)."""
    layers = []
    for i in range(n_layers):
        mixer = {"left": {"heads": width // 128, "kv_heads": max(1, width // 512), "dim": 128, "vdim": 128,
                          "mask": {"size": chunk}, "rot": {"base": 10000.0, "dims": 128}, "scale": 128 ** -0.5},
                 "right": {"heads": max(1, width // 256), "dim": 128, "vdim": right_vdim, "tau": 16.0}}
        if moe_every and i % moe_every == moe_every - 1:
            mlp = {"kind": "moe", "expert": {"ff": ff_mult * width // 8},
                   "router": {"experts": 16, "groups": {"count": 4, "keep": 2}, "top": 4},
                   "shared": {"ff": ff_mult * width // 2}}
        else:
            mlp = {"kind": "dense", "ff": ff_mult * width}
        layers.append({"type": "parallel", "mixer": mixer, "mlp": mlp})
    return SizizenConfig(vocab_size=vocab, width=width, layers=layers, eps=1e-5, name=f"sizizen-w{width}-l{n_layers}")
