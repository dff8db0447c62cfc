"""Dugazen: a decoder-only stack whose layers are listed one by one in config.json.

  layer         x += m nb1(mixer(n1(x))), then x += m nb2(ff(n2(x))): an RMS norm (weight 1 + w) in front of every
                sublayer and another on its output, m = `residual_mult`
  mixers        'channel_delta'   a delta-rule memory per head: every row of the [dim, vdim] state decays by a gate of
                                  its own, the value a key reads is corrected towards the token's value, and the
                                  read-out sees that write; short convolutions with SiLU behind q, k and v, unit-length
                                  queries and keys (possibly shared by a group of heads), a unit-RMS and a sigmoid
                                  gate per head on the output
                'attention'       grouped-query softmax attention over a sliding window: biases on every projection,
                                  queries and keys normed over the WHOLE projection before the split into heads,
                                  rotation of halves over the first rot.dims dimensions, values mixed with those the
                                  first mixing layer gave the same token, a sigmoid gate per output value
  feed-forward  dense, clamped gate: g = min(gate h, limit), u = clamp(up h, +-limit), down(g sigmoid(1.702 g) (u + 1));
                or none
  output        a table of its own, logits times `logit_scale`
The residual stream is fp32.

This module holds the configuration (every size and constant is read from config.json), the tensor names and a
random-weight builder for tests and benchmarks.  The compute path is core/layer/ragged_runner.py.
"""
import math
from dataclasses import dataclass, field
from typing import Dict, List

import torch

from .pagazen import PagazenModel

MIXERS = ("attention", "channel_delta")
GATE_SLOPE = 1.702          # the feed-forward's gate is g * sigmoid(GATE_SLOPE * g)
UNIT_EPS = 1e-6             # added to the squared length of a query or key of the delta rule


@dataclass
class DugazenConfig:
    vocab_size: int
    width: int
    layers: List[dict]
    eps: float = 1e-6
    residual_mult: float = 1.0
    logit_scale: float = 1.0
    name: str = "dugazen"
    architecture: str = "Dugazen"
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
    def from_json(cls, d: dict, name: str = "dugazen") -> "DugazenConfig":
        layers = d["layers"]
        mixed = None        # kv_heads * vdim of the layers that share the first one's values
        for i, layer in enumerate(layers):
            if layer["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {layer['type']!r}")
            m = layer["mixer"]
            H, G = int(m["heads"]), int(m["kv_heads"])
            if G <= 0 or H % G:
                raise ValueError(f"layer {i}: {H} heads do not divide over {G} key/value heads")
            if layer["type"] == "attention":
                rot = int(m["rot"]["dims"])
                if rot % 2 or not 0 <= rot <= int(m["dim"]):
                    raise ValueError(f"layer {i}: rotation over {rot} of {m['dim']} dimensions")
                if int(m["mask"]["size"]) < 1:
                    raise ValueError(f"layer {i}: mask {m['mask']!r}")
                if m.get("v_mix"):
                    width = G * int(m["vdim"])
                    if mixed not in (None, width):
                        raise ValueError(f"layer {i}: {width} values cannot be mixed with the first layer's {mixed}")
                    mixed = width
            elif int(m["conv"]) < 1:
                raise ValueError(f"layer {i}: a convolution of {m['conv']} taps")
            mlp = layer.get("mlp")
            if mlp is not None and mlp.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
        return cls(vocab_size=int(d["vocab"]), width=int(d["width"]), layers=layers, eps=float(d["norm"]["eps"]),
                   residual_mult=float(d.get("residual_mult", 1.0)), logit_scale=float(d.get("logit_scale", 1.0)),
                   name=name, raw=d)

    def to_json(self) -> dict:
        return {"architecture": self.architecture, "layers": self.layers, "logit_scale": self.logit_scale,
                "norm": {"eps": self.eps}, "residual_mult": self.residual_mult, "vocab": self.vocab_size,
                "width": self.width}

    def first_value_mix(self):
        """The first layer whose attention mixes values (the others take its values), or None."""
        for i, layer in enumerate(self.layers):
            if layer["type"] == "attention" and layer["mixer"].get("v_mix"):
                return i
        return None


# The two low-rank maps of a channel_delta mixer (decay gates and output gate) have an inner width of their own; no
# key of config.json gives it, the tensors' shapes do.
DEFAULT_RANK = 16


def tensor_shapes(cfg: DugazenConfig, rank: int = DEFAULT_RANK) -> Dict[str, tuple]:
    """Name -> shape of every tensor a checkpoint of this configuration holds (`rank`: inner width of the low-rank
    maps, which a checkpoint chooses by the shapes of its tensors)."""
    W = cfg.width
    out = {"embed": (cfg.vocab_size, W), "final.norm": (W,), "head": (cfg.vocab_size, W)}
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer["mixer"]
        H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
        out.update({p + "norm1": (W,), p + "norm1b": (W,)})
        if layer["type"] == "attention":
            out.update({p + "mix.q": (H * d, W), p + "mix.q.b": (H * d,), p + "mix.k": (G * d, W), p + "mix.k.b": (G * d,),
                        p + "mix.v": (G * dv, W), p + "mix.v.b": (G * dv,), p + "mix.q.norm": (H * d,),
                        p + "mix.k.norm": (G * d,), p + "mix.g": (H * dv, W), p + "mix.o": (W, H * dv), p + "mix.o.b": (W,)})
            if m.get("v_mix"):
                out[p + "mix.vmix"] = ()
        else:
            taps = int(m["conv"])
            out.update({p + "mix.q": (G * d, W), p + "mix.q.conv": (G * d, taps), p + "mix.k": (G * d, W),
                        p + "mix.k.conv": (G * d, taps), p + "mix.v": (H * dv, W), p + "mix.v.conv": (H * dv, taps),
                        p + "mix.b": (H, W), p + "mix.A_log": (H,), p + "mix.norm": (dv,), p + "mix.a1": (rank, W),
                        p + "mix.a2": (H * d, rank), p + "mix.dt_bias": (H * d,), p + "mix.g1": (rank, W),
                        p + "mix.g2": (H * dv, rank), p + "mix.o": (W, H * dv)})
        mlp = layer.get("mlp")
        if mlp is not None:
            ff = int(mlp["ff"])
            out.update({p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W),
                        p + "mlp.down": (W, ff)})
    return out


class DugazenModel(PagazenModel):
    """Configuration plus a name -> tensor source (`get(name)`): a checkpoint's files or a dict."""


def random_weights(cfg: DugazenConfig, seed: int = 0, dtype=torch.bfloat16, rank: int = DEFAULT_RANK) -> Dict[str, torch.Tensor]:
    """Random tensors of the right shapes and sensible ranges (projections ~ 1/sqrt(fan-in), offsets of norms near
    zero, plain norm weights near one, A_log and dt_bias so that decays spread over (0, 1), mixing weights inside it)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, rank).items():
        if name == "embed":
            t = torch.randn(shape, generator=g)
        elif name.endswith(".conv"):
            t = torch.randn(shape, generator=g) * 0.5
        elif len(shape) == 2:
            t = torch.randn(shape, generator=g) / math.sqrt(shape[1])
        elif name.endswith("mix.vmix"):
            t = 0.2 + 0.6 * torch.rand(shape, generator=g)
        elif name.endswith("A_log"):
            t = torch.rand(shape, generator=g) * 3.0 - 2.0
        elif name.endswith("dt_bias"):
            t = torch.rand(shape, generator=g) * 4.0 - 5.0
        elif name.endswith(".b"):
            t = torch.randn(shape, generator=g) * 0.3
        elif name.endswith(("mix.norm", "q.norm", "k.norm")):
            t = 1.0 + torch.randn(shape, generator=g) * 0.1
        else:
            t = torch.randn(shape, generator=g) * 0.1
        out[name] = t.to(dtype)
    return out


def build_random_model(cfg: DugazenConfig, seed: int = 0, rank: int = DEFAULT_RANK) -> DugazenModel:
    return DugazenModel(cfg, random_weights(cfg, seed, rank=rank))


def bench_config(width: int, n_layers: int, vocab: int = 32000, ff_mult: int = 4, every: int = 4,
                 window: int = 1024) -> DugazenConfig:
    """A configuration with the proportions of a served model: 128-wide heads; every `every`-th layer a windowed
    attention (one key/value head per four query heads), the others delta-rule memories; a feed-forward in every
    layer."""
    heads = max(1, width // 128)
    mlp = {"kind": "dense", "ff": ff_mult * width, "limit": 7.0}
    layers = []
    for i in range(n_layers):
        if i % every == every - 1:
            mixer = {"heads": heads, "kv_heads": max(1, heads // 4), "dim": 128, "vdim": 128, "mask": {"size": window},
                     "rot": {"base": 10000.0, "dims": 128}, "scale": 128 ** -0.5, "v_mix": True}
            layers.append({"type": "attention", "mixer": mixer, "mlp": mlp})
        else:
            mixer = {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4}
            layers.append({"type": "channel_delta", "mixer": mixer, "mlp": mlp})
    return DugazenConfig(vocab_size=vocab, width=width, layers=layers, eps=1e-6, residual_mult=1.0, logit_scale=1.0,
                         name=f"dugazen-w{width}-l{n_layers}")
