"""Small Sizizen configurations for the tests (none with the proportions of a real checkpoint) and an engine builder;
the helpers that feed a request in portions are those of ragged_util."""
import torch

from micro_vllm_amd.models.sizizen import SizizenConfig, build_random_model


def attention(heads=6, kv_heads=2, dim=40, vdim=24, chunk=37, rot=24, base=3000.0, scale=0.21):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
            "rot": {"base": base, "dims": rot}, "scale": scale}


def linear(heads=3, dim=40, vdim=56, tau=5.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def dense(ff=150):
    return {"kind": "dense", "ff": ff}


def moe(experts=12, groups=3, keep=2, top=4, ff=40, shared=72):
    d = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "groups": {"count": groups, "keep": keep}, "top": top}}
    if shared:
        d["shared"] = {"ff": shared}
    return d


def layer(left, right, mlp):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


def config_a():
    """Odd sizes everywhere, every layer another: head counts of the two mixers apart, chunks shorter and longer than a
    page, rotation over none / part / all of a head, routed and dense feed-forwards and none, with and without a shared
    expert."""
    return SizizenConfig(vocab_size=331, width=176, eps=1e-5, layers=[
        layer(attention(), linear(), moe()),
        layer(attention(heads=4, kv_heads=4, dim=24, vdim=40, chunk=70, rot=24), linear(heads=2, dim=72, vdim=20, tau=0.5), None),
        layer(attention(heads=2, kv_heads=1, dim=56, vdim=72, chunk=9, rot=10, base=70.0), linear(heads=5, dim=18, vdim=34, tau=30.0), dense()),
        layer(attention(heads=3, kv_heads=1, dim=16, vdim=80, chunk=130, rot=0, scale=0.4), linear(heads=1, dim=100, vdim=100, tau=1.0),
              moe(experts=10, groups=5, keep=3, top=3, ff=24, shared=0)),
    ])


def config_b():
    """Values that other configurations keep apart made equal or one: a head of its own per query head, one head, chunks
    of a page and of one token, one group of experts, one expert used, rotation over the whole head; widths the wave-tile
    projections and the matrix-core attention take (so the bf16 run uses both)."""
    return SizizenConfig(vocab_size=256, width=128, eps=1e-6, layers=[
        layer(attention(heads=2, kv_heads=2, dim=64, vdim=64, chunk=128, rot=64, base=100.0, scale=0.125), linear(heads=2, dim=64, vdim=64, tau=1.0), dense(128)),
        layer(attention(heads=6, kv_heads=2, dim=64, vdim=32, chunk=64, rot=32, scale=0.2), linear(heads=1, dim=128, vdim=128, tau=16.0),
              moe(experts=4, groups=1, keep=1, top=1, ff=64, shared=64)),
        layer(attention(heads=1, kv_heads=1, dim=32, vdim=32, chunk=1, rot=32, scale=0.2), linear(heads=4, dim=16, vdim=32, tau=2.0),
              moe(experts=6, groups=6, keep=6, top=6, ff=128, shared=0)),
    ])


def config_c():
    """Memories whose head shapes are beyond the chunked form's reach or at its end, one expert per group, most groups
    dropped."""
    return SizizenConfig(vocab_size=200, width=96, eps=1e-5, layers=[
        layer(attention(heads=4, kv_heads=2, dim=8, vdim=8, chunk=200, rot=2), linear(heads=1, dim=300, vdim=24, tau=8.0), dense(64)),
        layer(attention(heads=9, kv_heads=1, dim=32, vdim=136, chunk=33, rot=8), linear(heads=1, dim=250, vdim=200, tau=3.0),
              moe(experts=8, groups=8, keep=2, top=2, ff=50, shared=30)),
    ])


def random_config(seed):
    """A configuration drawn at random: layer order, head counts and widths (among them the shapes the matrix-core
    attention, the wave-tile projections and the chunked memory take and ones they do not), chunks from 1 to beyond the
    prompt, rotation over none / part / all of a head, dense and routed feed-forwards and none."""
    import random
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(2, 5)):
        kv = rng.choice([1, 2, 3])
        dim, vdim = rng.choice([(8, 8), (24, 40), (32, 32), (64, 64), (64, 32), (96, 96), (128, 64), (64, 128), (40, 56), (128, 128), (160, 20)])
        left = attention(kv * rng.choice([1, 2, 4, 9]), kv, dim, vdim, rng.choice([1, 2, 17, 64, 65, 100, 300]),
                         rng.choice([r for r in (0, 2, 8, 16, dim) if r <= dim]), rng.choice([50.0, 1e4, 1e6]),
                         rng.choice([0.1, dim ** -0.5, 0.5]))
        right = linear(rng.choice([1, 2, 3, 5]), rng.choice([8, 18, 32, 64, 100, 128, 150]), rng.choice([4, 8, 24, 33, 64, 100, 128, 144]),
                       rng.choice([0.7, 1.0, 4.0, 16.0]))
        kind = rng.random()
        mlp = None
        if kind < 0.35:
            mlp = dense(rng.choice([64, 150, 256]))
        elif kind < 0.85:
            groups, per = rng.choice([1, 2, 3, 4]), rng.choice([1, 2, 3, 5])
            keep = rng.randint(1, groups)
            mlp = moe(groups * per, groups, keep, rng.randint(1, min(6, keep * per)), rng.choice([24, 50, 64]), rng.choice([0, 30, 64]))
        layers.append(layer(left, right, mlp))
    return SizizenConfig(vocab_size=rng.choice([97, 256, 331, 1000]), width=rng.choice([48, 100, 192, 256]), layers=layers,
                         eps=rng.choice([1e-5, 1e-6]))


def make_engine(cfg, dtype=torch.float32, seed=0, pages=24, slots=4, rows=4, step_tokens=512, max_tokens=512, model=None,
                rank=16):
    from micro_vllm_amd.core.engine import InferenceEngine
    return InferenceEngine(model=model or build_random_model(cfg, seed, rank=rank), max_batch_size=rows,
                           max_prefill_tokens=step_tokens, n_blocks=pages, max_tokens=max_tokens, state_slots=slots,
                           dtype=dtype)
