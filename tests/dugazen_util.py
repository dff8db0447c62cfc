"""Small Dugazen configurations for the tests (none with the proportions of a real checkpoint) and an engine builder;
the helpers that feed a request in portions are those of ragged_util."""
import torch

from micro_vllm_amd.models.dugazen import DugazenConfig, build_random_model


def attention(heads=6, kv_heads=2, dim=40, vdim=24, window=37, rot=24, base=3000.0, scale=0.21, v_mix=True):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
            "rot": {"base": base, "dims": rot}, "scale": scale, "v_mix": v_mix}


def delta(heads=6, kv_heads=3, dim=40, vdim=56, conv=3):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def dense(ff=150, limit=0.9):
    return {"kind": "dense", "ff": ff, "limit": limit}


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def config_a():
    """Odd sizes everywhere, a memory first, query/key heads shared by two heads, three layers that mix values (the
    first of them behind one that does not), feed-forwards on either kind of mixer and absent from either."""
    return DugazenConfig(vocab_size=331, width=176, eps=1e-5, residual_mult=0.7, logit_scale=1.6, layers=[
        layer("channel_delta", delta(), dense()),
        layer("attention", attention(v_mix=False), None),
        layer("attention", attention(heads=4, kv_heads=2, dim=24, vdim=40, window=70, rot=24), dense(200, 2.5)),
        layer("channel_delta", delta(heads=4, kv_heads=1, dim=72, vdim=20, conv=5), None),
        layer("attention", attention(heads=2, kv_heads=2, dim=56, vdim=40, window=9, rot=10, base=70.0), dense(64, 0.5)),
        layer("attention", attention(heads=2, kv_heads=1, dim=16, vdim=80, window=130, rot=0, scale=0.4), None),
    ])


def config_b():
    """Values that other configurations keep apart made equal or one: a head of its own per query head, one head, one
    tap, a window of one token, unit multipliers, rotation over the whole head; widths the wave-tile projections and
    the matrix-core attention take (so the bf16 run uses both)."""
    return DugazenConfig(vocab_size=256, width=128, eps=1e-6, residual_mult=1.0, logit_scale=1.0, layers=[
        layer("attention", attention(heads=2, kv_heads=2, dim=64, vdim=64, window=65, rot=64, base=100.0, scale=0.125), dense(128, 7.0)),
        layer("channel_delta", delta(heads=1, kv_heads=1, dim=128, vdim=128, conv=1), dense(128, 7.0)),
        layer("attention", attention(heads=4, kv_heads=2, dim=32, vdim=64, window=1, rot=32, scale=0.2), dense(128, 7.0)),
        layer("channel_delta", delta(heads=2, kv_heads=2, dim=64, vdim=64, conv=2), dense(128, 7.0)),
    ])


def config_c():
    """No attention at all, memories whose head shapes differ, one of them beyond the chunked form's reach."""
    return DugazenConfig(vocab_size=200, width=96, eps=1e-6, residual_mult=1.3, logit_scale=0.25, layers=[
        layer("channel_delta", delta(heads=2, kv_heads=1, dim=200, vdim=24, conv=4), None),
        layer("channel_delta", delta(heads=3, kv_heads=3, dim=16, vdim=136, conv=4), dense(80, 1.2)),
    ])


def random_config(seed):
    """A configuration drawn at random: layer order, head counts and widths (among them the shapes the matrix-core
    attention, the wave-tile projections and the chunked memory take and ones they do not), windows from 1 to beyond
    the prompt, taps from 1 to 6, rotation over none / part / all of a head, with and without mixed values and
    feed-forwards."""
    import random
    rng = random.Random(seed)
    layers = []
    mixed = rng.choice([(1, 64), (2, 32), (2, 24), (1, 40)])      # kv_heads, vdim of the layers that mix values
    for i in range(rng.randint(2, 5)):
        mlp = dense(rng.choice([64, 150, 256]), rng.choice([0.3, 1.0, 7.0])) if rng.random() < 0.6 else None
        if rng.random() < 0.5:
            k = rng.choice([1, 2, 3])
            layers.append(layer("channel_delta", delta(k * rng.choice([1, 2, 4]), k, rng.choice([8, 20, 32, 64, 100, 128, 150]),
                                                       rng.choice([4, 8, 24, 32, 64, 100, 128]), rng.randint(1, 6)), mlp))
        else:
            mix = rng.random() < 0.7
            kv, vdim = mixed if mix else (rng.choice([1, 2, 3]), rng.choice([8, 32, 56, 128]))
            dim = rng.choice([8, 24, 32, 64, 128])
            layers.append(layer("attention", attention(
                kv * rng.choice([1, 2, 4, 9]), kv, dim, vdim, rng.choice([1, 2, 17, 64, 65, 100, 300]),
                rng.choice([r for r in (0, 2, 8, 16, dim) if r <= dim]), rng.choice([50.0, 1e4, 1e6]),
                rng.choice([0.1, dim ** -0.5, 0.5]), mix), mlp))
    return DugazenConfig(vocab_size=rng.choice([97, 256, 331, 1000]), width=rng.choice([48, 100, 192, 256]), layers=layers,
                         eps=rng.choice([1e-5, 1e-6]), residual_mult=rng.choice([0.3, 1.0, 1.4]),
                         logit_scale=rng.choice([0.5, 1.0, 3.0]))


def make_engine(cfg, dtype=torch.float32, seed=0, pages=24, slots=4, rows=4, step_tokens=512, max_tokens=512, model=None,
                rank=16):
    from micro_vllm_amd.core.engine import InferenceEngine
    return InferenceEngine(model=model or build_random_model(cfg, seed, rank=rank), max_batch_size=rows,
                           max_prefill_tokens=step_tokens, n_blocks=pages, max_tokens=max_tokens, state_slots=slots,
                           dtype=dtype)
