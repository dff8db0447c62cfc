"""Host-side parts of the Dugazen design (no GPU): configuration reader, tensor table, registry and checkpoint loading,
cache layout, and the plain restatement's own consistency (the delta rule against its closed forms, the decay's place in
the order of operations, norms over whole projections, rotation, the window's edge, mixed values, the clamped gate)."""
import json
import math
import os

import pytest
import torch

from dugazen_util import attention, config_a, config_b, config_c, dense, layer, random_config
from oracle import ref_dugazen as ref

D = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=D)


def test_config_reader_and_tensor_table(mv):
    from micro_vllm_amd.models.dugazen import DugazenConfig, tensor_shapes
    cfg = config_a()
    again = DugazenConfig.from_json(json.loads(json.dumps(cfg.to_json())))
    assert (again.vocab_size, again.width, again.eps, again.residual_mult, again.logit_scale) == (331, 176, 1e-5, 0.7, 1.6)
    assert again.num_hidden_layers == 6 and again.first_value_mix() == 2 and config_c().first_value_mix() is None
    s = tensor_shapes(again, rank=11)
    assert s["embed"] == s["head"] == (331, 176) and s["final.norm"] == (176,)
    assert s["l0.mix.q"] == s["l0.mix.k"] == (120, 176) and s["l0.mix.v"] == (336, 176) and s["l0.mix.v.conv"] == (336, 3)
    assert s["l0.mix.b"] == (6, 176) and s["l0.mix.A_log"] == (6,) and s["l0.mix.dt_bias"] == (240,) and s["l0.mix.norm"] == (56,)
    assert s["l0.mix.a1"] == s["l0.mix.g1"] == (11, 176) and s["l0.mix.a2"] == (240, 11) and s["l0.mix.g2"] == (336, 11)
    assert s["l0.mix.o"] == (176, 336) and s["l0.norm2b"] == (176,) and s["l0.mlp.up"] == (150, 176)
    assert s["l1.mix.q"] == (240, 176) and s["l1.mix.k.b"] == (80,) and s["l1.mix.v.b"] == (48,) and s["l1.mix.g"] == (144, 176)
    assert s["l1.mix.q.norm"] == (240,) and s["l1.mix.k.norm"] == (80,) and s["l1.mix.o.b"] == (176,)
    assert "l1.mix.vmix" not in s and s["l2.mix.vmix"] == () and "l1.norm2" not in s and s["l1.norm1b"] == (176,)
    for spoil in (lambda d: d["layers"][0].update(type="conv"), lambda d: d["layers"][0]["mlp"].update(kind="moe"),
                  lambda d: d["layers"][0]["mixer"].update(kv_heads=4), lambda d: d["layers"][0]["mixer"].update(conv=0),
                  lambda d: d["layers"][1]["mixer"]["rot"].update(dims=25), lambda d: d["layers"][1]["mixer"]["rot"].update(dims=42),
                  lambda d: d["layers"][1]["mixer"]["mask"].update(size=0), lambda d: d["layers"][4]["mixer"].update(vdim=44)):
        bad = json.loads(json.dumps(cfg.to_json()))
        spoil(bad)
        with pytest.raises(ValueError):
            DugazenConfig.from_json(bad)
    for seed in range(20):
        c = random_config(seed)
        assert DugazenConfig.from_json(json.loads(json.dumps(c.to_json()))).to_json() == c.to_json()


def test_registry_loads_a_checkpoint_directory(mv, tmp_path):
    from safetensors.torch import save_file
    from micro_vllm_amd.core.model_loader import load_model
    from micro_vllm_amd.models.dugazen import random_weights
    cfg = config_a()
    w = random_weights(cfg, 1, rank=5)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg.to_json()))
    model, tok = load_model(str(tmp_path))
    assert model.family == "ragged" and model.config.architecture == "Dugazen" and model.config.residual_mult == 0.7
    assert torch.equal(model.get("l2.mix.vmix"), w["l2.mix.vmix"]) and model.get("l0.mix.a1").shape == (5, 176)
    assert tok.encode("3 17 330") == [3, 17, 330]
    os.remove(tmp_path / "model.safetensors")
    del w["l0.mix.g2"]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError):
        load_model(str(tmp_path))


def test_cache_layout(mv):
    from micro_vllm_amd.core.layer.ragged_runner import RaggedRunner
    runner = RaggedRunner.__new__(RaggedRunner)
    for make in (config_a, config_b):
        cfg = make()
        runner.cfg, runner.width, runner.runs = cfg, cfg.width, cfg.layer_runs()
        kv, state = runner.cache_layout()
        assert sorted(list(kv) + list(state)) == list(range(len(cfg.layers)))
        if make is config_a:
            assert kv[1] == (2, 40, 24) and kv[5] == (1, 16, 80)
            assert state[0] == {"conv": (2, 2 * 120 + 336), "delta": (6, 40, 56)}
            assert state[3] == {"conv": (4, 2 * 72 + 80), "delta": (4, 72, 20)}
        else:
            assert state[1] == {"conv": (0, 384), "delta": (1, 128, 128)}        # one tap: nothing is carried


def test_restatement_delta_rule():
    T, H, n, p = 9, 2, 5, 3
    q, k, v = rnd(T, H, n, seed=1), ref.unit_vector(rnd(T, H, n, seed=2)), rnd(T, H, p, seed=3)
    one, beta = torch.ones(T, H, n, dtype=D), torch.ones(T, H, dtype=D)
    # no decay and beta 1 with unit keys: reading with the key just written gives its value
    o = ref.delta_rule(k, k, v, one, beta)
    assert torch.allclose(o, v, atol=1e-5)
    # orthogonal keys do not disturb each other: the state is the sum of the outer products
    eye = torch.eye(n, dtype=D)[:, None, :].expand(n, H, n)
    o, S = ref.delta_rule(eye, eye, v[:n], one[:n], beta[:n], torch.zeros(H, n, p, dtype=D))
    assert torch.allclose(S, v[:n].transpose(0, 1))
    # the decay acts before the correction, row by row: with one row decayed to nothing the value written there is gone
    gate = one.clone()
    gate[1, :, 0] = 0.0
    kk = torch.zeros(2, H, n, dtype=D)
    kk[:, :, 0] = 1.0
    half = torch.full((2, H), 0.5, dtype=D)
    _, S = ref.delta_rule(kk, kk, v[:2], gate[:2], half, torch.zeros(H, n, p, dtype=D))
    assert torch.allclose(S[:, 0], 0.5 * v[1])
    # the chunk identity the fast form rests on:  (I + diag(b) A) U = diag(b) (V - (G K) S0)
    g = torch.sigmoid(rnd(T, H, n, seed=4))
    b = torch.sigmoid(rnd(T, H, seed=5))
    S0 = rnd(H, n, p, seed=6)
    o, S = ref.delta_rule(q, k, v, g, b, S0)
    for h in range(H):
        G = torch.cumprod(g[:, h], 0)
        A = torch.tril((G * k[:, h]) @ (k[:, h] / G).T, -1)
        B = torch.tril((G * q[:, h]) @ (k[:, h] / G).T)
        U = torch.linalg.solve(torch.eye(T, dtype=D) + b[:, h, None] * A, b[:, h, None] * (v[:, h] - (G * k[:, h]) @ S0[h]))
        assert torch.allclose(o[:, h], (G * q[:, h]) @ S0[h] + B @ U)
        assert torch.allclose(S[h], G[-1][:, None] * S0[h] + (G[-1] / G * k[:, h]).T @ U)


def test_restatement_decay_convolution_unit_vectors():
    a, bias, a_log = rnd(4, 6), rnd(6, seed=1), torch.tensor([0.3, -1.0], dtype=D)
    g = ref.channel_decay(a, bias, a_log, 2)
    assert g.shape == (4, 2, 3)
    assert abs(float(g[2, 1, 0]) - math.exp(-math.exp(-1.0) * math.log1p(math.exp(float(a[2, 3] + bias[3]))))) < 1e-12
    big = ref.channel_decay(torch.tensor([[800.0, -800.0]], dtype=D), torch.zeros(2, dtype=D), torch.zeros(1, dtype=D), 1)
    assert float(big[0, 0, 0]) == math.exp(-800.0) and float(big[0, 0, 1]) == 1.0
    u, w = rnd(7, 3), rnd(3, 4, seed=1)
    y = ref.causal_conv(u, w)
    assert torch.allclose(y[0], w[:, 3] * u[0]) and torch.allclose(y[5], sum(w[:, j] * u[2 + j] for j in range(4)))
    x = torch.tensor([3e-4, 4e-4], dtype=D)
    assert torch.allclose(ref.unit_vector(x), x / math.sqrt(2.5e-7 + 1e-6))     # the constant counts for short vectors


def test_restatement_attention_parts():
    # rotation keeps lengths and depends on distances only; dimensions behind rot pass
    q, k = rnd(12, 1, 10), rnd(12, 1, 10, seed=1)
    q[:] = q[0]
    k[:] = k[0]
    rq, rk = ref.rotate_halves(q, 6, 50.0), ref.rotate_halves(k, 6, 50.0)
    assert torch.equal(rq[:, :, 6:], q[:, :, 6:]) and torch.equal(rq[0], q[0]) and not torch.allclose(rq[3], q[3])
    s = rq[:, 0] @ rk[:, 0].T
    assert torch.allclose(s[4, 1], s[9, 6]) and torch.allclose(rq.norm(dim=-1), q.norm(dim=-1))
    assert torch.allclose(rq[1, 0, 0], q[1, 0, 0] * math.cos(1) - q[1, 0, 3] * math.sin(1))
    # the window keeps the token itself and window - 1 before it
    v = rnd(12, 1, 4, seed=2)
    out = ref.window_attention(q, k, v, 0.3, 5)
    assert torch.allclose(out[9, 0], v[5:10, 0].mean(0))                        # equal keys: equal weights
    # norm over the whole projection: doubling one head's rows changes the others
    cfg = config_a()
    from micro_vllm_amd.models.dugazen import random_weights
    W = {n: t.to(D) for n, t in random_weights(cfg, 0).items()}
    m = cfg.layers[1]["mixer"]
    h = rnd(6, cfg.width, seed=3)
    base = ref.attention_mixer(h, W, "l1.mix.", m, 1e-5, [None])
    W["l1.mix.q"] = W["l1.mix.q"] * 3.0
    W["l1.mix.q.b"] = W["l1.mix.q.b"] * 3.0
    assert torch.allclose(ref.attention_mixer(h, W, "l1.mix.", m, 1e-5, [None]), base, atol=1e-4)
    W["l1.mix.q"][:40] *= 5.0
    assert not torch.allclose(ref.attention_mixer(h, W, "l1.mix.", m, 1e-5, [None]), base, atol=1e-3)


def test_restatement_mixed_values_and_clamped_gate():
    from micro_vllm_amd.models.dugazen import DugazenConfig, random_weights
    mix = attention(heads=2, kv_heads=1, dim=8, vdim=6, window=4, rot=4)
    cfg = DugazenConfig(vocab_size=50, width=32, eps=1e-6, layers=[layer("attention", mix, dense(20, 0.4)) for _ in range(3)])
    W = {n: t.to(D) for n, t in random_weights(cfg, 0).items()}
    toks = [3, 9, 1, 4, 4, 8]
    base = ref.forward(cfg.to_json(), W, toks)
    W["l0.mix.vmix"] = torch.tensor(0.9, dtype=D)             # the first layer's is not used
    assert torch.equal(ref.forward(cfg.to_json(), W, toks), base)
    W["l1.mix.vmix"] = W["l2.mix.vmix"] = torch.tensor(1.0, dtype=D)       # values of the first layer only
    only = ref.forward(cfg.to_json(), W, toks)
    for i in (1, 2):
        W[f"l{i}.mix.v"] = rnd(6, 32, seed=i)
    assert torch.allclose(ref.forward(cfg.to_json(), W, toks), only)
    # the gate is clamped from above only, the other factor on both sides
    eye = {"gate": torch.eye(4, dtype=D), "up": torch.eye(4, dtype=D), "down": torch.eye(4, dtype=D)}
    y = ref.clamped_ff(torch.tensor([[9.0, -9.0, 0.5, -0.5]], dtype=D), eye, "", 1.0)[0]
    sg = lambda z: 1 / (1 + math.exp(-1.702 * z))   # noqa: E731
    assert torch.allclose(y, torch.tensor([sg(1) * 2, 0.0, 0.5 * sg(0.5) * 1.5, -0.5 * sg(-0.5) * 0.5], dtype=D))
    eye["up"] = torch.zeros(4, 4, dtype=D)
    assert abs(float(ref.clamped_ff(torch.full((1, 4), -2.0, dtype=D), eye, "", 1.0)[0, 0]) + 2 * sg(-2)) < 1e-12
    # a prefix's logits do not depend on what follows
    for make in (config_a, config_b, config_c):
        c = make()
        Wc = random_weights(c, 2)
        t = [5, 9, 1, 0, 7, 7, 30]
        assert torch.allclose(ref.forward(c.to_json(), Wc, t[:4]), ref.forward(c.to_json(), Wc, t)[:4])
