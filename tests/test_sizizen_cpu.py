"""Host-side parts of the Sizizen design (no GPU): configuration reader, tensor table, registry and checkpoint loading,
cache layout, and the plain restatement's own consistency (gated linear attention against its closed forms, the decay,
norms, rotation, chunk edges, the group-limited choice, the order of norms and sums)."""
import json
import math
import os

import pytest
import torch

from oracle import ref_sizizen as ref
from sizizen_util import attention, config_a, config_b, config_c, dense, layer, linear, random_config

D = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=D)


def test_config_reader_and_tensor_table(mv):
    from micro_vllm_amd.models.sizizen import SizizenConfig, tensor_shapes
    cfg = config_a()
    again = SizizenConfig.from_json(json.loads(json.dumps(cfg.to_json())))
    assert (again.vocab_size, again.width, again.eps, again.num_hidden_layers) == (331, 176, 1e-5, 4)
    s = tensor_shapes(again, rank=11)
    assert s["embed"] == s["head"] == (331, 176) and s["final.norm"] == (176,)
    a = "l0.mix.left."
    assert s[a + "q"] == (240, 176) and s[a + "k.b"] == (80,) and s[a + "v"] == (48, 176) and s[a + "v.b"] == (48,)
    assert s[a + "q.norm"] == s[a + "k.norm"] == (40,) and s[a + "o"] == (176, 144) and s[a + "out"] == (176,)
    a = "l0.mix.right."
    assert s[a + "q"] == s[a + "k"] == (120, 176) and s[a + "v"] == s[a + "g"] == (168, 176) and s[a + "o"] == (176, 168)
    assert s[a + "a1"] == (11, 176) and s[a + "a2"] == (120, 11) and s[a + "a2.b"] == (120,) and s[a + "norm"] == (56,)
    assert s["l0.mlp.router"] == (12, 176) and s["l0.mlp.correction"] == (12,) and s["l0.mlp.e11.down"] == (176, 40)
    assert s["l0.mlp.shared.up"] == (72, 176) and "l3.mlp.shared.up" not in s and "l0.mlp.e0.gate" not in s
    assert "l1.norm2" not in s and s["l2.mlp.gate"] == (150, 176) and s["l2.norm2"] == (176,)

    def mixer(side, **kw):
        return lambda d: d["layers"][0]["mixer"][side].update(**kw)
    for spoil in (lambda d: d["layers"][0].update(type="attention"), lambda d: d["layers"][0]["mlp"].update(kind="other"),
                  mixer("left", kv_heads=4), mixer("left", kv_heads=0), mixer("left", rot={"base": 9.0, "dims": 25}),
                  mixer("left", rot={"base": 9.0, "dims": 42}), mixer("left", mask={"size": 0}), mixer("right", tau=0.0),
                  lambda d: d["layers"][0]["mlp"]["router"].update(top=9), lambda d: d["layers"][0]["mlp"]["router"].update(experts=13),
                  lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(keep=4)):
        bad = json.loads(json.dumps(cfg.to_json()))
        spoil(bad)
        with pytest.raises(ValueError):
            SizizenConfig.from_json(bad)
    for seed in range(20):
        c = random_config(seed)
        assert SizizenConfig.from_json(json.loads(json.dumps(c.to_json()))).to_json() == c.to_json()


def test_registry_loads_a_checkpoint_directory(mv, tmp_path):
    from safetensors.torch import save_file
    from micro_vllm_amd.core.model_loader import load_model
    from micro_vllm_amd.models.sizizen import random_weights
    cfg = config_a()
    w = random_weights(cfg, 1, rank=5)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg.to_json()))
    model, tok = load_model(str(tmp_path))
    assert model.family == "ragged" and model.config.architecture == "Sizizen" and model.config.eps == 1e-5
    assert torch.equal(model.get("l2.mix.right.a2.b"), w["l2.mix.right.a2.b"]) and model.get("l0.mix.right.a1").shape == (5, 176)
    assert tok.encode("3 17 330") == [3, 17, 330]
    os.remove(tmp_path / "model.safetensors")
    del w["l3.mlp.e9.down"]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError):
        load_model(str(tmp_path))


def test_cache_layout(mv):
    from micro_vllm_amd.core.layer.ragged_runner import RaggedRunner
    runner = RaggedRunner.__new__(RaggedRunner)
    for make in (config_a, config_b, config_c):
        cfg = make()
        runner.cfg, runner.width, runner.runs = cfg, cfg.width, cfg.layer_runs()
        kv, state = runner.cache_layout()
        assert sorted(kv) == sorted(state) == list(range(len(cfg.layers)))      # pages and a memory in every layer
        for i, lay in enumerate(cfg.layers):
            L, R = lay["mixer"]["left"], lay["mixer"]["right"]
            assert kv[i] == (L["kv_heads"], L["dim"], L["vdim"])
            assert list(state[i].values()) == [(R["heads"], R["dim"], R["vdim"])]


def test_restatement_gated_linear_attention():
    T, H, n, p = 9, 2, 5, 3
    q, k, v = rnd(T, H, n, seed=1), rnd(T, H, n, seed=2), rnd(T, H, p, seed=3)
    one = torch.ones(T, H, n, dtype=D)
    # no decay: causal sums of (q . k) v, the token itself included
    o = ref.gated_linear_attention(q, k, v, one)
    for h in range(H):
        assert torch.allclose(o[:, h], torch.tril(q[:, h] @ k[:, h].T) @ v[:, h])
    # the decay acts on the rows of key channels, before the token's own write
    gate = one.clone()
    gate[1, :, 0] = 0.0
    _, S = ref.gated_linear_attention(q[:2], k[:2], v[:2], gate[:2], torch.zeros(H, n, p, dtype=D))
    assert torch.allclose(S[:, 0], k[1, :, 0, None] * v[1])
    assert torch.allclose(S[:, 1], k[0, :, 1, None] * v[0] + k[1, :, 1, None] * v[1])
    # the chunk identity the fast form rests on
    g = torch.sigmoid(rnd(T, H, n, seed=4))
    S0 = rnd(H, n, p, seed=6)
    o, S = ref.gated_linear_attention(q, k, v, g, S0)
    for h in range(H):
        G = torch.cumprod(g[:, h], 0)
        B = torch.tril((G * q[:, h]) @ (k[:, h] / G).T)
        assert torch.allclose(o[:, h], (G * q[:, h]) @ S0[h] + B @ v[:, h])
        assert torch.allclose(S[h], G[-1][:, None] * S0[h] + (G[-1] / G * k[:, h]).T @ v[:, h])


def test_restatement_decay_and_norms():
    z = torch.tensor([-3.0, 0.0, 2.5, 800.0, -800.0], dtype=D)
    a = ref.channel_decay(z, 16.0)
    for i in range(3):
        assert abs(float(a[i]) - (1 / (1 + math.exp(-float(z[i])))) ** (1 / 16)) < 1e-14
    assert float(a[3]) == 1.0 and abs(float(a[4]) - math.exp(-50.0)) < 1e-30
    x = rnd(4, 10) + 100.0
    y = ref.layer_norm(x, torch.ones(10, dtype=D), 1e-5)
    assert torch.allclose(y.mean(-1), torch.zeros(4, dtype=D), atol=1e-12) and torch.allclose((y * y).mean(-1), torch.ones(4, dtype=D), atol=1e-4)
    assert torch.allclose(ref.layer_norm(x + 5.0, torch.ones(10, dtype=D), 1e-5), y)          # a shift is no news
    small = torch.tensor([3e-3, -3e-3], dtype=D)
    assert torch.allclose(ref.layer_norm(small, torch.ones(2, dtype=D), 1e-5), small / math.sqrt(9e-6 + 1e-5))   # eps inside the root
    assert torch.allclose(ref.rms_norm(small, torch.full((2,), 2.0, dtype=D), 1e-5), 2 * small / math.sqrt(9e-6 + 1e-5))


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
    # equal keys: the mean of the values from the chunk's start to the token
    v = rnd(12, 1, 4, seed=2)
    out = ref.chunked_attention(q, k, v, 0.3, 5)
    assert torch.allclose(out[9, 0], v[5:10, 0].mean(0)) and torch.allclose(out[10, 0], v[10, 0]) and torch.allclose(out[4, 0], v[:5, 0].mean(0))
    # two query heads share a key/value head: equal queries give equal outputs, other pairs do not
    q4 = rnd(12, 4, 10, seed=4)
    q4[:, 1], q4[:, 2] = q4[:, 0], q4[:, 0]
    o = ref.chunked_attention(q4, rnd(12, 2, 10, seed=5), rnd(12, 2, 4, seed=6), 0.3, 7)
    assert torch.equal(o[:, 0], o[:, 1]) and not torch.allclose(o[:, 0], o[:, 2])
    # the norm is each head's own: another head's rows do not matter
    cfg = config_a()
    from micro_vllm_amd.models.sizizen import random_weights
    W = {n: t.to(D) for n, t in random_weights(cfg, 0).items()}
    m, a = cfg.layers[0]["mixer"]["left"], "l0.mix.left."
    h = rnd(6, cfg.width, seed=3)
    base = ref.attention_mixer(h, W, a, m, 1e-5)
    for n in ("q", "q.b"):
        W[a + n] = W[a + n].clone()
        W[a + n][40:80] *= 7.0
    assert torch.allclose(ref.attention_mixer(h, W, a, m, 1e-5), base, atol=1e-4)
    W[a + "q.b"][:40] += 1.0
    assert not torch.allclose(ref.attention_mixer(h, W, a, m, 1e-5), base, atol=1e-3)


def test_restatement_group_limited_choice():
    eye = torch.eye(6, dtype=D)
    logit = lambda s: math.log(s / (1 - s))   # noqa: E731
    s = torch.tensor([0.9, 0.1, 0.6, 0.55, 0.5, 0.45], dtype=D)
    h = torch.tensor([logit(float(x)) for x in s], dtype=D)
    zero = torch.zeros(6, dtype=D)
    # pairs: worth 1.0, 1.15, 0.95 - two kept; the weights are the scores as they are
    got = ref.route(h, eye, zero, 3, 2, 3)
    assert [e for e, _ in got] == [0, 2, 3] and torch.allclose(torch.stack([w for _, w in got]), s[[0, 2, 3]])
    assert [e for e, _ in ref.route(h, eye, zero, 3, 1, 2)] == [2, 3]          # the best expert's group is not the best group
    # a correction moves the choice, also below zero, and leaves the weights alone
    corr = torch.tensor([-3.0, -3.0, -1.0, -1.0, 0.0, 0.0], dtype=D)
    got = ref.route(h, eye, corr, 3, 2, 4)
    assert [e for e, _ in got] == [4, 5, 2, 3] and torch.allclose(got[2][1], s[2])
    assert [e for e, _ in ref.route(h, eye, zero, 1, 1, 6)] == [0, 2, 3, 4, 5, 1]
    # worth counts the two largest of three only
    s3 = torch.tensor([0.5, 0.5, 0.49, 0.8, 0.3, 0.01], dtype=D)
    h3 = torch.tensor([logit(float(x)) for x in s3], dtype=D)
    assert [e for e, _ in ref.route(h3, eye, zero, 2, 1, 1)] == [3]


def test_restatement_stack():
    from micro_vllm_amd.models.sizizen import SizizenConfig, random_weights
    cfg = SizizenConfig(vocab_size=50, width=32, eps=1e-6, layers=[
        layer(attention(2, 1, 8, 6, 4, 4), linear(2, 6, 5, 3.0), dense(20)), layer(attention(2, 1, 8, 6, 3, 4), linear(1, 6, 5, 3.0), None)])
    W = {n: t.to(D) for n, t in random_weights(cfg, 0).items()}
    toks = [3, 9, 1, 4, 4, 8]
    base = ref.forward(cfg.to_json(), W, toks)
    # either branch passes a norm of its own: its size does not matter, its weight does
    W["l0.mix.left.o"] = W["l0.mix.left.o"] * 1000.0
    assert torch.allclose(ref.forward(cfg.to_json(), W, toks), base, atol=1e-4)
    W["l0.mix.left.out"] = W["l0.mix.left.out"] * 3.0
    assert not torch.allclose(ref.forward(cfg.to_json(), W, toks), base, atol=1e-2)
    # the first layer's input is the table's row as it is
    h = W["embed"][torch.tensor(toks)]
    W["l0.norm1"] = W["l0.norm1"] * 0
    W["l0.norm2"] = W["l0.norm2"] * 0
    W["l1.norm1"] = W["l1.norm1"] * 0
    assert torch.allclose(ref.forward(cfg.to_json(), W, toks), ref.layer_norm(h, W["final.norm"], 1e-6) @ W["head"].T)
    # dense: SiLU on the gate; experts: squared ReLU
    eye = {"gate": torch.eye(3, dtype=D), "up": torch.eye(3, dtype=D), "down": torch.eye(3, dtype=D)}
    x = torch.tensor([[2.0, -1.0, 0.0]], dtype=D)
    assert torch.allclose(ref.dense_ff(x, eye, ""), torch.sigmoid(x) * x * x) and torch.equal(ref.relu2_ff(x, eye, ""), torch.tensor([[4.0, 0.0, 0.0]], dtype=D))
    # a prefix's logits do not depend on what follows
    for make in (config_a, config_b, config_c):
        c = make()
        Wc = random_weights(c, 2)
        t = [5, 9, 1, 0, 7, 7, 30]
        assert torch.allclose(ref.forward(c.to_json(), Wc, t[:4]), ref.forward(c.to_json(), Wc, t)[:4])
