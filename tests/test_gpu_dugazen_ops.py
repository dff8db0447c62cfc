"""Each mechanism the Dugazen stack adds to the ragged family alone: the HIP kernel against the plain restatement in
oracle/ref_dugazen.py (fp64 on the CPU), on random inputs and on inputs built so that a fault shows (a key made dominant
just inside and just outside a window and at page borders, a memory that must hold one early write over hundreds of
tokens, gates of exactly zero and one, pages and slots dirtied before use, short vectors whose length the constant under
the root decides)."""
import math

import pytest
import torch

from oracle import ref_dugazen as ref

pytestmark = pytest.mark.gpu
DEV = "cuda"


@pytest.fixture(scope="module")
def ops():
    import micro_vllm_amd  # noqa: F401
    from micro_vllm_amd.kernel import ragged_ops
    return ragged_ops


def make_cache(kv=None, state=None, pages=16, slots=3, dtype=torch.float32, page=64, max_tokens=1024):
    from micro_vllm_amd.core.state_cache import HybridCacheManager
    cache = HybridCacheManager(pages, page, slots, kv or {}, state or {}, dtype=dtype, device=DEV, max_tokens=max_tokens,
                               max_rows=4, max_step_tokens=1024)
    for t in list(cache.k_caches.values()) + list(cache.v_caches.values()):
        t.fill_(9.0)                       # whatever a page or a slot held before
    for named in cache.states.values():
        for t in named.values():
            t.fill_(-7.0)
    order = list(cache._free_pages)        # pages in no particular order
    cache._free_pages.clear()
    cache._free_pages.extend(order[1::2] + order[0::2])
    return cache


def step_of(cache, rows):
    cache.reserve([(sid, len(t)) for sid, t in rows])
    st = cache.plan(rows)
    cache.advance([(sid, len(t)) for sid, t in rows])
    return st


def feed(cache, plan, fn):
    """plan = [[(seq, count)]]: runs fn(step, {seq: (first position, count, first token of the step)}) per step."""
    at = {}
    for rows in plan:
        st = step_of(cache, [(k, [0] * c) for k, c in rows])
        where, o = {}, 0
        for k, c in rows:
            where[k] = (at.get(k, 0), c, o)
            at[k] = at.get(k, 0) + c
            o += c
        fn(st, where)


def gather(seqs, where):
    return torch.cat([seqs[k][p:p + c] for k, (p, c, _) in where.items()]).float().to(DEV)


def scatter(got, out, where):
    for k, (_, c, o) in where.items():
        got[k].append(out[o:o + c].float().cpu().double())


# ----------------------------------------------------------------------------------------------- row-wise steps
@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("n", [203, 96, 1500, 3072, 5000, 9000])
def test_residual_step_between_two_norms(ops, f32, n):
    """Every width takes another form of the kernel: odd, in registers at 1 to 8 vectors a thread, beyond them."""
    g = torch.Generator().manual_seed(n)
    dt = torch.float32 if f32 else torch.bfloat16
    tol = 2e-5 if f32 else 4e-2
    T, eps, m = 7, 1e-5, 0.6
    x0, y = torch.randn(T, n, generator=g) * 2, torch.randn(T, n, generator=g)
    w, w2, b = (0.3 * torch.randn(n, generator=g) for _ in range(3))
    want = x0.double() + m * ref.offset_norm(y.double() + b.double(), w.double(), eps)
    x, h = x0.to(DEV), torch.empty(T, n, dtype=dt, device=DEV)
    ops.postnorm_residual(y.to(DEV), w.to(DEV), eps, x, h, bias=b.to(DEV), mult=m, next_w=w2.to(DEV))
    assert (x.cpu().double() - want).abs().max().item() < 1e-5
    assert (h.float().cpu().double() - ref.offset_norm(want, w2.double(), eps)).abs().max().item() < tol
    # without bias and next norm: h is the stream itself
    want = x0.double() + m * ref.offset_norm(y.double(), w.double(), eps)
    x = x0.to(DEV)
    ops.postnorm_residual(y.to(DEV), w.to(DEV), eps, x, h, mult=m)
    assert (x.cpu().double() - want).abs().max().item() < 1e-5 and torch.equal(h, x.to(dt))
    # two summands from column slices of wider buffers
    wide = torch.zeros(T, 2 * n + 4, device=DEV)
    wide[:, 4:4 + n] = y.to(DEV)
    x = x0.to(DEV)
    ops.postnorm_residual(wide[:, 4:4 + n], w.to(DEV), eps, x, h, y2=x0.to(DEV), s1=0.5, s2=-1.5, next_w=w2.to(DEV))
    want = x0.double() + ref.offset_norm(0.5 * y.double() - 1.5 * x0.double(), w.double(), eps)
    assert (x.cpu().double() - want).abs().max().item() < 1e-5
    assert (h.float().cpu().double() - ref.offset_norm(want, w2.double(), eps)).abs().max().item() < tol


@pytest.mark.parametrize("f32", [False, True])
def test_embedding_with_its_norm(ops, f32):
    g = torch.Generator().manual_seed(3)
    dt = torch.float32 if f32 else torch.bfloat16
    table, ids, w = torch.randn(50, 150, generator=g).to(dt), torch.tensor([3, 49, 0, 3], dtype=torch.int32), torch.randn(150, generator=g)
    x, h = torch.empty(4, 150, device=DEV), torch.empty(4, 150, dtype=dt, device=DEV)
    ops.embed_scaled(table.to(DEV), ids.to(DEV), 1.5, x, h, w=w.to(DEV), eps=1e-5, offset=1.0)
    want = table.double()[ids.long()] * 1.5
    assert (x.cpu().double() - want).abs().max().item() < 1e-6
    assert (h.float().cpu().double() - ref.offset_norm(want, w.double(), 1e-5)).abs().max().item() < (1e-5 if f32 else 5e-2)


@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("heads,p", [(3, 40), (2, 1100), (5, 1)])
def test_unit_rms_per_head_with_a_shared_weight_and_a_sigmoid_gate(ops, f32, heads, p):
    g = torch.Generator().manual_seed(4)
    T, n = 11, heads * p
    y, z, w = torch.randn(T, n, generator=g), 3 * torch.randn(T, n, generator=g), torch.randn(p, generator=g)
    out = torch.empty(T, n, dtype=torch.float32 if f32 else torch.bfloat16, device=DEV)
    ops.gated_group_norm(y.to(DEV), z.to(DEV), w.to(DEV), out, heads, False, 1e-5, sigmoid=True)
    want = (ref.rms_unit(y.double().view(T, heads, p), 1e-5) * w.double()).reshape(T, n) * torch.sigmoid(z.double())
    assert (out.float().cpu().double() - want).abs().max().item() < (1e-5 if f32 else 1e-2 * want.abs().max().item())


# ----------------------------------------------------------------------------------------------- attention
@pytest.mark.parametrize("H,G,d,dv,rot,mix,normed", [(6, 2, 40, 24, 24, 2, True), (2, 2, 64, 64, 64, 1, True),
                                                      (1, 1, 10, 130, 0, 0, True), (4, 1, 96, 8, 2, 2, False),
                                                      (16, 4, 128, 128, 128, 1, False)])
@pytest.mark.parametrize("f32", [False, True])
def test_projection_norm_rotation_values_into_pages(ops, H, G, d, dv, rot, mix, normed, f32):
    g = torch.Generator().manual_seed(d + rot)
    dt = torch.float32 if f32 else torch.bfloat16
    cq, ck, cv, eps, base, lam = H * d, G * d, G * dv, 1e-5, 90.0, 0.3
    lens = {"a": 150, "b": 9}
    raw = {k: 2 * torch.randn(n, cq + ck + cv, generator=g) for k, n in lens.items()}
    first = {k: torch.randn(n, cv, generator=g) for k, n in lens.items()}
    qb, kb, vb = (torch.randn(n, generator=g) for n in (cq, ck, cv))
    qn, kn = 1 + 0.3 * torch.randn(cq, generator=g), 1 + 0.3 * torch.randn(ck, generator=g)
    inv = (base ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / max(rot, 1))).to(DEV) if rot else None
    cache = make_cache(kv={0: (G, d, dv)}, dtype=dt)
    got = {k: [] for k in lens}

    def run(st, where):
        buf = torch.zeros(st.tokens, cq + ck + cv + 5, device=DEV)
        buf[:, :cq + ck + cv] = gather(raw, where)
        vf = gather(first, where).contiguous()
        args = dict(q_bias=qb.to(DEV), k_bias=kb.to(DEV), v_bias=vb.to(DEV))
        if normed:
            args.update(q_norm=qn.to(DEV), k_norm=kn.to(DEV))
        ops.qkv_norm_rotary_store(buf[:, :cq + ck + cv], cache.k_caches[0], cache.v_caches[0], st, H, G, d, dv, inv, rot, eps,
                                  v_first=vf if mix else None, mix=mix, lam=lam, **args)
        scatter(got, torch.cat([buf[:, :cq], vf], 1), where)
        assert bool((buf[:, cq + ck + cv:] == 0).all())

    feed(cache, [[("a", 70), ("b", 1)], [("b", 2), ("a", 1)], [("a", 79), ("b", 6)]], run)
    for k, n in lens.items():
        x = raw[k].double()
        q, kk, v = x[:, :cq] + qb.double(), x[:, cq:cq + ck] + kb.double(), x[:, cq + ck:] + vb.double()
        if normed:
            q, kk = ref.rms_unit(q, eps) * qn.double(), ref.rms_unit(kk, eps) * kn.double()
        if rot:
            q = ref.rotate_halves(q.view(n, H, d), rot, base).view(n, cq)
            kk = ref.rotate_halves(kk.view(n, G, d), rot, base).view(n, ck)
        out = torch.cat(got[k])
        assert (out[:, :cq] - q).abs().max().item() < 3e-5, k
        if mix == 1:
            assert (out[:, cq:] - v).abs().max().item() < 1e-5       # kept for the layers behind
        if mix == 2:
            v = (1 - lam) * v + lam * first[k].double()
        pages = cache.get_blocks(k)
        rows = torch.tensor([pages[i // 64] * 64 + i % 64 for i in range(n)])
        tol = 3e-5 if f32 else 0.02 * max(kk.abs().max().item(), v.abs().max().item())
        assert (cache.k_caches[0].view(-1, ck).float().cpu()[rows].double() - kk).abs().max().item() < tol
        assert (cache.v_caches[0].view(-1, cv).float().cpu()[rows].double() - v).abs().max().item() < tol


def attend(ops, q, k, v, gate, H, G, d, dv, scale, window, portions, f32=True, tiled=True, grouped=False, splits=None):
    """Whole rows q | k | v fed in portions through the page store and the windowed attention with an output gate."""
    dt = torch.float32 if f32 else torch.bfloat16
    cache = make_cache(kv={0: (G, d, dv)}, dtype=dt, pages=24, max_tokens=1536)
    T = q.shape[0]
    rows = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1), gate], 1).float()
    C = (H + G) * d + G * dv
    out, pos = [], 0
    for n in portions:
        st = step_of(cache, [("s", [0] * n)])
        buf = rows[pos:pos + n].to(DEV).contiguous()
        ops.qkv_norm_rotary_store(buf[:, :C], cache.k_caches[0], cache.v_caches[0], st, H, G, d, dv, None, 0, 1e-6)
        o = torch.empty(n, H * dv, dtype=dt, device=DEV)
        part, sp = None, 0
        if grouped:
            sp = splits or ops.window_attn_splits(n, H, G, window)
            part = torch.empty(n * H * sp * (dv + 2), device=DEV)
        ops.window_attn(buf[:, :H * d], cache.k_caches[0], cache.v_caches[0], o, st, None, H, G, d, dv, scale, window, tiled=tiled,
                        part=part, splits=sp, gate=buf[:, C:])
        out.append(o.float().cpu())
        pos += n
    return torch.cat(out)


@pytest.mark.parametrize("H,G,d,dv,window", [(6, 2, 40, 24, 37), (4, 1, 64, 64, 65), (2, 2, 128, 64, 300), (9, 1, 32, 32, 64),
                                             (3, 3, 8, 8, 1)])
def test_windowed_attention_with_an_output_gate(ops, H, G, d, dv, window):
    """All four forms (one workgroup per head, shared reads, shared reads cut into pieces, matrix cores) apply the gate."""
    g = torch.Generator().manual_seed(d + window)
    T, scale = 170, 0.2
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, G, d, generator=g), torch.randn(T, G, dv, generator=g)
    gate = 2 * torch.randn(T, H * dv, generator=g)
    want = ref.window_attention(q.double(), k.double(), v.double(), scale, window).reshape(T, -1) * torch.sigmoid(gate.double())
    args = (ops, q, k, v, gate, H, G, d, dv, scale, window)
    for portions in ([T], [3, 61, 2, 63, 1, 40], [130] + [1] * 40):
        for kw in (dict(), dict(grouped=True), dict(grouped=True, splits=3)):
            assert (attend(*args, portions, **kw).double() - want).abs().max().item() < 1e-4, (portions[:3], kw)
            assert (attend(*args, portions, f32=False, **kw).double() - want).abs().max().item() < 0.06, (portions[:3], kw)
        assert (attend(*args, portions, f32=False, tiled=False).double() - want).abs().max().item() < 0.06


@pytest.mark.parametrize("window", [64, 65, 71, 200])
@pytest.mark.parametrize("decode,f32,grouped", [(False, True, False), (True, True, True), (True, False, True), (False, False, False)])
def test_window_edge_with_a_dominant_key(ops, window, decode, f32, grouped):
    """One key wins the softmax wherever it is visible and carries a value of its own: the query window - 1 tokens later
    returns it, the next one does not - at the first token, at page borders and behind the first window."""
    H = G = 1
    d = dv = 32
    T = 2 * window + 80
    g = torch.Generator().manual_seed(window)
    q, k, v = torch.randn(T, H, d, generator=g) * 0.01, torch.randn(T, G, d, generator=g) * 0.01, torch.zeros(T, G, dv)
    gate = torch.full((T, dv), 30.0)                          # open
    marks = (0, 5, 63, 64, window + 3)
    for n, mark in enumerate(marks):
        k[mark, 0] = 0
        k[mark, 0, n] = 1.0
        v[mark, 0, 0] = 100.0 + mark
    portions = [window // 2, 2] + [1] * (T - window // 2 - 2) if decode else [T]
    for n, mark in enumerate(marks):
        qq = q.clone()
        for i in (mark + window - 1, mark + window):
            qq[i, 0] = 0
            qq[i, 0, n] = 1.0
        out = attend(ops, qq, k, v, gate, H, G, d, dv, 40.0, window, portions, f32=f32, grouped=grouped)
        inside, outside = out[mark + window - 1, 0].item(), out[mark + window, 0].item()
        assert abs(inside - (100.0 + mark)) < (1.0 if f32 else 2.5), (mark, inside)
        assert abs(outside - (100.0 + mark)) > 40.0, (mark, outside)


# ----------------------------------------------------------------------------------------------- delta rule
def delta_reference_prep(raw, conv, K, n, H, p):
    T = raw.shape[0]
    y = ref.silu(ref.causal_conv(raw, conv))
    q = ref.unit_vector(y[:, :K * n].view(T, K, n)) * n ** -0.5
    k = ref.unit_vector(y[:, K * n:2 * K * n].view(T, K, n))
    return torch.cat([q.reshape(T, -1), k.reshape(T, -1), y[:, 2 * K * n:]], 1)


@pytest.mark.parametrize("K,H,n,p,taps,low", [(2, 4, 40, 24, 4, 37), (1, 1, 7, 300, 1, 64), (3, 3, 128, 20, 2, 1), (1, 6, 200, 48, 5, 0)])
@pytest.mark.parametrize("f32", [False, True])
def test_convolutions_unit_vectors_and_beta_over_steps(ops, K, H, n, p, taps, low, f32):
    """Portions shorter and longer than the taps, steps of single tokens (the kept inputs then move on in the same
    launch), a sequence that takes over another one's slot."""
    g = torch.Generator().manual_seed(taps + n)
    dt = torch.float32 if f32 else torch.bfloat16
    C = 2 * K * n + H * p
    conv = torch.randn(C, taps, generator=g)
    seqs = {k: torch.randn(t, C + H + 3 + low, generator=g) for k, t in (("a", 40), ("b", 12), ("c", 4))}
    seqs["a"][7, :C] *= 1e-3           # a token whose short vectors the constant under the root decides
    cache = make_cache(kv={0: (1, 8, 8)}, state={0: {"conv": (taps - 1, C)}}, slots=2)
    got = {k: [] for k in seqs}
    wt = conv.t().contiguous().to(DEV)

    def run(st, where):
        proj = gather(seqs, where)
        out, beta = torch.empty(st.tokens, C, device=DEV), torch.empty(st.tokens, H, device=DEV)
        lo = torch.empty(st.tokens, low, dtype=dt, device=DEV)
        ops.delta_prep(proj, cache.states[0]["conv"], wt, out, beta, lo, st, K, n, H, p, C, C + H + 3, 1e-6)
        assert torch.equal(lo, proj[:, C + H + 3:].to(dt))
        scatter(got, torch.cat([out, beta], 1), where)

    feed(cache, [[("a", 5), ("b", 1)], [("a", 1), ("b", 1)], [("a", 1), ("b", 1)], [("b", 1), ("a", 1)], [("a", 2), ("b", 3)],
                 [("a", 30), ("b", 5)]], run)
    cache.free("b")
    feed(cache, [[("c", 1)], [("c", 1)], [("c", 2)]], run)   # takes b's slot
    for k, x in seqs.items():
        out = torch.cat(got[k])
        n_seen = out.shape[0]
        want = delta_reference_prep(x[:n_seen, :C].double(), conv.double(), K, n, H, p)
        assert (out[:, :C] - want).abs().max().item() < 2e-5, k
        assert (out[:, C:] - torch.sigmoid(x[:n_seen, C:C + H].double())).abs().max().item() < 1e-6


def delta_inputs(T, K, H, n, p, seed=0, spread=3.0):
    g = torch.Generator().manual_seed(seed)
    q = ref.unit_vector(torch.randn(T, K, n, generator=g)) * n ** -0.5
    k = ref.unit_vector(torch.randn(T, K, n, generator=g) + 0.7 * torch.randn(1, K, n, generator=g))    # keys that overlap
    d = dict(qkv=torch.cat([q.reshape(T, -1), k.reshape(T, -1), torch.randn(T, H * p, generator=g)], 1),
             a=spread * torch.randn(T, H * n, generator=g) - spread, z=2 * torch.randn(T, H * p, generator=g),
             beta=torch.sigmoid(2 * torch.randn(T, H, generator=g)))
    par = dict(dt_bias=torch.randn(H * n, generator=g), a_log=torch.randn(H, generator=g), norm=1 + 0.3 * torch.randn(p, generator=g))
    return d, par


def delta_want(d, par, K, H, n, p, eps):
    T = d["a"].shape[0]
    x = d["qkv"].double()
    src = [h // (H // K) for h in range(H)]
    gate = ref.channel_decay(d["a"].double(), par["dt_bias"].double(), par["a_log"].double(), H)
    o, S = ref.delta_rule(x[:, :K * n].view(T, K, n)[:, src], x[:, K * n:2 * K * n].view(T, K, n)[:, src],
                          x[:, 2 * K * n:].view(T, H, p), gate, d["beta"].double(), torch.zeros(H, n, p, dtype=torch.float64))
    y = ref.rms_unit(o, eps) * par["norm"].double() * torch.sigmoid(d["z"].double()).view(T, H, p)
    return y.reshape(T, H * p), S


def run_delta(ops, seqs, par, plan, K, H, n, p, eps, f32=True, chunked=True, cache=None):
    cache = cache or make_cache(kv={0: (1, 8, 8)}, state={0: {"S": (H, n, p)}}, slots=3)
    dev = {k: v.to(DEV) for k, v in par.items()}
    got = {k: [] for k in seqs}

    def run(st, where):
        t = {name: gather({k: s[name] for k, s in seqs.items()}, where) for name in ("qkv", "a", "z", "beta")}
        az = torch.cat([t["a"], t["z"]], 1)
        out = torch.empty(st.tokens, H * p, dtype=torch.float32 if f32 else torch.bfloat16, device=DEV)
        ops.delta_rule(t["qkv"], az[:, :H * n], az[:, H * n:], t["beta"], dev["dt_bias"], dev["a_log"], dev["norm"],
                       cache.states[0]["S"], out, st, K, H, n, p, eps, chunked=chunked)
        scatter(got, out, where)

    feed(cache, plan, run)
    states = {k: cache.states[0]["S"][cache.slot_of(k)].cpu().double() for k in seqs if cache.has(k)}
    return {k: torch.cat(v) for k, v in got.items() if v}, states


SHAPES = [(2, 4, 40, 56), (1, 1, 128, 128), (3, 3, 16, 8), (1, 2, 150, 100), (2, 2, 64, 200), (1, 3, 20, 30), (1, 1, 300, 24), (1, 1, 4, 1)]


@pytest.mark.parametrize("K,H,n,p", SHAPES)
def test_delta_rule_over_steps(ops, K, H, n, p):
    """Whole prompts, portions and single tokens of unequal rows, both forms; outputs and the state they leave."""
    eps = 1e-5
    lens = {"a": 210, "b": 33, "c": 5}
    data = {k: delta_inputs(t, K, H, n, p, seed=i) for i, (k, t) in enumerate(lens.items())}
    seqs, par = {k: d for k, (d, _) in data.items()}, data["a"][1]
    plans = ([[("a", 210), ("b", 33), ("c", 5)]],
             [[("a", 64), ("b", 2)], [("b", 30), ("a", 65), ("c", 1)], [("a", 1), ("b", 1), ("c", 4)], [("a", 17)], [("a", 63)]],
             [[("c", 5), ("a", 190), ("b", 17)]] + [[("a", 1), ("b", 1)]] * 16 + [[("a", 4)]])
    for plan in plans:
        for chunked in (True, False):
            got, states = run_delta(ops, seqs, par, plan, K, H, n, p, eps, chunked=chunked)
            for k in seqs:
                want, S = delta_want(seqs[k], par, K, H, n, p, eps)
                assert got[k].shape == want.shape
                assert (got[k] - want).abs().max().item() < 1e-4 * max(1.0, want.abs().max().item()), (k, chunked)
                assert (states[k] - S).abs().max().item() < 2e-5 * max(1.0, S.abs().max().item()), (k, chunked)
    got16, _ = run_delta(ops, seqs, par, plans[0], K, H, n, p, eps, f32=False)
    want, _ = delta_want(seqs["a"], par, K, H, n, p, eps)
    assert (got16["a"] - want).abs().max().item() < 1e-2 * max(1.0, want.abs().max().item())


@pytest.mark.parametrize("chunked", [True, False])
def test_delta_rule_with_gates_at_their_ends(ops, chunked):
    """Gate inputs from far below to far above: gates of exactly one beside gates that underflow to zero, in every mixture
    within a block and a chunk.  Quotients of their products would overflow; the two forms may not."""
    K, H, n, p, eps = 1, 2, 48, 32, 1e-5
    d, par = delta_inputs(200, K, H, n, p, seed=7)
    g = torch.Generator().manual_seed(8)
    d["a"] = torch.tensor([-300.0, -20.0, 0.0, 5.0, 60.0, 500.0])[torch.randint(0, 6, (200, H * n), generator=g)]
    d["a"][60:140] = torch.where(torch.rand(80, H * n, generator=g) < 0.97, torch.tensor(-300.0), torch.tensor(200.0))
    par["a_log"] = torch.tensor([1.5, -0.5])
    want, S = delta_want(d, par, K, H, n, p, eps)
    for plan in ([[("a", 200)]], [[("a", 100)], [("a", 3)], [("a", 97)]]):
        got, states = run_delta(ops, {"a": d}, par, plan, K, H, n, p, eps, chunked=chunked)
        assert bool(torch.isfinite(got["a"]).all())
        assert (got["a"] - want).abs().max().item() < 2e-4 * max(1.0, want.abs().max().item())
        assert (states["a"] - S).abs().max().item() < 2e-5


@pytest.mark.parametrize("chunked", [True, False])
def test_an_early_write_is_read_hundreds_of_tokens_later(ops, chunked):
    """Gates of one, one key direction written once at a chosen place (the first token, a block's and a chunk's edges) and
    left alone by all other keys: a query along it hundreds of tokens later returns that value; written again, the new one."""
    K = H = 1
    n, p, T, eps = 32, 16, 400, 1e-6
    for mark in (0, 1, 15, 16, 63, 64, 127):
        d, par = delta_inputs(T, K, H, n, p, seed=mark)
        d["a"].fill_(-400.0)
        d["z"].fill_(30.0)
        d["beta"].fill_(1.0)
        par["norm"].fill_(1.0)
        q, k, v = d["qkv"][:, :n], d["qkv"][:, n:2 * n], d["qkv"][:, 2 * n:]
        q[:, 0] = k[:, 0] = 0.0
        for i in (mark, 350):
            k[i] = 0.0
            k[i, 0] = 1.0
        for i in (340, 380):
            q[i] = 0.0
            q[i, 0] = 1.0
        got, _ = run_delta(ops, {"a": d}, par, [[("a", 200)], [("a", 1)], [("a", 199)]], K, H, n, p, eps, chunked=chunked)
        assert (got["a"][340] - ref.rms_unit(v[mark].double(), eps)).abs().max().item() < 1e-4, mark
        assert (got["a"][380] - ref.rms_unit(v[350].double(), eps)).abs().max().item() < 1e-4, mark
        want, _ = delta_want(d, par, K, H, n, p, eps)
        assert (got["a"] - want).abs().max().item() < 2e-4 * want.abs().max().item()


def test_delta_rule_slots_used_again(ops):
    K, H, n, p, eps = 1, 2, 24, 40, 1e-5
    a, par = delta_inputs(90, K, H, n, p, seed=1)
    b, _ = delta_inputs(70, K, H, n, p, seed=2)
    cache = make_cache(kv={0: (1, 8, 8)}, state={0: {"S": (H, n, p)}}, slots=1)
    run_delta(ops, {"a": a}, par, [[("a", 90)]], K, H, n, p, eps, cache=cache)
    for first in (1, 17, 64):
        for k in list(cache._slot):
            cache.free(k)
        got, _ = run_delta(ops, {"b": b}, par, [[("b", first)], [("b", 70 - first)]], K, H, n, p, eps, cache=cache)
        assert (got["b"] - delta_want(b, par, K, H, n, p, eps)[0]).abs().max().item() < 1e-4


def test_arguments_outside_the_kernels_limits_are_refused(ops):
    K, H, n, p = 1, 1, 16, 300                                # wider than a workgroup's columns
    d, par = delta_inputs(4, K, H, n, p)
    with pytest.raises(AssertionError):
        run_delta(ops, {"a": d}, par, [[("a", 4)]], K, H, n, p, 1e-5)
    with pytest.raises(AssertionError):
        run_delta(ops, {"a": delta_inputs(4, 2, 3, 16, 8)[0]}, delta_inputs(4, 2, 3, 16, 8)[1], [[("a", 4)]], 2, 3, 16, 8, 1e-5)
