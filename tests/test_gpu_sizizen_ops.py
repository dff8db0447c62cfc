"""Each mechanism the Sizizen stack adds to the ragged family alone: the HIP kernel against the plain restatement in
oracle/ref_sizizen.py (fp64 on the CPU), on random inputs and on inputs built so that a fault shows (a key made dominant
on either side of a chunk's edge and at page borders, a memory that must hold one early write over hundreds of tokens,
gates of exactly zero and one, rows with a mean far from zero, a best expert inside a dropped group, pages and slots
dirtied before use)."""
import pytest
import torch

from oracle import ref_sizizen as ref

pytestmark = pytest.mark.gpu
DEV = "cuda"


@pytest.fixture(scope="module")
def ops():
    import micro_vllm_amd  # noqa: F401
    from micro_vllm_amd.kernel import ragged_ops
    return ragged_ops


def make_cache(kv=None, state=None, pages=16, slots=3, dtype=torch.float32, page=64, max_tokens=1024, step_tokens=1024):
    from micro_vllm_amd.core.state_cache import HybridCacheManager
    cache = HybridCacheManager(pages, page, slots, kv or {}, state or {}, dtype=dtype, device=DEV, max_tokens=max_tokens,
                               max_rows=4, max_step_tokens=step_tokens)
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


# ----------------------------------------------------------------------------------------------- layer norm on outputs
@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("n", [203, 96, 1500, 3072, 5000, 9000, 7001])
@pytest.mark.parametrize("T", [5, 600])
def test_layer_norm_residual_step(ops, f32, n, T):
    """Every width takes another form of the kernel (odd ones value by value), few rows more threads than many.  A mean far
    from zero: the variance is that of the deviations, not a difference of large squares."""
    g = torch.Generator().manual_seed(n + T)
    dt = torch.float32 if f32 else torch.bfloat16
    tol, eps = (2e-5 if f32 else 5e-2), 1e-5
    T = T if n < 2000 else min(T, 520)
    x0, y, z = torch.randn(T, n, generator=g), torch.randn(T, n, generator=g) + 30.0, torch.randn(T, n, generator=g)
    w, w2, r1, r2 = (1 + 0.3 * torch.randn(n, generator=g) for _ in range(4))
    D = lambda t: t.double()   # noqa: E731
    d = lambda t: t.to(DEV)    # noqa: E731
    want = D(x0) + ref.layer_norm(D(y), D(w), eps)
    x, h = d(x0).clone(), torch.empty(T, n, dtype=dt, device=DEV)
    ops.layernorm_residual(x, d(y), d(w), eps, h)
    assert (x.cpu().double() - want).abs().max().item() < 3e-5 and torch.equal(h, x.to(dt))
    # the next norm out of the same launch; operands that are column slices of wider buffers
    wide = torch.zeros(T, 2 * n + 4, device=DEV)
    wide[:, 4:4 + n] = d(y)
    x = d(x0).clone()
    ops.layernorm_residual(x, wide[:, 4:4 + n], d(w), eps, h, next_w=d(w2))
    assert (x.cpu().double() - want).abs().max().item() < 3e-5
    assert (h.float().cpu().double() - ref.layer_norm(want, D(w2), eps)).abs().max().item() < tol
    # two branches, each normed over the width first
    v = 0.5 * (ref.rms_norm(D(y), D(r1), eps) + ref.rms_norm(D(z), D(r2), eps))
    want = D(x0) + ref.layer_norm(v, D(w), eps)
    for slot in (None, h):                 # with and without a copy in the activation type
        x = d(x0).clone()
        ops.layernorm_residual(x, d(y), d(w), eps, slot, branch=(d(r1), d(z), d(r2), 0.5))
        assert (x.cpu().double() - want).abs().max().item() < 5e-5
    assert torch.equal(h, x.to(dt))
    # the weighted sum of a token's expert rows, which lie anywhere, beside a shared row
    for top in (1, 4, 6):
        place = torch.randperm(T * top, generator=g).to(torch.int32)
        wts, rows = torch.rand(T, top, generator=g), torch.randn(T * top, n, generator=g) + 2.0
        v = (rows.double()[place.long()].view(T, top, n) * wts.double()[..., None]).sum(1)
        for shared in (None, z):
            full = v if shared is None else v + D(shared)
            want = D(x0) + ref.layer_norm(full, D(w), eps)
            x = d(x0).clone()
            ops.layernorm_residual(x, d(rows), d(w), eps, h, place=d(place), weights=d(wts), shared=None if shared is None else d(shared),
                                   next_w=d(w2))
            assert (x.cpu().double() - want).abs().max().item() < 3e-5
            assert (h.float().cpu().double() - ref.layer_norm(want, D(w2), eps)).abs().max().item() < tol
        if n > 4000:
            break


@pytest.mark.parametrize("f32", [False, True])
def test_layer_norm_of_chosen_rows_with_small_values(ops, f32):
    """Rows so small that the constant under the root decides, and a constant row."""
    g = torch.Generator().manual_seed(3)
    x, w = torch.randn(9, 150, generator=g) * 2, torch.randn(150, generator=g)
    x[4] *= 1e-3
    x[5] = 7.0
    out = torch.empty(4, 150, dtype=torch.float32 if f32 else torch.bfloat16, device=DEV)
    idx = torch.tensor([4, 0, 8, 5], dtype=torch.int32)
    ops.layernorm_gather(x.to(DEV), idx.to(DEV), w.to(DEV), 1e-5, out)
    want = ref.layer_norm(x.double()[idx.long()], w.double(), 1e-5)
    assert (out.float().cpu().double() - want).abs().max().item() < (2e-5 if f32 else 5e-2)
    out = torch.empty(9, 150, dtype=out.dtype, device=DEV)
    ops.layernorm_gather(x.to(DEV), None, w.to(DEV), 1e-5, out)
    assert (out.float().cpu().double() - ref.layer_norm(x.double(), w.double(), 1e-5)).abs().max().item() < (2e-5 if f32 else 5e-2)


@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("n", [64, 150, 333])
def test_squared_relu_aligned_and_not(ops, f32, n):
    v = torch.randn(7, n + 5, generator=torch.Generator().manual_seed(n)).to(DEV)
    for src in (v[:, :n], v[:, 1:n + 1], v[:, :n].contiguous()):
        out = torch.empty(7, n, dtype=torch.float32 if f32 else torch.bfloat16, device=DEV)
        ops.relu_squared(src, out)
        assert torch.equal(out, (src.clamp(min=0) ** 2).to(out.dtype))


# ----------------------------------------------------------------------------------------------- attention
@pytest.mark.parametrize("H,G,d,dv,rot,normed,low", [(6, 2, 40, 24, 24, True, 37), (2, 2, 64, 64, 64, True, 64), (1, 1, 10, 130, 0, True, 0),
                                                     (4, 1, 96, 8, 2, False, 1), (16, 4, 128, 128, 128, True, 128),
                                                     (3, 1, 200, 16, 30, True, 5), (2, 1, 400, 16, 400, True, 0)])
@pytest.mark.parametrize("f32", [False, True])
def test_norm_per_head_rotation_keys_and_values_into_pages(ops, H, G, d, dv, rot, normed, low, f32):
    """Steps of few tokens (a wave per head) and of many (eight heads a wave), rows dirtied beforehand, one head far larger
    than the others (a norm over more than the head would show it)."""
    g = torch.Generator().manual_seed(d + rot)
    dt = torch.float32 if f32 else torch.bfloat16
    cq, ck, cv, eps, base = H * d, G * d, G * dv, 1e-5, 90.0
    C = cq + ck + cv
    lens = {"a": 460, "b": 9}
    raw = {k: 2 * torch.randn(n, C + low, generator=g) for k, n in lens.items()}
    for x in raw.values():
        x[:, :d] *= 50.0
    qb, kb, vb = (torch.randn(n, generator=g) for n in (cq, ck, cv))
    qn, kn = 1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)
    inv = (base ** (-2.0 * torch.arange(rot // 2, dtype=torch.float64) / max(rot, 1))).to(DEV) if rot else None
    cache = make_cache(kv={0: (G, d, dv)}, dtype=dt)
    got = {k: [] for k in lens}

    def run(st, where):
        buf = torch.zeros(st.tokens, C + low + 5, device=DEV)
        buf[:, :C + low] = gather(raw, where)
        before = buf.clone()
        lo = torch.empty(st.tokens, low, dtype=dt, device=DEV) if low else None
        args = dict(q_bias=qb.to(DEV), k_bias=kb.to(DEV), v_bias=vb.to(DEV))
        if normed:
            args.update(q_norm=qn.to(DEV), k_norm=kn.to(DEV))
        ops.qkv_headnorm_rotary_store(buf[:, :C], cache.k_caches[0], cache.v_caches[0], st, H, G, d, dv, inv, rot, eps,
                                      low=buf[:, C:C + low] if low else None, low_out=lo, **args)
        scatter(got, buf[:, :cq], where)
        assert torch.equal(buf[:, cq:], before[:, cq:])
        if low:
            assert torch.equal(lo, buf[:, C:C + low].to(dt))

    feed(cache, [[("a", 70), ("b", 1)], [("b", 2), ("a", 1)], [("a", 389), ("b", 6)]], run)
    for k, n in lens.items():
        x = raw[k].double()
        q, kk, v = x[:, :cq] + qb.double(), x[:, cq:cq + ck] + kb.double(), x[:, cq + ck:C] + vb.double()
        q, kk = q.view(n, H, d), kk.view(n, G, d)
        if normed:
            q, kk = ref.rms_norm(q, qn.double(), eps), ref.rms_norm(kk, kn.double(), eps)
        if rot:
            q, kk = ref.rotate_halves(q, rot, base), ref.rotate_halves(kk, rot, base)
        q, kk = q.reshape(n, cq), kk.reshape(n, ck)
        scale = q.abs().max().item()
        assert (torch.cat(got[k]) - q).abs().max().item() < 3e-6 * max(scale, 10.0), k
        pages = cache.get_blocks(k)
        rows = torch.tensor([pages[i // 64] * 64 + i % 64 for i in range(n)])
        tol = 3e-5 if f32 else 0.02 * max(kk.abs().max().item(), v.abs().max().item())
        assert (cache.k_caches[0].view(-1, ck).float().cpu()[rows].double() - kk).abs().max().item() < tol
        assert (cache.v_caches[0].view(-1, cv).float().cpu()[rows].double() - v).abs().max().item() < tol


def test_rotation_with_adjacent_pairs_equals_halves_of_shuffled_dimensions(ops):
    g = torch.Generator().manual_seed(1)
    H, d, dv, rot = 2, 24, 8, 16
    raw = torch.randn(30, 3 * d + dv, generator=g)
    inv = (50.0 ** (-2.0 * torch.arange(8, dtype=torch.float64) / 16)).to(DEV)
    perm = torch.cat([torch.arange(0, 16, 2), torch.arange(1, 16, 2), torch.arange(16, 24)])
    cache = make_cache(kv={0: (1, d, dv)})
    a = raw.to(DEV)
    ops.qkv_headnorm_rotary_store(a, cache.k_caches[0], cache.v_caches[0], step_of(cache, [("a", [0] * 30)]), H, 1, d, dv, inv, rot, 1e-5,
                                  adjacent=True)
    b = raw.clone()
    b[:, :3 * d] = raw[:, :3 * d].view(30, 3, d)[:, :, perm].reshape(30, -1)
    b = b.to(DEV)
    ops.qkv_headnorm_rotary_store(b, cache.k_caches[0], cache.v_caches[0], step_of(cache, [("b", [0] * 30)]), H, 1, d, dv, inv, rot, 1e-5)
    assert torch.equal(a[:, :2 * d].view(30, 2, d)[:, :, perm.to(DEV)], b[:, :2 * d].view(30, 2, d))


def test_angles_far_from_the_start(ops):
    """Positions of hundreds of thousands: the angle is formed in fp64, so that the pair turns by what its position says."""
    import types
    d, rot, T = 8, 8, 3
    pos = torch.tensor([0, 99991, 777777], dtype=torch.int32)
    raw = torch.randn(T, 3 * d, generator=torch.Generator().manual_seed(2))
    inv = (10.0 ** (-2.0 * torch.arange(4, dtype=torch.float64) / 8))
    kc = torch.zeros(1, 64, 1, d, device=DEV)
    st = types.SimpleNamespace(tokens=T, page=64, max_page=0, tok_row=torch.arange(T, dtype=torch.int32, device=DEV), tok_pos=pos.to(DEV),
                               block_table=torch.full((T, 777777 // 64 + 1), 0, dtype=torch.int32, device=DEV))
    buf = raw.to(DEV)
    ops.qkv_headnorm_rotary_store(buf, kc, kc.clone(), st, 1, 1, d, d, inv.to(DEV), rot, 1e-5)
    a = pos.double()[:, None] * inv
    u, v = raw[:, :4].double(), raw[:, 4:8].double()
    want = torch.cat([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()], 1)
    assert (buf[:, :d].cpu().double() - want).abs().max().item() < 2e-6


def attend(ops, q, k, v, H, G, d, dv, scale, chunk, portions, f32=True, tiled=True, grouped=False, splits=None):
    """Whole rows q | k | v fed in portions through the page store and the attention within chunks."""
    dt = torch.float32 if f32 else torch.bfloat16
    cache = make_cache(kv={0: (G, d, dv)}, dtype=dt, pages=24, max_tokens=1536)
    T = q.shape[0]
    rows = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1).float()
    out, pos = [], 0
    for n in portions:
        st = step_of(cache, [("s", [0] * n)])
        buf = rows[pos:pos + n].to(DEV).contiguous()
        ops.qkv_headnorm_rotary_store(buf, cache.k_caches[0], cache.v_caches[0], st, H, G, d, dv, None, 0, 1e-6)
        o = torch.empty(n, H * dv, dtype=dt, device=DEV)
        part, sp = None, 0
        if grouped:
            sp = splits or ops.window_attn_splits(n, H, G, chunk)
            part = torch.empty(n * H * sp * (dv + 2), device=DEV)
        ops.window_attn(buf[:, :H * d], cache.k_caches[0], cache.v_caches[0], o, st, None, H, G, d, dv, scale, chunk, tiled=tiled,
                        part=part, splits=sp, chunked=True)
        out.append(o.float().cpu())
        pos += n
    return torch.cat(out)


@pytest.mark.parametrize("H,G,d,dv,chunk", [(6, 2, 40, 24, 37), (4, 1, 64, 64, 65), (2, 2, 128, 64, 300), (9, 1, 32, 32, 64), (6, 2, 64, 32, 64),
                                            (2, 1, 64, 32, 100), (3, 3, 8, 8, 1), (2, 1, 96, 96, 17)])
def test_attention_within_chunks(ops, H, G, d, dv, chunk):
    """All four forms (one workgroup per head, shared reads, shared reads cut into pieces, matrix cores), whole prompts,
    portions cut inside chunks, and decoding."""
    g = torch.Generator().manual_seed(d + chunk)
    T, scale = 210, 0.2
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, G, d, generator=g), torch.randn(T, G, dv, generator=g)
    want = ref.chunked_attention(q.double(), k.double(), v.double(), scale, chunk).reshape(T, -1)
    args = (ops, q, k, v, H, G, d, dv, scale, chunk)
    for portions in ([T], [3, 61, 2, 63, 1, 80], [150] + [1] * 60):
        for kw in (dict(), dict(grouped=True), dict(grouped=True, splits=3)):
            assert (attend(*args, portions, **kw).double() - want).abs().max().item() < 1e-4, (portions[:3], kw)
            assert (attend(*args, portions, f32=False, **kw).double() - want).abs().max().item() < 0.06, (portions[:3], kw)
        assert (attend(*args, portions, f32=False, tiled=False).double() - want).abs().max().item() < 0.06


@pytest.mark.parametrize("chunk", [16, 64, 65, 71, 192])
@pytest.mark.parametrize("decode,f32,grouped", [(False, True, False), (True, True, True), (True, False, True), (False, False, False),
                                                 (True, True, False)])
def test_chunk_edge_with_a_dominant_key(ops, chunk, decode, f32, grouped):
    """One key wins the softmax wherever it is visible and carries a value of its own: every query from it to its chunk's
    last position returns it, the next chunk's first does not - for the first and the last position of the first chunk,
    of a later one, and at page borders."""
    H = G = 1
    d = dv = 32
    T = 3 * chunk + 70
    g = torch.Generator().manual_seed(chunk)
    q, k, v = torch.randn(T, H, d, generator=g) * 0.01, torch.randn(T, G, d, generator=g) * 0.01, torch.zeros(T, G, dv)
    marks = (0, chunk - 1, chunk, 2 * chunk - 1, 63, 64, 2 * chunk + 1)
    for n, mark in enumerate(marks):
        k[mark, 0] = 0
        for m, other in enumerate(marks):
            if other == mark:              # positions that coincide share a key
                k[mark, 0, m] = 1.0
        v[mark, 0, 0] = 100.0 + mark
    portions = [chunk // 2, 2] + [1] * (T - chunk // 2 - 2) if decode else [T]
    for n, mark in enumerate(marks):
        end = mark // chunk * chunk + chunk - 1
        qq = q.clone()
        for i in {mark, (mark + end) // 2, end, end + 1}:
            qq[i, 0] = 0
            qq[i, 0, n] = 1.0
        out = attend(ops, qq, k, v, H, G, d, dv, 40.0, chunk, portions, f32=f32, grouped=grouped)
        for i in (mark, (mark + end) // 2, end):
            assert abs(out[i, 0].item() - (100.0 + mark)) < (1.0 if f32 else 2.5), (mark, i)
        assert abs(out[end + 1, 0].item() - (100.0 + mark)) > 40.0 or (end + 1) in marks, mark
        want = ref.chunked_attention(qq.double(), k.double(), v.double(), 40.0, chunk).reshape(T, -1)
        assert (out.double() - want).abs().max().item() < (1e-3 if f32 else 2.5)


# ----------------------------------------------------------------------------------------------- gated linear attention
def memory_inputs(T, H, n, p, seed=0, spread=3.0):
    g = torch.Generator().manual_seed(seed)
    d = dict(q=torch.randn(T, H * n, generator=g), k=torch.randn(T, H * n, generator=g), v=torch.randn(T, H * p, generator=g),
             z=spread * torch.randn(T, H * n, generator=g), g=2 * torch.randn(T, H * p, generator=g))
    par = dict(bias=torch.randn(H * n, generator=g), norm=1 + 0.3 * torch.randn(p, generator=g))
    return d, par


def memory_want(d, par, H, n, p, tau, eps, q_scale):
    T = d["q"].shape[0]
    x = {k: t.double() for k, t in d.items()}
    alpha = ref.channel_decay(x["z"] + par["bias"].double(), tau).view(T, H, n)
    o, S = ref.gated_linear_attention(q_scale * x["q"].view(T, H, n), x["k"].view(T, H, n), x["v"].view(T, H, p), alpha,
                                      torch.zeros(H, n, p, dtype=torch.float64))
    y = ref.rms_norm(o, par["norm"].double(), eps).reshape(T, H * p) * ref.silu(x["g"])
    return y, S


def run_memory(ops, seqs, par, plan, H, n, p, tau, eps, q_scale, f32=True, chunked=True, cache=None, shift=0):
    """`shift`: the projections' columns start that many floats into their rows (what the 16-byte reads cannot take)."""
    cache = cache or make_cache(kv={0: (1, 8, 8)}, state={0: {"S": (H, n, p)}}, slots=3)
    dev = {k: v.to(DEV) for k, v in par.items()}
    got = {k: [] for k in seqs}

    def run(st, where):
        t = {name: gather({k: s[name] for k, s in seqs.items()}, where) for name in ("q", "k", "v", "z", "g")}
        buf = torch.cat([torch.full((st.tokens, shift), 5.0, device=DEV), t["q"], t["k"], t["v"], t["g"]], 1)
        a, b, c = shift + H * n, shift + 2 * H * n, shift + 2 * H * n + H * p
        out = torch.empty(st.tokens, H * p, dtype=torch.float32 if f32 else torch.bfloat16, device=DEV)
        ops.gated_linear_attn(buf[:, shift:a], buf[:, a:b], buf[:, b:c], t["z"], dev["bias"], buf[:, c:], dev["norm"],
                              cache.states[0]["S"], out, st, H, n, p, tau, eps, q_scale=q_scale, chunked=chunked)
        scatter(got, out, where)

    feed(cache, plan, run)
    states = {k: cache.states[0]["S"][cache.slot_of(k)].cpu().double() for k in seqs if cache.has(k)}
    return {k: torch.cat(v) for k, v in got.items() if v}, states


SHAPES = [(4, 40, 56, 3.0, 0), (1, 128, 128, 16.0, 0), (3, 16, 8, 1.0, 1), (2, 150, 100, 0.5, 0), (2, 64, 200, 7.0, 0), (3, 18, 34, 2.0, 3),
          (1, 300, 24, 4.0, 0), (1, 4, 1, 1.0, 0), (1, 256, 256, 16.0, 0), (1, 33, 129, 5.0, 0)]


@pytest.mark.parametrize("H,n,p,tau,shift", SHAPES)
def test_gated_linear_attention_over_steps(ops, H, n, p, tau, shift):
    """Whole prompts, portions and single tokens of unequal rows, both forms; outputs and the state they leave."""
    eps, qs = 1e-5, n ** -0.5
    lens = {"a": 210, "b": 33, "c": 5}
    data = {k: memory_inputs(t, H, n, p, seed=i) for i, (k, t) in enumerate(lens.items())}
    seqs, par = {k: d for k, (d, _) in data.items()}, data["a"][1]
    wants = {k: memory_want(seqs[k], par, H, n, p, tau, eps, qs) for k in seqs}
    plans = ([[("a", 210), ("b", 33), ("c", 5)]],
             [[("a", 64), ("b", 2)], [("b", 30), ("a", 65), ("c", 1)], [("a", 1), ("b", 1), ("c", 4)], [("a", 17)], [("a", 63)]],
             [[("c", 5), ("a", 190), ("b", 17)]] + [[("a", 1), ("b", 1)]] * 16 + [[("a", 4)]])
    for plan in plans:
        for chunked in (True, False):
            got, states = run_memory(ops, seqs, par, plan, H, n, p, tau, eps, qs, chunked=chunked, shift=shift)
            for k, (want, S) in wants.items():
                assert got[k].shape == want.shape
                assert (got[k] - want).abs().max().item() < 1e-4 * max(1.0, want.abs().max().item()), (k, chunked)
                assert (states[k] - S).abs().max().item() < 2e-5 * max(1.0, S.abs().max().item()), (k, chunked)
    got16, _ = run_memory(ops, seqs, par, plans[0], H, n, p, tau, eps, qs, f32=False, shift=shift)
    want = wants["a"][0]
    assert (got16["a"] - want).abs().max().item() < 1e-2 * max(1.0, want.abs().max().item())


@pytest.mark.parametrize("chunked", [True, False])
def test_gates_at_their_ends(ops, chunked):
    """Decay logits from far below to far above: gates of exactly one beside gates that underflow to zero, in every mixture
    within a block and a chunk.  Quotients of their products would overflow; neither form may."""
    H, n, p, eps, tau = 2, 48, 32, 1e-5, 1.5
    d, par = memory_inputs(200, H, n, p, seed=7)
    g = torch.Generator().manual_seed(8)
    d["z"] = torch.tensor([400.0, 20.0, 0.0, -5.0, -90.0, -700.0])[torch.randint(0, 6, (200, H * n), generator=g)]
    d["z"][60:140] = torch.where(torch.rand(80, H * n, generator=g) < 0.97, torch.tensor(400.0), torch.tensor(-300.0))
    want, S = memory_want(d, par, H, n, p, tau, eps, 1.0)
    for plan in ([[("a", 200)]], [[("a", 100)], [("a", 3)], [("a", 97)]]):
        got, states = run_memory(ops, {"a": d}, par, plan, H, n, p, tau, eps, 1.0, chunked=chunked)
        assert bool(torch.isfinite(got["a"]).all())
        assert (got["a"] - want).abs().max().item() < 2e-4 * max(1.0, want.abs().max().item())
        assert (states["a"] - S).abs().max().item() < 2e-5 * max(1.0, S.abs().max().item())


@pytest.mark.parametrize("chunked", [True, False])
def test_gates_next_to_one_over_a_long_row(ops, chunked):
    """Gates of 1 - 1e-4 and nearer, hundreds of tokens: an error of the gate itself would be raised to that power."""
    H, n, p, eps = 1, 32, 16, 1e-6
    d, par = memory_inputs(900, H, n, p, seed=11, spread=1.0)
    d["z"] = d["z"] + 6.0
    par["bias"] = par["bias"] * 0.1
    want, S = memory_want(d, par, H, n, p, 16.0, eps, 0.3)
    got, states = run_memory(ops, {"a": d}, par, [[("a", 700)], [("a", 2)], [("a", 198)]], H, n, p, 16.0, eps, 0.3, chunked=chunked)
    assert (states["a"] - S).abs().max().item() < 2e-5 * S.abs().max().item()
    assert (got["a"] - want).abs().max().item() < 1e-4 * want.abs().max().item()


@pytest.mark.parametrize("chunked", [True, False])
def test_an_early_write_is_read_hundreds_of_tokens_later(ops, chunked):
    """Gates of one, one key direction written once at a chosen place (the first token, a block's and a chunk's edges) and
    left alone by all other keys: a query along it hundreds of tokens later returns that value; written again, the sum."""
    H, n, p, T, eps = 1, 32, 16, 400, 1e-6
    for mark in (0, 1, 15, 16, 63, 64, 127):
        d, par = memory_inputs(T, H, n, p, seed=mark)
        d["z"].fill_(500.0)
        d["g"].fill_(30.0)
        par["norm"].fill_(1.0)
        d["q"][:, 0] = d["k"][:, 0] = 0.0
        for i in (mark, 350):
            d["k"][i] = 0.0
            d["k"][i, 0] = 1.0
        for i in (340, 380):
            d["q"][i] = 0.0
            d["q"][i, 0] = 1.0
        got, _ = run_memory(ops, {"a": d}, par, [[("a", 200)], [("a", 1)], [("a", 199)]], H, n, p, 1.0, eps, 1.0, chunked=chunked)
        one = torch.ones(p, dtype=torch.float64)
        v = d["v"].double()
        assert (got["a"][340] - 30.0 * ref.rms_norm(v[mark], one, eps)).abs().max().item() < 3e-3, mark
        assert (got["a"][380] - 30.0 * ref.rms_norm(v[mark] + v[350], one, eps)).abs().max().item() < 3e-3, mark
        want, _ = memory_want(d, par, H, n, p, 1.0, eps, 1.0)
        assert (got["a"] - want).abs().max().item() < 2e-4 * want.abs().max().item()


def test_slots_used_again(ops):
    H, n, p, eps = 2, 24, 40, 1e-5
    a, par = memory_inputs(90, H, n, p, seed=1)
    b, _ = memory_inputs(70, H, n, p, seed=2)
    cache = make_cache(kv={0: (1, 8, 8)}, state={0: {"S": (H, n, p)}}, slots=1)
    run_memory(ops, {"a": a}, par, [[("a", 90)]], H, n, p, 2.0, eps, 1.0, cache=cache)
    for first in (1, 17, 64):
        for k in list(cache._slot):
            cache.free(k)
        got, _ = run_memory(ops, {"b": b}, par, [[("b", first)], [("b", 70 - first)]], H, n, p, 2.0, eps, 1.0, cache=cache)
        assert (got["b"] - memory_want(b, par, H, n, p, 2.0, eps, 1.0)[0]).abs().max().item() < 1e-4


def test_arguments_outside_the_kernels_limits_are_refused(ops):
    for H, n, p in ((1, 16, 300), (1, 600, 8), (1, 512, 256)):
        d, par = memory_inputs(4, H, n, p)
        with pytest.raises(AssertionError):
            run_memory(ops, {"a": d}, par, [[("a", 4)]], H, n, p, 1.0, 1e-5, 1.0)
    h, w = torch.zeros(3, 8, device=DEV), torch.zeros(6, 8, device=DEV)
    ids, wts = torch.zeros(3, 4, dtype=torch.int32, device=DEV), torch.zeros(3, 4, device=DEV)
    for groups, keep in ((4, 1), (3, 1), (2, 3), (0, 1)):      # uneven groups, too few experts left, more kept than there are
        with pytest.raises(AssertionError):
            ops.moe_route_grouped(h, w, None, ids, wts, groups, keep)


# ----------------------------------------------------------------------------------------------- routed experts
@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("T,E,groups,keep,top,W", [(37, 12, 3, 2, 4, 96), (5, 8, 8, 2, 2, 40), (3, 6, 1, 1, 6, 33), (130, 40, 4, 1, 6, 96),
                                                   (9, 96, 12, 5, 16, 200), (2, 1, 1, 1, 1, 24), (1, 256, 8, 4, 8, 512), (83, 100, 10, 3, 8, 208),
                                                   (65, 16, 4, 2, 4, 1024), (70, 256, 8, 4, 8, 48), (66, 300, 3, 1, 5, 64)])
@pytest.mark.parametrize("corrected", [True, False])
def test_group_limited_choice(ops, f32, T, E, groups, keep, top, W, corrected):
    g = torch.Generator().manual_seed(E + top)
    h = torch.randn(T, W, generator=g).to(torch.float32 if f32 else torch.bfloat16)
    wr = torch.randn(E, W, generator=g) * W ** -0.5 * 1.5
    corr = torch.randn(E, generator=g) - 1.0 if corrected else None      # choice scores mostly below zero
    ids, wts = torch.empty(T, top, dtype=torch.int32, device=DEV), torch.empty(T, top, device=DEV)
    ops.moe_route_grouped(h.to(DEV), wr.to(DEV), None if corr is None else corr.to(DEV), ids, wts, groups, keep)
    for t in range(T):
        want = ref.route(h[t].double(), wr.double(), corr.double() if corrected else torch.zeros(E, dtype=torch.float64), groups, keep, top)
        assert ids[t].tolist() == [e for e, _ in want], t
        assert (wts[t].cpu().double() - torch.stack([s for _, s in want])).abs().max().item() < 1e-6


def test_best_expert_of_a_dropped_group_and_negative_scores(ops):
    """One group holds the best expert but is worth less than two even ones: it is out, although what is left to choose
    from scores below zero (a dropped expert counts as nothing, not as zero).  Equal scores go to the lower index."""
    E, groups, keep, top, W = 8, 4, 2, 4, 8
    corr = torch.tensor([-0.2, -1.9, -0.9, -0.95, -0.9, -0.9, -2.5, -2.5])      # scores are all 1/2
    h, wr = torch.zeros(3, W), torch.randn(E, W)
    ids, wts = torch.empty(3, top, dtype=torch.int32, device=DEV), torch.empty(3, top, device=DEV)
    ops.moe_route_grouped(h.to(DEV), wr.to(DEV), corr.to(DEV), ids, wts, groups, keep)
    assert ids.tolist() == [[2, 4, 5, 3]] * 3 and bool((wts == 0.5).all())


@pytest.mark.parametrize("f32", [False, True])
@pytest.mark.parametrize("T", [3, 37])
@pytest.mark.parametrize("shared", [0, 56])
def test_routed_squared_relu_experts(ops, f32, T, shared):
    g = torch.Generator().manual_seed(T)
    dt = torch.float32 if f32 else torch.bfloat16
    E, groups, keep, top, W, ff, eps = 12, 4, 2, 3, 96, 40, 1e-5
    h = torch.randn(T, W, generator=g).to(dt)
    Wt = {"router": torch.randn(E, W, generator=g) * 0.2, "correction": torch.randn(E, generator=g) * 0.4 - 0.3}
    for e in range(E):
        Wt[f"e{e}.up"] = torch.randn(ff, W, generator=g).to(dt).float() / W ** 0.5
        Wt[f"e{e}.down"] = torch.randn(W, ff, generator=g).to(dt).float() / ff ** 0.5
    if shared:
        Wt["shared.up"], Wt["shared.down"] = (torch.randn(a, b, generator=g).to(dt).float() / b ** 0.5 for a, b in ((shared, W), (W, shared)))
    mlp = {"router": {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}}, "shared": {"ff": shared} if shared else None}
    Wt = {k: (v.to(dt) if ".up" in k or ".down" in k else v) for k, v in Wt.items()}
    want = ref.moe_ff(h.double(), {k: v.double() for k, v in Wt.items()}, "", mlp)
    hd = h.to(DEV)
    ids, wts = torch.empty(T, top, dtype=torch.int32, device=DEV), torch.empty(T, top, device=DEV)
    ops.moe_route_grouped(hd, Wt["router"].to(DEV), Wt["correction"].to(DEV), ids, wts, groups, keep)
    seg, order, place = (torch.empty(c, dtype=torch.int32, device=DEV) for c in (E + 1, T * top, T * top))
    ops.moe_plan(ids, seg, order, place, E)
    up = ops.linear_segments(hd, torch.stack([Wt[f"e{e}.up"] for e in range(E)]).to(DEV), torch.empty(T * top, ff, device=DEV), seg, order,
                             top, T)
    act = torch.empty(T * top, ff, dtype=dt, device=DEV)
    ops.relu_squared(up, act)
    down = ops.linear_segments(act, torch.stack([Wt[f"e{e}.down"] for e in range(E)]).to(DEV), torch.empty(T * top, W, device=DEV), seg,
                               None, 1, T)
    s_out = None
    if shared:
        s_act = torch.empty(T, shared, dtype=dt, device=DEV)
        ops.relu_squared(ops.AnyLinear(Wt["shared.up"].to(DEV))(hd), s_act)
        s_out = ops.AnyLinear(Wt["shared.down"].to(DEV))(s_act)
    x0, w = torch.randn(T, W, generator=g), 1 + 0.2 * torch.randn(W, generator=g)
    x = x0.to(DEV)
    ops.layernorm_residual(x, down, w.to(DEV), eps, place=place, weights=wts, shared=s_out)
    want = x0.double() + ref.layer_norm(want, w.double(), eps)
    assert (x.cpu().double() - want).abs().max().item() < (3e-5 if f32 else 4e-2)
