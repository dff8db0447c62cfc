"""Plain, slow restatement of the Sizizen layer stack: one function per mechanism, whole sequences, loops over
tokens and heads.  Shares nothing with the product path; the tests compare the engine against it.  Everything
runs in `dtype` (float64 by default) on the CPU.

Weights come as a dict name -> tensor with the checkpoint's names ('l<i>.mix.left.q', ...), the configuration as
the parsed config.json dict.

Notation.  L_w = layer norm with weight w, no bias; R_w = RMS norm with weight w.  No norm in front of a sublayer,
one behind it:
    x <- x + L1( M(x) );   x <- x + L2( F(x) )
M runs softmax attention over chunks of positions ('left') beside gated linear attention ('right') on the same
input and returns (R_left(left) + R_right(right)) / 2; F is a SiLU-gated feed-forward, a group-limited mixture of
squared-ReLU experts, or nothing.
"""
import math

import torch


def layer_norm(x, w, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(x):
    return x * torch.sigmoid(x)


def rotate_halves(x, rot, base):
    """x [T, heads, d]: dimension i < rot / 2 is paired with i + rot / 2; angle position * base^(-2 i / rot)."""
    out = x.clone()
    half = rot // 2
    for t in range(x.shape[0]):
        for i in range(half):
            a = t * base ** (-2.0 * i / rot)
            c, s = math.cos(a), math.sin(a)
            out[t, :, i] = x[t, :, i] * c - x[t, :, i + half] * s
            out[t, :, i + half] = x[t, :, i + half] * c + x[t, :, i] * s
    return out


def chunked_attention(q, k, v, scale, size):
    """q [T, H, d], k [T, G, d], v [T, G, dv]: softmax over the keys from the start of the token's chunk of `size`
    positions to the token itself."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for hd in range(H):
        g = hd // (H // G)
        for i in range(T):
            lo = (i // size) * size
            s = (k[lo:i + 1, g] @ q[i, hd]) * scale
            e = torch.exp(s - s.max())
            out[i, hd] = (e / e.sum()) @ v[lo:i + 1, g]
    return out


def attention_mixer(h, W, p, m, eps):
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = rms_norm((h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, d), W[p + "q.norm"], eps)
    k = rms_norm((h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, d), W[p + "k.norm"], eps)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(T, G, dv)
    rot, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
    q, k = rotate_halves(q, rot, base), rotate_halves(k, rot, base)
    o = chunked_attention(q, k, v, float(m["scale"]), int(m["mask"]["size"]))
    return o.reshape(T, H * dv) @ W[p + "o"].T


def channel_decay(z, tau):
    """sigmoid(z)^(1 / tau), through the logarithm: log sigmoid(z) = min(z, 0) - log(1 + e^-|z|)."""
    return torch.exp((torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-torch.abs(z)))) / tau)


def gated_linear_attention(q, k, v, alpha, state=None):
    """q, k, alpha [T, H, n]; v [T, H, p] -> o [T, H, p].  Per head, S [n, p] from zero: decay the rows, add the
    outer product of key and value, read with the query."""
    T, H, n = q.shape
    S = torch.zeros(H, n, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = alpha[t, h][:, None] * S[h] + torch.outer(k[t, h], v[t, h])
            out[t, h] = q[t, h] @ S[h]
    return out if state is None else (out, S)


def linear_mixer(h, W, p, m, eps):
    H, n, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = (h @ W[p + "q"].T).view(T, H, n) * n ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, n)
    v = (h @ W[p + "v"].T).view(T, H, dv)
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    o = gated_linear_attention(q, k, v, channel_decay(z, float(m["tau"])).view(T, H, n))
    o = rms_norm(o, W[p + "norm"], eps).reshape(T, H * dv)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps):
    left = attention_mixer(h, W, p + "left.", m["left"], eps)
    right = linear_mixer(h, W, p + "right.", m["right"], eps)
    return 0.5 * (rms_norm(left, W[p + "left.out"], eps) + rms_norm(right, W[p + "right.out"], eps))


def dense_ff(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def relu2_ff(h, W, p):
    u = torch.clamp(h @ W[p + "up"].T, min=0.0)
    return (u * u) @ W[p + "down"].T


def route(h, w_router, correction, groups, keep, top):
    """h [width] -> [(expert, weight)].  Experts come in `groups` equal runs of neighbours; a run is worth the sum of its
    two largest choice scores, and only experts of the `keep` best runs can be chosen."""
    s = torch.sigmoid(w_router @ h)
    choice = (s + correction).tolist()
    E = len(choice)
    per = E // groups
    worth = [sum(sorted(choice[g * per:(g + 1) * per], reverse=True)[:2]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: (-worth[g], g))[:keep]
    allowed = [e for e in range(E) if e // per in kept]
    chosen = sorted(allowed, key=lambda e: (-choice[e], e))[:top]
    return [(e, s[e]) for e in chosen]


def moe_ff(h, W, p, mlp):
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in route(h[t], W[p + "router"], W[p + "correction"], int(groups["count"]), int(groups["keep"]), int(r["top"])):
            out[t] = out[t] + s * relu2_ff(h[t:t + 1], W, p + f"e{e}.")[0]
    if mlp.get("shared"):
        out = out + relu2_ff(h, W, p + "shared.")
    return out


def forward(config, weights, tokens, dtype=torch.float64, residuals=None):
    """tokens: list of ids of ONE sequence from position 0 -> logits [T, vocab]."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = float(config["norm"]["eps"])
    x = W["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    for i, layer in enumerate(config["layers"]):
        p, mlp = f"l{i}.", layer.get("mlp")
        x = x + layer_norm(parallel_mixer(x, W, p + "mix.", layer["mixer"], eps), W[p + "norm1"], eps)
        if mlp is not None:
            y = dense_ff(x, W, p + "mlp.") if mlp["kind"] == "dense" else moe_ff(x, W, p + "mlp.", mlp)
            x = x + layer_norm(y, W[p + "norm2"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    return layer_norm(x, W["final.norm"], eps) @ W["head"].T
