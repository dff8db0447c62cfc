"""Plain, slow restatement of the Dugazen layer stack: one function per mechanism, whole sequences, loops over
tokens and heads.  Shares nothing with the product path; the tests compare the engine against it.  Everything
runs in `dtype` (float64 by default) on the CPU.

Weights come as a dict name -> tensor with the checkpoint's names ('l<i>.mix.q', ...), the configuration as the
parsed config.json dict.

Notation.  N = RMS norm with weight 1 + w.  A layer norms what a sublayer reads and what it returns:
    x <- x + m Nb1( M(N1(x)) );   x <- x + m Nb2( F(N2(x)) )
M is 'channel_delta' (a delta-rule memory S [dim, vdim] per head whose rows decay by a gate of their own) or
'attention' (windowed softmax attention, values mixed with those of the first such layer); F the clamped gated
feed-forward, or nothing.
"""
import math

import torch

UNIT_EPS = 1e-6
SLOPE = 1.702


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    return rms_unit(x, eps) * (1.0 + w)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-torch.abs(x)))


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] * u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] = y[t] + w[:, j] * u[s]
    return y


def channel_decay(a, dt_bias, a_log, heads):
    """a [T, heads * dim] -> gates [T, heads, dim] = exp(-exp(a_log_h) softplus(a + dt_bias))."""
    T = a.shape[0]
    return torch.exp(-torch.exp(a_log).view(1, heads, 1) * softplus(a + dt_bias).view(T, heads, -1))


def delta_rule(q, k, v, gate, beta, state=None):
    """q, k [T, H, n]; v [T, H, p]; gate [T, H, n]; beta [T, H] -> o [T, H, p].  Per head, S [n, p] from zero:
    decay the rows, correct the value the key reads, write, then read with q."""
    T, H, n = q.shape
    S = torch.zeros(H, n, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = gate[t, h][:, None] * S[h]
            u = beta[t, h] * (v[t, h] - k[t, h] @ S[h])
            S[h] = S[h] + torch.outer(k[t, h], u)
            out[t, h] = q[t, h] @ S[h]
    return out if state is None else (out, S)


def delta_mixer(h, W, p, m, eps):
    H, K, n, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]

    def short(name):
        return silu(causal_conv(h @ W[p + name].T, W[p + name + ".conv"]))

    q = unit_vector(short("q").view(T, K, n)) * n ** -0.5
    k = unit_vector(short("k").view(T, K, n))
    v = short("v").view(T, H, dv)
    src = [hd // (H // K) for hd in range(H)]
    beta = torch.sigmoid(h @ W[p + "b"].T)
    gate = channel_decay((h @ W[p + "a1"].T) @ W[p + "a2"].T, W[p + "dt_bias"], W[p + "A_log"], H)
    o = delta_rule(q[:, src], k[:, src], v, gate, beta)
    z = torch.sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T).view(T, H, dv)
    return (rms_unit(o, eps) * W[p + "norm"] * z).reshape(T, H * dv) @ W[p + "o"].T


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


def window_attention(q, k, v, scale, window):
    """q [T, H, d], k [T, G, d], v [T, G, dv]: softmax over the keys j with 0 <= i - j < window."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for hd in range(H):
        g = hd // (H // G)
        for i in range(T):
            lo = max(0, i - window + 1)
            s = (k[lo:i + 1, g] @ q[i, hd]) * scale
            e = torch.exp(s - s.max())
            out[i, hd] = (e / e.sum()) @ v[lo:i + 1, g]
    return out


def attention_mixer(h, W, p, m, eps, first):
    """`first`: a one-element list holding the values of the first mixing layer (None until that layer has run)."""
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = rms_unit(h @ W[p + "q"].T + W[p + "q.b"], eps) * W[p + "q.norm"]
    k = rms_unit(h @ W[p + "k"].T + W[p + "k.b"], eps) * W[p + "k.norm"]
    v = h @ W[p + "v"].T + W[p + "v.b"]
    rot, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
    q, k = rotate_halves(q.view(T, H, d), rot, base), rotate_halves(k.view(T, G, d), rot, base)
    if m.get("v_mix"):
        if first[0] is None:
            first[0] = v
        else:
            lam = W[p + "vmix"].reshape(())
            v = (1.0 - lam) * v + lam * first[0]
    o = window_attention(q, k, v.view(T, G, dv), float(m["scale"]), int(m["mask"]["size"])).reshape(T, H * dv)
    return (o * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T + W[p + "o.b"]


def clamped_ff(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(SLOPE * g) * (u + 1.0)) @ W[p + "down"].T


def forward(config, weights, tokens, dtype=torch.float64, residuals=None):
    """tokens: list of ids of ONE sequence from position 0 -> logits [T, vocab]."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps, mult = float(config["norm"]["eps"]), float(config["residual_mult"])
    x = W["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    first = [None]
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = offset_norm(x, W[p + "norm1"], eps)
        if layer["type"] == "channel_delta":
            y = delta_mixer(h, W, p + "mix.", m, eps)
        elif layer["type"] == "attention":
            y = attention_mixer(h, W, p + "mix.", m, eps, first)
        else:
            raise ValueError(layer["type"])
        x = x + mult * offset_norm(y, W[p + "norm1b"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = offset_norm(x, W[p + "norm2"], eps)
            x = x + mult * offset_norm(clamped_ff(h, W, p + "mlp.", float(mlp["limit"])), W[p + "norm2b"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    return (offset_norm(x, W["final.norm"], eps) @ W["head"].T) * float(config["logit_scale"])
