"""Plain CPU restatement of the Zomipel decoder, one function per mechanism: loops over tokens, heads and experts where that
is the clearest form, fp32 (or the dtype of its inputs, e.g. float64) throughout.  Test infrastructure only; nothing of the
product path is used here.

Notation: x (T, width) the residual rows of one sequence, positions 0 .. T-1; p the dict of tensors; all functions take the
tensors they need in the computing dtype.
"""
from __future__ import annotations

import math

import torch


def unit_rms(v, eps):
    """A row divided by its root mean square."""
    return v / torch.sqrt(torch.mean(v * v, dim=-1, keepdim=True) + eps)


def offset_rms_norm(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-torch.abs(z)))


# ---- attention -------------------------------------------------------------------------------------
def rotate(x, position, base, dims):
    """Rotation of the first `dims` entries of a head vector: entry i turns with entry i + dims/2 by position * base^(-2i/dims)."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = torch.tensor(position * base ** (-2.0 * i / dims), dtype=x.dtype)
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * torch.cos(a) - v * torch.sin(a)
        out[..., i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def sees(i, j, window, keep_first):
    """Does the query at position i see the key at position j?  window None: every earlier key."""
    return j <= i and (window is None or i - j < window or j < keep_first)


def window_attention(q, k, v, scale, window=None, keep_first=0, first=0):
    """Softmax attention of query rows at positions first, first+1, ... over the keys they see.  q (T,H,dk), k (S,G,dk),
    v (S,G,dv)."""
    T, H, _ = q.shape
    S, G = k.shape[:2]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        keys = [j for j in range(S) if sees(first + t, j, window, keep_first)]
        for h in range(H):
            g = h // (H // G)
            s = (k[keys, g] @ q[t, h]) * scale
            w = torch.exp(s - s.max())
            out[t, h] = (w / w.sum()) @ v[keys, g]
    return out


# ---- Mamba-2 ----------------------------------------------------------------------------------------
def causal_conv_silu(u, taps, bias, history=None):
    """Per channel: a sum over the last K inputs (the last tap is the current one's), bias, silu.  u (T,C), taps (C,K);
    history (K-1,C): inputs before the first row (None: zeros)."""
    T, C = u.shape
    K = taps.shape[1]
    if history is None:
        history = torch.zeros(K - 1, C, dtype=u.dtype)
    ext = torch.cat((history, u))
    out = torch.zeros_like(u)
    for t in range(T):
        for j in range(K):
            out[t] = out[t] + taps[:, j] * ext[t + j]
    return silu(out + bias)


def selective_state(x, B, C, dt, A, D, state=None):
    """The recurrence, token by token: S <- exp(A dt) S + dt B x^T, y = S^T C + D x.  x (T,H,P), B and C (T,G,N), dt (T,H) after
    softplus, A (H,) negative, D (H,).  Returns y (T,H,P) and the last states (H,N,P)."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, P, dtype=x.dtype) if state is None else state.clone()
    y = torch.zeros_like(x)
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = torch.exp(A[h] * dt[t, h]) * S[h] + dt[t, h] * torch.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
    return y, S


def gated_group_norm(y, z, w, groups, eps):
    """y silu(z), each of `groups` equal parts divided by its own root mean square, times w."""
    v = y * silu(z)
    parts = [unit_rms(part, eps) for part in torch.chunk(v, groups, dim=-1)]
    return torch.cat(parts, -1) * w


def mamba2(m, p, n, h, eps):
    """The mixer on the rows h of one sequence."""
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = torch.split(h @ p[n + "in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    xbc = causal_conv_silu(xbc, p[n + "conv"], p[n + "conv.b"])
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=-1)
    y, _ = selective_state(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + p[n + "dt_bias"]),
                           -torch.exp(p[n + "A_log"]), p[n + "D"])
    return gated_group_norm(y.reshape(T, inner), z, p[n + "norm"], m["norm_groups"], eps) @ p[n + "o"].T


def attention(m, p, n, h, eps):
    """The mixer on the rows h of one sequence."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ p[n + "q"].T + p[n + "q.b"]).view(T, H, dk)
    k = (h @ p[n + "k"].T + p[n + "k.b"]).view(T, G, dk)
    v = (h @ p[n + "v"].T + p[n + "v.b"]).view(T, G, dv)
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = torch.stack([rotate(q[t], t, base, dims) for t in range(T)])
    k = torch.stack([rotate(k[t], t, base, dims) for t in range(T)])
    a = window_attention(q, k, v, m["scale"], m["mask"]["size"], m["mask"]["keep_first"])
    return a.reshape(T, -1) @ p[n + "o"].T


MIXERS = {"attention": attention, "mamba2": mamba2}


# ---- feed-forward -------------------------------------------------------------------------------------
def gated_ff(p, n, h):
    return (silu(h @ p[n + ".gate"].T) * (h @ p[n + ".up"].T)) @ p[n + ".down"].T


def route(h, w, b, top):
    """Chosen experts of one row (largest logits first) and their weights: the softmax over the chosen logits."""
    z = w @ h + b
    chosen = sorted(range(len(z)), key=lambda e: -float(z[e]))[:top]
    s = torch.exp(z[chosen] - z[chosen].max())
    return chosen, s / s.sum()


def mixture(f, p, n, h):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(*route(h[t], p[n + "router"], p[n + "router.b"], f["router"]["top"])):
            out[t] = out[t] + w * gated_ff(p, n + f"e{e}", h[t])
    if f.get("shared") is not None:
        out = out + gated_ff(p, n + "shared", h) / (1.0 + torch.exp(-(h @ p[n + "shared.sg"].T)))
    return out


def feed_forward(f, p, n, h):
    if f is None:
        return torch.zeros_like(h)
    if f["kind"] == "dense":
        return gelu_tanh(h @ p[n + "up"].T) @ p[n + "down"].T
    return mixture(f, p, n, h)


# ---- the model ------------------------------------------------------------------------------------------
def layer_runs(config):
    """Layer indices in running order, and the places in that order in front of which the embedding output is added."""
    n, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return list(range(n)), []
    body = list(range(loop["start"], loop["stop"]))
    order = list(range(loop["start"])) + body * loop["times"] + list(range(loop["stop"], n))
    return order, [loop["start"] + i * len(body) for i in range(1, loop["times"])]


def forward(config, params, tokens, dtype=torch.float32, want_layers=False):
    """Logits (T, vocab) of one sequence, computed from scratch (no cache, no state)."""
    p = {n: t.to(dtype) for n, t in params.items()}
    eps = config["norm"]["eps"]
    x = x0 = p["embed"][torch.as_tensor(tokens)]
    order, again = layer_runs(config)
    after = []
    for place, i in enumerate(order):
        if place in again:
            x = x + x0
        layer, n = config["layers"][i], f"l{i}."
        h = offset_rms_norm(x, p[n + "norm1"], eps)
        x = x + (MIXERS[layer["type"]](layer["mixer"], p, n + "mix.", h, eps) + feed_forward(layer["mlp"], p, n + "mlp.", h))
        after.append(x)
    logits = offset_rms_norm(x, p["final.norm"], eps) @ p["embed"].T
    return (logits, torch.stack(after)) if want_layers else logits


def random_params(config, seed):
    """bf16 parameters of a configuration, of sizes that keep the residual stream near one, let the attention prefer single keys and
    give the recurrences memories between a few and a few hundred tokens."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s, std=1.0, mean=0.0: (torch.randn(*s, generator=g) * std + mean).to(torch.bfloat16)
    d, p = config["width"], {}
    w = lambda name, rows, cols, gain=1.0: p.__setitem__(name, r(rows, cols, std=gain / math.sqrt(cols)))

    def gated(n, ff):
        w(n + ".gate", ff, d, 1.5)
        w(n + ".up", ff, d, 1.5)
        w(n + ".down", d, ff, 1.0)

    p["embed"] = r(config["vocab"], d, std=0.7)
    p["final.norm"] = r(d, std=0.2)
    for i, layer in enumerate(config["layers"]):
        n, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        p[n + "norm1"] = r(d, std=0.2)
        if layer["type"] == "attention":
            for name, size, gain in (("q", m["heads"] * m["dim"], 1.6), ("k", m["kv_heads"] * m["dim"], 1.6), ("v", m["kv_heads"] * m["vdim"], 1.0)):
                w(f"{n}mix.{name}", size, d, gain)
                p[f"{n}mix.{name}.b"] = r(size, std=0.3)
            w(n + "mix.o", d, m["heads"] * m["vdim"])
        else:
            inner, bc = m["heads"] * m["vdim"], m["groups"] * m["state"]
            w(n + "mix.in", 2 * inner + 2 * bc + m["heads"], d)
            p[n + "mix.conv"] = r(inner + 2 * bc, m["conv"], std=0.6)
            p[n + "mix.conv.b"] = r(inner + 2 * bc, std=0.2)
            p[n + "mix.dt_bias"] = r(m["heads"], std=0.5, mean=-2.0)
            p[n + "mix.A_log"] = r(m["heads"], std=1.5, mean=-1.0)
            p[n + "mix.D"] = r(m["heads"], std=0.5, mean=0.5)
            p[n + "mix.norm"] = r(inner, std=0.2, mean=1.0)
            w(n + "mix.o", d, inner)
        if f is None:
            continue
        if f["kind"] == "dense":
            w(n + "mlp.up", f["ff"], d, 1.5)
            w(n + "mlp.down", d, f["ff"])
            continue
        for e in range(f["router"]["experts"]):
            gated(f"{n}mlp.e{e}", f["expert"]["ff"])
        w(n + "mlp.router", f["router"]["experts"], d, 2.0)
        p[n + "mlp.router.b"] = r(f["router"]["experts"], std=0.3)
        if f.get("shared") is not None:
            gated(n + "mlp.shared", f["shared"]["ff"])
            w(n + "mlp.shared.sg", 1, d, 1.5)
    return p
