"""Plain CPU restatement of the Zuzelorn decoder, one function per mechanism: loops over tokens and heads where that is the
clearest form, fp32 (or the dtype of its inputs, e.g. float64) throughout.  Test infrastructure only; nothing of the product
path is used here.

Notation: x (T, width) the residual rows of one sequence, positions 0 .. T-1; p the dict of tensors; all functions take the
tensors they need in the computing dtype.
"""
from __future__ import annotations

import math

import torch


def dynamic_tanh(x, alpha, w, b):
    """tanh(alpha x) w + b, element by element."""
    return torch.tanh(alpha * x) * w + b


def unit_rms(v, eps):
    """A row divided by its root mean square."""
    return v / torch.sqrt(torch.mean(v * v, dim=-1, keepdim=True) + eps)


def polynorm(z, coeffs, eps):
    a, b, c, e = (float(t) for t in coeffs)
    return a * unit_rms(z, eps) + b * unit_rms(z ** 2, eps) + c * unit_rms(z ** 3, eps) + e


def sink_attention(q, k, v, scale, temp, sink, first=0):
    """Causal attention of query rows at positions first, first+1, ... over all keys.  q (T,H,dk), k (S,G,dk), v (S,G,dv);
    temp, sink (H,): factor on a head's scores; extra score in its denominator (None: 1 / no sink)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for t in range(T):
            n = first + t + 1
            s = (k[:n, g] @ q[t, h]) * scale * (1.0 if temp is None else float(temp[h]))
            top = float(s.max()) if sink is None else max(float(s.max()), float(sink[h]))
            w = torch.exp(s - top)
            den = w.sum() + (0.0 if sink is None else math.exp(float(sink[h]) - top))
            out[t, h] = (w / den) @ v[:n, g]
    return out


def gate(y, h, w, b):
    """y times the logistic function of W h + b, element by element."""
    return y / (1.0 + torch.exp(-(h @ w.T + b)))


def _norm(p, name, x):
    return dynamic_tanh(x, p[name + ".alpha"], p[name], p[name + ".b"])


def forward(config, params, tokens, dtype=torch.float32, want_layers=False):
    """Logits (T, vocab) of one sequence, computed from scratch (no cache)."""
    p = {n: t.to(dtype) for n, t in params.items()}
    eps = config["norm"]["eps"]
    T = len(tokens)
    x = torch.stack([p["embed"][t] + p["pos"][i] for i, t in enumerate(tokens)])
    keys_values, after = {}, []
    for i, layer in enumerate(config["layers"]):
        m, n = layer["mixer"], f"l{i}."
        H, G = m["heads"], m["kv_heads"]
        h = _norm(p, n + "norm1", x)
        q = (h @ p[n + "mix.q"].T + p[n + "mix.q.b"]).view(T, H, m["dim"])
        if m.get("kv_from") is None:
            keys_values[i] = ((h @ p[n + "mix.k"].T + p[n + "mix.k.b"]).view(T, G, m["dim"]),
                              (h @ p[n + "mix.v"].T + p[n + "mix.v.b"]).view(T, G, m["vdim"]))
            k, v = keys_values[i]
        else:
            k, v = keys_values[m["kv_from"]]
        a = sink_attention(q, k, v, m["scale"], p[n + "mix.temp"], p[n + "mix.sink"])
        o = a.reshape(T, -1) @ p[n + "mix.o"].T + p[n + "mix.o.b"]
        x = x + _norm(p, n + "norm1b", gate(o, h, p[n + "rg1"], p[n + "rg1.b"]))
        if layer["mlp"] is not None:
            h = _norm(p, n + "norm2", x)
            f = polynorm(h @ p[n + "mlp.up"].T, p[n + "mlp.act"], eps) @ p[n + "mlp.down"].T
            x = x + _norm(p, n + "norm2b", gate(f, h, p[n + "rg2"], p[n + "rg2.b"]))
        after.append(x)
    logits = (_norm(p, "final.norm", x) @ p["head"].T) * config["logit_scale"]
    return (logits, torch.stack(after)) if want_layers else logits


def random_params(config, seed, sharpness=1.0):
    """Random bf16 tensors of a configuration.  Every bias, norm, temp and sink differs from a neutral value; `sharpness`
    scales the query weights (peaked attention: single keys matter)."""
    g = torch.Generator().manual_seed(seed)
    d = config["width"]

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)

    p = {"embed": rnd(config["vocab"], d), "pos": rnd(config["max_positions"], d, std=0.5),
         "head": rnd(config["vocab"], d, std=1.5 * d ** -0.5)}

    def norm(name):
        p[name] = rnd(d, std=0.3, mean=1.0)
        p[name + ".b"] = rnd(d, std=0.15)
        p[name + ".alpha"] = (0.4 + 0.4 * torch.rand((), generator=g)).to(torch.bfloat16)

    norm("final.norm")
    for i, layer in enumerate(config["layers"]):
        m, n = layer["mixer"], f"l{i}."
        for s in ("norm1", "norm1b"):
            norm(n + s)
        for name, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
            if name == "q" or m.get("kv_from") is None:
                p[n + "mix." + name] = rnd(rows, d, std=(1.4 * sharpness if name == "q" else 1.4) * d ** -0.5)
                p[n + "mix." + name + ".b"] = rnd(rows, std=0.3)
        p[n + "mix.temp"] = rnd(m["heads"], std=0.3, mean=1.4)
        p[n + "mix.sink"] = rnd(m["heads"], std=1.0, mean=1.5)
        p[n + "mix.o"] = rnd(d, m["heads"] * m["vdim"], std=2.0 * (m["heads"] * m["vdim"]) ** -0.5)
        p[n + "mix.o.b"] = rnd(d, std=0.2)
        p[n + "rg1"], p[n + "rg1.b"] = rnd(d, d, std=d ** -0.5), rnd(d, std=0.5, mean=0.5)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            for s in ("norm2", "norm2b"):
                norm(n + s)
            p[n + "mlp.up"], p[n + "mlp.down"] = rnd(ff, d, std=1.4 * d ** -0.5), rnd(d, ff, std=1.4 * ff ** -0.5)
            p[n + "mlp.act"] = torch.tensor([0.7, 0.4, 0.5, 0.3]).to(torch.bfloat16) + rnd(4, std=0.1)
            p[n + "rg2"], p[n + "rg2.b"] = rnd(d, d, std=d ** -0.5), rnd(d, std=0.5, mean=0.5)
    return p
