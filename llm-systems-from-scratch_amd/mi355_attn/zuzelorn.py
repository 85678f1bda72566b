"""Zuzelorn: a decoder with Dynamic Tanh norms, gated residuals, softmax sinks, key/value sharing between layers and PolyNorm.

With D(x) = tanh(alpha x) * w + b (the norm, per place its own alpha, w, b), token t at position p:

    x = E[t] + P[p]
    per layer:   h = D1(x);  x += D1b(sigmoid(R1 h + r1) * (Wo A(h) + bo))
                 h = D2(x);  x += D2b(sigmoid(R2 h + r2) * Wdown F(Wup h))            (layers with a feed-forward)
    logits = logit_scale * head Dfinal(x)

A: causal grouped-query attention without rotation, score = scale * temp_head * (q . k), an extra exp(sink_head) in the
softmax denominator; q, k, v = affine projections of h, or -- a layer with `kv_from` -- q of its own over the cached keys
and values of an earlier layer.  F(z) = a N(z) + b N(z^2) + c N(z^3) + e, N dividing a row by its root mean square.

Device work per layer: two merged projections ([q | k | v | gate] and [up | gate]) and two output projections as library
GEMMs; the cache write, attention (per-head scale and sink inside the kernels), PolyNorm, and one pass at the end of every
sublayer that applies bias, gate, norm and residual add and the norm in front of the next sublayer.  The residual stream,
norms, scores and softmax are fp32; with dtype "float32" everything is.  There is no CPU path.
"""
from __future__ import annotations

import torch

from . import ops
from .engine import BLOCK, AttentionLayer, PagedAttentionEngine, cache_head_dims
from .model import CachedLM
from .weights import Checkpoint, pad_heads, stack_rows


class ZuzelornLM(CachedLM):
    DTYPES = ("bfloat16", "float32")

    def __init__(self, config: dict, state_dict: dict, *, num_blocks: int | None = None, max_batch: int = 64,
                 dtype: str = "bfloat16", kv_dtype: str | None = None, decode_graphs: bool = False, device="cuda:0"):
        """config: the parsed config.json (vocab, width, max_positions, logit_scale, norm.eps, layers); state_dict: its
        tensors.  dtype "float32" computes everything in 32-bit; kv_dtype "fp8" keeps a bfloat16 model's cache as e4m3
        with scales.  num_blocks sizes every layer's pool (default: max_batch full contexts)."""
        if dtype not in self.DTYPES:
            raise ValueError(f"dtype must be one of {self.DTYPES}")
        self.config = dict(config)
        self.dtype = getattr(torch, dtype)
        if kv_dtype is None:
            kv_dtype = "bf16" if dtype == "bfloat16" else "fp32"
        if (kv_dtype == "fp32") != (dtype == "float32"):
            raise ValueError("a float32 model has an fp32 cache, a bfloat16 model a bf16 or fp8 one")
        dev = torch.device(device)
        d = self.width = config["width"]
        self.eps = float(config["norm"]["eps"])
        self.logit_scale = float(config.get("logit_scale", 1.0))
        context_length = config["max_positions"]
        ckpt = Checkpoint(state_dict, self.dtype, dev)
        raw, mat, vec = ckpt.raw, ckpt.matrix, ckpt.vector

        def norm(name):
            return float(raw(name + ".alpha").float()), vec(name, d), vec(name + ".b", d)

        self.emb = mat(raw("embed", config["vocab"], d))
        self.pos = mat(raw("pos", context_length, d))
        self.head = mat(raw("head", config["vocab"], d))
        self.final_norm = norm("final.norm")
        self.layers, attention = [], []
        for i, entry in enumerate(config["layers"]):
            if entry["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
            m, mlp, pre = entry["mixer"], entry.get("mlp"), f"l{i}."
            H, dk = m["heads"], m["dim"]
            G, dv = m.get("kv_heads", H), m.get("vdim", dk)
            kd, vd, _ = cache_head_dims(kv_dtype, dk, dv)
            # temp_head: its size scales the scores in the kernels; its sign moves into the head's query (exact)
            temp = raw(pre + "mix.temp", H).float()
            sign = torch.where(temp < 0, -1.0, 1.0).repeat_interleave(dk)
            w = [pad_heads(raw(pre + "mix.q", H * dk, d).float() * sign[:, None], H, dk, kd)]
            b = [pad_heads(raw(pre + "mix.q.b", H * dk).float() * sign, H, dk, kd)]
            src = m.get("kv_from")
            if src is None:
                for n, size, to in (("k", dk, kd), ("v", dv, vd)):
                    w.append(pad_heads(raw(pre + f"mix.{n}", G * size, d).float(), G, size, to))
                    b.append(pad_heads(raw(pre + f"mix.{n}.b", G * size).float(), G, size, to))
            w.append(raw(pre + "rg1", d, d).float())
            b.append(b[0].new_zeros(d))                     # (the gate's bias is added in fp32 where the gate is applied)
            w_in, starts = stack_rows(w)
            wo = pad_heads(raw(pre + "mix.o", d, H * dv).float().t(), H, dv, vd).t()
            ly = dict(H=H, G=G, kd=kd, vd=vd, own_kv=src is None, w_in=mat(w_in), b_in=mat(stack_rows(b)[0]), starts=starts,
                      wo=mat(wo), bo=vec(pre + "mix.o.b", d), rg1_b=vec(pre + "rg1.b", d), norm1=norm(pre + "norm1"),
                      norm1b=norm(pre + "norm1b"), ff=None)
            if mlp is not None:
                if mlp["kind"] != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
                ff = mlp["ff"]
                w_up, (_, gate_at) = stack_rows([raw(pre + "mlp.up", ff, d), raw(pre + "rg2", d, d)])
                ly.update(ff=ff, w_up=mat(w_up), gate_at=gate_at, wdown=mat(raw(pre + "mlp.down", d, ff)),
                          act=raw(pre + "mlp.act", 4).float().tolist(), rg2_b=vec(pre + "rg2.b", d), norm2=norm(pre + "norm2"),
                          norm2b=norm(pre + "norm2b"))
            self.layers.append(ly)
            # (a factor of exactly 0 would turn the kernels' masked scores of -inf into NaN)
            attention.append(AttentionLayer(H, G, dk, dv, kv_from=src, softmax_scale=m.get("scale"), rope=False,
                                            head_scale=temp.abs().clamp_min(1e-30).to(dev), sinks=vec(pre + "mix.sink", H)))
        if num_blocks is None:
            num_blocks = max_batch * ((context_length + BLOCK - 1) // BLOCK)
        self._serve(PagedAttentionEngine(num_blocks, context_length=context_length, max_batch=max_batch, kv_dtype=kv_dtype,
                                         device=dev, layers=attention), config["vocab"], decode_graphs)

    def _forward(self, token_ids, plan, attend, out_rows=None):
        T, d = token_ids.shape[0], self.width
        x = ops.embed_pos(self.emb, self.pos, token_ids, plan.positions)          # fp32; updated in place below
        h = ops.dyt_residual(x, norm=self.layers[0]["norm1"] if self.layers else self.final_norm, out_dtype=self.dtype)
        for i, ly in enumerate(self.layers):
            nxt = self.layers[i + 1]["norm1"] if i + 1 < len(self.layers) else self.final_norm
            H, G, kd, vd, at = ly["H"], ly["G"], ly["kd"], ly["vd"], ly["starts"]
            p = torch.addmm(ly["b_in"], h, ly["w_in"].T)
            q, k, v = p[:, :H * kd].view(T, H, kd), None, None
            if ly["own_kv"]:
                k = p[:, at[1]:at[1] + G * kd].view(T, G, kd)
                v = p[:, at[2]:at[2] + G * vd].view(T, G, vd)
            a = attend(i, plan, q, k, v)
            o = a.reshape(T, H * vd) @ ly["wo"].T
            h = ops.dyt_residual(x, o, sub_bias=ly["bo"], gate=p[:, at[-1]:at[-1] + d], gate_bias=ly["rg1_b"], post=ly["norm1b"],
                                 norm=ly["norm2"] if ly["ff"] else nxt, out_dtype=self.dtype)
            if ly["ff"]:
                u = h @ ly["w_up"].T
                f = ops.polynorm(u[:, :ly["ff"]], ly["act"], self.eps) @ ly["wdown"].T
                h = ops.dyt_residual(x, f, gate=u[:, ly["gate_at"]:ly["gate_at"] + d], gate_bias=ly["rg2_b"], post=ly["norm2b"],
                                     norm=nxt, out_dtype=self.dtype)
        if out_rows is not None:
            if out_rows.shape[0] == 0:
                return torch.empty(0, self.vocab_size, dtype=torch.float32, device=self.device)
            h = h[out_rows]
        return (h @ self.head.T).float() * self.logit_scale
