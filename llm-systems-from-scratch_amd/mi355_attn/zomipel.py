"""Zomipel: Mamba-2 and sliding-window attention layers with parallel feed-forwards, dense or mixtures of experts, run in a loop.

With N(x) = x / rms(x) * (1 + w), per layer and token

    h = N(x);   x += mixer(h) + ff(h)              logits = E N_final(x)

Mixers: grouped-query attention with biases, partial rotation and a sliding window that keeps the first tokens; Mamba-2
(convolution, selective state, gated group norm).  Feed-forwards: gelu; or `top` of `experts` gated layers, weighted by the
softmax over the chosen logits, plus an optional shared one behind a sigmoid gate; or none.  `loop` repeats a run of layers with
the same weights, every pass with a cache or state of its own and with the embedding output added in front of all but the first.

Device work per layer: one library GEMM for everything that reads h as a dense matrix ([q | k | v] or [z | x | B | C | dt], and
the dense or shared feed-forward's first projections); the mixer's kernels and the feed-forward's activation, which write side by
side into the rows of one matrix; one library GEMM that projects these rows out, i.e. adds mixer and feed-forward; router, grouping
and the grouped products of the experts; and one pass that adds all of it (and the embedding, in front of a repeated pass) to
the fp32 residual stream and norms it for the next layer.  With dtype "float32" everything is.  There is no CPU path.
"""
from __future__ import annotations

import torch

from . import ops
from .engine import BLOCK, AttentionLayer, PagedAttentionEngine, StateLayer, cache_head_dims
from .model import CachedLM
from .weights import Checkpoint, pad_heads, pad_to, pair_halves, stack_rows

DEFAULT_CONTEXT = 32768


def layer_runs(n_layers: int, loop: dict | None) -> tuple[list[int], set[int]]:
    """The layers in the order they run, and the places in that order where a repeated pass begins."""
    if loop is None:
        return list(range(n_layers)), set()
    start, stop, times = loop["start"], loop["stop"], loop["times"]
    if not 0 <= start < stop <= n_layers or times < 1:
        raise ValueError(f"loop {loop} does not fit {n_layers} layers")
    body = list(range(start, stop))
    return list(range(start)) + body * times + list(range(stop, n_layers)), {start + i * len(body) for i in range(1, times)}


class ZomipelLM(CachedLM):
    DTYPES = ("bfloat16", "float32")

    def __init__(self, config: dict, state_dict: dict, *, num_blocks: int | None = None, max_batch: int = 64,
                 context_length: int | None = None, dtype: str = "bfloat16", kv_dtype: str | None = None,
                 decode_graphs: bool = False, device="cuda:0"):
        """config: the parsed config.json (vocab, width, norm.eps, layers, loop); state_dict: its tensors.  The design sets no
        limit on positions: context_length (default: what the pool holds, or DEFAULT_CONTEXT) sizes the rotation tables and
        block tables.  num_blocks sizes every attention run's pool (default: max_batch full contexts).  dtype "float32"
        computes everything in 32-bit; kv_dtype "fp8" keeps a bfloat16 model's keys and values as e4m3 with scales."""
        if dtype not in self.DTYPES:
            raise ValueError(f"dtype must be one of {self.DTYPES}")
        self.config = dict(config)
        self.dtype = getattr(torch, dtype)
        if kv_dtype is None:
            kv_dtype = "bf16" if dtype == "bfloat16" else "fp32"
        if (kv_dtype == "fp32") != (dtype == "float32"):
            raise ValueError("a float32 model has an fp32 cache, a bfloat16 model a bf16 or fp8 one")
        if context_length is None:
            context_length = num_blocks * BLOCK if num_blocks is not None else DEFAULT_CONTEXT
        if num_blocks is None:
            num_blocks = max_batch * ((context_length + BLOCK - 1) // BLOCK)
        dev = torch.device(device)
        self.width = config["width"]
        self.eps = float(config["norm"]["eps"])
        self.h_cols = self.width + (-self.width % 64 if dtype == "bfloat16" else 0)      # (what the expert kernels read)
        ckpt = Checkpoint(state_dict, self.dtype, dev)
        self.emb = ckpt.matrix(ckpt.raw("embed", config["vocab"], self.width))
        self.final_norm = ckpt.vector("final.norm", self.width)
        layers, managed = [], []
        for i, entry in enumerate(config["layers"]):
            pre = f"l{i}."
            w_in, b_in, w_out = [], [], []               # rows of the projection of h, its biases; columns of the way out
            if entry["type"] == "attention":
                ly, mgr = self._attention(ckpt, pre + "mix.", entry["mixer"], kv_dtype, w_in, b_in, w_out)
            elif entry["type"] == "mamba2":
                ly, mgr = self._mamba2(ckpt, pre + "mix.", entry["mixer"], w_in, w_out)
            else:
                raise ValueError(f"layer {i}: unknown mixer {entry['type']!r}")
            n_mixer = len(w_in)
            ly.update(norm=ckpt.vector(pre + "norm1", self.width), ff=None, moe=None)
            ly.update(self._feed_forward(ckpt, pre + "mlp.", i, entry.get("mlp"), w_in, w_out))
            w, at = stack_rows(w_in)
            ly.update(w_in=ckpt.matrix(w), at=at[:n_mixer], ff_at=at[n_mixer:], b_in=None)
            if b_in:
                b = w.new_zeros(w.shape[0])
                for start, part in zip(at, b_in):
                    b[start:start + part.shape[0]] = part
                ly["b_in"] = ckpt.matrix(b)
            w, at = stack_rows([t.t() for t in w_out])
            ly.update(w_out=ckpt.matrix(w.t()), out_at=at)
            layers.append(ly)
            managed.append(mgr)
        order, self.again = layer_runs(len(layers), config.get("loop"))
        self.runs = [layers[i] for i in order]
        self._serve(PagedAttentionEngine(num_blocks, context_length=context_length, max_batch=max_batch, kv_dtype=kv_dtype,
                                         device=dev, layers=[managed[i] for i in order]), config["vocab"], decode_graphs)

    def _attention(self, ckpt, n, m, kv_dtype, w_in, b_in, w_out):
        d, H, G, dk, dv = self.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        kd, vd, _ = cache_head_dims(kv_dtype, dk, dv)
        dims = m["rot"]["dims"]
        for name, heads, size, to, turned in (("q", H, dk, kd, dims), ("k", G, dk, kd, dims), ("v", G, dv, vd, 0)):
            for parts, t in ((w_in, ckpt.raw(n + name, heads * size, d)), (b_in, ckpt.raw(f"{n}{name}.b", heads * size))):
                parts.append(pad_heads(pair_halves(t, heads, size, turned), heads, size, to))
        w_out.append(pad_heads(ckpt.raw(n + "o", d, H * dv).t(), H, dv, vd).t())
        mask = m["mask"]
        return (dict(type="attention", H=H, G=G, kd=kd, vd=vd),
                AttentionLayer(H, G, dk, dv, softmax_scale=float(m["scale"]), rope=dims > 0, rope_base=float(m["rot"]["base"]),
                               rope_dims=dims, window=mask["size"], keep_first=mask["keep_first"]))

    def _mamba2(self, ckpt, n, m, w_in, w_out):
        d, H, P, N, G, taps = self.width, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
        inner, channels = H * P, H * P + 2 * G * N
        w_in += torch.split(ckpt.raw(n + "in", inner + channels + H, d), [inner, channels, H])
        w_out.append(ckpt.raw(n + "o", d, inner))
        params = dict(conv=ckpt.vector(n + "conv", channels, taps).t().contiguous(), conv_b=ckpt.vector(n + "conv.b", channels),
                      dt_bias=ckpt.vector(n + "dt_bias", H), neg_a=-torch.exp(ckpt.vector(n + "A_log", H)),
                      d_skip=ckpt.vector(n + "D", H))
        return (dict(type="mamba2", inner=inner, gate_norm=ckpt.vector(n + "norm", inner), norm_groups=m["norm_groups"]),
                StateLayer(H, P, N, G, taps, params))

    def _feed_forward(self, ckpt, n, i, mlp, w_in, w_out):
        if mlp is None:
            return {}
        d = self.width
        if mlp["kind"] == "dense":
            w_in.append(ckpt.raw(n + "up", mlp["ff"], d))
            w_out.append(ckpt.raw(n + "down", d, mlp["ff"]))
            return dict(ff=mlp["ff"])
        if mlp["kind"] != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
        experts, top, ff, shared = mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"], mlp.get("shared")
        # the expert kernels walk k in steps of 64 elements of bf16: zeros behind the rows of h and behind ff
        step = 64 if self.dtype == torch.bfloat16 else 1
        gate_up, down = [], []
        for e in range(experts):
            gate_up += [pad_to(pad_to(ckpt.raw(f"{n}e{e}.{part}", ff, d), 0, step), 1, step) for part in ("gate", "up")]
            down.append(pad_to(ckpt.raw(f"{n}e{e}.down", d, ff), 1, step))
        rows, bias = [ckpt.raw(n + "router", experts, d)], [ckpt.raw(n + "router.b", experts)]
        out = {}
        if shared is not None:
            for part in ("gate", "up"):
                w_in.append(ckpt.raw(f"{n}shared.{part}", shared["ff"], d))
            w_out.append(ckpt.raw(n + "shared.down", d, shared["ff"]))
            rows.append(ckpt.raw(n + "shared.sg", 1, d))
            bias.append(bias[0].new_zeros(1))
            out["ff"] = shared["ff"]
        out["moe"] = dict(top=top, router=ckpt.matrix(pad_to(torch.cat(rows), 1, step)), shared=shared is not None,
                          bias=torch.cat(bias).to(device=ckpt.device, dtype=torch.float32),
                          gate_up=torch.stack([ckpt.matrix(torch.cat(gate_up[2 * e:2 * e + 2])) for e in range(experts)]),
                          down=torch.stack([ckpt.matrix(t) for t in down]))
        return out

    def _forward(self, token_ids, plan, attend, out_rows=None):
        return self._run(token_ids, plan, attend, out_rows)

    def _run(self, token_ids, plan, attend, out_rows=None, after_layer=None):
        """_forward; after_layer, when given, is called with the fp32 residual stream after every layer run."""
        T, d, dt = token_ids.shape[0], self.width, self.dtype
        norm = dict(weight_offset=1.0, eps=self.eps, out_dtype=dt, y_cols=self.h_cols)
        x, h = ops.residual_rms(None, self.runs[0]["norm"] if self.runs else self.final_norm, embed=self.emb, tokens=token_ids, **norm)
        for i, ly in enumerate(self.runs):
            hd = h[:, :d]
            p = hd @ ly["w_in"].T if ly["b_in"] is None else torch.addmm(ly["b_in"], hd, ly["w_in"].T)
            rows, at = torch.empty(T, ly["w_out"].shape[1], dtype=dt, device=x.device), ly["at"]
            if ly["type"] == "attention":
                H, G, kd, vd = ly["H"], ly["G"], ly["kd"], ly["vd"]
                attend(i, plan, p[:, :H * kd].view(T, H, kd), p[:, at[1]:at[1] + G * kd].view(T, G, kd),
                       p[:, at[2]:at[2] + G * vd].view(T, G, vd), out=rows[:, :H * vd].view(T, H, vd))
                used = H * vd
            else:
                used = ly["inner"]
                y = self.engine.advance_state(i, plan, p, at[1], at[2], out=rows[:, :used])
                ops.gated_norm(y, p[:, :used], ly["gate_norm"], ly["norm_groups"], self.eps, out=y)
            routed, moe = None, ly["moe"]
            shared_gate = None
            if moe is not None:
                ids, weights, shared_gate = ops.moe_route(h, moe["router"], moe["bias"], moe["top"], extra_row=moe["shared"])
                routed = ops.moe_experts(h, ids, weights, moe["gate_up"], moe["down"])
            if ly["ff"] is not None:
                ff, ff_at = ly["ff"], ly["ff_at"]
                ops.ff_act(p[:, ff_at[0]:ff_at[0] + ff], p[:, ff_at[1]:ff_at[1] + ff] if moe is not None else None,
                           row_gate=shared_gate, out=rows[:, ly["out_at"][1]:ly["out_at"][1] + ff])
            self._clear_gaps(rows, ly, used)
            again = i + 1 in self.again
            if after_layer is not None:                  # the stream itself, in front of what the next pass adds
                ops.residual_rms(x, None, sub=rows @ ly["w_out"].T, routed=routed, top=moe["top"] if moe else 1, out_dtype=dt)
                after_layer(x)
                sub = routed = None
            else:
                sub = rows @ ly["w_out"].T
            nxt = self.runs[i + 1]["norm"] if i + 1 < len(self.runs) else self.final_norm
            x, h = ops.residual_rms(x, nxt, sub=sub, routed=routed, top=moe["top"] if moe else 1, embed=self.emb if again else None,
                                    tokens=token_ids if again else None, **norm)
        if out_rows is not None:
            if out_rows.shape[0] == 0:
                return torch.empty(0, self.vocab_size, dtype=torch.float32, device=self.device)
            h = h[out_rows]
        return (h[:, :d] @ self.emb.T).float()

    @staticmethod
    def _clear_gaps(rows, ly, used):
        """The columns between the parts meet zero weights; they must hold numbers."""
        ends = ly["out_at"][1:] + [rows.shape[1]]
        for start, end in zip([used] + ([ly["out_at"][1] + ly["ff"]] if ly["ff"] is not None else []), ends):
            if start < end:
                rows[:, start:end] = 0
