"""Host logic around the Zuzelorn model, on the CPU: registry and configuration, cache geometry with layers that share keys
and values, weight layout (padding, stacking, sign of a head's factor), the trace replay loop and the command line -- and
the oracle itself against closed forms."""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

import mi355_attn
from mi355_attn import cli, zuzelorn
from mi355_attn.engine import AttentionLayer, PagedAttentionEngine, cache_head_dims
from oracle import zuzelorn_oracle as zo

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def attention(**kw):
    m = dict(heads=4, kv_heads=2, dim=24, vdim=16, scale=0.3)
    m.update(kw)
    return m


def config(layers, **kw):
    c = dict(architecture="Zuzelorn", vocab=37, width=40, max_positions=64, logit_scale=0.7, norm={"eps": 1e-5},
             layers=[{"type": "attention", "mixer": m, "mlp": f} for m, f in layers])
    c.update(kw)
    return c


FF = {"kind": "dense", "ff": 56}


# ---- oracle -------------------------------------------------------------------------------------
def test_oracle_attention_counts_the_sink_once_and_unscaled():
    q = torch.zeros(3, 2, 4)
    k, v = torch.randn(3, 1, 4), torch.ones(3, 1, 5)
    out = zo.sink_attention(q, k, v, scale=100.0, temp=torch.tensor([7.0, 1.0]), sink=torch.tensor([math.log(2.0), -math.inf]))
    for t in range(3):      # equal scores of 0: weights 1/(n + 2), and 1/n without a sink
        assert torch.allclose(out[t, 0], torch.full((5,), (t + 1) / (t + 3)), atol=1e-6)
        assert torch.allclose(out[t, 1], torch.ones(5), atol=1e-6)


def test_oracle_attention_equals_torch_softmax_attention_without_sink():
    q, k, v = torch.randn(9, 4, 8), torch.randn(9, 2, 8), torch.randn(9, 2, 6)
    got = zo.sink_attention(q, k, v, 0.4, None, None)
    kk, vv = (t.repeat_interleave(2, 1).transpose(0, 1) for t in (k, v))
    s = (q.transpose(0, 1) @ kk.transpose(1, 2)) * 0.4
    s = s.masked_fill(torch.ones(9, 9).triu(1).bool(), -math.inf)
    assert torch.allclose(got, (torch.softmax(s, -1) @ vv).transpose(0, 1), atol=1e-5)


def test_oracle_polynorm_and_gate_closed_forms():
    z = torch.tensor([[2.0, -2.0, 2.0, -2.0]])        # powers of constant size: every N is a sign pattern
    assert torch.allclose(zo.polynorm(z, (0.5, 0.25, 0.125, 3.0), 0.0), torch.tensor([[3.875, 2.625, 3.875, 2.625]]))
    h, w = torch.zeros(1, 3), torch.randn(4, 3)
    assert torch.allclose(zo.gate(torch.ones(1, 4), h, w, torch.full((4,), math.log(3.0))), torch.full((1, 4), 0.75))


def test_oracle_prefix_does_not_see_later_tokens():
    cfg = config([(attention(), FF), (attention(kv_from=0), None), (attention(heads=2, kv_heads=1), FF)])
    p = zo.random_params(cfg, 3)
    toks = [5, 1, 36, 7, 7, 20]
    full = zo.forward(cfg, p, toks)
    assert torch.allclose(full[:3], zo.forward(cfg, p, toks[:3]), atol=1e-5)
    assert not torch.allclose(full[3], full[4], atol=1e-2)        # same token, other position


# ---- registry and configuration ---------------------------------------------------------------------
def test_registry_picks_the_class_by_config():
    assert mi355_attn.model_class({"architecture": "Zuzelorn"}) is mi355_attn.ZuzelornLM
    assert mi355_attn.model_class({"d_model": 64}) is mi355_attn.CachedTransformerLM
    with pytest.raises(ValueError, match="unknown architecture"):
        mi355_attn.model_class({"architecture": "nothing"})


def test_float32_is_refused_for_a_model_that_has_no_such_path(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"vocab_size": 10}))
    with pytest.raises(mi355_attn.UnsupportedDtype):
        mi355_attn.load_model(str(tmp_path), dtype="float32")


def build(cfg, seed=1, **kw):
    return mi355_attn.ZuzelornLM(cfg, zo.random_params(cfg, seed), device="cpu", max_batch=2, **kw)


def test_weights_are_checked_against_the_configuration():
    cfg = config([(attention(), FF)])
    p = zo.random_params(cfg, 1)
    bad = dict(p)
    bad["l0.mix.q"] = p["l0.mix.q"][:-1]
    with pytest.raises(ValueError, match="l0.mix.q"):
        mi355_attn.ZuzelornLM(cfg, bad, device="cpu")
    del bad["l0.mix.q"]
    with pytest.raises(KeyError, match="l0.mix.q"):
        mi355_attn.ZuzelornLM(cfg, bad, device="cpu")
    for path, value in ((("type",), "other"), (("mlp", "kind"), "other")):
        c = json.loads(json.dumps(cfg))
        o = c["layers"][0]
        for key in path[:-1]:
            o = o[key]
        o[path[-1]] = value
        with pytest.raises(ValueError, match="other"):
            mi355_attn.ZuzelornLM(c, p, device="cpu")
    with pytest.raises(ValueError):
        build(cfg, dtype="float32", kv_dtype="bf16")
    with pytest.raises(ValueError):
        build(cfg, dtype="float16")


def test_projection_layout_pads_heads_and_folds_the_sign_of_a_heads_factor():
    cfg = config([(attention(), FF)])
    p = zo.random_params(cfg, 4)
    p["l0.mix.temp"] = torch.tensor([1.5, -0.75, 0.0, 2.0], dtype=torch.bfloat16)
    m = mi355_attn.ZuzelornLM(cfg, p, device="cpu", max_batch=2, dtype="float32")
    ly = m.layers[0]
    assert (ly["kd"], ly["vd"]) == (24, 16)
    mb = mi355_attn.ZuzelornLM(cfg, p, device="cpu", max_batch=2)
    lb = mb.layers[0]
    assert (lb["kd"], lb["vd"]) == (32, 32) and all(s % 8 == 0 for s in lb["starts"])
    h = torch.randn(5, 40)
    for mdl, l in ((m, ly), (mb, lb)):
        pr = h @ l["w_in"].float().T + l["b_in"].float()
        q = pr[:, :4 * l["kd"]].view(5, 4, l["kd"])
        want = (h @ p["l0.mix.q"].float().T + p["l0.mix.q.b"].float()).view(5, 4, 24) * torch.tensor([1.0, -1.0, 1.0, 1.0])[:, None]
        assert torch.allclose(q[..., :24], want, atol=1e-4) and bool((q[..., 24:] == 0).all())
        v = pr[:, l["starts"][2]:l["starts"][2] + 2 * l["vd"]].view(5, 2, l["vd"])
        assert torch.allclose(v[..., :16], (h @ p["l0.mix.v"].float().T + p["l0.mix.v.b"].float()).view(5, 2, 16), atol=1e-4)
        g = pr[:, l["starts"][-1]:l["starts"][-1] + 40]
        assert torch.allclose(g, h @ p["l0.rg1"].float().T, atol=1e-4)
        a = torch.randn(5, 4, 16)
        padded = torch.nn.functional.pad(a, (0, l["vd"] - 16)).reshape(5, -1)
        assert torch.allclose(padded @ l["wo"].float().T, a.reshape(5, -1) @ p["l0.mix.o"].float().T, atol=1e-4)
        scale = mdl.engine.layers[0].head_scale
        assert torch.allclose(scale, torch.tensor([1.5, 0.75, 1e-30, 2.0]))


# ---- cache geometry -------------------------------------------------------------------------------------
def test_cache_head_dims():
    assert cache_head_dims("bf16", 24, 24) == (32, 32, True)
    assert cache_head_dims("bf16", 64, 40) == (64, 64, True)
    assert cache_head_dims("bf16", 96, 128) == (128, 128, True)
    assert cache_head_dims("bf16", 130, 60) == (136, 64, False)
    assert cache_head_dims("fp32", 20, 33) == (24, 40, False)
    assert cache_head_dims("fp8", 16, 16) == (64, 64, True)
    for bad in (("fp8", 130, 16), ("bf16", 520, 8)):
        with pytest.raises(ValueError):
            cache_head_dims(*bad)


def test_layers_share_pools_and_bad_sharing_is_rejected():
    mk = lambda layers, **kw: PagedAttentionEngine(6, context_length=64, max_batch=2, device="cpu", layers=layers, **kw)
    L = lambda **kw: AttentionLayer(4, 2, 24, 16, rope=False, **kw)
    e = mk([L(), AttentionLayer(6, 3, 64, rope=False), L(kv_from=0), L(kv_from=0)], kv_dtype="bf16")
    assert e.k_caches[2] is e.k_caches[0] and e.v_caches[3] is e.v_caches[0] and e.k_caches[1] is not e.k_caches[0]
    assert tuple(e.k_caches[1].shape) == (6, 3, 16, 64) and e.shared == {0}
    e = mk([L(), L(kv_from=0)], kv_dtype="fp32")
    assert tuple(e.k_caches[0].shape) == (6, 2, 16, 24) and tuple(e.v_caches[1].shape) == (6, 2, 16, 16) and e.always_tables
    for bad in ([L(kv_from=0)], [L(), L(kv_from=1)], [L(), L(kv_from=0), L(kv_from=1)],
                [L(), AttentionLayer(4, 1, 24, 16, rope=False, kv_from=0)], [L(), AttentionLayer(4, 2, 80, 16, rope=False, kv_from=0)],
                [AttentionLayer(3, 2, 64, rope=False)], [AttentionLayer(4, 2, 24)]):
        with pytest.raises(ValueError):
            mk(bad)


def test_blocks_of_ended_requests_are_used_again():
    e = PagedAttentionEngine(4, context_length=64, max_batch=2, device="cpu", layers=[AttentionLayer(2, 1, 32, rope=False)])
    e.add_sequence(0)
    e.plan_prefill([0], [40])
    first = list(e.blocks[0])
    with pytest.raises(mi355_attn.OutOfBlocks):
        e.add_sequence(1)
        e.plan_prefill([1], [40])
    e.remove_sequence(0)
    plan = e.plan_prefill([1], [33])
    assert set(e.blocks[1]) <= set(range(4)) and set(e.blocks[1]) & set(first)
    assert plan.slots.tolist() == [e.blocks[1][t // 16] * 16 + t % 16 for t in range(33)]


# ---- trace replay and command line -----------------------------------------------------------------------
class FakeModel:
    """Logits row of a token = [sequence id, tokens so far, token]."""

    def __init__(self):
        self.lengths, self.next, self.freed = {}, 0, []

    def new_sequence(self):
        self.next += 1
        self.lengths[self.next] = 0
        return self.next

    def free_sequence(self, s):
        del self.lengths[s]
        self.freed.append(s)

    def step(self, sids, tokens, rows):
        out = []
        for s, ts in zip(sids, tokens):
            for t in ts:
                self.lengths[s] += 1
                out.append([float(s), float(self.lengths[s]), float(t)])
        return torch.tensor(out)[rows]


def test_replay_writes_wanted_rows_in_order_and_frees_ended_requests(tmp_path):
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [5, 6, 7], "want": [2, 0]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [8], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": [1, 2], "want": [1]}, {"id": "a", "tokens": [3], "want": [0]}], "end": ["b"]}]
    m, done = FakeModel(), []
    cli.replay(m, steps, str(tmp_path), done.append)
    read = lambda n: torch.frombuffer(bytearray((tmp_path / f"{n}.f32").read_bytes()), dtype=torch.float32).view(-1, 3).tolist()
    assert done == [0, 1, 2] and sorted(os.listdir(tmp_path)) == ["0.f32", "2.f32"]
    assert read(0) == [[1, 3, 7], [1, 1, 5]]
    assert read(2) == [[2, 2, 2], [3, 1, 3]]          # "a" after its end is a new sequence
    assert m.freed == [1, 2]
    with pytest.raises(ValueError):
        cli.replay(FakeModel(), [{"step": 0, "entries": [{"id": "a", "tokens": [5], "want": [1]}]}], str(tmp_path), done.append)


@pytest.mark.parametrize("tool", ["trace_run", "generate"])
def test_commands_answer_help(tool):
    res = subprocess.run([sys.executable, os.path.join(ROOT, "bin", tool), "--help"], capture_output=True, text=True, timeout=120)
    assert res.returncode == 0 and "--model" in res.stdout and os.access(os.path.join(ROOT, "bin", tool), os.X_OK)


def test_trace_run_ends_with_3_when_the_model_has_no_float32_path(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"vocab_size": 10}))
    res = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32",
                          "--out", str(tmp_path / "o"), "--max-tokens", "64"], capture_output=True, text=True, timeout=120, input="")
    assert res.returncode == 3


def test_serving_library_reports_what_it_lacks():
    from mi355_attn import _lib
    lib = _lib._ServingLib(mi355_attn.load())
    assert b"gfx950" in lib.mi355_version()
    lib.mi355_prefill_bwd.argtypes = []
    with pytest.raises(mi355_attn.LibraryMissing, match="mi355_prefill_bwd"):
        lib.mi355_prefill_bwd(None)


def test_operator_arguments_are_checked_on_the_host():
    f = torch.zeros(2, 8)
    with pytest.raises(ValueError):
        mi355_attn.dyt_residual(f, gate=f.bfloat16(), norm=(1.0, None, None))            # a gate without a sublayer result
    with pytest.raises(TypeError):
        mi355_attn.dyt_residual(f, f, norm=(1.0, None, None), out_dtype=torch.bfloat16)
    with pytest.raises(ValueError):
        mi355_attn.dyt_residual(f.bfloat16(), f)
    with pytest.raises(TypeError):
        mi355_attn.polynorm(f.half(), (1, 1, 1, 1), 1e-5)
    with pytest.raises(ValueError):
        mi355_attn.kv_cache_write(torch.zeros(1, 1, 8), torch.zeros(1, 1, 8), torch.zeros(1, 1, 16, 8), torch.zeros(2, 1, 16, 8),
                                  torch.zeros(1, dtype=torch.int64))
    with pytest.raises(ValueError):                                                     # CPU tensors never reach a kernel
        mi355_attn.polynorm(f, (1, 1, 1, 1), 1e-5)
    q, kc = torch.zeros(1, 2, 8), torch.zeros(1, 1, 16, 8)
    bt, cl = torch.zeros(1, 1, dtype=torch.int32), torch.ones(1, dtype=torch.int32)
    with pytest.raises(ValueError):
        mi355_attn.paged_attention_any(q, kc, kc, bt, cl, sinks=torch.zeros(3))
    with pytest.raises(ValueError):
        mi355_attn.paged_attention_any(q.bfloat16(), kc, kc, bt, cl)
    lib, z = mi355_attn.load(), None
    assert lib.mi355_paged_attn_any_fwd(z, z, z, z, 0, 0, 0, z, z, 0, 0, z, z, z, 1, 1, 1, 8, 8, 16, 1, 1.0, 2, z) == -1
    assert lib.mi355_kv_cache_write(z, z, z, z, z, 1, 1, 1, 8, 8, 8, 8, 2, z) == -1
    assert lib.mi355_polynorm_fwd(z, z, 1, 8, 8, 8, mi355_attn._lib.floats4((1, 1, 1, 1)), 1e-5, 0, z) == -1
    assert lib.mi355_embed_pos_fwd(z, z, z, z, z, 1, 8, 1, 1, 0, z) == -1
    assert lib.mi355_dyt_residual_fwd(z, z, z, z, 1.0, z, z, z, z, 1.0, z, z, z, 1, 8, 8, 8, 8, 0, z) == -1
