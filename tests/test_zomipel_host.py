"""Host logic around the Zomipel model, on the CPU: order of looped layers, registry and configuration, weight layout (stacked
projections, padded heads, turned pairs, experts), state slots, argument checks -- and the oracle itself against closed forms."""
import json
import math

import pytest
import torch

import mi355_attn
from mi355_attn.engine import AttentionLayer, PagedAttentionEngine, StateLayer
from mi355_attn.weights import pad_to, pair_halves
from mi355_attn.zomipel import layer_runs
from oracle import zomipel_oracle as zo


def attention(**kw):
    m = dict(heads=4, kv_heads=2, dim=24, vdim=16, scale=0.3, rot={"base": 50.0, "dims": 10}, mask={"size": 7, "keep_first": 2})
    m.update(kw)
    return {"type": "attention", "mixer": m}


def mamba(**kw):
    m = dict(heads=4, vdim=6, state=10, groups=2, norm_groups=3, conv=4)
    m.update(kw)
    return {"type": "mamba2", "mixer": m}


DENSE = {"kind": "dense", "ff": 44}
MOE = {"kind": "moe", "router": {"experts": 5, "top": 2}, "expert": {"ff": 20}, "shared": {"ff": 28}}


def config(*layers, **kw):
    c = dict(architecture="Zomipel", vocab=31, width=40, norm={"eps": 1e-4}, loop=None, layers=[dict(ly, mlp=f) for ly, f in layers])
    c.update(kw)
    return c


def build(cfg, seed=1, params=None, **kw):
    kw.setdefault("max_batch", 2)
    kw.setdefault("context_length", 64)
    return mi355_attn.ZomipelLM(cfg, params or zo.random_params(cfg, seed), device="cpu", **kw)


# ---- oracle ---------------------------------------------------------------------------------------------
def test_oracle_window_edges():
    """With equal scores the result is the mean over exactly the visible keys."""
    n, window, keep = 30, 6, 3
    q, k, v = torch.zeros(n, 2, 4), torch.randn(n, 1, 4), torch.eye(n)[:, None, :]
    out = zo.window_attention(q, k, v, 1.0, window, keep)
    for t in range(n):
        seen = sorted(set(range(max(0, t - window + 1), t + 1)) | set(range(min(keep, t + 1))))
        want = torch.zeros(n)
        want[seen] = 1.0 / len(seen)
        assert torch.allclose(out[t, 1], want, atol=1e-6), t
    assert torch.allclose(zo.window_attention(q[9:], k, v, 1.0, window, keep, first=9), out[9:], atol=1e-6)


def test_oracle_attention_without_window_equals_torch():
    q, k, v = torch.randn(9, 4, 8), torch.randn(9, 2, 8), torch.randn(9, 2, 6)
    kk, vv = (t.repeat_interleave(2, 1).transpose(0, 1) for t in (k, v))
    s = (q.transpose(0, 1) @ kk.transpose(1, 2)) * 0.4
    want = (torch.softmax(s.masked_fill(torch.ones(9, 9).triu(1).bool(), -math.inf), -1) @ vv).transpose(0, 1)
    for window, keep in ((None, 0), (9, 0), (1, 9), (4, 5)):
        got = zo.window_attention(q, k, v, 0.4, window, keep)
        assert torch.allclose(got, want, atol=1e-5) == (window != 4 or keep >= 9 - 4)


def test_oracle_rotation_keeps_relative_positions():
    q, k = torch.randn(12, dtype=torch.float64), torch.randn(12, dtype=torch.float64)
    dot = lambda a, b: float(zo.rotate(q, a, 20.0, 8) @ zo.rotate(k, b, 20.0, 8))
    assert abs(dot(7, 3) - dot(104, 100)) < 1e-9 and abs(dot(7, 3) - dot(7, 4)) > 1e-3
    turned = zo.rotate(q, 5, 20.0, 8)
    assert torch.equal(turned[8:], q[8:]) and torch.equal(zo.rotate(q, 0, 20.0, 8), q)
    z = torch.complex(q[1], q[5]) * torch.polar(torch.ones((), dtype=torch.float64), torch.tensor(5 * 20.0 ** -0.25, dtype=torch.float64))
    assert abs(turned[1] - z.real) < 1e-12 and abs(turned[5] - z.imag) < 1e-12


def test_oracle_state_equals_its_sum_over_tokens():
    """y_t = sum over s of exp(A (dt_(s+1) + .. + dt_t)) dt_s (C_t . B_s) x_s + D x_t."""
    T, H, P, G, N = 11, 4, 3, 2, 5
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    x, B, C, dt, A, D = r(T, H, P), r(T, G, N), r(T, G, N), r(T, H).abs(), -r(H).abs(), r(H)
    y, S = zo.selective_state(x, B, C, dt, A, D)
    for t in range(T):
        for h in range(H):
            want = D[h] * x[t, h]
            for s in range(t + 1):
                want = want + torch.exp(A[h] * dt[s + 1:t + 1, h].sum()) * dt[s, h] * (C[t, h // 2] @ B[s, h // 2]) * x[s, h]
            assert torch.allclose(y[t, h], want, atol=1e-10)
    y1, S1 = zo.selective_state(x[:4], B[:4], C[:4], dt[:4], A, D)
    y2, S2 = zo.selective_state(x[4:], B[4:], C[4:], dt[4:], A, D, S1)
    assert torch.allclose(torch.cat((y1, y2)), y, atol=1e-12) and torch.allclose(S2, S, atol=1e-12)


def test_oracle_convolution_and_norms():
    u, w, b = torch.randn(8, 3), torch.randn(3, 4), torch.randn(3)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(u.t()[None], (3, 0)), w[:, None], b, groups=3)[0].t()
    assert torch.allclose(zo.causal_conv_silu(u, w, b), torch.nn.functional.silu(want), atol=1e-5)
    assert torch.allclose(zo.causal_conv_silu(u[5:], w, b, history=u[2:5]), torch.nn.functional.silu(want)[5:], atol=1e-5)
    z, y = torch.full((1, 6), 40.0), torch.tensor([[3.0, -3.0, 3.0, 0.1, 0.1, -0.1]])       # silu(40) = 40; parts of equal size
    assert torch.allclose(zo.gated_group_norm(y, z, torch.ones(6), 2, 0.0), torch.sign(y), atol=1e-5)
    assert torch.allclose(zo.offset_rms_norm(torch.full((1, 4), -2.0), torch.tensor([0.0, 1.0, -1.0, 0.5]), 0.0),
                          torch.tensor([[-1.0, -2.0, 0.0, -1.5]]))


def test_oracle_router():
    chosen, w = zo.route(torch.zeros(3), torch.randn(4, 3), torch.log(torch.tensor([1.0, 6.0, 2.0, 0.5])), 2)
    assert chosen == [1, 2] and torch.allclose(w, torch.tensor([0.75, 0.25]))


def test_oracle_prefix_does_not_see_later_tokens():
    cfg = config((attention(), MOE), (mamba(), DENSE), loop={"start": 0, "stop": 2, "times": 2})
    p = zo.random_params(cfg, 3)
    a = zo.forward(cfg, p, [1, 2, 3, 4, 5, 6])
    b = zo.forward(cfg, p, [1, 2, 3, 9, 9])
    assert torch.allclose(a[:3], b[:3], atol=1e-5) and not torch.allclose(a[3], b[3], atol=1e-2)


# ---- order of layers -----------------------------------------------------------------------------------
def test_looped_layers():
    assert layer_runs(3, None) == ([0, 1, 2], set())
    assert layer_runs(4, {"start": 1, "stop": 3, "times": 3}) == ([0, 1, 2, 1, 2, 1, 2, 3], {3, 5})
    assert layer_runs(2, {"start": 0, "stop": 2, "times": 1}) == ([0, 1], set())
    for bad in ({"start": 1, "stop": 1, "times": 2}, {"start": 0, "stop": 3, "times": 2}, {"start": 0, "stop": 2, "times": 0}):
        with pytest.raises(ValueError):
            layer_runs(2, bad)
    for case in (None, {"start": 1, "stop": 3, "times": 3}, {"start": 0, "stop": 4, "times": 2}, {"start": 3, "stop": 4, "times": 4}):
        order, again = zo.layer_runs({"layers": [0] * 4, "loop": case})
        assert layer_runs(4, case) == (order, set(again))


def test_every_pass_has_a_cache_or_state_of_its_own_and_shares_weights():
    m = build(config((attention(), DENSE), (mamba(), None), loop={"start": 0, "stop": 2, "times": 2}))
    e = m.engine
    assert e.num_layers == 4 and m.runs[0] is m.runs[2] and m.runs[1] is m.runs[3] and m.again == {2}
    assert e.k_caches[0] is not e.k_caches[2] and e.k_caches[1] is None and sorted(e.ssm_states) == [1, 3]
    assert e.ssm_states[1].data_ptr() != e.ssm_states[3].data_ptr() and e.layers[1].params["conv"] is e.layers[3].params["conv"]


# ---- registry and configuration ------------------------------------------------------------------------------
def test_registry_picks_the_class_by_config():
    assert mi355_attn.model_class({"architecture": "Zomipel"}) is mi355_attn.ZomipelLM


def test_weights_and_configuration_are_checked():
    cfg = config((attention(), MOE), (mamba(), DENSE))
    p = zo.random_params(cfg, 1)
    for name in ("l0.mix.k.b", "l0.mlp.e3.down", "l0.mlp.shared.sg", "l1.mix.conv", "l1.mix.A_log", "l1.mlp.up", "final.norm"):
        bad = dict(p)
        bad[name] = p[name][:-1]
        with pytest.raises(ValueError, match=name.replace(".", r"\.")):
            build(cfg, params=bad)
        del bad[name]
        with pytest.raises(KeyError, match=name.replace(".", r"\.")):
            build(cfg, params=bad)
    for edit in (lambda c: c["layers"][0].update(type="other"), lambda c: c["layers"][1]["mlp"].update(kind="other")):
        c = json.loads(json.dumps(cfg))
        edit(c)
        with pytest.raises(ValueError, match="other"):
            build(c, params=p)
    for kw in (dict(dtype="float32", kv_dtype="bf16"), dict(kv_dtype="fp32"), dict(dtype="float16")):
        with pytest.raises(ValueError):
            build(cfg, **kw)


def test_what_the_configuration_says_reaches_the_engine():
    m = build(config((attention(), None), (mamba(), None)))
    a, s = m.engine.layers
    assert (a.n_q_heads, a.n_kv_heads, a.head_dim, a.v_dim, a.softmax_scale) == (4, 2, 24, 16, 0.3)
    assert (a.rope, a.rope_base, a.rope_dims, a.window, a.keep_first) == (True, 50.0, 10, 7, 2)
    assert (s.heads, s.vdim, s.state, s.groups, s.taps, s.channels) == (4, 6, 10, 2, 4, 24 + 40)
    assert not build(config((attention(rot={"base": 50.0, "dims": 0}), None))).engine.layers[0].rope


# ---- weight layout ---------------------------------------------------------------------------------------------
def test_pairs_are_adjacent_and_scores_stay():
    heads, size, dims = 3, 14, 8
    w = torch.arange(heads * size, dtype=torch.float32)
    got = pair_halves(w, heads, size, dims).view(heads, size)
    assert got[1].tolist() == [14 + i for i in (0, 4, 1, 5, 2, 6, 3, 7, 8, 9, 10, 11, 12, 13)]
    assert pair_halves(w, heads, size, 0).equal(w)
    assert pad_to(torch.ones(3, 5), 1, 4).tolist() == [[1.0] * 5 + [0.0] * 3] * 3 and pad_to(w, 0, 1) is w


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_attention_layer_layout(dtype):
    cfg = config((attention(), DENSE))
    p = zo.random_params(cfg, 4)
    m = build(cfg, params=p, dtype=dtype)
    ly = m.runs[0]
    kd, vd = ly["kd"], ly["vd"]
    assert (kd, vd) == ((32, 32) if dtype == "bfloat16" else (24, 16)) and all(a % 8 == 0 for a in ly["at"] + ly["ff_at"] + ly["out_at"])
    h = torch.randn(5, 40)
    pr = h @ ly["w_in"].float().T + ly["b_in"].float()
    order = [0, 5, 1, 6, 2, 7, 3, 8, 4, 9] + list(range(10, 24))                           # ten turned entries, pairs adjacent
    for at, name, heads, size, to, order in ((0, "q", 4, 24, kd, order), (ly["at"][1], "k", 2, 24, kd, order),
                                             (ly["at"][2], "v", 2, 16, vd, list(range(16)))):
        got = pr[:, at:at + heads * to].view(5, heads, to)
        want = (h @ p[f"l0.mix.{name}"].float().T + p[f"l0.mix.{name}.b"].float()).view(5, heads, size)[..., order]
        assert torch.allclose(got[..., :size], want, atol=1e-4) and bool((got[..., size:] == 0).all())
    up = pr[:, ly["ff_at"][0]:ly["ff_at"][0] + 44]
    assert torch.allclose(up, h @ p["l0.mlp.up"].float().T, atol=1e-4)
    a, f = torch.randn(5, 4, 16), torch.randn(5, 44)
    rows = torch.zeros(5, ly["w_out"].shape[1])
    rows[:, :4 * vd] = torch.nn.functional.pad(a, (0, vd - 16)).flatten(1)
    rows[:, ly["out_at"][1]:ly["out_at"][1] + 44] = f
    want = a.flatten(1) @ p["l0.mix.o"].float().T + f @ p["l0.mlp.down"].float().T
    assert torch.allclose(rows @ ly["w_out"].float().T, want, atol=1e-4)


def test_mamba_layer_layout():
    cfg = config((mamba(), MOE))
    p = zo.random_params(cfg, 4)
    m = build(cfg, params=p)
    ly, st = m.runs[0], m.engine.layers[0]
    h = torch.randn(5, 40)
    pr, want = h @ ly["w_in"].float().T, h @ p["l0.mix.in"].float().T
    for at, (a, b) in zip([0, ly["at"][1], ly["at"][2]], ((0, 24), (24, 88), (88, 92))):
        assert at % 8 == 0 and torch.allclose(pr[:, at:at + b - a], want[:, a:b], atol=1e-4)
    assert torch.equal(st.params["conv"], p["l0.mix.conv"].float().t()) and st.params["conv"].is_contiguous()
    assert torch.allclose(st.params["neg_a"], -torch.exp(p["l0.mix.A_log"].float()))
    for at, part in zip(ly["ff_at"], ("gate", "up")):
        assert torch.allclose(pr[:, at:at + 28], h @ p[f"l0.mlp.shared.{part}"].float().T, atol=1e-4)
    moe = ly["moe"]
    assert moe["router"].shape == (6, 64) and bool((moe["router"][:, 40:] == 0).all()) and m.h_cols == 64       # the gate's row is the last
    assert torch.equal(moe["router"][5, :40], p["l0.mlp.shared.sg"][0]) and float(moe["bias"][5]) == 0.0
    assert moe["gate_up"].shape == (5, 128, 64) and moe["down"].shape == (5, 40, 64)
    for e in range(5):
        for half, part in ((0, "gate"), (64, "up")):
            got = moe["gate_up"][e, half:half + 64]
            assert torch.equal(got[:20, :40], p[f"l0.mlp.e{e}.{part}"]) and int((got != 0).sum()) == int((got[:20, :40] != 0).sum())
        assert torch.equal(moe["down"][e, :, :20], p[f"l0.mlp.e{e}.down"]) and bool((moe["down"][e, :, 20:] == 0).all())
    f = build(cfg, params=p, dtype="float32").runs[0]["moe"]
    assert f["gate_up"].shape == (5, 40, 40) and f["down"].shape == (5, 40, 20)


# ---- state slots ---------------------------------------------------------------------------------------------------
def test_state_slots_are_given_back_and_used_again():
    layers = [StateLayer(2, 6, 4, 1, 3, {}), AttentionLayer(2, 1, 32, rope=False, window=5, keep_first=1)]
    e = PagedAttentionEngine(8, context_length=64, max_batch=2, device="cpu", layers=layers)
    assert tuple(e.conv_states[0].shape) == (2, 3, 20) and tuple(e.ssm_states[0].shape) == (2, 2, 4, 8) and e.ssm_states[0].dtype == torch.float32
    e.add_sequence(5)
    e.add_sequence(9)
    assert sorted(e.state_slots.values()) == [0, 1]
    with pytest.raises(mi355_attn.OutOfBlocks):
        e.add_sequence(10)
    assert 10 not in e.blocks                                             # a refused sequence leaves nothing behind
    plan = e.plan_prefill([9, 5], [3, 2])
    assert plan.state_slots.tolist() == [e.state_slots[9], e.state_slots[5]] and plan.positions.tolist() == [0, 1, 2, 0, 1]
    assert e.plan_decode([5]).state_slots.tolist() == [e.state_slots[5]]
    slot = e.state_slots[9]
    e.remove_sequence(9)
    e.add_sequence(10)
    assert e.state_slots[10] == slot and e.plan_prefill([10], [4]).positions.tolist() == [0, 1, 2, 3]
    assert not PagedAttentionEngine(8, context_length=64, max_batch=2, device="cpu", layers=layers[1:]).state_slots
    with pytest.raises(ValueError):
        PagedAttentionEngine(8, context_length=64, device="cpu", layers=[AttentionLayer(2, 1, 32, rope=False, window=-1)])
    with pytest.raises(ValueError):                                       # keys of a state layer cannot be shared
        PagedAttentionEngine(8, context_length=64, device="cpu", layers=[layers[0], AttentionLayer(2, 1, 32, rope=False, kv_from=0)])


# ---- argument checks -----------------------------------------------------------------------------------------------------
def test_operator_arguments_are_checked_on_the_host():
    f, b = torch.zeros(2, 64), torch.zeros(2, 64, dtype=torch.bfloat16)
    ids, wt = torch.zeros(2, 1, dtype=torch.int32), torch.ones(2, 1)
    for call in (lambda: mi355_attn.residual_rms(f, f[0]), lambda: mi355_attn.ff_act(b), lambda: mi355_attn.gated_norm(b, b, f[0], 1, 1e-5),
                 lambda: mi355_attn.gated_norm(b, b, f[0], 3, 1e-5), lambda: mi355_attn.moe_route(b, b, f[0, :2], 1),
                 lambda: mi355_attn.moe_experts(b, ids, wt, torch.zeros(1, 128, 64).bfloat16(), torch.zeros(1, 64, 64).bfloat16())):
        with pytest.raises((ValueError, TypeError)):                      # CPU tensors never reach a kernel
            call()
    lib, z = mi355_attn.load(), None
    assert lib.mi355_moe_route(z, z, z, z, z, z, 1, 64, 64, 64, 4, 1, 0, z) == -1
    assert lib.mi355_moe_group(z, 1, 4, z, z, z) == -1
    assert lib.mi355_ssm_decode(z, z) == -1 and lib.mi355_ssm_prefill(z, 0, z) == -1
