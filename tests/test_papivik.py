"""Papivik through the engine (scheduler, block manager, sequence slots, runner, ops) against
the plain float64 oracle of tests/papivik_oracle.py, on the CPU branch of the ops (the HIP
kernels are compared with these ops, and run the same engine suite, in test_papivik_gpu.py).
Small configurations with random weights; fp32 runs are compared tightly (a lost state, a stale
convolution input, a wrong key or a normaliser that starts elsewhere moves a logit by far more
than the tolerance), bf16 runs loosely."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import papivik_oracle as oracle
from bidetar_harness import engine, rel_err, replay, tokens, write_model
from aws_k8s_ansible_provisioner_amd.models.config import get_config
from aws_k8s_ansible_provisioner_amd.ops import stream as sops

FP32_TOL = 3e-4
F64 = torch.float64
REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def base_config():
    """Unequal layers: all three mixers (two of them twice, with other sizes), grouped and
    ungrouped heads, partial and full rotation, unequal convolutions, key and value sizes that
    differ, feed-forwards present and absent."""
    layers = [
        oracle.parallel_layer((4, 2, 8, 6), (4, 2, 6, 10), 0.5, 4, base=50.0, conv=(3, 4),
                              scales=(1.4, 0.7), ff=40),
        oracle.mlstm_layer(3, 6, 10, cap=7.0),
        oracle.lightning_layer(2, 7, 9, (0.8, 0.99), ff=24),
        oracle.parallel_layer((3, 3, 6, 6), (2, 2, 9, 5), 0.9, 6, base=900.0, conv=(4, 2),
                              scales=(0.6, 1.3)),
        oracle.mlstm_layer(2, 8, 4, cap=20.0, ff=16),
        oracle.lightning_layer(3, 4, 6, (1.0, 0.5, 0.95)),
    ]
    return oracle.make_config(width=36, vocab=47, layers=layers, embed_scale=0.7)


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    cfg = base_config()
    W = oracle.random_weights(cfg, seed=2)
    return cfg, W, write_model(tmp_path_factory.mktemp("papivik"), cfg, W)


@pytest.fixture(scope="module")
def reference(model):
    cfg, W, _ = model
    W64 = oracle.as_f64(W)
    reqs = {"a": tokens(75, cfg["vocab"], 1), "b": tokens(41, cfg["vocab"], 2),
            "c": tokens(23, cfg["vocab"], 3), "d": tokens(1, cfg["vocab"], 4),
            "e": tokens(64, cfg["vocab"], 5)}
    return reqs, {n: oracle.forward(cfg, W64, t)[0] for n, t in reqs.items()}


def check(got, want, names=None, tol=FP32_TOL):
    for n in names or got:
        e = rel_err(got[n], want[n])
        assert e.max().item() < tol, f"{n}: position {int(e.argmax())} off by {e.max().item():.2e}"


# ------------------------------------------------------------------ configuration, weights
def test_config_reader(model):
    cfg, W, path = model
    c = get_config(path)
    assert c.arch == "papivik" and c.embed_scale == 0.7 and not c.tie_embeddings
    assert [ls.type for ls in c.layer_specs] == ["parallel", "mlstm", "lightning", "parallel",
                                                 "mlstm", "lightning"]
    p = c.layer_specs[0].mixer
    a, r = p.left, p.right
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.conv) == (4, 2, 8, 6, 0.5, 3)
    assert (a.rot.dims, a.rot.base, a.rot.layout) == (4, 50.0, "half")
    assert a.head_norm and a.qk_norm_w and not (a.sink or a.gate or a.bias or a.shared_kv)
    assert (r.heads, r.qk_heads, r.dim, r.vdim, r.conv) == (4, 2, 6, 10, 4)
    assert (p.combine, p.left_scale, p.right_scale) == ("scale", 1.4, 0.7)
    m = c.layer_specs[1].mixer
    assert (m.heads, m.dim, m.vdim, m.cap) == (3, 6, 10, 7.0) and c.layer_specs[1].mlp is None
    t = c.layer_specs[2].mixer
    assert (t.heads, t.dim, t.vdim, t.decay) == (2, 7, 9, (0.8, 0.99))
    assert (t.act, t.k_scaled, t.out_norm, t.gate) == ("silu", False, "all", "sigmoid")
    assert c.layer_specs[0].mlp.act == "gelu" and c.layer_specs[0].mlp.ff == 40
    assert c.num_params() == sum(x.numel() for x in W.values())
    assert c.kv_bytes_per_token() == 2 * (2 * (8 + 6) + 3 * (6 + 6))


def test_config_reader_refuses_what_it_does_not_know(model):
    from aws_k8s_ansible_provisioner_amd.models.config import papivik_config

    for change in (lambda c: c["layers"][1].update(type="retention"),
                   lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3),
                   lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=10),
                   lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=3),
                   lambda c: c["layers"][0]["mixer"]["left"].update(conv=0),
                   lambda c: c["layers"][0]["mixer"]["right"].update(kv_heads=3),
                   lambda c: c["layers"][2]["mixer"].update(decay=[0.5]),
                   lambda c: c["layers"][2]["mixer"].update(decay=[0.5, 1.5]),
                   lambda c: c["layers"][0]["mlp"].update(kind="moe")):
        bad = copy.deepcopy(model[0])
        change(bad)
        with pytest.raises(ValueError):
            papivik_config("bad", bad)


def test_weights_round_trip(model):
    from aws_k8s_ansible_provisioner_amd.models.papivik import PapivikLM

    cfg, W, path = model
    m = PapivikLM(get_config(path), "cpu", dtype=torch.float32, max_model_len=64)
    m.load_state_dict(W)
    sd = m.state_dict()
    assert set(sd) == set(W)
    for k, t in W.items():
        assert tuple(sd[k].shape) == tuple(t.shape), k
        torch.testing.assert_close(sd[k].float(), t.float(), rtol=0, atol=0)
    assert m.weight_bytes() >= 4 * sum(t.numel() for t in W.values())
    bad = dict(W)
    bad["l1.mix.i.b"] = torch.zeros(2)
    with pytest.raises(ValueError):
        m.load_state_dict(bad)
    del bad["l1.mix.i.b"]
    with pytest.raises(KeyError):
        m.load_state_dict(bad)


def test_state_sizes(model):
    from aws_k8s_ansible_provisioner_amd.models.papivik import PapivikLM

    m = PapivikLM(get_config(model[2]), "cpu", dtype=torch.float32, max_model_len=64)
    m.allocate_state(3)
    n = sum(t[0].numel() * 4 for st in m.state for t in st)
    assert m.state_bytes_per_slot() == n
    assert all(t.shape[0] == 3 for st in m.state for t in st)


# ------------------------------------------------------------------ mechanisms alone
def test_post_norm_and_stream_copy():
    g = torch.Generator().manual_seed(0)
    x0, y = torch.randn(5, 24, generator=g), 3 * torch.randn(5, 24, generator=g)
    w, nw = torch.randn(24, generator=g), torch.randn(24, generator=g)
    want = x0.to(F64) + oracle.rms(y.to(F64), 1e-2) * w.to(F64)
    for nxt in (None, nw):
        x, out = x0.clone(), torch.zeros(5, 24)
        sops.stream_post_norm_add_norm(x, y, None, None, None, w, nxt, 1e-2, out)
        torch.testing.assert_close(x.to(F64), want, rtol=1e-5, atol=1e-5)
        exp = want if nxt is None else oracle.rms(want, 1e-2) * nw.to(F64)
        torch.testing.assert_close(out.to(F64), exp, rtol=1e-5, atol=1e-5)


def test_gelu():
    x = torch.linspace(-9, 9, 91).view(7, 13)
    out = torch.zeros(7, 13)
    sops.gelu_tanh(x, out)
    torch.testing.assert_close(out.to(F64), oracle.gelu_tanh(x.to(F64)), rtol=1e-5, atol=1e-6)


@pytest.mark.parametrize("rot_dims", [0, 4, 8])
def test_head_norm_rotation_and_cache(rot_dims):
    g = torch.Generator().manual_seed(rot_dims)
    T, H, G, D, Dv, BS = 8, 4, 2, 8, 6, 8
    N = H * D + G * (D + Dv) + 3
    proj = torch.randn(T, N, generator=g)
    qw, kw = torch.randn(D, generator=g), torch.randn(D, generator=g)
    slots = torch.tensor([8, 9, 10, 11, 3, -1, 17, 0])
    pos = torch.arange(T)
    cs = sops.rotary_table(64, rot_dims, 30.0) if rot_dims else None
    q, kc, vc = torch.zeros(T, H, D), torch.zeros(3, G, BS, D), torch.zeros(3, G, 1, Dv, 8)
    sops.head_norm_cache(proj, q, kc, vc, slots, H, G, D, Dv, 0, H * D, (H + G) * D, 1e-3, True,
                         False, qw, kw, cs, pos)
    p, rot = proj.to(F64), {"dims": rot_dims, "base": 30.0}
    wq = oracle.rotate_half(oracle.rms(p[:, :H * D].reshape(T, H, D), 1e-3) * qw.to(F64), rot)
    wk = oracle.rotate_half(oracle.rms(p[:, H * D:(H + G) * D].reshape(T, G, D), 1e-3)
                            * kw.to(F64), rot)
    torch.testing.assert_close(q.to(F64), wq, rtol=1e-5, atol=1e-5)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            torch.testing.assert_close(kc[s // BS, :, s % BS].to(F64), wk[t], rtol=1e-5, atol=1e-5)
            want = p[t, (H + G) * D:(H + G) * D + G * Dv].reshape(G, Dv)
            torch.testing.assert_close(vc[s // BS, :, 0, :, s % 8].to(F64), want)


def steps_of(cuts, slot=0):
    """(tensors of one step) per portion of one sequence: rows, slots, positions, q_start."""
    out, lo = [], 0
    for n in cuts:
        out.append((slice(lo, lo + n), torch.full((n,), slot, dtype=torch.int32),
                    torch.arange(lo, lo + n),
                    torch.tensor([0, n], dtype=torch.int32) if n > 1 else None))
        lo += n
    return out


CUTS = [[29], [1] * 29, [2, 3, 1, 7, 2, 14], [16, 13]]


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("taps,silu_from", [(4, 0), (3, 5), (1, 2), (2, 12)])
def test_convolution(cuts, taps, silu_from):
    g = torch.Generator().manual_seed(taps)
    C, N = 12, 16
    proj, cw = torch.randn(29, N, generator=g), torch.randn(C, taps, generator=g)
    want = oracle.causal_conv(proj[:, 3:3 + C].to(F64), cw.to(F64))
    want[:, silu_from:] = oracle.silu(want[:, silu_from:])
    state = torch.full((2, taps - 1, C), 5.0)       # stale contents of an earlier sequence
    for rows, slot, pos, qs in steps_of(cuts):
        out = torch.zeros(rows.stop - rows.start, C)
        sops.conv_silu(out, proj[rows], 3, cw, None, state, slot, pos, qs, silu_from)
        torch.testing.assert_close(out.to(F64), want[rows], rtol=1e-5, atol=1e-5)


def run_memory(cuts, proj, H, D, V, cap, ib, fb, nw, eps, state):
    outs = []
    o = [0, H * D, 2 * H * D, 2 * H * D + H * V, 2 * H * (D + V), 2 * H * (D + V) + H]
    for rows, slot, pos, qs in steps_of(cuts):
        out = torch.zeros(rows.stop - rows.start, H * V)
        sops.matrix_memory(out, proj[rows], *o, ib, fb, cap, state, nw, slot, pos, qs, H, D, V,
                           eps)
        outs.append(out)
    return torch.cat(outs)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("shift", [0.0, -9.0, 8.0])
def test_matrix_memory(cuts, shift):
    """shift moves the input gates: far below zero the running maximum falls from its start at
    zero only as fast as the forget gates let it, and the floor e^(-m) decides the divisor."""
    g = torch.Generator().manual_seed(7)
    H, D, V, cap, eps = 3, 5, 7, 12.0, 1e-4
    proj = torch.randn(29, 2 * H * (D + V) + 2 * H, generator=g)
    ib, fb = torch.randn(H, generator=g) + shift, torch.randn(H, generator=g) + 2
    nw = torch.randn(H * V, generator=g)
    p = proj.to(F64)
    q = p[:, :H * D].view(29, H, D) * D ** -0.5
    k, v = p[:, H * D:2 * H * D].view(29, H, D), p[:, 2 * H * D:2 * H * D + H * V].view(29, H, V)
    gate = p[:, 2 * H * D + H * V:2 * H * (D + V)]
    ig = cap * torch.tanh((p[:, -2 * H:-H] + ib) / cap)
    fg = oracle.log_sigmoid(cap * torch.tanh((p[:, -H:] + fb) / cap))
    o, (S, n, m) = oracle.mlstm_scan(q, k, v, ig, fg)
    want = oracle.rms(o, eps).reshape(29, H * V) * nw * oracle.sigmoid(gate)
    st = (torch.full((1, H, V, D), 3.0), torch.full((1, H, D), 3.0), torch.full((1, H), 3.0))
    got = run_memory(cuts, proj, H, D, V, cap, ib, fb, nw, eps, st)
    torch.testing.assert_close(got.to(F64), want, rtol=1e-4, atol=1e-5)
    torch.testing.assert_close(st[0][0].transpose(1, 2).to(F64), S, rtol=1e-4, atol=1e-5)
    torch.testing.assert_close(st[1][0].to(F64), n, rtol=1e-4, atol=1e-5)
    torch.testing.assert_close(st[2][0].to(F64), m, rtol=1e-4, atol=1e-5)


def test_matrix_memory_starts_its_maximum_at_zero():
    """One token with a closed input gate: with m = max(f + 0, i) the divisor's floor is e^(-m),
    far above |n . q|; a maximum that starts at minus infinity would give another output scale
    (seen through eps)."""
    q, k, v = (torch.ones(1, 1, 4, dtype=F64) for _ in range(3))
    i, f = torch.full((1, 1), -6.0, dtype=F64), torch.full((1, 1), -0.5, dtype=F64)
    o, (_, n, m) = oracle.mlstm_scan(q, k, v, i, f)
    assert m.item() == -0.5 and abs(n[0, 0].item() - np.exp(-5.5)) < 1e-12
    assert abs(o[0, 0, 0].item() - 4 * np.exp(-5.5) / (np.exp(0.5) + 1e-6)) < 1e-9


@pytest.mark.parametrize("cuts", CUTS)
def test_linear_attention(cuts):
    g = torch.Generator().manual_seed(9)
    H, D, V, eps = 3, 6, 5, 1e-4
    proj, nw = torch.randn(29, 2 * H * (D + V), generator=g), torch.randn(H * V, generator=g)
    decay = torch.tensor([1.0, 0.5, 0.97])
    p = oracle.silu(proj.to(F64))
    q, k = p[:, :H * D].view(29, H, D), p[:, H * D:2 * H * D].view(29, H, D)
    v = p[:, 2 * H * D:2 * H * D + H * V].view(29, H, V)
    o, S = oracle.decay_scan(q, k, v, decay.to(F64))
    gate = oracle.sigmoid(proj[:, 2 * H * D + H * V:].to(F64))
    want = oracle.rms(o.reshape(29, H * V), eps) * nw * gate
    st = torch.full((1, H, V, D), 3.0)
    outs = []
    for rows, slot, pos, qs in steps_of(cuts):
        out = torch.zeros(rows.stop - rows.start, H * V)
        sops.linear_attention(out, proj[rows], 0, H * D, 2 * H * D, 2 * H * D + H * V, decay, st,
                              nw, slot, pos, qs, H, D, V, eps)
        outs.append(out)
    torch.testing.assert_close(torch.cat(outs).to(F64), want, rtol=1e-4, atol=1e-5)
    torch.testing.assert_close(st[0].transpose(1, 2).to(F64), S, rtol=1e-4, atol=1e-5)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("H,G", [(4, 2), (3, 1), (2, 2)])
def test_gated_delta(cuts, H, G):
    g = torch.Generator().manual_seed(H)
    D, V, eps = 6, 5, 1e-4
    qkv = torch.randn(29, 2 * G * D + H * V, generator=g)
    qkv[11, G * D:2 * G * D] *= 40                  # a key whose length matters
    proj = torch.randn(29, H * V + 2 * H, generator=g)
    al, db = torch.randn(H, generator=g), torch.randn(H, generator=g) - 1
    nw = torch.randn(H * V, generator=g)
    p = qkv.to(F64)
    of = [h // (H // G) for h in range(H)]
    q = oracle.unit(p[:, :G * D].view(29, G, D))[:, of] * D ** -0.5
    k = oracle.unit(p[:, G * D:2 * G * D].view(29, G, D))[:, of]
    v = p[:, 2 * G * D:].view(29, H, V)
    b, a = proj[:, H * V:H * V + H].to(F64), proj[:, H * V + H:].to(F64)
    dec = torch.exp(-torch.exp(al.to(F64)) * oracle.softplus(a + db.to(F64)))
    o, S = oracle.delta_scan(q, k, v, oracle.sigmoid(b), dec)
    want = oracle.rms(o, eps).reshape(29, H * V) * nw * oracle.silu(proj[:, :H * V].to(F64))
    st = torch.full((1, H, V, D), 3.0)
    outs = []
    for rows, slot, pos, qs in steps_of(cuts):
        out = torch.zeros(rows.stop - rows.start, H * V)
        sops.gated_delta(out, qkv[rows], 0, G * D, 2 * G * D, proj[rows], 0, H * V, H * V + H, al,
                         db, st, nw, slot, pos, qs, H, G, D, V, eps)
        outs.append(out)
    torch.testing.assert_close(torch.cat(outs).to(F64), want, rtol=1e-4, atol=1e-5)
    torch.testing.assert_close(st[0].transpose(1, 2).to(F64), S, rtol=1e-4, atol=1e-5)
    # the read-out sees the current token's write: without it the first output is zero
    assert want[0].abs().max() > 0.01


def test_norm_gate_divides_before_the_norm():
    g = torch.Generator().manual_seed(1)
    y, gate = torch.randn(4, 12, generator=g), torch.randn(4, 12, generator=g)
    w = torch.randn(12, generator=g)
    den, floor = 50 * torch.randn(4, 3, generator=g), torch.rand(4, 3, generator=g)
    for act, f in (("sigmoid", oracle.sigmoid), ("silu", oracle.silu)):
        out = torch.zeros(4, 12)
        sops.norm_gate(out, y, gate, w, 3, 1e-2, act, den, floor)
        d = torch.maximum(den.abs(), floor).to(F64) + 1e-6
        want = oracle.rms(y.to(F64).view(4, 3, 4) / d[:, :, None], 1e-2).reshape(4, 12) * w \
            * f(gate.to(F64))
        torch.testing.assert_close(out.to(F64), want, rtol=1e-5, atol=1e-6)


# ------------------------------------------------------------------ the engine
def test_whole_prompts(model, reference):
    reqs, want = reference
    eng = engine(model[2], max_tokens=256)
    check(replay(eng, reqs, [[(n, len(t))] for n, t in reqs.items()]), want)


def test_token_by_token(model, reference):
    reqs, want = reference
    eng = engine(model[2], max_tokens=128)
    sub = {n: reqs[n] for n in ("c", "d", "b")}
    check(replay(eng, sub, [[(n, 1)] for n in sub for _ in range(len(sub[n]))]), want)


@pytest.mark.parametrize("sizes", [[2], [3, 5], [31, 2, 33], [32], [1, 2, 40, 7]])
def test_portions(model, reference, sizes):
    reqs, want = reference
    eng = engine(model[2], max_tokens=128)
    sched, i = [], 0
    for n in ("a", "b"):
        left = len(reqs[n])
        while left:
            c = min(left, sizes[i % len(sizes)])
            sched.append([(n, c)])
            left -= c
            i += 1
    check(replay(eng, {n: reqs[n] for n in ("a", "b")}, sched), want)


def test_unequal_batches_and_reuse(model, reference):
    """Portions beside single tokens, requests left out of steps, and a pool of six pages and
    three slots that seven requests use in turn (stale states and keys underneath)."""
    reqs, want = reference
    reqs = dict(reqs, f=reqs["c"][:], g=reqs["b"][:])
    want = dict(want, f=want["c"], g=want["b"])
    eng = engine(model[2], max_tokens=192, max_seqs=3)
    left = {n: len(t) for n, t in reqs.items()}
    rng = np.random.default_rng(5)
    live, waiting, sched = [], list(reqs), []
    while waiting or live:
        while waiting and len(live) < 3 and (waiting[0] != "e" or not live):
            live.append(waiting.pop(0))
            if sum(-(-len(reqs[x]) // 32) for x in live) > 6:
                waiting.insert(0, live.pop())
                break
        step = []
        for n in list(live):
            if len(live) > 1 and rng.random() < 0.2:
                continue
            c = min(left[n], int(rng.choice([1, 1, 2, 3, 17])))
            step.append((n, c))
            left[n] -= c
            if not left[n]:
                live.remove(n)
        if step:
            sched.append(step)
    check(replay(eng, reqs, sched), want)


def test_long_decode(model):
    cfg, W, path = model
    t = tokens(150, cfg["vocab"], 11)
    want = {"x": oracle.forward(cfg, oracle.as_f64(W), t)[0]}
    eng = engine(path, max_tokens=160)
    check(replay(eng, {"x": t}, [[("x", 5)]] + [[("x", 1)]] * 145), want, tol=1e-3)


def test_bf16_stays_near(model, reference):
    reqs, want = reference
    eng = engine(model[2], dtype="bfloat16", max_tokens=256)
    got = replay(eng, reqs, [[(n, len(t))] for n, t in reqs.items()])
    for n in reqs:
        assert rel_err(got[n], want[n]).median().item() < 0.2, n


def test_far_key_stands_out(tmp_path):
    """One attention layer whose query at the last position matches its own key and that of ONE
    equal token far back; the values' convolution takes the token before, so the two bring
    different values: leaving the far key out moves the logits."""
    cfg = oracle.make_config(24, 40, [oracle.parallel_layer((2, 1, 8, 8), (1, 1, 4, 4), 4.0, 0,
                                                            conv=(2, 1), scales=(1.0, 0.05))])
    W = oracle.random_weights(cfg, seed=4)
    for n, taps in (("q", [0.0, 1.0]), ("k", [0.0, 1.0]), ("v", [1.0, 0.0])):
        rows = W[f"l0.mix.left.{n}.conv"].shape[0]
        W[f"l0.mix.left.{n}.conv"] = torch.tensor([taps] * rows, dtype=torch.bfloat16)
    W["l0.mix.left.q"][8:] = W["l0.mix.left.q"][:8]
    W["l0.mix.left.k"] = W["l0.mix.left.q"][:8].clone()
    for n in ("q.norm", "k.norm"):
        W["l0.mix.left." + n] = torch.full((8,), 1.5, dtype=torch.bfloat16)
    path = write_model(tmp_path / "far", cfg, W)
    filler = [t for t in tokens(200, 40, 3) if t != 7][:120]
    t = filler[:3] + [7] + filler[3:] + [7]
    lost = filler[:3] + [filler[3]] + filler[3:] + [7]
    W64 = oracle.as_f64(W)
    want = oracle.forward(cfg, W64, t)[0]
    assert rel_err(oracle.forward(cfg, W64, lost)[0][-1:], want[-1:]).item() > 0.05
    for cuts in ([len(t)], [60, 2, len(t) - 63, 1]):
        eng = engine(path, max_tokens=160)
        check(replay(eng, {"x": t}, [[("x", c)] for c in cuts]), {"x": want})


OTHER = {
    "one_head": lambda: oracle.make_config(12, 19, [
        oracle.mlstm_layer(1, 1, 1), oracle.parallel_layer((1, 1, 2, 3), (1, 1, 1, 2), 1.0, 2,
                                                           conv=(1, 1)),
        oracle.lightning_layer(1, 2, 1, (0.9,))]),
    "no_attention": lambda: oracle.make_config(20, 31, [
        oracle.lightning_layer(2, 4, 6, (0.3, 0.999), ff=8), oracle.mlstm_layer(2, 6, 4, ff=12)]),
    "no_rotation": lambda: oracle.make_config(20, 31, [
        oracle.parallel_layer((6, 2, 4, 8), (6, 3, 4, 8), 0.7, 0, conv=(2, 5),
                              scales=(0.0, 1.0), ff=8)]),
    "wide_state": lambda: oracle.make_config(16, 23, [
        oracle.mlstm_layer(1, 40, 36, cap=2.0), oracle.lightning_layer(1, 33, 65, (0.95,)),
        oracle.parallel_layer((2, 2, 16, 16), (2, 1, 36, 40), 0.25, 16, conv=(5, 3))]),
}


@pytest.mark.parametrize("name", list(OTHER))
def test_other_sizes(name, tmp_path):
    cfg = OTHER[name]()
    W = oracle.random_weights(cfg, seed=len(name))
    path = write_model(tmp_path / name, cfg, W)
    t = tokens(70, cfg["vocab"], 2)
    want = {"x": oracle.forward(cfg, oracle.as_f64(W), t)[0]}
    eng = engine(path, max_tokens=96)
    check(replay(eng, {"x": t}, [[("x", c)] for c in (33, 2, 1, 20, 1, 1, 12)]), want)


# ------------------------------------------------------------------ generation, command lines
def greedy_reference(cfg, W64, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(oracle.forward(cfg, W64, t)[0][-1].argmax()))
    return t[len(prompt):]


def test_greedy_generation(model):
    from aws_k8s_ansible_provisioner_amd.engine.config import EngineConfig, SamplingParams
    from aws_k8s_ansible_provisioner_amd.engine.llm_engine import LLMEngine

    cfg, W, path = model
    eng = LLMEngine(EngineConfig(model=path, load_format="safetensors", weights_path=path,
                                 dtype="float32", max_model_len=64, max_num_seqs=2,
                                 max_num_batched_tokens=16, block_size=32, num_gpu_blocks=8,
                                 device="cpu"), log=lambda *a: None)
    prompts = [tokens(n, cfg["vocab"], 20 + n) for n in (21, 3, 9)]
    out = eng.generate(None, SamplingParams(max_tokens=7, temperature=0.0, ignore_eos=True),
                       prompt_ids=prompts)
    W64 = oracle.as_f64(W)
    for p, o in zip(prompts, out):
        assert list(o.output_ids) == greedy_reference(cfg, W64, p, 7)


def test_trace_runner_command(model, reference, tmp_path):
    cfg, _, path = model
    reqs, want = reference
    steps = [{"step": 0, "entries": [{"id": "b", "tokens": reqs["b"][:30], "want": [29]}],
              "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": reqs["b"][30:31], "want": []},
                                     {"id": "c", "tokens": reqs["c"], "want": [0, 22]}],
              "end": ["c"]},
             {"step": 2, "entries": [{"id": "b", "tokens": reqs["b"][31:], "want": [0, 9]}],
              "end": ["b"]}]
    r = subprocess.run([os.path.join(REPO, "bin", "trace_run"), "--model", path, "--dtype",
                        "float32", "--out", str(tmp_path), "--max-tokens", "128"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=300, env=dict(os.environ, AKAP_DEVICE="cpu"))
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1",
                                                                            "done 2"]
    got = [np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"])
           for i in range(3)]
    exp = [want["b"][[29]], want["c"][[0, 22]], want["b"][[31, 40]]]
    for g, e in zip(got, exp):
        assert rel_err(torch.from_numpy(g.astype(np.float64)), e).max().item() < FP32_TOL


def test_registry_sizes():
    c = get_config("papivik-w2048")
    assert c.hidden_size == 2048 and c.num_layers == 16 and c.layer_specs[-1].mlp is None
    assert [ls.type for ls in c.layer_specs[:4]] == ["mlstm", "parallel", "lightning", "parallel"]
    assert get_config("papivik-w4096").hidden_size == 4096
    assert get_config("tiny-papivik").layer_specs[1].mixer.left_scale == 1.2
