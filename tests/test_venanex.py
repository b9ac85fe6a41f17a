"""Venanex through the engine (scheduler, block manager, runner, ops) against the plain float64
oracle of tests/venanex_oracle.py, on the CPU branch of the ops (the same suite runs on the HIP
kernels in test_venanex_gpu.py).  Small configurations with random weights; fp32 runs are compared
tightly, bf16 runs loosely."""
import math

import pytest
import torch

import venanex_oracle as oracle
from bidetar_harness import engine, rel_err, replay, tokens, write_model
from aws_k8s_ansible_provisioner_amd import ops
from aws_k8s_ansible_provisioner_amd.models.config import get_config, venanex_config
from aws_k8s_ansible_provisioner_amd.models.transformer import AttnBatch
from aws_k8s_ansible_provisioner_amd.ops import stream as sops

FP32_TOL = 2e-4


def gen(seed):
    return torch.Generator().manual_seed(seed)


def base_config(**kw):
    """Unequal layers: both mixers, with and without feed-forward, with and without a shared
    expert, two chunk sizes (and none), a loop over the middle that starts after layer 0."""
    layers = [
        oracle.latent_layer(3, 8, 4, 6, 12, 10, mlp=oracle.experts(5, 2, 9, shared=7)),
        oracle.diff_layer(4, 2, 6, 10, chunk=20, mlp=oracle.experts(4, 1, 6, limit=0.6)),
        oracle.latent_layer(2, 6, 8, 10, 20, 14, base=7000.0, yarn=(3.0, 40, 6.0, 1.0), scale=0.3),
        oracle.diff_layer(3, 3, 4, 5, chunk=0, diff=0.35, scale=0.7,
                          mlp=oracle.experts(6, 3, 8, limit=2.0, shared=11, shared_limit=0.5)),
        oracle.diff_layer(6, 2, 5, 7, chunk=32, diff=0.8),
    ]
    return oracle.make_config(**{"width": 36, "vocab": 47, "layers": layers, "loop": (1, 4, 2), **kw})


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    cfg = base_config()
    W = oracle.random_weights(cfg, seed=2)
    return cfg, W, write_model(tmp_path_factory.mktemp("venanex"), cfg, W)


@pytest.fixture(scope="module")
def reference(model):
    cfg, W, _ = model
    reqs = {"a": tokens(75, cfg["vocab"], 1), "b": tokens(41, cfg["vocab"], 2),
            "c": tokens(23, cfg["vocab"], 3), "d": tokens(1, cfg["vocab"], 4),
            "e": tokens(64, cfg["vocab"], 5)}
    W64 = oracle.as_f64(W)
    return reqs, {n: oracle.forward(cfg, W64, t)[0] for n, t in reqs.items()}


def check(got, want, names=None, tol=FP32_TOL):
    for n in names or got:
        e = rel_err(got[n], want[n])
        assert e.max().item() < tol, f"{n}: position {int(e.argmax())} off by {e.max().item():.2e}"


# ------------------------------------------------------------------ configuration, weights
def test_config_reader(model):
    cfg, W, path = model
    c = get_config(path)
    assert c.arch == "venanex" and c.loop == (1, 4, 2) and c.loop_inject and c.tie_embeddings
    assert c.layer_runs() == [0, 1, 2, 3, 1, 2, 3, 4] and c.num_layers == 8
    assert c.hidden_size == 36 and c.vocab_size == 47
    m = [ls.mixer for ls in c.layer_specs]
    assert m[0].gate == "none" and m[0].gate_rows == 0 and m[0].rot.scaling is None
    assert m[2].rot.layout == "half" and m[2].rot.scaling["factor"] == 3.0 and m[2].scale == 0.3
    assert (m[1].diff, m[1].chunk, m[1].key_dim) == (0.6, 20, 12) and m[3].chunk == 0
    assert c.layer_specs[2].mlp is None and c.layer_specs[1].mlp.shared_ff == 0
    ml = c.layer_specs[3].mlp
    assert (ml.limit, ml.shared_limit, ml.shared_ff, ml.router.top) == (2.0, 0.5, 11, 3)
    assert ml.router.weigh == "input" and ml.shared_gate and not c.layer_specs[1].mlp.shared_gate
    assert c.num_params() == sum(v.numel() for v in W.values())
    # a cached token: latent + rotated part, or two keys and a value per key/value head; per pass
    row = {0: 16, 1: 2 * (12 + 10), 2: 28, 3: 3 * (8 + 5), 4: 2 * (10 + 7)}
    assert c.kv_bytes_per_token() == 2 * sum(row[i] for i in c.layer_runs())


def test_config_reader_loops_and_refusals():
    cfg = base_config(loop=None)
    assert not venanex_config("x", cfg).loop_inject and venanex_config("x", cfg).num_layers == 5
    one = venanex_config("x", base_config(loop=(0, 5, 1)))      # a single pass is injected too
    assert one.loop_inject and one.num_layers == 5
    for loop in [(2, 2, 2), (0, 6, 2), (1, 3, 0)]:
        with pytest.raises(ValueError):
            venanex_config("x", base_config(loop=loop))
    for change in (lambda ly: ly[0].update(type="attention_3"),
                   lambda ly: ly[0]["mixer"]["rot"].update(dims=2),
                   lambda ly: ly[2]["mixer"]["rot"]["scaling"].pop("fast"),
                   lambda ly: ly[1]["mixer"].update(kv_heads=3),
                   lambda ly: ly[1]["mixer"].update(rot={"base": 10.0, "dims": 2}),
                   lambda ly: ly[0]["mlp"].update(kind="dense"),
                   lambda ly: ly[0]["mlp"]["router"].update(top=6)):
        bad = base_config()
        change(bad["layers"])
        with pytest.raises(ValueError):
            venanex_config("x", bad)


def test_weights_round_trip(model):
    from aws_k8s_ansible_provisioner_amd.models.venanex import VenanexLM

    _, W, path = model
    m = VenanexLM(get_config(path), dtype=torch.float32, max_model_len=64)
    m.load_state_dict(W)
    sd = m.state_dict()
    assert set(sd) == set(W)
    for k, v in W.items():
        assert torch.equal(sd[k].float(), v.float()), k
    lam = oracle.diff_lambda(oracle.as_f64(W), "l3.", 0.35)
    assert abs(m.layers[3].lam_value - float(lam)) < 1e-6
    for k in ("l0.mix.uk", "loop.in", "l3.mlp.shared.sg", "l1.mix.lq2"):
        bad = dict(W)
        bad[k] = W[k][:-1] if W[k].shape[0] > 1 else W[k][:, :-1]
        with pytest.raises(ValueError):
            m.load_state_dict(bad)
        del bad[k]
        with pytest.raises(KeyError):
            m.load_state_dict(bad)
    with pytest.raises(ValueError):
        VenanexLM(get_config(path), dtype=torch.float16)


# ------------------------------------------------------------------ each mechanism alone
def test_layer_norm_step():
    """Rows with a mean far from zero; two addends; no norm on the way in; no norm on the way out
    (the stream itself, into a column slice); a fresh stream over NaNs."""
    g = gen(0)
    T, d, eps = 5, 22, 1e-3
    x0 = torch.randn(T, d, generator=g) + 4.0
    ya, yb = 3 * torch.randn(T, d, generator=g) - 7.0, torch.randn(T, d, generator=g)
    w1, w2 = 1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)
    ln = lambda v, w: oracle.layer_norm(v.double(), w.double(), eps)  # noqa: E731
    for a, b, pw, nw, fresh in [(ya, None, w1, w2, False), (ya, yb, w1, w2, False),
                                (ya, None, None, w2, True), (ya, yb, w1, None, False),
                                (ya, None, None, None, True)]:
        x = torch.full_like(x0, float("nan")) if fresh else x0.clone()
        wide = torch.zeros(T, 2 * d)
        sops.stream_layer_norm_step(x, a, b, pw, nw, eps, wide[:, d:], fresh=fresh)
        m = a.double() + (b.double() if b is not None else 0)
        want = (ln(m, pw) if pw is not None else m) + (0 if fresh else x0.double())
        torch.testing.assert_close(x.double(), want, rtol=1e-5, atol=1e-5)
        out = ln(want, nw) if nw is not None else want
        torch.testing.assert_close(wide[:, d:].double(), out, rtol=1e-5, atol=1e-5)
        assert wide[:, :d].abs().max() == 0
    assert (ln(x0, w1) - oracle.rms(x0.double(), eps) * w1.double()).abs().max() > 0.5


@pytest.mark.parametrize("dims,base,yarn", [(8, 50.0, None), (8, 7000.0, (3.0, 40, 6.0, 1.0)),
                                            (2, 10.0, (2.0, 64, 8.0, 1.0)),
                                            (16, 250.0, (8.0, 30, 1.0, 0.05)),
                                            (6, 90.0, (1.0, 16, 4.0, 4.0))])
def test_latent_preparation_and_query_rotation(dims, base, yarn):
    """Both latents are normed, the rotated part is not (it is made large); entries i and
    i + dims/2 turn together; frequencies below, inside and above the ramp; a cached row is
    [latent | rotated key]; slot -1 writes nothing."""
    g = gen(dims)
    T, Q, R, BS, NB, H, D = 6, 7, 10, 8, 3, 3, 5
    rot = {"base": base, "dims": dims, "scaling": dict(zip(("factor", "original", "fast", "slow"),
                                                           yarn)) if yarn else None}
    proj = torch.randn(T, Q + R + dims + 2, generator=g)
    proj[:, Q + R:Q + R + dims] *= 20.0
    qw, kw = 1 + 0.3 * torch.randn(Q, generator=g), 1 + 0.3 * torch.randn(R, generator=g)
    pos = torch.tensor([0, 1, 7, 29, 90, 5])
    slots = torch.tensor([3, 0, 7, 8, 23, -1])
    table = sops.rotary_table_yarn(96, dims, base, rot["scaling"])
    cq, cache = torch.zeros(T, Q), torch.zeros(NB, BS, R + dims)
    sops.latent_prep(proj, cq, cache, pos, slots, table, qw, kw, Q, R, dims, 0, Q, 1e-5, half=True)
    p64 = proj.double()
    torch.testing.assert_close(cq.double(), oracle.rms(p64[:, :Q], 1e-5) * qw.double(),
                               rtol=1e-5, atol=1e-5)
    c = oracle.rms(p64[:, Q:Q + R], 1e-5) * kw.double()
    kr = oracle.rotate(p64[:, Q + R:Q + R + dims], pos, rot)
    rows = cache.view(NB * BS, -1).double()
    torch.testing.assert_close(rows[slots[:-1]], torch.cat([c, kr], dim=1)[:-1], rtol=1e-5, atol=1e-4)
    written = torch.zeros(NB * BS, dtype=torch.bool)
    written[slots[:-1]] = True
    assert rows[~written].abs().max() == 0
    q = torch.randn(T, H, D + dims, generator=g)
    q0 = q.clone()
    sops.rotate_heads_(q, pos, table, D, half=True)
    assert torch.equal(q[..., :D], q0[..., :D])
    torch.testing.assert_close(q[..., D:].double(), oracle.rotate(q0[..., D:].double(), pos, rot),
                               rtol=1e-5, atol=1e-5)
    if yarn and yarn[0] > 1:
        plain = oracle.rotate(q0[..., D:].double(), pos, {**rot, "scaling": None})
        assert (plain - q[..., D:].double()).abs().max() > 0.05


def test_head_matmul_layouts():
    g = gen(1)
    a, w = torch.randn(3, 5, 6, generator=g), torch.randn(3, 4, 6, generator=g)
    want = torch.einsum("htk,hnk->htn", a, w)
    torch.testing.assert_close(sops.head_matmul(a, w), want)
    o = sops.head_matmul(a, w, w.transpose(1, 2).contiguous(), token_major=True)
    torch.testing.assert_close(o, want)
    assert o.transpose(0, 1).is_contiguous()


def attention_case(seqs, G, D, Dv, BS, seed, dtype=torch.float32, H=None):
    """seqs: (keys, rows) per sequence, single rows first; scattered pages filled with random keys
    and values.  Returns the batch, the caches and per sequence the keys [n, G, 2, D] and values
    [n, G, Dv] as written."""
    g = gen(seed)
    nb = [-(-kv // BS) for kv, _ in seqs]
    NB = sum(nb) + 2
    pages = torch.randperm(NB, generator=g).tolist()
    bt = torch.zeros(len(seqs), max(max(nb), 1) + 1, dtype=torch.int32)
    kc = torch.randn(NB, G, BS, 2 * D, generator=g).to(dtype)
    vt = torch.randn(NB, G, BS, Dv, generator=g).to(dtype)
    rows = []
    for b, (kv, _) in enumerate(seqs):
        ids = [pages.pop() for _ in range(nb[b])]
        bt[b, :nb[b]] = torch.tensor(ids, dtype=torch.int32)
        rows.append(ids)
    nd = next((i for i, (_, n) in enumerate(seqs) if n != 1), len(seqs))
    T = sum(n for _, n in seqs)
    starts = torch.tensor([0] + [n for _, n in seqs]).cumsum(0).int()
    pos = torch.cat([torch.arange(kv - n, kv) if kv else torch.zeros(n, dtype=torch.long)
                     for kv, n in seqs])
    ts, tr = [], []
    for b, (_, n) in enumerate(seqs):
        if b >= nd:
            ts += [b] * -(-n // 128)
            tr += list(range(0, n, 128))
    batch = AttnBatch(is_prefill=nd < len(seqs), positions=pos, slots=torch.zeros(T, dtype=torch.long),
                      block_tables=bt, seq_lens=torch.tensor([kv for kv, _ in seqs], dtype=torch.int32),
                      q_start=starts, tile_seq=torch.tensor(ts, dtype=torch.int32),
                      tile_row=torch.tensor(tr, dtype=torch.int32), tile_rows=128, num_decode=nd)

    def gather(b):
        kv = seqs[b][0]
        k = kc[rows[b]].permute(0, 2, 1, 3).reshape(-1, G, 2, D)[:kv]
        return k, vt[rows[b]].permute(0, 2, 1, 3).reshape(-1, G, Dv)[:kv]

    def where(b, j):
        return rows[b][j // BS], j % BS
    return batch, kc, vt, gather, where


def diff_want(batch, seqs, q, gather, gate, lam, diff, scale, chunk, eps, H, Dv):
    """The oracle on every sequence's keys, for its rows only."""
    want = torch.zeros(q.shape[0], H * Dv, dtype=torch.float64)
    for b, (kv, n) in enumerate(seqs):
        if kv == 0:
            continue
        k, v = gather(b)
        r0 = int(batch.q_start[b])
        pos = torch.arange(kv - n, kv)
        ok = oracle.chunk_mask(kv, chunk)[pos]
        o = oracle.diff_heads(q[r0:r0 + n].double().reshape(n, H, 2, -1), k.double(), v.double(), lam,
                              scale, diff, ok, eps)
        want[r0:r0 + n] = o.reshape(n, -1)
        if gate is not None:
            want[r0:r0 + n] *= torch.sigmoid(gate[r0:r0 + n].double())
    return want


def diff_run(batch, q, kc, vt, gate, H, lam, diff, scale, chunk, eps):
    out = torch.full((q.shape[0], H * vt.shape[3]), 9.0, dtype=q.dtype)
    sops.diff_attention(out, q, kc, sops.v_from_tokens(vt), batch, gate, H, lam, diff, scale, chunk,
                        eps, 512)
    return out


@pytest.mark.parametrize("H,G,D,Dv,chunk", [(4, 2, 6, 10, 20), (3, 3, 5, 3, 0), (6, 1, 8, 16, 7),
                                            (2, 2, 1, 1, 1), (4, 4, 16, 32, 64)])
def test_differential_attention(H, G, D, Dv, chunk):
    """Single rows, a prompt's first and later portions, any ratio of heads, a negative and a
    positive lambda, with and without gate."""
    seqs = [(33, 1), (20, 1), (1, 1), (45, 45), (70, 33), (2, 2)]
    batch, kc, vt, gather, _ = attention_case(seqs, G, D, Dv, 8, seed=H * D)
    g = gen(3)
    T = sum(n for _, n in seqs)
    wide = 2 * torch.randn(T, H * 2 * D + H * Dv + 3, generator=g)
    q, gate = wide[:, :H * 2 * D], wide[:, H * 2 * D:H * 2 * D + H * Dv]
    for lam, diff, gt in ((0.7, 0.4, gate), (-1.3, 0.8, None)):
        got = diff_run(batch, q, kc, vt, gt, H, lam, diff, 0.4, chunk, 1e-5)
        want = diff_want(batch, seqs, q, gather, gt, lam, diff, 0.4, chunk, 1e-5, H, Dv)
        torch.testing.assert_close(got.double(), want, rtol=2e-4, atol=2e-4)
        if chunk == 1:      # both maps rest on the query's own key: nothing to tell apart
            continue
        # the maps are not interchangeable, and 1 - diff counts
        for other in (diff_want(batch, seqs, q.reshape(T, H, 2, D).flip(2).reshape(T, -1),
                                lambda b: (gather(b)[0].flip(2), gather(b)[1]), gt, lam, diff, 0.4,
                                chunk, 1e-5, H, Dv),
                      diff_want(batch, seqs, q, gather, gt, lam, diff / 2, 0.4, chunk, 1e-5, H, Dv)):
            assert (other - want).abs().max() > 0.05


@pytest.mark.parametrize("far", [0, 39, 40, 41, 79, 80, 95])
@pytest.mark.parametrize("single", [True, False])
def test_one_key_at_a_chunk_edge(far, single):
    """One key is made to take nearly all the weight of map 1 wherever it is seen: rows of its own
    chunk from its position on must carry its value, every other row must not notice."""
    H, G, D, Dv, BS, chunk = 2, 1, 4, 6, 8, 40
    seqs = [(p + 1, 1) for p in (38, 39, 40, 60, 79, 80, 81, 95)] if single else [(96, 96)]
    batch, kc, vt, gather, where = attention_case(seqs, G, D, Dv, BS, seed=far)
    q = torch.randn(len(seqs) if single else 96, H * 2 * D, generator=gen(5))
    q[:, :D] = 1.0
    q[:, 2 * D:3 * D] = 1.0
    base = diff_run(batch, q, kc, vt, None, H, 0.5, 0.3, 0.5, chunk, 1e-5)
    for b, (kv, _) in enumerate(seqs):
        if far < kv:
            page, off = where(b, far)
            kc[page, :, off, :D] = 30.0
            vt[page, :, off] = 50.0 * torch.arange(1, Dv + 1) * (-1.0) ** torch.arange(Dv)
    got = diff_run(batch, q, kc, vt, None, H, 0.5, 0.3, 0.5, chunk, 1e-5)
    want = diff_want(batch, seqs, q, gather, None, 0.5, 0.3, 0.5, chunk, 1e-5, H, Dv)
    torch.testing.assert_close(got.double(), want, rtol=2e-4, atol=2e-4)
    for t, p in enumerate(batch.positions.tolist()):
        moved = (got[t] - base[t]).abs().max().item()
        seen = far <= p and far // chunk == p // chunk
        assert (moved > 0.05) if seen else (moved == 0.0), (p, moved)


def test_clamped_units():
    """Values on both sides of every clamp; the weight goes in ahead of the clamps (a weight on the
    output is far off); experts not chosen give zeros; the shared expert has a limit and a weight
    of its own; column slices."""
    g = gen(7)
    T, E, F_, Fs, top = 9, 4, 5, 3, 2
    gu = 3 * torch.randn(T, E * 2 * F_ + 2 * Fs + 4, generator=g)
    ids = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int()
    w, sw = torch.rand(T, top, generator=g), torch.rand(T, generator=g)
    out = torch.full((T, E * F_ + Fs), 9.0)
    sops.clamped_glu(gu[:, :-4], out, 1.1, ids, w, E, Fs, 0.4, sw)

    def unit(a, b, lim):
        a, b = torch.clamp(a, max=lim), torch.clamp(b, min=-lim, max=lim)
        return a * torch.sigmoid(1.702 * a) * (b + 1)

    want, late = torch.zeros(T, E * F_ + Fs).double(), torch.zeros(T, E * F_ + Fs).double()
    for t in range(T):
        for e, c in zip(ids[t].tolist(), w[t].double()):
            a, b = gu[t, e * 2 * F_:e * 2 * F_ + F_].double(), gu[t, e * 2 * F_ + F_:(e + 1) * 2 * F_].double()
            want[t, e * F_:(e + 1) * F_] = unit(c * a, c * b, 1.1)
            late[t, e * F_:(e + 1) * F_] = c * unit(a, b, 1.1)
        a, b = gu[t, E * 2 * F_:E * 2 * F_ + Fs].double(), gu[t, E * 2 * F_ + Fs:-4].double()
        late[t, E * F_:] = want[t, E * F_:] = sw[t].double() * unit(a, b, 0.4)
    torch.testing.assert_close(out.double(), want, rtol=1e-5, atol=1e-6)
    assert (late - want).abs().max() > 0.1
    plain = torch.empty(T, F_)
    sops.clamped_glu(gu[:, :2 * F_], plain, 0.0)            # a limit of zero
    torch.testing.assert_close(plain.double(), unit(gu[:, :F_].double(), gu[:, F_:2 * F_].double(), 0.0),
                               rtol=1e-5, atol=1e-6)
    only = torch.empty(T, Fs)
    sops.clamped_glu(gu[:, E * 2 * F_:-4], only, 0.0, None, None, 0, Fs, 0.4, sw)
    torch.testing.assert_close(only, out[:, E * F_:])


def test_router_with_a_gate_row():
    g = gen(8)
    h, router = torch.randn(20, 12, generator=g), torch.randn(7, 12, generator=g)
    ids, w, sg = sops.route_sigmoid(h, router, 3, gates=1)
    oid, ow = oracle.route(h.double(), router[:6].double(), 3)
    assert torch.equal(ids.long(), oid)
    torch.testing.assert_close(w.double(), ow, rtol=1e-5, atol=1e-6)
    torch.testing.assert_close(sg.double(), torch.sigmoid(h.double() @ router[6:].double().T),
                               rtol=1e-5, atol=1e-6)
    ids2, w2 = sops.route_sigmoid(h, router[:6], 3)         # without gate rows: unchanged
    assert torch.equal(ids, ids2) and torch.equal(w, w2)
    assert w.sum(dim=1).max() > 1.2                          # not renormalised


@pytest.mark.parametrize("layer", [0, 1, 3])
@pytest.mark.parametrize("small", [True, False])
def test_feed_forward_paths(model, layer, small):
    """All experts in one GEMM pair and expert-sorted rows, with and without a shared expert, one
    and several experts per token."""
    from aws_k8s_ansible_provisioner_amd.models.venanex import VenanexLM

    cfg, W, path = model
    m = VenanexLM(get_config(path), dtype=torch.float32, max_model_len=64)
    m.load_state_dict(W)
    h = 1.5 * torch.randn(40, cfg["width"], generator=gen(9))
    ya, yb = m._feed_forward(m.layers[layer], h, small)
    got = ya.double() + (yb.double() if yb is not None else 0)
    want = oracle.moe(h.double(), oracle.as_f64(W), f"l{layer}.", cfg["layers"][layer]["mlp"])
    torch.testing.assert_close(got, want, rtol=1e-4, atol=1e-4)


def test_grouped_expert_reference_with_clamped_units():
    """The CPU form of the core library's grouped expert feed-forward with clamped units."""
    g = gen(10)
    T, d, E, F_, top = 13, 8, 5, 6, 2
    h, w13 = torch.randn(T, d, generator=g), torch.randn(E, 2 * F_, d, generator=g)
    w2 = torch.randn(E, d, F_, generator=g)
    W = {"l.mlp.router": torch.randn(E, d, generator=g).double()}
    for e in range(E):
        W[f"l.mlp.e{e}.gate"], W[f"l.mlp.e{e}.up"] = w13[e, :F_].double(), w13[e, F_:].double()
        W[f"l.mlp.e{e}.down"] = w2[e].double()
    ids, w = oracle.route(h.double(), W["l.mlp.router"], top)
    got = ops.fused_moe(h, w13, w2, w.float(), ids.int(), clamp=(0.8, sops.CLAMPED_ALPHA))
    want = oracle.moe(h.double(), W, "l.", oracle.experts(E, top, F_, limit=0.8))
    torch.testing.assert_close(got.double(), want, rtol=1e-4, atol=1e-4)


# ------------------------------------------------------------------ whole model, schedules
def test_oracle_is_causal_and_sharp(model, reference):
    """A prefix gives the same logits, and every mechanism left out or done wrongly moves the
    logits by far more than the tolerance (the mistakes are planted in the oracle)."""
    cfg, W, _ = model
    reqs, want = reference
    W64 = oracle.as_f64(W)
    torch.testing.assert_close(oracle.forward(cfg, W64, reqs["a"][:30])[0], want["a"][:30],
                               rtol=1e-9, atol=1e-9)

    def moved(patch):
        with pytest.MonkeyPatch.context() as mp:
            patch(mp)
            return rel_err(oracle.forward(cfg, W64, reqs["a"])[0], want["a"])[25:].median().item()

    def swap(name, fn):
        return lambda mp: mp.setattr(oracle, name, fn)

    rms, mask, ln = oracle.rms, oracle.chunk_mask, oracle.layer_norm
    rotate, expert = oracle.rotate, oracle.expert
    wrong = {
        "norm keeps the mean": swap("layer_norm", lambda x, w, eps: rms(x, eps) * w),
        "chunk one token off": swap("chunk_mask", lambda T, n: mask(T + 1, n)[1:, 1:]),
        "no chunks": swap("chunk_mask", lambda T, n: mask(T, 0)),
        "lambda zero": swap("diff_lambda", lambda *a: torch.zeros((), dtype=torch.float64)),
        "no rotation": swap("rotate", lambda v, pos, rot: v),
        "no scaling": swap("rotate", lambda v, pos, rot: rotate(v, pos, {**rot, "scaling": None})),
        "positions one off": swap("rotate", lambda v, pos, rot: rotate(v, pos + (v.dim() == 3), rot)),
        "no clamp": swap("expert", lambda h, W, p, lim: expert(h, W, p, 1e9)),
        "no injection": swap("schedule", lambda c: [(i, False) for i in
                                                    venanex_config("x", c).layer_runs()]),
        "first pass not injected": swap("schedule", lambda c, s=oracle.schedule(cfg): [
            (i, e and k > 1) for k, (i, e) in enumerate(s)]),
    }
    for what, patch in wrong.items():
        assert moved(patch) > 20 * FP32_TOL, what
    assert oracle.layer_norm is ln


def test_whole_prompts(model, reference):
    reqs, want = reference
    eng = engine(model[2])
    check(replay(eng, reqs, [[(n, len(t))] for n, t in reqs.items()]), want)


def test_prefill_against_token_by_token(model, reference):
    reqs, want = reference
    eng = engine(model[2])
    one = {"a": reqs["a"]}
    check(replay(eng, one, [[("a", 1)]] * 75), want)            # every token decoded alone
    check(replay(eng, one, [[("a", 40)]] + [[("a", 1)]] * 35), want)


@pytest.mark.parametrize("sizes", [[2] * 37 + [1], [3, 2, 7, 2, 19, 2, 5, 33, 2],
                                   [31, 1, 1, 30, 2, 2, 8], [32, 32, 11], [20, 20, 20, 15],
                                   [19, 2, 18, 2, 34]])
def test_portions(model, reference, sizes):
    """Portions down to two tokens, cut before, on and after page and chunk borders."""
    reqs, want = reference
    assert sum(sizes) == 75
    eng = engine(model[2])
    check(replay(eng, {"a": reqs["a"]}, [[("a", s)] for s in sizes]), want)


def test_batches_of_unequal_requests(model, reference):
    reqs, want = reference
    eng = engine(model[2])
    sched = [[("a", 30), ("b", 2), ("c", 1)],
             [("a", 1), ("b", 20), ("c", 22), ("d", 1)],
             [("a", 1), ("b", 1), ("e", 33)],
             [("a", 1), ("b", 1)],                      # a pure decode step of two
             [("b", 17), ("e", 1)],                     # a is left out of a step
             [("a", 42), ("e", 30)]]
    check(replay(eng, reqs, sched), want)


def test_pages_are_used_again(model, reference):
    """A pool of 5 pages serves 7 requests one after another and side by side: later requests live
    in pages that hold other requests' latents, keys and values."""
    reqs, want = reference
    eng = engine(model[2], max_tokens=160, max_seqs=2)
    assert eng.runner.num_blocks == 5
    many = {f"{n}{i}": reqs[n] for i in range(2) for n in ("b", "c", "e")}
    many["a"] = reqs["a"]
    sched = [[("b0", 41), ("c0", 23)], [("e0", 64), ("c1", 22)], [("c1", 1)],
             [("a", 75), ("b1", 41)], [("e1", 10)], [("e1", 54)]]
    check(replay(eng, many, sched), {k: want[k[0]] for k in many})
    assert eng.sched.num_free_blocks() == 5 and eng.sched.num_running == 0


def test_first_tokens(model, reference):
    reqs, want = reference
    eng = engine(model[2])
    got = replay(eng, {"d": reqs["d"], "c": reqs["c"], "b": reqs["b"]},
                 [[("d", 1), ("c", 1), ("b", 2)], [("c", 2), ("b", 39)], [("c", 20)]])
    check(got, want, ["d", "c", "b"])


def sharp_config():
    """Large score scales: a softmax row rests on one or two keys."""
    return oracle.make_config(width=32, vocab=37, loop=(0, 2, 2), layers=[
        oracle.latent_layer(2, 8, 4, 8, 16, 12, scale=2.0),
        oracle.diff_layer(2, 1, 6, 8, chunk=48, scale=3.0, mlp=oracle.experts(3, 1, 8, shared=6))])


def test_a_far_token_that_stands_out(tmp_path):
    """One token far back (the first one, at a page border, just inside and outside the last
    queries' chunk) is replaced by the one that the last positions notice most, far above the
    tolerance: the engine must say the same, in a prompt and in decoding."""
    cfg = sharp_config()
    W = oracle.random_weights(cfg, seed=4)
    W64 = oracle.as_f64(W)
    path = write_model(tmp_path, cfg, W)
    toks = tokens(150, 37, 6)
    base = oracle.forward(cfg, W64, toks)[0]
    for at in (0, 31, 32, 95, 96, 143, 144):
        best = 0.0
        for tok in range(0, 37, 3):
            changed = toks[:at] + [tok] + toks[at + 1:]
            say = oracle.forward(cfg, W64, changed)[0]
            moved = rel_err(say, base)[145:].max().item()
            if moved > best:
                best, other, want = moved, changed, say
        assert best > 30 * FP32_TOL, (at, best)
        for sched in ([[("x", 150)]], [[("x", 100)], [("x", 44)]] + [[("x", 1)]] * 6):
            check(replay(engine(path), {"x": other}, sched), {"x": want})


def test_long_decoding(tmp_path):
    cfg = sharp_config()
    W = oracle.random_weights(cfg, seed=8)
    toks = tokens(230, 37, 9)
    want = {"a": oracle.forward(cfg, oracle.as_f64(W), toks)[0]}
    eng = engine(write_model(tmp_path, cfg, W))
    check(replay(eng, {"a": toks}, [[("a", 5)]] + [[("a", 1)]] * 225), want, tol=5e-4)


OTHER = {
    "ones": lambda: oracle.make_config(16, 19, loop=(0, 2, 1), layers=[
        oracle.latent_layer(1, 1, 2, 1, 1, 1, mlp=oracle.experts(1, 1, 1)),
        oracle.diff_layer(1, 1, 1, 1, chunk=1, mlp=oracle.experts(1, 1, 1, shared=1))]),
    "no_loop_only_latent": lambda: oracle.make_config(24, 31, [
        oracle.latent_layer(4, 6, 2, 4, 8, 8, yarn=(4.0, 16, 4.0, 0.5)),
        oracle.latent_layer(2, 4, 6, 8, 70, 3, mlp=oracle.experts(4, 4, 5))], eps=1e-3),
    "only_differential_whole_loop": lambda: oracle.make_config(20, 23, loop=(0, 3, 3), layers=[
        oracle.diff_layer(4, 4, 3, 6, chunk=9), oracle.diff_layer(2, 1, 8, 4, chunk=0, diff=0.0),
        oracle.diff_layer(6, 3, 2, 9, chunk=500, mlp=oracle.experts(7, 3, 4, limit=0.2))]),
    "loop_at_the_end": lambda: oracle.make_config(54, 19, loop=(2, 3, 4), eps=1e-6, layers=[
        oracle.latent_layer(5, 7, 6, 9, 13, 17),
        oracle.diff_layer(7, 7, 3, 2, chunk=31, mlp=oracle.experts(9, 2, 11, shared=3)),
        oracle.latent_layer(9, 5, 10, 4, 20, 9, mlp=oracle.experts(2, 1, 100, shared=100,
                                                                   shared_limit=7.0))]),
    "equal_sizes": lambda: oracle.make_config(32, 32, loop=(1, 3, 2), layers=[
        oracle.latent_layer(4, 8, 8, 8, 8, 8, mlp=oracle.experts(4, 2, 8, shared=8)),
        oracle.diff_layer(4, 4, 8, 8, chunk=32, mlp=oracle.experts(4, 2, 8, shared=8)),
        oracle.diff_layer(4, 4, 8, 8, chunk=32, mlp=oracle.experts(4, 2, 8, shared=8))]),
}


@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_configurations(tmp_path, name):
    cfg = OTHER[name]()
    W = oracle.random_weights(cfg, seed=len(name))
    W64 = oracle.as_f64(W)
    reqs = {"p": tokens(45, cfg["vocab"], 11), "q": tokens(38, cfg["vocab"], 12)}
    want = {n: oracle.forward(cfg, W64, t)[0] for n, t in reqs.items()}
    eng = engine(write_model(tmp_path, cfg, W))
    sched = [[("p", 17), ("q", 2)], [("p", 1), ("q", 30)], [("p", 27), ("q", 1)],
             [("q", 1)], [("q", 4)]]
    check(replay(eng, reqs, sched), want)


def test_portion_above_the_small_batch_threshold(tmp_path):
    """More rows than the all-experts path takes: the sorted path inside the engine."""
    cfg = oracle.make_config(24, 29, loop=(0, 1, 2), layers=[
        oracle.diff_layer(2, 1, 4, 6, chunk=64, mlp=oracle.experts(5, 2, 6, shared=4))])
    W = oracle.random_weights(cfg, seed=3)
    toks = tokens(300, 29, 1)
    want = {"a": oracle.forward(cfg, oracle.as_f64(W), toks)[0]}
    eng = engine(write_model(tmp_path, cfg, W))
    check(replay(eng, {"a": toks}, [[("a", 290)], [("a", 10)]]), want)


# ------------------------------------------------------------------ bf16, generation, CLI
def test_bfloat16_engine(model, reference):
    reqs, want = reference
    eng = engine(model[2], dtype="bfloat16")
    got = replay(eng, {"a": reqs["a"], "b": reqs["b"]},
                 [[("a", 30), ("b", 2)], [("a", 1), ("b", 39)], [("a", 44)]])
    for n in ("a", "b"):
        assert rel_err(got[n], want[n]).median().item() < 0.06


def greedy(path, cfg, W, prompts, device="cpu", **kw):
    from aws_k8s_ansible_provisioner_amd.engine.config import EngineConfig, SamplingParams
    from aws_k8s_ansible_provisioner_amd.engine.llm_engine import LLMEngine

    eng = LLMEngine(EngineConfig(model=path, load_format="safetensors", weights_path=path,
                                 dtype="float32", max_model_len=128, max_num_seqs=3,
                                 max_num_batched_tokens=32, block_size=32, num_gpu_blocks=12,
                                 device=device, gc_freeze=False, **kw), log=lambda *a: None)
    W64 = oracle.as_f64(W)
    for batch in prompts:
        outs = eng.generate(None, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True),
                            prompt_ids=batch)
        assert [len(o.output_ids) for o in outs] == [12] * len(batch)
        for p, o in zip(batch, outs):
            logits = oracle.forward(cfg, W64, p + list(o.output_ids))[0]
            for i, tok in enumerate(o.output_ids):
                row = logits[len(p) - 1 + i]
                assert row[tok] >= row.max() - 1e-3 * row.std(), (i, tok, int(row.argmax()))
    return eng


def test_greedy_generation_through_the_engine(model):
    """LLMEngine.generate (admission, chunked prefill, mixed steps, decode) picks the oracle's
    argmax token by token."""
    cfg, W, path = model
    prompts = [tokens(n, cfg["vocab"], 20 + n) for n in (30, 3, 17, 9, 66)]
    greedy(path, cfg, W, [prompts], enable_prefix_caching=False)


def test_prefix_cache_serves_this_design(model):
    """Nothing but pages belongs to a sequence, so a cached prefix may be reused: the second
    prompt takes two whole pages of the first and must still say what the oracle says."""
    cfg, W, path = model
    first = tokens(70, cfg["vocab"], 31)
    eng = greedy(path, cfg, W, [[first], [first[:66] + [1, 2, 3]]], enable_prefix_caching=True)
    assert eng.sched.prefix_stats()[0] > 0


def test_registry_model_runs():
    from aws_k8s_ansible_provisioner_amd.engine.config import EngineConfig, SamplingParams
    from aws_k8s_ansible_provisioner_amd.engine.llm_engine import LLMEngine

    eng = LLMEngine(EngineConfig(model="tiny-venanex", dtype="float32", max_model_len=64,
                                 max_num_seqs=2, max_num_batched_tokens=32, num_gpu_blocks=4,
                                 device="cpu", gc_freeze=False), log=lambda *a: None)
    outs = eng.generate(None, SamplingParams(max_tokens=4, temperature=0.7, seed=1, ignore_eos=True),
                        prompt_ids=[[5, 6, 7], [9] * 20])
    assert [len(o.output_ids) for o in outs] == [4, 4]
    assert all(math.isfinite(x) for x in eng.runner.model.embed.flatten()[:4].tolist())


def test_trace_run_command_line(model, reference, tmp_path):
    import json
    import os
    import subprocess
    import sys

    import numpy as np

    cfg, _, path = model
    reqs, want = reference
    a, c = reqs["a"], reqs["c"]
    steps = [
        {"step": 0, "entries": [{"id": "x", "tokens": a[:40], "want": [39, 0, 7]},
                                {"id": "y", "tokens": c[:1], "want": [0]}], "end": []},
        {"step": 1, "entries": [{"id": "y", "tokens": c[1:], "want": []}], "end": ["y"]},
        {"step": 2, "entries": [{"id": "x", "tokens": a[40:41], "want": [0]}], "end": []},
        {"step": 3, "entries": [{"id": "x", "tokens": a[41:], "want": [33]},
                                {"id": "z", "tokens": c, "want": [22, 21]}], "end": ["x", "z"]},
    ]
    repo = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(repo, "bin", "trace_run"), "--model", path,
                        "--dtype", "float32", "--out", str(out), "--max-tokens", "192",
                        "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True,
                       text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == \
        [f"done {i}" for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    V = cfg["vocab"]
    got0 = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, V)).double()
    exp0 = torch.stack([want["a"][39], want["a"][0], want["a"][7], want["c"][0]])
    assert rel_err(got0, exp0).max().item() < FP32_TOL
    got3 = torch.from_numpy(np.fromfile(out / "3.f32", dtype="<f4").reshape(-1, V)).double()
    exp3 = torch.stack([want["a"][74], want["c"][22], want["c"][21]])
    assert rel_err(got3, exp3).max().item() < FP32_TOL
