"""Papivik on the HIP kernels: every kernel against the PyTorch version of the same op (fp32 and
bf16 storage, odd sizes), then the engine -- mixed steps, hipGraph decode, a small page and slot
pool -- against the float64 oracle (tests/papivik_oracle.py), and greedy generation through
LLMEngine.generate."""
import pytest
import torch

import papivik_oracle as oracle
from bidetar_harness import engine, rel_err, replay, tokens, write_model
from aws_k8s_ansible_provisioner_amd.ops import stream as sops

pytestmark = pytest.mark.gpu
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def gen(seed):
    return torch.Generator().manual_seed(seed)


def close(a, b, dtype, scale=1.0):
    tol = 3e-5 if dtype == "float32" else 2e-2
    torch.testing.assert_close(a.float().cpu(), b.float().cpu(), rtol=tol, atol=tol * scale)


def both(fn):
    """fn(device) on the CPU and on the GPU; returns the two results."""
    return fn("cpu"), fn("cuda")


# ------------------------------------------------------------------ kernels against their ops
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("d", [24, 203, 2048, 4096])
def test_post_norm_kernel_without_a_following_norm(dtype, d):
    g, dt = gen(d), DT[dtype]
    x0, y = torch.randn(5, d, generator=g), (3 * torch.randn(5, d, generator=g)).to(dt)
    w = 1 + 0.3 * torch.randn(d, generator=g)

    def run(dev):
        x, o = x0.clone().to(dev), torch.zeros(5, d, dtype=dt, device=dev)
        sops.stream_post_norm_add_norm(x, y.to(dev), None, None, None, w.to(dev), None, 1e-5, o)
        return x, o
    c, n = both(run)
    close(n[0], c[0], "float32")
    close(n[1], c[1], dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("F_", [24, 333, 4096])
def test_gelu_kernel(dtype, F_):
    x = (4 * torch.randn(7, F_ + 8, generator=gen(F_))).to(DT[dtype])

    def run(dev):
        o = torch.zeros(7, F_, dtype=DT[dtype], device=dev)
        sops.gelu_tanh(x.to(dev)[:, :F_], o)
        return o
    c, n = both(run)
    close(n, c, dtype, scale=4.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,Dv,rot", [(4, 2, 32, 16, 8), (3, 1, 10, 7, 10), (8, 8, 128, 128, 64),
                                          (2, 2, 96, 40, 0), (2, 1, 256, 256, 256)])
def test_head_norm_rotation_kernel(dtype, H, G, D, Dv, rot):
    g, dt = gen(H * D), DT[dtype]
    T, BS, NB = 9, 8, 4
    N = H * D + G * (D + Dv) + 5
    proj = torch.randn(T, N, generator=g).to(dt)
    qw, kw = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.3 * torch.randn(D, generator=g)
    slots = torch.tensor([8, 9, 10, 11, 3, -1, 17, 0, 31])
    pos = torch.tensor([0, 1, 2, 37, 38, 5, 60, 61, 7])
    cs = sops.rotary_table(64, rot, 100.0) if rot else None

    def run(dev):
        q = torch.zeros(T, H, D, dtype=dt, device=dev)
        kc = torch.zeros(NB, G, BS, D, dtype=dt, device=dev)
        vc = torch.zeros(NB, G, BS // 8, Dv, 8, dtype=dt, device=dev)
        sops.head_norm_cache(proj.to(dev), q, kc, vc, slots.to(dev), H, G, D, Dv, 0, H * D,
                             (H + G) * D, 1e-6, True, False, qw.to(dev), kw.to(dev),
                             cs.to(dev) if cs is not None else None, pos.to(dev))
        return q, kc, vc
    c, n = both(run)
    for a, b in zip(n, c):
        close(a, b, dtype, scale=2.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,groups", [(48, 3), (512, 1), (645, 5), (4096, 32), (2048, 1)])
def test_norm_gate_kernel(dtype, n, groups):
    g, dt = gen(n), DT[dtype]
    T = 6
    y = 3 * torch.randn(T, n, generator=g)
    gate = torch.randn(T, n + 16, generator=g).to(dt)
    w = 1 + 0.2 * torch.randn(n, generator=g)
    den, fl = 4 * torch.randn(T, groups, generator=g), torch.rand(T, groups, generator=g)
    for act in ("sigmoid", "silu"):
        for d, f in ((None, None), (den, fl)):
            def run(dev):
                o = torch.zeros(T, n + 8, dtype=dt, device=dev)
                sops.norm_gate(o[:, :n], y.to(dev), gate.to(dev)[:, 8:8 + n], w.to(dev), groups,
                               1e-5, act, None if d is None else d.to(dev),
                               None if f is None else f.to(dev))
                return o
            c, k = both(run)
            close(k, c, dtype, scale=3.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("C,taps,silu_from,f32_out", [(48, 4, 16, False), (37, 3, 0, False),
                                                      (64, 1, 64, False), (512, 4, 510, True),
                                                      (24, 8, 7, False)])
def test_convolution_kernel(dtype, C, taps, silu_from, f32_out):
    g, dt = gen(C), DT[dtype]
    cw = 0.5 * torch.randn(C, taps, generator=g)
    steps = [[(0, 0, 37), (1, 0, 2)], [(1, 2, 1), (0, 37, 1)], [(0, 38, 19), (1, 3, 2), (2, 0, 1)],
             [(2, 1, 1), (-1, 0, 1), (1, 5, 1)], [(1, 0, 21)]]
    projs = [torch.randn(sum(n for _, _, n in st), C + 8, generator=g).to(dt) for st in steps]

    def run(dev):
        state = torch.full((3, taps - 1, C), 7.0, dtype=dt, device=dev)
        outs = []
        for st, proj in zip(steps, projs):
            slot, pos, qs = step_rows(st, dev)
            o = torch.zeros(proj.shape[0], C, dtype=torch.float32 if f32_out else dt, device=dev)
            sops.conv_silu(o, proj.to(dev), 4, cw.to(dev), None, state, slot, pos, qs, silu_from)
            outs.append(o)
        outs[3] = outs[3][[0, 2]]
        return outs + [state]
    c, n = both(run)
    for a, b in zip(n, c):
        close(a, b, dtype, scale=2.0)


def step_rows(step, dev):
    slot = torch.cat([torch.full((n,), s, dtype=torch.int32) for s, _, n in step]).to(dev)
    pos = torch.cat([torch.arange(p, p + n) for _, p, n in step]).to(dev)
    qs = None
    if not all(n == 1 for _, _, n in step):
        qs = torch.tensor([0] + [n for _, _, n in step]).cumsum(0).int().to(dev)
    return slot, pos, qs


# prompts in portions around the scan's and the chunks' sizes, a portion of two tokens, mixed
# steps whose leading rows are single tokens, single rows, a padding row, a slot used again from
# position 0 on top of stale contents
STEPS = [[(0, 0, 37), (1, 0, 2)], [(1, 2, 1), (0, 37, 1)], [(2, 0, 1), (0, 38, 90), (1, 3, 64)],
         [(2, 1, 1), (-1, 0, 1), (1, 67, 1)], [(0, 128, 1), (2, 2, 129), (1, 68, 2)],
         [(1, 0, 65), (0, 129, 63)]]
FIRST = [0, 0, 1, 0, 1, 0]


def run_steps(kind, dtype, H, G, D, V, dev, seed):
    """All STEPS through one recurrence op; returns every output and the final states."""
    g, dt = gen(seed), DT[dtype]
    HV = H * V
    nw = (1 + 0.3 * torch.randn(HV, generator=g)).to(dev)
    pa, pb = torch.randn(H, generator=g), torch.randn(H, generator=g)
    state = torch.full((3, H, V, D), 3.0, device=dev)
    extra = (torch.full((3, H, D), 3.0, device=dev), torch.full((3, H), 3.0, device=dev))
    outs = []
    for st, first in zip(STEPS, FIRST):
        T = sum(n for _, _, n in st)
        slot, pos, qs = step_rows(st, dev)
        qkv = torch.randn(T, 2 * G * D + HV + 8, generator=g)
        gates = torch.randn(T, HV + 2 * H, generator=g)
        # rows of a multiple of 8 elements, like the model's projections: the chunked form takes them
        gates = torch.nn.functional.pad(gates, (0, -(2 * G * D + 2 * HV + 2 * H) % 8))
        out = torch.zeros(T, HV + 8, dtype=dt, device=dev)
        if kind == "delta":
            qkv, proj = qkv.to(dt).to(dev), gates.to(dt).to(dev)
            sops.gated_delta(out[:, 8:], qkv, 0, G * D, 2 * G * D, proj, 0, HV, HV + H,
                             (0.7 * pa - 1).to(dev), (pb - 1).to(dev), state, nw, slot, pos, qs,
                             H, G, D, V, 1e-5, first)
        else:
            proj = torch.cat([qkv, gates], dim=1).to(dt).to(dev)
            o = (0, H * D, 2 * H * D, 2 * H * D + HV + 8)
            if kind == "mlstm":
                sops.matrix_memory(out[:, 8:], proj, *o, o[3] + HV, o[3] + HV + H,
                                   (2 * pa).to(dev), (pb + 2).to(dev), 9.0, (state,) + extra, nw,
                                   slot, pos, qs, H, D, V, 1e-5, first)
            else:
                sops.linear_attention(out[:, 8:], proj, *o, torch.sigmoid(3 + pa).to(dev), state,
                                      nw, slot, pos, qs, H, D, V, 1e-5, "silu", kind, "sigmoid",
                                      first)
        if any(s < 0 for s, _, _ in st):
            out = out[[0, 2]]                  # the padding row is left unwritten
        outs.append(out)
    return outs + [state] + (list(extra) if kind == "mlstm" else [])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,H,G,D,V", [
    ("mlstm", 3, 3, 5, 7), ("mlstm", 2, 2, 32, 64), ("mlstm", 2, 2, 128, 256),
    ("mlstm", 1, 1, 64, 32), ("mlstm", 2, 2, 96, 96),
    ("all", 3, 3, 6, 9), ("all", 2, 2, 32, 64), ("head", 4, 4, 128, 128), ("all", 1, 1, 64, 320),
    ("delta", 4, 2, 6, 10), ("delta", 4, 2, 32, 32), ("delta", 6, 2, 128, 128),
    ("delta", 2, 1, 64, 96), ("delta", 3, 3, 96, 64), ("delta", 2, 2, 256, 40)])
def test_recurrence_kernels(kind, H, G, D, V, dtype):
    a = run_steps(kind, dtype, H, G, D, V, "cpu", H * D + V)
    b = run_steps(kind, dtype, H, G, D, V, "cuda", H * D + V)
    ns = 3 if kind == "mlstm" else 1
    for i, (c, n) in enumerate(zip(a, b)):
        assert torch.isfinite(n).all(), i
        if i < len(a) - ns:
            close(n, c, dtype, scale=4.0)
        else:
            # (bf16: the chunked form rounds activated q, k, v of the plain recurrence once more)
            tol = 2e-4 if dtype == "float32" else 1e-2 if kind in ("all", "head") else 3e-4
            err = (n.cpu() - c).abs().max() / c.abs().max()
            assert err < tol, (i, err.item())


# ------------------------------------------------------------------ the engine
TOL = {"float32": 3e-4, "bfloat16": 0.35}


def check(got, want, dtype, names=None):
    for n in names or got:
        e = rel_err(got[n], want[n])
        assert e.max().item() < TOL[dtype], f"{n}: position {int(e.argmax())} off by {e.max().item():.2e}"


def base_config():
    layers = [
        oracle.parallel_layer((4, 2, 8, 6), (4, 2, 8, 16), 0.5, 4, base=50.0, conv=(3, 4),
                              scales=(1.4, 0.7), ff=40),
        oracle.mlstm_layer(3, 8, 16, cap=7.0),
        oracle.lightning_layer(2, 7, 9, (0.8, 0.99), ff=24),
        oracle.parallel_layer((3, 3, 32, 32), (2, 2, 32, 32), 0.3, 6, base=900.0, conv=(4, 2),
                              scales=(0.6, 1.3)),
        oracle.mlstm_layer(2, 32, 32, cap=20.0, ff=16),
        oracle.lightning_layer(3, 32, 64, (1.0, 0.5, 0.95)),
    ]
    return oracle.make_config(width=40, vocab=47, layers=layers, embed_scale=0.7)


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    cfg = base_config()
    W = oracle.random_weights(cfg, seed=2)
    W64 = oracle.as_f64(W)
    reqs = {"a": tokens(150, 47, 1), "b": tokens(41, 47, 2), "c": tokens(23, 47, 3),
            "d": tokens(1, 47, 4), "e": tokens(64, 47, 5)}
    want = {n: oracle.forward(cfg, W64, t)[0] for n, t in reqs.items()}
    return cfg, W, write_model(tmp_path_factory.mktemp("papivik"), cfg, W), reqs, want


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("eager", [False, True])
def test_schedules(model, dtype, eager):
    cfg, W, path, reqs, want = model
    eng = engine(path, dtype=dtype, max_tokens=512, device="cuda", eager=eager)
    whole = [[(n, len(t))] for n, t in reqs.items()]
    check(replay(eng, reqs, whole), want, dtype)
    sub = {n: reqs[n] for n in ("a", "b", "c", "d")}
    mixed = [[("a", 66), ("b", 2)], [("b", 1), ("a", 2), ("c", 9)], [("a", 1), ("b", 1), ("c", 1)],
             [("c", 13), ("b", 30)], [("a", 70), ("b", 1), ("d", 1)], [("a", 1), ("b", 1)],
             [("a", 1), ("b", 1)], [("b", 3)], [("a", 9), ("b", 1)]]
    check(replay(eng, sub, mixed), {n: want[n] for n in sub}, dtype)
    check(replay(eng, {"b": reqs["b"], "c": reqs["c"]}, [[("b", 1), ("c", 1)]] * 23 + [[("b", 1)]] * 18),
          want, dtype, ["b", "c"])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_small_pool_is_used_again(model, dtype):
    cfg, W, path, reqs, want = model
    eng = engine(path, dtype=dtype, max_tokens=128, max_seqs=2, device="cuda")
    for _ in range(2):
        for pair in (("b", "c"), ("e", "d"), ("c", "e")):
            sub = {n: reqs[n] for n in pair}
            n0, n1 = len(sub[pair[0]]), len(sub[pair[1]])
            sched = [[(pair[0], n0 - 1), (pair[1], 1)]] + ([[(pair[1], n1 - 1)]] if n1 > 1 else []) \
                + [[(pair[0], 1)]]
            check(replay(eng, sub, sched), want, dtype, pair)


def test_long_decode_through_graphs(model):
    cfg, W, path, _, _ = model
    t = tokens(260, 47, 11)
    want = {"x": oracle.forward(cfg, oracle.as_f64(W), t)[0]}
    eng = engine(path, max_tokens=288, device="cuda")
    got = replay(eng, {"x": t}, [[("x", 5)]] + [[("x", 1)]] * 255)
    assert rel_err(got["x"], want["x"]).max().item() < 2e-3


def test_greedy_generation(model):
    from aws_k8s_ansible_provisioner_amd.engine.config import EngineConfig, SamplingParams
    from aws_k8s_ansible_provisioner_amd.engine.llm_engine import LLMEngine

    cfg, W, path, _, _ = model
    eng = LLMEngine(EngineConfig(model=path, load_format="safetensors", weights_path=path,
                                 dtype="float32", max_model_len=128, max_num_seqs=2,
                                 max_num_batched_tokens=32, block_size=32, num_gpu_blocks=10,
                                 device="cuda", gc_freeze=False), log=lambda *a: None)
    prompts = [tokens(n, cfg["vocab"], 20 + n) for n in (41, 3, 9, 66)]
    outs = eng.generate(None, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True),
                        prompt_ids=prompts)
    W64 = oracle.as_f64(W)
    for p, o in zip(prompts, outs):
        logits = oracle.forward(cfg, W64, p + list(o.output_ids))[0]
        for i, tok in enumerate(o.output_ids):
            row = logits[len(p) - 1 + i]
            assert row[tok] >= row.max() - 1e-3 * row.std(), (i, tok, int(row.argmax()))


OTHER = {
    "one_head": lambda: oracle.make_config(16, 19, [
        oracle.mlstm_layer(1, 1, 1), oracle.parallel_layer((1, 1, 2, 3), (1, 1, 1, 2), 1.0, 2,
                                                           conv=(1, 1)),
        oracle.lightning_layer(1, 2, 1, (0.9,))]),
    "no_attention": lambda: oracle.make_config(24, 31, [
        oracle.lightning_layer(2, 4, 6, (0.3, 0.999), ff=8), oracle.mlstm_layer(2, 6, 4, ff=12)]),
    "no_rotation": lambda: oracle.make_config(24, 31, [
        oracle.parallel_layer((6, 2, 4, 8), (6, 3, 4, 8), 0.7, 0, conv=(2, 5), ff=8)]),
    "wide_state": lambda: oracle.make_config(16, 23, [
        oracle.mlstm_layer(1, 40, 36, cap=2.0), oracle.lightning_layer(1, 160, 65, (0.95,)),
        oracle.parallel_layer((2, 2, 16, 64), (2, 1, 36, 40), 0.25, 16, conv=(5, 3))]),
    "matrix_core": lambda: oracle.make_config(64, 23, [
        oracle.mlstm_layer(2, 64, 96, cap=11.0, ff=64), oracle.lightning_layer(2, 96, 32, (0.95, 0.0)),
        oracle.parallel_layer((4, 2, 64, 64), (4, 2, 64, 32), 0.15, 32, conv=(4, 4),
                              scales=(0.8, 1.1), ff=32)]),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(OTHER))
def test_other_configurations(tmp_path, name, dtype):
    cfg = OTHER[name]()
    W = oracle.random_weights(cfg, seed=len(name))
    reqs = {"p": tokens(145, cfg["vocab"], 11), "q": tokens(38, cfg["vocab"], 12)}
    W64 = oracle.as_f64(W)
    want = {n: oracle.forward(cfg, W64, t)[0] for n, t in reqs.items()}
    eng = engine(write_model(tmp_path, cfg, W), dtype=dtype, device="cuda")
    sched = [[("p", 67), ("q", 2)], [("p", 1), ("q", 30)], [("p", 77), ("q", 1)],
             [("q", 1)], [("q", 4)]]
    check(replay(eng, reqs, sched), want, dtype)


def test_registry_model_generates_with_sampling():
    from aws_k8s_ansible_provisioner_amd.engine.config import EngineConfig, SamplingParams
    from aws_k8s_ansible_provisioner_amd.engine.llm_engine import LLMEngine

    eng = LLMEngine(EngineConfig(model="tiny-papivik", dtype="bfloat16", max_model_len=256,
                                 max_num_seqs=4, max_num_batched_tokens=64, num_gpu_blocks=32,
                                 device="cuda", gc_freeze=False), log=lambda *a: None)
    outs = eng.generate(None, SamplingParams(max_tokens=20, temperature=0.8, top_p=0.9, seed=3,
                                             ignore_eos=True),
                        prompt_ids=[[5, 6, 7], [9] * 70, [1, 2], [3] * 33, [4] * 5])
    assert [len(o.output_ids) for o in outs] == [20] * 5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mid_size_engine_against_the_cpu_ops(tmp_path, dtype):
    """Sizes between the tiny oracle models and the benchmark's (matrix-core attention and
    chunks, 16-byte paths everywhere): the engine on the GPU against the same engine on the CPU
    ops, over a mixed schedule."""
    cfg = oracle.make_config(width=192, vocab=301, layers=[
        oracle.parallel_layer((8, 2, 64, 64), (8, 4, 64, 64), 0.11, 32, base=5000.0, ff=320),
        oracle.lightning_layer(4, 64, 64, (0.7, 0.9, 0.99, 0.999), ff=192),
        oracle.mlstm_layer(4, 64, 128, ff=192),
        oracle.parallel_layer((4, 1, 128, 128), (3, 1, 128, 64), 0.09, 128, conv=(2, 3),
                              scales=(0.9, 1.2))])
    W = oracle.random_weights(cfg, seed=11)
    path = write_model(tmp_path, cfg, W)
    reqs = {"a": tokens(330, 301, 1), "b": tokens(140, 301, 2), "c": tokens(61, 301, 3)}
    sched = [[("a", 200), ("b", 3)], [("a", 1), ("b", 100), ("c", 60)], [("a", 1), ("b", 1)],
             [("a", 128), ("b", 36), ("c", 1)]]
    want = replay(engine(path, dtype="float32", max_tokens=640, device="cpu"), reqs, sched)
    got = replay(engine(path, dtype=dtype, max_tokens=640, device="cuda"), reqs, sched)
    for n in reqs:
        e = rel_err(got[n], want[n])
        if dtype == "float32":
            assert e.max().item() < 1e-4, f"{n}: position {int(e.argmax())} off by {e.max().item():.2e}"
        else:
            assert e.median().item() < 0.05 and e.max().item() < 0.5, (n, e.median().item(),
                                                                       e.max().item())
