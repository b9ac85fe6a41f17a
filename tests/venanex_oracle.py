"""A plain float64 implementation of the Venanex design, one function per mechanism, written from
its equations.  It shares no code with the package: tests compare the engine with it.

Notation: x is the residual stream [T, d] of ONE sequence (positions 0 .. T-1), W a dict
name -> float64 tensor under the checkpoint's names, `cfg` the config.json dictionary, p the
prefix of a layer's tensors.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def as_f64(sd):
    return {k: v.to(F64) for k, v in sd.items()}


# ------------------------------------------------------------------------------------- norms
def layer_norm(x, w, eps):
    """Mean taken off, divided by the root of the mean squared deviation; weight, no bias."""
    c = x - x.mean(dim=-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(dim=-1, keepdim=True) + eps) * w


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


# ------------------------------------------------------------------------------------- rotation
def yarn_frequencies(rot):
    """(frequencies of the dims / 2 pairs, factor on cos and sin)."""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0

    def index_of(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(index_of(sc["fast"])), 0)
    hi = min(math.ceil(index_of(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(v, pos, rot):
    """v [T, ..., n]: entries i and i + dims/2 of the first dims turn together by pos f_i."""
    f, mag = yarn_frequencies(rot)
    half = rot["dims"] // 2
    out = v.clone()
    for i in range(half):
        a = pos.to(F64) * f[i]
        shape = [v.shape[0]] + [1] * (v.dim() - 2)
        c, s = (torch.cos(a) * mag).reshape(shape), (torch.sin(a) * mag).reshape(shape)
        out[..., i] = v[..., i] * c - v[..., i + half] * s
        out[..., i + half] = v[..., i + half] * c + v[..., i] * s
    return out


# ------------------------------------------------------------------------------------- mixers
def softmax_rows(s, ok):
    return torch.softmax(s.masked_fill(~ok, float("-inf")), dim=-1)


def latent_kv(h, W, p, m, eps, pos):
    """What a token leaves behind: the normed latent [T, R] and the rotated key part [T, r]."""
    R = m["kv_rank"]
    z = h @ W[p + "mix.dkv"].T
    return rms(z[:, :R], eps) * W[p + "mix.dkv.norm"], rotate(z[:, R:], pos, m["rot"])


def latent_mixer(h, W, p, m, eps):
    T, H, D, r, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    pos = torch.arange(T)
    c, kr = latent_kv(h, W, p, m, eps, pos)
    cq = rms(h @ W[p + "mix.dq"].T, eps) * W[p + "mix.dq.norm"]
    q = (cq @ W[p + "mix.uq"].T).reshape(T, H, D + r)
    qn, qr = q[..., :D], rotate(q[..., D:], pos, m["rot"])
    k = (c @ W[p + "mix.uk"].T).reshape(T, H, D)
    v = (c @ W[p + "mix.uv"].T).reshape(T, H, V)
    ok = pos[None, :] <= pos[:, None]
    o = torch.zeros(T, H, V, dtype=F64)
    for n in range(H):
        s = (qn[:, n] @ k[:, n].T + qr[:, n] @ kr.T) * m["scale"]
        o[:, n] = softmax_rows(s, ok) @ v[:, n]
    return o.reshape(T, H * V) @ W[p + "mix.o"].T


def chunk_mask(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    if size:
        ok = ok & (torch.div(i, size, rounding_mode="floor")
                   == torch.div(j, size, rounding_mode="floor"))
    return ok


def diff_lambda(W, p, diff):
    return (torch.exp((W[p + "mix.lq1"] * W[p + "mix.lk1"]).sum())
            - torch.exp((W[p + "mix.lq2"] * W[p + "mix.lk2"]).sum()) + diff)


def diff_heads(q, k, v, lam, scale, diff, ok, eps):
    """q [T, H, 2, D], k [T, G, 2, D], v [T, G, V] -> [T, H, V]: two softmax maps over the same
    values, the second taken off lam times, each head normed without a weight, times 1 - diff."""
    T, H, G, V = q.shape[0], q.shape[1], k.shape[1], v.shape[2]
    out = torch.zeros(T, H, V, dtype=F64)
    for n in range(H):
        g = n // (H // G)
        a = [softmax_rows(q[:, n, i] @ k[:, g, i].T * scale, ok) @ v[:, g] for i in (0, 1)]
        out[:, n] = rms(a[0] - lam * a[1], eps) * (1.0 - diff)
    return out


def attention_mixer(h, W, p, m, eps):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "mix.q"].T).reshape(T, H, 2, D)
    k = (h @ W[p + "mix.k"].T).reshape(T, G, 2, D)
    v = (h @ W[p + "mix.v"].T).reshape(T, G, V)
    ok = chunk_mask(T, (m.get("mask") or {}).get("size", 0))
    o = diff_heads(q, k, v, diff_lambda(W, p, m["diff"]), m["scale"], m["diff"], ok, eps)
    o = o.reshape(T, H * V) * torch.sigmoid(h @ W[p + "mix.g"].T)
    return o @ W[p + "mix.o"].T


# ------------------------------------------------------------------------------------- experts
def expert(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def route(h, Wr, top):
    """ids [T, top] by falling score, and the scores."""
    s = torch.sigmoid(h @ Wr.T)
    ids = torch.sort(s, dim=-1, descending=True, stable=True).indices[:, :top]
    return ids, s.gather(1, ids)


def moe(h, W, p, ml):
    ids, w = route(h, W[p + "mlp.router"], ml["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, we in zip(ids[t].tolist(), w[t]):
            out[t] += expert(we * h[t:t + 1], W, p + f"mlp.e{e}.", ml["expert"]["limit"])[0]
    if ml.get("shared"):
        sg = torch.sigmoid(h @ W[p + "mlp.shared.sg"].T)
        out = out + sg * expert(h, W, p + "mlp.shared.", ml["shared"]["limit"])
    return out


# ------------------------------------------------------------------------------------- the model
def layer(x, W, p, ly, eps):
    mix = latent_mixer if ly["type"] == "latent_attention" else attention_mixer
    y = mix(layer_norm(x, W[p + "norm1"], eps), W, p, ly["mixer"], eps)
    x = x + layer_norm(y, W[p + "norm1b"], eps)
    if ly.get("mlp") is not None:
        y = moe(layer_norm(x, W[p + "norm2"], eps), W, p, ly["mlp"])
        x = x + layer_norm(y, W[p + "norm2b"], eps)
    return x


def schedule(cfg):
    """(layer index, does a pass of the loop start here) in execution order."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    span = [(i, i == a) for i in range(a, b)]
    return ([(i, False) for i in range(a)] + span * lp["times"]
            + [(i, False) for i in range(b, n)])


def forward(cfg, W, tokens):
    """(logits [T, vocab], stream after every layer run [runs, T, d]) of one sequence."""
    eps = cfg["norm"]["eps"]
    x0 = W["embed"][torch.as_tensor(tokens)]
    x, after = x0, []
    for i, entry in schedule(cfg):
        if entry:
            x = torch.cat([x, x0], dim=-1) @ W["loop.in"].T
        x = layer(x, W, f"l{i}.", cfg["layers"][i], eps)
        after.append(x)
    return layer_norm(x, W["final.norm"], eps) @ W["embed"].T, torch.stack(after)


# ------------------------------------------------------------------------------------- test models
def latent_layer(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale=None, base=100.0, yarn=None,
                 mlp=None):
    """yarn = (factor, original, fast, slow) or None."""
    sc = dict(zip(("factor", "original", "fast", "slow"), yarn)) if yarn else None
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
                      "kv_rank": kv_rank, "q_rank": q_rank,
                      "scale": scale if scale is not None else (dim + rot_dim) ** -0.5,
                      "rot": {"base": base, "dims": rot_dim, "scaling": sc}}}


def diff_layer(heads, kv_heads, dim, vdim, chunk, diff=0.6, scale=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": diff,
         "scale": scale if scale is not None else dim ** -0.5}
    if chunk:
        m["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def experts(n, top, ff, limit=1.0, shared=None, shared_limit=2.0):
    ml = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
          "router": {"experts": n, "top": top}}
    if shared:
        ml["shared"] = {"ff": shared, "limit": shared_limit}
    return ml


def make_config(width, vocab, layers, loop=None, eps=1e-5):
    cfg = {"architecture": "Venanex", "layers": layers, "norm": {"eps": eps}, "vocab": vocab,
           "width": width}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def random_weights(cfg, seed=0):
    """Random tensors under the checkpoint's names, values that bfloat16 holds exactly.  The rows
    of the stream get a mean far from zero, so that a norm without its subtraction shows."""
    g = torch.Generator().manual_seed(seed)
    d = cfg["width"]

    def rnd(*shape, s=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * s + mean).to(torch.bfloat16)

    def lin(rows, cols, s=1.0):
        return rnd(rows, cols, s=s * cols ** -0.5)

    def gain(n):
        return rnd(n, s=0.2, mean=1.0)

    W = {"embed": rnd(cfg["vocab"], d, mean=0.5), "final.norm": gain(d)}
    if cfg.get("loop"):
        W["loop.in"] = lin(d, 2 * d, 1.2)
    for i, ly in enumerate(cfg["layers"]):
        p, m = f"l{i}.", ly["mixer"]
        H, D, V = m["heads"], m["dim"], m["vdim"]
        W[p + "norm1"], W[p + "norm1b"] = gain(d), rnd(d, s=0.2, mean=0.8)
        if ly["type"] == "latent_attention":
            R, r, Q = m["kv_rank"], m["rot_dim"], m["q_rank"]
            W[p + "mix.dq"], W[p + "mix.dq.norm"] = lin(Q, d), gain(Q)
            W[p + "mix.uq"] = lin(H * (D + r), Q, 1.6)
            W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = lin(R + r, d), gain(R)
            W[p + "mix.uk"], W[p + "mix.uv"] = lin(H * D, R, 1.6), lin(H * V, R)
        else:
            G = m["kv_heads"]
            W[p + "mix.q"], W[p + "mix.k"] = lin(H * 2 * D, d, 1.4), lin(G * 2 * D, d, 1.4)
            W[p + "mix.v"], W[p + "mix.g"] = lin(G * V, d), lin(H * V, d)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                W[p + "mix." + n] = rnd(D, s=0.5 * D ** -0.25)
        W[p + "mix.o"] = lin(d, H * V)
        ml = ly.get("mlp")
        if ml is None:
            continue
        W[p + "norm2"], W[p + "norm2b"] = gain(d), rnd(d, s=0.2, mean=0.8)
        W[p + "mlp.router"] = lin(ml["router"]["experts"], d, 2.0)
        names = [(f"e{e}.", ml["expert"]["ff"]) for e in range(ml["router"]["experts"])]
        if ml.get("shared"):
            names.append(("shared.", ml["shared"]["ff"]))
            W[p + "mlp.shared.sg"] = lin(1, d)
        for n, ff in names:
            W[p + f"mlp.{n}gate"], W[p + f"mlp.{n}up"] = lin(ff, d, 1.5), lin(ff, d, 1.5)
            W[p + f"mlp.{n}down"] = lin(d, ff, 2.0)
    return W
