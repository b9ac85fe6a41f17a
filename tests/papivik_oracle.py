"""Float64 oracle of the Papivik design, written from its equations: one function per mechanism,
whole sequences at once, token by token where the design is a recurrence, sharing no code with
the package.

Notation: positions count from 0; rms(v) = v / sqrt(mean(v^2) + eps) over the last axis; linear
weights are [out, in].  A model is (cfg, w): the config.json dictionary and a dictionary of
float64 tensors under the checkpoint's names.
"""
import math

import torch

F64 = torch.float64


def rms(v, eps):
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def log_sigmoid(z):
    return -softplus(-z)


def unit(v):
    return v / torch.sqrt((v * v).sum(dim=-1, keepdim=True) + 1e-6)


def causal_conv(u, cw):
    """u [T, C]; cw [C, taps] whose last column weighs the current token; zeros before the
    start; no bias."""
    T, C = u.shape
    taps = cw.shape[1]
    out = torch.zeros(T, C, dtype=F64)
    for t in range(T):
        for j in range(taps):
            src = t - (taps - 1 - j)
            if src >= 0:
                out[t] = out[t] + cw[:, j] * u[src]
    return out


# ----------------------------------------------------------------------------- recurrences
def mlstm_scan(q, k, v, i, f):
    """q, k [T, H, D] (q scaled), v [T, H, V], log gates i, f [T, H].  Returns o [T, H, V] and
    the last (S [H, D, V], n [H, D], m [H])."""
    T, H, D = q.shape
    V = v.shape[2]
    S = torch.zeros(H, D, V, dtype=F64)
    n = torch.zeros(H, D, dtype=F64)
    m = torch.zeros(H, dtype=F64)
    out = torch.zeros(T, H, V, dtype=F64)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        m = m_new
        den = torch.maximum((n * q[t]).sum(dim=-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(dim=1) / den[:, None]
    return out, (S, n, m)


def decay_scan(q, k, v, decay):
    """S <- decay_h S + k v^T, o = S^T q; decay [H]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out, S


def delta_scan(q, k, v, beta, g):
    """q, k [T, H, D] (already one per value head), v [T, H, V], beta and decay g [T, H]:
    S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(dim=1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out, S


# ----------------------------------------------------------------------------- attention
def rotate_half(x, rot):
    """x [T, H, D]: the first rot.dims entries of every head, entry i paired with i + dims/2."""
    if not rot or not rot.get("dims"):
        return x
    dims = int(rot["dims"])
    half = dims // 2
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / dims) for i in range(half)], dtype=F64)
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * f[None, :]
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    out = x.clone()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def causal_attention(q, k, v, scale):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; head h reads key/value head h // (H / G)."""
    T, H, D = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    hide = torch.triu(torch.ones(T, T, dtype=torch.bool), diagonal=1)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(hide, float("-inf"))
        e = torch.exp(s - s.max(dim=1, keepdim=True).values)
        out[:, h] = (e / e.sum(dim=1, keepdim=True)) @ v[:, g]
    return out


# ----------------------------------------------------------------------------- mixers
def mlstm(h, w, p, m, eps):
    T = h.shape[0]
    H, D, V, cap = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"])
    q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, V)
    i = cap * torch.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = log_sigmoid(cap * torch.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    o, _ = mlstm_scan(q, k, v, i, f)
    o = rms(o, eps).reshape(T, H * V) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def lightning(h, w, p, m, eps):
    T = h.shape[0]
    H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(h @ w[p + "q"].T).view(T, H, D)
    k = silu(h @ w[p + "k"].T).view(T, H, D)
    v = silu(h @ w[p + "v"].T).view(T, H, V)
    o, _ = decay_scan(q, k, v, torch.tensor(m["decay"], dtype=F64))
    o = rms(o.reshape(T, H * V), eps) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def conv_attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = causal_conv(h @ w[p + "q"].T, w[p + "q.conv"]).view(T, H, D)
    k = causal_conv(h @ w[p + "k"].T, w[p + "k.conv"]).view(T, G, D)
    v = causal_conv(h @ w[p + "v"].T, w[p + "v.conv"]).view(T, G, Dv)
    q = rotate_half(rms(q, eps) * w[p + "q.norm"], m.get("rot"))
    k = rotate_half(rms(k, eps) * w[p + "k.norm"], m.get("rot"))
    o = causal_attention(q, k, v, float(m["scale"]))
    return o.reshape(T, H * Dv) @ w[p + "o"].T


def gated_delta(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D, V = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(causal_conv(h @ w[p + "q"].T, w[p + "q.conv"])).view(T, G, D)
    k = silu(causal_conv(h @ w[p + "k"].T, w[p + "k.conv"])).view(T, G, D)
    v = silu(causal_conv(h @ w[p + "v"].T, w[p + "v.conv"])).view(T, H, V)
    q, k = unit(q) * D ** -0.5, unit(k)
    of = torch.tensor([x // (H // G) for x in range(H)])
    beta = sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o, _ = delta_scan(q[:, of], k[:, of], v, beta, g)
    o = rms(o, eps) * w[p + "norm"] * silu(h @ w[p + "g"].T).view(T, H, V)
    return o.reshape(T, H * V) @ w[p + "o"].T


def parallel(h, w, p, m, eps):
    return float(m["left_scale"]) * conv_attention(h, w, p + "left.", m["left"], eps) \
        + float(m["right_scale"]) * gated_delta(h, w, p + "right.", m["right"], eps)


MIXERS = {"mlstm": mlstm, "lightning": lightning, "parallel": parallel}


# ----------------------------------------------------------------------------- the model
def forward(cfg, w, tokens):
    """Logits [T, vocab] of one sequence and the residual stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    after = []
    for i, ly in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[ly["type"]](x, w, p + "mix.", ly["mixer"], eps)
        x = x + rms(y, eps) * w[p + "norm1"]
        if ly.get("mlp") is not None:
            y = gelu_tanh(x @ w[p + "mlp.up"].T) @ w[p + "mlp.down"].T
            x = x + rms(y, eps) * w[p + "norm2"]
        after.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T, torch.stack(after)


# ----------------------------------------------------------------------------- test models
def random_weights(cfg, seed=0):
    """Random weights under the checkpoint's names, values a bf16 file can hold (bf16 tensors).
    Gate biases and decays sit in a range where a state neither dies at once nor stays for
    ever."""
    gen = torch.Generator().manual_seed(seed)
    d = int(cfg["width"])

    def rnd(*shape, s=1.0, mean=0.0):
        return (torch.randn(*shape, generator=gen) * s + mean).to(torch.bfloat16)

    def lin(rows, cols):
        return rnd(rows, cols, s=cols ** -0.5)

    w = {"embed": rnd(int(cfg["vocab"]), d, s=1.0 / float(cfg["embedding"]["scale"])),
         "final.norm": rnd(d, s=0.2, mean=1.0), "head": lin(int(cfg["vocab"]), d)}
    for i, ly in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", ly["mixer"]
        w[f"l{i}.norm1"] = rnd(d, s=0.2, mean=1.0)
        if ly["type"] in ("mlstm", "lightning"):
            H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
            for name, rows in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V)):
                w[p + name] = lin(rows, d)
            w[p + "o"] = lin(d, H * V)
            w[p + "norm"] = rnd(H * V, s=0.2, mean=1.0)
            if ly["type"] == "mlstm":
                w[p + "i"], w[p + "f"] = lin(H, d), lin(H, d)
                w[p + "i.b"], w[p + "f.b"] = rnd(H, s=1.5), rnd(H, s=1.0, mean=3.0)
        else:
            a, r = m["left"], m["right"]
            q = p + "left."
            H, G, D, Dv = int(a["heads"]), int(a["kv_heads"]), int(a["dim"]), int(a["vdim"])
            for name, rows in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                w[q + name] = lin(rows, d)
                w[q + name + ".conv"] = rnd(rows, int(a["conv"]), s=0.6)
            w[q + "q.norm"], w[q + "k.norm"] = rnd(D, s=0.3, mean=1.2), rnd(D, s=0.3, mean=1.2)
            w[q + "o"] = lin(d, H * Dv)
            q = p + "right."
            H, G, D, V = int(r["heads"]), int(r["kv_heads"]), int(r["dim"]), int(r["vdim"])
            for name, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
                w[q + name] = lin(rows, d)
                w[q + name + ".conv"] = rnd(rows, int(r["conv"]), s=0.6)
            w[q + "b"], w[q + "a"] = lin(H, d), lin(H, d)
            w[q + "A_log"], w[q + "dt_bias"] = rnd(H, s=0.7, mean=-0.5), rnd(H, s=1.0, mean=-2.0)
            w[q + "norm"] = rnd(V, s=0.2, mean=1.0)
            w[q + "g"], w[q + "o"] = lin(H * V, d), lin(d, H * V)
        if ly.get("mlp") is not None:
            ff = int(ly["mlp"]["ff"])
            w[f"l{i}.norm2"] = rnd(d, s=0.2, mean=1.0)
            w[f"l{i}.mlp.up"], w[f"l{i}.mlp.down"] = lin(ff, d), lin(d, ff)
    return w


def as_f64(weights):
    return {k: v.to(F64) for k, v in weights.items()}


def dense(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def mlstm_layer(heads, dim, vdim, cap=15.0, ff=0):
    return {"type": "mlstm", "mlp": dense(ff),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def lightning_layer(heads, dim, vdim, decay, ff=0):
    return {"type": "lightning", "mlp": dense(ff),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def parallel_layer(att, delta, scale, rot_dims, base=100.0, conv=(4, 4), scales=(1.0, 1.0), ff=0):
    """att = (heads, kv_heads, dim, vdim), delta the same of the delta rule."""
    keys = ("heads", "kv_heads", "dim", "vdim")
    left = dict(zip(keys, att), conv=conv[0], scale=scale,
                rot={"base": base, "dims": rot_dims})
    right = dict(zip(keys, delta), conv=conv[1])
    return {"type": "parallel", "mlp": dense(ff),
            "mixer": {"left": left, "right": right, "left_scale": scales[0],
                      "right_scale": scales[1]}}


def make_config(width, vocab, layers, eps=1e-5, embed_scale=1.0):
    return {"architecture": "Papivik", "embedding": {"scale": embed_scale}, "layers": layers,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}
