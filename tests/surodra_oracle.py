"""A slow, whole-sequence implementation of the Surodra design, one function per mechanism, written from its equations
and sharing no code with the package: the oracle of tests/test_surodra.py.  Everything runs in fp32 (or fp64) on the CPU
over one whole sequence at a time; there is no cache, no batching and no portioning here.

Notation: x residual [L, W]; N squashing norm; a layer computes x <- x + m mixer(N1 x), then x <- x + m ff(N2 x).
"""
import json
import math
import os

import torch


# ---- norms ---------------------------------------------------------------------------------------------------------
def squash_norm(x, alpha, w, b):
    """No statistics at all: every value is squashed on its own."""
    return torch.tanh(alpha * x) * w + b


def unit_rms(y, eps):
    return y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)


def unit_vector(y):
    return y / torch.sqrt((y * y).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- short causal convolution ----------------------------------------------------------------------------------------
def short_conv(u, w):
    """u [L, C], w [C, taps]:  y[t] = sum_j w[:, j] u[t - taps + 1 + j], zeros before the sequence."""
    L, C = u.shape
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u])
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + w[:, j] * padded[j: j + L]
    return y


# ---- rotation --------------------------------------------------------------------------------------------------------
def rotate(x, rot):
    """x [L, heads, D]: value i < dims / 2 and value i + dims / 2 form a pair, turned by position * f_i."""
    dims = int((rot or {}).get("dims", 0) or 0)
    if dims == 0:
        return x
    L, n = x.shape[0], dims // 2
    f = torch.tensor([rot["base"] ** (-2.0 * i / dims) for i in range(n)], dtype=torch.float64)
    if rot.get("scaling"):
        f = f / rot["scaling"]["factor"]
    ang = torch.arange(L, dtype=torch.float64)[:, None] * f[None, :]
    c, s = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
    a, b = x[..., :n], x[..., n: dims]
    return torch.cat([a * c - b * s, b * c + a * s, x[..., dims:]], dim=-1)


# ---- recurrences, token by token -----------------------------------------------------------------------------------
def decayed_memory(q, k, v, decay):
    """q, k, decay [L, H, D], v [L, H, E]:  S_t = diag(decay_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t."""
    L, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(L):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def delta_memory(q, k, v, g, beta):
    """q, k [L, H, D], v [L, H, E], g, beta [L, H]: decay, correct the value read at k, write, read at q."""
    L, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(L):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


# ---- mixers ------------------------------------------------------------------------------------------------------------
def delta_mixer(h, w, m, eps):
    L = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w[n].T, w[n + ".conv"])) for n in ("q", "k", "v"))
    q = unit_vector(q.view(L, G, D)) * D ** -0.5
    k = unit_vector(k.view(L, G, D))
    own = torch.arange(H) // (H // G)
    beta = torch.sigmoid(h @ w["b"].T)
    g = torch.exp(-torch.exp(w["A_log"]) * torch.log1p(torch.exp(h @ w["a"].T + w["dt_bias"])))
    o = delta_memory(q[:, own], k[:, own], v.view(L, H, E), g, beta)
    o = unit_rms(o, eps) * w["norm"] * silu(h @ w["g"].T).view(L, H, E)
    return o.reshape(L, H * E) @ w["o"].T


def sink_attention(h, w, m, eps):
    L = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms(h @ w["q"].T, eps) * w["q.norm"]            # over the whole projection, not per head
    k = unit_rms(h @ w["k"].T, eps) * w["k.norm"]
    v = (h @ w["v"].T).view(L, G, E)
    q, k = rotate(q.view(L, H, D), m.get("rot")), rotate(k.view(L, G, D), m.get("rot"))
    seen = torch.arange(L)[None, :] <= torch.arange(L)[:, None]
    gate = torch.sigmoid(h @ w["g"].T)
    out = []
    for n in range(H):
        g = n // (H // G)
        s = (q[:, n] @ k[:, g].T) * m["scale"]
        s = s.masked_fill(~seen, float("-inf"))
        top = torch.maximum(s.max(-1, keepdim=True).values, w["sink"][n])
        e = torch.exp(s - top)
        p = e / (e.sum(-1, keepdim=True) + torch.exp(w["sink"][n] - top))
        out.append((p @ v[:, g]) * gate[:, n: n + 1])
    return torch.cat(out, -1) @ w["o"].T


def gated_linear_mixer(h, w, m, eps):
    L = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(L, H, D) * D ** -0.5
    k = (h @ w["k"].T).view(L, H, D)
    v = (h @ w["v"].T).view(L, H, E)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    alpha = torch.sigmoid(z) ** (1.0 / m["tau"])
    o = unit_rms(decayed_memory(q, k, v, alpha.view(L, H, D)), eps) * w["norm"]
    return (o.reshape(L, H * E) * silu(h @ w["g"].T)) @ w["o"].T


def parallel_mixer(h, w, m, eps):
    def part(side):
        return {n[len(side) + 1:]: t for n, t in w.items() if n.startswith(side + ".")}
    lw, rw = part("left"), part("right")
    a = unit_rms(sink_attention(h, lw, m["left"], eps), eps) * lw["out"]
    b = unit_rms(gated_linear_mixer(h, rw, m["right"], eps), eps) * rw["out"]
    return 0.5 * (a + b)


def retention_mixer(h, w, m, eps):
    L = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ w["q"].T).view(L, H, D), m.get("rot"))
    k = rotate((h @ w["k"].T).view(L, H, D), m.get("rot")) * D ** -0.5
    v = (h @ w["v"].T).view(L, H, E)
    decay = torch.tensor(m["decay"], dtype=h.dtype)[None, :, None].expand(L, H, D)
    o = unit_rms(decayed_memory(q, k, v, decay), eps)
    return (o.reshape(L, H * E) * silu(h @ w["g"].T)) @ w["o"].T


MIXERS = {"delta": delta_mixer, "parallel": parallel_mixer, "retention": retention_mixer}


def feed_forward(h, w):
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


# ---- the stack -----------------------------------------------------------------------------------------------------------
def run_list(n, loop):
    """(layer, pass, is this the first layer of a pass?) in running order."""
    if not loop:
        return [(i, 0, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return [(i, 0, False) for i in range(a)] + \
        [(i, t, i == a) for t in range(loop["times"]) for i in range(a, b)] + [(i, 0, False) for i in range(b, n)]


def sub(weights, prefix):
    return {n[len(prefix):]: t for n, t in weights.items() if n.startswith(prefix)}


def forward(cfg, weights, tokens, dtype=torch.float32, want_layers=False):
    """tokens: list of ids.  Logits [L, vocab]; with ``want_layers`` also the residual after every layer run."""
    W = {n: t.to(dtype) for n, t in weights.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]

    def norm(x, name):
        return squash_norm(x, W[name + ".alpha"], W[name], W[name + ".b"])
    e = W["embed"][torch.tensor(tokens)]
    x, trail = e, []
    for i, t, first in run_list(len(cfg["layers"]), cfg.get("loop")):
        spec = cfg["layers"][i]
        if first:
            if t > 0:
                x = x + e
            x = x + W["loop.step"][t]
        x = x + mult * MIXERS[spec["type"]](norm(x, f"l{i}.norm1"), sub(W, f"l{i}.mix."), spec["mixer"], eps)
        if spec.get("mlp"):
            x = x + mult * feed_forward(norm(x, f"l{i}.norm2"), sub(W, f"l{i}.mlp."))
        trail.append(x)
    y = norm(x, "final.norm") @ W["head"].T * cfg["logit_scale"]
    y = cfg["logit_softcap"] * torch.tanh(y / cfg["logit_softcap"])
    return (y, torch.stack(trail)) if want_layers else y


# ---- small random models ---------------------------------------------------------------------------------------------
def _mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def _rot(dims, base, factor=None):
    if not dims:
        return {}
    return {"rot": {"base": base, "dims": dims, **({"scaling": {"factor": factor}} if factor else {})}}


def delta_layer(heads=4, kv_heads=2, dim=12, vdim=20, conv=4, ff=40):
    return {"type": "delta", "mlp": _mlp(ff),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def parallel_layer(heads=4, kv_heads=2, dim=12, vdim=20, rot_dims=8, base=300.0, factor=3.0, scale=0.3, right_heads=3,
                   right_dim=8, right_vdim=12, tau=5.0, rank=7, ff=40):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, **_rot(rot_dims, base, factor)}
    layer = {"type": "parallel", "mlp": _mlp(ff),
             "mixer": {"left": left, "right": {"heads": right_heads, "dim": right_dim, "vdim": right_vdim, "tau": tau}}}
    return layer, rank


def retention_layer(heads=3, dim=12, vdim=20, decay=(0.9, 0.97, 0.995), rot_dims=12, base=500.0, ff=None):
    return {"type": "retention", "mlp": _mlp(ff),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay), **_rot(rot_dims, base)}}


def make_config(layers, vocab=96, width=48, eps=1e-2, loop=None, mult=0.35, logit_scale=0.7, cap=9.0):
    """(config, ranks of the decay projections by layer); ``layers`` may hold (layer, rank) pairs."""
    ranks = {i: l[1] for i, l in enumerate(layers) if isinstance(l, tuple)}
    cfg = {"architecture": "Surodra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
           "logit_scale": logit_scale, "logit_softcap": cap,
           "layers": [l[0] if isinstance(l, tuple) else l for l in layers]}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg, ranks


def make_weights(cfg, ranks, seed=0):
    g = torch.Generator().manual_seed(seed)
    Wd, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def lin(o, i, s=1.0):
        return rnd(o, i, s=s / math.sqrt(i))

    def near1(*shape):
        return 1.0 + rnd(*shape, s=0.15)
    W = {"embed": rnd(V, Wd), "head": lin(V, Wd, 6.0)}

    def norm(name):
        W.update({name: near1(Wd), name + ".b": rnd(Wd, s=0.2), name + ".alpha": 0.5 + 0.3 * torch.rand((), generator=g)})
    norm("final.norm")
    if cfg.get("loop"):
        W["loop.step"] = rnd(cfg["loop"]["times"], Wd, s=0.6)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        norm(p + "norm1")
        if L["type"] == "delta":
            H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            W.update({p + "mix.q": lin(G * D, Wd, 2.0), p + "mix.k": lin(G * D, Wd, 2.0), p + "mix.v": lin(H * E, Wd, 2.0),
                      p + "mix.b": lin(H, Wd, 2.0), p + "mix.a": lin(H, Wd, 2.0), p + "mix.g": lin(H * E, Wd, 2.0),
                      p + "mix.o": lin(Wd, H * E, 1.5), p + "mix.A_log": rnd(H, s=0.5) - 1.0, p + "mix.dt_bias": rnd(H) - 2.0,
                      p + "mix.norm": near1(E)})
            for n, c in (("q", G * D), ("k", G * D), ("v", H * E)):
                W[p + f"mix.{n}.conv"] = rnd(c, m["conv"], s=0.8)
        elif L["type"] == "retention":
            H, D, E = m["heads"], m["dim"], m["vdim"]
            W.update({p + "mix.q": lin(H * D, Wd, 2.0), p + "mix.k": lin(H * D, Wd, 2.0), p + "mix.v": lin(H * E, Wd, 2.0),
                      p + "mix.g": lin(H * E, Wd, 2.0), p + "mix.o": lin(Wd, H * E, 1.5)})
        else:
            a, b, R = m["left"], m["right"], ranks[i]
            H, G, D, E = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            W.update({p + "mix.left.q": lin(H * D, Wd, 2.0), p + "mix.left.k": lin(G * D, Wd, 2.0),
                      p + "mix.left.v": lin(G * E, Wd, 2.0), p + "mix.left.q.norm": 1.5 * near1(H * D),
                      p + "mix.left.k.norm": 1.5 * near1(G * D), p + "mix.left.sink": rnd(H) + 1.0,
                      p + "mix.left.g": lin(H, Wd, 2.0), p + "mix.left.o": lin(Wd, H * E),
                      p + "mix.left.out": 2.0 * near1(Wd)})
            H, D, E = b["heads"], b["dim"], b["vdim"]
            W.update({p + "mix.right.q": lin(H * D, Wd, 2.0), p + "mix.right.k": lin(H * D, Wd, 2.0),
                      p + "mix.right.v": lin(H * E, Wd, 2.0), p + "mix.right.g": lin(H * E, Wd, 2.0),
                      p + "mix.right.o": lin(Wd, H * E), p + "mix.right.norm": near1(E), p + "mix.right.a1": lin(R, Wd, 2.0),
                      p + "mix.right.a2": lin(H * D, R, 2.0), p + "mix.right.a2.b": rnd(H * D) + 1.0,
                      p + "mix.right.out": 2.0 * near1(Wd)})
        if L.get("mlp"):
            norm(p + "norm2")
            ff = L["mlp"]["ff"]
            W.update({p + "mlp.gate": lin(ff, Wd, 2.5), p + "mlp.up": lin(ff, Wd, 2.5), p + "mlp.down": lin(Wd, ff, 2.0)})
    # the checkpoint holds bfloat16: round once, so that oracle and engine read the same numbers
    return {k: v.to(torch.bfloat16) for k, v in W.items()}


def save_checkpoint(folder, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in W.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def logit_error(got, want):
    """Root mean square difference over the vocabulary with the mean taken off, relative to the logits' own spread."""
    d = torch.as_tensor(got).float() - torch.as_tensor(want).float()
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / torch.as_tensor(want).float().std(-1).clamp_min(1e-6)).max().item()
