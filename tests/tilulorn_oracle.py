"""A slow, whole-sequence implementation of the Tilulorn design, one function per mechanism, written from its equations
and sharing no code with the package: the oracle of tests/test_tilulorn.py.  Everything runs in fp32 (or fp64) on the CPU
over one whole sequence at a time; there is no cache, no batching and no portioning here.

Notation: x residual [L, W]; N(y) = y / rms(y) * w; a layer computes x <- x + mixer(N1 x), then x <- x + ff(N2 x).
"""
import json
import math
import os

import torch


# ---- norms ---------------------------------------------------------------------------------------------------------
def unit_rms(y, eps):
    return y / torch.sqrt((y * y).mean(-1, keepdim=True) + eps)


def rms_norm(y, w, eps):
    return unit_rms(y, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


# ---- rotation --------------------------------------------------------------------------------------------------------
def plain_frequencies(dims, base):
    return [base ** (-2.0 * i / dims) for i in range(dims // 2)]


def yarn_frequencies(dims, base, factor, original, fast, slow):
    def turn_dim(turns):
        return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(turn_dim(fast)), 0), min(math.ceil(turn_dim(slow)), dims - 1)
    out = []
    for i, f in enumerate(plain_frequencies(dims, base)):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * r + f * (1 - r))
    return out


def turn(x, freqs, pairs, size=1.0):
    """x [L, heads, D]; pair i of ``pairs`` (two index lists) turns by position * freqs[i]; cos and sin times ``size``."""
    L = x.shape[0]
    ang = torch.arange(L, dtype=torch.float64)[:, None] * torch.tensor(freqs, dtype=torch.float64)[None, :]
    c, s = (size * torch.cos(ang)).to(x.dtype)[:, None, :], (size * torch.sin(ang)).to(x.dtype)[:, None, :]
    first, second = pairs
    a, b = x[..., first], x[..., second]
    y = x.clone()
    y[..., first] = a * c - b * s
    y[..., second] = b * c + a * s
    return y


def rotate_neighbours(x, rot):
    """Values 2i and 2i + 1 form a pair; every frequency divided by the factor."""
    dims = int((rot or {}).get("dims", 0) or 0)
    if dims == 0:
        return x
    factor = rot["scaling"]["factor"] if rot.get("scaling") else 1.0
    f = [v / factor for v in plain_frequencies(dims, rot["base"])]
    return turn(x, f, (list(range(0, dims, 2)), list(range(1, dims, 2))))


def rotate_halves_yarn(x, rot):
    """Values i and i + dims / 2 form a pair; frequencies of long wavelengths divided by the factor."""
    dims = int((rot or {}).get("dims", 0) or 0)
    if dims == 0:
        return x
    f, size = plain_frequencies(dims, rot["base"]), 1.0
    sc = rot.get("scaling")
    if sc:
        f = yarn_frequencies(dims, rot["base"], sc["factor"], sc["original"], sc["fast"], sc["slow"])
        size = 0.1 * math.log(sc["factor"]) + 1.0
    return turn(x, f, (list(range(dims // 2)), list(range(dims // 2, dims))), size)


# ---- mixers ------------------------------------------------------------------------------------------------------------
def latent_mixer(h, w, m, eps):
    """Keys and values come out of one normed latent per token; one rotated key part serves every head."""
    L = h.shape[0]
    H, D, P, E, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (rms_norm(h @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).view(L, H, D + P)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :R], w["dkv.norm"], eps)
    k = (c @ w["uk"].T).view(L, H, D)
    v = (c @ w["uv"].T).view(L, H, E)
    k_rot = rotate_halves_yarn(down[:, None, R:], m.get("rot"))[:, 0]
    q_rot = rotate_halves_yarn(q[..., D:], m.get("rot"))
    unseen = torch.arange(L)[None, :] > torch.arange(L)[:, None]
    gate = torch.sigmoid(h @ w["g"].T)
    out = []
    for n in range(H):
        s = (q[:, n, :D] @ k[:, n].T + q_rot[:, n] @ k_rot.T) * m["scale"]
        p = torch.softmax(s.masked_fill(unseen, float("-inf")), -1)
        out.append((p @ v[:, n]) * gate[:, n: n + 1])
    return torch.cat(out, -1) @ w["o"].T


def window_mixer(h, w, m, eps):
    """Sliding-window attention whose values are its keys before norm and rotation; a sink in every denominator."""
    L = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    k_raw = h @ w["k"].T
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps)             # over the whole projection, not per head
    k = rms_norm(k_raw, w["k.norm"], eps)
    v = k_raw.view(L, G, D)
    q, k = rotate_neighbours(q.view(L, H, D), m.get("rot")), rotate_neighbours(k.view(L, G, D), m.get("rot"))
    back = torch.arange(L)[:, None] - torch.arange(L)[None, :]
    seen = back >= 0
    if m.get("mask"):
        seen = seen & (back < m["mask"]["size"])
    gate = torch.sigmoid(h @ w["g"].T)
    out = []
    for n in range(H):
        g = n // (H // G)
        s = ((q[:, n] @ k[:, g].T) * m["scale"]).masked_fill(~seen, float("-inf"))
        top = torch.maximum(s.max(-1, keepdim=True).values, w["sink"][n])
        e = torch.exp(s - top)
        p = e / (e.sum(-1, keepdim=True) + torch.exp(w["sink"][n] - top))
        out.append((p @ v[:, g]) * gate[:, n: n + 1])
    return torch.cat(out, -1) @ w["o"].T


def shifted_mix(h, mu):
    """h + (h' - h) mu, h' the row of the token before (zeros before the first)."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def bonus_memory(r, k, v, decay, u):
    """r, k, decay [L, H, D], v [L, H, E], u [H, D]: read the old memory plus the own token through the bonus, then fade
    and write:  o_t = (S + diag(u) k_t v_t^T)^T r_t,  S <- diag(decay_t) S + k_t v_t^T."""
    L, H, D = r.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=r.dtype)
    out = []
    for t in range(L):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out.append(((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1))
        S = decay[t][:, :, None] * S + kv
    return torch.stack(out)


def wkv_mixer(h, w, m, eps):
    L = h.shape[0]
    H, D = m["heads"], m["dim"]
    mix = {s: shifted_mix(h, w["mu." + s]) for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[s].T).view(L, H, D) for s in "rkv")
    z = torch.tanh(mix["w"] @ w["w1"].T) @ w["w2"].T + w["w0"]
    decay = torch.exp(-torch.exp(z)).view(L, H, D)
    o = unit_rms(bonus_memory(r, k, v, decay, w["u"]), eps).reshape(L, H * D) * w["norm"]
    return (o * silu(mix["g"] @ w["g"].T)) @ w["o"].T


MIXERS = {"latent_attention": latent_mixer, "attention": window_mixer, "wkv": wkv_mixer}


# ---- feed-forward ------------------------------------------------------------------------------------------------------
def table_experts(h, w, tokens):
    """The token id alone picks the experts; each counts 1 / (how many a token has)."""
    out = torch.zeros_like(h)
    for t, tok in enumerate(tokens):
        row = w["table"][tok].tolist()
        for e in row:
            e = int(e)
            a = silu(w[f"e{e}.gate"] @ h[t]) * (w[f"e{e}.up"] @ h[t])
            out[t] += (w[f"e{e}.down"] @ a) / len(row)
    return out


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
    W = {n: t.to(dtype) if t.is_floating_point() else t for n, t in weights.items()}
    eps = cfg["norm"]["eps"]
    e = W["embed"][torch.tensor(tokens)]
    x, trail = e, []
    for i, t, first in run_list(len(cfg["layers"]), cfg.get("loop")):
        spec = cfg["layers"][i]
        if first:
            x = torch.cat([x, e], -1) @ W["loop.in"].T + W["loop.step"][t]
        x = x + MIXERS[spec["type"]](rms_norm(x, W[f"l{i}.norm1"], eps), sub(W, f"l{i}.mix."), spec["mixer"], eps)
        if spec.get("mlp"):
            x = x + table_experts(rms_norm(x, W[f"l{i}.norm2"], eps), sub(W, f"l{i}.mlp."), tokens)
        trail.append(x)
    y = rms_norm(x, W["final.norm"], eps) @ W["head"].T
    return (y, torch.stack(trail)) if want_layers else y


# ---- small random models ---------------------------------------------------------------------------------------------
def _mlp(ff, experts, top):
    return None if ff is None else {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def latent_layer(heads=3, dim=12, rot_dim=8, vdim=20, kv_rank=24, q_rank=28, base=300.0, scaling=(3.0, 24, 4.0, 0.5),
                 scale=0.25, ff=24, experts=5, top=2):
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mlp": _mlp(ff, experts, top),
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "scale": scale, "rot": rot}}


def window_layer(heads=4, kv_heads=2, dim=12, window=21, rot_dims=8, base=200.0, factor=2.5, scale=0.3, ff=20, experts=4,
                 top=1):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": window}}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims, **({"scaling": {"factor": factor}} if factor else {})}
    return {"type": "attention", "mlp": _mlp(ff, experts, top), "mixer": m}


def wkv_layer(heads=3, dim=12, rank=5, ff=16, experts=3, top=3):
    return {"type": "wkv", "mlp": _mlp(ff, experts, top), "mixer": {"heads": heads, "dim": dim}}, rank


def make_config(layers, vocab=96, width=48, eps=5e-2, loop=None):
    """(config, ranks of the decay projections by layer); ``layers`` may hold (layer, rank) pairs."""
    ranks = {i: l[1] for i, l in enumerate(layers) if isinstance(l, tuple)}
    cfg = {"architecture": "Tilulorn", "vocab": vocab, "width": width, "norm": {"eps": eps},
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
    W = {"embed": rnd(V, Wd), "head": lin(V, Wd, 4.0), "final.norm": near1(Wd)}
    if cfg.get("loop"):
        W["loop.in"] = torch.cat([0.6 * torch.eye(Wd) + lin(Wd, Wd, 0.3), lin(Wd, Wd, 0.8)], -1)
        W["loop.step"] = rnd(cfg["loop"]["times"], Wd, s=0.6)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        x = p + "mix."
        W[p + "norm1"] = near1(Wd)
        if L["type"] == "wkv":
            H, D = m["heads"], m["dim"]
            W.update({x + s: lin(H * D, Wd, 1.0 if s in "rk" else 2.0) for s in "rkvg"})
            W.update({x + "mu." + s: torch.rand(Wd, generator=g) * 0.9 for s in "rkvgw"})
            W.update({x + "w1": lin(ranks[i], Wd, 1.5), x + "w2": lin(H * D, ranks[i], 1.5), x + "w0": rnd(H * D) - 2.5,
                      x + "u": 0.5 + rnd(H, D, s=0.5), x + "norm": near1(H * D), x + "o": lin(Wd, H * D)})
        elif L["type"] == "attention":
            H, G, D = m["heads"], m["kv_heads"], m["dim"]
            W.update({x + "q": lin(H * D, Wd, 2.0), x + "k": lin(G * D, Wd, 2.0), x + "q.norm": 1.5 * near1(H * D),
                      x + "k.norm": 1.5 * near1(G * D), x + "sink": rnd(H) + 1.0, x + "g": lin(H, Wd, 2.0),
                      x + "o": lin(Wd, H * D)})
        else:
            H, D, P, E, R, Q = (m[n] for n in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            W.update({x + "dq": lin(Q, Wd, 2.0), x + "dq.norm": near1(Q), x + "uq": lin(H * (D + P), Q, 1.5),
                      x + "dkv": lin(R + P, Wd, 2.0), x + "dkv.norm": near1(R), x + "uk": lin(H * D, R, 1.5),
                      x + "uv": lin(H * E, R, 2.0), x + "g": lin(H, Wd, 2.0), x + "o": lin(Wd, H * E)})
        if L.get("mlp"):
            ff, n, top = L["mlp"]["expert"]["ff"], L["mlp"]["router"]["experts"], L["mlp"]["router"]["top"]
            W[p + "norm2"] = near1(Wd)
            for e in range(n):
                W.update({p + f"mlp.e{e}.gate": lin(ff, Wd, 2.0), p + f"mlp.e{e}.up": lin(ff, Wd, 2.0),
                          p + f"mlp.e{e}.down": lin(Wd, ff)})
            W[p + "mlp.table"] = torch.stack([torch.randperm(n, generator=g)[:top] for _ in range(V)]).to(torch.int32)
    # the checkpoint holds bfloat16: round once, so that oracle and engine read the same numbers
    return {k: v.to(torch.bfloat16) if v.is_floating_point() else v for k, v in W.items()}


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
