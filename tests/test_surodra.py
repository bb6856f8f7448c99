"""Surodra (per-head gated delta rule, softmax attention with sinks beside gated linear attention, retention, squashing
norms over an fp32 residual, a loop with a step row and the embedding output added between passes, soft-capped logits)
against the slow oracle of tests/surodra_oracle.py: every mechanism alone, then whole models through the engine's own
scheduler, page pool, state slots and step function -- on the CPU backend (fp32) and, marked gpu, through the HIP kernels
(fp32 and bf16).  Small random models are written to disk as checkpoints, so the loader and the configuration reader run
too."""
import pytest
import torch

import surodra_oracle as O
from vllm_distributed_amd import ops

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
CASES = [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)]
OP_CASES = [("cpu", torch.float32), pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
            pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)]
# 16-bit: models this narrow (48 values per row) average little rounding away; the crafted cases move by more
TOL = {"float32": 3e-4, "bfloat16": 0.12}
OP_TOL = {torch.float32: 3e-5, torch.bfloat16: 2.5e-2}


@pytest.fixture(autouse=True)
def _seed():
    torch.manual_seed(0)


def rel(got, want):
    got, want = got.float().cpu(), want.float().cpu()
    return ((got - want).norm() / want.norm().clamp_min(1e-20)).item()


def mixed_layers():
    """Every mixer with unequal sizes, with and without a feed-forward."""
    return [O.retention_layer(ff=24), O.delta_layer(), O.parallel_layer(ff=None), O.delta_layer(heads=3, kv_heads=1, dim=20,
                                                                                         vdim=8, conv=2, ff=None),
            O.parallel_layer(heads=3, kv_heads=3, dim=8, vdim=8, rot_dims=0, right_heads=1, right_dim=20, right_vdim=4,
                             tau=1.0, rank=1)]


def matrix_core_layers():
    """Heads of the widths the matrix-core attention kernels take in 16-bit runs, and recurrent heads of whole matrix
    tiles."""
    return [O.parallel_layer(heads=4, kv_heads=2, dim=64, vdim=64, rot_dims=32, scale=0.12, right_heads=2, right_dim=32,
                             right_vdim=64, ff=None),
            O.delta_layer(heads=4, kv_heads=2, dim=64, vdim=32),
            O.parallel_layer(heads=2, kv_heads=1, dim=128, vdim=128, rot_dims=128, factor=None, scale=0.09, right_heads=1,
                             right_dim=64, right_vdim=128, rank=16, ff=24),
            O.retention_layer(heads=2, dim=32, vdim=64, decay=(0.95, 0.999), rot_dims=32)]


def recurrent_layers():
    """No attention layer at all: the page pool is book-keeping only, every mixer lives in state slots."""
    return [O.delta_layer(heads=2, kv_heads=2, dim=32, vdim=16, conv=3), O.retention_layer(),
            O.delta_layer(heads=1, kv_heads=1, dim=5, vdim=70, conv=1, ff=None)]


LAYER_SETS = {"mixed": mixed_layers, "matrix_core": matrix_core_layers, "recurrent_only": recurrent_layers}
LOOPS = {"mixed": (1, 4, 2), "matrix_core": (0, 4, 2), "recurrent_only": (0, 2, 3)}


# ---- driving the engine ------------------------------------------------------------------------------------------
def run_schedule(folder, dtype, device, prompts, schedule, max_tokens, block_size=16, eager=True):
    """``schedule``: steps of (request, token count); every request ends when its tokens are used up.  Returns
    request -> logits [tokens, vocab] in the order the tokens ran."""
    from vllm_distributed_amd.entrypoints.trace_replay import TraceReplayer
    r = TraceReplayer(folder, dtype, max_tokens, block_size=block_size, device=device, enforce_eager=eager)
    at = {k: 0 for k in prompts}
    got = {k: [] for k in prompts}
    try:
        for step in schedule:
            entries, end = [], []
            for rid, n in step:
                lo, hi = at[rid], at[rid] + n
                entries.append({"id": rid, "tokens": prompts[rid][lo:hi], "want": list(range(n))})
                at[rid] = hi
                if hi == len(prompts[rid]):
                    end.append(rid)
            rows = torch.from_numpy(r.step(entries, end))
            o = 0
            for rid, n in step:
                got[rid].append(rows[o:o + n])
                o += n
    finally:
        r.shutdown()
    assert all(at[k] == len(prompts[k]) for k in prompts)
    return {k: torch.cat(v) for k, v in got.items()}


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def check(cfg, W, prompts, got, dtype):
    for rid, p in prompts.items():
        err = O.logit_error(got[rid], O.forward(cfg, W, p))
        assert err < TOL[dtype], f"request {rid}: logits differ by {err:.2e} of their spread"


def model(tmp_path, layers, seed=0, **kw):
    cfg, ranks = O.make_config(layers, **kw)
    W = O.make_weights(cfg, ranks, seed)
    return O.save_checkpoint(str(tmp_path / "m"), cfg, W), cfg, W


def pages(lens, bs, spare=3):
    """Scattered pages for sequences of the given lengths: (block table, number of blocks)."""
    nblk = sum(-(-n // bs) for n in lens) + spare
    perm = torch.randperm(nblk - 1) + 1
    table = torch.zeros(len(lens), max(-(-n // bs) for n in lens), dtype=torch.int32)
    o = 0
    for s, n in enumerate(lens):
        k = -(-n // bs)
        table[s, :k] = perm[o:o + k].int()
        o += k
    return table, nblk


def dev_(t, dev):
    return t.to(dev) if t is not None else None


# ---- mechanisms alone ----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("W_", [40, 301, 516, 1100, 2056, 4104])
def test_residual_under_squashing_norm(dev, dt, W_):
    """Up to two branches, plain or divided by their root mean square, an activation row and a step row, then the squash
    -- with values in its linear range, around its bend and far beyond it."""
    T, eps, coef = 5, 1e-2, 0.35
    alpha, w, b = torch.tensor([0.8]), 1 + 0.2 * torch.randn(W_), 0.3 * torch.randn(W_)
    wa, wb, step = 1 + 0.2 * torch.randn(W_), 1 + 0.2 * torch.randn(W_), torch.randn(W_)
    big = torch.randn(T, W_ + 8).to(dt)
    y0, y1, e = big[:, :W_], torch.randn(T, W_).to(dt), torch.randn(T, W_).to(dt)      # y0: rows with a pitch
    x0 = torch.randn(T, W_) * torch.tensor([0.01, 0.3, 1.0, 5.0, 60.0])[:, None]
    cases = [([], None, None), ([(y0, None)], None, None), ([(y1, wa)], None, step), ([(y0, wa), (y1, wb)], e, step),
             ([(y0, None), (y1, wb)], None, None), ([], e, step)]
    for branches, extra, st in cases:
        want = x0.clone()
        total = sum((O.unit_rms(y.float(), eps) * v if v is not None else y.float()) for y, v in branches)
        want = want + coef * total
        if extra is not None:
            want = want + extra.float()
        if st is not None:
            want = want + st
        x = x0.clone().to(dev)
        on_dev = [((big.to(dev)[:, :W_] if y is y0 else y.to(dev)), dev_(v, dev)) for y, v in branches]
        h = ops.residual_squash_norm(x, on_dev, coef, eps, alpha.to(dev), w.to(dev), b.to(dev), dt, dev_(extra, dev),
                                     dev_(st, dev))
        torch.testing.assert_close(x.cpu(), want, atol=2e-5, rtol=1e-5)
        exact = O.squash_norm(want, alpha, w, b)
        torch.testing.assert_close(h.float().cpu(), exact, atol=2e-6 if dt == torch.float32 else 8e-3,
                                   rtol=2e-6 if dt == torch.float32 else 8e-3)


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("scale,cap", [(0.4, 3.0), (1.0, 0.0), (2.0, 30.0)])
def test_scaled_and_capped_logits(dev, dt, scale, cap):
    x = (torch.randn(7, 301) * torch.logspace(-3, 2, 301)).to(dt)
    y = x.float() * scale
    want = cap * torch.tanh(y / cap) if cap else y
    got = ops.scaled_softcap(x.to(dev), scale, cap)
    assert got.dtype == torch.float32
    torch.testing.assert_close(got.cpu(), want, atol=1e-6, rtol=2e-6)


def test_linearly_scaled_frequencies():
    from vllm_distributed_amd.layers.rotary import half_split_cos_sin
    x = torch.randn(50, 2, 20)
    for rot in ({"base": 77.0, "dims": 12, "scaling": {"factor": 2.5}}, {"base": 1e4, "dims": 20}):
        n = rot["dims"] // 2
        sc = rot.get("scaling")
        cs = half_split_cos_sin(50, rot["dims"], rot["base"], dict(kind="linear", **sc) if sc else None,
                                torch.device("cpu"))[:50, None]
        a, b = x[..., :n], x[..., n: 2 * n]
        c, s = cs[..., :n], cs[..., n:]
        got = torch.cat([a * c - b * s, b * c + a * s, x[..., 2 * n:]], -1)
        torch.testing.assert_close(got, O.rotate(x, rot), atol=1e-5, rtol=1e-5)


# (heads, key heads, D, Dv, rotated, page size): any-size kernel and, in 16 bits, the matrix-core forms
ATTN = [(4, 2, 12, 20, 8, 16), (3, 1, 20, 8, 0, 32), (1, 1, 5, 7, 4, 16), (8, 2, 64, 64, 16, 16), (4, 4, 128, 128, 128, 32),
        (2, 1, 72, 40, 6, 16), (16, 1, 64, 64, 12, 16), (4, 2, 96, 96, 32, 32), (2, 2, 256, 256, 48, 16)]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,G,D,E,rot,bs", ATTN)
def test_attention_with_projection_norm_sink_and_head_gate(dev, dt, H, G, D, E, rot, bs):
    """Ragged batch on scattered pages -- a decoded token, a portion behind cached context that starts inside a page, a
    whole prompt -- against the oracle of each sequence.  Rows of unequal size, so that a norm per head instead of one
    over the projection is far off."""
    from vllm_distributed_amd.layers.rotary import half_split_cos_sin
    eps, scale = 1e-3, 2.0 * D ** -0.5
    lens, news = [75, 53, 20], [1, 11, 20]
    nq, nk, nv = H * D, G * D, G * E
    Wd = nq + nk + nv + H
    xs = []
    for n in lens:
        x = torch.randn(n, Wd)
        x[:, :D] *= 3.0                                   # head 0 carries most of the queries' size
        xs.append(x.to(dt))
    eye = torch.eye(Wd)
    w = {"q": eye[:nq], "k": eye[nq: nq + nk], "v": eye[nq + nk: nq + nk + nv], "g": eye[nq + nk + nv:],
         "q.norm": 1 + 0.3 * torch.randn(nq), "k.norm": 1 + 0.3 * torch.randn(nk), "sink": 2.0 * torch.randn(H) + 1,
         "o": torch.eye(H * E)}
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale}
    if rot:
        m["rot"] = {"base": 60.0, "dims": rot, "scaling": {"factor": 1.5}}
    want = torch.cat([O.sink_attention(x.float(), w, m, eps)[n - k:] for x, n, k in zip(xs, lens, news)])
    no_sink = torch.cat([O.sink_attention(x.float(), dict(w, sink=torch.full((H,), -1e9)), m, eps)[n - k:]
                         for x, n, k in zip(xs, lens, news)])
    assert rel(no_sink, want) > 0.1
    table, nblk = pages(lens, bs)
    kc = torch.zeros(nblk, G, bs, D, dtype=dt, device=dev)
    vc = torch.zeros(nblk, G, E, bs, dtype=dt, device=dev)
    cs = half_split_cos_sin(128, rot, 60.0, dict(kind="linear", factor=1.5), torch.device(dev)) if rot else None
    sink = w["sink"].to(dev)
    mfma = ops.masked_attention_mfma_ok(H, G, D, E, 1, sink, dt, dev == "cuda")

    def write(rows, pos, slots):
        return ops.qk_norm_rope_cache(rows.to(dev), H, G, D, E, 1, w["q.norm"].to(dev), w["k.norm"].to(dev), cs, pos.to(dev),
                                      rot, eps, kc, vc, slots.to(dev), by_map=mfma, whole_norm=True)
    for s, (n, k) in enumerate(zip(lens, news)):          # context first, as earlier steps would have
        if n - k:
            pos = torch.arange(n - k)
            write(xs[s][: n - k], pos, table[s, pos // bs].long() * bs + pos % bs)
    pos = torch.cat([torch.arange(n - k, n) for n, k in zip(lens, news)])
    slots = torch.cat([table[s, torch.arange(n - k, n) // bs].long() * bs + torch.arange(n - k, n) % bs
                       for s, (n, k) in enumerate(zip(lens, news))])
    rows = torch.cat([x[n - k:] for x, n, k in zip(xs, lens, news)])
    qn = write(rows, pos, slots)
    qsl = torch.tensor([0] + list(torch.tensor(news).cumsum(0)), dtype=torch.int32).to(dev)
    sl = torch.tensor(lens, dtype=torch.int32).to(dev)
    gate = rows.to(dev)[:, Wd - H:]
    if mfma:
        pq = (qsl[1:] - qsl[1]).contiguous()
        for splits in (1, 3):
            got = ops.masked_softmax_attention_mfma(qn, kc, vc, table.to(dev), sl, qsl, pq, 1, 1, 2, int(sum(news[1:])), 1,
                                                    splits, max(news), scale, H, sink=sink, gate=gate)
            assert rel(got, want) < OP_TOL[dt], splits
    got = ops.masked_softmax_attention(qn.view(-1, H, D), kc, vc, table.to(dev), sl, qsl, scale, sink=sink, gate=gate,
                                       max_query_len=max(news))
    assert rel(got, want) < OP_TOL[dt]


# portions of two sequences: short ones take the token-by-token form, longer ones the chunk-parallel form; portions that
# end inside, at and just behind blocks of sixteen tokens and chunks of 64 and 128
PORTIONS = [[(0, 2), (1, 4)], [(0, 17)], [(1, 1), (0, 1)], [(1, 140), (0, 129)], [(0, 16), (1, 33)], [(0, 1), (1, 64)],
            [(0, 65), (1, 3)], [(1, 1), (0, 1)]]
TOTAL = [sum(n for st in PORTIONS for s, n in st if s == q) for q in (0, 1)]


def in_portions(xs, dev, dt, launch):
    """Runs PORTIONS through ``launch(x, qsl, lens, table, max_new, first_long, positions)``; both splits of the step's
    sequences (short ones announced as such, or not) are used in turn."""
    slot = torch.tensor([[4], [2]], dtype=torch.int32, device=dev)
    done, got = [0, 0], [[], []]
    for turn, step in enumerate(PORTIONS):
        order = sorted(step, key=lambda a: a[1] > 1)
        x = torch.cat([xs[s][done[s]: done[s] + n] for s, n in order]).to(dt).to(dev)
        pos = torch.cat([torch.arange(done[s], done[s] + n) for s, n in order]).to(dev)
        qsl = torch.tensor([0] + list(torch.tensor([n for _, n in order]).cumsum(0)), dtype=torch.int32, device=dev)
        lens = torch.tensor([done[s] + n for s, n in order], dtype=torch.int32, device=dev)
        few = sum(n == 1 for _, n in order) if turn % 2 == 0 else 0
        out = launch(x, qsl, lens, slot[[s for s, _ in order]], max(n for _, n in order), few, pos).cpu()
        o = 0
        for s, n in order:
            got[s].append(out[o:o + n])
            o += n
            done[s] += n
    assert done == TOTAL
    return [torch.cat(g) for g in got]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,G,D,E,taps", [(4, 2, 12, 20, 3), (3, 1, 64, 32, 2), (1, 1, 37, 130, 4), (2, 2, 130, 64, 4),
                                          (6, 3, 128, 128, 3), (5, 1, 32, 7, 2)])
def test_delta_rule_with_a_decay_per_head(dev, dt, H, G, D, E, taps):
    """Portions in state slots that hold stale content, against the oracle on the whole sequences."""
    eps = 1e-4
    C = 2 * G * D + H * E
    Wd = C + H * E + 2 * H
    xs = [torch.randn(n, Wd).to(dt).float() for n in TOTAL]
    eye = torch.eye(Wd)
    P = {"q": eye[: G * D], "k": eye[G * D: 2 * G * D], "v": eye[2 * G * D: C], "g": eye[C: C + H * E],
         "b": eye[C + H * E: C + H * E + H], "a": eye[C + H * E + H:], "q.conv": torch.randn(G * D, taps),
         "k.conv": torch.randn(G * D, taps), "v.conv": torch.randn(H * E, taps), "A_log": torch.randn(H) * 1.5 - 2,
         "dt_bias": torch.randn(H), "norm": 1 + 0.2 * torch.randn(E), "o": torch.eye(H * E)}
    P = {k: (v.to(dt).float() if k.endswith("conv") else v) for k, v in P.items()}
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E}
    want = [O.delta_mixer(x, P, m, eps) for x in xs]
    conv_w = torch.cat([P["q.conv"], P["k.conv"], P["v.conv"]]).to(dt).to(dev)
    conv_state = torch.full((5, C, taps - 1), 7.0, device=dev, dtype=dt)
    state = torch.full((5, H, E, D), 3.0, device=dev)

    def launch(x, qsl, lens, tbl, longest, few, pos):
        xc = ops.causal_conv1d(x[:, :C], conv_w, None, conv_state, qsl, lens, tbl, longest)
        return ops.gated_delta_rule_head(xc, x[:, C + H * E + H:], x[:, C + H * E: C + H * E + H], x[:, C: C + H * E],
                                         P["A_log"].to(dev), P["dt_bias"].to(dev), P["norm"].to(dev), state, qsl, lens, tbl,
                                         H, G, D, E, eps, longest, few)
    got = in_portions(xs, dev, dt, launch)
    for g, w in zip(got, want):
        assert rel(g, w) < OP_TOL[dt]
    assert (state[[0, 1, 3]] == 3.0).all()                # nobody else's slot


# (heads, D, Dv, tau, decays of the channels): ordinary ones, ones that vanish within a few tokens (their running products
# underflow inside a block), and a mixture
GLA = [(3, 12, 20, 5.0, 1.0), (2, 64, 128, 12.0, 0.0), (1, 5, 70, 1.0, 1.0), (2, 128, 64, 0.3, -3.0), (1, 33, 8, 1.0, -6.0),
       (2, 160, 36, 8.0, 1.0), (1, 32, 300, 2.0, -2.0)]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,D,E,tau,bias", GLA)
def test_gated_linear_attention(dev, dt, H, D, E, tau, bias):
    eps = 1e-4
    nk, nv = H * D, H * E
    Wd = 3 * nk + 2 * nv
    xs = [torch.randn(n, Wd).to(dt).float() for n in TOTAL]
    eye = torch.eye(Wd)
    P = {"q": eye[:nk], "k": eye[nk: 2 * nk], "v": eye[2 * nk: 2 * nk + nv], "g": eye[2 * nk + nv: 2 * nk + 2 * nv],
         "a1": eye[2 * nk + 2 * nv:], "a2": torch.eye(nk), "a2.b": 3.0 * torch.randn(nk) + bias,
         "norm": 1 + 0.2 * torch.randn(E), "o": torch.eye(nv)}
    want = [O.gated_linear_mixer(x, P, {"heads": H, "dim": D, "vdim": E, "tau": tau}, eps) for x in xs]
    state = torch.full((5, H, E, D), 3.0, device=dev)

    def launch(x, qsl, lens, tbl, longest, few, pos):
        return ops.linear_attention(x[:, :nk], x[:, nk: 2 * nk], x[:, 2 * nk: 2 * nk + nv],
                                    x[:, 2 * nk + nv: 2 * nk + 2 * nv], P["norm"].to(dev), state, qsl, lens, tbl, H, D, E,
                                    eps, longest, z=x[:, 2 * nk + 2 * nv:], z_bias=P["a2.b"].to(dev), tau=tau,
                                    q_scale=D ** -0.5, first_long_seq=few)
    got = in_portions(xs, dev, dt, launch)
    for g, w in zip(got, want):
        assert rel(g, w) < OP_TOL[dt]
    assert (state[[0, 1, 3]] == 3.0).all()


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,D,E,rot,decay", [(3, 12, 20, 12, (0.5, 0.97, 0.999)), (2, 64, 64, 64, (0.99, 1.0)),
                                             (1, 40, 130, 16, (0.9,)), (2, 128, 128, 96, (0.0, 0.998)),
                                             (1, 6, 5, 4, (0.8,)), (1, 256, 70, 8, (0.01,)), (4, 16, 32, 0, (0.9,) * 4)])
def test_retention(dev, dt, H, D, E, rot, decay):
    """Fixed decays, one of them zero (nothing survives a token) and one of them one (nothing fades)."""
    from vllm_distributed_amd.layers.linear_attention import MIN_LOG_DECAY
    from vllm_distributed_amd.layers.rotary import half_split_cos_sin
    eps = 1e-4
    nk, nv = H * D, H * E
    xs = [torch.randn(n, 2 * nk + 2 * nv).to(dt).float() for n in TOTAL]
    eye = torch.eye(2 * nk + 2 * nv)
    P = {"q": eye[:nk], "k": eye[nk: 2 * nk], "v": eye[2 * nk: 2 * nk + nv], "g": eye[2 * nk + nv:], "o": torch.eye(nv)}
    m = {"heads": H, "dim": D, "vdim": E, "decay": decay}
    if rot:
        m["rot"] = {"base": 900.0, "dims": rot}
    want = [O.retention_mixer(x, P, m, eps) for x in xs]
    state = torch.full((5, H, E, D), 3.0, device=dev)
    cs = half_split_cos_sin(max(TOTAL), rot, 900.0, None, torch.device(dev)) if rot else None
    ld = torch.tensor(decay).log().clamp_min(MIN_LOG_DECAY).to(dev)

    def launch(x, qsl, lens, tbl, longest, few, pos):
        return ops.linear_attention(x[:, :nk], x[:, nk: 2 * nk], x[:, 2 * nk: 2 * nk + nv], x[:, 2 * nk + nv:], None, state,
                                    qsl, lens, tbl, H, D, E, eps, longest, log_decay=ld, cos_sin=cs,
                                    positions=pos if rot else None, rot=rot, k_scale=D ** -0.5, first_long_seq=few)
    got = in_portions(xs, dev, dt, launch)
    for g, w in zip(got, want):
        assert rel(g, w) < OP_TOL[dt]
    assert (state[[0, 1, 3]] == 3.0).all()


# ---- configuration and loading -----------------------------------------------------------------------------------------
def test_rank_of_the_decay_projection_comes_from_its_shape(tmp_path):
    from vllm_distributed_amd.config import load_hf_config
    folder, cfg, _ = model(tmp_path, [O.parallel_layer(rank=11)])
    hf = load_hf_config(folder)
    assert hf.architectures == ["SurodraForCausalLM"] and hf.layers[0]["mixer"]["right"]["decay_rank"] == 11
    assert hf.hidden_size == cfg["width"] and hf.vocab_size == cfg["vocab"]


def test_tensor_without_a_place_is_refused(tmp_path):
    from vllm_distributed_amd.entrypoints.trace_replay import TraceReplayer
    folder, cfg, W = model(tmp_path, [O.retention_layer()])
    O.save_checkpoint(folder, cfg, dict(W, **{"l0.mix.norm": torch.ones(3)}))
    with pytest.raises(ValueError, match="no place"):
        TraceReplayer(folder, "float32", 64, device="cpu", enforce_eager=True)


def test_unknown_mixer_is_refused():
    from vllm_distributed_amd.models.surodra import normalise_config
    cfg, _ = O.make_config([O.retention_layer()])
    cfg["layers"][0] = dict(cfg["layers"][0], type="conv_only")
    with pytest.raises(ValueError, match="unknown mixer"):
        normalise_config(cfg)


# ---- whole models through the engine --------------------------------------------------------------------------------
VARIANTS = {
    "mixed_looped": dict(layers=mixed_layers(), loop=(1, 4, 2)),
    "no_loop": dict(layers=mixed_layers()[:4]),
    "loop_over_everything": dict(layers=mixed_layers()[1:3], loop=(0, 2, 3)),
    "loop_once_at_the_end": dict(layers=mixed_layers()[:3], loop=(2, 3, 1)),
    "matrix_core": dict(layers=matrix_core_layers(), loop=(1, 3, 2), width=64),
    "delta_only": dict(layers=[O.delta_layer(heads=1, kv_heads=1, dim=40, vdim=8, conv=1, ff=None),
                               O.delta_layer(heads=6, kv_heads=3, dim=16, vdim=4, conv=5)], loop=(1, 2, 2), mult=1.0),
    "parallel_only": dict(layers=[O.parallel_layer(heads=1, kv_heads=1, dim=4, vdim=6, rot_dims=2, factor=None, ff=None),
                                  O.parallel_layer(heads=6, kv_heads=2, dim=10, vdim=4, rot_dims=10, right_heads=2,
                                                   right_dim=4, right_vdim=40, tau=12.0, rank=20)], cap=2.0, eps=1e-6),
    "retention_only": dict(layers=[O.retention_layer(heads=1, dim=40, vdim=8, decay=(0.99,), rot_dims=0),
                                   O.retention_layer(heads=2, dim=6, vdim=36, decay=(0.7, 0.9999), rot_dims=4, ff=17)],
                           loop=(0, 1, 4), logit_scale=1.0),
    "odd_widths": dict(layers=[O.delta_layer(heads=3, kv_heads=3, dim=7, vdim=9, conv=3, ff=13),
                               O.parallel_layer(heads=3, kv_heads=1, dim=6, vdim=5, rot_dims=4, right_heads=3, right_dim=5,
                                                right_vdim=7, rank=3, ff=9),
                               O.retention_layer(heads=2, dim=6, vdim=5, decay=(0.9, 0.99), rot_dims=6)],
                       width=45, vocab=37, loop=(0, 2, 2), eps=1e-3),
}


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("name", list(VARIANTS))
def test_whole_prompt(tmp_path, dev, dtype, name):
    kw = dict(VARIANTS[name])
    folder, cfg, W = model(tmp_path, kw.pop("layers"), seed=3, **kw)
    prompts = {"a": tokens(85, cfg["vocab"], 1), "b": tokens(1, cfg["vocab"], 2)}
    got = run_schedule(folder, dtype, dev, prompts, [[("a", 85)], [("b", 1)]], 112)
    check(cfg, W, prompts, got, dtype)


def test_the_loops_additions_matter():
    """The oracle itself: the step rows of every pass, the sinks and the soft cap change the logits by far more than the
    fp32 tolerance of the comparisons above and below."""
    cfg, ranks = O.make_config(mixed_layers(), loop=(1, 4, 2))
    W = O.make_weights(cfg, ranks, 3)
    p = tokens(12, cfg["vocab"], 1)
    full = O.forward(cfg, W, p)
    for k, row in (("loop.step", 0), ("loop.step", 1), ("l2.mix.left.sink", None)):
        t = W[k].clone()
        if row is None:
            t[:] = -60.0
        else:
            t[row] = 0
        assert O.logit_error(O.forward(cfg, dict(W, **{k: t}), p), full) > 0.05, (k, row)
    assert O.logit_error(O.forward(dict(cfg, logit_softcap=1e6), W, p), full) > 0.02


@pytest.mark.parametrize("dev", DEVICES)
def test_residual_after_every_layer_run(tmp_path, dev):
    """The framework's residual after every layer run against the oracle's trail (looped layers count each time): what
    the next pass adds (embedding output, step row) is taken off again, since it joins in the same launch."""
    from vllm_distributed_amd.entrypoints.trace_replay import TraceReplayer
    folder, cfg, W = model(tmp_path, mixed_layers(), seed=1, loop=(1, 4, 3))
    p = tokens(20, cfg["vocab"], 1)
    _, trail = O.forward(cfg, W, p, want_layers=True)
    r = TraceReplayer(folder, "float32", 64, device=dev, enforce_eager=True)
    seen = []
    mdl = r.core.model_executor.worker.model_runner.model

    def keep(mod, args, out):
        x, extra, step = args[0], args[5], args[6]
        y = x.clone()
        y = y - extra.float() if extra is not None else y
        y = y - step.float() if step is not None else y
        seen.append(y[: len(p)].cpu())
    hooks = [b.register_forward_hook(keep) for b in mdl.layers]
    try:
        seen.clear()
        r.step([{"id": "a", "tokens": p, "want": [0]}], ["a"])
    finally:
        for h in hooks:
            h.remove()
        r.shutdown()
    assert len(seen) == len(trail) == 11
    torch.testing.assert_close(torch.stack(seen), trail, atol=3e-4, rtol=3e-4)


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("layers", list(LAYER_SETS))
def test_prefill_equals_decoding_token_by_token(tmp_path, dev, dtype, layers):
    folder, cfg, W = model(tmp_path, LAYER_SETS[layers](), seed=4, loop=LOOPS[layers])
    p = tokens(70, cfg["vocab"], 5)
    got = run_schedule(folder, dtype, dev, {"a": p}, [[("a", 11)]] + [[("a", 1)]] * 59, 80)
    check(cfg, W, {"a": p}, got, dtype)
    whole = run_schedule(folder, dtype, dev, {"a": p}, [[("a", 70)]], 80)
    assert O.logit_error(got["a"], whole["a"]) < TOL[dtype]


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("block_size", [16, 32])
@pytest.mark.parametrize("layers", list(LAYER_SETS))
def test_portions_down_to_two_tokens(tmp_path, dev, dtype, block_size, layers):
    folder, cfg, W = model(tmp_path, LAYER_SETS[layers](), seed=6, loop=LOOPS[layers])
    p = tokens(140, cfg["vocab"], 7)
    cuts = [2, 3, 11, 2, 16, 1, 17, 2, 7, 12, 1, 1, 15, 18, 32]
    assert sum(cuts) == 140
    got = run_schedule(folder, dtype, dev, {"a": p}, [[("a", n)] for n in cuts], 160, block_size=block_size)
    check(cfg, W, {"a": p}, got, dtype)


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("layers", list(LAYER_SETS))
def test_unequal_requests_share_steps_and_reuse_pages_and_slots(tmp_path, dev, dtype, layers):
    """Seven requests over four slots and a pool of 10 pages: portions beside single tokens, requests that sit out
    steps, pages and slots of finished requests taken by later ones; each against itself alone (the oracle)."""
    folder, cfg, W = model(tmp_path, LAYER_SETS[layers](), seed=8, loop=LOOPS[layers])
    V = cfg["vocab"]
    prompts = {"a": tokens(40, V, 1), "b": tokens(17, V, 2), "c": tokens(1, V, 3), "d": tokens(33, V, 4),
               "e": tokens(48, V, 5), "f": tokens(9, V, 6), "g": tokens(30, V, 7)}
    sched = [[("a", 13), ("b", 2)], [("a", 1), ("b", 15), ("c", 1)], [("a", 20), ("d", 16)],
             [("d", 1), ("a", 1)], [("a", 5), ("d", 16)],                       # a, b, c, d done: their pages return
             [("e", 31), ("f", 2)], [("e", 1), ("f", 1), ("g", 2)], [("g", 28), ("e", 1)],
             [("e", 15), ("f", 6)]]
    got = run_schedule(folder, dtype, dev, prompts, sched, 160)
    check(cfg, W, prompts, got, dtype)


NEEDLES = {
    "delta": O.delta_layer(heads=2, kv_heads=1, dim=8, vdim=8, conv=2, ff=None),
    "left": O.parallel_layer(heads=2, kv_heads=1, dim=8, vdim=8, rot_dims=0, scale=0.3, right_heads=2, right_dim=8,
                             right_vdim=8, tau=14.0, ff=None),
    "right": O.parallel_layer(heads=2, kv_heads=1, dim=8, vdim=8, rot_dims=0, scale=0.3, right_heads=2, right_dim=8,
                              right_vdim=8, tau=14.0, ff=None),
    "retention": O.retention_layer(heads=2, dim=8, vdim=8, decay=(0.9999, 0.9998), rot_dims=0),
}


def needle_model(kind):
    """One layer.  Token 0 is a 'needle' that alone fills key direction 0 of head 0; every other token's query looks
    there, so the logits of all later positions hang on whether the needle is still seen or remembered."""
    cfg, ranks = O.make_config([NEEDLES[kind]], vocab=64, width=32, mult=1.5)
    W = {k: v.float() for k, v in O.make_weights(cfg, ranks, 11).items()}
    emb = 0.2 * W["embed"]
    emb[:, 0] = 0
    emb[:, 2] = 3.0                                    # every token is mostly e2 ...
    emb[0] = 0
    emb[0, 0] = 3.0                                    # ... except the needle, alone along e0
    W["embed"] = emb
    W["l0.norm1"], W["l0.norm1.b"], W["l0.norm1.alpha"] = torch.ones(32), torch.zeros(32), torch.tensor(1.0)
    p = "l0.mix." + (kind + "." if kind in ("left", "right") else "")
    q, k = 0.03 * W[p + "q"], 0.03 * W[p + "k"]
    q[0], k[0] = 0, 0
    q[0, 2] = k[0, 0] = 4.0
    W[p + "q"], W[p + "k"] = q, k
    if kind == "delta":
        W[p + "A_log"][:] = -9.0
        for n in ("q", "k"):
            W[p + n + ".conv"][0] = torch.tensor([0.25, 1.0])
        W[p + "b"] = torch.abs(W[p + "b"])             # (mostly) whole writes
    if kind in ("left", "right"):                      # the other side is silent
        W["l0.mix." + ("right" if kind == "left" else "left") + ".out"][:] = 0.0
    if kind == "left":
        W[p + "sink"][0] = 3.0
        W[p + "q.norm"][:] = 3.0
        W[p + "k.norm"][:] = 3.0
    if kind == "right":
        W[p + "a2.b"][:] = 9.0
    return cfg, {k: v.to(torch.bfloat16) for k, v in W.items()}


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("kind", list(NEEDLES))
def test_far_token_decides(tmp_path, dev, dtype, kind):
    """The needle at the first position, at the last of a page, at the first of the next one, and far back behind
    hundreds of others; seen from the same portion, from later portions and from decoded tokens."""
    cfg, W = needle_model(kind)
    folder = O.save_checkpoint(str(tmp_path / "m"), cfg, W)
    body = [t % 63 + 1 for t in tokens(460, 64, 12)]
    prompts = {"first": [0] + body[:99], "page_end": body[:15] + [0] + body[15:60],
               "page_start": body[:16] + [0] + body[16:60],
               "far": body[:3] + [0] + body[3:440]}
    sched = [[("first", 1), ("page_end", 16)], [("first", 60), ("page_end", 2)], [("first", 1), ("page_end", 30)],
             [("first", 38), ("page_end", 13)], [("page_start", 17), ("far", 150)], [("page_start", 1), ("far", 200)],
             [("page_start", 41), ("far", 1)], [("page_start", 1), ("far", 2)], [("page_start", 1), ("far", 1)],
             [("far", 86)], [("far", 1)]]
    got = run_schedule(folder, dtype, dev, prompts, sched, 640)
    check(cfg, W, prompts, got, dtype)
    for rid, p in prompts.items():                     # without the needle the last position reads quite different
        at = p.index(0)
        other = p[:at] + [body[200]] + p[at + 1:]
        change = O.logit_error(O.forward(cfg, W, other)[-1], O.forward(cfg, W, p)[-1])
        assert change > 2 * TOL["bfloat16"], (rid, change)


@pytest.mark.parametrize("dev", DEVICES)
def test_greedy_generation_through_llm(tmp_path, dev):
    """The engine's own entry point and scheduler: greedy continuation of three prompts of unequal length equals
    the oracle's (recomputed from scratch for every token)."""
    from vllm_distributed_amd import LLM, SamplingParams
    folder, cfg, W = model(tmp_path, mixed_layers(), seed=9, loop=(1, 4, 2))
    V = cfg["vocab"]
    prompts = [tokens(19, V, 1), tokens(3, V, 2), tokens(33, V, 3)]
    llm = LLM(model=folder, skip_tokenizer_init=True, dtype="float32", device=dev, max_model_len=128, max_num_seqs=4,
              max_num_batched_tokens=24, enable_chunked_prefill=True, gpu_memory_utilization=0.1, enforce_eager=True)
    outs = llm.generate(prompt_token_ids=prompts, sampling_params=SamplingParams(temperature=0, max_tokens=10,
                                                                                 ignore_eos=True))
    llm.shutdown()
    for p, o in zip(prompts, outs):
        seq = list(p)
        for tok in o.outputs[0].token_ids:
            logits = O.forward(cfg, W, seq)[-1]
            best = int(logits.argmax())
            assert tok == best or logits[best] - logits[tok] < 1e-3, (len(seq), tok, best)
            seq.append(tok)
        assert len(o.outputs[0].token_ids) == 10


@pytest.mark.parametrize("dev", DEVICES)
def test_long_decoding_keeps_the_state(tmp_path, dev):
    """300 single tokens after a short prompt: nothing drifts against the oracle's whole-sequence run."""
    folder, cfg, W = model(tmp_path, mixed_layers()[:4], seed=12, loop=(1, 3, 2))
    p = tokens(305, cfg["vocab"], 13)
    got = run_schedule(folder, "float32", dev, {"a": p}, [[("a", 5)]] + [[("a", 1)]] * 300, 320)
    check(cfg, W, {"a": p}, got, "float32")


@pytest.mark.gpu
@pytest.mark.parametrize("layers", list(LAYER_SETS))
def test_decode_graphs_equal_eager(tmp_path, layers):
    """Single decoded tokens through captured graphs (several replays with other work between them) give the
    eager logits."""
    folder, cfg, W = model(tmp_path, LAYER_SETS[layers](), seed=10, loop=LOOPS[layers])
    V = cfg["vocab"]
    prompts = {"a": tokens(30, V, 1), "b": tokens(22, V, 2)}
    sched = [[("a", 10), ("b", 4)]] + [[("a", 1), ("b", 1)]] * 18 + [[("a", 2)]]
    eager = run_schedule(folder, "bfloat16", "cuda", prompts, sched, 64, eager=True)
    graph = run_schedule(folder, "bfloat16", "cuda", prompts, sched, 64, eager=False)
    for k in prompts:
        torch.testing.assert_close(graph[k], eager[k], atol=1e-3, rtol=1e-3)
    check(cfg, W, prompts, graph, "bfloat16")
