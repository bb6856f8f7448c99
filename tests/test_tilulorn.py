"""Tilulorn (latent attention with YaRN frequencies and a gate per head, window attention whose values are its keys,
RWKV-style time mixing, experts chosen by token id, a loop whose passes start from a product of the residual and the
embedding output) against the slow oracle of tests/tilulorn_oracle.py: every mechanism alone, then whole models through the
engine's own scheduler, page pool, state slots and step function -- on the CPU backend (fp32) and, marked gpu, through the
HIP kernels (fp32 and bf16).  Small random models are written to disk as checkpoints, so the loader and the configuration
reader run too."""
import math

import pytest
import torch

import tilulorn_oracle as O
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
    return [O.window_layer(), O.latent_layer(), O.wkv_layer(), O.latent_layer(heads=2, dim=20, rot_dim=4, vdim=8, kv_rank=40,
                                                                         q_rank=16, scaling=None, ff=None),
            O.window_layer(heads=3, kv_heads=3, dim=20, window=1, rot_dims=0, ff=None),
            O.wkv_layer(heads=2, dim=20, rank=16, ff=None)]


def matrix_core_layers():
    """Heads, latents and experts of the widths the matrix-core kernels take in 16-bit runs."""
    return [O.latent_layer(heads=4, dim=32, rot_dim=32, vdim=32, kv_rank=64, q_rank=48, scale=0.12, ff=128, experts=3, top=2),
            O.window_layer(heads=4, kv_heads=2, dim=64, window=33, rot_dims=64, scale=0.1, ff=None),
            O.wkv_layer(heads=2, dim=64, rank=32, ff=128, experts=4, top=1),
            O.window_layer(heads=2, kv_heads=1, dim=128, window=17, rot_dims=32, factor=None, scale=0.09, ff=None)]


def recurrent_layers():
    """No attention layer at all: the page pool is book-keeping only, every mixer lives in state slots."""
    return [O.wkv_layer(heads=1, dim=32, rank=1, ff=12, experts=2, top=1), O.wkv_layer(heads=5, dim=7, rank=20, ff=None)]


def attention_layers():
    """No recurrent layer."""
    return [O.latent_layer(heads=1, dim=8, rot_dim=16, vdim=40, kv_rank=12, q_rank=60, ff=None),
            O.window_layer(heads=6, kv_heads=2, dim=8, window=9, rot_dims=4, ff=13, experts=1, top=1)]


LAYER_SETS = {"mixed": mixed_layers, "matrix_core": matrix_core_layers, "recurrent_only": recurrent_layers,
              "attention_only": attention_layers}
LOOPS = {"mixed": (1, 4, 2), "matrix_core": (0, 4, 2), "recurrent_only": (0, 2, 3), "attention_only": (1, 2, 2)}
WIDTHS = {"matrix_core": 128}


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


def layer_set(tmp_path, name, seed):
    return model(tmp_path, LAYER_SETS[name](), seed=seed, loop=LOOPS[name], width=WIDTHS.get(name, 48))


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


def slots_of(table, s, pos, bs):
    return table[s, pos // bs].long() * bs + pos % bs


# ---- mechanisms alone ----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("W_", [40, 301, 516, 1024, 2048, 4104])
def test_residual_step_row_and_cast(dev, dt, W_):
    """A sub-layer's output and a row for every token join the residual; then a norm, or the residual itself into a part of
    a wider buffer."""
    T, eps = 5, 1e-2
    w, step = 1 + 0.2 * torch.randn(W_), torch.randn(W_)
    y = torch.randn(T, W_).to(dt)
    x0 = torch.randn(T, W_) * torch.tensor([0.01, 0.3, 1.0, 5.0, 60.0])[:, None]
    tol = dict(atol=2e-6, rtol=2e-5) if dt == torch.float32 else dict(atol=8e-3, rtol=8e-3)
    for sub, st, norm in ((True, None, True), (False, step, True), (True, step, False), (True, None, False),
                          (False, None, True)):
        want = x0 + (y.float() if sub else 0) + (st if st is not None else 0)
        x = x0.clone().to(dev)
        wide = torch.full((T, 2 * W_), 9.0, dtype=dt, device=dev)
        h = ops.gated_residual_group_norm(x, [(y.to(dev), None, None, None, None)] if sub else [],
                                          w.to(dev) if norm else None, 1, eps, dt, step=st.to(dev) if st is not None else None,
                                          cast_to=None if norm else wide[:, :W_])
        torch.testing.assert_close(x.cpu(), want, atol=1e-5, rtol=1e-5)
        if norm:
            torch.testing.assert_close(h.float().cpu(), O.rms_norm(want, w, eps), **tol)
        else:
            torch.testing.assert_close(wide[:, :W_].float().cpu(), want, **tol)
            assert (wide[:, W_:] == 9.0).all()


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("shape", [(4, 5, 48, 32), (4, 1, 20, 64), (2, 33, 24, 40), (3, 200, 64, 128), (4, 300, 36, 96),
                                   (2, 7, 5, 17)])
def test_grouped_products_and_fp32_product(dev, dt, shape):
    G, M, n, K = shape
    x, w = torch.randn(G, M, K).to(dt), torch.randn(G, n, K).to(dt)
    got = ops.grouped_linear(x.to(dev), w.to(dev))
    for g in range(G):
        assert rel(got[g], x[g].float() @ w[g].float().T) < OP_TOL[dt]
    y = ops.linear_f32(x[0].to(dev), w[0].to(dev))
    assert y.dtype == torch.float32
    torch.testing.assert_close(y.cpu(), x[0].float() @ w[0].float().T, atol=2e-4, rtol=2e-4)


def test_yarn_frequencies_and_magnitude():
    """The framework's table against the equations: ramps that start below zero, end behind the last dimension, have no
    length, or are all on one side."""
    from vllm_distributed_amd.layers.rotary import half_split_cos_sin
    from vllm_distributed_amd.models.tilulorn import yarn_scaling
    x = torch.randn(70, 2, 24)
    for dims, base, sc in ((16, 300.0, (3.0, 24, 4.0, 0.5)), (24, 1e4, (8.0, 4096, 32.0, 1.0)), (8, 50.0, (2.0, 6, 1.0, 1.0)),
                           (20, 777.0, (1.0, 100, 16.0, 2.0)), (12, 20.0, (5.0, 100000, 2.0, 1.0))):
        rot = {"base": base, "dims": dims, "scaling": dict(zip(("factor", "original", "fast", "slow"), sc))}
        n = dims // 2
        cs = half_split_cos_sin(70, dims, base, yarn_scaling(rot), torch.device("cpu"))[:70, None]
        a, b = x[..., :n], x[..., n: dims]
        c, s = cs[..., :n], cs[..., n:]
        got = torch.cat([a * c - b * s, b * c + a * s, x[..., dims:]], -1)
        torch.testing.assert_close(got, O.rotate_halves_yarn(x, rot), atol=1e-5, rtol=1e-5)
    plain = O.rotate_halves_yarn(x, {"base": 300.0, "dims": 16})
    assert rel(O.rotate_halves_yarn(x, {"base": 300.0, "dims": 16, "scaling": {"factor": 3.0, "original": 24, "fast": 4.0,
                                                                              "slow": 0.5}}), plain) > 0.3


# (heads, plain, rotated, value, latent, page size): the kernel for any sizes and, in 16 bits, the matrix-core form
LATENT = [(3, 12, 8, 20, 24, 16), (5, 7, 6, 9, 33, 32), (1, 32, 16, 8, 100, 16), (4, 32, 32, 32, 64, 16),
          (16, 48, 32, 64, 128, 32), (2, 24, 64, 40, 512, 16)]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,D,P,E,R,bs", LATENT)
def test_latent_attention_with_half_split_rotation_and_head_gate(dev, dt, H, D, P, E, R, bs):
    """Ragged batch on scattered pages -- a decoded token, a portion behind cached context that starts inside a page, a whole
    prompt -- through cache write, attention and gate, against the oracle on whole sequences.  The queries arrive with the
    key up-projection folded in, as the layer makes them."""
    from vllm_distributed_amd.layers.rotary import half_split_cos_sin
    from vllm_distributed_amd.models.tilulorn import yarn_scaling
    eps, scale = 1e-3, 1.5 * (D + P) ** -0.5
    lens, news = [75, 53, 20], [1, 11, 20]
    nq = H * (D + P)
    Wd = nq + R + P + H
    xs = [torch.randn(n, Wd).to(dt) for n in lens]
    eye = torch.eye(Wd)
    rot = {"base": 40.0, "dims": P, "scaling": {"factor": 4.0, "original": 30, "fast": 6.0, "slow": 0.6}}
    w = {"dq": eye[:nq], "dq.norm": torch.ones(nq), "uq": torch.eye(nq), "dkv": eye[nq: nq + R + P],
         "dkv.norm": 1 + 0.3 * torch.randn(R), "uk": torch.randn(H * D, R) / math.sqrt(R), "uv": torch.randn(H * E, R) /
         math.sqrt(R), "g": eye[nq + R + P:], "o": torch.eye(H * E)}
    m = {"heads": H, "dim": D, "rot_dim": P, "vdim": E, "kv_rank": R, "scale": scale, "rot": rot}
    keep = O.rms_norm
    try:                                    # the queries as they are: their latent's norm is another op
        O.rms_norm = lambda y, wt, e: y if wt is w["dq.norm"] else keep(y, wt, e)
        want = torch.cat([O.latent_mixer(x.float(), w, m, eps)[n - k:] for x, n, k in zip(xs, lens, news)])
    finally:
        O.rms_norm = keep
    table, nblk = pages(lens, bs)
    mfma = dev == "cuda" and dt == torch.bfloat16 and (R + P, R) in ops.MLA_KERNEL_SIZES
    kc = torch.zeros(nblk, bs, R + P, dtype=dt, device=dev)
    vt = torch.zeros(nblk, R, bs, dtype=dt, device=dev) if mfma else None
    cs = half_split_cos_sin(128, P, rot["base"], yarn_scaling(rot), torch.device(dev))
    w_uk = w["uk"].view(H, D, R)

    def write(rows, pos, slots):
        n = rows.shape[0]
        q = rows[:, :nq].float().view(n, H, D + P)
        qf = torch.zeros(n, H, R + P)
        qf[..., :R] = torch.einsum("thd,hdr->thr", q[..., :D], w_uk)
        qf = qf.to(dt).to(dev)
        r = rows.to(dev)
        ops.latent_norm_rope_cache(r[:, :nq], r[:, nq: nq + R + P], w["dkv.norm"].to(dev), cs, pos.to(dev), qf, kc,
                                   slots.to(dev), H, D, P, R, P, eps, vt, "halves")
        return qf
    for s, (n, k) in enumerate(zip(lens, news)):
        if n - k:
            pos = torch.arange(n - k)
            write(xs[s][: n - k], pos, slots_of(table, s, pos, bs))
    pos = torch.cat([torch.arange(n - k, n) for n, k in zip(lens, news)])
    slots = torch.cat([slots_of(table, s, torch.arange(n - k, n), bs) for s, (n, k) in enumerate(zip(lens, news))])
    rows = torch.cat([x[n - k:] for x, n, k in zip(xs, lens, news)])
    qf = write(rows, pos, slots)
    qsl = torch.tensor([0] + list(torch.tensor(news).cumsum(0)), dtype=torch.int32).to(dev)
    sl = torch.tensor(lens, dtype=torch.int32).to(dev)
    gate = rows.to(dev)[:, Wd - H:]

    def finish(lat):
        o = torch.bmm(lat.float().transpose(0, 1), w["uv"].view(H, E, R).transpose(1, 2).contiguous().to(dev))
        return ops.head_gate_rows(o.to(dt).transpose(0, 1), gate)
    if mfma:
        lat = torch.empty(qf.shape[0], H, R, dtype=dt, device=dev)
        for splits in (1, 3):
            ops.mla_attention(lat[:1], qf[:1], kc, vt, table.to(dev)[:1], sl[:1], qsl[:2], scale, 1, splits, 1.0)
            ops.mla_attention(lat[1:], qf[1:], kc, vt, table.to(dev)[1:], sl[1:], (qsl[1:] - qsl[1]).contiguous(), scale,
                              max(news), 1, 1.0)
            assert rel(finish(lat), want) < OP_TOL[dt]
    lat = ops.latent_window_attention(qf, kc, table.to(dev), sl, qsl, scale, 0, R, max(news))
    assert rel(finish(lat), want) < OP_TOL[dt]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,E", [(3, 20), (1, 7), (16, 64), (5, 128)])
def test_gate_of_head_rows(dev, dt, H, E):
    """Heads-first outputs (as a batched product leaves them) and token-first ones, gates out of wider rows."""
    T = 9
    a, g = torch.randn(H, T, E).to(dt), torch.randn(T, H + 5).to(dt)
    want = (a.float().transpose(0, 1) * torch.sigmoid(g[:, 3: 3 + H].float())[..., None]).reshape(T, H * E)
    for v in (a.to(dev).transpose(0, 1), a.transpose(0, 1).contiguous().to(dev)):
        got = ops.head_gate_rows(v, g.to(dev)[:, 3: 3 + H])
        assert got.dtype == dt and got.is_contiguous() and rel(got, want) < (1e-6 if dt == torch.float32 else 5e-3)


# (heads, key heads, D, window, rotated, page size): any-size kernel and, in 16 bits, the matrix-core forms
ATTN = [(4, 2, 12, 21, 8, 16), (3, 1, 20, 1, 0, 32), (1, 1, 5, 7, 4, 16), (8, 2, 64, 17, 64, 16), (4, 4, 128, 40, 128, 32),
        (2, 1, 72, 16, 6, 16), (16, 1, 64, 100, 16, 16), (4, 2, 96, 33, 32, 32), (2, 2, 256, 13, 48, 16)]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,G,D,window,rot,bs", ATTN)
def test_window_attention_over_key_values(dev, dt, H, G, D, window, rot, bs):
    """The values are the keys as projected: before norm and rotation.  Decoded token, portion and prompt on scattered
    pages; one key that carries nearly all the weight sits just inside and just outside the window of the last queries."""
    from vllm_distributed_amd.layers.rotary import half_split_cos_sin
    eps, scale = 1e-3, 2.0 * D ** -0.5
    lens, news = [75, 53, 20], [1, 11, 20]
    nq, nk = H * D, G * D
    Wd = nq + nk + H
    xs = []
    for n in lens:
        x = torch.randn(n, Wd)
        x[:, :D] *= 3.0                                   # head 0 carries most of the queries' size
        at = n - window                                   # the last query's oldest visible key, and its neighbour before
        for p in (at, at - 1):
            if p >= 0:
                x[p, nq: nq + nk] *= 12.0
        xs.append(x.to(dt))
    eye = torch.eye(Wd)
    w = {"q": eye[:nq], "k": eye[nq: nq + nk], "g": eye[nq + nk:], "q.norm": 1 + 0.3 * torch.randn(nq),
         "k.norm": 1 + 0.3 * torch.randn(nk), "sink": 2.0 * torch.randn(H) + 1, "o": torch.eye(H * D)}
    m = {"heads": H, "kv_heads": G, "dim": D, "scale": scale, "mask": {"size": window}}
    if rot:
        m["rot"] = {"base": 60.0, "dims": rot, "scaling": {"factor": 1.5}}

    def oracle(w_, m_):
        return torch.cat([O.window_mixer(x.float(), w_, m_, eps)[n - k:] for x, n, k in zip(xs, lens, news)])
    want = oracle(w, m)
    assert rel(oracle(dict(w, sink=torch.full((H,), -1e9)), m), want) > 0.1
    last = [sum(news[: s + 1]) - 1 for s, n in enumerate(lens) if n > window]
    assert not last or rel(oracle(w, dict(m, mask={"size": window + 1}))[last], want[last]) > 0.05
    table, nblk = pages(lens, bs)
    kc = torch.zeros(nblk, G, bs, D, dtype=dt, device=dev)
    vc = torch.zeros(nblk, G, D, bs, dtype=dt, device=dev)
    cs = half_split_cos_sin(128, rot, 60.0, dict(kind="linear", factor=1.5), torch.device(dev)) if rot else None
    sink = w["sink"].to(dev)
    mfma = ops.masked_attention_mfma_ok(H, G, D, D, 1, sink, dt, dev == "cuda")

    def write(rows, pos, slots):
        return ops.qk_norm_rope_cache(rows.to(dev), H, G, D, D, 1, w["q.norm"].to(dev), w["k.norm"].to(dev), cs, pos.to(dev),
                                      rot, eps, kc, vc, slots.to(dev), by_map=mfma, pairing="neighbours", whole_norm=True,
                                      key_values=True)
    for s, (n, k) in enumerate(zip(lens, news)):          # context first, as earlier steps would have
        if n - k:
            pos = torch.arange(n - k)
            write(xs[s][: n - k], pos, slots_of(table, s, pos, bs))
    pos = torch.cat([torch.arange(n - k, n) for n, k in zip(lens, news)])
    slots = torch.cat([slots_of(table, s, torch.arange(n - k, n), bs) for s, (n, k) in enumerate(zip(lens, news))])
    rows = torch.cat([x[n - k:] for x, n, k in zip(xs, lens, news)])
    qn = write(rows, pos, slots)
    qsl = torch.tensor([0] + list(torch.tensor(news).cumsum(0)), dtype=torch.int32).to(dev)
    sl = torch.tensor(lens, dtype=torch.int32).to(dev)
    gate = rows.to(dev)[:, Wd - H:]
    if mfma:
        pq = (qsl[1:] - qsl[1]).contiguous()
        for splits in (1, 3):
            got = ops.masked_softmax_attention_mfma(qn, kc, vc, table.to(dev), sl, qsl, pq, 1, 1, 2, int(sum(news[1:])), 1,
                                                    splits, max(news), scale, H, window, sink=sink, gate=gate)
            assert rel(got, want) < OP_TOL[dt], splits
    got = ops.masked_softmax_attention(qn.view(-1, H, D), kc, vc, table.to(dev), sl, qsl, scale, window, sink=sink, gate=gate,
                                       max_query_len=max(news))
    assert rel(got, want) < OP_TOL[dt]


# portions of two sequences: short ones take the token-by-token form, longer ones the chunk-parallel form; portions that
# end inside, at and just behind blocks of sixteen tokens and chunks of 64 and 128
PORTIONS = [[(0, 2), (1, 4)], [(0, 17)], [(1, 1), (0, 1)], [(1, 140), (0, 129)], [(0, 16), (1, 33)], [(0, 1), (1, 64)],
            [(0, 65), (1, 3)], [(1, 1), (0, 1)]]
TOTAL = [sum(n for st in PORTIONS for s, n in st if s == q) for q in (0, 1)]


def in_portions(xs, dev, dt, launch):
    """Runs PORTIONS through ``launch(x, qsl, lens, table, max_new, first_long)``; both splits of the step's sequences (short
    ones announced as such, or not) are used in turn."""
    slot = torch.tensor([[4], [2]], dtype=torch.int32, device=dev)
    done, got = [0, 0], [[], []]
    for turn, step in enumerate(PORTIONS):
        order = sorted(step, key=lambda a: a[1] > 1)
        x = torch.cat([xs[s][done[s]: done[s] + n] for s, n in order]).to(dt).to(dev)
        qsl = torch.tensor([0] + list(torch.tensor([n for _, n in order]).cumsum(0)), dtype=torch.int32, device=dev)
        lens = torch.tensor([done[s] + n for s, n in order], dtype=torch.int32, device=dev)
        few = sum(n == 1 for _, n in order) if turn % 2 == 0 else 0
        out = launch(x, qsl, lens, slot[[s for s, _ in order]], max(n for _, n in order), few).cpu()
        o = 0
        for s, n in order:
            got[s].append(out[o:o + n])
            o += n
            done[s] += n
    assert done == TOTAL
    return [torch.cat(g) for g in got]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("M,W_", [(5, 48), (1, 7), (3, 1030), (8, 260)])
def test_token_shift(dev, dt, M, W_):
    """Mixes with the row before, across portions and slots with stale content."""
    xs = [torch.randn(n, W_).to(dt).float() for n in TOTAL]
    mu = torch.rand(M, W_)
    state = torch.full((5, 1, W_), 7.0, dtype=dt, device=dev)

    def launch(x, qsl, lens, tbl, longest, few):
        wide = torch.cat([x, x], -1)                       # rows with a pitch
        got = ops.token_shift_mix(wide[:, :W_], mu.to(dev), state, qsl, lens, tbl, longest)
        assert got.shape == (M, x.shape[0], W_)
        return got.transpose(0, 1).reshape(x.shape[0], M * W_)
    got = in_portions(xs, dev, dt, launch)
    for g, x in zip(got, xs):
        want = torch.stack([O.shifted_mix(x, mu[i]) for i in range(M)], 1).reshape(x.shape[0], M * W_)
        torch.testing.assert_close(g.float(), want, atol=1e-5 if dt == torch.float32 else 3e-2, rtol=1e-5 if dt ==
                                   torch.float32 else 1e-2)
    assert (state[[0, 1, 3]] == 7.0).all()                 # nobody else's slot
    assert (state[4, 0].float().cpu() == xs[0][-1]).all() and (state[2, 0].float().cpu() == xs[1][-1]).all()


# (heads, D, pre-activations around): slow decays, ordinary ones, ones that vanish within a token (running products
# underflow inside a block), and all of them side by side
WKV = [(3, 12, -3.0, 1.0), (2, 64, -5.0, 1.5), (1, 5, 0.0, 1.0), (2, 128, -1.0, 2.5), (1, 33, 2.0, 3.0), (2, 160, -2.0, 1.0),
       (4, 32, -4.0, 3.0), (1, 300, -3.0, 1.0)]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("H,D,bias,spread", WKV)
def test_memory_with_bonus_and_doubly_exponential_decay(dev, dt, H, D, bias, spread):
    """Portions in state slots that hold stale content, against the oracle on the whole sequences; the bonus is large, so
    that a token entering its own read-out through the memory instead is far off."""
    eps = 1e-4
    n = H * D
    xs = [torch.randn(L, 5 * n).to(dt).float() for L in TOTAL]
    u, w0, norm = 2.0 + torch.randn(H, D), spread * torch.randn(n) + bias, 1 + 0.2 * torch.randn(n)

    def oracle(x, bonus):
        r, k, v, g, z = (x[:, i * n: (i + 1) * n] for i in range(5))
        decay = torch.exp(-torch.exp(z + w0)).view(-1, H, D)
        o = O.bonus_memory(r.view(-1, H, D), k.view(-1, H, D), v.view(-1, H, D), decay, bonus)
        return O.unit_rms(o, eps).reshape(-1, n) * norm * O.silu(g)
    want = [oracle(x, u) for x in xs]
    assert rel(oracle(xs[0], torch.ones_like(u)), want[0]) > 0.05
    state = torch.full((5, H, D, D), 3.0, device=dev)

    def launch(x, qsl, lens, tbl, longest, few):
        r, k, v, g, z = (x[:, i * n: (i + 1) * n] for i in range(5))
        return ops.linear_attention(r, k, v, g, norm.to(dev), state, qsl, lens, tbl, H, D, D, eps, longest, z=z,
                                    z_bias=w0.to(dev), decay_exp=True, bonus=u.reshape(-1).to(dev), first_long_seq=few)
    got = in_portions(xs, dev, dt, launch)
    for g, w in zip(got, want):
        assert rel(g, w) < OP_TOL[dt]
    assert (state[[0, 1, 3]] == 3.0).all()


@pytest.mark.parametrize("dev,dt", OP_CASES)
def test_options_of_the_memory_combine(dev, dt):
    """A bonus beside sigmoid decays, doubly exponential decays without a bonus, and values wider than the keys."""
    H, D, E, eps = 2, 32, 80, 1e-4
    n, nv = H * D, H * E
    xs = [torch.randn(L, 3 * n + 2 * nv).to(dt).float() for L in TOTAL]
    u, norm, zb = torch.randn(H, D), 1 + 0.2 * torch.randn(E), torch.randn(n)
    state = torch.full((5, H, E, D), 3.0, device=dev)

    def split(x):
        return torch.split(x, [n, n, nv, nv, n], -1)
    for bonus in (u, None):
        def launch(x, qsl, lens, tbl, longest, few):
            q, k, v, g, z = split(x)
            kw = dict(bonus=bonus.reshape(-1).to(dev), tau=3.0) if bonus is not None else dict(decay_exp=True)
            return ops.linear_attention(q, k, v, g, norm.to(dev), state, qsl, lens, tbl, H, D, E, eps, longest, z=z,
                                        z_bias=zb.to(dev), first_long_seq=few, **kw)
        got = in_portions(xs, dev, dt, launch)
        for g_, x in zip(got, xs):
            q, k, v, g, z = split(x)
            q, k, v, z = q.view(-1, H, D), k.view(-1, H, D), v.view(-1, H, E), (z + zb).view(-1, H, D)
            if bonus is not None:
                o = O.bonus_memory(q, k, v, torch.sigmoid(z) ** (1 / 3.0), bonus)
            else:                                          # reading behind the write is a bonus of one beside faded memory
                f = torch.exp(-torch.exp(z))
                o = O.bonus_memory(q * f, k, v, f, torch.zeros(H, D)) + (q * k).sum(-1, keepdim=True) * v
            want = (O.unit_rms(o, eps) * norm).reshape(-1, nv) * O.silu(g)
            assert rel(g_, want) < OP_TOL[dt]


@pytest.mark.parametrize("dev,dt", OP_CASES)
@pytest.mark.parametrize("E,top,W_,ff", [(5, 2, 48, 24), (3, 3, 40, 17), (1, 1, 64, 8), (4, 1, 128, 128), (8, 5, 256, 384)])
def test_experts_chosen_by_token_id(dev, dt, E, top, W_, ff):
    """Every width the expert kernels have a form for, few and many tokens, tokens that occur repeatedly."""
    V = 30
    for T in (3, 150):
        toks = tokens(T, V, T)
        h = torch.randn(T, W_).to(dt)
        w = {"table": torch.stack([torch.randperm(E)[:top] for _ in range(V)]).int()}
        for e in range(E):
            for nm, shape in (("gate", (ff, W_)), ("up", (ff, W_)), ("down", (W_, ff))):
                w[f"e{e}.{nm}"] = (torch.randn(*shape) / math.sqrt(shape[1])).to(dt).float()
        want = O.table_experts(h.float(), w, toks)
        w13 = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)]).to(dt).to(dev)
        w2 = torch.stack([w[f"e{e}.down"] for e in range(E)]).to(dt).to(dev)
        ids = w["table"][torch.tensor(toks)].to(dev)
        got = ops.fused_moe(h.to(dev), w13, w2, torch.full((T, top), 1.0 / top, device=dev), ids)
        assert rel(got, want) < OP_TOL[dt], T


# ---- configuration and loading -----------------------------------------------------------------------------------------
def test_rank_of_the_decay_projection_comes_from_its_shape(tmp_path):
    from vllm_distributed_amd.config import load_hf_config
    folder, cfg, _ = model(tmp_path, [O.wkv_layer(rank=11)])
    hf = load_hf_config(folder)
    assert hf.architectures == ["TilulornForCausalLM"] and hf.layers[0]["mixer"]["decay_rank"] == 11
    assert hf.hidden_size == cfg["width"] and hf.vocab_size == cfg["vocab"]


@pytest.mark.parametrize("name,t,match", [
    ("l0.mix.b", torch.ones(3), "no place"), ("l0.mlp.table", torch.full((96, 3), 3, dtype=torch.int32), "outside"),
    ("l0.mlp.table", torch.zeros((96, 2), dtype=torch.int32), "expected integers")])
def test_tensors_that_do_not_fit_are_refused(tmp_path, name, t, match):
    from vllm_distributed_amd.entrypoints.trace_replay import TraceReplayer
    folder, cfg, W = model(tmp_path, [O.wkv_layer()])
    O.save_checkpoint(folder, cfg, dict(W, **{name: t}))
    with pytest.raises(ValueError, match=match):
        TraceReplayer(folder, "float32", 64, device="cpu", enforce_eager=True)


def test_unknown_mixer_and_feed_forward_are_refused():
    from vllm_distributed_amd.models.tilulorn import normalise_config
    cfg, _ = O.make_config([O.window_layer()])
    with pytest.raises(ValueError, match="unknown mixer"):
        normalise_config(dict(cfg, layers=[dict(cfg["layers"][0], type="conv_only")]))
    with pytest.raises(ValueError, match="unknown feed-forward"):
        normalise_config(dict(cfg, layers=[dict(cfg["layers"][0], mlp={"kind": "dense", "ff": 8})]))


# ---- whole models through the engine --------------------------------------------------------------------------------
VARIANTS = {
    "mixed_looped": dict(layers=mixed_layers(), loop=(1, 4, 2)),
    "no_loop": dict(layers=mixed_layers()[:4]),
    "loop_over_everything": dict(layers=mixed_layers()[1:3], loop=(0, 2, 3)),
    "loop_once_at_the_end": dict(layers=mixed_layers()[:3], loop=(2, 3, 1)),
    "loop_of_one_layer_many_times": dict(layers=mixed_layers()[:3], loop=(1, 2, 4)),
    "matrix_core": dict(layers=matrix_core_layers(), loop=(1, 3, 2), width=128),
    "latent_only": dict(layers=[O.latent_layer(heads=1, dim=4, rot_dim=4, vdim=6, kv_rank=8, q_rank=5, ff=None),
                                O.latent_layer(heads=6, dim=10, rot_dim=2, vdim=4, kv_rank=16, q_rank=40, experts=2, top=2)],
                        eps=1e-6),
    "window_only": dict(layers=[O.window_layer(heads=1, kv_heads=1, dim=40, window=2, rot_dims=40, factor=None),
                                O.window_layer(heads=6, kv_heads=3, dim=6, window=500, rot_dims=2, ff=None)], eps=1e-6),
    "wkv_only": dict(layers=[O.wkv_layer(heads=1, dim=40, rank=3, ff=None), O.wkv_layer(heads=6, dim=4, rank=33, top=1)],
                     loop=(0, 1, 4)),
    "odd_widths": dict(layers=[O.window_layer(heads=3, kv_heads=1, dim=7, window=10, rot_dims=6, ff=13, experts=3, top=2),
                               O.latent_layer(heads=3, dim=5, rot_dim=6, vdim=7, kv_rank=9, q_rank=11, ff=9),
                               O.wkv_layer(heads=3, dim=5, rank=2, ff=7)], width=45, vocab=37, loop=(0, 2, 2), eps=1e-3),
}


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("name", list(VARIANTS))
def test_whole_prompt(tmp_path, dev, dtype, name):
    kw = dict(VARIANTS[name])
    folder, cfg, W = model(tmp_path, kw.pop("layers"), seed=5, **kw)
    prompts = {"a": tokens(85, cfg["vocab"], 1), "b": tokens(1, cfg["vocab"], 2)}
    got = run_schedule(folder, dtype, dev, prompts, [[("a", 85)], [("b", 1)]], 112)
    check(cfg, W, prompts, got, dtype)


def test_the_parts_matter():
    """The oracle itself: step rows, both halves of the loop's product, sinks, bonus, gates, expert tables and window change
    the logits by far more than the fp32 tolerance of the comparisons above and below."""
    cfg, ranks = O.make_config(mixed_layers(), loop=(1, 4, 2))
    W = O.make_weights(cfg, ranks, 3)
    p = tokens(40, cfg["vocab"], 1)
    full = O.forward(cfg, W, p)

    def changed(**new):
        return O.logit_error(O.forward(cfg, dict(W, **{k.replace("__", "."): v for k, v in new.items()}), p), full)
    for row in (0, 1):
        t = W["loop.step"].clone()
        t[row] = 0
        assert changed(loop__step=t) > 0.05
    for half in (slice(0, 48), slice(48, 96)):
        t = W["loop.in"].clone()
        t[:, half] = 0
        assert changed(loop__in=t) > 0.05
    assert changed(l0__mix__sink=torch.full_like(W["l0.mix.sink"], -60.0)) > 0.02
    assert changed(l2__mix__u=torch.ones_like(W["l2.mix.u"])) > 0.02
    assert changed(l2__mix__mu__w=torch.zeros_like(W["l2.mix.mu.w"])) > 2e-3
    assert changed(l1__mix__g=torch.zeros_like(W["l1.mix.g"])) > 0.02
    assert changed(l1__mlp__table=W["l1.mlp.table"].flip(0)) > 0.05
    wide = dict(cfg, layers=[dict(l, mixer=dict(l["mixer"], mask={"size": 22})) if i == 0 else l
                             for i, l in enumerate(cfg["layers"])])
    assert O.logit_error(O.forward(wide, W, p), full) > 0.01


@pytest.mark.parametrize("dev", DEVICES)
def test_residual_after_every_layer_run(tmp_path, dev):
    """The framework's residual after every layer run against the oracle's trail (looped layers count each time)."""
    from vllm_distributed_amd.entrypoints.trace_replay import TraceReplayer
    folder, cfg, W = model(tmp_path, mixed_layers(), seed=1, loop=(1, 4, 3))
    p = tokens(20, cfg["vocab"], 1)
    _, trail = O.forward(cfg, W, p, want_layers=True)
    r = TraceReplayer(folder, "float32", 64, device=dev, enforce_eager=True)
    seen = []
    mdl = r.core.model_executor.worker.model_runner.model
    hooks = [b.register_forward_hook(lambda mod, args, out: seen.append(args[0][: len(p)].clone().cpu())) for b in mdl.layers]
    try:
        r.step([{"id": "a", "tokens": p, "want": [0]}], ["a"])
    finally:
        for h in hooks:
            h.remove()
        r.shutdown()
    assert len(seen) == len(trail) == 12
    torch.testing.assert_close(torch.stack(seen), trail, atol=3e-4, rtol=3e-4)


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("layers", list(LAYER_SETS))
def test_prefill_equals_decoding_token_by_token(tmp_path, dev, dtype, layers):
    folder, cfg, W = layer_set(tmp_path, layers, 4)
    p = tokens(70, cfg["vocab"], 5)
    got = run_schedule(folder, dtype, dev, {"a": p}, [[("a", 11)]] + [[("a", 1)]] * 59, 80)
    check(cfg, W, {"a": p}, got, dtype)
    whole = run_schedule(folder, dtype, dev, {"a": p}, [[("a", 70)]], 80)
    assert O.logit_error(got["a"], whole["a"]) < TOL[dtype]


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("block_size", [16, 32])
@pytest.mark.parametrize("layers", list(LAYER_SETS))
def test_portions_down_to_two_tokens(tmp_path, dev, dtype, block_size, layers):
    folder, cfg, W = layer_set(tmp_path, layers, 6)
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
    folder, cfg, W = layer_set(tmp_path, layers, 8)
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
    "latent_attention": O.latent_layer(heads=2, dim=8, rot_dim=8, vdim=8, kv_rank=16, q_rank=16, scale=0.6, ff=None),
    "wkv": O.wkv_layer(heads=2, dim=8, rank=4, ff=None),
    "attention": O.window_layer(heads=2, kv_heads=1, dim=8, window=37, rot_dims=0, scale=0.6, ff=None),
}


def needle_model(kind):
    """One layer.  Token 0 is a 'needle' that alone fills key direction 0 of head 0; every other token's query looks
    there, so the logits of all later positions hang on whether the needle is still seen or remembered."""
    cfg, ranks = O.make_config([NEEDLES[kind]], vocab=64, width=32)
    W = {k: v.float() if v.is_floating_point() else v for k, v in O.make_weights(cfg, ranks, 11).items()}
    emb = 0.2 * W["embed"]
    emb[:, 0] = 0
    emb[:, 2] = 3.0                                    # every token is mostly e2 ...
    emb[0] = 0
    emb[0, 0] = 3.0                                    # ... except the needle, alone along e0
    W["embed"] = emb
    W["l0.norm1"] = torch.ones(32)
    p = "l0.mix."
    W[p + "o"] *= 5.0 if kind == "latent_attention" else 1.5
    if kind == "latent_attention":                     # the needle's latent has a direction of its own
        W[p + "dq"] *= 0.05
        W[p + "dq"][0] = 0
        W[p + "dq"][0, 2] = 4.0
        W[p + "dq.norm"][:] = 1.0
        W[p + "uq"] *= 0.05
        W[p + "uq"][0, 0] = 3.0
        W[p + "dkv"] *= 0.3
        W[p + "dkv"][0] = 0
        W[p + "dkv"][0, 0] = 4.0
        W[p + "dkv.norm"][:] = 1.0
        W[p + "uk"] *= 0.05
        W[p + "uk"][0, 0] = 3.0
        W[p + "g"][0] = 0
        W[p + "g"][0, 2] = 1.0
    elif kind == "attention":
        for n in ("q", "k"):
            W[p + n] *= 0.3 if n == "k" else 0.03
        W[p + "q"][0], W[p + "k"][0] = 0, 0
        W[p + "q"][0, 2] = W[p + "k"][0, 0] = 4.0
        W[p + "sink"][:] = 2.0
        W[p + "q.norm"][:] = 2.0
        W[p + "k.norm"][:] = 2.0
    else:
        for n in ("r", "k"):
            W[p + n] *= 0.03
            W[p + n][0] = 0
        W[p + "r"][0, 2] = W[p + "k"][0, 0] = 4.0
        for s in "rkvgw":
            W[p + "mu." + s][:] = 0.1
        W[p + "w0"][:] = -9.0                          # hardly any fading
        W[p + "w2"] *= 0.1
    return cfg, {k: v.to(torch.bfloat16) if v.is_floating_point() else v for k, v in W.items()}


@pytest.mark.parametrize("dev,dtype", CASES)
@pytest.mark.parametrize("kind", list(NEEDLES))
def test_far_token_decides(tmp_path, dev, dtype, kind):
    """The needle at the first position, at the last of a page, at the first of the next one, and far back behind
    hundreds of others; seen from the same portion, from later portions and from decoded tokens.  Window attention: it is
    seen up to the window's edge -- in a prompt portion and by decoded tokens -- and then gone."""
    cfg, W = needle_model(kind)
    folder = O.save_checkpoint(str(tmp_path / "m"), cfg, W)
    body = [t % 63 + 1 for t in tokens(460, 64, 12)]
    prompts = {"first": [0] + body[:99], "page_end": body[:15] + [0] + body[15:60],
               "page_start": body[:16] + [0] + body[16:60],
               "far": body[:3] + [0] + body[3:440]}
    sched = [[("first", 1), ("page_end", 16)], [("first", 30), ("page_end", 2)], [("first", 1), ("page_end", 30)]] + \
        [[("first", 1), ("page_end", 1)]] * 8 + \
        [[("first", 60), ("page_end", 5)], [("page_start", 17), ("far", 150)], [("page_start", 1), ("far", 200)],
         [("page_start", 41), ("far", 1)], [("page_start", 1), ("far", 2)], [("page_start", 1), ("far", 1)],
         [("far", 86)], [("far", 1)]]
    got = run_schedule(folder, dtype, dev, prompts, sched, 640)
    check(cfg, W, prompts, got, dtype)
    for rid, p in prompts.items():                     # without the needle the positions that see it read quite different
        at = p.index(0)
        other = p[:at] + [body[200]] + p[at + 1:]
        a, b = O.forward(cfg, W, other), O.forward(cfg, W, p)
        if kind == "attention":
            inside, outside = at + 36, at + 37
            assert O.logit_error(a[inside], b[inside]) > 2 * TOL["bfloat16"], rid
            assert O.logit_error(a[outside], b[outside]) < 1e-5, rid
        else:
            assert O.logit_error(a[-1], b[-1]) > 2 * TOL["bfloat16"], (rid, O.logit_error(a[-1], b[-1]))


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
    folder, cfg, W = layer_set(tmp_path, layers, 10)
    V = cfg["vocab"]
    prompts = {"a": tokens(30, V, 1), "b": tokens(22, V, 2)}
    sched = [[("a", 10), ("b", 4)]] + [[("a", 1), ("b", 1)]] * 18 + [[("a", 2)]]
    eager = run_schedule(folder, "bfloat16", "cuda", prompts, sched, 64, eager=True)
    graph = run_schedule(folder, "bfloat16", "cuda", prompts, sched, 64, eager=False)
    for k in prompts:
        torch.testing.assert_close(graph[k], eager[k], atol=1e-3, rtol=1e-3)
    check(cfg, W, prompts, graph, "bfloat16")
