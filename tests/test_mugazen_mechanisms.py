"""Mugazen's mechanisms one at a time: each framework op (CPU reference
and, marked gpu, the HIP kernel) against the plain float64 oracle function
of the same mechanism. Where random inputs would hide a fault — a far key
among hundreds, a sink, the order of decay, write and read — inputs are
made so that it shows."""

import math
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import mugazen_oracle as O  # noqa: E402

from agentainer_amd import ops  # noqa: E402
from agentainer_amd.models.llama import AttnMetadata  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64


@pytest.fixture(autouse=True)
def _true_fp32():
    torch.backends.cuda.matmul.allow_tf32 = False


def rnd(*shape, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).bfloat16().float()


def close(got, want, dtype, tol32=2e-5, tol16=2e-2):
    tol = tol32 if dtype == torch.float32 else tol16
    err = float((got.double().cpu() - want).abs().max()
                / want.abs().max().clamp(min=1e-6))
    assert err < tol, err


def i32(device, *vals):
    return torch.tensor(vals, dtype=torch.int32, device=device)


# ------------------------------------------------------------- embedding

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [40, 50, 2304, 4352])
def test_position_embedding_norm(device, dtype, W):
    V, P, scale, eps = 30, 17, 5.0, 1e-2
    embed, pos, nw = rnd(V, W, seed=1), rnd(P, W, seed=2, scale=2.0), rnd(
        W, seed=3)
    ids = torch.tensor([4, 4, 29, 0, 11])
    at = torch.tensor([0, 16, 3, 3, 1], dtype=torch.int32)
    want = O.rms_norm(embed.double()[ids] * scale + pos.double()[at.long()],
                      nw.double(), eps)
    x = torch.empty(5, W, device=device)
    x0 = torch.empty(5, W, device=device)
    ops.position_embed_norm(
        x, ids.to(device), at.to(device),
        embed.to(device=device, dtype=dtype),
        pos.to(device=device, dtype=dtype), scale, nw.to(device), eps,
        x_copy=x0)
    close(x, want, torch.float32)
    assert torch.equal(x, x0)
    # the position vector is not scaled: the same ids at another place differ
    assert float((x[0] - x[1]).abs().max()) > 0.05


# ------------------------------------------------- residual update + norm

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [64, 50, 1200, 4096, 4100])
def test_sandwich_residual_with_pass_inputs(device, dtype, W):
    """x += N(y; post); x += rows + vec; h = N(x; pre) — every optional
    part on and off; the mean of x is far from zero, so a layer norm in
    place of the RMS norm would show."""
    T, eps = 5, 1e-3
    x0 = rnd(T, W, seed=1, scale=2.0) + 3.0
    y, rows, vec = rnd(T, W, seed=2, scale=4.0), rnd(T, W, seed=3), rnd(
        W, seed=4)
    post, pre = rnd(W, seed=5), rnd(W, seed=6)
    d = lambda t: t.to(device)                       # noqa: E731
    for use_y in (True, False):
        for use_rows, use_vec in ((0, 0), (0, 1), (1, 1)):
            for use_h in (True, False):
                want = x0.double()
                if use_y:
                    want = want + O.rms_norm(y.double(), post.double(), eps)
                if use_vec:
                    want = want + vec.double()
                if use_rows:
                    want = want + rows.double()
                x = d(x0.clone())
                h = (torch.empty(T, W, device=device, dtype=dtype)
                     if use_h else None)
                ops.residual_update_norm(
                    x, y.to(device=device, dtype=dtype) if use_y else None,
                    ops.UPDATE_UNIT_RMS if use_y else ops.UPDATE_NONE, None,
                    None, d(post), eps, d(pre) if use_h else None, None, h,
                    rms_norm=True, add_rows=d(rows) if use_rows else None,
                    add_vec=d(vec) if use_vec else None)
                close(x, want, torch.float32, 2e-6)
                if use_h:
                    close(h, O.rms_norm(want, pre.double(), eps), dtype)
    # eps sits inside both roots: tiny rows are not blown up
    x = d(torch.zeros(1, W))
    tiny = rnd(1, W, seed=9, scale=1e-3)
    h = torch.empty(1, W, device=device)
    ops.residual_update_norm(x, d(tiny), ops.UPDATE_UNIT_RMS, None, None,
                             d(post), eps, d(pre), None, h, rms_norm=True)
    want = O.rms_norm(tiny.double(), post.double(), eps)
    close(x, want, torch.float32)
    close(h, O.rms_norm(want, pre.double(), eps), torch.float32)


# -------------------------------------------------------- narrow projection

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,N,K", [(1, 1, 64), (3, 8, 40), (70, 33, 256),
                                   (17, 130, 72), (2100, 64, 512),
                                   (2100, 20, 96), (5, 6, 50), (33, 16, 4096),
                                   (8200, 70, 96), (8200, 60, 264),
                                   (4100, 150, 520)])
def test_narrow_projection_keeps_32_bits(device, dtype, T, N, K):
    wide = rnd(T, K + 8, seed=1)
    x = wide[:, 8:]                      # a view with an offset
    w, b = rnd(N, K, seed=2), rnd(N, seed=3)
    want = x.double() @ w.double().T + b.double()
    got = ops.narrow_linear(wide.to(device=device, dtype=dtype)[:, 8:],
                            w.to(device=device, dtype=dtype), b.to(device))
    assert got.dtype == torch.float32
    # exact products, fp32 sums: far below bf16 rounding in both modes
    close(got, want, torch.float32, 2e-5)
    got = ops.narrow_linear(x.contiguous().to(device=device, dtype=dtype),
                            w.to(device=device, dtype=dtype))
    close(got, want - b.double(), torch.float32, 2e-5)


# ------------------------------------------------------------- delta rule

def run_scan(device, rows, q, k, v, pre, bias, rate, strength, S, decode,
             q_scale=1.0, dtype=torch.float32):
    """rows: [(slot, first token, n tokens, tokens before)] of one batch;
    q.. are per-sequence dicts keyed by slot."""
    cat = lambda d: torch.cat([d[s][a:a + n] for s, a, n, _ in rows])  # noqa: E731
    T = sum(n for _s, _a, n, _b in rows)
    H, Dv = next(iter(v.values())).shape[1:]
    out = torch.zeros(T, H, Dv, device=device)
    starts, acc = [], 0
    for _s, _a, n, _b in rows:
        starts.append(acc)
        acc += n
    dev = lambda t, dt=torch.float32: t.to(device=device, dtype=dt)  # noqa: E731
    ops.matrix_memory_scan(
        ops.SCAN_DELTA_HEAD, out, dev(cat(q), dtype), dev(cat(k), dtype),
        dev(cat(v), dtype), dev(cat(pre)), dev(bias), dev(rate),
        dev(cat(strength)), q_scale, 0.0, S, None, None,
        torch.tensor([s for s, *_ in rows], device=device),
        i32(device, *[b + n for _s, _a, n, b in rows]),
        None if decode else i32(device, *starts),
        None if decode else i32(device, *[n for _s, _a, n, _b in rows]))
    return out.double().cpu()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 16, 12), (3, 1, 24, 40),
                                      (2, 2, 64, 64), (6, 3, 6, 5),
                                      (4, 4, 128, 128), (2, 1, 200, 96)])
def test_head_decay_delta_rule(device, H, G, D, Dv):
    """Two sequences side by side in unequal portions (down to two tokens),
    then one token each; both slots still hold a stranger's memory when
    their sequences start."""
    n = {0: 23, 2: 14}
    mk = lambda seed, *sh: {s: rnd(t, *sh, seed=seed + s) for s, t in n.items()}  # noqa: E731
    q, v, strength, pre = mk(1, G, D), mk(20, H, Dv), mk(30, H), mk(40, H)
    k = {s: O.unit_vector(rnd(t, G, D, seed=10 + s)).bfloat16().float()
         for s, t in n.items()}
    rate, bias = rnd(H, seed=50, scale=0.5) - 0.5, rnd(H, seed=51) - 1.5
    want = {s: O.delta_recurrence(
        q[s].double() * 0.25, k[s].double(), v[s].double(),
        O.delta_decay(pre[s].double(), rate.double(), bias.double()),
        O.sigmoid(strength[s].double())) for s in n}
    S = rnd(4, H, Dv, D, seed=60).to(device)        # dirty slots
    keep = S[[1, 3]].clone()
    got = {s: [] for s in n}
    at = {s: 0 for s in n}
    for step in ([(0, 11), (2, 2)], [(0, 2), (2, 9)], [(0, 1), (2, 1)],
                 [(2, 2), (0, 8)], [(0, 1)]):
        rows = [(s, at[s], m, at[s]) for s, m in step]
        o = run_scan(device, rows, q, k, v, pre, bias, rate, strength, S,
                     all(m == 1 for _s, m in step), q_scale=0.25)
        p = 0
        for s, m in step:
            got[s].append(o[p:p + m])
            p += m
            at[s] += m
    for s in n:
        assert torch.allclose(torch.cat(got[s]), want[s], atol=3e-5,
                              rtol=1e-4)
    assert torch.equal(S[[1, 3]], keep)             # nobody else's memory


@pytest.mark.parametrize("device", DEVICES)
def test_delta_rule_order_of_decay_write_and_read(device):
    """One channel, numbers that tell the orders apart: the memory decays
    BEFORE it is compared with v, and the read-out sees the write of its
    own token."""
    one = {0: torch.ones(2, 1, 1)}
    v = {0: torch.tensor([[[1.0]], [[3.0]]])}
    pre = {0: torch.tensor([[0.0], [0.4]])}
    strength = {0: torch.tensor([[0.0], [1.0]])}
    rate, bias = torch.tensor([0.3]), torch.tensor([0.2])
    b = [0.5, 1 / (1 + math.exp(-1.0))]
    g = math.exp(-math.exp(0.3) * math.log1p(math.exp(0.6)))
    s1 = b[0] * 1.0
    s2 = g * s1 + b[1] * (3.0 - g * s1)
    S = torch.full((1, 1, 1, 1), 99.0, device=device)
    o = run_scan(device, [(0, 0, 2, 0)], one, one, v, pre, bias, rate,
                 strength, S, False)
    assert abs(float(o[0]) - s1) < 1e-6 and abs(float(o[1]) - s2) < 1e-6
    assert abs(float(S) - s2) < 1e-6
    # a unit key with full strength overwrites: the old value is gone
    full = {0: torch.tensor([[60.0], [60.0]])}
    o = run_scan(device, [(0, 0, 2, 0)], one, one, v, pre, bias, rate, full,
                 S, False)
    assert abs(float(o[1]) - 3.0) < 1e-5


@pytest.mark.parametrize("device", DEVICES)
def test_delta_memory_reaches_far_back(device):
    """One strong write, then 300 tokens that neither write nor (almost)
    decay: the value is still there, decayed by exactly 300 factors."""
    T = 301
    q = {1: torch.zeros(T, 1, 8)}
    q[1][:, 0, 0] = 1.0
    v = {1: torch.zeros(T, 1, 4)}
    v[1][0, 0] = torch.tensor([1.0, -2.0, 3.0, 4.0])
    strength = {1: torch.full((T, 1), -80.0)}
    strength[1][0] = 80.0
    pre = {1: torch.full((T, 1), -6.0)}
    zero = torch.zeros(1)
    S = torch.zeros(3, 1, 4, 8, device=device)
    g = math.exp(-math.log1p(math.exp(-6.0)))
    o = run_scan(device, [(1, 0, T - 1, 0)], q, q, v, pre, zero, zero,
                 strength, S, False)
    o1 = run_scan(device, [(1, T - 1, 1, T - 1)], q, q, v, pre, zero, zero,
                  strength, S, True)
    for row, steps in ((o[150, 0], 150), (o1[0, 0], 300)):
        want = v[1][0, 0].double() * g ** steps
        assert torch.allclose(row, want, rtol=2e-4)


def step_metadata(device, at, n, slot, page, perm, decode):
    pos = torch.arange(at, at + n)
    return AttnMetadata(
        page_table=perm.to(torch.int32).view(1, -1).to(device),
        seq_lens=i32(device, at + n),
        slot_mapping=(perm[pos // page] * page + pos % page).to(device),
        positions=pos.to(dtype=torch.int32, device=device),
        is_prefill=not decode, query_starts=i32(device, 0),
        query_lens=i32(device, n), max_qlen=n,
        state_slots=torch.tensor([slot], device=device))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mx", [
    O.delta_layer(heads=4, kv_heads=2, dim=16, vdim=24, conv=4),
    O.delta_layer(heads=3, kv_heads=3, dim=10, vdim=7, conv=2),
    O.delta_layer(heads=6, kv_heads=1, dim=32, vdim=16, conv=1)])
def test_delta_mixer_module(device, dtype, mx):
    from agentainer_amd.models.mugazen import config_from_dict
    from agentainer_amd.models.pekarax import MatrixMemoryMixer

    W, eps = 40, 1e-4
    cfg = O.make_config([(mx, None)], width=W, eps=eps)
    w = O.random_weights(cfg, seed=2)
    c = config_from_dict(cfg)
    h = rnd(29, W, seed=5)
    want = O.delta_mixer(h.double(), {k: t.double() for k, t in w.items()},
                         "l0.mix.", mx["mixer"], eps)
    mod = MatrixMemoryMixer(W, c.layers[0].delta, eps, dtype).to(device)
    mod.load(lambda n: w["l0.mix." + n].to(device=device, dtype=dtype))
    state = {k: torch.full((3, *s), 7.0, device=device)
             for k, s in c.state_shapes()[0].items()}
    perm, got, at = torch.arange(1, 9), [], 0
    for n in (2, 9, 2, 1, 1, 11, 1, 2):
        md = step_metadata(device, at, n, 1, 4, perm, n == 1 and at > 0)
        got.append(mod(h[at:at + n].to(device=device, dtype=dtype), None,
                       state, md).float().cpu())
        at += n
    close(torch.cat(got), want, dtype, 1e-4, 4e-2)


# ------------------------------------------------------- latent attention

def paged_rows(c, page, rp, device, dtype, seed=0):
    """Scatter [n, R] latents into shuffled pages of a zero-padded pool."""
    n, R = c.shape
    n_pages = -(-n // page)
    perm = (torch.randperm(n_pages + 3, generator=torch.Generator()
                           .manual_seed(seed))[:n_pages] + 1)
    pool = torch.zeros(n_pages + 5, page, rp, dtype=dtype)
    for j in range(n):
        pool[perm[j // page], j % page, :R] = c[j].to(dtype)
    return pool.to(device), perm.to(torch.int32).view(1, -1).to(device)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,R,page,n,simple", [
    (4, 32, 16, 300, False), (3, 96, 4, 90, False), (20, 128, 16, 150, False),
    (5, 256, 8, 70, False), (2, 512, 16, 80, False), (1, 64, 16, 40, False),
    (6, 64, 16, 90, True)])
def test_latent_attention_sink_and_head_gate(device, dtype, H, R, page, n,
                                             simple, monkeypatch):
    """Sinks of very different weight — one that takes nearly everything,
    one that is invisible — and a planted key near the start that only two
    queries ask for: as one prompt, as a later portion and decoded."""
    monkeypatch.setattr(ops, "LATENT_SIMPLE", simple)
    scale = R ** -0.5
    q, c = rnd(n, H, R, seed=1), rnd(n, R, seed=2)
    sink = torch.linspace(-8.0, 7.0, H) if H > 1 else torch.tensor([3.0])
    far = min(page, 5)                       # first row of a page or inside
    for i in (n - 2, n - 1):
        q[i] = 0.0
        q[i, :, 0] = 1.0
    c[:, 0] = 0.0
    c[far] = 0.0
    c[far, 0] = 14.0 / scale                 # beats hundreds of keys
    c[far, 1] = 9.0
    q, c = q.to(dtype).float(), c.to(dtype).float()
    kv = c.double().unsqueeze(1).expand(n, H, R)
    plain = O.sink_softmax_attention(q.double(), kv, kv, scale, sink.double())
    assert float(plain[n - 1, :, 1].min()) > 8.0      # the far key is seen
    no_sink = O.sink_softmax_attention(q.double(), kv, kv, scale,
                                       torch.full((H,), -1e4).double())
    assert float((plain[0] - no_sink[0]).abs().max()) > 0.2 * float(
        no_sink[0].abs().max())                       # and so is the sink
    gate = rnd(n, H + 8, seed=3, scale=2.0).to(dtype)
    want = plain * O.sigmoid(gate[:, :H].double()).unsqueeze(-1)
    pool, table = paged_rows(c, page, R, device, dtype)
    ql = q.transpose(0, 1).contiguous().to(device=device, dtype=dtype)
    sd = sink.to(device)
    gd = gate.to(device)[:, :H]                       # a strided view
    causal = 1 << 30

    def call(lo, hi, decode=False, s=sd, g=gd):
        out = torch.empty(H, hi - lo, R, device=device, dtype=dtype)
        ops.latent_window_attention(
            out, ql[:, lo:hi].contiguous(), pool, table, i32(device, hi),
            None if decode else i32(device, 0),
            None if decode else i32(device, hi - lo), scale, causal,
            max_qlen=hi - lo, sink=s, head_gate=None if g is None
            else g[lo:hi])
        return out.transpose(0, 1)

    close(call(0, n), want, dtype)
    lo = n - 7
    close(call(lo, n), want[lo:n], dtype)
    for i in (0, 1, page - 1, page, n - 2, n - 1):
        close(call(i, i + 1, decode=True), want[i:i + 1], dtype)
    close(call(lo, n, g=None), plain[lo:n], dtype)
    close(call(n - 1, n, decode=True, g=None), plain[n - 1:], dtype)
    close(call(lo, n, s=None, g=None), no_sink[lo:n], dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mx,n", [
    (O.latent_layer(heads=4, dim=32, vdim=16, q_rank=40, kv_rank=48), 140),
    (O.latent_layer(heads=3, dim=9, vdim=20, q_rank=11, kv_rank=10,
                    scale=0.21), 50),
    (O.latent_layer(heads=1, dim=16, vdim=8, q_rank=24, kv_rank=128), 60)])
def test_latent_attention_module_over_paged_pool(device, dtype, mx, n):
    """The serving module (absorbed key map, value map after the sum, sink
    and gate inside the kernels) against the oracle's expanded keys and
    values: portions, then decoded tokens."""
    from agentainer_amd.models.lelitar import LatentAttention
    from agentainer_amd.models.mugazen import config_from_dict

    W, eps, page = 48, 1e-4, 8
    cfg = O.make_config([(mx, None)], width=W, eps=eps)
    w = O.random_weights(cfg, seed=3)
    w["l0.mix.uq"] *= 4.0                   # peaked scores
    mc = config_from_dict(cfg).layers[0].latent
    h = rnd(n, W, seed=7)
    want = O.latent_mixer(h.double(), {k: t.double() for k, t in w.items()},
                          "l0.mix.", mx["mixer"], eps)
    mod = LatentAttention(W, mc, eps, dtype).to(device)
    mod.load(lambda name: w["l0.mix." + name].to(device=device, dtype=dtype))
    perm = torch.randperm(-(-n // page), generator=torch.Generator()
                          .manual_seed(1)) + 1
    pool = torch.zeros(perm.numel() + 2, page, mc.padded_rank, device=device,
                       dtype=dtype)
    got, at = [], 0
    for m in [n - 15, 2, 7] + [1] * 6:
        md = step_metadata(device, at, m, 0, page, perm, m == 1)
        got.append(mod(h[at:at + m].to(device=device, dtype=dtype), pool,
                       md).float().cpu())
        at += m
    close(torch.cat(got), want, dtype, 1e-4, 6e-2)


# ----------------------------------------------------------- feed-forward

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F,limit", [(24, 1.0), (30, 0.75), (64, 7.0)])
def test_clamped_dense_unit(device, dtype, F, limit):
    """Values beyond both clamps: the gate is capped from above only, the
    up branch on both sides."""
    from agentainer_amd.models.mugazen import ClampedFeedForward

    z = rnd(9, 2 * F, seed=1, scale=3.0 * limit)
    out = torch.empty(9, F, device=device, dtype=dtype)
    ops.routed_clamped_glu(out, z.to(device=device, dtype=dtype), None, 1,
                           limit, 1.702)
    want = O.clamped_unit(z.double()[:, :F], z.double()[:, F:], limit)
    close(out, want, dtype)
    assert float(z[:, :F].min()) < -limit and float(z[:, :F].max()) > limit
    W = 20
    w = {"gate": rnd(F, W, seed=2), "up": rnd(F, W, seed=3),
         "down": rnd(W, F, seed=4, scale=0.3)}
    h = rnd(6, W, seed=5)
    mod = ClampedFeedForward(W, F, limit, dtype).to(device)
    mod.load(lambda n: w[n].to(device=device, dtype=dtype))
    want = O.dense_ff(h.double(), {k: t.double() for k, t in w.items()}, "",
                      {"limit": limit})
    close(mod(h.to(device=device, dtype=dtype)), want, dtype, 2e-5, 3e-2)


def expert_case(E, top, F, W, seed=0):
    w = {"router": rnd(E, W, seed=seed + 1), "router.b": rnd(
        E, seed=seed + 2, scale=3.0)}
    for e in range(E):
        for k, (nm, a, b) in enumerate((("gate", F, W), ("up", F, W),
                                        ("down", W, F))):
            w[f"e{e}.{nm}"] = rnd(a, b, seed=seed + 10 + 3 * e + k, scale=0.4)
    return w, {"router": {"experts": E, "top": top}, "expert": {"ff": F}}


def expert_module(E, top, F, W, w, device, dtype):
    from agentainer_amd.models.mugazen import (MugazenFeedForwardConfig,
                                               TopSoftmaxExperts)
    mod = TopSoftmaxExperts(W, MugazenFeedForwardConfig(
        "moe", F, experts=E, top=top), dtype).to(device)
    mod.load(lambda n: w[n].to(device=device, dtype=dtype))
    return mod


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,top", [(8, 2), (5, 5), (7, 1), (70, 3), (1, 1)])
def test_router_softmax_over_chosen_logits(device, E, top):
    """Bias decides some choices AND enters the weights; the weights are the
    softmax over the chosen logits only and sum to one."""
    W = 24
    w, ml = expert_case(E, top, 4, W)
    mod = expert_module(E, top, 4, W, w, device, torch.float32)
    h = rnd(40, W, seed=77)
    got = mod.route(h.to(device)).double().cpu()
    want = torch.zeros(40, E, dtype=F64)
    w64 = {k: t.double() for k, t in w.items()}
    for t, chosen in enumerate(O.route(h.double(), w64, "", ml["router"])):
        for e, x in chosen:
            want[t, e] = x
    assert torch.allclose(got, want, atol=2e-6)
    assert torch.allclose(got.sum(-1), torch.ones(40, dtype=F64), atol=1e-5)
    if E > top:
        w64["router.b"] = torch.zeros(E, dtype=F64)
        other = O.route(h.double(), w64, "", ml["router"])
        assert any({e for e, _ in c} != set(want[t].nonzero().view(-1).tolist())
                   for t, c in enumerate(other))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,F", [(6, 2, 12), (4, 4, 5), (9, 1, 16)])
def test_experts_stacked_and_gathered(device, dtype, E, top, F):
    W = 24
    w, ml = expert_case(E, top, F, W, seed=100)
    # choices far from ties, so bf16 rows choose the same experts
    w["router.b"] = 12.0 * torch.arange(E, dtype=torch.float32)
    mod = expert_module(E, top, F, W, w, device, dtype)
    h = rnd(33, W, seed=78, scale=0.5)
    want = O.expert_mixture(h.double(), {k: t.double() for k, t in w.items()},
                            "", ml)
    hd = h.to(device=device, dtype=dtype)
    close(mod(hd, allow_gather=False), want, dtype, 2e-5, 3e-2)
    mod.SPARSE_MIN_TOKENS = 1
    close(mod(hd), want, dtype, 2e-5, 3e-2)


# ------------------------------------------------------------ config reader

def test_config_reader_runs_and_cache_entries():
    from agentainer_amd.models.mugazen import config_from_dict

    d = O.make_config([(O.delta_layer(), O.dense_mlp()),
                       (O.latent_layer(kv_rank=40), O.moe_mlp()),
                       (O.delta_layer(conv=2), None)], loop=(1, 3, 3),
                      max_positions=77)
    c = config_from_dict(d)
    assert [(r.layer, r.loop_pass, r.enters) for r in c.runs()] == [
        (0, None, False), (1, 0, True), (2, 0, False), (1, 1, True),
        (2, 1, False), (1, 2, True), (2, 2, False)]
    assert [(i, t) for i, t, _e in c.runs()] == O.run_order(d)
    assert c.n_layers == 7 and c.max_position == 77
    layout = c.cache_layout()
    assert layout.kv_shapes == [None, (64,), None, (64,), None, (64,), None]
    assert [bool(s) for s in layout.state_shapes] == [True, False, True,
                                                      False, True, False, True]
    assert c.kv_bytes_per_token(2) == 3 * 64 * 2
    for bad in (dict(start=2, stop=1, times=2), dict(start=0, stop=4, times=1),
                dict(start=0, stop=1, times=0)):
        with pytest.raises(ValueError):
            config_from_dict(dict(d, loop=bad))
    for key, val in (("type", "attention"), ("mlp", {"kind": "gated"})):
        broken = dict(d, layers=[dict(d["layers"][0], **{key: val})])
        broken.pop("loop")
        with pytest.raises(ValueError):
            config_from_dict(broken)
    plain = dict(d)
    plain.pop("loop")
    assert [r.layer for r in config_from_dict(plain).runs()] == [0, 1, 2]
