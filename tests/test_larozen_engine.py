"""Larozen through the serving engine (one cache entry per layer RUN, K/V
pools with shortened value rows, recurrent state slots, varlen + decode
paths, scheduler) against the plain float64 oracle. Every scenario runs on
CPU (reference ops) and, marked gpu, on the MI355X (HIP kernels, captured
decode graph). Models are small random ones in float32 so that a pass that
reads another pass's memory, a lost state, a position that is one off or a
missing sink shows far above the tolerance."""

import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import larozen_oracle as O  # noqa: E402

from agentainer_amd.config import load_config  # noqa: E402
from agentainer_amd.engine.llm import GenRequest, LLMEngine  # noqa: E402
from agentainer_amd.store import Store  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]


def make_instance(tmp_path, cfg, weights, device, dtype="float32", page=4,
                  pool_tokens=512, slots=4, **extra):
    path = str(tmp_path / "ckpt")
    O.save_checkpoint(path, cfg, weights)
    conf = load_config(path="/nonexistent.yaml", env={})
    conf.data["store"]["path"] = str(tmp_path / "root")
    e = conf.data["engine"]
    e.update(sync_mode=True, async_decode=False, prefill_stream=False,
             prefix_sharing=False, dtype=dtype, kv_page_size=page,
             kv_pool_tokens=pool_tokens,
             max_seqs=slots + (1 if device == "cuda" else 0),
             max_pages_per_seq=-(-pool_tokens // page),
             max_batch_tokens=1 << 20)
    e.update(extra)
    store = Store(str(tmp_path / "root" / "state"), sync="never")
    if device == "cuda":
        torch.backends.cuda.matmul.allow_tf32 = False
    eng = LLMEngine(store, conf, device=device,
                    state_root=str(tmp_path / "root"))
    return eng, eng._get_instance(path), path


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(3, cfg["vocab"], (n,), generator=g).tolist()


def replay(inst, reqs, schedule):
    """schedule: list of steps, each [(request id, n tokens)]. Every
    position's logits are collected. Returns {id: [T, V] tensor}."""
    at = {i: 0 for i in reqs}
    got = {i: [] for i in reqs}
    for step in schedule:
        entries, want = [], []
        for i, n in step:
            entries.append((i, reqs[i][at[i]:at[i] + n]))
            want.append(list(range(n)))
            at[i] += n
        lg = inst.forward_step(entries, want).float().cpu()
        k = 0
        for i, n in step:
            got[i].append(lg[k:k + n])
            k += n
        for i, _n in step:
            if at[i] == len(reqs[i]):
                inst.release(i)
    return {i: torch.cat(v) for i, v in got.items() if v}


def check(got, cfg, weights, reqs, tol=3e-4):
    for i, toks in reqs.items():
        want = O.forward(toks, weights, cfg).float()
        assert got[i].shape == want.shape
        err = float((got[i] - want).abs().max() / want.abs().max())
        assert err < tol, f"request {i}: relative error {err:.3e}"


def cuts(total, sizes):
    out, k = [], 0
    while total > 0:
        n = min(sizes[k % len(sizes)], total)
        out.append(n)
        total -= n
        k += 1
    return out


def small_config(order="apa", **kw):
    """order: a / p = attention / parallel with a feed-forward, A / P =
    without one."""
    table = {"a": (O.attention_layer, 56), "p": (O.parallel_layer, 40),
             "A": (O.attention_layer, None), "P": (O.parallel_layer, None)}
    kw.setdefault("loop", (0, 2, 2))
    return O.make_config([(table[c][0](), table[c][1]) for c in order], **kw)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("order,loop", [("aApPa", (1, 3, 3)), ("pa", (0, 1, 2)),
                                        ("Ap", (1, 2, 1)), ("ap", None)])
def test_layer_runs_match_oracle_residual_trace(tmp_path, device, order, loop):
    """Run by run: the fp32 residual after every layer of every pass."""
    cfg = small_config(order=order, loop=loop)
    w = O.random_weights(cfg, seed=1)
    eng, inst, _ = make_instance(tmp_path, cfg, w, device)
    toks = tokens_for(cfg, 19, 1)
    trace = []
    want = O.forward(toks, w, cfg, trace).float()
    inst.model.residual_trace = []
    got = inst.forward_step([("a", toks)], [list(range(19))]).float().cpu()
    runs = inst.model.residual_trace
    inst.model.residual_trace = None
    assert len(runs) == len(trace) == len(O.run_order(cfg))
    for k, (a, b) in enumerate(zip(runs, trace)):
        # engine rows may carry bucket padding past the real tokens
        err = float((a[:19].cpu() - b.float()).abs().max() / b.abs().max())
        assert err < 1e-4, f"run {k}: {err:.3e}"
    assert float((got - want).abs().max() / want.abs().max()) < 3e-4


@pytest.mark.parametrize("device", DEVICES)
def test_prefill_equals_token_by_token_decode(tmp_path, device):
    """Whole prompt in one step == one token per step from the first token
    on (memories, convolution tails and pools carried per run)."""
    cfg = small_config()
    w = O.random_weights(cfg, seed=2)
    eng, inst, _ = make_instance(tmp_path, cfg, w, device)
    reqs = {"a": tokens_for(cfg, 30, 2), "b": tokens_for(cfg, 30, 2)}
    got = replay(inst, {"a": reqs["a"]}, [[("a", 30)]])
    got.update(replay(inst, {"b": reqs["b"]}, [[("b", 1)] for _ in range(30)]))
    check(got, cfg, w, reqs)
    assert float((got["a"] - got["b"]).abs().max()) < 1e-3


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("sizes", [[2], [3, 2, 7], [5, 1, 1, 2], [13, 2]])
def test_portions_of_several_sizes(tmp_path, device, sizes):
    """Portions cut mid-page, mid-chunk of the scan, and shorter than the
    convolution's reach (the tail is shifted, not replaced), then a decoded
    tail."""
    cfg = small_config(order="paP", loop=(1, 3, 2))
    w = O.random_weights(cfg, seed=3)
    eng, inst, _ = make_instance(tmp_path, cfg, w, device, page=4)
    toks = tokens_for(cfg, 41, 3)
    sched = [[("a", n)] for n in cuts(33, sizes)] + [[("a", 1)]] * 8
    check(replay(inst, {"a": toks}, sched), cfg, w, {"a": toks})


@pytest.mark.parametrize("device", DEVICES)
def test_mixed_batches_and_reuse_of_pages_and_slots(tmp_path, device):
    """Unequal requests side by side — portions beside single tokens — in
    a pool too small for all of them at once: pages and state slots of
    finished requests go to the next ones, whose first token must start
    from zero memory although the slot still holds the last owner's."""
    cfg = small_config(order="pap", loop=(0, 2, 2))
    w = O.random_weights(cfg, seed=4)
    eng, inst, _ = make_instance(tmp_path, cfg, w, device, page=4,
                                 pool_tokens=112, slots=4)
    reqs = {i: tokens_for(cfg, n, 10 + k) for k, (i, n) in enumerate(
        [("a", 40), ("b", 17), ("c", 3), ("d", 28), ("e", 36), ("f", 1)])}
    sched = [
        [("a", 16), ("b", 9)],
        [("a", 16), ("b", 1), ("c", 2)],
        [("a", 1), ("b", 1), ("c", 1)],             # pure decode batch
        [("a", 1), ("b", 6), ("d", 2)],             # c's slot reused by d
        [("a", 6), ("d", 26), ("f", 1)],            # a, b, d, f finish
        [("e", 30)],                                # reuses pages and a slot
        [("e", 1)], [("e", 1)], [("e", 4)],
    ]
    free0 = inst.kvm.free_pages
    got = replay(inst, reqs, sched)
    check(got, cfg, w, reqs)
    assert inst.kvm.free_pages == free0          # everything given back
    assert len(inst.kvm._free_slots) == 4
    # each request alone gives the same logits as inside the batches
    for i in ("b", "d"):
        alone = replay(inst, {i: reqs[i]}, [[(i, len(reqs[i]))]])
        assert float((alone[i] - got[i]).abs().max()) < 1e-3


@pytest.mark.parametrize("device", DEVICES)
def test_long_sequence_page_borders_long_decode(tmp_path, device):
    """150 tokens, half of them decoded one by one over many page borders
    and many steps of the query factor."""
    cfg = small_config(order="ap", loop=(0, 2, 2))
    w = O.random_weights(cfg, seed=5)
    eng, inst, _ = make_instance(tmp_path, cfg, w, device, page=8,
                                 pool_tokens=256)
    toks = tokens_for(cfg, 150, 5)
    sched = [[("a", 70)], [("a", 9)]] + [[("a", 1)]] * 71
    check(replay(inst, {"a": toks}, sched), cfg, w, {"a": toks})


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("path", ["tied", "left", "right"])
def test_far_tokens_are_really_read(tmp_path, device, path):
    """Exchanging one token near the start changes the logits 60 tokens
    later, decoded ones included, exactly as the oracle says: through either
    attention with one score standing out, or through a state-space memory
    that hardly decays (the other paths switched off)."""
    cfg = small_config(order="a" if path == "tied" else "p", loop=(0, 1, 2))
    w = O.random_weights(cfg, seed=12)
    if path == "tied":
        w["l0.mix.q"] *= 4.0                      # peaked softmax
    elif path == "left":
        w["l0.mix.left.q.norm"] *= 4.0
        w["l0.mix.right.out"] *= 0.0
    else:
        # decays close to one
        w["l0.mix.right.A_log"] = w["l0.mix.right.A_log"] - 7.0
        w["l0.mix.left.out"] *= 0.0
    w = {k: t.bfloat16().float() for k, t in w.items()}
    toks = tokens_for(cfg, 64, 12)
    other = list(toks)
    other[2] = (toks[2] + 17) % cfg["vocab"]
    reqs = {"a": toks, "b": other}
    eng, inst, _ = make_instance(tmp_path, cfg, w, device)
    got = replay(inst, reqs, [[("a", 40), ("b", 40)]]
                 + [[("a", 1), ("b", 1)]] * 24)
    check(got, cfg, w, reqs)
    d = (got["a"] - got["b"])[-1]
    want = (O.forward(toks, w, cfg) - O.forward(other, w, cfg))[-1].float()
    assert float(want.abs().max()) > 2e-3
    assert float((d - want).abs().max()) < 0.1 * float(want.abs().max())


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_and_query_factor_steps(tmp_path, device):
    """The first tokens, where sinks weigh most, and positions around the
    steps of the query factor, each as the first row of a portion, inside
    one, and decoded."""
    layer = O.parallel_layer(left=O.left_mixer(every=6, coef=1.5))
    cfg = O.make_config([(layer, 24)], loop=None)
    w = O.random_weights(cfg, seed=14)
    w["l0.mix.left.sink"] = (w["l0.mix.left.sink"] + 2.0).bfloat16().float()
    eng, inst, _ = make_instance(tmp_path, cfg, w, device)
    toks = tokens_for(cfg, 20, 14)
    for sched in ([5, 1, 5, 1, 1, 5, 2], [1] * 20, [4, 3, 4, 1, 8], [20]):
        got = replay(inst, {"a": toks}, [[("a", n)] for n in sched])
        check(got, cfg, w, {"a": toks}, 1e-4)
    # a factor that is one position late would be seen
    cfg2 = O.make_config([(O.parallel_layer(left=O.left_mixer(
        every=7, coef=1.5)), 24)], loop=None)
    a, b = O.forward(toks, w, cfg), O.forward(toks, w, cfg2)
    assert float((a[5] - b[5]).abs().max()) > 1e-2
    assert float((a[4] - b[4]).abs().max()) == 0.0


@pytest.mark.parametrize("device", DEVICES)
def test_passes_keep_separate_memories(tmp_path, device):
    """Running the group another number of times, or not feeding the
    embedding in, changes the logits; the engine follows the oracle in every
    variant, a single pass included, decoded tokens included."""
    cfg = small_config(order="apA", loop=(0, 2, 3))
    w = O.random_weights(cfg, seed=13)
    toks = tokens_for(cfg, 20, 13)
    sched = [[("a", 12)]] + [[("a", 1)]] * 8
    seen = []
    for k, (times, cut) in enumerate(((3, False), (2, False), (1, False),
                                      (2, True))):
        c = dict(cfg, loop=dict(cfg["loop"], times=times))
        v = dict(w)
        if cut:
            v["loop.in"] = w["loop.in"].clone()
            v["loop.in"][:, cfg["width"]:] = 0.0
        eng, inst, _ = make_instance(tmp_path / str(k), c, v, device)
        got = replay(inst, {"a": toks}, sched)
        check(got, c, v, {"a": toks})
        seen.append(got["a"])
    for i in range(len(seen)):
        for j in range(i):
            assert float((seen[i] - seen[j]).abs().max()) > 1e-2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("layers,kw", [
    # values that a usual model makes equal (or 1) all differ here
    ([(O.attention_layer(heads=6, kv_heads=3, dim=20, rot_dims=6, base=77.0,
                         scale=0.4, softcap=2.5), 44),
      (O.parallel_layer(O.left_mixer(heads=5, kv_heads=5, dim=8, vdim=20,
                                     coef=1.1, every=3),
                        O.right_mixer(heads=6, vdim=9, state=14, groups=3,
                                      conv=5, norm_groups=2)), None),
      (O.attention_layer(heads=2, kv_heads=1, dim=4, rot_dims=4), 12)],
     dict(width=40, loop=(1, 3, 2))),
    ([(O.parallel_layer(O.left_mixer(heads=1, kv_heads=1, dim=24, vdim=8,
                                     every=1),
                        O.right_mixer(heads=1, vdim=36, state=4, groups=1,
                                      conv=1, norm_groups=1)), 20),
      (O.attention_layer(heads=7, kv_heads=7, dim=12, rot_dims=2), None)],
     dict(width=32, eps=1e-3, loop=(1, 2, 4))),
    ([(O.parallel_layer(O.left_mixer(heads=8, kv_heads=1, dim=4, vdim=12),
                        O.right_mixer(heads=8, vdim=4, state=33, groups=8,
                                      conv=2, norm_groups=8)), 28),
      (O.parallel_layer(O.left_mixer(heads=2, kv_heads=2, dim=40, vdim=6,
                                     coef=0.0),
                        O.right_mixer(heads=4, vdim=10, state=20, groups=1,
                                      conv=4, norm_groups=5)), 8),
      (O.attention_layer(heads=4, kv_heads=4, dim=36, rot_dims=0), 16)],
     dict(width=64, loop=(2, 3, 1))),
    ([(O.attention_layer(), 30), (O.parallel_layer(), 30)],
     dict(width=50, loop=None)),
])
def test_other_sizes(tmp_path, device, layers, kw):
    cfg = O.make_config(layers, vocab=300, **kw)
    w = O.random_weights(cfg, seed=6)
    eng, inst, _ = make_instance(tmp_path, cfg, w, device, page=4)
    reqs = {"a": tokens_for(cfg, 23, 6), "b": tokens_for(cfg, 9, 7)}
    sched = [[("a", 11), ("b", 2)], [("a", 2), ("b", 1)],
             [("a", 1), ("b", 1)], [("a", 9), ("b", 5)]]
    check(replay(inst, reqs, sched), cfg, w, reqs)


@pytest.mark.parametrize("device", DEVICES)
def test_checkpoint_offload_restore(tmp_path, device):
    """A sequence's pages AND its per-run state (memories, convolution
    tails) survive offload to host and restore into other pages and another
    slot."""
    cfg = small_config()
    w = O.random_weights(cfg, seed=8)
    eng, inst, _ = make_instance(tmp_path, cfg, w, device, page=4)
    toks = tokens_for(cfg, 30, 8)
    inst.forward_step([("pre", toks[:5])], [[0]])  # takes the first slot
    a = inst.forward_step([("a", toks[:21])], [[20]]).float().cpu()
    ck = inst.kvm.offload("a", free=True)
    assert not inst.kvm.has_seq("a") and ck.state is not None
    inst.release("pre")
    inst.forward_step([("x", toks[:9])], [[0]])    # dirty pages and slots
    inst.forward_step([("y", toks[3:9])], [[0]])
    inst.kvm.restore("a", ck)
    b = inst.forward_step([("a", toks[21:])], [list(range(9))]).float().cpu()
    want = O.forward(toks, w, cfg).float()
    assert float((a[0] - want[20]).abs().max() / want.abs().max()) < 3e-4
    assert float((b - want[21:]).abs().max() / want.abs().max()) < 3e-4


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_scheduler(tmp_path, device):
    """Deploy the checkpoint directory as an agent and generate greedily
    through the engine's own scheduler (chunked admission: the step token
    budget is smaller than the prompt), against oracle argmax decoding."""
    from agentainer_amd.registry import Manager

    cfg = small_config(vocab=300)
    w = O.random_weights(cfg, seed=9)
    eng, inst0, path = make_instance(tmp_path, cfg, w, device, page=4,
                                     pool_tokens=400, slots=8,
                                     max_batch_tokens=8)
    conf = load_config(path="/nonexistent.yaml", env={})
    manager = Manager(eng.store, eng, conf)
    agents = [manager.deploy(name=f"g{k}", model=path,
                             sampling={"max_tokens": 12}) for k in range(2)]
    inst = eng._instances[path]
    assert inst.stateful and not inst.async_decode and not inst.prefix_sharing
    reqs = []
    for k, ag in enumerate(agents):
        manager.start(ag.id)
        prompt = tokens_for(cfg, 21 + 6 * k, 20 + k)
        r = GenRequest(agent_id=ag.id, prompt_tokens=prompt, max_new=12,
                       temperature=0.0, top_p=1.0, seed=0)
        b = inst.binding(ag.id)
        with inst._lock:
            b.queue.put(r)
            inst._pump_agent(b)
        reqs.append(r)
    for _ in range(200):
        inst.step()
        if all(r.done.is_set() for r in reqs):
            break
    for r in reqs:
        assert r.done.is_set() and not r.error, r.error
        # the sampler reads bf16 logits: every generated token must be the
        # oracle's argmax up to that rounding, given the tokens before it
        seq = list(r.prompt_tokens)
        assert 1 <= len(r.generated) <= 12
        for k, t in enumerate(r.generated):
            lg = O.forward(seq, w, cfg)[-1]
            assert float(lg[t]) >= float(lg.max()) - 0.01 * float(lg.abs().max()), (k, t)
            seq.append(t)
        assert (len(r.generated) == 12
                or r.generated[-1] == inst.tokenizer.eos_id)


def test_named_random_init_model_is_registered(tmp_path):
    """`deploy tiny-larozen` resolves through the family registry."""
    from agentainer_amd.models import registry

    assert registry.family_of("tiny-larozen") == "Larozen"
    assert registry.build_target("tiny-larozen") == "gated+masked+recurrent"
    conf = load_config(path="/nonexistent.yaml", env={})
    conf.data["store"]["path"] = str(tmp_path / "root")
    conf.data["engine"].update(sync_mode=True, kv_pool_tokens=128,
                               max_seqs=8)
    eng = LLMEngine(Store(str(tmp_path / "root" / "state"), sync="never"),
                    conf, device="cpu", state_root=str(tmp_path / "root"))
    eng.validate_model("tiny-larozen")
    inst = eng._get_instance("tiny-larozen")
    lg = inst.forward_step([("a", [5, 6, 7, 8])], [[3]])
    assert lg.shape == (1, 512) and bool(torch.isfinite(lg).all())
    # three layers, the last two of them twice: five cache entries; tied
    # values keep 16 of 32 coordinates
    assert [tuple(c[1].shape[1:]) for c in inst.kvm.caches] == [
        (2, 16, 16), (1, 16, 32), (2, 16, 16), (1, 16, 32), (2, 16, 16)]
    assert [bool(s) for s in inst.kvm.states] == [False, True, False, True,
                                                  False]


@pytest.mark.gpu
@pytest.mark.parametrize("layers,kw", [
    ([(O.attention_layer(heads=6, kv_heads=3, dim=64, rot_dims=24), 256),
      (O.parallel_layer(O.left_mixer(heads=4, kv_heads=1, dim=32, vdim=64,
                                     every=40),
                        O.right_mixer(heads=6, vdim=32, state=64, groups=3,
                                      conv=4, norm_groups=2)), 192)],
     dict(width=128, loop=(0, 2, 2))),
    # sizes the tile and vector kernels do not take
    ([(O.parallel_layer(O.left_mixer(heads=3, kv_heads=1, dim=20, vdim=12),
                        O.right_mixer(heads=3, vdim=11, state=10, groups=1,
                                      conv=2, norm_groups=3)), 60),
      (O.attention_layer(heads=3, kv_heads=3, dim=20, rot_dims=10), 70)],
     dict(width=72, loop=(1, 2, 3)))])
def test_bf16_serving_path_close_to_oracle(tmp_path, layers, kw):
    """bf16 serving precision (captured decode graph): logits stay within
    bf16 rounding of the oracle, and graph replays keep agreeing with it
    step after step."""
    cfg = O.make_config(layers, vocab=300, **kw)
    w = O.random_weights(cfg, seed=11)
    eng, inst, _ = make_instance(tmp_path, cfg, w, "cuda", dtype="bfloat16",
                                 page=16, pool_tokens=512)
    reqs = {"a": tokens_for(cfg, 120, 1), "b": tokens_for(cfg, 75, 2)}
    sched = ([[("a", 64), ("b", 3)], [("a", 30), ("b", 50)]]
             + [[("a", 1), ("b", 1)]] * 22 + [[("a", 4)]])
    got = replay(inst, reqs, sched)
    assert inst.use_graph and inst._graphs, "decode graph was not captured"
    for i, toks in reqs.items():
        want = O.forward(toks, w, cfg).float()
        d = got[i] - want
        d = d - d.mean(-1, keepdim=True)
        rel = d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
        assert float(rel.max()) < 0.08, rel
        assert float(rel.median()) < 0.03, float(rel.median())
