"""Lomazen on the CPU: the package's host side (configuration, weight stacking, model wiring with looped layers, ScheduleBatch /
ForwardBatch, the layered cache and request pools, TraceReplayer, Scheduler) runs with the CPU stand-in ops (tests/cpu_ops.py)
and every logit is compared with the plain whole-sequence implementation in oracle/lomazen_ref.py.  The HIP kernels have
their own file (test_lomazen_gpu.py); here the arithmetic is the stand-in's, the bookkeeping is the package's."""
import math

import pytest
import torch

import lomazen_cases as cases
import lomazen_util as lu
from oracle import lomazen_ref as ref

TOL = 2e-5


@pytest.fixture(autouse=True)
def _cpu_backend():
    import cpu_ops
    from sglang_custom_amd import ops_backend
    from sglang_custom_amd.distributed import parallel_state

    prev = ops_backend._backend
    ops_backend.set_ops_backend(cpu_ops)
    parallel_state.init_distributed_environment(1, 0)
    yield
    ops_backend.set_ops_backend(prev)


@pytest.fixture(scope="module")
def model():
    cfg = lu.make_config()
    return cfg, lu.make_weights(cfg, seed=3)


def test_oracle_restatements_agree():
    """The oracle's attention against explicit sums over the visible keys, its difference from the two maps' own weights, its
    rotation against complex multiplication, its walk over looped layers against hand-made lists."""
    g = torch.Generator().manual_seed(0)
    T, d, dv = 13, 6, 4
    q, k, v = (torch.randn(T, *s, generator=g, dtype=torch.float64) for s in ((2, 2, d), (1, 2, d), (1, dv)))
    a = [ref.causal_attention(q[:, :, m], k[:, :, m], v, 0.7, 2.0) for m in (0, 1)]
    for t in (0, 5, 12):
        for h in (0, 1):
            s = torch.tensor([2.0 * math.tanh(0.7 * float(q[t, h, 1] @ k[j, 0, 1]) / 2.0) for j in range(t + 1)], dtype=torch.float64)
            w = torch.exp(s) / torch.exp(s).sum()
            assert float((a[1][t, h] - w @ v[: t + 1, 0]).abs().max()) < 1e-12
    o = ref.difference_attention(q, k, v, 0.7, 0.4, 0.25, 1e-5)
    raw = [ref.causal_attention(q[:, :, m], k[:, :, m], v, 0.7) for m in (0, 1)]
    e = raw[0] - 0.4 * raw[1]
    assert float((o - 0.75 * e / torch.sqrt(e.pow(2).mean(-1, keepdim=True) + 1e-5)).abs().max()) < 1e-12
    f, pos = ref.frequencies(d, 30.0), torch.arange(T)
    z = torch.view_as_complex(q[:, 0, 0].reshape(T, d // 2, 2).contiguous()) * torch.exp(1j * pos[:, None] * f[None])
    assert float((ref.rotate(q[:, 0, :1], pos, f, True)[:, 0].reshape(T, -1, 2) - torch.view_as_real(z)).abs().max()) < 1e-12
    halves = torch.cat([q[:, 0, 0, 0::2], q[:, 0, 0, 1::2]], -1)[:, None]
    r = ref.rotate(halves, pos, f, False)[:, 0]
    assert float((torch.stack([r[:, : d // 2], r[:, d // 2:]], -1) - torch.view_as_real(z)).abs().max()) < 1e-12
    walk = ref.layer_walk(dict(layers=[0] * 4, loop=dict(start=1, stop=3, times=2)))
    assert walk == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert ref.layer_walk(dict(layers=[0] * 2)) == [(0, None), (1, None)]


@pytest.mark.parametrize("kind", ["attention", "attention_2"])
@pytest.mark.parametrize("mlp", ["none", "dense", "moe", "moe_top1"])
def test_each_mixer_alone(kind, mlp):
    """One-layer models: whole, cut, and token by token."""
    mixer = dict(attention=lu.attention(), attention_2=lu.attention_2())[kind]
    ff = dict(none=None, dense=lu.dense(24), moe=lu.moe(top=3), moe_top1=lu.moe(top=1))[mlp]
    cfg = lu.make_config(layers=[(mixer, ff)], loop=None)
    w = lu.make_weights(cfg, seed=1)
    prompts = lu.random_prompts(cfg, [25])
    mr = lu.build_runner(cfg, w)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 25)]], TOL)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 7)], [("r0", 2)]] + [[("r0", 1)] for _ in range(16)], TOL)
    assert lu.pools_are_whole(mr)


def test_whole_prompt_then_token_by_token(model):
    cfg, w = model
    prompts = lu.random_prompts(cfg, [31])
    mr = lu.build_runner(cfg, w)
    want = {"r0": ref.forward(cfg, w, prompts["r0"])}
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 31)]], TOL, want_all=want)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 1)] for _ in range(31)], TOL, want_all=want)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 9)]] + [[("r0", 1)] for _ in range(22)], TOL, want_all=want)
    assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("sizes", [[2, 2, 2, 3, 5, 2, 7, 1, 1, 2, 6], [1, 4, 4, 4, 4, 4, 4, 2, 3, 3], [31, 2]])
def test_portions_of_any_size(model, sizes):
    cfg, w = model
    prompts = lu.random_prompts(cfg, [sum(sizes)], seed=5)
    mr = lu.build_runner(cfg, w)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", k)] for k in sizes], TOL)
    assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("page_size", [1, 4, 6])
def test_mixed_batches_reuse_slots_and_pages(model, page_size):
    """Unequal requests side by side -- portions beside single tokens, a request that sits a step out, requests that end
    while others go on -- in a pool so small that cache rows and request rows are all handed out again."""
    cfg, w = model
    prompts = lu.random_prompts(cfg, [27, 9, 1, 12, 30, 6], seed=7)
    sched = [[("r0", 5), ("r1", 2)], [("r0", 1), ("r1", 7), ("r2", 1)], [("r0", 4), ("r3", 3)], [("r3", 1)],
             [("r0", 1), ("r3", 1)], [("r0", 16), ("r3", 7), ("r4", 2)], [("r4", 1), ("r5", 1)], [("r4", 1), ("r5", 1)],
             [("r4", 19), ("r5", 4)], [("r4", 1)], [("r4", 6)]]
    mr = lu.build_runner(cfg, w, max_total_tokens=72, max_running_requests=3, page_size=page_size)
    want = {k: ref.forward(cfg, w, p) for k, p in prompts.items()}
    for _ in range(2):         # the second time on the used pools: stale rows
        lu.replay_and_compare(mr, cfg, w, prompts, sched, TOL, want_all=want)
        assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("loop", [None, (0, 5, 2), (0, 1, 3), (4, 5, 2), (2, 2, 4), (1, 3, 1), (0, 5, 1)])
def test_loops(loop):
    """Around the first, the last, all, one or no layers; once; several times: runs, caches, the start of every pass."""
    cfg = lu.make_config(loop=loop)
    w = lu.make_weights(cfg, seed=3)
    prompts = lu.random_prompts(cfg, [17, 6], seed=2)
    mr = lu.build_runner(cfg, w, max_total_tokens=48)
    if loop == (2, 2, 4):       # a loop over nothing has no passes
        walk = [(i, None) for i in range(5)]
        bare = {k: v for k, v in cfg.items() if k != "loop"}
    else:
        walk, bare = ref.layer_walk(cfg), cfg
    mc = mr.model_config
    assert mc.layer_runs == [i for i, _ in walk] and mc.pass_starts == [t for _, t in walk] and mr.token_to_kv_pool.layer_num == len(walk)
    assert len({b.data_ptr() for b in mr.token_to_kv_pool.k_buffer}) == len(walk), "every run has a cache of its own"
    assert mr.req_to_token_pool.state_pool is None
    streams, got = [], []
    want = ref.forward(bare, w, prompts["r0"], streams=streams)
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    mr.model.model.capture_streams = got
    out = TraceReplayer(mr).step([dict(id="x", tokens=prompts["r0"], want=list(range(17)))], ["x"])
    mr.model.model.capture_streams = None
    assert lu.rel_err(out, want) < TOL and len(got) == len(streams) == len(walk)
    for a, b in zip(got, streams):
        assert float((a.double() - b).abs().max()) < 1e-3, "the stream after every layer run"
    lu.replay_and_compare(mr, bare, w, prompts, [[("r0", 6), ("r1", 1)], [("r0", 1), ("r1", 3)], [("r0", 9), ("r1", 2)], [("r0", 1)]], TOL)


def test_equal_and_unit_sizes():
    """Sizes that a model may happen to make equal or 1: one head, widths of 1 and 2, no rotation, no bands, one expert, all experts,
    width equal to the vocabulary, no factor on the logits, no cap, a difference whose two maps count alike."""
    layers = [(lu.attention(heads=1, kv_heads=1, dim=2, vdim=1), lu.moe(experts=1, top=1, ff=1)),
              (lu.attention_2(heads=1, kv_heads=1, dim=1, vdim=2, rot_dims=0), lu.dense(1)),
              (lu.attention(heads=8, kv_heads=1, dim=8, vdim=8, softcap=None, rot_dims=0), lu.moe(experts=4, top=4, ff=16)),
              (lu.attention_2(heads=16, kv_heads=16, dim=2, vdim=2, rot_dims=2, diff=0.0), None),
              (lu.attention(heads=4, kv_heads=4, dim=4, vdim=4, scaling=False), lu.dense(16)),
              (lu.attention_2(heads=2, kv_heads=2, dim=4, vdim=4, rot_dims=4), None)]
    cfg = lu.make_config(layers=layers, width=16, vocab=16, logit_scale=None, loop=(2, 3, 2))
    w = lu.make_weights(cfg, seed=11)
    prompts = lu.random_prompts(cfg, [14, 5], seed=1)
    mr = lu.build_runner(cfg, w, max_total_tokens=32)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 3), ("r1", 1)], [("r0", 1), ("r1", 1)], [("r0", 10), ("r1", 3)]], 1e-4)


def test_prefix_cache_serves_the_design(model):
    """Nothing but cache rows is kept per sequence: requests that share a prompt's start share its rows, loops included."""
    from sglang_custom_amd.managers.schedule_batch import Req
    from sglang_custom_amd.managers.scheduler import Scheduler
    from sglang_custom_amd.sampling.sampling_params import SamplingParams

    cfg, w = model
    mr = lu.build_runner(cfg, w)
    sch = Scheduler(mr, enable_radix_cache=True)
    shared = lu.random_prompts(cfg, [12], seed=4)["r0"]
    asks = {"a": shared + [3, 4], "b": shared + [5], "c": shared[:9] + [1, 2, 3]}
    for k, p in asks.items():
        sch.add_request(Req(k, p, SamplingParams(temperature=0, max_new_tokens=4)))
        done = sch.run_until_done()
        assert done[k].output_ids == ref.greedy(cfg, w, p, 4), k


def test_cache_rows_are_what_the_next_step_reads(model):
    """Cutting a prompt must hand over exactly what each run keeps: corrupting a key or a value row of ONE run changes the next
    portion's logits, and every run has its own."""
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    cfg, w = model
    toks = lu.random_prompts(cfg, [16], seed=2)["r0"]
    mr = lu.build_runner(cfg, w)
    kvp = mr.token_to_kv_pool
    assert mr.model_config.layer_runs == [0, 1, 2, 3, 1, 2, 3, 4] and mr.model_config.pass_starts == [None, 0, None, None, 1, None, None, None]
    assert [tuple(b.shape[1:]) for b in kvp.k_buffer] == [(3, 20), (2, 12), (2, 12), (1, 20), (2, 12), (2, 12), (1, 20), (5, 8)]
    assert [tuple(b.shape[1:]) for b in kvp.v_buffer] == [(3, 14), (2, 10), (2, 16), (1, 6), (2, 10), (2, 16), (1, 6), (5, 12)]
    want = ref.forward(cfg, w, toks)
    rp = TraceReplayer(mr)
    assert lu.rel_err(rp.step([dict(id="a", tokens=toks[:12], want=list(range(12)))]), want[:12]) < TOL
    bad = []
    for buffers in (kvp.k_buffer, kvp.v_buffer):
        for run in range(8):
            rp2 = TraceReplayer(mr)
            rp2.step([dict(id="b", tokens=toks[:12], want=[])])
            buffers[run][mr.req_to_token_pool.req_to_token[rp2.live["b"].req_pool_idx, 4].long()] += 2.0
            bad.append(lu.rel_err(rp2.step([dict(id="b", tokens=toks[12:13], want=[0])], ["b"]), want[12:13]))
    assert min(bad) > 1e-4, bad
    assert lu.rel_err(rp.step([dict(id="a", tokens=toks[12:], want=[0, 1, 2, 3])], ["a"]), want[12:]) < TOL
    assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("chunk,mixed", [(None, False), (6, False), (6, True)])
def test_greedy_generation_through_the_scheduler(model, chunk, mixed):
    """The package's own entry point: requests queued at the Scheduler, prompts chunked by its policy, decode batches
    (and decode tokens riding prefill batches) formed by it, tokens picked by the Sampler."""
    from sglang_custom_amd.managers.schedule_batch import Req
    from sglang_custom_amd.managers.scheduler import Scheduler
    from sglang_custom_amd.sampling.sampling_params import SamplingParams

    cfg, w = model
    prompts = lu.random_prompts(cfg, [11, 3, 7, 15, 1], seed=9)
    mr = lu.build_runner(cfg, w, max_total_tokens=96, max_running_requests=3, chunked_prefill_size=chunk, enable_mixed_chunk=mixed)
    sch = Scheduler(mr)
    for k, p in prompts.items():
        sch.add_request(Req(k, p, SamplingParams(temperature=0, max_new_tokens=6)))
    done = sch.run_until_done()
    for k, p in prompts.items():
        assert done[k].output_ids == ref.greedy(cfg, w, p, 6), k
    assert lu.pools_are_whole(mr)
    if chunk:
        assert sch.num_prefill_batches > 3


def test_capture_needs_nothing_of_the_other_families(model, monkeypatch):
    """A library built for this family alone lacks the split-KV decode kernels: preparing, capturing and replaying a step must not ask
    for their plan or counters."""
    import cpu_ops
    from sglang_custom_amd import build
    from sglang_custom_amd.model_executor.forward_batch_info import ForwardMode

    cfg, w = model
    assert "attn_causal.hip" in build.FAMILY_SOURCES["Lomazen"] and "attn_decode.hip" not in build.FAMILY_SOURCES["Lomazen"]
    mr = lu.build_runner(cfg, w)

    def absent(*_a, **_k):
        raise RuntimeError("not in this library")

    monkeypatch.setattr(cpu_ops, "decode_num_splits", absent, raising=False)
    b, two = mr.attn_backend, torch.ones(2, dtype=torch.int64)
    b.init_cuda_graph_state(2, 2)
    b.init_forward_metadata_capture_cuda_graph(2, 2, two, two, None, ForwardMode.DECODE, None)
    assert b.forward_metadata is not None
    b.init_forward_metadata_replay_cuda_graph(2, two, two, 2, None, ForwardMode.DECODE, None, two)
    assert b._lse is None and b._tickets is None


def test_planted_mistakes_show(model):
    """Each branch of the design left out of the oracle moves the logits far past the tolerance: what the comparisons above rest on."""
    cfg, w = model
    toks = lu.random_prompts(cfg, [18], seed=6)["r0"]
    want = ref.forward(cfg, w, toks)

    def moved(change_cfg=None, change_w=None):
        c = lu.make_config()
        if change_cfg:
            change_cfg(c)
        w2 = dict(w)
        if change_w:
            change_w(w2)
        return lu.rel_err(ref.forward(c, w2, toks), want)

    def scale_of(i, name, value):
        return lambda c: c["layers"][i]["mixer"].__setitem__(name, value)

    errors = dict(cap=moved(scale_of(1, "softcap", None)), bands=moved(lambda c: c["layers"][1]["mixer"]["rot"].pop("scaling")),
                  rotation=moved(lambda c: c["layers"][0]["mixer"].pop("rot")), diff=moved(scale_of(0, "diff", 0.31)),
                  lam=moved(None, lambda x: x.__setitem__("l0.mix.lq1", -x["l0.mix.lq1"])), step=moved(None, lambda x: x.__setitem__("loop.step", x["loop.step"].flip(0))),
                  entry=moved(None, lambda x: x.__setitem__("loop.in", torch.cat([x["loop.in"][:, 48:], x["loop.in"][:, :48]], 1))),
                  gate=moved(None, lambda x: x.__setitem__("l1.mix.g", 0 * x["l1.mix.g"])), head_gate=moved(None, lambda x: x.__setitem__("l2.mix.g", 0 * x["l2.mix.g"])),
                  passes=moved(lambda c: c["loop"].__setitem__("times", 1)), top=moved(lambda c: c["layers"][1]["mlp"]["router"].__setitem__("top", 1)))
    assert min(errors.values()) > 50 * TOL, errors


def test_configuration_is_read_not_assumed():
    from sglang_custom_amd.configs.model_config import ModelConfig
    from sglang_custom_amd.models.registry import get_model_class

    mc = ModelConfig(lu.make_config(), dtype="float32")
    assert mc.architecture == "Lomazen" and get_model_class(mc.architecture).__name__ == "LomazenForCausalLM"
    assert mc.layer_runs == [0, 1, 2, 3, 1, 2, 3, 4] and mc.num_hidden_layers == 8 and mc.loop_times == 2
    assert mc.kv_layer_shapes == [(3, 20, 14), (2, 12, 10), (2, 12, 16), (1, 20, 6), (2, 12, 10), (2, 12, 16), (1, 20, 6), (5, 8, 12)]
    assert mc.logit_scale == 1.5 and mc.rms_norm_eps == 1e-5 and mc.v_head_dim == 16 and not mc.needs_sequence_state
    for path, value in ((("layers", 1, "type"), "something_else"), (("layers", 0, "mlp", "kind"), "other"),
                        (("layers", 1, "mlp", "router", "top"), 6), (("layers", 1, "mixer", "rot", "dims"), 14),
                        (("layers", 1, "mixer", "rot", "dims"), 5), (("layers", 0, "mixer", "kv_heads"), 2), (("layers", 0, "mixer", "scale"), 0.0),
                        (("loop", "stop"), 6), (("loop", "start"), 5), (("loop", "times"), 0)):
        bad = lu.make_config()
        node = bad
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = value
        with pytest.raises(ValueError):
            ModelConfig(bad)


# ---- the stand-in ops themselves against the oracle's functions: the same cases the HIP kernels run on the GPU
def test_standins_norms_entry_units():
    import cpu_ops

    cases.check_norm_add_norm(cpu_ops, "cpu", torch.float32)
    cases.check_pass_entry(cpu_ops, "cpu", torch.float32)
    cases.check_pass_entry_layer("cpu", torch.float32)
    cases.check_gated_unit(cpu_ops, "cpu", torch.float32)
    cases.check_moe_layer("cpu", torch.float32, 9)
    cases.check_moe_layer("cpu", torch.float32, 5, top=1)


def test_standins_rotation_and_attention():
    import cpu_ops

    cases.check_frequencies()
    cases.check_rotate_write(cpu_ops, "cpu", torch.float32)
    cases.check_rotate_write(cpu_ops, "cpu", torch.float32, interleaved=False, unit_norm=False, rot=6)
    cases.check_rotate_write(cpu_ops, "cpu", torch.float32, rot=0)
    for maps, gate in ((1, "feature"), (2, "head"), (1, None)):
        cases.check_attention(cpu_ops, "cpu", torch.float32, maps=maps, gate=gate, cap=3.0 if maps == 1 else 0.0, T=50, cuts=(17, 2, 30, 1), decode_tail=1)
        cases.check_batch_of_unequal(cpu_ops, "cpu", torch.float32, maps=maps)
    cases.check_score_cap(cpu_ops, "cpu", torch.float32)
    cases.check_difference(cpu_ops, "cpu", torch.float32)
    cases.check_rotation_decides(cpu_ops, "cpu", torch.float32)
