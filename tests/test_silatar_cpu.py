"""Silatar on the CPU: the package's host side (configuration, weight stacking, model wiring with looped layers, ScheduleBatch /
ForwardBatch, the latent / request / state pools, TraceReplayer, Scheduler) runs with the CPU stand-in ops (tests/cpu_ops.py)
and every logit is compared with the plain whole-sequence implementation in oracle/silatar_ref.py.  The HIP kernels have
their own file (test_silatar_gpu.py); here the arithmetic is the stand-in's, the bookkeeping is the package's."""
import math

import pytest
import torch

import silatar_cases as cases
import silatar_util as su
from oracle import silatar_ref as ref

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
    cfg = su.make_config()
    return cfg, su.make_weights(cfg, seed=3)


def test_oracle_restatements_agree():
    """The oracle's recurrence against a closed form -- weights exp(sum of later log forgets + log in) over all earlier tokens,
    divided by max(|their q.k sum|, 1): e^m cancels between numerator and denominator but for the 1e-6 -- and its attention
    against explicit softmaxes."""
    g = torch.Generator().manual_seed(0)
    T, d, dv = 17, 5, 4
    q, k, v = (torch.randn(T, 1, n, generator=g, dtype=torch.float64) for n in (d, d, dv))
    i, f = torch.randn(T, 1, generator=g, dtype=torch.float64) * 2, -torch.rand(T, 1, generator=g, dtype=torch.float64)
    o = ref.matrix_memory(q, k, v, i, f)
    for t in (0, 1, 9, 16):
        wt = torch.tensor([math.exp(float(f[s + 1: t + 1].sum() + i[s])) for s in range(t + 1)], dtype=torch.float64)
        qk = k[: t + 1, 0] @ q[t, 0]
        want = (wt * qk) @ v[: t + 1, 0] / max(abs(float((wt * qk).sum())), 1.0)
        assert float((o[t, 0] - want).abs().max()) < 2e-5 * max(1.0, float(want.abs().max()))
    a = ref.causal_softmax_attention(q, k, v, 0.7)
    for t in (0, 8, 16):
        p = torch.softmax(0.7 * (k[: t + 1, 0] @ q[t, 0]), 0)
        assert float((a[t, 0] - p @ v[: t + 1, 0]).abs().max()) < 1e-12
    assert ref.layer_runs(dict(layers=[0] * 5, loop=dict(start=1, stop=3, times=3))) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert ref.layer_runs(dict(layers=[0] * 3)) == [0, 1, 2]


@pytest.mark.parametrize("kind", ["latent_attention", "mlstm"])
@pytest.mark.parametrize("mlp", ["none", "dense", "moe", "moe_top1_no_shared"])
def test_each_mixer_alone(kind, mlp):
    """One-layer models: whole, cut, and token by token."""
    mixer = dict(latent_attention=su.latent(), mlstm=su.mlstm())[kind]
    ff = dict(none=None, dense=su.dense(24), moe=su.moe(top=3), moe_top1_no_shared=su.moe(top=1, shared=None))[mlp]
    cfg = su.make_config(layers=[(mixer, ff)], loop=None)
    w = su.make_weights(cfg, seed=1)
    prompts = su.random_prompts(cfg, [25])
    mr = su.build_runner(cfg, w)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 25)]], TOL)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 7)], [("r0", 2)]] + [[("r0", 1)] for _ in range(16)], TOL)
    assert su.pools_are_whole(mr)


def test_whole_prompt_then_token_by_token(model):
    cfg, w = model
    prompts = su.random_prompts(cfg, [31])
    mr = su.build_runner(cfg, w)
    want = {"r0": ref.forward(cfg, w, prompts["r0"])}
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 31)]], TOL, want_all=want)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 1)] for _ in range(31)], TOL, want_all=want)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 9)]] + [[("r0", 1)] for _ in range(22)], TOL, want_all=want)
    assert su.pools_are_whole(mr)


@pytest.mark.parametrize("sizes", [[2, 2, 2, 3, 5, 2, 7, 1, 1, 2, 6], [1, 4, 4, 4, 4, 4, 4, 2, 3, 3], [31, 2]])
def test_portions_of_any_size(model, sizes):
    cfg, w = model
    prompts = su.random_prompts(cfg, [sum(sizes)], seed=5)
    mr = su.build_runner(cfg, w)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", k)] for k in sizes], TOL)
    assert su.pools_are_whole(mr)


@pytest.mark.parametrize("page_size", [1, 4, 6])
def test_mixed_batches_reuse_slots_and_pages(model, page_size):
    """Unequal requests side by side -- portions beside single tokens, a request that sits a step out, requests that end
    while others go on -- in a pool so small that rows, request rows and state slots are all handed out again."""
    cfg, w = model
    prompts = su.random_prompts(cfg, [27, 9, 1, 12, 30, 6], seed=7)
    sched = [[("r0", 5), ("r1", 2)], [("r0", 1), ("r1", 7), ("r2", 1)], [("r0", 4), ("r3", 3)], [("r3", 1)],
             [("r0", 1), ("r3", 1)], [("r0", 16), ("r3", 7), ("r4", 2)], [("r4", 1), ("r5", 1)], [("r4", 1), ("r5", 1)],
             [("r4", 19), ("r5", 4)], [("r4", 1)], [("r4", 6)]]
    mr = su.build_runner(cfg, w, max_total_tokens=72, max_running_requests=3, page_size=page_size)
    want = {k: ref.forward(cfg, w, p) for k, p in prompts.items()}
    for _ in range(2):         # the second time on the used pools: stale rows, stale matrices, stale normalisers
        su.replay_and_compare(mr, cfg, w, prompts, sched, TOL, want_all=want)
        assert su.pools_are_whole(mr)


@pytest.mark.parametrize("loop", [None, (0, 5, 2), (0, 1, 3), (4, 5, 2), (2, 2, 4), (1, 3, 1), (0, 5, 1)])
def test_loops(loop):
    """Around the first, the last, all, one or no layers; once; several times: runs, caches and states."""
    cfg = su.make_config(loop=loop)
    w = su.make_weights(cfg, seed=3)
    prompts = su.random_prompts(cfg, [17, 6], seed=2)
    mr = su.build_runner(cfg, w, max_total_tokens=48)
    runs = ref.layer_runs(cfg)
    kinds = [cfg["layers"][i]["type"] for i in runs]
    assert mr.model_config.layer_runs == runs and mr.token_to_kv_pool.layer_num == len(runs)
    assert [b is not None for b in mr.token_to_kv_pool.kv_buffer] == [k == "latent_attention" for k in kinds]
    assert sorted(mr.req_to_token_pool.state_pool.matrices) == [r for r, k in enumerate(kinds) if k == "mlstm"]
    streams, got = [], []
    want = ref.forward(cfg, w, prompts["r0"], streams=streams)
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    mr.model.model.capture_streams = got
    out = TraceReplayer(mr).step([dict(id="x", tokens=prompts["r0"], want=list(range(17)))], ["x"])
    mr.model.model.capture_streams = None
    assert su.rel_err(out, want) < TOL and len(got) == len(streams) == len(runs)
    for a, b in zip(got, streams):
        assert float((a.double() - b).abs().max()) < 1e-3, "the stream after every layer run"
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 6), ("r1", 1)], [("r0", 1), ("r1", 3)], [("r0", 9), ("r1", 2)], [("r0", 1)]], TOL)


def test_equal_and_unit_sizes():
    """Sizes that a model may happen to make equal or 1: one head, head and value widths of 1 and 2, a rank of 1, no rotated
    part, no rotation, no stretching, one expert, all experts, a limit that clamps nothing, width equal to the vocabulary, no cap on
    the logits, equal sizes everywhere."""
    layers = [(su.latent(heads=1, dim=2, rot_dim=2, vdim=1, kv_rank=3), su.moe(experts=1, top=1, ff=1, shared=(1, 5.0))),
              (su.mlstm(heads=1, dim=1, vdim=2, gate_cap=1.0), su.dense(1)),
              (su.latent(heads=2, dim=8, rot_dim=0, vdim=8, kv_rank=8, rot_dims=0), su.moe(experts=4, top=4, ff=16, limit=1e9, shared=(16, 1e9))),
              (su.mlstm(heads=16, dim=1, vdim=2), None),
              (su.latent(heads=4, dim=4, rot_dim=4, vdim=4, kv_rank=4, rot_dims=0), su.dense(16)),
              (su.latent(heads=2, dim=4, rot_dim=6, vdim=4, kv_rank=6, rot_dims=2, scaling=False), None)]
    cfg = su.make_config(layers=layers, width=16, vocab=16, softcap=None, loop=(2, 3, 2))
    w = su.make_weights(cfg, seed=11)
    prompts = su.random_prompts(cfg, [14, 5], seed=1)
    mr = su.build_runner(cfg, w, max_total_tokens=32)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 3), ("r1", 1)], [("r0", 1), ("r1", 1)], [("r0", 10), ("r1", 3)]], 1e-4)


def test_attention_only_model_shares_prefixes():
    """Without recurrent layers nothing but cache rows is kept, so the prefix cache serves the design, loops included."""
    from sglang_custom_amd.managers.schedule_batch import Req
    from sglang_custom_amd.managers.scheduler import Scheduler
    from sglang_custom_amd.sampling.sampling_params import SamplingParams

    cfg = su.make_config(layers=[(su.latent(), su.dense()), (su.latent(heads=2, kv_rank=12), None)], loop=(0, 2, 2))
    w = su.make_weights(cfg, seed=2)
    mr = su.build_runner(cfg, w)
    assert mr.req_to_token_pool.state_pool is None
    prompts = su.random_prompts(cfg, [20, 7], seed=3)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 6), ("r1", 7)], [("r0", 13)], [("r0", 1)]], TOL)
    sch = Scheduler(mr, enable_radix_cache=True)
    shared = su.random_prompts(cfg, [12], seed=4)["r0"]
    asks = {"a": shared + [3, 4], "b": shared + [5], "c": shared[:9] + [1, 2, 3]}
    for k, p in asks.items():
        sch.add_request(Req(k, p, SamplingParams(temperature=0, max_new_tokens=4)))
        done = sch.run_until_done()
        assert done[k].output_ids == ref.greedy(cfg, w, p, 4), k


def test_state_is_what_the_next_step_reads(model):
    """Cutting a prompt must hand over exactly what each run keeps: corrupting the matrix, the normaliser, the running maximum or
    the cache rows of ONE run changes the next portion's logits, and every run has its own."""
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    cfg, w = model
    toks = su.random_prompts(cfg, [16], seed=2)["r0"]
    mr = su.build_runner(cfg, w)
    pool, kvp = mr.req_to_token_pool.state_pool, mr.token_to_kv_pool
    assert mr.model_config.layer_runs == [0, 1, 2, 3, 1, 2, 3, 4]
    assert sorted(pool.matrices) == sorted(pool.vectors) == [0, 3, 6]
    assert pool.matrices[0].shape[1:] == (2, 14, 9) and pool.vectors[0].shape[1:] == (2, 1, 15) and pool.matrices[3].data_ptr() != pool.matrices[6].data_ptr()
    assert [None if b is None else b.shape[1] for b in kvp.kv_buffer] == [None, 28, 13, None, 28, 13, None, 45]
    for m in list(pool.matrices.values()) + list(pool.vectors.values()):
        m.fill_(123.0)
    want = ref.forward(cfg, w, toks)
    rp = TraceReplayer(mr)
    assert su.rel_err(rp.step([dict(id="a", tokens=toks[:12], want=list(range(12)))]), want[:12]) < TOL
    bad = []
    for kind, run in [("matrices", r) for r in (0, 3, 6)] + [("vectors", r) for r in (0, 3, 6)] + [("maximum", 6)] + [("rows", r) for r in (1, 2, 4, 5, 7)]:
        rp2 = TraceReplayer(mr)
        rp2.step([dict(id="b", tokens=toks[:12], want=[])])
        s2 = rp2.live["b"].state_slot
        if kind == "rows":
            kvp.kv_buffer[run][mr.req_to_token_pool.req_to_token[rp2.live["b"].req_pool_idx, 4].long()] += 2.0
        elif kind == "maximum":
            pool.vectors[run][s2, ..., -1] += 1.0
        else:
            getattr(pool, kind)[run][s2] += 0.5
        bad.append(su.rel_err(rp2.step([dict(id="b", tokens=toks[12:13], want=[0])], ["b"]), want[12:13]))
    assert min(bad) > 1e-4, bad
    assert su.rel_err(rp.step([dict(id="a", tokens=toks[12:], want=[0, 1, 2, 3])], ["a"]), want[12:]) < TOL
    assert su.pools_are_whole(mr)


@pytest.mark.parametrize("chunk,mixed", [(None, False), (6, False), (6, True)])
def test_greedy_generation_through_the_scheduler(model, chunk, mixed):
    """The package's own entry point: requests queued at the Scheduler, prompts chunked by its policy, decode batches
    (and decode tokens riding prefill batches) formed by it, tokens picked by the Sampler."""
    from sglang_custom_amd.managers.schedule_batch import Req
    from sglang_custom_amd.managers.scheduler import Scheduler
    from sglang_custom_amd.sampling.sampling_params import SamplingParams

    cfg, w = model
    prompts = su.random_prompts(cfg, [11, 3, 7, 15, 1], seed=9)
    mr = su.build_runner(cfg, w, max_total_tokens=96, max_running_requests=3, chunked_prefill_size=chunk, enable_mixed_chunk=mixed)
    sch = Scheduler(mr)
    for k, p in prompts.items():
        sch.add_request(Req(k, p, SamplingParams(temperature=0, max_new_tokens=6)))
    done = sch.run_until_done()
    for k, p in prompts.items():
        assert done[k].output_ids == ref.greedy(cfg, w, p, 6), k
    assert su.pools_are_whole(mr)
    if chunk:
        assert sch.num_prefill_batches > 3


def test_prefix_cache_is_refused_with_recurrent_layers(model):
    from sglang_custom_amd.managers.scheduler import Scheduler

    cfg, w = model
    with pytest.raises(ValueError):
        Scheduler(su.build_runner(cfg, w), enable_radix_cache=True)


def test_configuration_is_read_not_assumed():
    from sglang_custom_amd.configs.model_config import ModelConfig
    from sglang_custom_amd.models.registry import get_model_class

    mc = ModelConfig(su.make_config(), dtype="float32")
    assert mc.architecture == "Silatar" and get_model_class(mc.architecture).__name__ == "SilatarForCausalLM"
    assert mc.layer_runs == [0, 1, 2, 3, 1, 2, 3, 4] and mc.num_hidden_layers == 8
    assert mc.latent_kv == [None, (20, 8), (9, 4), None, (20, 8), (9, 4), None, (33, 12)]
    assert mc.recurrent_layer_shapes == [(2, 14, 9), None, None, (3, 8, 12), None, None, (3, 8, 12), None]
    assert mc.final_logit_softcapping == 12.0 and mc.rms_norm_eps == 1e-5 and mc.v_head_dim == 33
    for path, value in ((("layers", 1, "type"), "something_else"), (("layers", 0, "mlp", "kind"), "other"),
                        (("layers", 1, "mlp", "router", "top"), 6), (("layers", 1, "mixer", "rot", "dims"), 10),
                        (("layers", 1, "mixer", "rot", "dims"), 5), (("layers", 0, "mixer", "gate_cap"), 0.0),
                        (("loop", "stop"), 6), (("loop", "start"), 5), (("loop", "times"), 0)):
        bad = su.make_config()
        node = bad
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = value
        with pytest.raises(ValueError):
            ModelConfig(bad)


# ---- the stand-in ops themselves against the oracle's functions: the same cases the HIP kernels run on the GPU
def test_standins_norms_projections_units():
    import cpu_ops

    cases.check_norm_add_norm(cpu_ops, "cpu", torch.float32)
    cases.check_head_norm_gate(cpu_ops, "cpu", torch.float32)
    cases.check_project_f32(cpu_ops, "cpu", torch.float32)
    cases.check_gelu(cpu_ops, "cpu", torch.float32)
    cases.check_clamped_glu(cpu_ops, "cpu", torch.float32)
    cases.check_moe_layer("cpu", torch.float32, 9)
    cases.check_moe_layer("cpu", torch.float32, 5, top=1, shared=None)


def test_standins_latent_attention():
    import cpu_ops

    cases.check_frequencies()
    cases.check_latent_rows(cpu_ops, "cpu", torch.float32)
    cases.check_latent_rows(cpu_ops, "cpu", torch.float32, rot_dims=0)
    cases.check_latent_attention(cpu_ops, "cpu", torch.float32, T=60, cuts=(17, 2, 40, 1), decode_tail=1)
    cases.check_latent_attention(cpu_ops, "cpu", torch.float32, T=50, H=1, rank=5, dr=6, rot_dims=4, cuts=(25, 25), page=8)
    cases.check_shared_key_part(cpu_ops, "cpu", torch.float32)


def test_standins_matrix_memory():
    import cpu_ops

    cases.check_matrix_memory(cpu_ops, "cpu", torch.float32, cuts=(20, 2, 1, 22))
    cases.check_matrix_memory(cpu_ops, "cpu", torch.float32, cuts=(3, 40, 1, 1), decode_tail=2, dv=70)
    cases.check_matrix_memory_planted(cpu_ops, "cpu", torch.float32)
    cases.check_matrix_memory_batch(cpu_ops, "cpu", torch.float32)
