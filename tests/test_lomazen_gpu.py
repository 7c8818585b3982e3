"""Lomazen on the GPU: every HIP kernel the family added or extended against the plain functions of oracle/lomazen_ref.py
(lomazen_cases.py holds the cases), then the whole engine (ModelRunner, pools, TraceReplayer, Scheduler) in fp32 and bf16
against the whole-sequence oracle, decode steps eager and captured.  Where random numbers would hide a fault -- one key among
hundreds, a key that must not be seen yet, a score far past the cap, two maps that cancel, stale rows in reused slots -- the
inputs are built so that it shows."""
import pytest
import torch

import lomazen_cases as cases
import lomazen_util as lu
from oracle import lomazen_ref as ref

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(autouse=True)
def _product_ops():
    from sglang_custom_amd import ops_backend
    from sglang_custom_amd.distributed import parallel_state

    ops_backend.set_ops_backend(None)      # the HIP library (get_ops() loads it and raises if it is missing)
    parallel_state.init_distributed_environment(1, 0)
    yield


def ops():
    from sglang_custom_amd.ops_backend import get_ops

    return get_ops()


# ---------------------------------------------------------------------------------------------- kernels, one by one
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [48, 33, 1024, 2056, 4096, 5000, 8192, 9000, 16384])
def test_norms_around_a_sublayer_and_the_start_of_a_pass(dtype, D):
    cases.check_norm_add_norm(ops(), DEV, dtype, D=D)
    cases.check_norm_add_norm(ops(), DEV, dtype, D=D, T=1, n_rows=1)
    cases.check_pass_entry(ops(), DEV, dtype, D=D)


@pytest.mark.parametrize("dtype", DTYPES)
def test_pass_entry_layer_and_gated_unit(dtype):
    cases.check_pass_entry_layer(DEV, dtype)
    cases.check_pass_entry_layer(DEV, dtype, T=130, D=72, V=31, times=2)
    cases.check_gated_unit(ops(), DEV, dtype)
    cases.check_gated_unit(ops(), DEV, dtype, ff=37)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,kw", [(1, {}), (9, {}), (70, dict(top=3)), (300, dict(experts=4, top=1)), (40, dict(D=60, ff=20)),
                                  (900, dict(experts=3, top=2, D=128, ff=64)), (2200, dict(experts=3, top=2, D=128, ff=128)),
                                  (33, dict(experts=9, top=8)), (5, dict(experts=1, top=1, D=33, ff=7))])
def test_mixture_of_squared_relu_experts(dtype, T, kw):
    cases.check_moe_layer(DEV, dtype, T, **kw)


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_norms_and_cache_rows(dtype):
    cases.check_frequencies()
    for kw in (dict(), dict(rot=0), dict(interleaved=False), dict(interleaved=False, rot=6), dict(d=16, rot=16, W=24), dict(d=64, rot=64, R=10, S=5, W=440),
               dict(d=56, rot=20, interleaved=False, unit_norm=False, R=12, S=4, W=208), dict(d=128, rot=64, interleaved=False, R=64, S=16, W=2048, T=3),
               dict(d=256, rot=128, R=5, S=5, W=40), dict(d=7, rot=4, W=9, off=3), dict(d=24, rot=20, R=3, S=1, W=8), dict(d=33, rot=32, interleaved=False, W=5),
               dict(d=600, rot=2, R=2, S=1, W=8), dict(d=2, rot=2, R=1, S=1, W=1)):
        cases.check_rotate_write(ops(), DEV, dtype, **kw)


# head counts and widths: whole matrix-core tiles, widths padded to them, widths without 16-byte rows, one head, more heads than a
# tile's columns or rows, widths past what the matrix-core kernels take
SHAPES = [(10, 5, 1, 64, 88), (6, 2, 2, 56, 104), (16, 4, 1, 128, 128), (8, 2, 2, 128, 256), (6, 2, 1, 16, 24), (3, 3, 2, 40, 8), (1, 1, 1, 8, 8), (20, 1, 1, 72, 64),
          (40, 2, 2, 24, 40), (140, 1, 1, 32, 16), (5, 5, 1, 11, 13), (4, 2, 2, 7, 20), (2, 1, 1, 256, 256), (2, 2, 1, 200, 136), (2, 1, 2, 136, 48), (3, 1, 1, 264, 300),
          (6, 3, 2, 64, 128), (12, 12, 1, 88, 120)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,maps,d,dv", SHAPES)
def test_attention(dtype, H, G, maps, d, dv):
    gate = "feature" if maps == 1 else "head"
    for T, cuts, page, singles, decode, splits in ((150, (150,), 1, 0, 0, 1), (150, (17, 2, 100, 30, 1), 1, 1, 0, 1), (140, (130,) + (1,) * 10, 16, 0, 10, 3),
                                                   (100, (50, 2, 47, 1), 6, 0, 1, 1), (70, (64, 2, 2, 1, 1), 64, 2, 0, 2), (3, (1, 1, 1), 1, 0, 3, 1)):
        cases.check_attention(ops(), DEV, dtype, H=H, G=G, maps=maps, d=d, dv=dv, T=T, cuts=cuts, cap=4.0 if maps == 1 and T == 150 else 0.0,
                              gate=gate if T != 70 else None, page=page, singles_tail=singles, decode_tail=decode, splits=splits)
    cases.check_attention(ops(), DEV, dtype, H=H, G=G, maps=maps, d=d, dv=dv, T=40, cuts=(33, 6, 1), gate="head" if maps == 1 else "feature", decode_tail=1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(maps=2), dict(H=4, G=4, d=64, dv=32, page=32), dict(H=2, G=1, maps=2, d=56, dv=104, page=16)])
def test_attention_one_key_among_hundreds(dtype, kw):
    cases.check_attention_planted(ops(), DEV, dtype, **kw)


@pytest.mark.parametrize("dtype", DTYPES)
def test_score_cap_difference_batches_rotation(dtype):
    cases.check_score_cap(ops(), DEV, dtype)
    cases.check_score_cap(ops(), DEV, dtype, H=3, G=1, d=70, dv=9)
    cases.check_difference(ops(), DEV, dtype)
    cases.check_difference(ops(), DEV, dtype, H=6, G=2, d=56, dv=104)
    for maps in (1, 2):
        cases.check_batch_of_unequal(ops(), DEV, dtype, maps=maps)
        cases.check_batch_of_unequal(ops(), DEV, dtype, maps=maps, H=8, G=8, d=64, dv=128)
    cases.check_rotation_decides(ops(), DEV, dtype)
    cases.check_rotation_decides(ops(), DEV, dtype, d=64)


def test_what_the_launch_refuses():
    """Shapes the kernels do not take come back as errors from the host side, before anything is launched."""
    from sglang_custom_amd._lib import Mi355Error

    with pytest.raises(Mi355Error):
        cases.check_attention(ops(), DEV, torch.bfloat16, H=2, G=1, d=600, dv=16, T=5, cuts=(5,))
    with pytest.raises(Mi355Error):
        cases.check_attention(ops(), DEV, torch.float32, H=2, G=1, d=16, dv=520, T=5, cuts=(5,))


# ---------------------------------------------------------------------------------------------- the engine
CASES = [("float32", 3e-5), ("bfloat16", 6e-2)]


def _model(dtype, **kw):
    """fp32: the CPU tests' small model.  bf16: the same order of layers with larger widths, every token using every expert of
    its mixtures (see lomazen_util.default_layers)."""
    if dtype == "float32":
        cfg = lu.make_config(**kw)
        return cfg, lu.make_weights(cfg, seed=3)
    layers = [(lu.attention_2(heads=4, kv_heads=4, dim=24, vdim=40), lu.dense(96)), (lu.attention(heads=6, kv_heads=2, dim=32, vdim=24), lu.moe(top=5, ff=48)),
              (lu.attention_2(heads=4, kv_heads=2, dim=16, vdim=32, rot_dims=0), None),
              (lu.attention(heads=2, kv_heads=1, dim=40, vdim=24, softcap=None, base=50.0, rot_dims=16, scaling=False), lu.moe(experts=3, top=3, ff=40)),
              (lu.attention(heads=5, kv_heads=5, dim=24, vdim=48, softcap=1.5), lu.dense(64))]
    cfg = lu.make_config(layers=layers, width=96, vocab=101, **kw)
    return cfg, lu.make_weights(cfg, seed=3)


@pytest.mark.parametrize("dtype,tol", CASES)
@pytest.mark.parametrize("kind", ["attention", "attention_2"])
def test_each_mixer_alone(dtype, tol, kind):
    mixer = dict(attention=lu.attention(dim=16, vdim=16), attention_2=lu.attention_2(dim=16, vdim=32))[kind]
    cfg = lu.make_config(layers=[(mixer, None)], loop=(0, 1, 2))
    w = lu.make_weights(cfg, seed=1)
    prompts = lu.random_prompts(cfg, [90])
    mr = lu.build_runner(cfg, w, dtype=dtype, device=DEV)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 90)]], tol)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 37)], [("r0", 2)], [("r0", 40)]] + [[("r0", 1)] for _ in range(11)], tol)
    assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("dtype,tol", CASES)
@pytest.mark.parametrize("graph", [True, False])
def test_portions_and_batches(dtype, tol, graph):
    cfg, w = _model(dtype)
    prompts = lu.random_prompts(cfg, [27, 9, 1, 12, 30, 6], seed=7)
    sched = [[("r0", 5), ("r1", 2)], [("r0", 1), ("r1", 7), ("r2", 1)], [("r0", 4), ("r3", 3)], [("r3", 1)],
             [("r0", 1), ("r3", 1)], [("r0", 16), ("r3", 7), ("r4", 2)], [("r4", 1), ("r5", 1)], [("r4", 1), ("r5", 1)],
             [("r4", 19), ("r5", 4)], [("r4", 1)], [("r4", 6)]]
    want = {k: ref.forward(cfg, w, p) for k, p in prompts.items()}
    for page in (1, 6):
        mr = lu.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=72, max_running_requests=3, page_size=page, disable_cuda_graph=not graph,
                             cuda_graph_bs=[2, 4])
        assert (mr.graph_runner is not None) == graph
        for _ in range(2):       # the second time over used slots
            lu.replay_and_compare(mr, cfg, w, prompts, sched, tol, want_all=want)
            assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("dtype,tol", CASES)
def test_long_decode(dtype, tol):
    """Other sizes than the small default's: heads of 64 and 128 on the matrix cores in bf16, two maps over 128-wide values, a loop around
    everything but the ends; a 170-token decode on captured steps, pages of 16, key ranges in the decode steps."""
    layers = [(lu.attention(heads=4, kv_heads=2, dim=64, vdim=32, scale=0.2, softcap=8.0, base=10000.0, rot_dims=32,
                            scaling=dict(factor=8.0, low=1.0, high=4.0, original=64)), lu.dense(96)),
              (lu.attention_2(heads=4, kv_heads=2, dim=64, vdim=128, scale=0.1, rot_dims=32), lu.moe(experts=4, top=4, ff=64)),
              (lu.attention(heads=8, kv_heads=8, dim=128, vdim=72, scale=0.2, softcap=None), None),
              (lu.attention_2(heads=2, kv_heads=1, dim=32, vdim=96, diff=0.5), lu.dense(64))]
    cfg = lu.make_config(layers=layers, width=128, vocab=211, loop=(1, 3, 3), logit_scale=0.7, eps=1e-6)
    w = lu.make_weights(cfg, seed=5)
    mr = lu.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=512, max_running_requests=4, page_size=16, cuda_graph_bs=[1, 4])
    assert mr.graph_runner is not None
    p = lu.random_prompts(cfg, [300, 90, 3, 60], seed=8)
    want = {k: ref.forward(cfg, w, x) for k, x in p.items()}
    lu.replay_and_compare(mr, cfg, w, {"r0": p["r0"]}, [[("r0", 300)]], tol, want_all=want)
    lu.replay_and_compare(mr, cfg, w, {"r0": p["r0"]}, [[("r0", 130)]] + [[("r0", 1)]] * 170, tol, want_all=want)
    sched = [[("r0", 64), ("r1", 64), ("r2", 2)], [("r0", 29), ("r1", 2), ("r2", 1), ("r3", 16)], [("r0", 168), ("r1", 3), ("r3", 3)],
             [("r0", 2), ("r1", 16), ("r3", 35)], [("r0", 30), ("r1", 4), ("r3", 5)]] + [[("r0", 1), ("r1", 1), ("r3", 1)]] + [[("r0", 1)]] * 6
    for _ in range(2):
        lu.replay_and_compare(mr, cfg, w, p, sched, tol, want_all=want)
        assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("dtype,tol", CASES)
def test_sizes_that_are_multiples_of_nothing(dtype, tol):
    """Width 100, vocabulary 77, heads of 21 / 13 / 37, odd feed-forward widths, pages of 5: no 16-byte row anywhere in 16 bits, no
    whole tile."""
    layers = [(lu.attention(heads=3, kv_heads=1, dim=21, vdim=13, base=77.0, rot_dims=6), lu.moe(experts=3, top=3, ff=51)),
              (lu.attention_2(heads=3, kv_heads=3, dim=21, vdim=37, rot_dims=14), lu.dense(71)),
              (lu.attention(heads=10, kv_heads=5, dim=11, vdim=23, rot_dims=10, softcap=2.0), None)]
    cfg = lu.make_config(layers=layers, width=100, vocab=77, loop=(0, 2, 2), logit_scale=0.9)
    w = lu.make_weights(cfg, seed=21)
    mr = lu.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=200, max_running_requests=3, page_size=5)
    p = lu.random_prompts(cfg, [83, 41, 6], seed=4)
    want = {k: ref.forward(cfg, w, x) for k, x in p.items()}
    sched = [[("r0", 33), ("r1", 2)], [("r0", 2), ("r1", 30), ("r2", 1)], [("r0", 40), ("r1", 1), ("r2", 5)], [("r0", 1), ("r1", 1)],
             [("r0", 1), ("r1", 7)]] + [[("r0", 1)]] * 6
    for _ in range(2):
        lu.replay_and_compare(mr, cfg, w, p, sched, tol, want_all=want)
        assert lu.pools_are_whole(mr)


def test_equal_and_unit_sizes():
    """The sizes of the CPU test of this name, in fp32: norms over one or two features amplify 16-bit rounding without bound."""
    layers = [(lu.attention(heads=1, kv_heads=1, dim=2, vdim=1), lu.moe(experts=1, top=1, ff=1)),
              (lu.attention_2(heads=1, kv_heads=1, dim=1, vdim=2, rot_dims=0), lu.dense(1)),
              (lu.attention(heads=8, kv_heads=1, dim=8, vdim=8, softcap=None, rot_dims=0), lu.moe(experts=4, top=4, ff=16)),
              (lu.attention_2(heads=16, kv_heads=16, dim=2, vdim=2, rot_dims=2, diff=0.0), None),
              (lu.attention(heads=4, kv_heads=4, dim=4, vdim=4, scaling=False), lu.dense(16)),
              (lu.attention_2(heads=2, kv_heads=2, dim=4, vdim=4, rot_dims=4), None)]
    cfg = lu.make_config(layers=layers, width=16, vocab=16, logit_scale=None, loop=(2, 3, 2))
    w = lu.make_weights(cfg, seed=11)
    prompts = lu.random_prompts(cfg, [14, 5], seed=1)
    mr = lu.build_runner(cfg, w, dtype="float32", device=DEV, max_total_tokens=32)
    lu.replay_and_compare(mr, cfg, w, prompts, [[("r0", 3), ("r1", 1)], [("r0", 1), ("r1", 1)], [("r0", 10), ("r1", 3)]], 1e-4)
    assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_logits_do_not_depend_on_cuts_or_company(dtype):
    """One request whole, in portions, and beside others on other slots: the same logits up to the rounding of differently
    shaped products."""
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    cfg, w = _model(dtype)
    p = lu.random_prompts(cfg, [40, 25], seed=13)
    mr = lu.build_runner(cfg, w, dtype=dtype, device=DEV)
    rp = TraceReplayer(mr)
    whole = rp.step([dict(id="a", tokens=p["r0"], want=list(range(40)))], ["a"]).double().cpu()
    parts = []
    for lo, hi in ((0, 3), (3, 5), (5, 30), (30, 31), (31, 32), (32, 40)):
        parts.append(rp.step([dict(id="z", tokens=p["r1"][lo:min(hi, 25)] or [1], want=[]), dict(id="b", tokens=p["r0"][lo:hi], want=list(range(hi - lo)))]))
    rp.finish("b")
    rp.finish("z")
    parts = torch.cat(parts).double().cpu()
    assert float(lu.row_errors(parts, whole).max()) < (2e-5 if dtype == "float32" else 8e-2)
    assert lu.pools_are_whole(mr)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_steps_match_eager_steps(dtype):
    """The same decode steps eager and captured, several replays with eager work between them, batch sizes that are padded: equal up to
    the number of key ranges a step is cut into."""
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    cfg, w = _model(dtype)
    p = lu.random_prompts(cfg, [30, 22, 9], seed=17)
    outs = []
    for graph in (False, True):
        mr = lu.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=160, disable_cuda_graph=not graph, cuda_graph_bs=[2, 4])
        rp, rows = TraceReplayer(mr), []
        rp.step([dict(id=k, tokens=p[k][:3], want=[]) for k in p])
        for i in range(3, 30):
            live = [k for k in p if i < len(p[k])]
            rows.append(rp.step([dict(id=k, tokens=p[k][i:i + 1], want=[0]) for k in live]).cpu())
            if i % 7 == 0:
                rp.step([dict(id=f"other{i}", tokens=p["r0"][:i], want=[0])], [f"other{i}"])     # eager work on other slots
        for k in p:
            rp.finish(k)
        assert lu.pools_are_whole(mr)
        outs.append(torch.cat(rows).double())
    assert float(lu.row_errors(outs[1], outs[0]).max()) < (2e-5 if dtype == "float32" else 6e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_scheduler(dtype):
    """The engine's own entry point, prompts chunked and decode tokens riding prefill batches.  fp32 must give the
    oracle's tokens; bf16 must give the same tokens whether a prompt is chunked or not, up to a near-tie."""
    from sglang_custom_amd.managers.schedule_batch import Req
    from sglang_custom_amd.managers.scheduler import Scheduler
    from sglang_custom_amd.sampling.sampling_params import SamplingParams

    cfg, w = _model(dtype)
    prompts = lu.random_prompts(cfg, [11, 3, 7, 15, 1], seed=9)
    outs = []
    for chunk, mixed in ((None, False), (6, True)):
        mr = lu.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=96, max_running_requests=3,
                             chunked_prefill_size=chunk, enable_mixed_chunk=mixed)
        sch = Scheduler(mr)
        for k, p in prompts.items():
            sch.add_request(Req(k, p, SamplingParams(temperature=0, max_new_tokens=6)))
        done = sch.run_until_done()
        outs.append({k: done[k].output_ids for k in prompts})
        assert lu.pools_are_whole(mr)
    if dtype == "float32":
        for k, p in prompts.items():
            assert outs[0][k] == outs[1][k] == ref.greedy(cfg, w, p, 6), k
    else:
        assert sum(outs[0][k] == outs[1][k] for k in prompts) >= len(prompts) - 1


@pytest.mark.parametrize("dtype,tol", CASES)
def test_command_line_replay_of_a_model_folder(tmp_path, dtype, tol):
    """bin/trace_run as a user starts it: a model folder on disk, steps on standard input, logits in files; four live
    requests at most, a pool that the requests' total would not fit into."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np

    from test_seturax_gpu import _write_model_folder

    layers = [(lu.attention_2(heads=2, kv_heads=1, dim=32, vdim=24), lu.dense(48)), (lu.attention(heads=5, kv_heads=5, dim=16, vdim=24), lu.moe(experts=3, top=3, ff=40)),
              (lu.attention(heads=6, kv_heads=2, dim=24, vdim=32, softcap=2.0), None)]
    cfg = lu.make_config(layers=layers, width=64, vocab=83, loop=(1, 3, 2), logit_scale=0.8)
    w = lu.make_weights(cfg, seed=17)
    _write_model_folder(tmp_path, cfg, w)
    prompts = lu.random_prompts(cfg, [70, 33, 1, 64, 40], seed=6)
    sched = [[("r0", 40), ("r1", 2)], [("r0", 1), ("r1", 30), ("r2", 1), ("r3", 7)], [("r0", 29), ("r1", 1), ("r3", 57)],
             [("r4", 2)], [("r4", 1)], [("r4", 37)]]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    lines, want, at = [], [], {k: 0 for k in prompts}
    full = {k: ref.forward(cfg, w, p) for k, p in prompts.items()}
    for n, step in enumerate(sched):
        entries, rows, end = [], [], []
        for name, cnt in step:
            lo, hi = at[name], at[name] + cnt
            asked = list(range(0, cnt, 3)) + ([cnt - 1] if (cnt - 1) % 3 else [])
            entries.append({"id": name, "tokens": prompts[name][lo:hi], "want": asked})
            rows.append(full[name][lo:hi][asked])
            at[name] = hi
            if hi == len(prompts[name]):
                end.append(name)
        lines.append(json.dumps({"step": n, "entries": entries, "end": end}))
        want.append(torch.cat(rows))
    lines.append(json.dumps({"step": len(sched), "entries": [], "end": []}))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "192"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=300, cwd=root)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.split("\n") if x.startswith("done")] == [f"done {n}" for n in range(len(sched) + 1)]
    errors = []
    for n, expect in enumerate(want):
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"]).copy())
        assert got.shape == expect.shape
        errors.append(lu.row_errors(got, expect))
    assert lu.within(torch.cat(errors), tol, dtype != "float32"), [float(e.max()) for e in errors]
    assert not (out / f"{len(sched)}.f32").exists()
