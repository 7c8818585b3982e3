"""Silatar on the GPU: every HIP kernel the family added or extended against the plain functions of oracle/silatar_ref.py
(silatar_cases.py holds the cases), then the whole engine (ModelRunner, pools, TraceReplayer, Scheduler) in fp32 and bf16
against the whole-sequence oracle.  Where random numbers would hide a fault -- one key among hundreds, a key that must not be
seen yet, a value written hundreds of tokens back, the start of the running maximum, a factor on an input instead of an output,
stale rows and stale state in reused slots -- the inputs are built so that it shows."""
import pytest
import torch

import silatar_cases as cases
import silatar_util as su
from oracle import silatar_ref as ref

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
def test_norms_around_a_sublayer(dtype, D):
    cases.check_norm_add_norm(ops(), DEV, dtype, D=D)
    cases.check_norm_add_norm(ops(), DEV, dtype, D=D, T=1, n_rows=1)


@pytest.mark.parametrize("dtype", DTYPES)
def test_head_norm_with_a_weight_per_head(dtype):
    cases.check_head_norm_gate(ops(), DEV, dtype)
    cases.check_head_norm_gate(ops(), DEV, dtype, H=1, dv=130)
    cases.check_head_norm_gate(ops(), DEV, dtype, T=70, H=8, dv=64)


@pytest.mark.parametrize("dtype", DTYPES)
def test_small_projections_and_units(dtype):
    cases.check_project_f32(ops(), DEV, dtype)
    cases.check_gelu(ops(), DEV, dtype)
    for ff in (24, 33, 8, 2600):
        cases.check_clamped_glu(ops(), DEV, dtype, ff=ff)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,kw", [(1, {}), (9, {}), (70, dict(top=3)), (300, dict(experts=4, top=1)), (40, dict(D=60, ff=20, shared=None)),
                                  (900, dict(experts=3, top=2, D=128, ff=64)), (2200, dict(experts=3, top=2, D=128, ff=128)),
                                  (33, dict(experts=9, top=8, limit=0.3))])
def test_mixture_with_weights_on_the_inputs(dtype, T, kw):
    cases.check_moe_layer(DEV, dtype, T, **kw)


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_rows(dtype):
    cases.check_frequencies()
    cases.check_latent_rows(ops(), DEV, dtype)
    cases.check_latent_rows(ops(), DEV, dtype, rot_dims=0)
    cases.check_latent_rows(ops(), DEV, dtype, T=3, q_cols=0, rank=512, dr=64, rot_dims=64)
    cases.check_latent_rows(ops(), DEV, dtype, rank=7, dr=2, rot_dims=2)


# head counts and widths: whole matrix-core tiles, widths that are multiples of nothing, one head, more heads than a workgroup's
# rows, a rank too wide for the matrix-core kernel
SHAPES = [(4, 32, 16, 16), (6, 96, 16, 16), (1, 20, 6, 4), (16, 512, 64, 64), (3, 130, 10, 10), (40, 64, 8, 0), (70, 32, 16, 8), (2, 520, 8, 8), (5, 16, 0, 0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,rank,dr,rot", SHAPES)
def test_latent_attention(dtype, H, rank, dr, rot):
    for T, cuts, page, tail, splits in ((150, (150,), 1, 0, 1), (150, (17, 2, 100, 30, 1), 1, 1, 1), (140, (130,) + (1,) * 10, 16, 10, 3),
                                        (100, (50, 2, 47, 1), 6, 1, 1), (70, (64, 2, 2, 1, 1), 64, 2, 2)):
        s = splits if rank <= 512 else 1
        cases.check_latent_attention(ops(), DEV, dtype, H=H, rank=rank, dr=dr, rot_dims=rot, T=T, cuts=cuts, page=page, decode_tail=tail, splits=s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_attention_one_key_among_hundreds(dtype):
    cases.check_latent_attention_planted(ops(), DEV, dtype)
    cases.check_latent_attention_planted(ops(), DEV, dtype, H=20, rank=48, dr=8, page=32)
    cases.check_shared_key_part(ops(), DEV, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv", [(3, 12, 20), (2, 32, 32), (4, 64, 48), (2, 128, 128), (6, 1, 1), (3, 40, 70), (1, 200, 33), (2, 256, 64)])
def test_matrix_memory(dtype, H, dk, dv):
    whole = None
    for cuts, tail in (((45,), 0), ((20, 2, 1, 22), 0), ((3, 40, 1, 1), 2), ((1,) * 45, 45), ((17, 16, 12), 0)):
        got = cases.check_matrix_memory(ops(), DEV, dtype, H=H, dk=dk, dv=dv, cuts=cuts, decode_tail=tail)
        whole = got if whole is None else whole
        assert torch.equal(got, whole), "the same bits however the sequence is cut"
    cases.check_matrix_memory(ops(), DEV, dtype, H=H, dk=dk, dv=dv, cuts=(45,), cap=40.0, gate_std=12.0)


@pytest.mark.parametrize("dtype", DTYPES)
def test_matrix_memory_far_writes_floor_and_batches(dtype):
    cases.check_matrix_memory_planted(ops(), DEV, dtype)
    cases.check_matrix_memory_batch(ops(), DEV, dtype)
    cases.check_matrix_memory_batch(ops(), DEV, dtype, H=3, dk=96, dv=130)


# ---------------------------------------------------------------------------------------------- the engine
CASES = [("float32", 3e-5), ("bfloat16", 6e-2)]


def _model(dtype, **kw):
    """fp32: the CPU tests' small model.  bf16: the same order of layers with larger widths, every token using every expert of
    its mixtures (see silatar_util.default_layers)."""
    if dtype == "float32":
        cfg = su.make_config(**kw)
        return cfg, su.make_weights(cfg, seed=3)
    layers = [(su.mlstm(heads=2, dim=24, vdim=40), su.dense(96)), (su.latent(heads=4, dim=24, rot_dim=16, vdim=24, kv_rank=48), su.moe(top=5, ff=48)),
              (su.latent(heads=3, dim=16, rot_dim=8, vdim=32, kv_rank=40, scaling=False), None),
              (su.mlstm(heads=3, dim=32, vdim=24, gate_cap=15.0), su.moe(experts=3, top=3, ff=40, shared=None)),
              (su.latent(heads=1, dim=40, rot_dim=24, vdim=48, kv_rank=56, rot_dims=12, base=50.0), su.dense(64))]
    cfg = su.make_config(layers=layers, width=96, vocab=101, **kw)
    return cfg, su.make_weights(cfg, seed=3)


@pytest.mark.parametrize("dtype,tol", CASES)
@pytest.mark.parametrize("kind", ["latent_attention", "mlstm"])
def test_each_mixer_alone(dtype, tol, kind):
    mixer = dict(latent_attention=su.latent(kv_rank=32), mlstm=su.mlstm(dim=24, vdim=24))[kind]
    cfg = su.make_config(layers=[(mixer, None)], loop=(0, 1, 2))
    w = su.make_weights(cfg, seed=1)
    prompts = su.random_prompts(cfg, [90])
    mr = su.build_runner(cfg, w, dtype=dtype, device=DEV)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 90)]], tol)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 37)], [("r0", 2)], [("r0", 40)]] + [[("r0", 1)] for _ in range(11)], tol)
    assert su.pools_are_whole(mr)


@pytest.mark.parametrize("dtype,tol", CASES)
def test_portions_and_batches(dtype, tol):
    cfg, w = _model(dtype)
    prompts = su.random_prompts(cfg, [27, 9, 1, 12, 30, 6], seed=7)
    sched = [[("r0", 5), ("r1", 2)], [("r0", 1), ("r1", 7), ("r2", 1)], [("r0", 4), ("r3", 3)], [("r3", 1)],
             [("r0", 1), ("r3", 1)], [("r0", 16), ("r3", 7), ("r4", 2)], [("r4", 1), ("r5", 1)], [("r4", 1), ("r5", 1)],
             [("r4", 19), ("r5", 4)], [("r4", 1)], [("r4", 6)]]
    want = {k: ref.forward(cfg, w, p) for k, p in prompts.items()}
    for page in (1, 6):
        mr = su.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=72, max_running_requests=3, page_size=page)
        for _ in range(2):       # the second time over used slots and state
            su.replay_and_compare(mr, cfg, w, prompts, sched, tol, want_all=want)
            assert su.pools_are_whole(mr)


@pytest.mark.parametrize("dtype,tol", CASES)
def test_long_decode(dtype, tol):
    """Other sizes than the small default's: heads of 64 / 32 on the matrix cores in bf16, key widths past 64 in the matrix
    memory, a loop around everything but the ends; a 170-token decode, pages of 16, key ranges in the decode steps."""
    layers = [(su.latent(heads=4, dim=64, rot_dim=32, vdim=32, kv_rank=128, scale=0.12, base=10000.0,
                         scaling=dict(factor=8.0, original=64, fast=8.0, slow=1.0)), su.dense(96)),
              (su.mlstm(heads=4, dim=72, vdim=40, gate_cap=10.0), su.moe(experts=4, top=4, ff=64, limit=1.5, shared=(32, 0.6))),
              (su.latent(heads=8, dim=24, rot_dim=16, vdim=24, kv_rank=64, scale=0.2), None),
              (su.mlstm(heads=2, dim=32, vdim=96), su.dense(64))]
    cfg = su.make_config(layers=layers, width=128, vocab=211, loop=(1, 3, 3), softcap=20.0, eps=1e-6)
    w = su.make_weights(cfg, seed=5)
    mr = su.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=512, max_running_requests=4, page_size=16)
    p = su.random_prompts(cfg, [300, 90, 3, 60], seed=8)
    want = {k: ref.forward(cfg, w, x) for k, x in p.items()}
    su.replay_and_compare(mr, cfg, w, {"r0": p["r0"]}, [[("r0", 300)]], tol, want_all=want)
    su.replay_and_compare(mr, cfg, w, {"r0": p["r0"]}, [[("r0", 130)]] + [[("r0", 1)]] * 170, tol, want_all=want)
    sched = [[("r0", 64), ("r1", 64), ("r2", 2)], [("r0", 29), ("r1", 2), ("r2", 1), ("r3", 16)], [("r0", 168), ("r1", 3), ("r3", 3)],
             [("r0", 2), ("r1", 16), ("r3", 35)], [("r0", 30), ("r1", 4), ("r3", 5)]] + [[("r0", 1), ("r1", 1), ("r3", 1)]] + [[("r0", 1)]] * 6
    for _ in range(2):
        su.replay_and_compare(mr, cfg, w, p, sched, tol, want_all=want)
        assert su.pools_are_whole(mr)


@pytest.mark.parametrize("dtype,tol", CASES)
def test_sizes_that_are_multiples_of_nothing(dtype, tol):
    """Width 100, vocabulary 77, heads of 21 / 13 / 37, ranks of 29 and 51, odd feed-forward widths, pages of 5: no 16-byte row
    anywhere in 16 bits, no whole tile."""
    layers = [(su.latent(heads=3, dim=21, rot_dim=10, vdim=13, kv_rank=29, rot_dims=6, base=77.0), su.moe(experts=3, top=3, ff=51, shared=(27, 0.9))),
              (su.mlstm(heads=3, dim=21, vdim=37, gate_cap=7.0), su.dense(71)),
              (su.latent(heads=5, dim=11, rot_dim=6, vdim=23, kv_rank=51, scale=0.3), None)]
    cfg = su.make_config(layers=layers, width=100, vocab=77, loop=(0, 2, 2), softcap=9.0)
    w = su.make_weights(cfg, seed=21)
    mr = su.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=200, max_running_requests=3, page_size=5)
    p = su.random_prompts(cfg, [83, 41, 6], seed=4)
    want = {k: ref.forward(cfg, w, x) for k, x in p.items()}
    sched = [[("r0", 33), ("r1", 2)], [("r0", 2), ("r1", 30), ("r2", 1)], [("r0", 40), ("r1", 1), ("r2", 5)], [("r0", 1), ("r1", 1)],
             [("r0", 1), ("r1", 7)]] + [[("r0", 1)]] * 6
    for _ in range(2):
        su.replay_and_compare(mr, cfg, w, p, sched, tol, want_all=want)
        assert su.pools_are_whole(mr)


def test_equal_and_unit_sizes():
    """The sizes of the CPU test of this name, in fp32: norms over one or two features amplify 16-bit rounding without bound."""
    layers = [(su.latent(heads=1, dim=2, rot_dim=2, vdim=1, kv_rank=3), su.moe(experts=1, top=1, ff=1, shared=(1, 5.0))),
              (su.mlstm(heads=1, dim=1, vdim=2, gate_cap=1.0), su.dense(1)),
              (su.latent(heads=2, dim=8, rot_dim=0, vdim=8, kv_rank=8, rot_dims=0), su.moe(experts=4, top=4, ff=16, limit=1e9, shared=(16, 1e9))),
              (su.mlstm(heads=16, dim=1, vdim=2), None),
              (su.latent(heads=4, dim=4, rot_dim=4, vdim=4, kv_rank=4, rot_dims=0), su.dense(16)),
              (su.latent(heads=2, dim=4, rot_dim=6, vdim=4, kv_rank=6, rot_dims=2, scaling=False), None)]
    cfg = su.make_config(layers=layers, width=16, vocab=16, softcap=None, loop=(2, 3, 2))
    w = su.make_weights(cfg, seed=11)
    prompts = su.random_prompts(cfg, [14, 5], seed=1)
    mr = su.build_runner(cfg, w, dtype="float32", device=DEV, max_total_tokens=32)
    su.replay_and_compare(mr, cfg, w, prompts, [[("r0", 3), ("r1", 1)], [("r0", 1), ("r1", 1)], [("r0", 10), ("r1", 3)]], 1e-4)
    assert su.pools_are_whole(mr)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_logits_do_not_depend_on_cuts_or_company(dtype):
    """One request whole, in portions, and beside others on other slots: the same logits up to the rounding of differently
    shaped products."""
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    cfg, w = _model(dtype)
    p = su.random_prompts(cfg, [40, 25], seed=13)
    mr = su.build_runner(cfg, w, dtype=dtype, device=DEV)
    rp = TraceReplayer(mr)
    whole = rp.step([dict(id="a", tokens=p["r0"], want=list(range(40)))], ["a"]).double().cpu()
    parts = []
    for lo, hi in ((0, 3), (3, 5), (5, 30), (30, 31), (31, 32), (32, 40)):
        parts.append(rp.step([dict(id="z", tokens=p["r1"][lo:min(hi, 25)] or [1], want=[]), dict(id="b", tokens=p["r0"][lo:hi], want=list(range(hi - lo)))]))
    rp.finish("b")
    rp.finish("z")
    parts = torch.cat(parts).double().cpu()
    assert float(su.row_errors(parts, whole).max()) < (2e-5 if dtype == "float32" else 8e-2)
    assert su.pools_are_whole(mr)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_scheduler(dtype):
    """The engine's own entry point, prompts chunked and decode tokens riding prefill batches.  fp32 must give the
    oracle's tokens; bf16 must give the same tokens whether a prompt is chunked or not, up to a near-tie."""
    from sglang_custom_amd.managers.schedule_batch import Req
    from sglang_custom_amd.managers.scheduler import Scheduler
    from sglang_custom_amd.sampling.sampling_params import SamplingParams

    cfg, w = _model(dtype)
    prompts = su.random_prompts(cfg, [11, 3, 7, 15, 1], seed=9)
    outs = []
    for chunk, mixed in ((None, False), (6, True)):
        mr = su.build_runner(cfg, w, dtype=dtype, device=DEV, max_total_tokens=96, max_running_requests=3,
                             chunked_prefill_size=chunk, enable_mixed_chunk=mixed)
        sch = Scheduler(mr)
        for k, p in prompts.items():
            sch.add_request(Req(k, p, SamplingParams(temperature=0, max_new_tokens=6)))
        done = sch.run_until_done()
        outs.append({k: done[k].output_ids for k in prompts})
        assert su.pools_are_whole(mr)
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

    layers = [(su.mlstm(heads=2, dim=32, vdim=24), su.dense(48)), (su.latent(heads=5, dim=16, rot_dim=16, vdim=24, kv_rank=40), su.moe(experts=3, top=3, ff=40)),
              (su.mlstm(heads=3, dim=16, vdim=32, gate_cap=9.0), None)]
    cfg = su.make_config(layers=layers, width=64, vocab=83, loop=(1, 3, 2), softcap=8.0)
    w = su.make_weights(cfg, seed=17)
    _write_model_folder(tmp_path, cfg, w)
    prompts = su.random_prompts(cfg, [70, 33, 1, 64, 40], seed=6)
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
        errors.append(su.row_errors(got, expect))
    assert su.within(torch.cat(errors), tol, dtype != "float32"), [float(e.max()) for e in errors]
    assert not (out / f"{len(sched)}.f32").exists()
