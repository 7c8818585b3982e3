"""Shared pieces of the Lomazen tests: small random models in checkpoint form and the replay of a schedule with every
logit compared against the whole-sequence oracle (oracle/lomazen_ref.py)."""
import torch

from fudonex_util import pools_are_whole  # noqa: F401  (generic helper)
from gatarax_util import row_errors, within
from oracle import lomazen_ref as ref
from seturax_util import build_runner, random_prompts, rel_err  # noqa: F401  (generic helpers)


def attention(heads=6, kv_heads=2, dim=12, vdim=10, scale=0.4, softcap=5.0, base=500.0, rot_dims=None, scaling=True):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if softcap:
        m["softcap"] = softcap
    dims = dim if rot_dims is None else rot_dims
    if dims:
        m["rot"] = dict(base=base, dims=dims)
        if scaling:
            m["rot"]["scaling"] = dict(factor=4.0, low=0.5, high=3.0, original=24) if scaling is True else dict(scaling)
    return dict(type="attention", mixer=m)


def attention_2(heads=3, kv_heads=3, dim=10, vdim=14, scale=0.3, diff=0.3, base=900.0, rot_dims=6):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, diff=diff)
    if rot_dims:
        m["rot"] = dict(base=base, dims=rot_dims)
    return dict(type="attention_2", mixer=m)


def dense(ff=40):
    return dict(kind="dense", ff=ff)


def moe(experts=5, top=2, ff=18):
    return dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))


def default_layers(every_expert=False):
    """Both mixers, both feed-forwards and none, unlike sizes throughout.  every_expert: each token uses all experts of its
    mixtures, so that a 16-bit run and a float64 oracle cannot part ways over a close call between two scores (the weights
    still differ from token to token)."""
    a, b = (moe(top=5), moe(experts=3, top=3)) if every_expert else (moe(), moe(experts=7, top=1))
    return [(attention_2(), dense()), (attention(), a), (attention_2(heads=4, kv_heads=2, dim=6, vdim=16, diff=0.55, rot_dims=0), None),
            (attention(heads=2, kv_heads=1, dim=20, vdim=6, softcap=None, base=50.0, rot_dims=8, scaling=False), b),
            (attention(heads=5, kv_heads=5, dim=8, vdim=12, softcap=1.5), dense(24))]


def make_config(layers=None, width=48, vocab=53, loop=(1, 4, 2), logit_scale=1.5, eps=1e-5):
    """layers: list of (mixer spec, mlp spec or None)."""
    if layers is None:
        layers = default_layers()
        assert loop is None or loop[1] <= len(layers)
    cfg = dict(architecture="Lomazen", vocab=vocab, width=width, norm=dict(eps=eps),
               layers=[dict(type=m["type"], mixer={k: (dict(v) if isinstance(v, dict) else v) for k, v in m["mixer"].items()}, mlp=f)
                       for m, f in layers])
    if loop:
        cfg["loop"] = dict(start=loop[0], stop=loop[1], times=loop[2])
    if logit_scale is not None:
        cfg["logit_scale"] = logit_scale
    return cfg


def make_weights(cfg, seed=0):
    """Checkpoint-named tensors with bf16-representable values, so that a bf16 and an fp32 run read the same numbers."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, std=1.0, mean=0.0):
        return (mean + std * torch.randn(*shape, generator=g)).to(torch.bfloat16)

    def norm(n):
        return rnd(n, std=0.1, mean=1.0)

    w = {"embed": rnd(V, D), "final.norm": norm(D)}
    if cfg.get("loop"):
        w["loop.in"] = rnd(D, 2 * D, std=(2 * D) ** -0.5)
        w["loop.step"] = rnd(cfg["loop"]["times"], D, std=0.5)
    for i, spec in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", spec["mixer"], spec["mlp"]
        x = p + "mix."
        w[p + "norm1"], w[p + "norm1b"] = norm(D), norm(D)
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        maps = 2 if spec["type"] == "attention_2" else 1
        w[x + "q"], w[x + "k"] = rnd(H * maps * d, D, std=1.5 * D ** -0.5), rnd(G * maps * d, D, std=1.5 * D ** -0.5)
        w[x + "v"] = rnd(G * dv, D, std=D ** -0.5)
        w[x + "g"] = rnd(H * dv if maps == 1 else H, D, std=1.5 * D ** -0.5)
        w[x + "o"] = rnd(D, H * dv, std=(H * dv) ** -0.5)
        if maps == 2:
            for n in ("lq1", "lk1", "lq2", "lk2"):
                w[x + n] = rnd(d, std=0.3 * d ** -0.5)
        if mlp is None:
            continue
        w[p + "norm2"], w[p + "norm2b"] = norm(D), norm(D)
        y = p + "mlp."
        if mlp["kind"] == "dense":
            w[y + "gate"], w[y + "up"] = rnd(mlp["ff"], D, std=D ** -0.5), rnd(mlp["ff"], D, std=D ** -0.5)
            w[y + "down"] = rnd(D, mlp["ff"], std=mlp["ff"] ** -0.5)
            continue
        for e in range(mlp["router"]["experts"]):
            w[f"{y}e{e}.up"], w[f"{y}e{e}.down"] = rnd(mlp["expert"]["ff"], D, std=D ** -0.5), rnd(D, mlp["expert"]["ff"], std=mlp["expert"]["ff"] ** -0.5)
        w[y + "router"] = rnd(mlp["router"]["experts"], D, std=D ** -0.5)
    return w


def replay_and_compare(runner, cfg, weights, prompts, schedule, tol, want_all=None):
    """schedule: list of steps, each a list of (request name, token count).  Every token's logits are asked for and
    compared with the oracle's logits of the whole prompt; a request ends with its last token.  Returns the worst error."""
    from sglang_custom_amd.managers.trace_replay import TraceReplayer

    sixteen = runner.dtype != torch.float32
    want = want_all if want_all is not None else {k: ref.forward(cfg, weights, p) for k, p in prompts.items()}
    rp, at, errors = TraceReplayer(runner), {k: 0 for k in prompts}, []
    for step in schedule:
        entries, rows, end = [], [], []
        for name, n in step:
            lo, hi = at[name], at[name] + n
            entries.append(dict(id=name, tokens=prompts[name][lo:hi], want=list(range(n))))
            rows.append(want[name][lo:hi])
            at[name] = hi
            if hi == len(prompts[name]):
                end.append(name)
        e = row_errors(rp.step(entries, end), torch.cat(rows))
        worst = float(e.max())
        assert worst < (3 * tol if sixteen else tol), f"step {step}: logits differ from the whole-sequence oracle by {worst:.3g} (limit {tol})"
        errors.append(e)
    assert all(at[k] == len(p) for k, p in prompts.items()), "the schedule does not cover the prompts"
    assert not rp.live
    e = torch.cat(errors)
    assert within(e, tol, sixteen), f"{int((e >= tol).sum())} of {e.numel()} rows differ by more than {tol}"
    return float(e.max())
