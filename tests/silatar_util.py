"""Shared pieces of the Silatar tests: small random models in checkpoint form and the replay of a schedule with every
logit compared against the whole-sequence oracle (oracle/silatar_ref.py)."""
import torch

from fudonex_util import pools_are_whole  # noqa: F401  (generic helper)
from gatarax_util import row_errors, within
from oracle import silatar_ref as ref
from seturax_util import build_runner, random_prompts, rel_err  # noqa: F401  (generic helpers)


def latent(heads=3, dim=12, rot_dim=8, vdim=10, kv_rank=20, scale=0.25, base=500.0, rot_dims=None, scaling=True):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale)
    dims = rot_dim if rot_dims is None else rot_dims
    if dims:
        m["rot"] = dict(base=base, dims=dims)
        if scaling:
            m["rot"]["scaling"] = dict(factor=4.0, original=16, fast=2.0, slow=0.5) if scaling is True else dict(scaling)
    return dict(type="latent_attention", mixer=m)


def mlstm(heads=2, dim=14, vdim=9, gate_cap=6.0):
    return dict(type="mlstm", mixer=dict(heads=heads, dim=dim, vdim=vdim, gate_cap=gate_cap))


def dense(ff=40):
    return dict(kind="dense", ff=ff)


def moe(experts=5, top=2, ff=18, limit=0.8, shared=(22, 1.1)):
    m = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff, limit=limit))
    if shared:
        m["shared"] = dict(ff=shared[0], limit=shared[1])
    return m


def default_layers(every_expert=False):
    """Both mixers, both feed-forwards and none, unlike sizes throughout.  every_expert: each token uses all experts of its
    mixtures, so that a 16-bit run and a float64 oracle cannot part ways over a close call between two scores (the weights
    still differ from token to token)."""
    a, b = (moe(top=5), moe(experts=3, top=3, shared=None)) if every_expert else (moe(), moe(experts=7, top=1, shared=None))
    return [(mlstm(), dense()), (latent(), a), (latent(heads=2, dim=6, rot_dim=4, vdim=16, kv_rank=9, scaling=False), None),
            (mlstm(heads=3, dim=8, vdim=12, gate_cap=15.0), b),
            (latent(heads=1, dim=20, rot_dim=12, vdim=6, kv_rank=33, rot_dims=6, base=50.0), dense(24))]


def make_config(layers=None, width=48, vocab=53, loop=(1, 4, 2), softcap=12.0, eps=1e-5):
    """layers: list of (mixer spec, mlp spec or None)."""
    if layers is None:
        layers = default_layers()
        assert loop is None or loop[1] <= len(layers)
    cfg = dict(architecture="Silatar", vocab=vocab, width=width, norm=dict(eps=eps),
               layers=[dict(type=m["type"], mixer={k: (dict(v) if isinstance(v, dict) else v) for k, v in m["mixer"].items()}, mlp=f)
                       for m, f in layers])
    if loop:
        cfg["loop"] = dict(start=loop[0], stop=loop[1], times=loop[2])
    if softcap:
        cfg["logit_softcap"] = softcap
    return cfg


def make_weights(cfg, seed=0):
    """Checkpoint-named tensors with bf16-representable values, so that a bf16 and an fp32 run read the same numbers."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, std=1.0, mean=0.0):
        return (mean + std * torch.randn(*shape, generator=g)).to(torch.bfloat16)

    def norm(n):
        return rnd(n, std=0.1, mean=1.0)

    w = {"embed": rnd(V, D), "head": rnd(V, D, std=2 * D ** -0.5), "final.norm": norm(D)}
    for i, spec in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", spec["mixer"], spec["mlp"]
        x = p + "mix."
        w[p + "norm1"], w[p + "norm1b"] = norm(D), norm(D)
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if spec["type"] == "latent_attention":
            w[x + "q"] = rnd(H * (d + m["rot_dim"]), D, std=1.5 * D ** -0.5)
            w[x + "dkv"] = rnd(m["kv_rank"] + m["rot_dim"], D, std=D ** -0.5)
            w[x + "dkv.norm"] = norm(m["kv_rank"])
            w[x + "uk"] = rnd(H * d, m["kv_rank"], std=1.5 * m["kv_rank"] ** -0.5)
            w[x + "uv"] = rnd(H * dv, m["kv_rank"], std=m["kv_rank"] ** -0.5)
        else:
            for n, rows in (("q", H * d), ("v", H * dv), ("g", H * dv)):
                w[x + n] = rnd(rows, D, std=D ** -0.5)
            # keys that resemble the queries: a token's own write then always shows in its read-out.  With independent ones the
            # terms of a read-out now and then nearly cancel, and the norm that follows divides the rounding of 16-bit inputs by
            # the small rest (any 16-bit implementation shows those rows)
            w[x + "k"] = (w[x + "q"].float() + 0.5 * rnd(H * d, D, std=D ** -0.5).float()).to(torch.bfloat16)
            for n, mean in (("i", -0.5), ("f", 2.0)):
                w[x + n] = rnd(H, D, std=2 * D ** -0.5)
                w[x + n + ".b"] = rnd(H, std=0.7, mean=mean)
            w[x + "norm"] = norm(H * dv)
        w[x + "o"] = rnd(D, H * dv, std=(H * dv) ** -0.5)
        if mlp is None:
            continue
        w[p + "norm2"], w[p + "norm2b"] = norm(D), norm(D)
        y = p + "mlp."
        if mlp["kind"] == "dense":
            w[y + "up"], w[y + "down"] = rnd(mlp["ff"], D, std=D ** -0.5), rnd(D, mlp["ff"], std=mlp["ff"] ** -0.5)
            continue
        parts = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        if mlp.get("shared"):
            parts.append(("shared.", mlp["shared"]["ff"]))
            w[y + "shared.sg"] = rnd(1, D, std=2 * D ** -0.5)
        for n, ff in parts:
            w[y + n + "gate"], w[y + n + "up"] = rnd(ff, D, std=2 * D ** -0.5), rnd(ff, D, std=2 * D ** -0.5)     # past the limits often
            w[y + n + "down"] = rnd(D, ff, std=ff ** -0.5)
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
