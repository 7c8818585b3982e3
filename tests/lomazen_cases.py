"""Checks of single Lomazen mechanisms against the oracle's functions (oracle/lomazen_ref.py), written once for any ops
object: the HIP kernels on the GPU (test_lomazen_gpu.py) and the CPU stand-ins (test_lomazen_cpu.py).  Every case builds
the request table, positions and cache by hand, so that slots, pages and cuts are the case's to choose."""
import math

import torch

from oracle import lomazen_ref as ref
from verozen_cases import Table, _bf, _close, _tol


# ------------------------------------------------------------------------------------------- norms around a sublayer
def check_norm_add_norm(ops, device, dtype, T=7, D=48, eps=1e-5, n_rows=2):
    g = torch.Generator().manual_seed(0)
    dev = lambda t: t.to(dtype).to(device)
    x = torch.randn(T, D, generator=g) * 3 + 5.0
    y = _bf(torch.randn(T, D + 8, generator=g) * 4 - 6.0)             # a large mean, which this norm keeps
    w1, w2 = (_bf(1 + 0.2 * torch.randn(D, generator=g)) for _ in range(2))
    big = _bf(torch.randn(3 * T + 2, D, generator=g) * 2)
    rows = torch.randint(0, 3 * T + 2, (T, n_rows), generator=g, dtype=torch.int32)
    coef = torch.rand(T, n_rows, generator=g)
    picked = big[rows.long()]
    branches = [("one branch", y[:, 8:], dict(y=dev(y)[:, 8:])), ("picked rows", picked.sum(1), dict(y=dev(big), rows=rows.to(device))),
                ("weighted rows", (picked * coef.double()[..., None]).sum(1), dict(y=dev(big), rows=rows.to(device), coef=coef.to(device)))]
    for what, b, kw in branches:
        want = x.double() + ref.rms_norm(b, w1, eps)
        for nxt in ("norm", "copy", "none"):
            xd, kw2 = x.clone().to(device), dict(kw)
            h = ops.rmsnorm_residual_add_next(xd, kw2.pop("y"), dev(w1), dev(w2) if nxt == "norm" else None, eps, copy=nxt == "copy", **kw2)
            _close(xd, want, 3e-6, f"{what}: norm of the output added to the stream")
            if nxt == "none":
                assert h is None
                continue
            assert h.dtype == dtype
            _close(h, ref.rms_norm(want, w2, eps) if nxt == "norm" else want, _tol(dtype), f"{what}: {nxt} of the new stream")
    # eps sits inside the root: a tiny branch is not blown up to unit size
    tiny = torch.full((1, D), 2.0 ** -9, dtype=torch.float64)
    xd = torch.zeros(1, D, device=device)
    ops.rmsnorm_residual_add_next(xd, dev(tiny), dev(torch.ones(D)), None, 1e-2)
    _close(xd, ref.unit_rms(tiny, 1e-2), 1e-4, "a branch much smaller than the root of eps")


def check_pass_entry(ops, device, dtype, T=9, D=48, V=17, eps=1e-5):
    g = torch.Generator().manual_seed(1)
    y = _bf(torch.randn(T, D + 8, generator=g))
    table, step = torch.randn(V, D, generator=g), torch.randn(D, generator=g)
    w = _bf(1 + 0.2 * torch.randn(D, generator=g))
    ids = torch.randint(0, V, (T,), generator=g)
    ids[0], ids[-1] = 0, V - 1
    x = torch.full((T, D), 1e6, device=device)                        # what was there is replaced, not added to
    h = ops.pass_entry(x, y.to(dtype).to(device)[:, 8:], table.to(device), ids.to(device), step.to(device), w.to(dtype).to(device), eps)
    want = y[:, 8:] + table.double()[ids] + step.double()
    _close(x, want, 1e-6, "the stream at the start of a pass")
    _close(h, ref.rms_norm(want, w, eps), _tol(dtype), "the pass's first norm")


def check_pass_entry_layer(device, dtype, T=6, D=32, V=13, times=3):
    """The layer: W [x; e] + step_t from a product of the stream's half and a table of the embedding's half."""
    from sglang_custom_amd.layers.post_norm import PassEntry

    g = torch.Generator().manual_seed(2)
    w_in, step, e = _bf(torch.randn(D, 2 * D, generator=g) * D ** -0.5), _bf(torch.randn(times, D, generator=g)), _bf(torch.randn(V, D, generator=g))
    wn = _bf(1 + 0.1 * torch.randn(D, generator=g))
    m = PassEntry(D, times, V, 1e-5, dtype, device)
    m.set_weights(w_in.to(torch.bfloat16), step.to(torch.bfloat16), e.to(torch.bfloat16))
    m.stream_proj.quant_method.process_weights_after_loading(m.stream_proj)
    ids = torch.randint(0, V, (T,), generator=g)
    x = _bf(torch.randn(T, D, generator=g))
    for t in range(times):
        xd = x.float().to(device)
        h = m(xd, x.to(dtype).to(device), ids.to(device), t, wn.to(dtype).to(device))
        want = ref.enter_pass(x, e[ids], w_in, step[t])
        _close(xd, want, 3e-6 if dtype == torch.float32 else 6e-3, f"pass {t}")
        _close(h, ref.rms_norm(want, wn, 1e-5), _tol(dtype), f"pass {t}, first norm")


# ------------------------------------------------------------------------------------------- mixture, dense unit
def check_gated_unit(ops, device, dtype, T=5, ff=24):
    g = torch.Generator().manual_seed(3)
    gu = _bf(torch.randn(T, 2 * ff, generator=g) * 2)
    d = gu.to(dtype).to(device)
    _close(ops.gelu_tanh_and_mul(d[:, :ff], d[:, ff:]), ref.gelu_tanh(gu[:, :ff]) * gu[:, ff:], 1e-5 if dtype == torch.float32 else 8e-3, "tanh-GELU unit")


def check_moe_layer(device, dtype, T, experts=6, top=2, D=64, ff=32, seed=5):
    """The mixture layer itself (through the current ops backend) against the oracle.  Every token's router logits are set
    well apart, so that 16-bit rounding of the rows cannot change a choice; some experts get no token, one gets many."""
    from sglang_custom_amd.models.lomazen import LomazenMoE

    g = torch.Generator().manual_seed(seed)
    mlp = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))
    h = _bf(torch.randn(T, D, generator=g))
    h[:, :experts] = 0
    order = torch.stack([torch.randperm(max(experts - 1, 1), generator=g) for _ in range(T)])    # the last expert is never chosen
    order[: T // 2, 0] = 0
    for t in range(T):
        seen = [int(order[t, 0])] + [int(e) for e in order[t, 1:] if int(e) != int(order[t, 0])]
        for j, e in enumerate(seen[:top]):
            h[t, e] = 3.0 - 0.5 * j
        if experts > 1:
            h[t, experts - 1] = -3.0
    w = {f"e{e}.{n}": _bf(torch.randn(a, b, generator=g) * b ** -0.5) for e in range(experts) for n, a, b in (("up", ff, D), ("down", D, ff))}
    w["router"] = torch.zeros(experts, D, dtype=torch.float64)
    w["router"][:, :experts] = torch.eye(experts, dtype=torch.float64)
    want = ref.moe_ff(h, w, "", mlp)
    m = LomazenMoE(D, mlp, dtype, device)
    m.gate_weight.data.copy_(w["router"])
    m.experts.w_up.data.copy_(torch.stack([w[f"e{e}.up"] for e in range(experts)]))
    m.experts.w_down.data.copy_(torch.stack([w[f"e{e}.down"] for e in range(experts)]))
    out = m(h.to(dtype).to(device))
    got = (out["y"].double().cpu()[out["rows"].cpu().long()] * out["coef"].double().cpu()[..., None]).sum(1)
    _close(got, want, 2e-5 if dtype == torch.float32 else 2e-2, f"mixture of {experts} experts, {top} per token, {T} tokens")
    if 1 < top <= experts // 2:       # the scores are those of a softmax over ALL experts: the chosen ones' do not add up to one
        total = out["coef"].double().cpu().sum(1)
        assert float(total.max()) < 0.999
        _close(total, ref.choose(h @ w["router"].T, top)[1].sum(1), 1e-4 if dtype == torch.float32 else 1e-2, "sums of the chosen scores")


# ------------------------------------------------------------------------------------------- rotation and cache rows
def check_frequencies():
    """The package's frequency table against the oracle's: bands that keep, blend and divide; all of one kind; an empty ramp."""
    from sglang_custom_amd.layers.rotary_embedding import banded_pair_inv_freq

    kinds = set()
    for dims, base, sc in ((16, 500.0, dict(factor=4.0, low=0.5, high=3.0, original=24)), (48, 90000.0, dict(factor=16.0, low=1.5, high=6.0, original=700)),
                           (12, 10000.0, None), (6, 100.0, dict(factor=2.0, low=1.0, high=2.0, original=100000)), (4, 10.0, dict(factor=3.0, low=50.0, high=60.0, original=9)),
                           (32, 3000.0, dict(factor=8.0, low=2.0, high=2.0, original=512)), (2, 77.0, dict(factor=1.0, low=1.0, high=4.0, original=8))):
        got, want, plain = banded_pair_inv_freq(base, dims, sc), ref.frequencies(dims, base, sc), ref.frequencies(dims, base)
        assert got.dtype == torch.float32 and got.numel() == dims // 2
        assert float(((got.double() - want).abs() / want).max()) < 1e-7, (dims, base, sc)
        if sc and dims == 48:
            r = plain / want
            kinds = {"kept" if x < 1.0001 else "divided" if abs(x - 16.0) < 1e-6 else "blended" for x in r.tolist()}
    assert kinds == {"kept", "divided", "blended"}


class KVSetup:
    """Cache rows of one sequence scattered over slots through a request-table row; every row is stale until it is written."""

    def __init__(self, device, dtype, T, k_shape, v_shape, row=3, page=1, seed=5):
        g = torch.Generator().manual_seed(seed)
        self.tab = Table(device)
        if page == 1:
            n = T + 70
            slots = torch.randperm(n - 1, generator=g)[:T] + 1
        else:
            n = (T // page + 4) * page
            pages = torch.randperm(n // page - 1, generator=g) + 1
            slots = (pages[:, None] * page + torch.arange(page)[None, :]).reshape(-1)[:T]
        self.slots, self.row = slots.to(device), row
        self.k = torch.full((n + page,) + tuple(k_shape), 50.0, dtype=dtype, device=device)
        self.v = torch.full((n + page,) + tuple(v_shape), 50.0, dtype=dtype, device=device)
        self.tab.req_to_token[row, :T] = slots.to(torch.int32).to(device)


def check_rotate_write(ops, device, dtype, T=11, R=6, S=2, d=12, W=20, rot=8, interleaved=True, unit_norm=True, off=8, eps=1e-5):
    g = torch.Generator().manual_seed(6)
    f = ref.frequencies(rot, 300.0, dict(factor=4.0, low=0.5, high=3.0, original=24)) if rot else torch.zeros(1)
    p = _bf(torch.randn(T, off + (R + S) * d + W, generator=g) * 2)
    pos = torch.arange(T) + 900
    pos[0] = 0
    s = KVSetup(device, dtype, T, (S, d), (1, W))
    pd = p.to(dtype).to(device)
    q, k, v = pd[:, off: off + R * d], pd[:, off + R * d: off + (R + S) * d], pd[:, off + (R + S) * d:]
    got = ops.qkv_rotate_write(q.unflatten(1, (R, d)), k.unflatten(1, (S, d)), v, pos.to(device), f.float().to(device), rot, interleaved, unit_norm, eps,
                               s.k, s.v, s.slots.long())
    z = p[:, off: off + (R + S) * d].reshape(T, R + S, d)
    z = ref.rotate(z, pos, f, interleaved) if rot else z
    z = ref.unit_rms(z, eps) if unit_norm else z
    tol = 3e-4 if dtype == torch.float32 else _tol(dtype)
    what = f"{R}+{S} rows of {d}, rotation over {rot}, {'neighbours' if interleaved else 'halves'}"
    _close(got, z[:, :R], tol, "queries: " + what)
    _close(s.k[s.slots.long()], z[:, R:], tol, "keys in their cache rows: " + what)
    assert torch.equal(s.v[s.slots.long()].cpu().view(T, W), pd[:, off + (R + S) * d:].cpu()), "values are copied"
    untouched = torch.ones(s.k.shape[0], dtype=torch.bool)
    untouched[s.slots.cpu().long()] = False
    assert float((s.k.cpu()[untouched] - 50.0).abs().max()) == 0.0 and float((s.v.cpu()[untouched] - 50.0).abs().max()) == 0.0


# ------------------------------------------------------------------------------------------- attention
def run_attention(ops, device, dtype, q, k, v, cuts, scale, cap=0.0, lam=0.0, out_scale=1.0, eps=1e-5, gate=None, page=1, singles_tail=0,
                  decode_tail=0, splits=1):
    """q [T, H, maps, d], k [T, G, maps, d], v [T, G, dv].  A token's own and later rows are written only when its step comes, so a
    kernel that looks ahead reads stale rows.  The last singles_tail tokens go one by one as runs of one, the last decode_tail as
    decode steps."""
    T, H, maps, d = q.shape
    G, dv = v.shape[1], v.shape[2]
    s = KVSetup(device, dtype, T, (G, maps * d), (G, dv), page=page)
    kd, vd = k.reshape(T, G, maps * d).to(dtype).to(device), v.to(dtype).to(device)
    qd = q.to(dtype).to(device)
    gd = None
    if gate is not None:        # a column block of a wider row
        gd = torch.zeros(T, gate.shape[1] + 16, dtype=dtype)
        gd[:, 8: 8 + gate.shape[1]] = gate.to(dtype)
        gd = gd.to(device)[:, 8: 8 + gate.shape[1]]
    bq = ops.causal_attention_run_tokens(H, G, maps, d, dv, dtype)
    assert bq > 0
    outs, at = [], 0
    for n in cuts:
        decode = n == 1 and at >= T - decode_tail
        single = n == 1 and at >= T - singles_tail
        b = s.tab.batch([(s.row, at, n)])
        s.k[s.slots[at:at + n].long()] = kd[at:at + n]
        s.v[s.slots[at:at + n].long()] = vd[at:at + n]
        o = torch.full((n, H, dv), 9.0, dtype=dtype, device=device)
        kw = {}
        if not decode:
            runs = [[i, min(bq, n - i)] for i in range(0, n, bq)]
            kw = dict(tok_req=b["tok_req"], runs=torch.tensor(runs, dtype=torch.int32, device=device), max_run=1 if single or bq == 1 else bq)
        ops.causal_attention(qd[at:at + n], s.k, s.v, o, s.tab.req_to_token, b["req_pool_indices"], b["positions"], scale, cap=cap, lam=lam,
                             out_scale=out_scale, eps=eps, gate=None if gd is None else gd[at:at + n], num_splits=splits if decode or single else 1, **kw)
        outs.append(o.cpu())
        at += n
    assert at == T
    return torch.cat(outs)


def attend(q, k, v, scale, cap=0.0, lam=0.0, diff=0.0, eps=1e-5, gate=None):
    T, H, maps, _ = q.shape
    if maps == 1:
        o = ref.causal_attention(q[:, :, 0], k[:, :, 0], v, scale, cap or None)
    else:
        o = ref.difference_attention(q, k, v, scale, lam, diff, eps)
    if gate is not None:
        o = o * torch.sigmoid(gate.view(T, H, -1))
    return o


def check_attention(ops, device, dtype, H=6, G=2, maps=1, d=16, dv=24, T=150, cuts=(150,), cap=0.0, gate="feature", page=1, singles_tail=0,
                    decode_tail=0, splits=1):
    g = torch.Generator().manual_seed(7)
    q, k, v = (_bf(torch.randn(T, n, *s, generator=g)) for n, s in ((H, (maps, d)), (G, (maps, d)), (G, (dv,))))
    z = None if gate is None else _bf(torch.randn(T, H * dv if gate == "feature" else H, generator=g))
    scale, lam, diff = 1.7 * d ** -0.5, 0.45, 0.3
    want = attend(q, k, v, scale, cap, lam, diff, gate=z)
    got = run_attention(ops, device, dtype, q, k, v, cuts, scale, cap=cap, lam=lam, out_scale=1.0 - diff if maps == 2 else 1.0, gate=z, page=page,
                        singles_tail=singles_tail, decode_tail=decode_tail, splits=splits)
    _close(got, want, 3e-5 if dtype == torch.float32 else 2e-2,
           f"attention ({H}/{G} heads of {maps} x {d} / {dv}, cap {cap}, gate {gate}) cut into {list(cuts)[:6]}, pages of {page}, {splits} ranges")


def check_attention_planted(ops, device, dtype, H=6, G=2, maps=1, d=16, dv=16, T=400, page=1):
    """One key in hundreds whose score stands out: at position 0, far back, at every edge of a 32- or 64-row tile and of a page, the
    token itself, and the token just after, which must not be seen -- in prompts, portions, single tokens and decode steps with and
    without key ranges.  With two maps the key stands out in ONE of them, and the other map's average is taken off."""
    for m in range(maps):
        for cuts, singles, decode, splits in (((T,), 0, 0, 1), ((33, 31, 2, 2, 61, 3, T - 132), 0, 0, 1), ((T - 3, 1, 1, 1), 0, 3, 1), ((T - 3, 1, 1, 1), 3, 0, 5),
                                              ((T - 3, 1, 1, 1), 0, 3, 2), ((T - 9,) + (1,) * 9, 0, 9, 13)):
            for key in (0, 1, 31, 32, 63, 64, 65, 127, 128, 255, 256, T - 4, T - 2, T - 1):
                q, k = torch.zeros(T, H, maps, d, dtype=torch.float64), torch.zeros(T, G, maps, d, dtype=torch.float64)
                v = torch.zeros(T, G, dv, dtype=torch.float64)
                v[:, :, 2] = torch.arange(T, dtype=torch.float64).remainder(7.0)[:, None] / 8.0       # values that differ from row to row
                v[key, :, 1] = 4.0
                q[:, :, m, d - 1] = 4.0
                k[key, :, m, d - 1] = 4.0                                                            # score 16 against 0 elsewhere
                want = attend(q, k, v, 1.0, lam=0.5)
                got = run_attention(ops, device, dtype, q, k, v, cuts, 1.0, lam=0.5, page=page, singles_tail=singles, decode_tail=decode, splits=splits).double()
                err = float((got - want).abs().max())
                assert err < (2e-5 if dtype == torch.float32 else 1.5e-2) * 4.0, (m, cuts[:6], splits, key, err)
                if maps == 1 and key + 1 < T:
                    assert float(got[key, :, 1].min()) > 3.9
                if key > 0:
                    assert float(got[key - 1, :, 1].abs().max()) == 0.0, "a later key is not seen"


def check_score_cap(ops, device, dtype, H=4, G=2, d=8, dv=8, T=70):
    """Two keys with raw scores far apart and far past the cap come out with almost equal weights; without the cap the larger takes
    all.  Negative scores are capped too, and small ones pass almost unchanged."""
    q, k, v = torch.zeros(T, H, 1, d, dtype=torch.float64), torch.zeros(T, G, 1, d, dtype=torch.float64), torch.zeros(T, G, dv, dtype=torch.float64)
    q[..., 0] = 8.0
    k[..., 0] = -100.0
    k[3, :, 0, 0], k[40, :, 0, 0], k[50, :, 0, 0] = 30.0, 60.0, 0.125
    v[3, :, 0], v[40, :, 1], v[50, :, 2] = 1.0, 1.0, 1.0
    v[:, :, 7] = 1.0
    for cuts, tail, splits in (((T,), 0, 1), ((60, 2, 7, 1), 1, 2)):
        for cap in (4.0, 30.0, 0.0):
            want = attend(q, k, v, 1.0, cap)
            got = run_attention(ops, device, dtype, q, k, v, cuts, 1.0, cap=cap, decode_tail=tail, splits=splits)
            assert bool(torch.isfinite(got).all())
            _close(got, want, 3e-5 if dtype == torch.float32 else 1e-2, f"cap {cap}")
        got = run_attention(ops, device, dtype, q, k, v, cuts, 1.0, cap=4.0, decode_tail=tail, splits=splits)
        assert abs(float(got[T - 1, 0, 0]) - float(got[T - 1, 0, 1])) < 2e-3 and float(got[T - 1, 0, 0]) > 0.4
        assert float(run_attention(ops, device, dtype, q, k, v, cuts, 1.0, decode_tail=tail, splits=splits)[T - 1, 0, 1]) > 0.99


def check_difference(ops, device, dtype, H=2, G=1, d=8, dv=16, T=40):
    """The first token: both maps are the same one value, so the difference is (1 - lambda) v, over its root mean square a unit vector in
    the direction of v; lambda past 1 turns it round.  A lambda of 0 leaves map 1 alone.  eps keeps a difference of nothing at nothing."""
    g = torch.Generator().manual_seed(11)
    q, k, v = (_bf(torch.randn(T, n, *s, generator=g)) for n, s in ((H, (2, d)), (G, (2, d)), (G, (dv,))))
    tol = 3e-5 if dtype == torch.float32 else 2e-2
    for lam, sign in ((0.3, 1.0), (2.5, -1.0), (0.0, 1.0), (-0.7, 1.0)):
        for cuts, tail in (((T,), 0), ((1, 2, T - 5, 1, 1), 2)):
            got = run_attention(ops, device, dtype, q, k, v, cuts, 0.9, lam=lam, out_scale=0.8, decode_tail=tail)
            _close(got, attend(q, k, v, 0.9, lam=lam, diff=0.2), tol, f"difference with lambda {lam}")
            _close(got[0, 0], sign * 0.8 * ref.unit_rms(v[0, 0], 1e-5), tol, "the first token")
    same = run_attention(ops, device, dtype, q[:, :, :1].repeat(1, 1, 2, 1), k[:, :, :1].repeat(1, 1, 2, 1), v, (T,), 0.9, lam=1.0)
    assert float(same.abs().max()) < (1e-3 if dtype == torch.float32 else 2e-2), "equal maps cancel"


def check_batch_of_unequal(ops, device, dtype, H=6, G=2, maps=1, d=16, dv=24):
    """Three sequences in one step -- a prompt, a portion, a single token -- as runs and singles of one batch, against each alone."""
    g = torch.Generator().manual_seed(13)
    parts = [(0, 0, 70), (2, 45, 33), (1, 129, 1)]
    tab = Table(device)
    slots = torch.randperm(400, generator=g) + 1
    k_cache, v_cache = torch.full((402, G, maps * d), 50.0, dtype=dtype, device=device), torch.full((402, G, dv), 50.0, dtype=dtype, device=device)
    seqs, at = [], 0
    for row, p0, n in parts:
        L = p0 + n
        q, k, v = (_bf(torch.randn(L, m, *s, generator=g)) for m, s in ((H, (maps, d)), (G, (maps, d)), (G, (dv,))))
        sl = slots[at:at + L].to(device)
        tab.req_to_token[row, :L] = sl.to(torch.int32)
        k_cache[sl], v_cache[sl] = k.reshape(L, G, maps * d).to(dtype).to(device), v.to(dtype).to(device)
        seqs.append((q, attend(q, k, v, 0.4, cap=6.0 if maps == 1 else 0.0, lam=0.4, diff=0.25)))
        at += L
    b = tab.batch(parts)
    q = torch.cat([s[0][p0:p0 + n] for s, (_, p0, n) in zip(seqs, parts)]).to(dtype).to(device)
    out = torch.full((q.shape[0], H, dv), 9.0, dtype=dtype, device=device)
    bq = ops.causal_attention_run_tokens(H, G, maps, d, dv, dtype)
    runs, singles, t0 = [], [], 0
    for _, _, n in parts:
        if n == 1 or bq == 1:
            singles += [[t, 1] for t in range(t0, t0 + n)]
        else:
            runs += [[t, min(bq, t0 + n - t)] for t in range(t0, t0 + n, bq)]
        t0 += n
    for r, mx, sp in ((runs, bq, 1), (singles, 1, 3)):
        if r:
            before = out.clone()
            ops.causal_attention(q, k_cache, v_cache, out, tab.req_to_token, b["req_pool_indices"], b["positions"], 0.4, cap=6.0 if maps == 1 else 0.0, lam=0.4,
                                 out_scale=0.75 if maps == 2 else 1.0, eps=1e-5, tok_req=b["tok_req"], runs=torch.tensor(r, dtype=torch.int32, device=device),
                                 max_run=mx, num_splits=sp)
            listed = torch.zeros(q.shape[0], dtype=torch.bool)
            for t, n in r:
                listed[t:t + n] = True
            assert torch.equal(out.cpu()[~listed], before.cpu()[~listed]), "tokens that are not listed are left alone"
    _close(out, torch.cat([s[1][p0:p0 + n] for s, (_, p0, n) in zip(seqs, parts)]), 3e-5 if dtype == torch.float32 else 2e-2, "unequal sequences in one batch")


def check_rotation_decides(ops, device, dtype, d=16, T=70):
    """Rotation-matched content: a query at position p finds the key at p - 5 in either pairing, through rotate-and-write and attention."""
    g = torch.Generator().manual_seed(9)
    for neighbours in (True, False):
        f = ref.frequencies(d, 20.0)
        base = torch.randn(1, 1, d, generator=g, dtype=torch.float64).expand(T, 1, d)
        back = _bf(ref.rotate(base.clone(), torch.full((T,), -5), f, neighbours))
        base = _bf(base)
        v = _bf(torch.eye(16, dtype=torch.float64)[torch.arange(T) % 16])[:, None]
        s = KVSetup(device, dtype, T, (1, d), (1, 16))
        dev = lambda t: t.to(dtype).to(device)
        pos = torch.arange(T).to(device)
        q = ops.qkv_rotate_write(dev(back), dev(base), dev(v[:, 0]), pos, f.float().to(device), d, neighbours, True, 1e-6, s.k, s.v, s.slots.long())
        b = s.tab.batch([(s.row, 0, T)])
        out = torch.empty(T, 1, 16, dtype=dtype, device=device)
        ops.causal_attention(q.view(T, 1, 1, d), s.k, s.v, out, s.tab.req_to_token, b["req_pool_indices"][:1].expand(T).contiguous(), b["positions"], 8.0)
        o = out.double().cpu()[T - 1, 0]
        assert int(o.argmax()) == (T - 1 - 5) % 16 and float(o.max()) > 2 * float(o.sort().values[-2]), (neighbours, o)
        assert abs(float(o.sum()) - 1.0) < 1e-2 and math.isfinite(float(o.sum()))
