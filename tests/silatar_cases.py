"""Checks of single Silatar mechanisms against the oracle's functions (oracle/silatar_ref.py), written once for any ops
object: the HIP kernels on the GPU (test_silatar_gpu.py) and the CPU stand-ins (test_silatar_cpu.py).  Every case builds
the request table, positions and state pool by hand, so that slots, pages and cuts are the case's to choose."""
import math

import torch

from oracle import silatar_ref as ref
from verozen_cases import Table, _bf, _close, _tol


def _segs(b, decode):
    return {} if decode else dict(tok_req=b["tok_req"], seg_start=b["seg_start"], seg_len=b["seg_len"])


# ------------------------------------------------------------------------------------------- norms around a sublayer
def check_norm_add_norm(ops, device, dtype, T=7, D=48, eps=1e-5, n_rows=2):
    g = torch.Generator().manual_seed(0)
    dev = lambda t: t.to(dtype).to(device)
    x = torch.randn(T, D, generator=g) * 3 + 20.0                     # a large mean, which the norm takes off
    y = _bf(torch.randn(T, D + 8, generator=g) * 4 - 6.0)
    w1, w2 = (_bf(1 + 0.2 * torch.randn(D, generator=g)) for _ in range(2))
    for next_norm in (True, False):
        xd = x.clone().to(device)
        h = ops.layernorm_residual_add(xd, dev(y)[:, 8:], dev(w1), dev(w2) if next_norm else None, eps)
        want = x.double() + ref.layer_norm(y[:, 8:], w1, eps)
        _close(xd, want, 2e-6, "layer norm of the output added to the stream")
        assert (h is not None) == next_norm
        if next_norm:
            assert h.dtype == dtype
            _close(h, ref.layer_norm(want, w2, eps), _tol(dtype), "the next norm of the new stream")
    # a token's expert rows and a gated second branch
    big = _bf(torch.randn(3 * T + 2, D, generator=g) * 2)
    rows = torch.randint(0, 3 * T + 2, (T, n_rows), generator=g, dtype=torch.int32)
    y2 = _bf(torch.randn(T, D, generator=g) * 3)
    gate = torch.randn(T, 5, generator=g) * 2
    b = big[rows.long()].sum(1)
    for second in (False, True):
        xd = x.clone().to(device)
        kw = dict(y2=dev(y2), y2_gate=gate.to(device)[:, 3]) if second else {}
        h = ops.layernorm_residual_add(xd, dev(big), dev(w1), dev(w2), eps, rows=rows.to(device), **kw)
        want = x.double() + ref.layer_norm(b + (torch.sigmoid(gate[:, 3:4].double()) * y2 if second else 0.0), w1, eps)
        _close(xd, want, 3e-6, "sum of picked rows" + (" and a gated branch" if second else ""))
        _close(h, ref.layer_norm(want, w2, eps), _tol(dtype), "the next norm")
    # eps sits inside the root: a branch of tiny deviations is not blown up to unit size
    tiny = torch.full((1, D), 0.5, dtype=torch.float64)
    tiny[0, 0] += 2.0 ** -8
    xd = torch.zeros(1, D, device=device)
    ops.layernorm_residual_add(xd, dev(tiny), dev(torch.ones(D)), None, 1e-2)
    _close(xd, ref.layer_norm(tiny, torch.ones(D, dtype=torch.float64), 1e-2), 2e-4, "tiny deviations")


def check_head_norm_gate(ops, device, dtype, T=5, H=3, dv=20, eps=1e-5):
    g = torch.Generator().manual_seed(3)
    o = torch.randn(T, H, dv, generator=g) * 4
    z = _bf(torch.randn(T, H * dv + 6, generator=g))
    w = _bf(1 + 0.3 * torch.randn(H * dv, generator=g))
    got = ops.head_rmsnorm_gate_act(o.to(device), w.to(dtype).to(device), z.to(dtype).to(device)[:, 6:], eps, dtype, "sigmoid")
    want = ref.unit_rms(o.double(), eps).reshape(T, H * dv) * w * torch.sigmoid(z[:, 6:])
    _close(got, want, _tol(dtype), "head norm with a weight per head, sigmoid gate")


# ------------------------------------------------------------------------------------------- small projections, activations
def check_project_f32(ops, device, dtype):
    """Unrounded in 16 bits, and a row's numbers are the same bits whatever lies beside it."""
    g = torch.Generator().manual_seed(1)
    for T, N, K, off in ((37, 19, 96, 0), (1, 1, 8, 0), (300, 5, 264, 8), (33, 17, 100, 0), (5, 40, 37, 3), (16, 16, 4096, 0)):
        x = _bf(torch.randn(T, K + off, generator=g))
        w = _bf(torch.randn(N, K, generator=g))
        xd, wd = x.to(dtype).to(device)[:, off:], w.to(dtype).to(device)
        got = ops.project_f32(xd, wd)
        assert got.dtype == torch.float32 and tuple(got.shape) == (T, N)
        _close(got, x[:, off:] @ w.T, 3e-6, f"small projection {T} x {N} x {K}")
        if dtype != torch.float32:
            for t in (0, T // 2, T - 1):
                assert torch.equal(ops.project_f32(xd[t:t + 1], wd)[0], got[t]), "a row does not depend on the batch"


def check_gelu(ops, device, dtype):
    g = torch.Generator().manual_seed(2)
    for T, d, off in ((9, 64, 8), (3, 4104, 0), (5, 33, 1), (70, 8, 0)):
        z = _bf(torch.randn(T, d + off, generator=g) * 3)
        got = ops.activation(z.to(dtype).to(device)[:, off:], "gelu_erf")
        _close(got, ref.gelu_erf(z[:, off:]), 1e-5 if dtype == torch.float32 else 5e-3, "erf-GELU")
    # the erf form, not the tanh approximation: they differ by about 5e-4 near 2.2
    z = torch.full((1, 8), -2.25)
    got = float(ops.activation(z.to(device), "gelu_erf")[0, 0])
    assert abs(got - float(ref.gelu_erf(torch.tensor(-2.25, dtype=torch.float64)))) < 2e-6


def check_clamped_glu(ops, device, dtype, ff=24, limit=0.75):
    g = torch.Generator().manual_seed(4)
    P = 11
    a = _bf(torch.randn(P, 2 * ff, generator=g) * 2)
    ad = a.to(dtype).to(device)
    _close(ops.clamped_glu(ad, limit, 1.702), ref.clamped_unit(a[:, :ff], a[:, ff:], limit), _tol(dtype), "clamped unit")
    rows = torch.tensor([[7, 2], [0, 10], [5, 4]], dtype=torch.int32)
    coef = torch.tensor([[0.25, 1.0], [0.5, 0.125], [0.9, 0.3]])
    got = ops.clamped_glu(ad, limit, 1.702, rows=rows.to(device), coef=coef.to(device))
    for r, c in zip(rows.reshape(-1).tolist(), coef.reshape(-1).tolist()):
        _close(got[r], ref.clamped_unit(c * a[r, :ff], c * a[r, ff:], limit), _tol(dtype), "clamped unit of a scaled row")
    # planted: the gate is clamped from above alone, the other half on both sides; the scale comes before the clamps
    L = limit
    cases = [(5.0, 0.0, L * _sig(1.702 * L)), (-5.0, 0.0, -5.0 * _sig(-1.702 * 5.0)), (0.5, 9.0, 0.5 * _sig(0.851) * (L + 1)),
             (0.5, -9.0, 0.5 * _sig(0.851) * (1 - L))]
    a = torch.zeros(1, 2 * ff, dtype=torch.float64)
    for i, (gt, up, _) in enumerate(cases):
        a[0, i], a[0, ff + i] = gt, up
    got = ops.clamped_glu(a.to(dtype).to(device), limit, 1.702)[0].double().cpu()
    for i, (_, _, want) in enumerate(cases):
        assert abs(float(got[i]) - want) < _tol(dtype) * max(abs(want), 0.05), (i, float(got[i]), want)
    one = torch.zeros(1, 1, dtype=torch.int32, device=device)
    got = ops.clamped_glu(torch.full((1, 2 * ff), 2.0, dtype=dtype, device=device), limit, 1.702, rows=one, coef=torch.full((1, 1), 0.125, device=device))
    assert abs(float(got[0, 0]) - 0.25 * _sig(1.702 * 0.25) * 1.25) < 2e-2, "0.125 * 2 is under the limit: scaled before the clamp"


def _sig(z):
    return 1.0 / (1.0 + math.exp(-z))


def check_moe_layer(device, dtype, T, experts=6, top=2, D=64, ff=32, limit=0.8, shared=(40, 1.3), seed=5):
    """The mixture layer itself (through the current ops backend) against the oracle.  Every token's router logits are set
    well apart, so that 16-bit rounding of the rows cannot change a choice; some experts get no token, one gets many."""
    from sglang_custom_amd.models.silatar import SilatarMoE

    g = torch.Generator().manual_seed(seed)
    mlp = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff, limit=limit))
    if shared:
        mlp["shared"] = dict(ff=shared[0], limit=shared[1])
    h = _bf(torch.randn(T, D, generator=g))
    h[:, :experts] = 0
    order = torch.stack([torch.randperm(experts - 1, generator=g) for _ in range(T)])            # the last expert is never chosen
    order[: T // 2, 0] = 0
    for t in range(T):
        seen = [int(order[t, 0])] + [int(e) for e in order[t, 1:] if int(e) != int(order[t, 0])]
        for j, e in enumerate(seen[:top]):
            h[t, e] = 3.0 - 0.5 * j
        h[t, experts - 1] = -3.0
    w = {}
    names = [(f"e{e}.", ff) for e in range(experts)] + ([("shared.", shared[0])] if shared else [])
    for n, f in names:
        w[n + "gate"], w[n + "up"], w[n + "down"] = (_bf(torch.randn(a, b, generator=g) * 2 * b ** -0.5) for a, b in ((f, D), (f, D), (D, f)))
    w["router"] = torch.zeros(experts, D, dtype=torch.float64)
    w["router"][:, :experts] = torch.eye(experts, dtype=torch.float64)
    if shared:
        w["shared.sg"] = _bf(torch.randn(1, D, generator=g) * D ** -0.5)
    want = ref.moe_ff(h, w, "", mlp)
    m = SilatarMoE(D, mlp, dtype, device)
    m.gate_weight.data.copy_(torch.cat([w["router"]] + ([w["shared.sg"]] if shared else [])))
    m.experts.w_up.data.copy_(torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(experts)]))
    m.experts.w_down.data.copy_(torch.stack([w[f"e{e}.down"] for e in range(experts)]))
    if shared:
        m.shared_gate_up.weight.data.copy_(torch.cat([w["shared.gate"], w["shared.up"]]))
        m.shared_down.weight.data.copy_(w["shared.down"])
        for lin in (m.shared_gate_up, m.shared_down):
            lin.quant_method.process_weights_after_loading(lin)
    out = m(h.to(dtype).to(device))
    y = out["y"].double().cpu()
    got = y[out["rows"].cpu().long()].sum(1)
    if shared:
        got = got + torch.sigmoid(out["y2_gate"].double().cpu())[:, None] * out["y2"].double().cpu()
    _close(got, want, 2e-5 if dtype == torch.float32 else 2e-2, f"mixture of {experts} experts, {top} per token, {T} tokens")
    # the weight is a factor on the input: with it on the output the result is visibly another one
    ids, s = ref.choose(h @ w["router"].T, top)
    other = torch.stack([sum(s[t, j] * ref.expert(h[t], w, f"e{int(ids[t, j])}.", limit) for j in range(top)) for t in range(min(T, 4))])
    here = torch.stack([sum(ref.expert(s[t, j] * h[t], w, f"e{int(ids[t, j])}.", limit) for j in range(top)) for t in range(min(T, 4))])
    assert float((other - here).abs().max()) > 0.05


# ------------------------------------------------------------------------------------------- latent rows and attention
class LatentSetup:
    """Cache rows of one sequence scattered over slots through a request-table row."""

    def __init__(self, device, dtype, T, width, row=3, page=1, seed=5):
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
        self.cache = torch.full((n + page, width), 50.0, dtype=dtype, device=device)       # stale rows that nothing may read
        self.tab.req_to_token[row, :T] = slots.to(torch.int32).to(device)


def check_latent_rows(ops, device, dtype, T=11, q_cols=30, rank=20, dr=12, rot_dims=8, eps=1e-5):
    g = torch.Generator().manual_seed(6)
    f, mag = ref.stretched_frequencies(rot_dims, 300.0, dict(factor=4.0, original=64, fast=4.0, slow=0.5)) if rot_dims else (torch.zeros(1), 1.0)
    a = _bf(torch.randn(T, q_cols + rank + dr + 3, generator=g) * 2)
    w = _bf(1 + 0.1 * torch.randn(rank, generator=g))
    pos = torch.arange(T) + 900
    pos[0] = 0
    s = LatentSetup(device, dtype, T, rank + dr)
    fd = f.float().to(device)
    ops.latent_rows_write(a.to(dtype).to(device), q_cols, w.to(dtype).to(device), pos.to(device), s.slots.long(), fd, s.cache, rank, dr,
                          rot_dims, True, mag, eps)
    c = ref.unit_rms(a[:, q_cols: q_cols + rank], eps) * w
    r = a[:, None, q_cols + rank: q_cols + rank + dr]
    if rot_dims:
        r = ref.rotate_neighbours(r, pos, f, mag)
    tol = 3e-4 if dtype == torch.float32 else _tol(dtype)
    _close(s.cache[s.slots.long()], torch.cat([c, r[:, 0]], 1), tol, "latent norm and rotated key part in their cache rows")
    untouched = torch.ones(s.cache.shape[0], dtype=torch.bool)
    untouched[s.slots.cpu().long()] = False
    assert float((s.cache.cpu()[untouched] - 50.0).abs().max()) == 0.0


def run_latent_attention(ops, device, dtype, qa, qr, c, r, scale, f, mag, rot_dims, cuts, page=1, decode_tail=0, splits=1):
    """qa [T, H, rank], qr [T, H, dr] unrotated, c [T, rank], r [T, dr] rotated rows.  A token's own and later rows are written
    only when its step comes, so a kernel that looks ahead reads stale rows."""
    T, H, rank = qa.shape
    dr = qr.shape[2]
    s = LatentSetup(device, dtype, T, rank + dr, page=page)
    rows = torch.cat([c, r], 1).to(dtype).to(device)
    bq = ops.latent_window_attention_block_tokens(H, rank, dr, dtype)
    assert bq > 0
    qad = qa.to(dtype).to(device).transpose(0, 1).contiguous().transpose(0, 1)      # head-major, as the batched product leaves it
    wide = torch.zeros(T, H, dr + 16, dtype=dtype)
    wide[..., 16:] = qr.to(dtype)
    qrd = wide.to(device)[..., 16:]
    outs, at = [], 0
    for n in cuts:
        decode = at >= T - decode_tail and n == 1
        b = s.tab.batch([(s.row, at, n)])
        s.cache[s.slots[at:at + n].long()] = rows[at:at + n]
        o = torch.zeros((n, H, rank), dtype=dtype, device=device)
        blocks = None if decode else torch.tensor([[i, min(bq, n - i)] for i in range(0, n, bq)], dtype=torch.int32, device=device)
        ops.latent_window_attention(qad[at:at + n], qrd[at:at + n], s.cache, o, s.tab.req_to_token, b["req_pool_indices"], b["positions"], None,
                                    f.float().to(device), rot_dims, 0, scale, tok_req=None if decode else b["tok_req"], blocks=blocks,
                                    num_splits=splits if decode and dtype != torch.float32 else 1, interleaved=True, rot_mag=mag)
        outs.append(o.cpu())
        at += n
    assert at == T
    return torch.cat(outs)


def _attend(qa, qr, c, r, scale, f, mag, rot_dims):
    T, H, _ = qa.shape
    if rot_dims:
        qr = ref.rotate_neighbours(qr, torch.arange(T), f, mag)
    k = torch.cat([c, r], 1)[:, None].expand(T, H, -1)
    return ref.causal_softmax_attention(torch.cat([qa, qr], -1), k, c[:, None].expand(T, H, -1), scale)


def check_latent_attention(ops, device, dtype, H=4, rank=32, dr=16, rot_dims=16, T=150, cuts=(150,), page=1, decode_tail=0, splits=1):
    g = torch.Generator().manual_seed(7)
    f, mag = ref.stretched_frequencies(rot_dims, 300.0, dict(factor=4.0, original=64, fast=4.0, slow=0.5)) if rot_dims else (torch.zeros(1), 1.0)
    qa, qr = _bf(torch.randn(T, H, rank, generator=g)), _bf(torch.randn(T, H, dr, generator=g))
    c, r = _bf(torch.randn(T, rank, generator=g)), _bf(torch.randn(T, dr, generator=g))
    scale = 1.7 / math.sqrt(rank + dr)
    want = _attend(qa, qr, c, r, scale, f, mag, rot_dims)
    got = run_latent_attention(ops, device, dtype, qa, qr, c, r, scale, f, mag, rot_dims, cuts, page=page, decode_tail=decode_tail, splits=splits)
    _close(got, want, 3e-5 if dtype == torch.float32 else 2e-2, f"latent attention ({H} heads, rank {rank} + {dr}) cut into {list(cuts)[:6]}, pages of {page}")


def check_latent_attention_planted(ops, device, dtype, rank=32, dr=16, H=3, T=400, page=1):
    """One key in hundreds whose score stands out: at position 0, far back, at every edge of a 32-row tile and of a page, the token
    itself, and the token just after, which must not be seen -- in prompts, portions and decode steps with and without key
    ranges."""
    f = torch.zeros(max(dr // 2, 1))
    cuts_of = [((T,), 0, 1), ((33, 31, 2, 2, T - 68), 0, 1), ((T - 3, 1, 1, 1), 3, 1), ((T - 3, 1, 1, 1), 3, 4), ((T - 40,) + (1,) * 40, 40, 3)]
    for cuts, tail, splits in cuts_of:
        for key in (0, 1, 31, 32, 33, 63, 64, 200, T - 4, T - 3, T - 2, T - 1):
            qa = torch.zeros(T, H, rank, dtype=torch.float64)
            c = torch.zeros(T, rank, dtype=torch.float64)
            c[:, 2] = torch.arange(T, dtype=torch.float64).remainder(7.0) / 8.0          # values that differ from row to row
            c[key, 1] = 4.0
            qa[:, :, 1] = 4.0                                                             # score 16 against 0 elsewhere
            zq, zr = torch.zeros(T, H, dr, dtype=torch.float64), torch.zeros(T, dr, dtype=torch.float64)
            want = _attend(qa, zq, c, zr, 1.0, f, 1.0, 0)
            got = run_latent_attention(ops, device, dtype, qa, zq, c, zr, 1.0, f, 1.0, 0, cuts, page=page, decode_tail=tail, splits=splits).double()
            tol = 1e-5 if dtype == torch.float32 else 1.5e-2
            err = float((got - want).abs().max())
            assert err < tol * 4.0, (cuts[:6], splits, key, err)
            if key + 1 < T:
                assert float(got[key, 0, 1]) > 3.9
            if key > 0:
                assert float(got[key - 1, :, 1].abs().max()) == 0.0, "a later key is not seen"


def check_shared_key_part(ops, device, dtype, T=70, H=2, rank=16, dr=8):
    """The rotated part alone decides: a query at position p with rotation-matched content finds the key at p - 5, whatever the
    magnitude on cos and sin; the pairing is of neighbouring features."""
    f, mag = ref.stretched_frequencies(dr, 20.0, dict(factor=4.0, original=64, fast=4.0, slow=0.5))
    g = torch.Generator().manual_seed(9)
    base = torch.randn(1, 1, dr, generator=g, dtype=torch.float64).expand(T, 1, dr)
    r = ref.rotate_neighbours(base, torch.arange(T), f, mag)[:, 0]
    qr = ref.rotate_neighbours(base.expand(T, H, dr).clone(), torch.full((T,), -5), f, 1.0)
    qr, r = _bf(qr), _bf(r)
    c = _bf(torch.eye(rank, dtype=torch.float64)[torch.arange(T) % rank])
    qa = torch.zeros(T, H, rank, dtype=torch.float64)
    want = _attend(qa, qr, c, r, 8.0, f, mag, dr)
    got = run_latent_attention(ops, device, dtype, qa, qr, c, r, 8.0, f, mag, dr, (T,))
    _close(got, want, 2e-3 if dtype == torch.float32 else 8e-2, "scores from the shared rotated part")
    p = T - 1
    assert float(want[p, 0, (p - 5) % rank]) > 2 * float(want[p, 0, (p - 4) % rank]) and float(want[p, 0].sum()) > 0.99


def check_frequencies():
    """The package's frequency table against the oracle's, also where the two ends of the ramp meet or cross."""
    from sglang_custom_amd.layers.rotary_embedding import scaled_pair_inv_freq

    for dims, base, sc in ((8, 500.0, dict(factor=4.0, original=16, fast=2.0, slow=0.5)), (24, 9000.0, dict(factor=8.0, original=512, fast=24.0, slow=2.0)),
                           (12, 10000.0, None), (6, 100.0, dict(factor=2.0, original=4096, fast=1.0, slow=1.0)),
                           (4, 10.0, dict(factor=3.0, original=100000, fast=0.001, slow=0.0001)), (2, 77.0, dict(factor=1.0, original=8, fast=64.0, slow=32.0))):
        got, mag = scaled_pair_inv_freq(base, dims, sc)
        want, mw = ref.stretched_frequencies(dims, base, sc)
        assert got.dtype == torch.float32 and got.numel() == dims // 2
        assert float(((got.double() - want).abs() / want).max()) < 1e-7 and abs(mag - mw) < 1e-12, (dims, base, sc)


# ------------------------------------------------------------------------------------------- matrix memory
def run_matrix_memory(ops, device, dtype, q, k, v, zi, zf, bi, bf, cap, q_scale, cuts, decode_tail=0, slot=2, state=None):
    T, H, dk = q.shape
    dv = v.shape[2]
    tab = Table(device)
    tab.req_to_state[4] = slot
    blocks = -(-dv // ops.MATRIX_MEMORY_VALUE_BLOCK)
    if state is None:
        state = (torch.full((5, H, dk, dv), 77.0, dtype=torch.float32, device=device),        # stale: position 0 must not read it
                 torch.full((5, H, blocks, dk + 1), 33.0, dtype=torch.float32, device=device))
    wide = torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1).to(dtype).to(device)      # column blocks of one projection
    qd, kd = wide[:, : H * dk].view(T, H, dk), wide[:, H * dk: 2 * H * dk].view(T, H, dk)
    vd = wide[:, 2 * H * dk:].view(T, H, dv)
    gates = torch.cat([zi, zf], 1).float().to(device)
    outs, at = [], 0
    for n in cuts:
        decode = at >= T - decode_tail and n == 1
        b = tab.batch([(4, at, n)])
        o = torch.empty((n, H, dv), dtype=torch.float32, device=device)
        ops.matrix_memory(qd[at:at + n], kd[at:at + n], vd[at:at + n], gates[at:at + n, :H], gates[at:at + n, H:], bi.float().to(device),
                          bf.float().to(device), o, state[0], state[1], tab.req_to_state, b["req_pool_indices"], b["positions"], q_scale, cap,
                          **_segs(b, decode))
        outs.append(o.cpu())
        at += n
    assert at == T
    for z in (0, 1, 3, 4):
        assert float((state[0][z] - 77.0).abs().max()) == 0.0 and float((state[1][z] - 33.0).abs().max()) == 0.0, "only the sequence's slot is written"
    return torch.cat(outs), state


def _gates(zi, zf, bi, bf, cap):
    return ref.capped(zi + bi, cap), ref.log_sigmoid(ref.capped(zf + bf, cap))


def check_matrix_memory(ops, device, dtype, H=3, dk=12, dv=20, T=45, cuts=(45,), decode_tail=0, cap=5.0, gate_std=2.0):
    g = torch.Generator().manual_seed(8)
    q, k, v = (_bf(torch.randn(T, H, n, generator=g)) for n in (dk, dk, dv))
    zi, zf = (gate_std * torch.randn(T, H, generator=g).float().double() for _ in range(2))
    bi, bf = _bf(torch.randn(H, generator=g)), _bf(torch.randn(H, generator=g) + 2.0)
    want = ref.matrix_memory(q * 0.3, k, v, *_gates(zi, zf, bi, bf, cap))
    got, state = run_matrix_memory(ops, device, dtype, q, k, v, zi, zf, bi, bf, cap, 0.3, cuts, decode_tail=decode_tail)
    # per row: a read-out is a quotient, and rows differ in size
    scale = want.abs().amax(-1, keepdim=True).clamp_min(1e-3)
    err = float(((got.double() - want).abs() / scale).max())
    assert err < 3e-4, f"matrix memory ({H} heads of {dk}/{dv}) cut into {list(cuts)[:6]}: {err:.3g}"
    nm = state[1][2]
    assert torch.equal(nm, nm[:, :1].expand_as(nm).contiguous()), "every block's copy of the normaliser is the same"
    return got


def check_matrix_memory_planted(ops, device, dtype):
    """Hand-made gates.  Head 0 never forgets (f = 0 to rounding), head 1 halves per token; a token far back under a key of its
    own is read in full / not at all.  The running maximum starts at 0: a first write of e^-6 is weighed against e^0 (result
    e^-6 v, not v).  Where the floor e^-m rules, |n . q| does not divide.  A large input gate takes over completely, in
    finite numbers."""
    H, dk, dv, T, cap = 2, 8, 40, 300, 90.0

    def logit(x):            # the gate logit whose capped value is x
        return cap * math.atanh(x / cap)

    q, k, v = (torch.zeros(T, H, n, dtype=torch.float64) for n in (dk, dk, dv))
    zi = torch.full((T, H), logit(-60.0), dtype=torch.float64)                # writes nothing to speak of
    zf = torch.zeros(T, H, dtype=torch.float64)
    zf[:, 0] = logit(60.0)
    k[:, :, 1] = 1.0
    for t in (3, 250):
        k[t] = 0
    k[3, :, 0] = 1.0
    v[3, :, 2], v[3, :, 37] = 2.0, -3.0
    zi[3] = logit(-6.0)
    q[3, :, 0] = q[200, :, 0] = q[249, :, 0] = 1.0
    k[250, :, 5] = 1.0
    v[250, :, 39] = 7.0
    zi[250] = logit(80.0)
    q[250, :, 5] = 1.0
    q[251, :, 0] = 1.0
    q[299, :, 5] = 0.5
    b0 = torch.zeros(H, dtype=torch.float64)
    want = ref.matrix_memory(q, k, v, *_gates(zi, zf, b0, b0, cap))
    e6 = math.exp(-6.0)
    for cuts, tail in (((T,), 0), ((2, 2, 16, 17, 200, 13, 1, 1, T - 252), 0), ((3, 1, 245, 1, 1) + (1,) * 49, 51)):
        got, state = run_matrix_memory(ops, device, dtype, q, k, v, zi, zf, b0, b0, cap, 1.0, cuts, decode_tail=tail)
        assert bool(torch.isfinite(got).all()) and bool(torch.isfinite(state[0][2]).all())
        for t in (3, 200, 249):
            assert abs(float(got[t, 0, 2]) / (2.0 * e6) - 1) < 1e-4 and abs(float(got[t, 0, 37]) / (-3.0 * e6) - 1) < 1e-4, (cuts[:5], t)
        assert abs(float(got[250, 0, 39]) - 7.0) < 1e-4 and abs(float(got[250, 1, 39]) - 7.0) < 1e-4
        assert abs(float(got[251, 0, 2])) < 1e-6, "what came before a much larger write is gone"
        assert abs(float(got[299, 0, 39]) - 7.0) < 1e-4, "|n . q| divides: the size of q cancels"
        scale = want.abs().amax(-1, keepdim=True).clamp_min(1e-6)
        assert float(((got.double() - want).abs() / scale).max()) < 1e-3


def check_matrix_memory_batch(ops, device, dtype, H=2, dk=20, dv=36):
    """Three sequences in one step -- a new one, one that goes on, one with a single token -- against each alone; a slot that is
    used again by a new sequence starts from zero."""
    g = torch.Generator().manual_seed(12)
    lens, done = [19, 30, 25], [0, 13, 24]
    seqs = []
    for n in lens:
        q, k, v = (_bf(torch.randn(n, H, m, generator=g)) for m in (dk, dk, dv))
        zi, zf = (2.0 * torch.randn(n, H, generator=g).float().double() for _ in range(2))
        seqs.append((q, k, v, zi, zf))
    b0 = torch.zeros(H, dtype=torch.float64)
    want = [ref.matrix_memory(s[0], s[1], s[2], *_gates(s[3], s[4], b0, b0, 4.0)) for s in seqs]
    tab = Table(device)
    tab.req_to_state[:6] = torch.tensor([1, 3, 2, 0, 0, 0], dtype=torch.int32)
    blocks = -(-dv // ops.MATRIX_MEMORY_VALUE_BLOCK)
    state, norm = torch.full((5, H, dk, dv), 9.0, device=device), torch.full((5, H, blocks, dk + 1), 9.0, device=device)

    def step(parts):
        b = tab.batch(parts)
        cat = [torch.cat([seqs[r][i][p0:p0 + n] for r, p0, n in parts]) for i in range(5)]
        o = torch.empty((cat[0].shape[0], H, dv), dtype=torch.float32, device=device)
        ops.matrix_memory(*(t.to(dtype).to(device) for t in cat[:3]), *(t.float().to(device) for t in cat[3:]), b0.float().to(device),
                          b0.float().to(device), o, state, norm, tab.req_to_state, b["req_pool_indices"], b["positions"], 1.0, 4.0, **_segs(b, False))
        at = 0
        for r, p0, n in parts:
            w = want[r][p0:p0 + n]
            assert float(((o[at:at + n].cpu().double() - w).abs() / w.abs().amax(-1, keepdim=True).clamp_min(1e-3)).max()) < 3e-4, (parts, r)
            at += n

    for _ in range(2):              # the second time over used slots
        step([(2, 0, done[2]), (1, 0, done[1])])
        step([(0, 0, 19), (1, 13, 17), (2, 24, 1)])
