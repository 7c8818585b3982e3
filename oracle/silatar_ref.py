"""Plain, slow restatement of the Silatar design for checking the product path: one function per mechanism, whole
sequences at once, no cache, no state hand-over, no batching, float64 by default.  Test infrastructure only; nothing
under sglang_custom_amd/ imports it and it imports nothing from there.

Notation: x [T, D] is the residual stream of ONE sequence at positions 0..T-1; weights come in a dict under their
checkpoint names (linear weights [out, in], applied as x @ W.T).

  stream      x_0 = E[token];  per layer run  x <- x + L(mixer(L(x; n1)); n1b);  x <- x + L(ff(L(x; n2)); n2b)
  L           layer norm with a weight and no bias, (y - mean) / sqrt(var + eps) * w
  order       the layers in turn, except that layers a .. b-1 are walked r times in a row (same weights, nothing shared
              between the walks but the stream)
  mixer       "latent_attention": causal softmax attention whose per-head keys and values are linear in one small normed
              latent per token, plus one rotated key part that the heads share.  "mlstm": a matrix memory per head with an
              exponential input gate, a sigmoid forget gate, a normaliser and a running maximum that keeps both finite.
  ff          "dense": down(gelu(up h)); "moe": top-k experts fed with s_e h (s_e the sigmoid score), a clamped gated unit,
              plus a shared expert times a sigmoid gate; or none
  output      logits = c * tanh(H L(x; n_f) / c)
"""
import math
from typing import Dict, List, Optional

import torch


# ----------------------------------------------------------------------------------- small pieces
def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_erf(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


def capped(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


# ----------------------------------------------------------------------------------- rotation
def stretched_frequencies(dims: int, base: float, scaling: Optional[dict]):
    """(f_i for i < dims / 2, factor on cos and sin).  With scaling {factor, original, fast, slow}: the pair that turns t
    times over `original` positions sits at index dims ln(original / (2 pi t)) / (2 ln base); from the (floored) index for
    `fast` to the (ceiled) index for `slow` the frequency goes over, linearly in the index, from f_i to f_i / factor."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return torch.tensor(f, dtype=torch.float64), 1.0
    factor = float(scaling["factor"])
    index = {}
    for key in ("fast", "slow"):
        index[key] = dims * math.log(float(scaling["original"]) / (2.0 * math.pi * float(scaling[key]))) / (2.0 * math.log(base))
    first, last = max(math.floor(index["fast"]), 0), min(math.ceil(index["slow"]), dims - 1)
    width = max(last - first, 0.001)
    for i in range(dims // 2):
        r = min(1.0, max(0.0, (i - first) / width))
        f[i] = r * f[i] / factor + (1.0 - r) * f[i]
    return torch.tensor(f, dtype=torch.float64), 1.0 + 0.1 * math.log(factor)


def rotate_neighbours(x: torch.Tensor, positions: torch.Tensor, freqs: torch.Tensor, mag: float) -> torch.Tensor:
    """x [T, H, d]: features 2 i and 2 i + 1 (i < len(freqs)) turn together by positions * freqs[i]; the rest pass."""
    out = x.clone()
    for i in range(freqs.numel()):
        ang = positions.to(torch.float64) * freqs[i]
        c, s = (mag * torch.cos(ang)).to(x.dtype)[:, None], (mag * torch.sin(ang)).to(x.dtype)[:, None]
        a, b = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = a * c - b * s
        out[..., 2 * i + 1] = b * c + a * s
    return out


# ----------------------------------------------------------------------------------- mixers
def causal_softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """q, k [T, H, d], v [T, H, dv] -> [T, H, dv]."""
    T, H, _ = q.shape
    mask = torch.ones(T, T, dtype=torch.bool).tril()
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = (q[:, h] @ k[:, h].T * scale).masked_fill(~mask, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, h]
    return out


def latent_rows(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mx: dict, eps: float):
    """(c [T, rank] normed latent, r [T, rot] rotated shared key part): what a cache holds of each token."""
    rank = mx["kv_rank"]
    y = h @ w[p + "dkv"].T
    c = unit_rms(y[:, :rank], eps) * w[p + "dkv.norm"]
    r = y[:, None, rank:]
    rot = mx.get("rot")
    if rot and rot["dims"]:
        f, mag = stretched_frequencies(rot["dims"], float(rot["base"]), rot.get("scaling"))
        r = rotate_neighbours(r, torch.arange(h.shape[0]), f, mag)
    return c, r[:, 0]


def latent_attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mx: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, dn, dr, dv = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, dn + dr)
    qn, qr = q[..., :dn], q[..., dn:]
    c, r = latent_rows(h, w, p, mx, eps)
    rot = mx.get("rot")
    if rot and rot["dims"]:
        f, mag = stretched_frequencies(rot["dims"], float(rot["base"]), rot.get("scaling"))
        qr = rotate_neighbours(qr, torch.arange(T), f, mag)
    kn = (c @ w[p + "uk"].T).view(T, H, dn)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    k = torch.cat([kn, r[:, None, :].expand(T, H, dr)], -1)
    o = causal_softmax_attention(torch.cat([qn, qr], -1), k, v, float(mx["scale"]))
    return o.reshape(T, H * dv) @ w[p + "o"].T


def matrix_memory(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, log_in: torch.Tensor, log_forget: torch.Tensor) -> torch.Tensor:
    """q (already scaled), k [T, H, d], v [T, H, dv], log_in, log_forget [T, H] -> o [T, H, dv].  With m_0 = 0, S_0 = 0,
    n_0 = 0:  m' = max(f + m, i);  (S, n) <- e^(f + m - m') (S, n) + e^(i - m') (k v^T, k);  m <- m';
    o = S^T q / (max(|n . q|, e^-m) + 1e-6)."""
    T, H, d = q.shape
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        S = torch.zeros(d, v.shape[2], dtype=q.dtype)
        n = torch.zeros(d, dtype=q.dtype)
        m = torch.zeros((), dtype=q.dtype)
        for t in range(T):
            m_new = torch.maximum(log_forget[t, h] + m, log_in[t, h])
            keep, write = torch.exp(log_forget[t, h] + m - m_new), torch.exp(log_in[t, h] - m_new)
            S = keep * S + write * torch.outer(k[t, h], v[t, h])
            n = keep * n + write * k[t, h]
            m = m_new
            out[t, h] = (S.T @ q[t, h]) / (torch.maximum((n @ q[t, h]).abs(), torch.exp(-m)) + 1e-6)
    return out


def mlstm_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mx: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv, cap = mx["heads"], mx["dim"], mx["vdim"], float(mx["gate_cap"])
    q = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, dv)
    log_in = capped(h @ w[p + "i"].T + w[p + "i.b"], cap)
    log_forget = log_sigmoid(capped(h @ w[p + "f"].T + w[p + "f.b"], cap))
    o = unit_rms(matrix_memory(q, k, v, log_in, log_forget), eps).reshape(T, H * dv)
    return (o * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ----------------------------------------------------------------------------------- feed-forward
def clamped_unit(gate: torch.Tensor, up: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = torch.clamp(gate, max=limit), torch.clamp(up, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def expert(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, limit: float) -> torch.Tensor:
    return clamped_unit(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit) @ w[p + "down"].T


def choose(z: torch.Tensor, top: int):
    """Router logits [T, E] -> (ids [T, top], sigmoid scores of those [T, top]); the lower index on a tie."""
    s = torch.sigmoid(z)
    ids = torch.argsort(s, dim=-1, descending=True, stable=True)[:, :top]
    return ids, torch.gather(s, 1, ids)


def moe_ff(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mlp: dict) -> torch.Tensor:
    ids, s = choose(h @ w[p + "router"].T, mlp["router"]["top"])
    rows = []
    for t in range(h.shape[0]):
        y = torch.zeros_like(h[t])
        for j in range(ids.shape[1]):
            y = y + expert(s[t, j] * h[t], w, f"{p}e{int(ids[t, j])}.", float(mlp["expert"]["limit"]))
        rows.append(y)
    y = torch.stack(rows)
    if mlp.get("shared"):
        y = y + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert(h, w, p + "shared.", float(mlp["shared"]["limit"]))
    return y


def dense_ff(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return gelu_erf(h @ w[p + "up"].T) @ w[p + "down"].T


# ----------------------------------------------------------------------------------- the model
def layer_runs(config: dict) -> List[int]:
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return list(range(n))
    a, b, r = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    return list(range(a)) + list(range(a, b)) * r + list(range(b, n))


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64, streams: Optional[list] = None):
    """Logits [T, vocab] of one sequence; `streams` (a list) receives the residual stream after every layer run."""
    w = {n: t.to(dtype) if t.is_floating_point() else t for n, t in weights.items()}
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)]
    for i in layer_runs(config):
        spec, p = config["layers"][i], f"l{i}."
        mixer = {"latent_attention": latent_attention_mixer, "mlstm": mlstm_mixer}[spec["type"]]
        y = mixer(layer_norm(x, w[p + "norm1"], eps), w, p + "mix.", spec["mixer"], eps)
        x = x + layer_norm(y, w[p + "norm1b"], eps)
        mlp = spec.get("mlp")
        if mlp is not None:
            h = layer_norm(x, w[p + "norm2"], eps)
            y = dense_ff(h, w, p + "mlp.") if mlp["kind"] == "dense" else moe_ff(h, w, p + "mlp.", mlp)
            x = x + layer_norm(y, w[p + "norm2b"], eps)
        if streams is not None:
            streams.append(x.clone())
    logits = layer_norm(x, w["final.norm"], eps) @ w["head"].T
    cap = config.get("logit_softcap")
    return capped(logits, float(cap)) if cap else logits


def greedy(config: dict, weights: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    """n tokens, each the arg-max of the whole-sequence logits at the last position (the lowest id on a tie)."""
    toks, out = list(prompt), []
    for _ in range(n):
        nxt = int(torch.argmax(forward(config, weights, toks)[-1]))
        out.append(nxt)
        toks.append(nxt)
    return out
