"""Plain, slow restatement of the Lomazen design for checking the product path: one function per mechanism, whole
sequences at once, no cache, no batching, float64 by default.  Test infrastructure only; nothing under sglang_custom_amd/
imports it and it imports nothing from there.

Notation: x [T, D] is the residual stream of ONE sequence at positions 0..T-1; weights come in a dict under their
checkpoint names (linear weights [out, in], applied as x @ W.T).

  stream      x = e = E[token];  per layer run  x <- x + N(mixer(N(x; n1)); n1b);  x <- x + N(ff(N(x; n2)); n2b)
  N           RMS norm with a weight, y / sqrt(mean y^2 + eps) * w
  order       the layers in turn, except that layers a .. b-1 are walked r times in a row; pass t of that walk starts from
              x <- W_in [x; e] + step_t
  mixer       "attention": grouped causal softmax attention; queries and keys are rotated (neighbouring features, some
              frequencies divided) and divided by their root mean square, scores are capped, the result is gated feature by
              feature.  "attention_2": the difference of two such softmaxes over the same values (rotation in halves, no norm, no
              cap), normed per head, gated head by head.
  ff          "dense": down(gelu(gate h) * up h); "moe": the top experts of a softmax, each down(relu(up h)^2); or none
  output      logits = s * E N(x; n_f)
"""
import math
from typing import Dict, List, Optional, Tuple

import torch


# ----------------------------------------------------------------------------------- small pieces
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * w


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def capped(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


# ----------------------------------------------------------------------------------- rotation
def frequencies(dims: int, base: float, scaling: Optional[dict] = None) -> torch.Tensor:
    """f_i, i < dims / 2.  With scaling {factor, low, high, original}: a pair of wavelength l = 2 pi / f keeps f when
    original / l > high, turns at f / factor when original / l < low, and at a blend of the two between, linear in
    original / l."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling:
        factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
        for i, fi in enumerate(f):
            turns = original * fi / (2.0 * math.pi)
            if turns > high:
                continue
            if turns < low:
                f[i] = fi / factor
            else:
                s = (turns - low) / (high - low)
                f[i] = (1.0 - s) * fi / factor + s * fi
    return torch.tensor(f, dtype=torch.float64)


def rotate(x: torch.Tensor, positions: torch.Tensor, freqs: torch.Tensor, neighbours: bool) -> torch.Tensor:
    """x [T, H, d]: the first 2 n features (n = len(freqs)) form pairs (2 i, 2 i + 1), or (i, i + n), which turn by
    positions * freqs[i]; the rest pass."""
    out, n = x.clone(), freqs.numel()
    for i in range(n):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + n)
        ang = positions.to(torch.float64) * freqs[i]
        c, s = torch.cos(ang).to(x.dtype)[:, None], torch.sin(ang).to(x.dtype)[:, None]
        out[..., a] = x[..., a] * c - x[..., b] * s
        out[..., b] = x[..., b] * c + x[..., a] * s
    return out


# ----------------------------------------------------------------------------------- mixers
def causal_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, cap: Optional[float] = None) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; query head h reads key / value head h // (H / G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    mask = torch.ones(T, T, dtype=torch.bool).tril()
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        s = q[:, h] @ k[:, h // per].T * scale
        if cap:
            s = capped(s, cap)
        out[:, h] = torch.softmax(s.masked_fill(~mask, -math.inf), -1) @ v[:, h // per]
    return out


def difference_factor(lq1, lk1, lq2, lk2, diff: float) -> torch.Tensor:
    return torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum()) + diff


def difference_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, lam, diff: float, eps: float) -> torch.Tensor:
    """q [T, H, 2, d], k [T, G, 2, d], v [T, G, dv] -> [T, H, dv]: (map 1 - lam * map 2) over its root mean square, times
    1 - diff."""
    a1 = causal_attention(q[:, :, 0], k[:, :, 0], v, scale)
    a2 = causal_attention(q[:, :, 1], k[:, :, 1], v, scale)
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def rotated(x: torch.Tensor, rot: Optional[dict], neighbours: bool) -> torch.Tensor:
    if not rot or not rot["dims"]:
        return x
    return rotate(x, torch.arange(x.shape[0]), frequencies(rot["dims"], float(rot["base"]), rot.get("scaling")), neighbours)


def attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mx: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, d)
    k = (h @ w[p + "k"].T).view(T, G, d)
    v = (h @ w[p + "v"].T).view(T, G, dv)
    q, k = (unit_rms(rotated(z, mx.get("rot"), True), eps) for z in (q, k))
    o = causal_attention(q, k, v, float(mx["scale"]), mx.get("softcap")).reshape(T, H * dv)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def attention_2_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mx: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = rotated((h @ w[p + "q"].T).view(T, 2 * H, d), mx.get("rot"), False).view(T, H, 2, d)
    k = rotated((h @ w[p + "k"].T).view(T, 2 * G, d), mx.get("rot"), False).view(T, G, 2, d)
    v = (h @ w[p + "v"].T).view(T, G, dv)
    diff = float(mx["diff"])
    lam = difference_factor(w[p + "lq1"], w[p + "lk1"], w[p + "lq2"], w[p + "lk2"], diff)
    o = difference_attention(q, k, v, float(mx["scale"]), lam, diff, eps)
    return (o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]).reshape(T, H * dv) @ w[p + "o"].T


# ----------------------------------------------------------------------------------- feed-forward
def dense_ff(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return torch.clamp(h @ w[p + "up"].T, min=0.0) ** 2 @ w[p + "down"].T


def choose(z: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits [T, E] -> (ids [T, top], those experts' softmax scores); the lower index on a tie."""
    s = torch.softmax(z, -1)
    ids = torch.argsort(s, dim=-1, descending=True, stable=True)[:, :top]
    return ids, torch.gather(s, 1, ids)


def moe_ff(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mlp: dict) -> torch.Tensor:
    ids, s = choose(h @ w[p + "router"].T, mlp["router"]["top"])
    rows = []
    for t in range(h.shape[0]):
        y = torch.zeros_like(h[t])
        for j in range(ids.shape[1]):
            y = y + s[t, j] * expert(h[t], w, f"{p}e{int(ids[t, j])}.")
        rows.append(y)
    return torch.stack(rows)


# ----------------------------------------------------------------------------------- the model
def layer_walk(config: dict) -> List[Tuple[int, Optional[int]]]:
    """(layer, number of the pass that starts right before it, or None) of every layer run."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, r = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    out = [(i, None) for i in range(a)]
    for t in range(r):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def enter_pass(x: torch.Tensor, e: torch.Tensor, w_in: torch.Tensor, step: torch.Tensor) -> torch.Tensor:
    return torch.cat([x, e], -1) @ w_in.T + step


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64, streams: Optional[list] = None):
    """Logits [T, vocab] of one sequence; `streams` (a list) receives the residual stream after every layer run."""
    w = {n: t.to(dtype) if t.is_floating_point() else t for n, t in weights.items()}
    eps = float(config["norm"]["eps"])
    e = w["embed"][torch.tensor(tokens)]
    x = e
    for i, t in layer_walk(config):
        if t is not None:
            x = enter_pass(x, e, w["loop.in"], w["loop.step"][t])
        spec, p = config["layers"][i], f"l{i}."
        mixer = {"attention": attention_mixer, "attention_2": attention_2_mixer}[spec["type"]]
        y = mixer(rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", spec["mixer"], eps)
        x = x + rms_norm(y, w[p + "norm1b"], eps)
        mlp = spec.get("mlp")
        if mlp is not None:
            h = rms_norm(x, w[p + "norm2"], eps)
            y = dense_ff(h, w, p + "mlp.") if mlp["kind"] == "dense" else moe_ff(h, w, p + "mlp.", mlp)
            x = x + rms_norm(y, w[p + "norm2b"], eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T * float(config.get("logit_scale", 1.0))


def greedy(config: dict, weights: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    """n tokens, each the arg-max of the whole-sequence logits at the last position (the lowest id on a tie)."""
    toks, out = list(prompt), []
    for _ in range(n):
        nxt = int(torch.argmax(forward(config, weights, toks)[-1]))
        out.append(nxt)
        toks.append(nxt)
    return out
