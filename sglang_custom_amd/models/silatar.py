"""Silatar: a decoder-only model on an fp32 residual stream with a layer norm (weight, no bias) on BOTH sides of every
sublayer, x <- x + L(mixer(L(x))), x <- x + L(ff(L(x))), some of whose layers run several times in a row with the same
weights.  The mixer is, layer by layer,

  latent_attention   causal softmax attention over a latent cache: per token one RMS-normed latent c and one rotated key part
                     that the heads share; per-head keys W_uk c and values W_uv c exist only in absorbed form.  Rotation of
                     neighbouring features, with frequencies and a magnitude stretched for long sequences.
  mlstm              a matrix memory per head: exponential input gate and sigmoid forget gate, both from capped logits, a
                     normaliser and a running maximum beside the matrix; the read-out is RMS-normed per head and multiplied by
                     a sigmoid gate per feature.

The feed-forward is dense with an erf-GELU, a mixture of clamped gated experts whose sigmoid scores are factors on the
experts' INPUTS, plus a shared expert behind a sigmoid gate, or absent.  The logits are capped by a tanh.
(No counterpart in the reference; the module layout follows its model files, python/sglang/srt/models/deepseek_v2.py for the
latent attention and the mixture.)

Per layer run (T tokens, width D), besides the GEMMs' own launches:

  latent_attention   in_proj [q | kv latent | shared key part]; LatentWindowAttention.write_rows (latent norm, rotation, cache row);
                     W_uk per head; LatentWindowAttention (rotation of q inside); W_uv per head; o
  mlstm              in_proj [q | k | v | g] and, in unrounded fp32, [i | f]; MatrixMemory; HeadNormGate; o
  LayerNormResidualAdd   x += L(y) in place, and the layer norm in front of the next sublayer              1 launch, fp32
  dense              up, gelu, down
  moe                router and shared gate logits in unrounded fp32 (one projection); route, align, grouped GEMM, clamped
                     unit, grouped GEMM; the shared expert's two GEMMs and clamped unit; the sum over a token's rows and the
                     gated shared branch happen in the LayerNormResidualAdd that follows

Norms, positions and angles, attention scores / weights, router, gates of the recurrence, recurrent state and the residual sum
are fp32 in every dtype; `dtype` is what the projections read and write.  Caches and states belong to layer RUNS: run r of the
configuration's layer_runs uses cache layer r, whichever layer's weights it reads.  Every size comes from the configuration,
layer by layer.  Tensor parallelism is not implemented for this family (its head counts need not divide)."""
from typing import Dict

import torch
from torch import nn

from ..distributed.parallel_state import get_tensor_model_parallel_world_size
from ..layers.activation import Activation, ClampedGLU
from ..layers.latent_window_attention import LatentWindowAttention
from ..layers.linear import PerHeadLinear, ReplicatedLinear
from ..layers.linear_recurrence import HeadNormGate, MatrixMemory
from ..layers.logits_processor import LogitsProcessor
from ..layers.moe import GroupedExperts, GroupedTopKRouter
from ..layers.post_norm import LayerNormResidualAdd
from ..layers.rotary_embedding import scaled_pair_inv_freq
from ..layers.token_shift import ShiftedLayerNorm
from ..layers.vocab_parallel_embedding import ParallelLMHead
from ..ops_backend import get_ops


class SilatarLatentAttention(nn.Module):
    def __init__(self, hidden: int, mx: dict, eps: float, layer_id: int, dtype, device):
        super().__init__()
        H, dn, dr, dv, rank = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
        self.H, self.dn, self.dr, self.dv, self.rank, self.eps = H, dn, dr, dv, rank, float(eps)
        self.q_width = H * (dn + dr)
        self.in_proj = ReplicatedLinear(hidden, self.q_width + rank + dr, dtype, device)       # [q | kv latent | shared key part]
        self.kv_norm = nn.Parameter(torch.ones(rank, dtype=dtype, device=device), requires_grad=False)
        self.uk = PerHeadLinear(H, dn, rank, dtype, device)      # absorbed: q_nope -> latent (the transpose of the key expansion)
        self.uv = PerHeadLinear(H, rank, dv, dtype, device)
        self.o_proj = ReplicatedLinear(H * dv, hidden, dtype, device)
        rot = mx.get("rot") or {}
        dims = int(rot.get("dims", 0))
        freqs, mag = scaled_pair_inv_freq(rot["base"], dims, rot.get("scaling")) if dims else (torch.zeros(1), 1.0)
        self.attn = LatentWindowAttention(H, rank, dr, mx["scale"], 0, layer_id, rot_dims=dims, rot_base=1.0, device=device,
                                          with_sink=False, interleaved=True, inv_freq=freqs, rot_mag=mag)

    def forward(self, positions, h, forward_batch, run: int):
        T, H = h.shape[0], self.H
        p = self.in_proj(h)[0]
        self.attn.write_rows(p, self.q_width, self.kv_norm.data, self.eps, positions, forward_batch, cache_layer=run)
        q = p[:, : self.q_width].view(T, H, self.dn + self.dr)
        qa = self.uk(q[..., : self.dn])
        o_lat = torch.empty((H, T, self.rank), dtype=h.dtype, device=h.device).transpose(0, 1)
        self.attn(qa, q[..., self.dn:], None, forward_batch, o_lat, cache_layer=run)
        return self.o_proj(self.uv(o_lat).reshape(T, H * self.dv))[0]


class SilatarMatrixMemory(nn.Module):
    def __init__(self, hidden: int, mx: dict, eps: float, layer_id: int, dtype, device):
        super().__init__()
        H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
        self.H, self.d, self.dv = H, d, dv
        self.in_proj = ReplicatedLinear(hidden, 2 * H * d + 2 * H * dv, dtype, device)         # [q | k | v | g]
        self.gate_weight = nn.Parameter(torch.zeros(2 * H, hidden, dtype=dtype, device=device), requires_grad=False)    # [i | f]
        self.memory = MatrixMemory(H, d, dv, mx["gate_cap"], device, q_scale=d ** -0.5)
        self.norm_gate = HeadNormGate(dv, eps, dtype, device, with_weight=True, gate_act="sigmoid", heads=H)
        self.o_proj = ReplicatedLinear(H * dv, hidden, dtype, device)

    def forward(self, positions, h, forward_batch, run: int):
        T, H, d, dv = h.shape[0], self.H, self.d, self.dv
        p = self.in_proj(h)[0]
        gates = get_ops().project_f32(h, self.gate_weight.data)
        q, k = p[:, : H * d].view(T, H, d), p[:, H * d: 2 * H * d].view(T, H, d)
        v = p[:, 2 * H * d: 2 * H * d + H * dv].view(T, H, dv)
        o = self.memory(q, k, v, gates, forward_batch, cache_layer=run)
        return self.o_proj(self.norm_gate(o, p[:, 2 * H * d + H * dv:]))[0]


class SilatarMLP(nn.Module):
    def __init__(self, hidden: int, ff: int, dtype, device):
        super().__init__()
        self.up = ReplicatedLinear(hidden, ff, dtype, device)
        self.act = Activation("gelu_erf")
        self.down = ReplicatedLinear(ff, hidden, dtype, device)

    def forward(self, h):
        """-> what LayerNormResidualAdd takes besides the stream and the next norm."""
        return dict(y=self.down(self.act(self.up(h)[0]))[0])


class SilatarMoE(nn.Module):
    def __init__(self, hidden: int, mlp: dict, dtype, device):
        super().__init__()
        r, e, s = mlp["router"], mlp["expert"], mlp.get("shared")
        self.E = r["experts"]
        # rows [experts | gate of the shared expert]: both logits of one projection, unrounded
        self.gate_weight = nn.Parameter(torch.zeros(self.E + (1 if s else 0), hidden, dtype=dtype, device=device), requires_grad=False)
        self.router = GroupedTopKRouter(hidden, self.E, r["top"], 1, 1, 1.0, device, group_best=1, renorm=False, with_correction=False,
                                        with_weight=False)
        self.experts = GroupedExperts(hidden, e["ff"], self.E, dtype, device, activation="clamped_glu", limit=e["limit"])
        self.shared_gate_up = ReplicatedLinear(hidden, 2 * s["ff"], dtype, device) if s else None
        self.shared_act = ClampedGLU(s["limit"]) if s else None
        self.shared_down = ReplicatedLinear(s["ff"], hidden, dtype, device) if s else None

    def forward(self, h):
        logits = get_ops().project_f32(h, self.gate_weight.data)
        ids, weights = self.router.route(logits[:, : self.E])
        y, rows = self.experts(h, ids, weights)
        out = dict(y=y, rows=rows)
        if self.shared_down is not None:
            out.update(y2=self.shared_down(self.shared_act(self.shared_gate_up(h)[0]))[0], y2_gate=logits[:, self.E])
        return out


_MIXERS = {"latent_attention": SilatarLatentAttention, "mlstm": SilatarMatrixMemory}


class SilatarDecoderLayer(nn.Module):
    def __init__(self, config, layer_id: int, dtype, device):
        super().__init__()
        spec = config.layer_specs[layer_id]
        D, eps, mlp = config.hidden_size, config.rms_norm_eps, spec.get("mlp")
        self.kind = spec["type"]
        self.norm1 = nn.Parameter(torch.ones(D, dtype=dtype, device=device), requires_grad=False)
        self.mixer = _MIXERS[self.kind](D, spec["mixer"], eps, layer_id, dtype, device)
        self.add1 = LayerNormResidualAdd(D, eps, dtype, device)
        self.mlp = None
        if mlp is not None:
            self.norm2 = nn.Parameter(torch.ones(D, dtype=dtype, device=device), requires_grad=False)
            self.mlp = SilatarMLP(D, mlp["ff"], dtype, device) if mlp["kind"] == "dense" else SilatarMoE(D, mlp, dtype, device)
            self.add2 = LayerNormResidualAdd(D, eps, dtype, device)

    def forward(self, positions, x, h, forward_batch, run: int, next_norm):
        """x: the fp32 stream, updated in place; h: its normed copy for the mixer; next_norm: the weight of the norm that reads
        the stream after this run.  Returns that norm's result."""
        y = self.mixer(positions, h, forward_batch, run)
        h = self.add1(x, y, self.norm2.data if self.mlp is not None else next_norm)
        if self.mlp is not None:
            h = self.add2(x, next_weight=next_norm, **self.mlp(h))
        return h


class SilatarModel(nn.Module):
    def __init__(self, config, dtype, device):
        super().__init__()
        D = config.hidden_size
        self.layer_runs = list(config.layer_runs)
        self.embed = nn.Parameter(torch.zeros(config.vocab_size, D, dtype=dtype, device=device), requires_grad=False)
        self.layers = nn.ModuleList([SilatarDecoderLayer(config, i, dtype, device) for i in range(len(config.layer_specs))])
        self.norm = ShiftedLayerNorm(D, config.rms_norm_eps, dtype, device)
        self.capture_streams = None     # a list here receives the fp32 residual after every layer run (tests, debugging)

    def forward(self, input_ids, positions, forward_batch):
        x = get_ops().embedding(input_ids, self.embed.data).float()
        runs = [self.layers[i] for i in self.layer_runs]
        norms = [layer.norm1.data for layer in runs] + [self.norm.weight.data]
        h = get_ops().layernorm_shift(x, norms[0], self.norm.eps)
        for r, layer in enumerate(runs):
            h = layer(positions, x, h, forward_batch, r, norms[r + 1])
            if self.capture_streams is not None:
                self.capture_streams.append(x.clone())
        return h


class SilatarForCausalLM(nn.Module):
    supports_hip_graph = False    # a captured decode step pads the batch with row 0 of the request table, whose state slot it would overwrite

    def __init__(self, config, dtype=torch.bfloat16, device="cuda", quant_method_factory=None):
        super().__init__()
        if quant_method_factory is not None:
            raise NotImplementedError("Silatar runs unquantised (its norms, router, gates and residual are fp32 by design)")
        if get_tensor_model_parallel_world_size() != 1:
            raise NotImplementedError("Silatar: tensor parallelism is not implemented")
        self.config = config
        self.dtype = dtype
        self.needs_sequence_state = bool(config.needs_sequence_state)
        self.model = SilatarModel(config, dtype, device)
        self.lm_head = ParallelLMHead(config.vocab_size, config.hidden_size, dtype, device)
        self.logits_processor = LogitsProcessor(config)
        self.to(device)

    def sequence_state_spec(self) -> dict:
        cfg = self.config
        matrices = {r: s for r, s in enumerate(cfg.recurrent_layer_shapes) if s is not None}
        vectors = {r: self.model.layers[cfg.layer_runs[r]].mixer.memory.state_vectors() for r in matrices}
        return dict(layer_num=0, hidden=cfg.hidden_size, matrices=matrices, vectors=vectors)

    @torch.no_grad()
    def forward(self, input_ids, positions, forward_batch):
        hidden_states = self.model(input_ids, positions, forward_batch)
        return self.logits_processor(input_ids, hidden_states, self.lm_head, forward_batch)

    @torch.no_grad()
    def load_weights(self, weights: Dict[str, torch.Tensor]) -> None:
        """Checkpoint names: embed, head, final.norm, l<i>.{norm1, norm1b}, with a feed-forward l<i>.{norm2, norm2b}; a latent
        attention's l<i>.mix.{q, dkv, dkv.norm, uk, uv, o}; an mlstm's l<i>.mix.{q, k, v, g, i, i.b, f, f.b, norm, o}; dense
        l<i>.mlp.{up, down}; moe l<i>.mlp.{router, e<j>.gate, e<j>.up, e<j>.down, shared.gate, shared.up, shared.down, shared.sg};
        linear weights [out, in].  Projections that read the same rows are stacked, the experts' weights are stacked per layer, uk
        and uv are split per head."""

        def put(param, value):
            assert tuple(param.shape) == tuple(value.shape), f"shape {tuple(value.shape)} for a parameter {tuple(param.shape)}"
            param.data.copy_(value.to(dtype=param.dtype), non_blocking=True)

        def stack(*names):
            return torch.cat([weights[n] for n in names], 0)

        m = self.model
        put(m.embed, weights["embed"])
        put(m.norm.weight, weights["final.norm"])
        put(self.lm_head.weight, weights["head"])
        for i, layer in enumerate(m.layers):
            p, mx, mlp = f"l{i}.", layer.mixer, layer.mlp
            x = p + "mix."
            put(layer.norm1, weights[p + "norm1"])
            put(layer.add1.weight, weights[p + "norm1b"])
            if layer.kind == "latent_attention":
                put(mx.in_proj.weight, stack(x + "q", x + "dkv"))
                put(mx.kv_norm, weights[x + "dkv.norm"])
                put(mx.uk.weight, weights[x + "uk"].view(mx.H, mx.dn, mx.rank).transpose(1, 2))
                put(mx.uv.weight, weights[x + "uv"].view(mx.H, mx.dv, mx.rank))
            else:
                put(mx.in_proj.weight, stack(x + "q", x + "k", x + "v", x + "g"))
                put(mx.gate_weight, stack(x + "i", x + "f"))
                put(mx.memory.in_bias, weights[x + "i.b"])
                put(mx.memory.forget_bias, weights[x + "f.b"])
                put(mx.norm_gate.weight, weights[x + "norm"])
            put(mx.o_proj.weight, weights[x + "o"])
            if mlp is None:
                continue
            put(layer.norm2, weights[p + "norm2"])
            put(layer.add2.weight, weights[p + "norm2b"])
            y = p + "mlp."
            if isinstance(mlp, SilatarMLP):
                put(mlp.up.weight, weights[y + "up"])
                put(mlp.down.weight, weights[y + "down"])
                continue
            put(mlp.experts.w_up, torch.stack([stack(f"{y}e{e}.gate", f"{y}e{e}.up") for e in range(mlp.E)]))
            put(mlp.experts.w_down, torch.stack([weights[f"{y}e{e}.down"] for e in range(mlp.E)]))
            if mlp.shared_down is None:
                put(mlp.gate_weight, weights[y + "router"])
            else:
                put(mlp.gate_weight, stack(y + "router", y + "shared.sg"))
                put(mlp.shared_gate_up.weight, stack(y + "shared.gate", y + "shared.up"))
                put(mlp.shared_down.weight, weights[y + "shared.down"])
        self.process_weights_after_loading()

    def process_weights_after_loading(self) -> None:
        for module in self.modules():
            if isinstance(module, ReplicatedLinear):
                module.quant_method.process_weights_after_loading(module)
            elif isinstance(module, PerHeadLinear):
                module.process_weights_after_loading()

    @torch.no_grad()
    def init_random_weights(self, seed: int = 0, std: float = 0.02) -> None:
        dev = self.lm_head.weight.device
        g = torch.Generator(device=dev).manual_seed(seed)
        for name, p in self.named_parameters():
            w = torch.randn(p.shape, generator=g, device=p.device, dtype=torch.float32)
            if name.endswith("norm1") or name.endswith("norm2") or name.endswith("kv_norm") or name.endswith("norm.weight") \
                    or name.endswith("add1.weight") or name.endswith("add2.weight") or name.endswith("norm_gate.weight"):
                p.data.copy_((1.0 + 0.1 * w).to(p.dtype))
            elif name.endswith("forget_bias"):
                p.data.copy_((3.0 + 0.5 * w).to(p.dtype))       # memories that last
            elif name.endswith("in_bias"):
                p.data.copy_((0.5 * w).to(p.dtype))
            elif name.endswith("embed"):
                p.data.copy_(w.to(p.dtype))
            else:
                p.data.copy_((w * (std if p.dim() < 2 else p.shape[-1] ** -0.5)).to(p.dtype))
        self.process_weights_after_loading()
