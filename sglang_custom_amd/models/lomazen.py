"""Lomazen: a decoder-only model on an fp32 residual stream with an RMS norm on BOTH sides of every sublayer,
x <- x + N(mixer(N(x))), x <- x + N(ff(N(x))), some of whose layers run several times in a row with the same weights; every such
pass starts from a projection of the stream and the token's embedding, plus a vector of its own.  The mixer is, layer by layer,

  attention     grouped causal softmax attention: queries and keys rotated in neighbouring features with banded frequencies and
                divided by their root mean square, scores capped by a tanh, the result gated feature by feature.
  attention_2   the difference of two softmax attentions over the same values (rotation in halves), divided by its root mean square
                per head, gated head by head.

The feed-forward is dense with a tanh-GELU gate, a mixture of squared-relu experts weighted by their softmax scores, or absent.
The head is the embedding table; logits are multiplied by a constant.  (No counterpart in the reference; the module layout
follows its model files, python/sglang/srt/models/llama.py.)

Per layer run (T tokens, width D), besides the GEMMs' own launches:

  mixer               in_proj [q | k | v | gate]; CausalAttention.rotate_and_write (rotation, norms, cache rows); CausalAttention
                      (both maps, their difference, its norm and the gate inside); o                     2 launches
  RMSNormResidualAdd  x += N(y) in place, and the norm in front of the next sublayer                     1 launch, fp32
  dense               gate | up, gated unit, down
  moe                 router logits in unrounded fp32, route, align, grouped GEMM (squared relu in it), grouped GEMM; the weighted
                      sum over a token's experts happens in the RMSNormResidualAdd that follows
  PassEntry           one product of the stream's half; embedding half, sum and the next norm in one launch

Norms, positions and angles, attention scores / weights, router and the residual sum are fp32 in every dtype; `dtype` is what
the projections read and write.  Caches belong to layer RUNS: run r of the configuration's layer_runs uses cache layer r, whichever
layer's weights it reads.  Every size comes from the configuration, layer by layer.  Nothing but cache rows is kept per sequence, so
the prefix cache and captured decode steps serve this family.  Tensor parallelism is not implemented for it (its head counts need
not divide)."""
from typing import Dict

import torch
from torch import nn

from ..distributed.parallel_state import get_tensor_model_parallel_world_size
from ..layers.activation import GeluTanhAndMul
from ..layers.causal_attention import CausalAttention
from ..layers.linear import ReplicatedLinear
from ..layers.logits_processor import LogitsProcessor
from ..layers.moe import GroupedExperts, GroupedTopKRouter
from ..layers.post_norm import PassEntry, RMSNormResidualAdd
from ..layers.pre_norm import OffsetRMSNorm
from ..layers.rotary_embedding import banded_pair_inv_freq
from ..layers.vocab_parallel_embedding import ParallelLMHead
from ..ops_backend import get_ops


class LomazenAttention(nn.Module):
    """Both mixers: maps 1 (unit-norm queries and keys, capped scores, a gate per feature) or 2 (their difference, a gate per head)."""

    def __init__(self, hidden: int, mx: dict, maps: int, eps: float, dtype, device):
        super().__init__()
        H, d = mx["heads"], mx["dim"]
        G, dv = mx.get("kv_heads", H), mx.get("vdim", d)
        self.H, self.dv, self.maps = H, dv, maps
        self.widths = (H * maps * d, G * maps * d, G * dv, H * dv if maps == 1 else H)      # q | k | v | gate
        # whole groups of eight rows, so that the rows of the projection's result stay 16-byte aligned
        self.in_proj = ReplicatedLinear(hidden, -(-sum(self.widths) // 8) * 8, dtype, device)
        self.o_proj = ReplicatedLinear(H * dv, hidden, dtype, device)
        rot = mx.get("rot") or {}
        dims = int(rot.get("dims", 0))
        self.diff = float(mx["diff"]) if maps == 2 else None
        if maps == 2:
            # fp32 whatever the model dtype: lambda is exp(lq1 . lk1) - exp(lq2 . lk2) + diff
            self.lambda_vectors = nn.Parameter(torch.zeros(4, d, dtype=torch.float32, device=device), requires_grad=False)
        self.attn = CausalAttention(H, G, d, dv, mx["scale"], device, maps=maps, score_cap=float(mx.get("softcap") or 0.0) if maps == 1 else 0.0,
                                    rot_dims=dims, inv_freq=banded_pair_inv_freq(rot["base"], dims, rot.get("scaling")) if dims else None,
                                    interleaved=maps == 1, unit_norm=maps == 1, eps=eps, out_scale=1.0 - self.diff if maps == 2 else 1.0)

    def set_lambda(self) -> None:
        if self.maps == 2:
            lq1, lk1, lq2, lk2 = self.lambda_vectors.data.double().cpu()
            self.attn.map_factor = float(torch.exp((lq1 * lk1).sum()) - torch.exp((lq2 * lk2).sum()) + self.diff)

    def forward(self, positions, h, forward_batch, run: int):
        T, (nq, nk, nv, ng) = h.shape[0], self.widths
        p = self.in_proj(h)[0]
        q = self.attn.rotate_and_write(p[:, :nq], p[:, nq: nq + nk], p[:, nq + nk: nq + nk + nv], positions, forward_batch, run)
        o = torch.empty((T, self.H, self.dv), dtype=h.dtype, device=h.device)
        self.attn(q, forward_batch, o, run, gate=p[:, nq + nk + nv: nq + nk + nv + ng])
        return self.o_proj(o.view(T, self.H * self.dv))[0]


class LomazenMLP(nn.Module):
    def __init__(self, hidden: int, ff: int, dtype, device):
        super().__init__()
        self.ff = ff
        self.gate_up = ReplicatedLinear(hidden, 2 * ff, dtype, device)
        self.act = GeluTanhAndMul()
        self.down = ReplicatedLinear(ff, hidden, dtype, device)

    def forward(self, h):
        """-> what RMSNormResidualAdd takes besides the stream and the next norm."""
        gu = self.gate_up(h)[0]
        return dict(y=self.down(self.act(gu[:, : self.ff], gu[:, self.ff:]))[0])


class LomazenMoE(nn.Module):
    def __init__(self, hidden: int, mlp: dict, dtype, device):
        super().__init__()
        r = mlp["router"]
        self.E = r["experts"]
        self.gate_weight = nn.Parameter(torch.zeros(self.E, hidden, dtype=dtype, device=device), requires_grad=False)
        self.router = GroupedTopKRouter(hidden, self.E, r["top"], 1, 1, 1.0, device, score_fn="softmax", group_best=1, renorm=False,
                                        with_correction=False, with_weight=False)
        self.experts = GroupedExperts(hidden, mlp["expert"]["ff"], self.E, dtype, device, activation="relu2")

    def forward(self, h):
        ids, weights = self.router.route(get_ops().project_f32(h, self.gate_weight.data))
        y, rows = self.experts(h, ids)
        return dict(y=y, rows=rows, coef=weights)


class LomazenDecoderLayer(nn.Module):
    def __init__(self, config, layer_id: int, dtype, device):
        super().__init__()
        spec = config.layer_specs[layer_id]
        D, eps, mlp = config.hidden_size, config.rms_norm_eps, spec.get("mlp")
        self.norm1 = nn.Parameter(torch.ones(D, dtype=dtype, device=device), requires_grad=False)
        self.mixer = LomazenAttention(D, spec["mixer"], 2 if spec["type"] == "attention_2" else 1, eps, dtype, device)
        self.add1 = RMSNormResidualAdd(D, eps, dtype, device)
        self.mlp = None
        if mlp is not None:
            self.norm2 = nn.Parameter(torch.ones(D, dtype=dtype, device=device), requires_grad=False)
            self.mlp = LomazenMLP(D, mlp["ff"], dtype, device) if mlp["kind"] == "dense" else LomazenMoE(D, mlp, dtype, device)
            self.add2 = RMSNormResidualAdd(D, eps, dtype, device)

    def forward(self, positions, x, h, forward_batch, run: int, next_norm):
        """x: the fp32 stream, updated in place; h: its normed copy for the mixer; next_norm: the weight of the norm that reads the
        stream after this run, or None where a pass starts.  Returns that norm's result, or the stream in the activation dtype."""
        y = self.mixer(positions, h, forward_batch, run)
        h = self.add1(x, y, self.norm2.data if self.mlp is not None else next_norm)
        if self.mlp is not None:
            h = self.add2(x, next_weight=next_norm, **self.mlp(h))
        return h


class LomazenModel(nn.Module):
    def __init__(self, config, dtype, device):
        super().__init__()
        D, eps = config.hidden_size, config.rms_norm_eps
        self.layer_runs, self.pass_starts = list(config.layer_runs), list(config.pass_starts)
        self.embed = nn.Parameter(torch.zeros(config.vocab_size, D, dtype=dtype, device=device), requires_grad=False)
        self.layers = nn.ModuleList([LomazenDecoderLayer(config, i, dtype, device) for i in range(len(config.layer_specs))])
        self.entry = PassEntry(D, config.loop_times, config.vocab_size, eps, dtype, device) if config.loop_times else None
        self.norm = OffsetRMSNorm(D, eps, dtype, device, offset=0.0)
        self.capture_streams = None     # a list here receives the fp32 residual after every layer run (tests, debugging)

    def forward(self, input_ids, positions, forward_batch):
        h = get_ops().embedding(input_ids, self.embed.data)
        x = h.float() if h.dtype != torch.float32 else h.clone()
        runs = [self.layers[i] for i in self.layer_runs]
        # the norm in front of every run and the last one; None: a pass starts there, which wants the stream itself
        norms = [None if t is not None else layer.norm1.data for layer, t in zip(runs, self.pass_starts)] + [self.norm.weight.data]
        if norms[0] is not None:
            h = get_ops().offset_rmsnorm(x, norms[0], self.norm.eps, 0.0)
        for r, layer in enumerate(runs):
            if self.pass_starts[r] is not None:
                h = self.entry(x, h, input_ids, self.pass_starts[r], layer.norm1.data)
            h = layer(positions, x, h, forward_batch, r, norms[r + 1])
            if self.capture_streams is not None:
                self.capture_streams.append(x.clone())
        return h


class LomazenForCausalLM(nn.Module):
    supports_hip_graph = True     # padded rows of a captured step attend to the request table's row 0 and write the sink slot

    def __init__(self, config, dtype=torch.bfloat16, device="cuda", quant_method_factory=None):
        super().__init__()
        if quant_method_factory is not None:
            raise NotImplementedError("Lomazen runs unquantised (its norms, router and residual are fp32 by design)")
        if get_tensor_model_parallel_world_size() != 1:
            raise NotImplementedError("Lomazen: tensor parallelism is not implemented")
        self.config = config
        self.dtype = dtype
        self.needs_sequence_state = False
        self.model = LomazenModel(config, dtype, device)
        self.lm_head = ParallelLMHead(config.vocab_size, config.hidden_size, dtype, device)
        self.lm_head.weight = self.model.embed
        self.logits_processor = LogitsProcessor(config, logit_scale=config.logit_scale if config.logit_scale != 1.0 else None)
        self.to(device)

    @torch.no_grad()
    def forward(self, input_ids, positions, forward_batch):
        hidden_states = self.model(input_ids, positions, forward_batch)
        return self.logits_processor(input_ids, hidden_states, self.lm_head, forward_batch)

    @torch.no_grad()
    def load_weights(self, weights: Dict[str, torch.Tensor]) -> None:
        """Checkpoint names: embed, final.norm, with a loop loop.in [D, 2 D] (stream first) and loop.step [passes, D]; l<i>.{norm1,
        norm1b}, with a feed-forward l<i>.{norm2, norm2b}; l<i>.mix.{q, k, v, g, o}, of an attention_2 also l<i>.mix.{lq1, lk1, lq2,
        lk2}; dense l<i>.mlp.{gate, up, down}; moe l<i>.mlp.{router, e<j>.up, e<j>.down}; linear weights [out, in].  Projections that
        read the same rows are stacked, the experts' weights are stacked per layer."""

        def put(param, value):
            assert tuple(param.shape) == tuple(value.shape), f"shape {tuple(value.shape)} for a parameter {tuple(param.shape)}"
            param.data.copy_(value.to(dtype=param.dtype), non_blocking=True)

        def stack(*names):
            return torch.cat([weights[n] for n in names], 0)

        m = self.model
        put(m.embed, weights["embed"])
        put(m.norm.weight, weights["final.norm"])
        if m.entry is not None:
            m.entry.set_weights(weights["loop.in"], weights["loop.step"], weights["embed"])
        for i, layer in enumerate(m.layers):
            p, mx, mlp = f"l{i}.", layer.mixer, layer.mlp
            x = p + "mix."
            put(layer.norm1, weights[p + "norm1"])
            put(layer.add1.weight, weights[p + "norm1b"])
            for n, rows in zip("qkvg", mx.widths):
                assert weights[x + n].shape[0] == rows, f"{x + n}: {tuple(weights[x + n].shape)} for {rows} rows"
            w = stack(x + "q", x + "k", x + "v", x + "g")
            pad = mx.in_proj.weight.shape[0] - w.shape[0]
            put(mx.in_proj.weight, torch.cat([w, w.new_zeros(pad, w.shape[1])]) if pad else w)
            put(mx.o_proj.weight, weights[x + "o"])
            if mx.maps == 2:
                put(mx.lambda_vectors, torch.stack([weights[x + n].float() for n in ("lq1", "lk1", "lq2", "lk2")]))
            if mlp is None:
                continue
            put(layer.norm2, weights[p + "norm2"])
            put(layer.add2.weight, weights[p + "norm2b"])
            y = p + "mlp."
            if isinstance(mlp, LomazenMLP):
                put(mlp.gate_up.weight, stack(y + "gate", y + "up"))
                put(mlp.down.weight, weights[y + "down"])
                continue
            put(mlp.gate_weight, weights[y + "router"])
            put(mlp.experts.w_up, torch.stack([weights[f"{y}e{e}.up"] for e in range(mlp.E)]))
            put(mlp.experts.w_down, torch.stack([weights[f"{y}e{e}.down"] for e in range(mlp.E)]))
        self.process_weights_after_loading()

    def process_weights_after_loading(self) -> None:
        for module in self.modules():
            if isinstance(module, ReplicatedLinear):
                module.quant_method.process_weights_after_loading(module)
            elif isinstance(module, LomazenAttention):
                module.set_lambda()

    @torch.no_grad()
    def init_random_weights(self, seed: int = 0, std: float = 0.02) -> None:
        dev = self.lm_head.weight.device
        g = torch.Generator(device=dev).manual_seed(seed)
        for name, p in self.named_parameters():
            if name.endswith("embed_table"):
                continue                      # made from the weights below
            w = torch.randn(p.shape, generator=g, device=p.device, dtype=torch.float32)
            if name.endswith("norm1") or name.endswith("norm2") or name.endswith("norm.weight") or name.endswith("add1.weight") \
                    or name.endswith("add2.weight"):
                p.data.copy_((1.0 + 0.1 * w).to(p.dtype))
            elif name.endswith("lambda_vectors"):
                p.data.copy_(0.1 * w)
            elif name.endswith("embed") or name.endswith("lm_head.weight"):
                p.data.copy_(w.to(p.dtype))
            else:
                p.data.copy_((w * (std if p.dim() < 2 else p.shape[-1] ** -0.5)).to(p.dtype))
        if self.model.entry is not None:
            D = self.config.hidden_size
            w_in = torch.randn(D, 2 * D, generator=g, device=dev, dtype=torch.float32) * (2 * D) ** -0.5
            self.model.entry.set_weights(w_in.to(self.dtype), self.model.entry.step.data.clone(), self.model.embed.data)
        self.process_weights_after_loading()
