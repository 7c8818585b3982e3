"""Norms of a model that normalises AFTER the residual sum, on an fp32 residual stream (no counterpart in the
reference, whose models norm before their sublayers and keep the residual in the activation dtype):

  GroupRMSNorm        x <- N(c x + branch) * w in place, N = RMS norm over `groups` equal consecutive parts of the row,
                      each divided by its own sqrt(mean(part^2) + eps).  The branch is a [T, D] tensor or a weighted sum
                      of rows of a larger tensor (the chosen experts' outputs of a mixture).  One launch, which also
                      writes the activation-dtype copy of the new x that the next projections read.
  NormedResidualAdd   x <- x + mult * ls * y / sqrt(mean(y^2) + eps) * (offset + w) in place, same second output: a norm on a
                      sublayer's OUTPUT; offset 1 for a weight stored around zero, ls an optional per-channel layer scale.
  LayerNormResidualAdd  x <- x + LN(y) w in place, LN the layer norm without bias, and in the same launch the layer norm in front
                      of whatever reads the stream next: h = LN(x) w_next.  y may be the sum of a token's expert rows plus a
                      gated second branch.  Which norm comes next is the caller's: layers may run in another order than they
                      are stored in.
  RMSNormResidualAdd  the same sandwich with RMS norms: x <- x + N(y) w, h = N(x) w_next, N(y) = y / sqrt(mean(y^2) + eps).  y may be a
                      token's expert rows times factors; without a next norm h is x in the activation dtype if asked for.
  PassEntry           the start of a pass over layers that run several times: x <- W [x; e] + step_t, e the token's embedding.  W
                      acts on the two halves separately, so the embedding's part is one fp32 row per vocabulary entry, made
                      when weights are loaded, and a pass multiplies by the stream's half alone; the sum, and the first norm of
                      the pass, are one launch.

groups, eps and c are constructor arguments; all arithmetic is fp32 whatever the activation dtype."""
from typing import Optional

import torch
from torch import nn

from ..ops_backend import get_ops
from .linear import ReplicatedLinear


class GroupRMSNorm(nn.Module):
    def __init__(self, hidden: int, groups: int, eps: float, dtype, device, residual_scale: float = 1.0):
        super().__init__()
        assert groups >= 1 and hidden % groups == 0
        self.groups, self.eps, self.residual_scale = int(groups), float(eps), float(residual_scale)
        self.weight = nn.Parameter(torch.ones(hidden, dtype=dtype, device=device), requires_grad=False)

    def forward(self, x: torch.Tensor, branch: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None,
                coef: Optional[torch.Tensor] = None) -> torch.Tensor:
        """x fp32 [T, D], updated in place; returns its copy in the weight's dtype.  rows int32 [T, n] / coef fp32 [T, n]:
        the branch of token t is sum_j coef[t, j] * branch[rows[t, j]]."""
        return get_ops().scaled_add_group_rmsnorm(x, branch, self.residual_scale, self.weight.data, self.groups, self.eps,
                                                  rows=rows, coef=coef, inplace=True)

    def normed(self, x: torch.Tensor) -> torch.Tensor:
        """N(x) * w in the weight's dtype; x is left as it is (a model's last norm)."""
        return get_ops().scaled_add_group_rmsnorm(x, None, 1.0, self.weight.data, self.groups, self.eps, inplace=False)


class NormedResidualAdd(nn.Module):
    def __init__(self, hidden: int, eps: float, dtype, device, offset: float = 0.0, mult: float = 1.0, layer_scale: bool = False):
        super().__init__()
        self.eps, self.offset, self.mult = float(eps), float(offset), float(mult)
        self.weight = nn.Parameter((torch.zeros if offset else torch.ones)(hidden, dtype=dtype, device=device), requires_grad=False)
        self.layer_scale = nn.Parameter(torch.ones(hidden, dtype=dtype, device=device), requires_grad=False) if layer_scale else None

    def forward(self, x: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
        if self.offset == 0.0 and self.mult == 1.0 and self.layer_scale is None:
            return get_ops().rmsnorm_residual_add(x, y, self.weight.data, self.eps)
        return get_ops().rmsnorm_residual_add(x, y, self.weight.data, self.eps, offset=self.offset, mult=self.mult,
                                              layer_scale=self.layer_scale.data if self.layer_scale is not None else None)


class LayerNormResidualAdd(nn.Module):
    def __init__(self, hidden: int, eps: float, dtype, device):
        super().__init__()
        self.eps = float(eps)
        self.weight = nn.Parameter(torch.ones(hidden, dtype=dtype, device=device), requires_grad=False)

    def forward(self, x: torch.Tensor, y: torch.Tensor, next_weight: Optional[torch.Tensor], rows: Optional[torch.Tensor] = None,
                y2: Optional[torch.Tensor] = None, y2_gate: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
        """x fp32 [T, D], updated in place; returns LN(x) * next_weight in the weight's dtype."""
        return get_ops().layernorm_residual_add(x, y, self.weight.data, next_weight, self.eps, rows=rows, y2=y2, y2_gate=y2_gate)


class RMSNormResidualAdd(nn.Module):
    def __init__(self, hidden: int, eps: float, dtype, device):
        super().__init__()
        self.eps = float(eps)
        self.weight = nn.Parameter(torch.ones(hidden, dtype=dtype, device=device), requires_grad=False)

    def forward(self, x: torch.Tensor, y: torch.Tensor, next_weight: Optional[torch.Tensor], rows: Optional[torch.Tensor] = None,
                coef: Optional[torch.Tensor] = None) -> torch.Tensor:
        """x fp32 [T, D], updated in place; returns N(x) * next_weight, or x (next_weight None), in the weight's dtype."""
        return get_ops().rmsnorm_residual_add_next(x, y, self.weight.data, next_weight, self.eps, rows=rows, coef=coef, copy=True)


class PassEntry(nn.Module):
    def __init__(self, hidden: int, times: int, vocab: int, eps: float, dtype, device):
        super().__init__()
        self.eps = float(eps)
        self.stream_proj = ReplicatedLinear(hidden, hidden, dtype, device)       # the half of W that reads the stream
        self.step = nn.Parameter(torch.zeros(times, hidden, dtype=torch.float32, device=device), requires_grad=False)
        self.embed_table = nn.Parameter(torch.zeros(vocab, hidden, dtype=torch.float32, device=device), requires_grad=False)

    def set_weights(self, w: torch.Tensor, step: torch.Tensor, embed: torch.Tensor) -> None:
        """w [hidden, 2 hidden] = [stream | embedding], embed [vocab, hidden] as the model reads it."""
        D = self.step.shape[1]
        assert w.shape == (D, 2 * D) and step.shape == self.step.shape and embed.shape == self.embed_table.shape
        dev, dt = self.embed_table.device, self.stream_proj.weight.dtype
        self.stream_proj.weight.data.copy_(w[:, :D].to(dt))
        self.step.data.copy_(step.to(torch.float32))
        half = w[:, D:].to(device=dev, dtype=dt).float().contiguous()
        for lo in range(0, embed.shape[0], 8192):
            rows = embed[lo: lo + 8192].to(device=dev, dtype=dt).float().contiguous()
            self.embed_table.data[lo: lo + 8192] = get_ops().linear(rows, half)

    def forward(self, x: torch.Tensor, h: torch.Tensor, input_ids: torch.Tensor, t: int, next_weight: torch.Tensor) -> torch.Tensor:
        """x fp32 [T, D], replaced in place; h its copy in the activation dtype; returns N(x) * next_weight."""
        y = self.stream_proj(h)[0]
        return get_ops().pass_entry(x, y, self.embed_table.data, input_ids, self.step.data[t], next_weight, self.eps)
