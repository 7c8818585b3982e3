"""CausalAttention: the per-layer hand-off to the attention backend for softmax attention over every earlier token whose cached
keys and values have per-layer widths (RadixAttention's role, python/sglang/srt/layers/radix_attention.py:59-108, for mechanisms
the reference does not have):

    s_j = (q_i . k_j) * scale,   cap > 0: s_j <- cap tanh(s_j / cap),   a = softmax over j <= i of s_j, times v_j

with one or two score maps per head over the same values.  Two maps (difference attention): a_1 - lambda a_2, divided by its
root mean square (eps), times out_scale; lambda is one number per layer, set when weights are loaded.  The result may be
multiplied by the sigmoid of a logit per head or per feature.

rotate_and_write() comes first: queries and keys rotated (first rot_dims features of every map; neighbouring features or halves)
and, with unit_norm, divided by their root mean square; keys and values go to their cache rows.  A call names the cache layer it
works on: one set of weights can run several times per step over rows of its own.  Scores and weights are fp32 in every
dtype."""
from typing import Optional

import torch
from torch import nn

from ..ops_backend import get_ops


class CausalAttention(nn.Module):
    def __init__(self, num_heads: int, num_kv_heads: int, head_dim: int, v_head_dim: int, scaling: float, device, maps: int = 1,
                 score_cap: float = 0.0, rot_dims: int = 0, inv_freq: Optional[torch.Tensor] = None, interleaved: bool = False,
                 unit_norm: bool = False, eps: float = 1e-6, out_scale: float = 1.0):
        super().__init__()
        assert num_heads % num_kv_heads == 0 and maps in (1, 2) and 0 <= rot_dims <= head_dim and rot_dims % 2 == 0
        self.tp_q_head_num, self.tp_k_head_num, self.tp_v_head_num = num_heads, num_kv_heads, num_kv_heads
        self.qk_head_dim, self.v_head_dim, self.maps = head_dim, v_head_dim, int(maps)
        self.scaling, self.score_cap, self.eps = float(scaling), float(score_cap or 0.0), float(eps)
        self.rot_dims, self.interleaved, self.unit_norm = int(rot_dims), bool(interleaved), bool(unit_norm)
        self.map_factor, self.out_scale = 0.0, float(out_scale)
        self.register_buffer("inv_freq", (torch.zeros(1) if inv_freq is None else inv_freq.to(torch.float32)).to(device), persistent=False)

    def rotate_and_write(self, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, positions: torch.Tensor, forward_batch,
                         cache_layer: int) -> torch.Tensor:
        """q [T, H * maps * d], k [T, G * maps * d], v [T, G * dv] (column blocks of one projection) -> queries [T, H, maps, d]."""
        T, d = q.shape[0], self.qk_head_dim
        k_cache, v_cache = forward_batch.token_to_kv_pool.get_kv_buffer(cache_layer)
        out = get_ops().qkv_rotate_write(q.unflatten(1, (self.tp_q_head_num * self.maps, d)), k.unflatten(1, (self.tp_k_head_num * self.maps, d)), v,
                                         positions, self.inv_freq, self.rot_dims, self.interleaved, self.unit_norm, self.eps, k_cache, v_cache,
                                         forward_batch.out_cache_loc)
        return out.view(T, self.tp_q_head_num, self.maps, d)

    def forward(self, q: torch.Tensor, forward_batch, out: torch.Tensor, cache_layer: int, gate: Optional[torch.Tensor] = None) -> torch.Tensor:
        return forward_batch.attn_backend.forward_causal(q, self, forward_batch, out, cache_layer, gate=gate)
