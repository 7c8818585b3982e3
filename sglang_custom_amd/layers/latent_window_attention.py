"""LatentWindowAttention: the per-layer hand-off to the attention backend for attention over a latent KV cache, over a
sliding window with a softmax sink or over every earlier token (RadixAttention's role,
python/sglang/srt/layers/radix_attention.py:59-108, for a mechanism the reference does not have).  Holds what the backend
reads: head count, latent rank, rope width, how many of the rope features rotate, at which frequencies, in which pairing and
with which magnitude, window (0: none), scale, layer id, and the per-head sink (or none).

The heads share one cache row per token, [c (rank) | rotated rope key]; queries come in absorbed form (q_nope W_uk
per head, rank wide) with their rope part unrotated, and the result per head is the attention-weighted sum of c,
times sigmoid(gate) when gate logits are given.  A call may name the cache layer it works on: one set of weights can then run
several times per step over rows of their own."""
from typing import Optional

import torch
from torch import nn

from ..ops_backend import get_ops
from .rotary_embedding import rotate_half_inv_freq


class LatentWindowAttention(nn.Module):
    def __init__(self, num_heads: int, kv_rank: int, rope_dim: int, scaling: float, window: int, layer_id: int,
                 rot_dims: int, rot_base: float, device, with_sink: bool = True, interleaved: bool = False,
                 inv_freq: Optional[torch.Tensor] = None, rot_mag: float = 1.0):
        """inv_freq: the rotation's frequencies when they are not rot_base^(-2 i / rot_dims), with rot_mag the factor on cos and
        sin that comes with them; interleaved: feature 2 i turns with 2 i + 1 instead of i with i + rot_dims / 2."""
        super().__init__()
        assert 0 <= rot_dims <= rope_dim and rot_dims % 2 == 0 and window >= 0
        self.tp_q_head_num = num_heads
        self.kv_rank = kv_rank
        self.rope_dim = rope_dim
        self.rot_dims = rot_dims
        self.scaling = float(scaling)
        self.window = int(window)
        self.layer_id = layer_id
        self.interleaved, self.rot_mag = bool(interleaved), float(rot_mag)
        self.sink = nn.Parameter(torch.zeros(num_heads, dtype=torch.float32, device=device), requires_grad=False) if with_sink else None
        freqs = rotate_half_inv_freq(rot_base, rot_dims) if inv_freq is None else inv_freq.to(torch.float32)
        self.register_buffer("inv_freq", freqs.to(device), persistent=False)

    def write_rows(self, a: torch.Tensor, q_cols: int, kv_weight: torch.Tensor, eps: float, positions: torch.Tensor, forward_batch,
                   cache_layer: Optional[int] = None) -> None:
        """The step's cache rows from a = [q_cols columns left alone | kv latent | rope key | ...]."""
        cache = forward_batch.token_to_kv_pool.get_key_buffer(self.layer_id if cache_layer is None else cache_layer)
        get_ops().latent_rows_write(a, q_cols, kv_weight, positions, forward_batch.out_cache_loc, self.inv_freq, cache, self.kv_rank,
                                    self.rope_dim, self.rot_dims, self.interleaved, self.rot_mag, eps)

    def forward(self, qa: torch.Tensor, qr: torch.Tensor, gate, forward_batch, out: torch.Tensor,
                cache_layer: Optional[int] = None) -> torch.Tensor:
        return forward_batch.attn_backend.forward_latent_window(qa, qr, gate, self, forward_batch, out, cache_layer=cache_layer)
