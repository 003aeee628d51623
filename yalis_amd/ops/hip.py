"""The kernel library: ctypes bindings of the HIP kernels in ``yalis_amd/csrc``.

Every method takes torch tensors on the GPU, checks what the kernels assume, and
launches on torch's current stream.  There is no other implementation behind these
methods: when the library cannot be built or loaded, constructing ``HipOps``
raises.  Plain matrix products of many rows in bfloat16 go to the vendor library
(hipBLASLt, called from ``csrc/library_gemm.hip``; the reference uses cuBLAS in the same
places, yalis/external/model.py:449,462-466,717-722); few-row products, every float32
product and everything else are the hand-written kernels.
"""
from __future__ import annotations

import ctypes
from typing import Optional, Tuple

import torch

from .build import load_kernels

_F32, _BF16 = 0, 1
_c_int = ctypes.c_int
_c_float = ctypes.c_float
_c_size_t = ctypes.c_size_t
_c_u64 = ctypes.c_ulonglong
_vp = ctypes.c_void_p


class KernelError(RuntimeError):
    pass


class StaleWorkspace(KernelError):
    """A result that lives in the library's workspace was consumed after the workspace had
    been handed to a later launch."""


def _code(dtype: torch.dtype) -> int:
    if dtype == torch.float32:
        return _F32
    if dtype == torch.bfloat16:
        return _BF16
    raise KernelError(f"kernels take float32 and bfloat16 only, got {dtype}")


def _ptr(t: Optional[torch.Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


_SIGNATURES = {
    "yk_abi_version": ([], _c_int),
    "yk_cache_tiled": ([_c_int, _c_int, _c_int], _c_int),
    "yk_embed": ([_vp, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _c_float, _vp], _c_int),
    "yk_add_rmsnorm": (
        [_vp, _vp, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_float, _c_int, _vp, _c_int, _vp, _vp],
        _c_int,
    ),
    "yk_rope_append": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp,
         _c_int, _c_int, _c_int, _vp, _vp, _vp, _c_int, _vp],
        _c_int,
    ),
    "yk_add_bias": ([_vp, _c_int, _c_int, _vp, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _vp], _c_int),
    "yk_gated_act": ([_vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_float, _vp], _c_int),
    "yk_norm_add": (
        [_vp, _vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_float, _vp, _c_int, _c_int, _c_float, _vp, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_sum_norm": (
        [_vp, _vp, _c_int, _c_int, _c_int, _c_float, _vp, _vp, _c_int, _c_int, _c_int, _c_float, _vp, _c_float, _vp, _c_float, _vp, _c_int,
         _c_int, _c_float, _vp, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_embed_pairs": (
        [_vp, _vp, _c_int, _c_int, _c_float, _vp, _c_int, _c_u64, _c_u64, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_token_shift_mix": ([_vp, _c_int, _vp, _c_int, _vp, _vp, _vp, _vp, _vp, _vp, _c_int, _c_int, _vp], _c_int),
    "yk_low_rank": ([_vp, _c_int, _c_int, _vp, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _vp], _c_int),
    "yk_act_rows": ([_vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_int, _vp], _c_int),
    "yk_gemm_mfma_skinny_grouped": (
        [_vp, _c_size_t, _c_int, _vp, _vp, _c_int, _vp, _c_size_t, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_round_rows": ([_vp, _vp, _c_int, _c_size_t, _vp], _c_int),
    "yk_qkv_prepare": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _c_int,
         _c_int, _c_float, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_float, _vp, _vp, _c_int, _c_int, _vp, _vp, _vp, _c_int,
         _c_int, _vp, _vp, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_qk_row_scales": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _c_int, _c_float, _vp, _c_float, _c_int, _vp, _vp],
        _c_int,
    ),
    "yk_attn_masked": (
        [_vp, _c_int, _vp, _vp, _vp, _c_int, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float,
         _c_float, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp,
         _c_int, _vp, _c_int, _c_int, _c_float, _c_float, _c_float, _vp],
        _c_int,
    ),
    "yk_attn_finish": (
        [_vp, _c_int, _vp, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int,
         _vp],
        _c_int,
    ),
    "yk_causal_conv": ([_vp, _c_int, _c_int, _vp, _vp, _c_int, _vp, _vp, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp], _c_int),
    "yk_sandwich_norm": (
        [_vp, _vp, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _c_float, _c_int, _c_float, _vp, _vp, _c_float, _c_int, _c_int, _vp, _vp,
         _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_activation": ([_vp, _c_int, _c_int, _c_int, _c_int, _vp, _c_int, _c_size_t, _vp], _c_int),
    "yk_scale_rows": ([_vp, _c_float, _c_float, _c_size_t, _vp], _c_int),
    "yk_embed_norm": ([_vp, _vp, _c_int, _c_int, _vp, _c_float, _vp, _c_int, _c_int, _c_int, _vp], _c_int),
    "yk_streams_norm": (
        [_vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_float, _vp, _vp, _vp, _vp, _vp, _vp, _c_int, _c_float,
         _c_int, _vp, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_scan_inputs": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_float, _c_int, _vp, _c_int, _vp],
        _c_int,
    ),
    "yk_decay_scan_chunks_ok": ([_c_int, _c_int, _c_int, _c_int], _c_int),
    "yk_decay_scan_chunks_bytes": ([_c_int, _c_int, _c_int, _c_int, _c_int, _c_int], _c_size_t),
    "yk_decay_scan_chunks": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _vp, _c_int, _vp, _c_int, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_float, _c_int,
         _vp, _vp, _c_size_t, _vp, _vp],
        _c_int,
    ),
    "yk_decay_scan_step": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _c_int, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_float, _c_int, _vp, _vp, _vp],
        _c_int,
    ),
    "yk_moe_router_share": ([_vp, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _c_int, _vp, _vp, _c_int, _vp], _c_int),
    "yk_latent_prepare": (
        [_vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_float, _vp, _c_int, _c_int, _c_int, _vp, _vp, _vp, _vp, _c_int, _c_int, _vp, _vp,
         _c_int, _vp, _c_int, _vp],
        _c_int,
    ),
    "yk_latent_mfma_ok": ([_c_int, _c_int, _c_int], _c_int),
    "yk_latent_mfma_tile_tokens": ([_c_int], _c_int),
    "yk_latent_mfma_workspace": ([_c_int, _c_int, _c_int, _c_int], _c_size_t),
    "yk_latent_attention_mfma": (
        [_vp, _vp, _vp, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_int, _vp, _vp, _c_size_t, _vp, _vp],
        _c_int,
    ),
    "yk_head_linear": (
        [_vp, _c_int, _c_int, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _c_int, _vp, _c_int, _c_int,
         _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_head_linear_mfma_ok": ([_c_int, _c_int, _c_int], _c_int),
    "yk_head_linear_mfma": (
        [_vp, _c_int, _c_int, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _c_int, _vp, _c_int, _c_int,
         _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_latent_tile_tokens": ([_c_int], _c_int),
    "yk_latent_attention": ([_vp, _vp, _c_int, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _vp, _vp, _vp], _c_int),
    "yk_linear_state_scan": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _vp, _c_int, _c_int, _c_float, _c_float, _c_int, _vp, _c_int,
         _c_int, _vp, _vp, _c_float, _vp, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _vp, _vp],
        _c_int,
    ),
    "yk_gated_head_norm": (
        [_vp, _vp, _c_int, _c_float, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_conv_state_push": ([_vp, _c_int, _c_int, _vp, _vp, _vp, _vp, _c_int, _c_int, _c_int, _vp], _c_int),
    "yk_rglru_gates": ([_vp, _c_int, _vp, _vp, _vp, _vp, _vp, _c_int, _c_float, _vp, _vp, _c_int, _c_int, _c_int, _vp, _vp, _vp], _c_int),
    "yk_rglru_gates_mfma_ok": ([_c_int, _c_int], _c_int),
    "yk_rglru_scan_chunked": (
        [_vp, _vp, _vp, _c_int, _vp, _c_int, _c_int, _vp, _vp, _vp, _vp, _vp, _vp, _c_int, _vp, _vp, _vp, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_rglru_scan": ([_vp, _vp, _vp, _c_int, _vp, _c_int, _c_int, _vp, _vp, _vp, _vp, _vp, _vp, _c_int, _c_int, _c_int, _vp], _c_int),
    "yk_moe_max_tiles": ([_c_int, _c_int, _c_int], _c_int),
    "yk_moe_mfma_ok": ([_c_int, _c_int, _c_int], _c_int),
    "yk_moe_router_topk": ([_vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _vp, _vp, _vp], _c_int),
    "yk_moe_combine": ([_vp, _c_int, _c_int, _c_int, _vp, _c_int, _c_float, _vp, _c_int, _c_int, _vp, _vp], _c_int),
    "yk_moe_route": ([_vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _vp, _vp], _c_int),
    "yk_moe_gate_up": (
        [_vp, _c_int, _c_int, _vp, _c_int, _vp, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float,
         _c_float, _vp, _c_int, _vp],
        _c_int,
    ),
    "yk_moe_down": ([_vp, _c_int, _vp, _c_int, _vp, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp], _c_int),
    "yk_gemm_fma": (
        [_vp, _c_int, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_gemm_skinny_splits": ([_c_int, _c_int, _c_int, _c_int], _c_int),
    "yk_gemm_skinny_force": ([_c_int, _c_int, _c_int], _c_int),
    "yk_gemm_skinny_wide": ([_c_int], _c_int),
    "yk_gemm_library": ([_vp, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _c_size_t, _vp, _vp], _c_int),
    "yk_gemm_library_tune": ([_c_int], _c_int),
    "yk_gemm_mfma_skinny": (
        [_vp, _vp, _vp, _c_int, _vp, _c_size_t, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_gemm_tile": (
        [_vp, _vp, _vp, _c_int, _vp, _c_size_t, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_gemm_tile_splits": ([_c_int, _c_int, _c_int], _c_int),
    "yk_gemm_tile_grouped": (
        [_vp, _c_int, _vp, _c_int, _vp, _c_size_t, _c_int, _vp, _c_int, _c_int, _vp, _vp, _vp, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
    "yk_gemm_tile_force": ([_c_int], _c_int),
    "yk_attn_generic": (
        [_vp, _c_int, _vp, _vp, _vp, _c_int, _vp, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_int, _vp],
        _c_int,
    ),
    "yk_attn_mfma_supported": ([_c_int], _c_int),
    "yk_attn_heads_per_tile": ([_c_int, _c_int], _c_int),
    "yk_attn_long_tile_tokens": ([_c_int, _c_int, _c_int], _c_int),
    "yk_attn_tokens_per_tile": ([_c_int, _c_int], _c_int),
    "yk_attn_mfma_workspace": ([_c_int, _c_int, _c_int, _c_int, _c_int], _c_size_t),
    "yk_attn_mfma_prefill": (
        [_vp, _c_int, _vp, _vp, _vp, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_int, _c_int, _c_int, _vp, _c_size_t, _c_int, _c_int, _c_float, _vp, _c_int, _vp, _c_int,
         _c_int, _c_float, _c_float, _c_float, _vp],
        _c_int,
    ),
    "yk_attn_mfma": (
        [_vp, _c_int, _vp, _vp, _vp, _vp, _c_int, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_int, _c_int, _c_int, _vp, _c_size_t, _c_int, _c_int, _c_float, _vp, _c_int, _vp, _c_int,
         _c_int, _c_float, _c_float, _c_float, _vp],
        _c_int,
    ),
    "yk_attn_mfma_rope": (
        [_vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _vp, _vp, _c_int,
         _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _c_float, _c_int, _c_int, _c_int, _vp, _c_size_t, _c_int, _vp],
        _c_int,
    ),
    "yk_attn_combine": ([_vp, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _c_size_t, _vp], _c_int),
    "yk_gemm_skinny_from_attention_ok": ([_c_int, _c_int, _c_int], _c_int),
    "yk_gemm_mfma_skinny_from_attention": (
        [_vp, _c_size_t, _vp, _c_int, _c_int, _c_int, _c_int, _c_int, _vp, _vp, _c_int, _vp, _c_size_t, _c_int, _c_int, _c_int, _c_int, _c_int, _vp],
        _c_int,
    ),
}
# the libraries that are built and loaded when first used (choosing tokens; the benchmark's probes)
_LATER_SIGNATURES = {
    "sampling": {
        "yk_abi_version": ([], _c_int),
        "yk_argmax": ([_vp, _vp, _c_int, _c_int, _vp, _c_size_t, _vp], _c_int),
        "yk_sample": ([_vp, _vp, _c_int, _c_int, _vp, _vp, _vp, _vp, _vp, _c_int, _vp, _c_size_t, _vp, _vp], _c_int),
        "yk_sample_workspace_bytes": ([_c_int, _c_int], _c_size_t),
    },
    "probe": {
        "yk_abi_version": ([], _c_int),
        "yk_probe_stream_read": ([_vp, _c_size_t, _c_int, _c_int, _vp, _vp], _c_int),
        "yk_probe_mfma_bf16": ([_c_int, _c_int, _vp, _vp], _c_int),
    },
}
_ABI = 24

# Rows of x up to which the hand-written matrix-core kernel runs a bfloat16 product;
# above it the vendor library does.
SKINNY_MAX_ROWS = 64
# Waves the attention launch aims at when it decides how far to split the keys.
ATTN_TARGET_WAVES = 1024
# Tokens of a step up to which an attention leaves its splits unmerged for the product that
# follows.  Every workgroup of that product merges its own slice of them again, so the saved
# kernel pays for few tokens only.  Measured at the 8B shape, 1,024-token contexts (ms a step,
# merged by a kernel of its own / by the product): 1 token 3.439 / 3.381, 2 tokens 3.471 /
# 3.427, 3 tokens 3.505 / 3.499, 4 tokens 3.506 / 3.526, 8 tokens 3.635 / 3.695.  The kernel
# takes up to 16.
MERGE_IN_PRODUCT_MAX_TOKENS = 2


class SplitSum:
    """The unreduced K slices of a product: float32 [slices, rows, columns] whose sum over
    the first axis is the result.  The kernels that consume a projection (norm, rotary +
    append, gated activation) add the slices themselves, which saves a pass over memory
    of its own.  ``out_dtype`` is the dtype the product was asked for: the consumers round
    the sum to it, so that a value does not depend on whether its product came reduced or
    as slices.  It lives in the library's workspace: consume it before the next product
    is launched.  One that the library made carries the workspace's generation number, and
    the library refuses (``StaleWorkspace``) to consume it once a later product has taken
    the workspace."""

    def __init__(self, tensor: torch.Tensor, out_dtype: torch.dtype = torch.float32, owner=None, generation: int = 0):
        self.tensor = tensor
        self.owner, self.generation = owner, generation
        self.shape = tuple(tensor.shape[1:])
        self.n_splits = tensor.shape[0]
        self.out_dtype = out_dtype
        self.dtype = torch.float32
        self.device = tensor.device

    @property
    def round_sum(self) -> int:
        return int(self.out_dtype == torch.bfloat16)

    def check_live(self) -> None:
        if self.owner is not None and self.generation != self.owner._gemm_gen:
            raise StaleWorkspace(
                "a product's unreduced slices (SplitSum) were consumed after a later product had been launched: the "
                "library's workspace holds that product's slices now.  Consume a linear(..., partial_ok=True) result "
                "(norm, rotary + append, gated activation, .reduce()) before the next linear, or ask without partial_ok")

    def reduce(self) -> torch.Tensor:
        """The product itself, float32 (for code that does not add the slices itself)."""
        self.check_live()
        return self.tensor.sum(0).to(self.out_dtype).float()

    def float(self) -> torch.Tensor:
        return self.reduce()


class EmbeddedRows:
    """The rows of an embedding table that a step's tokens name, not yet gathered: it stands
    for a tensor [tokens, width] with which a residual stream starts.  The norm kernel that
    comes first gathers the rows itself (``add_rmsnorm`` with this as ``delta`` fills the
    residual and normalises it in one pass); ``gather()`` gives the tensor (float32)."""

    def __init__(self, ops, token_ids: torch.Tensor, table: torch.Tensor):
        self.ops, self.token_ids, self.table = ops, token_ids, table
        self.shape = (token_ids.numel(), table.shape[1])
        self.dtype = torch.float32
        self.device = table.device

    def gather(self) -> torch.Tensor:
        return self.ops.embed(self.token_ids, self.table)

    def float(self) -> torch.Tensor:
        return self.gather()


class SplitAttention:
    """The output of an attention whose keys were split across workgroups, not yet merged:
    it stands for a bfloat16 tensor [tokens, heads * head_dim].  ``HipOps.linear`` merges the
    splits while it stages them as its input where its kernel can (up to 16 tokens), which
    saves the merging kernel; ``merge()`` gives the tensor itself.  It lives in the library's
    workspace: consume it before the next attention (or anything else that takes that
    workspace: choosing tokens) is launched; the library refuses a stale one."""

    def __init__(self, ops, workspace, tiles, token_cols, n_tokens, n_heads, n_kv, head_dim, n_splits):
        self.ops, self.workspace, self.tiles, self.token_cols = ops, workspace, tiles, token_cols
        self.generation = ops._ws_gen
        self.n_heads, self.n_kv, self.head_dim, self.n_splits = n_heads, n_kv, head_dim, n_splits
        self.shape = (n_tokens, n_heads * head_dim)
        self.dtype = torch.bfloat16
        self.device = workspace.device

    def check_live(self) -> None:
        if self.generation != self.ops._ws_gen:
            raise StaleWorkspace(
                "an attention's unmerged splits (SplitAttention) were consumed after a later launch had taken the "
                "library's workspace; hand them to linear() or merge() before the next attention")

    def merge(self) -> torch.Tensor:
        ops = self.ops
        self.check_live()
        out = torch.empty(self.shape, dtype=self.dtype, device=self.device)
        ops._check(
            ops.lib.yk_attn_combine(
                out.data_ptr(), self.tiles.data_ptr(), self.tiles.shape[0], self.head_dim, self.n_heads, self.n_kv,
                self.n_splits, self.workspace.data_ptr(), self.workspace.numel(), ops._stream(),
            )
        )
        return out


class RopeInLaunch:
    """What ``HipOps.attention`` needs to rotate and append inside its own launch: the float32
    tables [positions, rotary_dim / 2] (None with rotary_dim 0), how pairs are formed, and
    whether the projection's rows hold keys and values to append (False: queries only, the
    pages already hold this step's keys and values)."""

    def __init__(self, cos, sin, rotary_dim: int, interleaved: bool, append: bool):
        self.cos, self.sin, self.rotary_dim, self.interleaved, self.append = cos, sin, int(rotary_dim), bool(interleaved), bool(append)


class HipOps:
    def __init__(self, device: str = "cuda:0"):
        if not torch.cuda.is_available():
            raise KernelError("HipOps needs a GPU: torch.cuda.is_available() is False")
        self.device = torch.device(device)
        self.lib = self._bind(load_kernels(), _SIGNATURES)
        self._later: dict = {}
        self._answers: dict = {}
        self._device_index = self.device.index if self.device.index is not None else torch.cuda.current_device()
        # the quick way to the current stream's handle, where this torch has it
        self._raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)
        self._workspace: Optional[torch.Tensor] = None  # attention splits, argmax parts
        self._library_workspace: Optional[torch.Tensor] = None  # the vendor library's scratch
        self._gemm_workspace: Optional[torch.Tensor] = None  # K slices of products
        # how often each workspace has been handed out: what lives in one (SplitSum,
        # SplitAttention) remembers the number and is refused once it has moved on
        self._ws_gen = 0
        self._gemm_gen = 0
        # page ids a workgroup of the long-span attention keeps in LDS (more: looked up in the
        # block table one by one); tests lower it to walk that path with short tables
        self.long_span_pages_in_lds = 2048

    # ------------------------------------------------------------------ helpers
    @staticmethod
    def _bind(lib, signatures):
        lib.yk_last_error.restype = ctypes.c_char_p
        for name, (args, res) in signatures.items():
            fn = getattr(lib, name)
            fn.argtypes = args
            fn.restype = res
        if lib.yk_abi_version() != _ABI:
            raise KernelError("kernel library and bindings disagree; rebuild (python -c 'import __graft_entry__ as g; g.build()')")
        return lib

    def _library(self, name: str):
        """A library beside the step's kernels, built and loaded at its first use."""
        if name not in self._later:
            self._later[name] = self._bind(load_kernels(name), _LATER_SIGNATURES[name])
        return self._later[name]

    def _stream(self) -> int:
        """The raw handle of torch's current stream on this device (asked for at every
        launch: a graph capture switches streams)."""
        if self._raw_stream is not None:
            return self._raw_stream(self._device_index)
        return torch.cuda.current_stream(self.device).cuda_stream

    def _check(self, rc: int, lib=None) -> None:
        if rc != 0:
            raise KernelError((lib or self.lib).yk_last_error().decode())

    def _grown(self, have: Optional[torch.Tensor], floats: int) -> torch.Tensor:
        if have is not None and have.numel() >= floats:
            return have
        if have is not None and torch.cuda.is_current_stream_capturing():
            # kernels already recorded hold the old buffer's address
            raise KernelError(f"a scratch buffer would have to grow to {floats} floats while a graph is being captured; "
                              "reserve_workspaces() before the capture must ask for more")
        return torch.empty(max(floats, 1 << 22), dtype=torch.float32, device=self.device)

    def _ws(self, floats: int) -> torch.Tensor:
        """Float32 scratch that grows and is reused (stream order keeps uses apart)."""
        self._workspace = self._grown(self._workspace, floats)
        self._ws_gen += 1
        return self._workspace

    def _gemm_ws(self, floats: int) -> torch.Tensor:
        self._gemm_workspace = self._grown(self._gemm_workspace, floats)
        self._gemm_gen += 1
        return self._gemm_workspace

    def reserve_workspaces(self, rows: int, products=()) -> None:
        """Make the scratch buffers large enough for steps of ``rows`` tokens before a graph is
        captured (a buffer must not be replaced while a capture is running: that raises).
        ``products``: the (n, k) of the weight matrices the step multiplies ``rows`` rows by; the
        unreduced K slices of each take slices x rows x n floats."""
        need = 1 << 24
        if rows <= SKINNY_MAX_ROWS:
            for n, k in products:
                if k >= 8 and k % 8 == 0:
                    need = max(need, self._ask("yk_gemm_skinny_splits", rows, n, k, 0) * rows * n)
        self._ws(1 << 24)
        self._gemm_ws(need)

    def force_skinny_plan(self, chunk: int = 0, waves: int = 0, slices: int = 0) -> None:
        """For tests and measurements: force the few-row product's chunk length (128 / 256), waves a
        workgroup and number of K slices (0: the library decides); call without arguments to clear."""
        self._check(self.lib.yk_gemm_skinny_force(int(chunk), int(waves), int(slices)))
        self._answers = {k: v for k, v in self._answers.items() if k[0] not in ("yk_gemm_skinny_splits", "yk_gemm_skinny_from_attention_ok")}

    def wide_skinny_products(self, mode: int = 1) -> None:
        """For tests and measurements: when few-row products of 33 to 64 rows run in the wide form
        (32 x 32 x 16 matrix-core products): 0 never, 1 where the library's rule says so (the
        default: an unsliced K of 8,192 and more), 2 always."""
        self._check(self.lib.yk_gemm_skinny_wide(int(mode)))

    def tune_library_products(self, on: bool = True) -> None:
        """Whether new shapes of up to 256 rows get the vendor library's first candidate (the
        default: the same choice, and the same bits, in every process) or the fastest of its
        candidates, timed when the shape is first met (the choice then depends on the run)."""
        self._check(self.lib.yk_gemm_library_tune(int(bool(on))))

    def workspaces(self):
        """The scratch buffers in use, for whoever must keep them alive (a captured graph)."""
        return (self._workspace, self._gemm_workspace)

    def _ask(self, name: str, *args: int) -> int:
        """A size question to the library (tile sizes, slices, workspace needs): the answers
        depend on the arguments alone, so each is asked once."""
        key = (name, args)
        got = self._answers.get(key)
        if got is None:
            got = self._answers[key] = getattr(self.lib, name)(*args)
        return got

    @staticmethod
    def _rows(t: torch.Tensor, what: str) -> None:
        if t.dim() != 2 or t.stride(1) != 1:
            raise KernelError(f"{what}: expected a 2-D tensor with contiguous rows, got shape {tuple(t.shape)} strides {t.stride()}")

    # ---------------------------------------------------------- sizes a part may ask
    def check_attention_sizes(self, n_heads: int, n_kv: int, head_dim: int, page_size: int) -> None:
        if n_heads % n_kv:
            raise KernelError(f"attention: {n_heads} heads are not a multiple of {n_kv} kv heads")
        if head_dim % 16 or not 16 <= head_dim <= 256:
            raise KernelError(f"attention: head_dim must be a multiple of 16 between 16 and 256, got {head_dim}")
        if page_size % 16:
            raise KernelError(f"attention: page_size must be a multiple of 16, got {page_size}")

    def attention_tokens_per_tile(self, n_heads: int, n_kv: int) -> int:
        return self._ask("yk_attn_tokens_per_tile", n_heads, n_kv)

    def attention_long_span_tile(self, n_heads: int, n_kv: int, col_tiles: int = 1) -> int:
        """Tokens per tile of the kernel for long spans (one workgroup a tile) when a wave
        has ``col_tiles`` (1 or 2) column tiles."""
        return self._ask("yk_attn_long_tile_tokens", n_heads, n_kv, col_tiles)

    @staticmethod
    def attention_long_col_tiles(workgroups: int, fewest_keys: int) -> int:
        """Column tiles per wave for a step's long spans.  ``workgroups``: how many the
        larger tiles (two column tiles a wave) would make; ``fewest_keys``: the fewest keys
        any of the spans has cached before it.  Two where those workgroups fill the GPU twice
        over, or where no span starts from nothing: every block of keys staged through LDS
        then serves twice the columns, and where the tiles are few the keys are split across
        workgroups (``attention_long_splits``).  One for prompts from nothing: they have tiles
        with a few keys and tiles with all of them, which small tiles balance better.
        Measured on the 8B shape (us, one / two, each with its own splits): a whole 2,048-token
        prompt 70 / 77, a whole 4,096-token one 232 / 204, 2,048 tokens against 6,144 cached
        396 / 318, four 512-token portions against 3,584 cached 228 / 182, a 480-token portion
        against 3,616 cached 72 / 65, against 7,200 cached 116 / 103, two such portions
        124 / 111."""
        return 2 if workgroups >= 1024 or fewest_keys >= 1024 else 1

    # ------------------------------------------------------------------ embedding
    def embed(self, token_ids: torch.Tensor, table: torch.Tensor, positions=None, position_table=None, scale: float = 1.0) -> torch.Tensor:
        """float32 rows table[id] * scale (+ position_table[position], a learned vector per absolute position, summed in
        float32)."""
        self._rows(table, "embed table")
        n = token_ids.numel()
        if position_table is not None:
            self._rows(position_table, "position table")
            if (position_table.dtype != table.dtype or position_table.shape[1] != table.shape[1] or not position_table.is_contiguous()
                    or positions is None or positions.numel() != n or positions.dtype != torch.int32):
                raise KernelError("embed: the position table has the embedding table's dtype and width, and every token an int32 position")
        out = torch.empty((n, table.shape[1]), dtype=torch.float32, device=table.device)
        self._check(
            self.lib.yk_embed(
                token_ids.data_ptr(), table.data_ptr(), _code(table.dtype), out.data_ptr(), n,
                table.shape[1], table.shape[0], _ptr(positions) if position_table is not None else None, _ptr(position_table),
                0 if position_table is None else position_table.shape[0], float(scale), self._stream(),
            )
        )
        return out

    def embed_pairs(self, token_ids, table, scale, pair_table, buckets, mul_prev, mul_cur, state, ctx, act_dtype):
        """(float32 rows table[id] * scale + pair_table[(before * mul_prev + id * mul_cur) mod buckets], the same rounded to
        ``act_dtype``).  The token before a span's first one is ``state`` [slots, 1] (int32, negative: none, which takes
        the pair table's row ``buckets``); it is left at the span's last token."""
        n, width = token_ids.numel(), table.shape[1]
        if table.dim() != 2 or not table.is_contiguous() or not pair_table.is_contiguous() or tuple(pair_table.shape) != (buckets + 1, width) \
                or pair_table.dtype != table.dtype:
            raise KernelError(f"embed_pairs: the pairs' table {tuple(pair_table.shape)} does not match {buckets} buckets and a row for none, of {width}")
        if state.dtype != torch.int32 or tuple(state.shape[1:]) != (1,) or token_ids.dtype != torch.int32:
            raise KernelError("embed_pairs: a request's last token is one int32")
        a = ctx.arrays
        out = torch.empty((n, width), dtype=torch.float32, device=table.device)
        rounded = None if act_dtype == torch.float32 else torch.empty((n, width), dtype=act_dtype, device=table.device)
        self._check(self.lib.yk_embed_pairs(
            token_ids.data_ptr(), table.data_ptr(), _code(table.dtype), table.shape[0], float(scale), pair_table.data_ptr(), int(buckets),
            int(mul_prev), int(mul_cur), state.data_ptr(), a["token_seq"].data_ptr(), a["seq_qstart"].data_ptr(), a["seq_qlen"].data_ptr(),
            a["state_slots"].data_ptr(), out.data_ptr(), _ptr(rounded), n, width, self._stream()))
        return out, (out if rounded is None else rounded)

    def embedded_rows(self, token_ids: torch.Tensor, table: torch.Tensor):
        """(an uninitialised float32 residual [tokens, width], the ``EmbeddedRows`` that the
        first ``add_rmsnorm`` fills it from): the embedding without a kernel of its own."""
        self._rows(table, "embed table")
        residual = torch.empty((token_ids.numel(), table.shape[1]), dtype=torch.float32, device=table.device)
        return residual, EmbeddedRows(self, token_ids, table)

    # ----------------------------------------------------------------------- norm
    def rmsnorm(self, x, weight, eps, unit_offset, out_dtype):
        """norm(x) * weight for rows ``x`` [N, width] that are no residual stream (a tensor, or a
        ``SplitSum`` whose slices are summed on the way); nothing is written but the result."""
        n_splits, round_sum, src = 1, 0, x
        if isinstance(x, SplitAttention):
            x = src = x.merge()
        if isinstance(x, SplitSum):
            x.check_live()
            n_splits, round_sum, src = x.n_splits, x.round_sum, x.tensor
        else:
            self._rows(x, "norm input")
            if not x.is_contiguous():
                raise KernelError("norm input must be contiguous")
        n, width = x.shape
        if weight.numel() != width:
            raise KernelError(f"norm weight has {weight.numel()} elements, rows have {width}")
        out = torch.empty((n, width), dtype=out_dtype, device=src.device)
        self._check(
            self.lib.yk_add_rmsnorm(
                None, src.data_ptr(), _code(src.dtype), n_splits, round_sum, None, weight.data_ptr(), _code(weight.dtype),
                out.data_ptr(), _code(out_dtype), n, n, width, float(eps), int(bool(unit_offset)), None, 0, None, self._stream(),
            )
        )
        return out

    def _norm(self, residual, delta, rows, weight, eps, unit_offset, out_dtype, n_out, row=None):
        self._rows(residual, "residual")
        if row is not None and (rows is not None or row.dtype != torch.float32 or row.numel() != residual.shape[1] or not row.is_contiguous()):
            raise KernelError("add_rmsnorm: the vector for every token is contiguous float32 [width], and the residual is written back")
        if residual.dtype != torch.float32 or not residual.is_contiguous():
            raise KernelError("the residual stream must be contiguous float32")
        width = residual.shape[1]
        if weight.numel() != width:
            raise KernelError(f"norm weight has {weight.numel()} elements, rows have {width}")
        n_splits, round_sum = 1, 0
        table_ids, table_rows = None, 0
        if isinstance(delta, EmbeddedRows):
            if rows is not None or tuple(delta.shape) != tuple(residual.shape):
                raise KernelError(f"embedded rows {tuple(delta.shape)} start a residual of their own shape, got {tuple(residual.shape)}")
            table_ids, delta = delta.token_ids, delta.table
            self._rows(delta, "embedding table")
            if not delta.is_contiguous() or table_ids.dtype != torch.int32:
                raise KernelError("the embedding table must be contiguous and the token ids int32")
            table_rows = delta.shape[0]
        elif isinstance(delta, SplitSum):
            delta.check_live()
            n_splits, round_sum, delta = delta.n_splits, delta.round_sum, delta.tensor
            if tuple(delta.shape[1:]) != tuple(residual.shape):
                raise KernelError(f"delta {tuple(delta.shape[1:])} does not match the residual {tuple(residual.shape)}")
        elif delta is not None and (tuple(delta.shape) != tuple(residual.shape) or not delta.is_contiguous()):
            raise KernelError(f"delta {tuple(delta.shape)} does not match the residual {tuple(residual.shape)}")
        out = torch.empty((n_out, width), dtype=out_dtype, device=residual.device)
        self._check(
            self.lib.yk_add_rmsnorm(
                residual.data_ptr(), _ptr(delta), 0 if delta is None else _code(delta.dtype), n_splits, round_sum,
                _ptr(rows), weight.data_ptr(), _code(weight.dtype), out.data_ptr(), _code(out_dtype),
                n_out, residual.shape[0], width, float(eps), int(bool(unit_offset)), _ptr(table_ids), table_rows, _ptr(row),
                self._stream(),
            )
        )
        return out

    def add_rmsnorm(self, residual, delta, weight, eps, unit_offset, out_dtype, row=None):
        """residual (float32, in place) += delta (+ ``row``, one float32 vector [width] for every token); returns the
        normed rows."""
        return self._norm(residual, delta, None, weight, eps, unit_offset, out_dtype, residual.shape[0], row=row)

    def gather_add_rmsnorm(self, residual, delta, rows, weight, eps, unit_offset, out_dtype):
        return self._norm(residual, delta, rows, weight, eps, unit_offset, out_dtype, rows.numel())

    # --------------------------------------------------------------------- linear
    def linear(self, x: torch.Tensor, w: torch.Tensor, out_dtype: torch.dtype, partial_ok: bool = False, bias=None):
        """x [M, K] . w [N, K]^T (+ bias [N]) -> [M, N].  With ``partial_ok`` (and no bias) the
        result may come as a ``SplitSum`` for a consumer that adds the slices itself."""
        if bias is not None:
            # the product in float32, the bias added there, one rounding (as a product that adds
            # the bias to its accumulators rounds: the reference's biased Linear)
            acc = self.linear(x, w, torch.float32, partial_ok=False)
            if bias.numel() != acc.shape[1] or not bias.is_contiguous():
                raise KernelError(f"linear: bias has {bias.numel()} elements, the product {acc.shape[1]} columns")
            y = acc if out_dtype == torch.float32 else torch.empty(acc.shape, dtype=out_dtype, device=acc.device)
            if y.shape[0]:
                self._check(self.lib.yk_add_bias(acc.data_ptr(), _code(acc.dtype), acc.stride(0), y.data_ptr(), _code(y.dtype),
                                                 y.stride(0), bias.data_ptr(), _code(bias.dtype), y.shape[0], y.shape[1],
                                                 self._stream()))
            return y
        if isinstance(x, SplitAttention):
            y = self._linear_from_attention(x, w, out_dtype, partial_ok)
            if y is not None:
                return y
            x = x.merge()
        self._rows(x, "linear input")
        self._rows(w, "linear weight")
        m, k = x.shape
        n = w.shape[0]
        if w.shape[1] != k:
            raise KernelError(f"linear: input has {k} columns, weight has {w.shape[1]}")
        if m == 0:
            return torch.empty((0, n), dtype=out_dtype, device=x.device)
        bf = torch.bfloat16
        aligned = k % 8 == 0 and x.stride(0) % 8 == 0 and w.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0 and w.data_ptr() % 16 == 0
        if x.dtype == bf and w.dtype == bf and aligned:
            if out_dtype == bf and self.long_matrix_tiles(m, n, k):
                return self.gemm_tile(x, w, bf, partial_ok)
            if m > SKINNY_MAX_ROWS and out_dtype == bf and not self.few_library_tiles(m, n):
                return self.gemm_library(x, w, bf)  # vendor library, bfloat16 in and out
            if m > SKINNY_MAX_ROWS and out_dtype == torch.float32:
                # vendor library, float32 accumulators stored as they are (the output head for
                # more than 64 wanted rows: the few-row kernel would stream the table once per 64)
                return self.gemm_library(x, w, torch.float32)
            return self.gemm_mfma_skinny(x, w, out_dtype, partial_ok)
        return self.gemm_fma(x, w, out_dtype)

    @staticmethod
    def long_matrix_tiles(m: int, n: int, k: int) -> bool:
        """Whether a product of 65 to 256 rows is ``gemm_tile``'s: where the matrix is at least twice
        as long as it is wide (a down projection), so that tiles of 128 x 128 cut along K occupy
        the GPU and the slices are long.  Measured in replayed graphs (us, vendor library's first
        candidate / few-row kernel / tiles): 8B down-proj (4,096 x 14,336) at 72 rows 36.6 / 37.2 /
        25.6, at 128 57.9 / 35.4 / 27.0, at 192 77.5 / 65.9 / 49.3, at 256 45.9 / - / 47.5; 3B
        (3,072 x 8,192) at 128 32.9 / 19.6 / 17.7, at 192 45.3 / 27.5 / 28.5; 70B (8,192 x 28,672) at
        128 200 / 167 / 110, at 256 314 / - / 200; 1B (2,048 x 8,192) at 192 22.9 / 19.7 / 18.2.  On
        squarer matrices the three are within a tenth of each other up to 128 rows, and from 384
        rows on the library wins everywhere."""
        return SKINNY_MAX_ROWS < m <= 256 and k >= 2 * n and k >= 4096

    @staticmethod
    def few_library_tiles(m: int, n: int) -> bool:
        """Whether a product of 65 to 128 rows is still the few-row kernel's: where the vendor
        library's output tiles (256 columns wide) would be too few to occupy the GPU's 256
        compute units, while the few-row kernel divides K among workgroups.  Measured in replayed
        graphs with the library's fastest candidate (us, few-row kernel / library), 8B shapes at
        128 rows: o-proj 13.8 / 15.3, down-proj 38.7 / 52.1, but qkv 23.7 / 16.6 and gate/up
        96 / 58; at 160 rows o-proj 20.2 / 16.4, down-proj 65.6 / 58.7.  3B shapes at 128 rows:
        o-proj 10.9 / 11.4, down-proj 20.6 / 22.9, qkv 13.7 / 13.2.  So: up to 128 rows and up to
        4,096 columns."""
        return m <= 128 and -(-n // 256) <= 16

    def _linear_from_attention(self, x: "SplitAttention", w: torch.Tensor, out_dtype, partial_ok: bool):
        """The few-row product fed by attention's unmerged splits, or None where it does not
        apply (the caller then merges them first)."""
        x.check_live()
        m, k = x.shape
        n = w.shape[0]
        if (w.dim() != 2 or w.dtype != torch.bfloat16 or w.shape[1] != k or w.stride(1) != 1 or w.stride(0) % 8
                or w.data_ptr() % 16 or not self._ask("yk_gemm_skinny_from_attention_ok", m, n, k)):
            return None
        splits = self._ask("yk_gemm_skinny_splits", m, n, k, 0)
        keep = bool(partial_ok and splits > 1)
        ws = self._gemm_ws(splits * m * n) if splits > 1 else None
        y = None if keep else torch.empty((m, n), dtype=out_dtype, device=w.device)
        rc = self.lib.yk_gemm_mfma_skinny_from_attention(
            x.workspace.data_ptr(), x.workspace.numel(), x.token_cols.data_ptr(), x.tiles.shape[0], x.n_splits,
            x.n_heads, x.n_kv, x.head_dim, w.data_ptr(), _ptr(y), _code(out_dtype), _ptr(ws),
            0 if ws is None else ws.numel(), m, n, w.stride(0), n, int(keep), self._stream(),
        )
        if rc < 0:
            raise KernelError(self.lib.yk_last_error().decode())
        if keep:
            return SplitSum(ws[: rc * m * n].view(rc, m, n), out_dtype, self, self._gemm_gen)  # rc: the slices the launch wrote
        return y

    LIBRARY_WORKSPACE_BYTES = 64 << 20

    def gemm_library(self, x: torch.Tensor, w: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
        """x [M, K] . w [N, K]^T in the vendor library: bfloat16 operands with 16-byte aligned rows,
        float32 accumulation, the result bfloat16 or float32.  Every shape's algorithm is chosen
        when the shape is first met (the library's first candidate, or with
        ``tune_library_products`` the fastest for up to 256 rows) and kept."""
        m, k = x.shape
        n = w.shape[0]
        if x.dtype != torch.bfloat16 or w.dtype != torch.bfloat16 or w.shape[1] != k or x.stride(1) != 1 or w.stride(1) != 1:
            raise KernelError(f"gemm_library: operands {tuple(x.shape)} {x.dtype} and {tuple(w.shape)} {w.dtype}")
        if self._library_workspace is None:
            self._library_workspace = torch.empty(self.LIBRARY_WORKSPACE_BYTES, dtype=torch.uint8, device=self.device)
        y = torch.empty((m, n), dtype=out_dtype, device=x.device)
        self._check(self.lib.yk_gemm_library(
            x.data_ptr(), w.data_ptr(), y.data_ptr(), _code(out_dtype), m, n, k, x.stride(0), w.stride(0), n,
            self._library_workspace.data_ptr(), self._library_workspace.numel(), None, self._stream()))
        return y

    def gemm_tile(self, x, w, out_dtype, partial_ok: bool = False):
        """x [M, K] . w [N, K]^T in tiles of 128 x 128 on the matrix cores (bfloat16 operands with
        16-byte aligned rows): the kernel for some dozens to a few hundred rows against long
        matrices.  Where its plan cuts K the result comes as a ``SplitSum`` (with ``partial_ok``)
        or is summed here."""
        m, k = x.shape
        n = w.shape[0]
        splits = self._ask("yk_gemm_tile_splits", m, n, k)
        ws = self._gemm_ws(splits * m * n) if splits > 1 else None
        y = None if splits > 1 else torch.empty((m, n), dtype=out_dtype, device=x.device)
        rc = self.lib.yk_gemm_tile(
            x.data_ptr(), w.data_ptr(), _ptr(y), _code(out_dtype), _ptr(ws), 0 if ws is None else ws.numel(),
            m, n, k, x.stride(0), w.stride(0), n, self._stream(),
        )
        if rc < 0:
            raise KernelError(self.lib.yk_last_error().decode())
        if rc == 0:
            return y
        part = SplitSum(ws[: rc * m * n].view(rc, m, n), out_dtype, self, self._gemm_gen)
        return part if partial_ok else part.reduce().to(out_dtype)

    def force_tile_slices(self, slices: int = 0) -> None:
        """For tests and measurements: force the K slices of ``gemm_tile`` (0: the library decides)."""
        self._check(self.lib.yk_gemm_tile_force(int(slices)))
        self._answers = {k: v for k, v in self._answers.items() if k[0] != "yk_gemm_tile_splits"}

    def gemm_fma(self, x, w, out_dtype):
        m, k = x.shape
        n = w.shape[0]
        y = torch.empty((m, n), dtype=out_dtype, device=x.device)
        self._check(
            self.lib.yk_gemm_fma(
                x.data_ptr(), _code(x.dtype), w.data_ptr(), _code(w.dtype), y.data_ptr(), _code(out_dtype),
                m, n, k, x.stride(0), w.stride(0), n, self._stream(),
            )
        )
        return y

    # ---------------------------------------------------------- gate/up + activation
    GATE_UP_GROUP = 8  # rows of the packed matrix alternate: 8 of gate, their 8 of up

    def pack_gate_up(self, w_gate: torch.Tensor, w_up: torch.Tensor) -> Tuple[torch.Tensor, int]:
        """One matrix for both projections and the group size of its row order: 0 = [gate; up];
        8 = eight gate rows, then their eight up rows, and so on, which lets the few-row
        product apply the activation itself (the reference keeps gate and up in one matrix
        with rows interleaved too, yalis/external/model.py:717-722)."""
        inter = w_gate.shape[0]
        g = self.GATE_UP_GROUP
        if w_gate.dtype == torch.bfloat16 and w_up.dtype == torch.bfloat16 and inter % g == 0:
            k = w_gate.shape[1]
            packed = self._rows_apart(2 * inter, k, w_gate.device)
            packed.view(inter // g, 2, g, k)[:, 0].copy_(w_gate.view(inter // g, g, k))
            packed.view(inter // g, 2, g, k)[:, 1].copy_(w_up.view(inter // g, g, k))
            return packed, g
        return torch.cat([w_gate, w_up], dim=0).contiguous(), 0

    # Rows of a streamed bfloat16 matrix that would lie a multiple of 4 KiB apart are kept 128 bytes
    # further apart.  Workgroups of the few-row product that walk all of K in step (gate/up, the
    # output head: their K is not sliced) ask, at every moment, for addresses a whole number of
    # rows apart, and rows 4 KiB apart crowd onto few memory channels.  Up to 32 rows of x the
    # product answers that by starting its workgroups at different places of K; with more rows
    # they must stay in step (they share the staged rows of x through L2: started apart, gate/up
    # at 64 rows went 50 -> 64 us), and the gap between rows does it instead: 8B shape, us, rows 8 KiB
    # apart / 128 bytes more: gate/up at 64 rows of x 52.0 / 45.6, at 48 48.0 / 42.6, the head at 64
    # 221 / 197, at 48 212 / 184; at 32 rows and fewer no difference (42.2 / 43.3, 37.0 / 37.5).  The
    # sliced products (qkv, o-proj, down-proj) are better off without (qkv at 64 rows 14.0 / 15.7),
    # and so are rows of 16 KiB (the 70B shape's gate/up at 64 / 8 rows 196 / 223, 151 / 178): the
    # gap is for rows of 4 and 8 KiB (the 1B shape's head at 64 rows 120 / 110).
    ROW_GAP = 64  # elements

    @staticmethod
    def _rows_crowd(k: int) -> bool:
        return 2 * k in (4096, 8192)

    def _rows_apart(self, rows: int, k: int, device) -> torch.Tensor:
        """An uninitialised bfloat16 [rows, k], its rows 128 bytes further apart where that pays."""
        if self._rows_crowd(k):
            return torch.empty((rows, k + self.ROW_GAP), dtype=torch.bfloat16, device=device)[:, :k]
        return torch.empty((rows, k), dtype=torch.bfloat16, device=device)

    def streamed_matrix(self, w: torch.Tensor) -> torch.Tensor:
        """``w`` as a part should keep it when all it does with it is multiply few rows by it with
        K unsliced (an output head): ``w`` itself, or a copy with its rows 128 bytes further apart
        (see above)."""
        if w.dim() != 2 or w.dtype != torch.bfloat16 or not w.is_contiguous() or not self._rows_crowd(w.shape[1]):
            return w
        out = self._rows_apart(w.shape[0], w.shape[1], w.device)
        out.copy_(w)
        return out

    def gate_up_act(self, x: torch.Tensor, w_gate_up: torch.Tensor, group: int, activation: str, out_dtype: torch.dtype) -> torch.Tensor:
        """act(x . gate^T) * (x . up^T) -> [M, intermediate], ``w_gate_up`` and ``group`` as
        ``pack_gate_up`` gave them.  Few rows of bfloat16 whose product is not split over K
        run as one kernel; otherwise the product, then the activation kernel."""
        act = {"silu": 1, "gelu_tanh": 2}.get(activation if isinstance(activation, str) else None)
        if act is None:
            self.gated_kind(activation)  # raises for an unknown one
            act = 0  # a gated pair that the product's epilogue does not have: product, then the activation kernel
        self._rows(x, "gate/up input")
        m, k = x.shape
        n = w_gate_up.shape[0]
        bf = torch.bfloat16
        fused = (
            act > 0 and group == self.GATE_UP_GROUP and 0 < m <= SKINNY_MAX_ROWS and x.dtype == bf and w_gate_up.dtype == bf and out_dtype == bf
            and w_gate_up.shape[1] == k and k % 8 == 0 and x.stride(0) % 8 == 0 and w_gate_up.stride(0) % 8 == 0
            and x.data_ptr() % 16 == 0 and w_gate_up.data_ptr() % 16 == 0 and n % 16 == 0
            and self._ask("yk_gemm_skinny_splits", m, n, k, 1) == 1
        )
        if not fused:
            return self.gated_act(self.linear(x, w_gate_up, out_dtype, partial_ok=True), activation, out_dtype, group=group)
        y = torch.empty((m, n // 2), dtype=bf, device=x.device)
        rc = self.lib.yk_gemm_mfma_skinny(
            x.data_ptr(), w_gate_up.data_ptr(), y.data_ptr(), _code(bf), None, 0,
            m, n, k, x.stride(0), w_gate_up.stride(0), n // 2, 0, act, self._stream(),
        )
        if rc < 0:
            self._check(rc)
        return y

    def gemm_mfma_skinny(self, x, w, out_dtype, partial_ok: bool = False):
        m, k = x.shape
        n = w.shape[0]
        splits = self._ask("yk_gemm_skinny_splits", m, n, k, 0)
        keep = bool(partial_ok and splits > 1)
        ws = self._gemm_ws(splits * m * n) if splits > 1 else None
        y = None if keep else torch.empty((m, n), dtype=out_dtype, device=x.device)
        rc = self.lib.yk_gemm_mfma_skinny(
            x.data_ptr(), w.data_ptr(), _ptr(y), _code(out_dtype), _ptr(ws), 0 if ws is None else ws.numel(),
            m, n, k, x.stride(0), w.stride(0), n, int(keep), 0, self._stream(),
        )
        if rc < 0:
            raise KernelError(self.lib.yk_last_error().decode())
        if keep:
            return SplitSum(ws[: rc * m * n].view(rc, m, n), out_dtype, self, self._gemm_gen)  # rc: the slices the launch wrote
        return y

    # ------------------------------------------------- rotary + append to the cache
    def rope_append(self, qkv, n_heads, n_kv, head_dim, positions, cos, sin, rotary_dim,
                    interleaved, k_cache, v_cache, slots, page_size) -> torch.Tensor:
        """Rotates the query heads, appends rotated keys and values to the pages; returns
        the tensor whose rows start with the rotated queries (``qkv`` itself, rotated in
        place, or a new [N, n_heads * head_dim] tensor when ``qkv`` is a SplitSum)."""
        n_splits, round_sum = 1, 0
        src = qkv
        if isinstance(qkv, SplitSum):
            qkv.check_live()
            n_splits, round_sum, src = qkv.n_splits, qkv.round_sum, qkv.tensor
            n, cols = qkv.shape
            act = k_cache.dtype if n_kv else torch.bfloat16
            q_out = torch.empty((n, n_heads * head_dim), dtype=act, device=src.device)
            src_stride = cols
        else:
            self._rows(qkv, "qkv")
            n, cols = qkv.shape
            q_out = qkv
            src_stride = qkv.stride(0)
        if cols != (n_heads + 2 * n_kv) * head_dim:
            raise KernelError(f"qkv rows have {cols} elements, expected {(n_heads + 2 * n_kv) * head_dim}")
        if positions.numel() != n or (n_kv > 0 and slots.numel() != n):
            raise KernelError("positions/slots do not match the number of tokens")
        max_pos = 0
        if rotary_dim:
            if cos.dtype != torch.float32 or sin.dtype != torch.float32 or cos.shape != sin.shape or cos.shape[1] != rotary_dim // 2:
                raise KernelError("rotary tables must be float32 [positions, rotary_dim/2]")
            max_pos = cos.shape[0]
        if n_kv > 0:
            if k_cache.dtype != q_out.dtype or v_cache.dtype != q_out.dtype:
                raise KernelError("cache and activations differ in dtype")
            if tuple(k_cache.shape[1:]) != (n_kv, page_size, head_dim) or tuple(v_cache.shape[1:]) != (n_kv, head_dim, page_size):
                raise KernelError(f"cache pages have shapes {tuple(k_cache.shape)}, {tuple(v_cache.shape)}")
        self._check(
            self.lib.yk_rope_append(
                src.data_ptr(), _code(src.dtype), n_splits, round_sum, src_stride, q_out.data_ptr(), _code(q_out.dtype),
                q_out.stride(0), n, n_heads, n_kv, head_dim,
                positions.data_ptr(), _ptr(cos) if rotary_dim else None, _ptr(sin) if rotary_dim else None,
                rotary_dim, int(bool(interleaved)), max_pos,
                _ptr(k_cache) if n_kv else None, _ptr(v_cache) if n_kv else None,
                _ptr(slots) if n_kv else None, page_size, self._stream(),
            )
        )
        return q_out

    # ------------------------------------------------------------------ attention
    @staticmethod
    def attention_plan(column_groups: int, key_blocks: int) -> Tuple[int, int]:
        """(waves per workgroup, splits across workgroups) for the short-span kernel: the
        keys of a column group are divided until the launch has about ATTN_TARGET_WAVES
        waves, first among the waves of a workgroup (merged through LDS, no second kernel),
        then across workgroups (merged by the combine kernel)."""
        par = max(1, min(-(-ATTN_TARGET_WAVES // max(1, column_groups)), key_blocks))
        if par == 1:
            return 1, 1
        return 4, max(1, min(-(-par // 4), 256))

    @staticmethod
    def attention_long_splits(workgroups: int, key_blocks: int, col_tiles: int = 1) -> int:
        """Splits of the keys for the long-span kernel: one where the tiles alone fill the GPU
        (a prompt of a few thousand tokens); more where few tiles meet a long context (a
        portion of a prompt whose earlier portions are cached): as many as still leave all
        workgroups on the GPU at once (three a compute unit with one column tile a wave, two
        with two; a second, partly filled round costs more than the finer split gains: a
        480-token portion against 3,616 cached, one column tile, 3 / 4 / 5 splits 71.8 / 76.4 /
        73.3 us; two column tiles, 3 / 4 / 5 splits 74.3 / 64.5 / 76.9), at least 8 key blocks
        a split."""
        slots = 768 if col_tiles == 1 else 512
        return max(1, min(slots // max(1, workgroups), key_blocks // 8, 16))

    @staticmethod
    def rope_in_launch(rotation, append: bool) -> "RopeInLaunch":
        """What ``attention(rope=)`` takes, from a position encoding's ``Rotation`` (None: no
        rotation, the launch only appends) and whether the projection's rows hold keys and
        values to append."""
        if rotation is None:
            return RopeInLaunch(None, None, 0, False, append)
        return RopeInLaunch(rotation.cos, rotation.sin, rotation.rotary_dim, rotation.interleaved, append)

    def attention_can_rotate(self, act_dtype: torch.dtype, head_dim: int) -> bool:
        """Whether ``attention`` takes ``rope=`` for such a mixer: the matrix-core kernel for
        short spans can rotate queries and append keys and values itself."""
        return act_dtype == torch.bfloat16 and bool(self._ask("yk_attn_mfma_supported", head_dim))

    def attention_takes_sink(self, act_dtype: torch.dtype, head_dim: int) -> bool:
        """Whether ``attention`` takes ``sink=`` at these sizes (the matrix-core kernels do; elsewhere sinks are
        ``attention_masked``'s)."""
        return self.attention_can_rotate(act_dtype, head_dim)

    def attention_takes_maps(self, act_dtype: torch.dtype, head_dim: int) -> bool:
        """Whether ``attention`` takes ``differential=`` where both maps of a head together are ``head_dim`` wide."""
        return self.attention_can_rotate(act_dtype, head_dim)

    def attention(self, qkv, n_heads, n_kv, head_dim, k_cache, v_cache, page_size,
                  scale, window, ctx, group, tiles, long_tiles=None, plan=None, long_plan=None,
                  long_col_tiles: int = 1, token_cols=None, rope: Optional["RopeInLaunch"] = None,
                  keep_first: int = 0, softcap: float = 0.0, distance_bias=None, sink=None, chunked: bool = False,
                  differential=None):
        """Queries are the first n_heads heads of each row of ``qkv`` (whatever follows
        them in the row is skipped); keys and values come from the cache through the
        block table of ``group``.  ``long_tiles`` hold up to
        ``attention_long_span_tile(n_heads, n_kv, long_col_tiles)`` tokens each.  ``plan``
        overrides ``attention_plan`` and ``long_plan`` ``attention_long_splits`` (tests,
        measurements).  With ``token_cols`` (``attention_token_columns`` of the same short
        tiles) the caller takes a ``SplitAttention`` as well: what a step of up to 16 tokens,
        none of them in a long tile, leaves when its keys were split across workgroups.

        ``keep_first`` / ``softcap`` (matrix-core kernels only; other sizes are ``attention_masked``'s): with a
        window, the first ``keep_first`` keys of a request stay visible below it; scores times the scale
        are squashed to softcap * tanh(s / softcap); ``distance_bias`` (float32 [distances, n_heads]): row
        min(p - j, distances - 1) is added to head h's scaled (and squashed) score of key j for the query at p;
        ``chunked``: the window begins anew at every multiple of its size instead of sliding.

        ``differential`` (lambda, eps, gain; matrix-core kernels only): every head brings two query rows, one per map with
        zeros where the other map's keys are (``qkv_prepare(query_maps=2)``; ``n_heads`` counts these rows), and the result
        [N, n_heads / 2 * head_dim] is (a1 - lambda a2) divided by its root mean square per head and times gain.

        ``rope`` (only where ``attention_can_rotate``, and only for steps whose spans are single
        tokens): ``qkv`` is then the projection's raw output (a tensor or a ``SplitSum``) and
        the launch does what ``rope_append`` would have done before it: it rotates the queries
        and, with ``rope.append``, rotates the tokens' keys, uses them and their values, and
        stores both in the pages."""
        if rope is not None:
            return self._attention_rope(qkv, n_heads, n_kv, head_dim, k_cache, v_cache, page_size, scale, window,
                                        ctx, group, tiles, plan, token_cols, rope)
        self._rows(qkv, "qkv")
        n = qkv.shape[0]
        bt = ctx.arrays[f"block_table_g{group}"]
        if tuple(k_cache.shape[1:]) != (n_kv, page_size, head_dim) or tuple(v_cache.shape[1:]) != (n_kv, head_dim, page_size):
            raise KernelError(f"cache pages have shapes {tuple(k_cache.shape)}, {tuple(v_cache.shape)}")
        if k_cache.dtype != qkv.dtype:
            raise KernelError("cache and activations differ in dtype")
        maps = 1 if differential is None else 2
        lam, map_eps, gain = (0.0, 0.0, 1.0) if differential is None else (float(v) for v in differential)
        if maps == 2 and (n_heads % (2 * n_kv) or sink is not None or distance_bias is not None):
            raise KernelError("attention: two maps are two query rows a head, without sinks and biases per distance")
        out = torch.empty((n, n_heads // maps * head_dim), dtype=qkv.dtype, device=qkv.device)
        use_mfma = (
            qkv.dtype == torch.bfloat16
            and self._ask("yk_attn_mfma_supported", head_dim)
            and qkv.stride(0) % 8 == 0
            and qkv.data_ptr() % 16 == 0
        )
        if (keep_first or softcap or distance_bias is not None or sink is not None or chunked or maps == 2) and not use_mfma:
            raise KernelError("attention: kept first keys, chunks, squashed scores, biases per distance and sinks outside the matrix-core kernels' sizes are attention_masked's")
        # keys any query of the step reads at most (a chunk's queries read no other chunk's)
        reach = min(ctx.max_ctx, int(window)) if chunked else ctx.max_ctx
        if sink is not None and (sink.dtype != torch.float32 or sink.numel() != n_heads or not sink.is_contiguous()):
            raise KernelError("attention: the sinks are contiguous float32 [heads]")
        if distance_bias is not None and (distance_bias.dtype != torch.float32 or distance_bias.dim() != 2 or not distance_bias.is_contiguous()
                                          or distance_bias.shape[1] != n_heads or distance_bias.shape[0] < 1):
            raise KernelError("attention: the distance bias is contiguous float32 [distances, heads]")
        bias_rows = 0 if distance_bias is None else distance_bias.shape[0]
        if use_mfma and long_tiles is not None and long_tiles.shape[0] > 0:
            n_long = long_tiles.shape[0]
            hpt = self._ask("yk_attn_heads_per_tile", n_heads, n_kv)
            groups = n_long * n_kv * (-(-(n_heads // n_kv) // hpt))
            long_splits = long_plan if long_plan is not None else self.attention_long_splits(groups, max(1, -(-reach // 64)), int(long_col_tiles))
            ws_floats = self._ask("yk_attn_mfma_workspace", 4 * long_col_tiles * n_long, n_heads, n_kv, head_dim, long_splits)
            ws = self._ws(ws_floats) if ws_floats else None
            self._check(
                self.lib.yk_attn_mfma_prefill(
                    qkv.data_ptr(), qkv.stride(0), out.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(),
                    long_tiles.data_ptr(), n_long, bt.data_ptr(), bt.shape[1], page_size, head_dim,
                    n_heads, n_kv, float(scale), int(window), long_splits, int(long_col_tiles), _ptr(ws),
                    0 if ws is None else ws.numel(), int(self.long_span_pages_in_lds), int(keep_first), float(softcap),
                    _ptr(distance_bias), bias_rows, _ptr(sink), int(bool(chunked)), maps, lam, map_eps, gain, self._stream(),
                )
            )
        if use_mfma and tiles.shape[0] == 0:
            return out
        if use_mfma:
            n_tiles = tiles.shape[0]
            hpt = self._ask("yk_attn_heads_per_tile", n_heads, n_kv)
            chunks = -(-(n_heads // n_kv) // hpt)
            key_blocks = max(1, -(-reach // 64))
            waves, splits = plan or self.attention_plan(n_tiles * n_kv * chunks, key_blocks)
            ws_floats = self._ask("yk_attn_mfma_workspace", n_tiles, n_heads, n_kv, head_dim, splits)
            ws = self._ws(ws_floats) if ws_floats else None
            leave = bool(token_cols is not None and splits > 1 and n <= MERGE_IN_PRODUCT_MAX_TOKENS and (long_tiles is None or long_tiles.shape[0] == 0)
                         and sink is None and maps == 1)  # (a sink joins, and maps meet, in the merge kernel)
            self._check(
                self.lib.yk_attn_mfma(
                    qkv.data_ptr(), qkv.stride(0), out.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(),
                    tiles.data_ptr(), n_tiles, bt.data_ptr(), bt.shape[1], page_size, head_dim, n_heads, n_kv,
                    float(scale), int(window), waves, splits, _ptr(ws), 0 if ws is None else ws.numel(), int(leave),
                    int(keep_first), float(softcap), _ptr(distance_bias), bias_rows, _ptr(sink), int(bool(chunked)),
                    maps, lam, map_eps, gain, self._stream(),
                )
            )
            if leave:
                return SplitAttention(self, ws, tiles, token_cols, n, n_heads, n_kv, head_dim, splits)
        else:
            self._check(
                self.lib.yk_attn_generic(
                    qkv.data_ptr(), qkv.stride(0), out.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(),
                    _code(qkv.dtype), ctx.arrays["positions"].data_ptr(), ctx.arrays["token_seq"].data_ptr(),
                    bt.data_ptr(), bt.shape[1], n, page_size, head_dim, n_heads, n_kv, float(scale), int(window),
                    self._stream(),
                )
            )
        return out

    def _attention_rope(self, qkv, n_heads, n_kv, head_dim, k_cache, v_cache, page_size, scale, window,
                        ctx, group, tiles, plan, token_cols, rope: "RopeInLaunch"):
        n_splits_src, round_sum, src = 1, 0, qkv
        if isinstance(qkv, SplitSum):
            qkv.check_live()
            n_splits_src, round_sum, src = qkv.n_splits, qkv.round_sum, qkv.tensor
            n, cols = qkv.shape
            src_stride = cols
        else:
            self._rows(qkv, "qkv")
            n, cols = qkv.shape
            src_stride = qkv.stride(0)
        if ctx.max_qlen != 1 or tiles.shape[0] != n:
            raise KernelError("attention with rotary inside takes steps of single tokens only")
        if not self.attention_can_rotate(k_cache.dtype, head_dim):
            raise KernelError("attention with rotary inside needs bfloat16 pages and a head size of 64 or 128")
        if cols != (n_heads + (2 * n_kv if rope.append else 0)) * head_dim:
            raise KernelError(f"projection rows have {cols} elements, expected {(n_heads + (2 * n_kv if rope.append else 0)) * head_dim}")
        if tuple(k_cache.shape[1:]) != (n_kv, page_size, head_dim) or tuple(v_cache.shape[1:]) != (n_kv, head_dim, page_size):
            raise KernelError(f"cache pages have shapes {tuple(k_cache.shape)}, {tuple(v_cache.shape)}")
        max_pos = 0
        if rope.rotary_dim:
            cos, sin = rope.cos, rope.sin
            if cos.dtype != torch.float32 or sin.dtype != torch.float32 or cos.shape != sin.shape or cos.shape[1] != rope.rotary_dim // 2:
                raise KernelError("rotary tables must be float32 [positions, rotary_dim/2]")
            max_pos = cos.shape[0]
        bt = ctx.arrays[f"block_table_g{group}"]
        out = torch.empty((n, n_heads * head_dim), dtype=torch.bfloat16, device=src.device)
        hpt = self._ask("yk_attn_heads_per_tile", n_heads, n_kv)
        chunks = -(-(n_heads // n_kv) // hpt)
        key_blocks = max(1, -(-ctx.max_ctx // 64))
        waves, splits = plan or self.attention_plan(n * n_kv * chunks, key_blocks)
        ws_floats = self._ask("yk_attn_mfma_workspace", n, n_heads, n_kv, head_dim, splits)
        ws = self._ws(ws_floats) if ws_floats else None
        leave = bool(token_cols is not None and splits > 1 and n <= MERGE_IN_PRODUCT_MAX_TOKENS)
        self._check(
            self.lib.yk_attn_mfma_rope(
                src.data_ptr(), _code(src.dtype), n_splits_src, round_sum, src_stride, n,
                _ptr(rope.cos) if rope.rotary_dim else None, _ptr(rope.sin) if rope.rotary_dim else None,
                int(rope.rotary_dim), int(bool(rope.interleaved)), max_pos, int(bool(rope.append)),
                out.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), tiles.data_ptr(), n, bt.data_ptr(), bt.shape[1],
                page_size, head_dim, n_heads, n_kv, float(scale), int(window), waves, splits, _ptr(ws),
                0 if ws is None else ws.numel(), int(leave), self._stream(),
            )
        )
        if leave:
            return SplitAttention(self, ws, tiles, token_cols, n, n_heads, n_kv, head_dim, splits)
        return out

    # ----------------------------------------------------------------- activation
    # gated pairs the kernels know: name -> (code, number of constants)
    GATED_KINDS = {"silu": (0, 0), "gelu_tanh": (1, 0), "clamped_swish": (2, 2)}

    @classmethod
    def gated_kind(cls, activation) -> Tuple[int, float, float]:
        """(code, p0, p1) of an activation given as a name or as (name, constants...):
        ("clamped_swish", limit, slope) is min(g, limit) * sigmoid(slope * min(g, limit)) *
        (clamp(u, -limit, limit) + 1)."""
        name, consts = (activation, ()) if isinstance(activation, str) else (activation[0], tuple(activation[1:]))
        if name not in cls.GATED_KINDS:
            raise KernelError(f"unknown activation {name!r}")
        code, n = cls.GATED_KINDS[name]
        if len(consts) != n:
            raise KernelError(f"activation {name!r} takes {n} constants, got {len(consts)}")
        p = [float(c) for c in consts] + [0.0, 0.0]
        return code, p[0], p[1]

    @classmethod
    def plain_kind(cls, activation) -> int:
        """The code of a plain (ungated) activation: "silu", "gelu_tanh", "relu2" (the square of relu)."""
        if activation not in cls.ACTIVATION_KINDS:
            raise KernelError(f"activation {activation!r} is not offered (offered: {sorted(cls.ACTIVATION_KINDS)})")
        return cls.ACTIVATION_KINDS[activation]

    def gated_act(self, gu, activation, out_dtype: Optional[torch.dtype] = None, group: int = 0) -> torch.Tensor:
        """act(gate) * up (or another gated pair, see ``gated_kind``) for gate/up columns [gate | up]
        (group 0) or alternating in groups of ``group`` columns (see ``pack_gate_up``)."""
        n_splits, round_sum = 1, 0
        src = gu
        if isinstance(gu, SplitSum):
            gu.check_live()
            n_splits, round_sum, src = gu.n_splits, gu.round_sum, gu.tensor
            rows, cols = gu.shape
            out_dtype = out_dtype or torch.bfloat16
        else:
            self._rows(gu, "gate/up")
            if not gu.is_contiguous():
                raise KernelError("gate/up must be contiguous")
            rows, cols = gu.shape
            out_dtype = out_dtype or gu.dtype
        if cols % 2:
            raise KernelError("gate/up must have an even number of columns")
        act, p0, p1 = self.gated_kind(activation)
        inter = cols // 2
        out = torch.empty((rows, inter), dtype=out_dtype, device=src.device)
        self._check(
            self.lib.yk_gated_act(src.data_ptr(), _code(src.dtype), n_splits, round_sum, out.data_ptr(), _code(out_dtype),
                                  rows, inter, act, int(group), p0, p1, self._stream())
        )
        return out

    # ------------------------------------------------- a branch joins through its own norm
    def round_rows(self, x: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
        """A float32 stream rounded to the activation dtype (the stream itself when that is float32)."""
        if out_dtype == torch.float32:
            return x
        if x.dtype != torch.float32 or not x.is_contiguous():
            raise KernelError("round_rows takes a contiguous float32 tensor")
        out = torch.empty(x.shape, dtype=out_dtype, device=x.device)
        self._check(self.lib.yk_round_rows(x.data_ptr(), out.data_ptr(), _code(out_dtype), x.numel(), self._stream()))
        return out

    def norm_add(self, residual, branch, weight, eps, unit_offset, out_dtype, expert_rows=None, expert_weight: float = 1.0):
        """residual (float32 [N, width], in place) += norm(branch) * weight, where branch is a tensor, a
        ``SplitSum``, and / or ``expert_rows`` (float32 [N * top, width], of which a token takes
        ``expert_weight`` times the sum of its top rows); returns the new residual in ``out_dtype``
        (the residual itself for float32)."""
        self._rows(residual, "residual")
        if residual.dtype != torch.float32 or not residual.is_contiguous():
            raise KernelError("the residual stream must be contiguous float32")
        n, width = residual.shape
        if weight.numel() != width:
            raise KernelError(f"norm weight has {weight.numel()} elements, rows have {width}")
        n_splits, round_sum, src = 1, 0, branch
        if isinstance(branch, SplitAttention):
            branch = src = branch.merge()
        if isinstance(branch, SplitSum):
            branch.check_live()
            n_splits, round_sum, src = branch.n_splits, branch.round_sum, branch.tensor
        if branch is not None and (tuple(branch.shape) != (n, width) or not src.is_contiguous()):
            raise KernelError(f"branch {tuple(branch.shape)} does not match the residual {(n, width)}")
        top = 0
        if expert_rows is not None:
            if expert_rows.dtype != torch.float32 or not expert_rows.is_contiguous() or expert_rows.dim() != 2 \
                    or expert_rows.shape[1] != width or (n and expert_rows.shape[0] % n):
                raise KernelError(f"expert rows {tuple(expert_rows.shape)} do not match the residual {(n, width)}")
            top = expert_rows.shape[0] // n if n else 1
        out = None if out_dtype == torch.float32 else torch.empty((n, width), dtype=out_dtype, device=residual.device)
        self._check(
            self.lib.yk_norm_add(
                residual.data_ptr(), _ptr(src), 0 if src is None else _code(src.dtype), n_splits, round_sum,
                _ptr(expert_rows), top, float(expert_weight), weight.data_ptr(), _code(weight.dtype), int(bool(unit_offset)),
                float(eps), _ptr(out), _BF16, n, width, self._stream(),
            )
        )
        return residual if out is None else out

    def sum_norm(self, residual, terms, branch_scale, branch_weight, residual_scale, weight, eps, unit_offset, out_dtype):
        """residual (float32 [N, width], in place) = norm(residual_scale * residual + branch_scale * (sum of the terms) *
        branch_weight) * weight; returns it in ``out_dtype`` (itself for float32).  ``terms``: one or two of (rows, weight,
        eps): a tensor or a ``SplitSum``, divided by its root mean square and multiplied by its weight, or, with weight
        None, as it is.  ``branch_weight`` [width] or None."""
        self._rows(residual, "residual")
        if residual.dtype != torch.float32 or not residual.is_contiguous():
            raise KernelError("the residual stream must be contiguous float32")
        n, width = residual.shape
        if not 1 <= len(terms) <= 2:
            raise KernelError("sum_norm takes one or two terms")
        args = []
        for rows, w, e in terms:
            n_splits, round_sum, src = 1, 0, rows
            if isinstance(rows, SplitAttention):
                rows = src = rows.merge()
            if isinstance(rows, SplitSum):
                rows.check_live()
                n_splits, round_sum, src = rows.n_splits, rows.round_sum, rows.tensor
            if tuple(rows.shape) != (n, width) or not src.is_contiguous():
                raise KernelError(f"branch {tuple(rows.shape)} does not match the residual {(n, width)}")
            args += [src.data_ptr(), _code(src.dtype), n_splits, round_sum, float(e), _ptr(w)]
        if len(terms) == 1:
            args += [None, 0, 1, 0, 0.0, None]
        for w in [t[1] for t in terms] + [branch_weight, weight]:
            if w is not None and (w.numel() != width or not w.is_contiguous() or w.dtype != weight.dtype):
                raise KernelError("sum_norm: the weights are contiguous, as wide as the rows and of one dtype")
        out = None if out_dtype == torch.float32 else torch.empty((n, width), dtype=out_dtype, device=residual.device)
        self._check(self.lib.yk_sum_norm(
            residual.data_ptr(), *args, float(branch_scale), _ptr(branch_weight), float(residual_scale), weight.data_ptr(), _code(weight.dtype),
            int(bool(unit_offset)), float(eps), _ptr(out), n, width, self._stream()))
        return residual if out is None else out

    # ------------------------------------- attention with prepared heads, kept first keys, a finish
    def masked_pages_tiled(self, dtype: torch.dtype, head_dim: int, value_dim: int, page_size: int) -> bool:
        return head_dim == value_dim and self.cache_tiled(dtype, head_dim, page_size)

    def qkv_prepare(self, qkv, n_heads, n_kv, head_dim, value_dim, positions, act_dtype, q_norm=None, k_norm=None,
                    qk_eps: float = 0.0, rotation=None, value_norm_eps=None, value_rotation=None,
                    k_cache=None, v_cache=None, slots=None, page_size: int = 0, bias=None, row_scales=None,
                    norm_over_projection: bool = False, values_from_keys: bool = False, unweighted_norm: bool = False,
                    query_maps: int = 1) -> torch.Tensor:
        """From a projection's rows [q | k | v | ...] (a tensor or a ``SplitSum``): normed (weights
        ``q_norm`` / ``k_norm`` of head_dim elements, or none) and rotated queries [N, n_heads * head_dim];
        normed, rotated keys and unit-normed (``value_norm_eps``), rotated (``value_rotation``) values
        into the pages (``n_kv`` 0: queries only).  ``bias`` (float32, one number per column of the projection)
        is added first.  ``values_from_keys``: the rows are [q | k | ...] and a token's values are its keys as
        projected (biased, before the norm).  ``norm_over_projection``: the weights are as wide as the q (k)
        projection and no root mean square is taken here: it comes with ``row_scales`` (float32 [N, 2], from
        ``qk_row_scales``), which multiply a token's queries (column 0) and keys (column 1) after the weights.
        ``unweighted_norm``: every head is divided by its root mean square (``qk_eps`` under the root) and that is all.
        ``query_maps`` = m > 1: a head's elements are m maps side by side, and the queries come as [N, n_heads * m * head_dim],
        a row per head and map with zeros where the other maps' elements are."""
        n_splits, round_sum, src = 1, 0, qkv
        if isinstance(qkv, SplitSum):
            qkv.check_live()
            n_splits, round_sum, src = qkv.n_splits, qkv.round_sum, qkv.tensor
            n, cols = qkv.shape
            stride = cols
        else:
            self._rows(qkv, "qkv")
            n, cols = qkv.shape
            stride = qkv.stride(0)
        if cols < n_heads * head_dim + n_kv * (head_dim + (0 if values_from_keys else value_dim)):
            raise KernelError(f"qkv rows have {cols} elements, fewer than the heads need")
        if values_from_keys and value_dim != head_dim:
            raise KernelError("qkv_prepare: values that are the keys are as wide as the keys")
        if bias is not None and (bias.dtype != torch.float32 or bias.numel() < cols or not bias.is_contiguous()):
            raise KernelError("qkv_prepare: the bias is contiguous float32 with a number per column of the projection")
        if row_scales is not None and (row_scales.dtype != torch.float32 or tuple(row_scales.shape) != (n, 2) or not row_scales.is_contiguous()):
            raise KernelError("qkv_prepare: the rows' scales are contiguous float32 [N, 2]")
        if norm_over_projection and (row_scales is None or q_norm is None or (n_kv > 0 and k_norm is None)):
            raise KernelError("qkv_prepare: a norm over the whole projection takes its weights and the rows' scales")
        if positions.numel() != n or (n_kv > 0 and slots.numel() != n):
            raise KernelError("positions/slots do not match the number of tokens")
        if query_maps < 1 or head_dim % query_maps:
            raise KernelError(f"qkv_prepare: heads of {head_dim} do not divide into {query_maps} maps")
        q_out = torch.empty((n, n_heads * query_maps * head_dim), dtype=act_dtype, device=src.device)
        tiled = False
        if n_kv > 0:
            if k_cache.dtype != act_dtype or v_cache.dtype != act_dtype:
                raise KernelError("cache and activations differ in dtype")
            if tuple(k_cache.shape[1:]) != (n_kv, page_size, head_dim) or tuple(v_cache.shape[1:]) != (n_kv, value_dim, page_size):
                raise KernelError(f"cache pages have shapes {tuple(k_cache.shape)}, {tuple(v_cache.shape)}")
            tiled = self.masked_pages_tiled(act_dtype, head_dim, value_dim, page_size)
        norm_w = q_norm if q_norm is not None else k_norm
        if q_norm is not None and k_norm is not None and q_norm.dtype != k_norm.dtype:
            raise KernelError("query and key norm weights differ in dtype")
        for w, heads in ((q_norm, n_heads), (k_norm, n_kv)):
            want = heads * head_dim if norm_over_projection else head_dim
            if w is not None and not (norm_over_projection and heads == 0) and (w.numel() != want or not w.is_contiguous()):
                raise KernelError(f"a norm's weight has {w.numel()} elements, {want} are normed together")
        qk_norm = int(q_norm is not None or k_norm is not None) * (2 if norm_over_projection else 1)
        if qk_norm and (q_norm is None or k_norm is None):
            raise KernelError("queries and keys are normed together or not at all")
        if unweighted_norm:
            if qk_norm:
                raise KernelError("qkv_prepare: a norm without weights takes none")
            qk_norm = 1
        for r in (rotation, value_rotation):
            if r is not None and (r.cos.dtype != torch.float32 or r.cos.shape != r.sin.shape or r.cos.shape[1] != r.rotary_dim // 2):
                raise KernelError("rotary tables must be float32 [positions, rotary_dim/2]")
        if value_rotation is not None and value_rotation.rotary_dim != value_dim:
            raise KernelError("values rotate over all of value_dim")
        self._check(
            self.lib.yk_qkv_prepare(
                src.data_ptr(), _code(src.dtype), n_splits, round_sum, stride, q_out.data_ptr(), _code(act_dtype),
                q_out.stride(0), n, n_heads, n_kv, head_dim, value_dim, positions.data_ptr(), _ptr(q_norm), _ptr(k_norm),
                _F32 if norm_w is None else _code(norm_w.dtype), qk_norm, float(qk_eps),
                None if rotation is None else rotation.cos.data_ptr(), None if rotation is None else rotation.sin.data_ptr(),
                0 if rotation is None else rotation.rotary_dim, int(bool(rotation is not None and rotation.interleaved)),
                0 if rotation is None else rotation.cos.shape[0],
                int(value_norm_eps is not None), float(value_norm_eps or 0.0),
                None if value_rotation is None else value_rotation.cos.data_ptr(),
                None if value_rotation is None else value_rotation.sin.data_ptr(),
                int(bool(value_rotation is not None and value_rotation.interleaved)),
                0 if value_rotation is None else value_rotation.cos.shape[0],
                _ptr(k_cache) if n_kv else None, _ptr(v_cache) if n_kv else None, _ptr(slots) if n_kv else None,
                int(page_size), int(tiled), _ptr(bias), _ptr(row_scales), int(bool(values_from_keys)), int(query_maps), self._stream(),
            )
        )
        return q_out

    def qk_row_scales(self, proj, n_q_cols: int, n_k_cols: int, positions, bias=None, eps=None, temperature=None) -> torch.Tensor:
        """float32 [N, 2]: what a token's queries (column 0) and keys (column 1) are multiplied with as wholes.  With
        ``eps``: 1 / sqrt(mean(x^2) + eps) over the first ``n_q_cols`` columns of the projection (a tensor or a
        ``SplitSum``) plus ``bias``, and over the next ``n_k_cols``.  With ``temperature`` = (coef, every): the queries'
        factor 1 + coef ln(floor((p + 1) / every) + 1) at position p on top."""
        n_splits, round_sum, src = 1, 0, proj
        if isinstance(proj, SplitSum):
            proj.check_live()
            n_splits, round_sum, src = proj.n_splits, proj.round_sum, proj.tensor
            n, cols = proj.shape
            stride = cols
        else:
            self._rows(proj, "projection")
            n, cols = proj.shape
            stride = proj.stride(0)
        if cols < n_q_cols + n_k_cols or positions.numel() != n or positions.dtype != torch.int32:
            raise KernelError("qk_row_scales: the projection holds the query and key columns, and every token has an int32 position")
        if bias is not None and (bias.dtype != torch.float32 or bias.numel() < n_q_cols + n_k_cols or not bias.is_contiguous()):
            raise KernelError("qk_row_scales: the bias is contiguous float32 with a number per column")
        coef, every = (0.0, 0) if temperature is None else (float(temperature[0]), int(temperature[1]))
        out = torch.empty((n, 2), dtype=torch.float32, device=src.device)
        self._check(self.lib.yk_qk_row_scales(src.data_ptr(), _code(src.dtype), n_splits, round_sum, stride, n, int(n_q_cols), int(n_k_cols),
                                              _ptr(bias), int(eps is not None), float(eps or 0.0), positions.data_ptr(), coef, every,
                                              out.data_ptr(), self._stream()))
        return out

    @staticmethod
    def _gate_source(gate, n: int):
        """(tensor, splits, round_sum, row stride) of the projection whose columns hold per-head gates."""
        if gate is None:
            return None, 1, 0, 0
        if isinstance(gate, SplitSum):
            gate.check_live()
            return gate.tensor, gate.n_splits, gate.round_sum, gate.shape[1]
        return gate, 1, 0, gate.stride(0)

    def attention_masked(self, q, n_heads, n_kv, head_dim, value_dim, k_cache, v_cache, page_size, scale, ctx, group,
                         window: int = 0, keep_first: int = 0, softcap: float = 0.0, value_rotation=None,
                         gate=None, gate_col: int = 0, gate_elems: int = 1, distance_bias=None, sink=None,
                         chunked: bool = False, differential=None) -> torch.Tensor:
        """softmax over the keys j <= p with (p - j < window or j < keep_first) of q . k * scale
        (squashed by ``softcap`` * tanh(s / ``softcap``) when set), times the values [N, n_heads *
        value_dim]; then, with ``value_rotation``, every head's output turned back by its token's
        position, and, with ``gate`` (the projection, a tensor or ``SplitSum``, whose columns
        ``gate_col`` + h hold the heads' gates), multiplied by the sigmoid of its gate (``gate_elems`` = value_dim:
        a gate per output element, in the columns ``gate_col`` + h * value_dim + d).  ``distance_bias`` (float32
        [distances, n_heads]): row min(p - j, distances - 1) is added to the scaled scores of head h.  ``sink`` (float32
        [n_heads]): exp(sink[h]) joins head h's denominator once; it has no key and no value.  ``chunked``: the window
        begins anew at every multiple of its size (keys j with floor(j / window) = floor(p / window)).  ``differential``
        (lambda, eps, gain): a head's queries and keys are two maps side by side, each with a softmax of its own over its
        half's scores; the head's output is (a1 - lambda a2) divided by its root mean square and times gain."""
        if differential is not None and (head_dim % 2 or sink is not None or distance_bias is not None):
            raise KernelError("attention_masked: two maps divide a head in halves and go without sinks and biases per distance")
        lam, map_eps, gain = (0.0, 0.0, 1.0) if differential is None else (float(v) for v in differential)
        self._rows(q, "queries")
        if sink is not None and (sink.dtype != torch.float32 or sink.numel() != n_heads or not sink.is_contiguous()):
            raise KernelError("attention_masked: the sinks are contiguous float32 [heads]")
        if distance_bias is not None and (distance_bias.dtype != torch.float32 or distance_bias.dim() != 2 or not distance_bias.is_contiguous()
                                          or distance_bias.shape[1] != n_heads or distance_bias.shape[0] < 1):
            raise KernelError("attention_masked: the distance bias is contiguous float32 [distances, heads]")
        n = q.shape[0]
        bt = ctx.arrays[f"block_table_g{group}"]
        if tuple(k_cache.shape[1:]) != (n_kv, page_size, head_dim) or tuple(v_cache.shape[1:]) != (n_kv, value_dim, page_size):
            raise KernelError(f"cache pages have shapes {tuple(k_cache.shape)}, {tuple(v_cache.shape)}")
        if k_cache.dtype != q.dtype:
            raise KernelError("cache and activations differ in dtype")
        out = torch.empty((n, n_heads * value_dim), dtype=q.dtype, device=q.device)
        gsrc, gsplits, ground, gstride = self._gate_source(gate, n)
        vr = value_rotation
        self._check(
            self.lib.yk_attn_masked(
                q.data_ptr(), q.stride(0), out.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), _code(q.dtype),
                ctx.arrays["positions"].data_ptr(), ctx.arrays["token_seq"].data_ptr(), bt.data_ptr(), bt.shape[1], n,
                page_size, head_dim, value_dim, n_heads, n_kv, float(scale), float(softcap or 0.0), int(window or 0),
                int(keep_first or 0), int(self.masked_pages_tiled(q.dtype, head_dim, value_dim, page_size)),
                None if vr is None else vr.cos.data_ptr(), None if vr is None else vr.sin.data_ptr(),
                int(bool(vr is not None and vr.interleaved)), 0 if vr is None else vr.cos.shape[0],
                _ptr(gsrc), 0 if gsrc is None else _code(gsrc.dtype), gsplits, ground, gstride, int(gate_col), int(gate_elems),
                _ptr(distance_bias), 0 if distance_bias is None else distance_bias.shape[0], _ptr(sink), int(bool(chunked)),
                1 if differential is None else 2, lam, map_eps, gain, self._stream(),
            )
        )
        return out

    def attention_finish(self, out, positions, n_heads, value_dim, value_rotation=None, gate=None, gate_col: int = 0,
                         gate_elems: int = 1):
        """In place on an attention's output [N, n_heads * value_dim]: the turn back by the position
        and the gate, as ``attention_masked`` applies them itself."""
        n = out.shape[0]
        gsrc, gsplits, ground, gstride = self._gate_source(gate, n)
        vr = value_rotation
        self._check(
            self.lib.yk_attn_finish(
                out.data_ptr(), _code(out.dtype), positions.data_ptr(), n, value_dim, n_heads,
                None if vr is None else vr.cos.data_ptr(), None if vr is None else vr.sin.data_ptr(),
                int(bool(vr is not None and vr.interleaved)), 0 if vr is None else vr.cos.shape[0],
                _ptr(gsrc), 0 if gsrc is None else _code(gsrc.dtype), gsplits, ground, gstride, int(gate_col), int(gate_elems),
                self._stream(),
            )
        )
        return out

    # ------------------------------------------------ short convolution + gated linear recurrence
    def causal_conv(self, x, weight, bias, state, ctx, act: Optional[str] = None, move_state: bool = False) -> torch.Tensor:
        """Per channel, u_t = bias + sum_j weight[c, j] * x_(t - (taps - 1 - j)) over each request's
        span; inputs before the span come from ``state`` [slots, taps - 1, channels] (not changed here unless
        ``move_state``: it then takes in each request's span, as ``conv_state_push`` would; in a step of single
        tokens the same launch does it).  ``x`` [N, channels] may be a view with a row stride.  ``act`` = "silu":
        applied to u (float32) before it is rounded."""
        if act not in (None, "silu"):
            raise KernelError(f"causal_conv: activation {act!r} is not offered")
        n, channels = x.shape
        taps = weight.shape[1]
        if x.stride(1) != 1 or tuple(weight.shape) != (channels, taps) or not weight.is_contiguous():
            raise KernelError("causal_conv: x must have unit column stride and weight be [channels, taps]")
        if bias is not None and (bias.dtype != weight.dtype or bias.numel() != channels):
            raise KernelError("causal_conv: bias does not match the weight")
        if taps > 1 and (state.dtype != x.dtype or tuple(state.shape[1:]) != (taps - 1, channels)):
            raise KernelError(f"causal_conv: state {tuple(state.shape)} does not hold {taps - 1} inputs of {channels} channels")
        out = torch.empty((n, channels), dtype=x.dtype, device=x.device)
        a = ctx.arrays
        inside = bool(move_state and taps > 1 and ctx.max_qlen == 1)
        self._check(
            self.lib.yk_causal_conv(
                x.data_ptr(), x.stride(0), _code(x.dtype), weight.data_ptr(), _ptr(bias), _code(weight.dtype), _ptr(state),
                a["token_seq"].data_ptr(), a["seq_qstart"].data_ptr(), a["state_slots"].data_ptr(), out.data_ptr(),
                n, channels, taps, int(act == "silu"), int(inside), self._stream(),
            )
        )
        if move_state and taps > 1 and not inside:
            self.conv_state_push(x, state, ctx)
        return out

    # ------------------------------------------------- norms on both sides of a branch, plain feed-forward
    def sandwich_norm(self, residual, branch, post, scale, pre, rows, out_dtype):
        """residual (float32 [N, width], in place unless ``rows`` picks some of them) += scale *
        post(branch); returns pre(residual) in ``out_dtype``, or None without ``pre``.  ``post`` and
        ``pre`` are (weight, bias or None, eps, centred) or None (``post`` None: the branch is added as
        it is); ``branch`` a tensor, a ``SplitSum`` or None.  Without a residual: pre(branch)."""
        n_splits, round_sum, src = 1, 0, branch
        if isinstance(branch, SplitAttention):
            branch = src = branch.merge()
        if isinstance(branch, SplitSum):
            branch.check_live()
            n_splits, round_sum, src = branch.n_splits, branch.round_sum, branch.tensor
        ref = residual if residual is not None else branch
        if ref is None:
            raise KernelError("sandwich_norm: neither a residual nor a branch")
        n, width = ref.shape
        if residual is not None and (residual.dtype != torch.float32 or not residual.is_contiguous() or residual.dim() != 2):
            raise KernelError("the residual stream must be contiguous float32 rows")
        if branch is not None and (tuple(branch.shape) != (n, width) or not src.is_contiguous()):
            raise KernelError(f"branch {tuple(branch.shape)} does not match the rows {(n, width)}")
        if post is not None and branch is None:
            raise KernelError("sandwich_norm: a branch's norm without a branch")
        w_dtype = None
        for c in (post, pre):
            if c is None:
                continue
            w, b = c[0], c[1]
            if w.numel() != width or not w.is_contiguous() or (b is not None and (b.numel() != width or b.dtype != w.dtype or not b.is_contiguous())):
                raise KernelError(f"sandwich_norm: a norm's weight or bias does not fit rows of {width}")
            if w_dtype not in (None, w.dtype):
                raise KernelError("sandwich_norm: the two norms' weights differ in dtype")
            w_dtype = w.dtype
        n_out = n
        if rows is not None:
            if residual is None or rows.dtype != torch.int32 or not rows.is_contiguous():
                raise KernelError("sandwich_norm: gathered rows need a residual and an int32 index")
            n_out = rows.numel()
        out = torch.empty((n_out, width), dtype=out_dtype, device=ref.device) if pre is not None else None
        pa = post if post is not None else (None, None, 0.0, False)
        pb = pre if pre is not None else (None, None, 0.0, False)
        self._check(self.lib.yk_sandwich_norm(
            _ptr(residual), _ptr(src), 0 if src is None else _code(src.dtype), n_splits, round_sum, n,
            _ptr(pa[0]), _ptr(pa[1]), float(pa[2]), int(bool(pa[3])), float(scale), _ptr(pb[0]), _ptr(pb[1]), float(pb[2]),
            int(bool(pb[3])), 0 if w_dtype is None else _code(w_dtype), _ptr(rows), _ptr(out), _code(out_dtype), n_out, width,
            self._stream()))
        return out

    ACTIVATION_KINDS = {"silu": 0, "gelu_tanh": 1, "relu2": 2}

    def activation(self, x, kind: str, out_dtype: torch.dtype) -> torch.Tensor:
        """act(x) elementwise in float32, rounded once; ``x`` a tensor or a product's unreduced slices."""
        if kind not in self.ACTIVATION_KINDS:
            raise KernelError(f"activation {kind!r} is not offered (offered: {sorted(self.ACTIVATION_KINDS)})")
        n_splits, round_sum, src = 1, 0, x
        if isinstance(x, SplitSum):
            x.check_live()
            n_splits, round_sum, src = x.n_splits, x.round_sum, x.tensor
        if not src.is_contiguous():
            raise KernelError("activation: the input must be contiguous")
        out = torch.empty(tuple(x.shape), dtype=out_dtype, device=src.device)
        self._check(self.lib.yk_activation(src.data_ptr(), _code(src.dtype), n_splits, round_sum, self.ACTIVATION_KINDS[kind],
                                           out.data_ptr(), _code(out_dtype), out.numel(), self._stream()))
        return out

    def scale_rows(self, x: torch.Tensor, s: float, softcap: float = 0.0) -> torch.Tensor:
        """x (contiguous float32) *= s, in place; with ``softcap`` c, x = c tanh(s x / c)."""
        if x.dtype != torch.float32 or not x.is_contiguous():
            raise KernelError("scale_rows takes a contiguous float32 tensor")
        self._check(self.lib.yk_scale_rows(x.data_ptr(), float(s), float(softcap), x.numel(), self._stream()))
        return x

    # ------------------------------------------------------------- a stream kept as several copies
    def embed_norm(self, token_ids, table, weight, eps, copies: int) -> torch.Tensor:
        """float32 [N, copies, width]: table[id] divided by its root mean square and times ``weight``, the same in every copy."""
        if table.dim() != 2 or not table.is_contiguous() or weight.dtype != table.dtype or weight.numel() != table.shape[1] or not weight.is_contiguous():
            raise KernelError("embed_norm: a contiguous table and a weight as wide as its rows, of one dtype")
        if token_ids.dtype != torch.int32:
            raise KernelError("embed_norm: token ids are int32")
        n, width = token_ids.numel(), table.shape[1]
        out = torch.empty((n, int(copies), width), dtype=torch.float32, device=table.device)
        self._check(self.lib.yk_embed_norm(token_ids.data_ptr(), table.data_ptr(), _code(table.dtype), table.shape[0], weight.data_ptr(), float(eps),
                                           out.data_ptr(), n, width, int(copies), self._stream()))
        return out

    def streams_norm(self, residual, y, experts, mix, out, read, rows, weight, eps, unit_offset, out_dtype) -> torch.Tensor:
        """``residual`` float32 [N, streams, width], in place: x_t <- sum_s mix[s, t] x_s + out[t] b, where b is ``y`` (a tensor, a
        ``SplitSum`` or None) plus, with ``experts`` = (rows, top, weight, row weights or None), a mixture's uncombined rows as
        ``moe_combine`` sums them; ``mix`` [streams, streams] and ``out`` [streams] float32, None: nothing is pending.  Returns
        norm(sum_s read[s] x_s) * weight in ``out_dtype`` (``read`` None: the plain sum).  With ``rows`` (int32) those
        tokens' rows only, and the residual is left as it is."""
        if residual.dim() != 3 or residual.dtype != torch.float32 or not residual.is_contiguous():
            raise KernelError("streams_norm: the copies are contiguous float32 [N, streams, width]")
        n, streams, width = residual.shape
        for t, count in ((mix, streams * streams), (out, streams), (read, streams)):
            if t is not None and (t.dtype != torch.float32 or t.numel() != count or not t.is_contiguous()):
                raise KernelError("streams_norm: the tables are contiguous float32 [streams, streams] and [streams]")
        if weight.numel() != width or not weight.is_contiguous() or (mix is None) != (out is None):
            raise KernelError(f"streams_norm: the norm's weight has {weight.numel()} elements, rows have {width}")
        if isinstance(y, SplitAttention):
            y = y.merge()
        n_splits, round_sum, src = 1, 0, y
        if isinstance(y, SplitSum):
            y.check_live()
            n_splits, round_sum, src = y.n_splits, y.round_sum, y.tensor
        if y is not None and (tuple(y.shape) != (n, width) or not src.is_contiguous()):
            raise KernelError(f"streams_norm: the branch {tuple(y.shape)} does not match the stream {(n, width)}")
        erows, top, eweight, rweights = experts if experts is not None else (None, 0, 1.0, None)
        if erows is not None and (erows.dtype != torch.float32 or not erows.is_contiguous() or tuple(erows.shape) != (n * top, width)):
            raise KernelError(f"streams_norm: expert rows {tuple(erows.shape)} do not match the stream {(n, width)}")
        if rweights is not None and (rweights.dtype != torch.float32 or rweights.numel() != n * top or not rweights.is_contiguous()):
            raise KernelError("streams_norm: the rows' weights are contiguous float32, one per row")
        if rows is not None and rows.dtype != torch.int32:
            raise KernelError("streams_norm: picked rows are int32")
        n_out = n if rows is None else rows.numel()
        h = torch.empty((n_out, width), dtype=out_dtype, device=residual.device)
        self._check(self.lib.yk_streams_norm(
            residual.data_ptr(), n, streams, width, _ptr(src), 0 if src is None else _code(src.dtype), n_splits, round_sum, _ptr(erows), int(top),
            float(eweight), _ptr(rweights), _ptr(mix), _ptr(out), _ptr(read), _ptr(rows), weight.data_ptr(), _code(weight.dtype), float(eps),
            int(bool(unit_offset)), h.data_ptr(), _code(out_dtype), n_out, self._stream()))
        return h

    # ------------------------------------------------------------- attention over one latent per token
    def latent_prepare(self, proj, q_rank, q_norm, eps, act_dtype, kv_col=0, kv_rank=0, rot_dim=0, kv_norm=None, rotation=None,
                       positions=None, pages=None, slots=None, page_size=0, values=None) -> torch.Tensor:
        """From the stacked down-projection's rows ``proj`` [N, >= q_rank (+ sections)]: the query
        latent rmsnorm(proj[:, :q_rank]) * q_norm [N, q_rank]; and, with ``kv_rank`` > 0, each token's
        page row [rmsnorm(proj[:, kv_col : kv_col + kv_rank]) * kv_norm | the next rot_dim elements turned
        by the token's position] written at its slot of ``pages`` [pages, 1, page_size, kv_rank + rot_dim], and
        the normed latent once more, transposed, into ``values`` [pages, 1, kv_rank, page_size] where given."""
        self._rows(proj, "latent_prepare input")
        n = proj.shape[0]
        if proj.dtype != act_dtype:
            raise KernelError("latent_prepare: the projection comes in the activation dtype")
        if q_norm.numel() != q_rank or not q_norm.is_contiguous():
            raise KernelError("latent_prepare: the query latent's norm weight does not fit")
        c_q = torch.empty((n, q_rank), dtype=act_dtype, device=proj.device)
        cos = sin = None
        max_pos = inter = 0
        if kv_rank:
            if kv_norm is None or kv_norm.numel() != kv_rank or kv_norm.dtype != q_norm.dtype or not kv_norm.is_contiguous():
                raise KernelError("latent_prepare: the latent's norm weight does not fit")
            if pages is None or pages.dtype != act_dtype or not pages.is_contiguous() or pages.dim() != 4 or pages.shape[1] != 1 \
                    or pages.shape[2] != page_size or pages.shape[3] != kv_rank + rot_dim:
                raise KernelError(f"latent_prepare: pages {None if pages is None else tuple(pages.shape)} do not hold rows of {kv_rank + rot_dim}")
            if values is not None and (values.dtype != act_dtype or not values.is_contiguous()
                                       or tuple(values.shape) != (pages.shape[0], 1, kv_rank, page_size)):
                raise KernelError(f"latent_prepare: transposed pages {tuple(values.shape)} do not match the pages")
            if rot_dim:
                if rotation is None or rotation.rotary_dim != rot_dim:
                    raise KernelError("latent_prepare: the rotation must cover the rotated part exactly")
                cos, sin, max_pos, inter = rotation.cos, rotation.sin, rotation.cos.shape[0], int(rotation.interleaved)
        self._check(self.lib.yk_latent_prepare(
            proj.data_ptr(), proj.stride(0), _code(proj.dtype), q_rank, q_norm.data_ptr(), _code(q_norm.dtype), float(eps),
            c_q.data_ptr(), kv_col, kv_rank, rot_dim, _ptr(kv_norm), _ptr(positions), _ptr(cos), _ptr(sin), inter, max_pos,
            _ptr(pages) if kv_rank else None, _ptr(values) if kv_rank else None, page_size, _ptr(slots) if kv_rank else None, n,
            self._stream()))
        return c_q

    # tokens from which the per-head products run on the matrix cores (where sizes and types allow)
    HEAD_LINEAR_MFMA_FROM = 33

    def head_weights_transposed(self, w: torch.Tensor) -> Optional[torch.Tensor]:
        """What ``head_linear`` takes as ``w_t``: the weights [heads, in, out] once more as [heads, out, in],
        where the matrix-core form may use them (bfloat16, sizes it is built for); else None."""
        if w.dtype != torch.bfloat16 or w.dim() != 3 or not self._ask("yk_head_linear_mfma_ok", w.shape[1], w.shape[2], 0):
            return None
        return w.transpose(1, 2).contiguous()

    def head_linear(self, x, w, n_heads, in_dim, out_dim, out_dtype, tail=0, rotation=None, positions=None, gate=None, gate_col=0,
                    w_t=None, gate_elems=1):
        """Per head, out[n, h, :out_dim] = x[n, h, :in_dim] . w[h] with w [heads, in_dim, out_dim]
        (float32 sums).  ``tail`` further elements of every head of x follow the product in the output,
        turned by the token's position (``rotation``, ``positions``); ``gate`` [N, >= gate_col + heads]:
        head h's output is multiplied by sigmoid(gate[n, gate_col + h]) (``gate_elems`` = out_dim: element o of it by
        sigmoid(gate[n, gate_col + h * out_dim + o])).  ``w_t`` (``head_weights_transposed``):
        with it, products of many tokens run on the matrix cores (a float32 input as two bfloat16 parts)."""
        self._rows(x, "head_linear input")
        n = x.shape[0]
        if tuple(w.shape) != (n_heads, in_dim, out_dim) or not w.is_contiguous() or x.shape[1] != n_heads * (in_dim + tail):
            raise KernelError(f"head_linear: input {tuple(x.shape)} and weight {tuple(w.shape)} do not fit {n_heads} heads of {in_dim} (+{tail}) -> {out_dim}")
        out = torch.empty((n, n_heads * (out_dim + tail)), dtype=out_dtype, device=x.device)
        if gate is not None:
            self._rows(gate, "head_linear gate")
            if gate_elems not in (1, out_dim) or gate.shape[0] != n or gate.shape[1] < gate_col + n_heads * gate_elems:
                raise KernelError("head_linear: the gate's rows do not hold a column per head (or per output element)")
        cos = sin = None
        inter = 0
        if tail:
            if rotation is None or rotation.rotary_dim != tail or positions is None:
                raise KernelError("head_linear: the tail needs a rotation that covers it exactly, and positions")
            cos, sin, inter = rotation.cos, rotation.sin, int(rotation.interleaved)
        gate_ok = gate is None or (gate.dtype == out_dtype if x.dtype == torch.float32 else False)
        if (w_t is not None and n >= self.HEAD_LINEAR_MFMA_FROM and tuple(w_t.shape) == (n_heads, out_dim, in_dim) and w_t.is_contiguous()
                and w_t.dtype == torch.bfloat16 and self._ask("yk_head_linear_mfma_ok", in_dim, out_dim, tail)
                and x.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0 and (in_dim + tail) % 8 == 0 and gate_ok
                and ((x.dtype, out_dtype) in ((torch.bfloat16, torch.float32), (torch.float32, torch.bfloat16)))
                and (x.dtype == torch.float32 or gate is None)):
            self._check(self.lib.yk_head_linear_mfma(
                x.data_ptr(), x.stride(0), _code(x.dtype), w_t.data_ptr(), out.data_ptr(), _code(out_dtype), n_heads, in_dim, out_dim,
                tail, _ptr(positions), _ptr(cos), _ptr(sin), inter, _ptr(gate), 0 if gate is None else _code(gate.dtype),
                0 if gate is None else gate.stride(0), gate_col, int(gate_elems), n, self._stream()))
            return out
        self._check(self.lib.yk_head_linear(
            x.data_ptr(), x.stride(0), _code(x.dtype), w.data_ptr(), _code(w.dtype), out.data_ptr(), _code(out_dtype), n_heads, in_dim,
            out_dim, tail, _ptr(positions), _ptr(cos), _ptr(sin), inter, _ptr(gate), 0 if gate is None else _code(gate.dtype),
            0 if gate is None else gate.stride(0), gate_col, int(gate_elems), n, self._stream()))
        return out

    def latent_attention_on_matrix_cores(self, act_dtype: torch.dtype, kv_rank: int, rot_dim: int, page_size: int) -> bool:
        """Whether ``latent_attention`` has its matrix-core form for these sizes; that form reads the
        latent a second time from transposed pages (``values``), which the caller then has to keep."""
        return act_dtype == torch.bfloat16 and bool(self._ask("yk_latent_mfma_ok", kv_rank, rot_dim, page_size))

    def latent_tile_tokens(self, n_heads: int, matrix_cores: bool = False) -> int:
        """Consecutive tokens of a request that one tile of ``latent_attention`` takes."""
        return self._ask("yk_latent_mfma_tile_tokens" if matrix_cores else "yk_latent_tile_tokens", n_heads)

    @staticmethod
    def latent_attention_splits(n_tiles: int, n_heads: int, max_ctx: int) -> int:
        """Into how many workgroups the matrix-core form divides the keys of a tile: none while the
        tiles alone make some hundreds of waves; else as many as that takes, each with at least 128 keys."""
        waves = n_tiles * -(-n_heads // 16)
        return max(1, min(-(-512 // max(waves, 1)), max(1, -(-max_ctx // 32) // 4), 64))

    def latent_attention(self, q_lat, pages, n_heads, kv_rank, rot_dim, scale, ctx, group, page_size, tiles=None, values=None,
                         splits: Optional[int] = None, sink=None) -> torch.Tensor:
        """Causal softmax attention of ``q_lat`` (float32 [N, heads * (kv_rank + rot_dim)]) over the page
        rows [c | kr] of each token's request: scores q . row * scale, the result sum_j p_j c_j as
        float32 [N, heads * kv_rank].  ``tiles``: the step's spans cut into ``latent_tile_tokens`` tokens
        (rows of request, first token, count, first position).  ``sink`` (float32 [heads]): exp(sink_h) joins the
        softmax's denominator of head h, a score with no key and no value."""
        n = q_lat.shape[0]
        width = kv_rank + rot_dim
        if sink is not None and (sink.dtype != torch.float32 or sink.numel() != n_heads or not sink.is_contiguous()):
            raise KernelError("latent_attention: the sinks are contiguous float32, one per head")
        if q_lat.dtype != torch.float32 or not q_lat.is_contiguous() or q_lat.shape[1] != n_heads * width:
            raise KernelError("latent_attention: queries are contiguous float32 [N, heads * (kv_rank + rot_dim)]")
        if pages.dim() != 4 or pages.shape[1] != 1 or pages.shape[2] != page_size or pages.shape[3] != width or not pages.is_contiguous():
            raise KernelError(f"latent_attention: pages {tuple(pages.shape)} do not hold rows of {width}")
        if tiles is None:
            tiles = ctx.arrays[f"latent_tiles_{self.latent_tile_tokens(n_heads)}"]
        bt = ctx.arrays[f"block_table_g{group}"]
        out = torch.empty((n, n_heads * kv_rank), dtype=torch.float32, device=q_lat.device)
        if values is not None:
            # the matrix-core form: ``tiles`` are cut for it (latent_tile_tokens(heads, True))
            if tiles is None or not self.latent_attention_on_matrix_cores(pages.dtype, kv_rank, rot_dim, page_size) or not values.is_contiguous() \
                    or values.dtype != pages.dtype or tuple(values.shape) != (pages.shape[0], 1, kv_rank, page_size):
                raise KernelError("latent_attention: transposed pages are for the matrix-core form, with tiles cut for it")
            if splits is None:  # (given: tests and measurements force a number)
                splits = self.latent_attention_splits(tiles.shape[0], n_heads, int(ctx.max_ctx))
            floats = self.lib.yk_latent_mfma_workspace(tiles.shape[0], n_heads, kv_rank, splits)
            ws = self._ws(floats) if floats else None
            self._check(self.lib.yk_latent_attention_mfma(
                q_lat.data_ptr(), pages.data_ptr(), values.data_ptr(), tiles.data_ptr(), tiles.shape[0], bt.data_ptr(), bt.shape[1],
                page_size, n_heads, kv_rank, rot_dim, float(scale), splits, _ptr(sink), _ptr(ws), 0 if ws is None else ws.numel(), out.data_ptr(),
                self._stream()))
            return out
        self._check(self.lib.yk_latent_attention(
            q_lat.data_ptr(), pages.data_ptr(), _code(pages.dtype), tiles.data_ptr(), tiles.shape[0], bt.data_ptr(), bt.shape[1],
            page_size, n_heads, kv_rank, rot_dim, float(scale), _ptr(sink), out.data_ptr(), self._stream()))
        return out

    # ---------------------------------------------------------------- a matrix per head as the memory
    def conv_state_push(self, x, state, ctx) -> None:
        """``state`` [slots, keep, channels] (a request's last inputs of a convolution, oldest first)
        takes in each request's span of ``x`` [N, channels]."""
        n, channels = x.shape
        if x.stride(1) != 1 or state.dtype != x.dtype or state.dim() != 3 or state.shape[2] != channels or not state.is_contiguous():
            raise KernelError("conv_state_push: the state does not match the inputs")
        a = ctx.arrays
        self._check(self.lib.yk_conv_state_push(
            x.data_ptr(), x.stride(0), _code(x.dtype), state.data_ptr(), a["seq_qstart"].data_ptr(), a["seq_qlen"].data_ptr(),
            a["state_slots"].data_ptr(), a["seq_qstart"].numel(), state.shape[1], channels, self._stream()))

    def linear_state_scan(self, qkv, n_heads, n_kv, dim, vdim, state, ctx, q_scale=1.0, unit_eps=None, decay=None, beta=None,
                          columns=None, skip=None, bonus=None):
        """The recurrence S <- diag(a) S; u = v or beta (v - S^T k); S += k u^T; o = S^T q over each
        request's span, S [slots, heads, dim, vdim] float32 updated in place.  ``qkv`` [N, >= 2 * kv_heads *
        dim + heads * vdim]: columns [q | k | v].  ``unit_eps``: q and k are divided by sqrt(sum of squares +
        unit_eps) first; q is multiplied by ``q_scale``.  ``decay``: ("head", x, col, A_log, dt_bias): a =
        exp(-exp(A_log) softplus(x[:, col + h] + dt_bias)); ("channel", z, col, bias, tau): a_i = sigmoid(z[:,
        col + h * dim + i] + bias)^(1 / tau); ("channel_softplus", z, col, A_log, dt_bias): a_i = exp(-exp(A_log_h)
        softplus(z[:, col + h * dim + i] + dt_bias)); ("channel_exp", z, col, bias): a_i = exp(-exp(z[:, col + h * dim + i] +
        bias)); x, z float32; ("fixed", a): a constant per head, a float32 [heads].  ``beta``: (x, col) -> sigmoid(x[:, col + h]), x float32 or of ``qkv``'s dtype, or
        None for plain writes, or "step": u = dt v with the step dt = softplus(x[:, col + h] + dt_bias) of the head's
        decay.  ``columns`` = (q, k, v): where the kv heads' queries and keys and the heads' values start in a row
        (default 0, n_kv * dim, 2 * n_kv * dim).  ``skip`` (float32 [heads]): o += skip_h v.  ``bonus`` (float32
        [heads, dim], plain writes): o = (S + diag(bonus) k v^T)^T q of the memory before the token's decay and write.
        Returns o float32 [N, heads * vdim]."""
        self._rows(qkv, "linear_state_scan input")
        n = qkv.shape[0]
        if state.dtype != torch.float32 or not state.is_contiguous() or tuple(state.shape[1:]) != (n_heads, dim, vdim):
            raise KernelError(f"linear_state_scan: state {tuple(state.shape)} does not hold {n_heads} matrices of {dim} x {vdim}")
        if decay[0] == "fixed":
            decay = ("fixed", None, 0, decay[1])
        kind, src, col = decay[0], decay[1], int(decay[2])
        need = n_heads if kind == "head" else n_heads * dim
        write_mode = 0 if beta is None else (2 if isinstance(beta, str) else 1)
        if isinstance(beta, str) and (beta != "step" or kind != "head"):
            raise KernelError("linear_state_scan: a write by the step goes with the decay per head")
        if write_mode != 1:
            beta = None
        q_col, k_col, v_col = columns if columns is not None else (0, n_kv * dim, 2 * n_kv * dim)
        if skip is not None and (skip.dtype != torch.float32 or skip.numel() != n_heads or not skip.is_contiguous()):
            raise KernelError("linear_state_scan: the skip is contiguous float32, one number per head")
        if bonus is not None and (bonus.dtype != torch.float32 or bonus.numel() != n_heads * dim or not bonus.is_contiguous() or write_mode or skip is not None):
            raise KernelError("linear_state_scan: the bonus is contiguous float32 [heads, dim] and goes with plain writes and no skip")
        for t, what, cols in (((src, "decay", col + need),) if src is not None else ()) + (((beta[0], "beta", int(beta[1]) + n_heads),) if beta is not None else ()):
            if (t.dtype != torch.float32 and not (what == "beta" and t.dtype == qkv.dtype)) or t.dim() != 2 or t.stride(1) != 1 or t.shape[0] != n or t.shape[1] < cols:
                raise KernelError(f"linear_state_scan: the {what}'s input must be float32 rows of at least {cols} columns")
        if kind == "head":
            p0, p1, tau = decay[3], decay[4], 1.0
            ok = all(p.dtype == torch.float32 and p.numel() == n_heads and p.is_contiguous() for p in (p0, p1))
        elif kind == "channel":
            p0, p1, tau = decay[3], None, float(decay[4])
            ok = p0.dtype == torch.float32 and p0.numel() == n_heads * dim and p0.is_contiguous()
        elif kind == "channel_softplus":
            p0, p1, tau = decay[3], decay[4], 1.0
            ok = all(p.dtype == torch.float32 and p.numel() == size and p.is_contiguous() for p, size in ((p0, n_heads), (p1, n_heads * dim)))
        elif kind == "channel_exp":
            p0, p1, tau = decay[3], None, 1.0
            ok = p0.dtype == torch.float32 and p0.numel() == n_heads * dim and p0.is_contiguous()
        elif kind == "fixed":
            p0, p1, tau = decay[3], None, 1.0
            ok = p0.dtype == torch.float32 and p0.numel() == n_heads and p0.is_contiguous()
        else:
            raise KernelError(f"linear_state_scan: unknown kind of decay {kind!r}")
        if not ok:
            raise KernelError("linear_state_scan: the decay's constants must be contiguous float32 of the heads' size")
        a = ctx.arrays
        mode = {"head": 0, "channel": 1, "channel_softplus": 2, "channel_exp": 3, "fixed": 4}[kind]
        beta_f32 = beta is not None and beta[0].dtype == torch.float32
        # where tokens are many their decays per channel are made first, once for all the columns that read them
        many = mode not in (0, 4) and n > 4 * a["seq_qstart"].numel()
        decays = torch.empty((n, n_heads * dim), dtype=torch.float32, device=qkv.device) if many else None
        out = torch.empty((n, n_heads * vdim), dtype=torch.float32, device=qkv.device)
        self._check(self.lib.yk_linear_state_scan(
            qkv.data_ptr(), qkv.stride(0), _code(qkv.dtype), n_heads, n_kv, dim, vdim, state.data_ptr(), a["seq_qstart"].data_ptr(),
            a["seq_qlen"].data_ptr(), a["state_slots"].data_ptr(), a["seq_qstart"].numel(), n, float(q_scale),
            -1.0 if unit_eps is None else float(unit_eps), mode, _ptr(src), 0 if src is None else src.stride(0), col,
            p0.data_ptr(), _ptr(p1), tau, beta[0].data_ptr() if beta_f32 else None, 0 if beta is None else beta[0].stride(0),
            0 if beta is None else int(beta[1]), out.data_ptr(), int(q_col), int(k_col), int(v_col), write_mode, _ptr(skip),
            beta[0].data_ptr() if beta is not None and not beta_f32 else None, _ptr(bonus), _ptr(decays), self._stream()))
        return out

    @staticmethod
    def fixed_decay_chunk() -> int:
        """Tokens of a span that meet in products in ``fixed_decay_scan``."""
        return 64

    def scan_inputs(self, proj, n_heads, dim, vdim, k_scale=1.0, rotation=None, positions=None, act=None) -> torch.Tensor:
        """float32 rows [q | k | v] as they enter a recurrence, from a projection's rows [q | k | v | ...]: ``act`` ("silu") on all
        three, ``rotation`` on q and k by the tokens' positions, k times ``k_scale``."""
        self._rows(proj, "scan_inputs input")
        if act not in (None, "silu"):
            raise KernelError(f"scan_inputs: activation {act!r} is not offered")
        n = proj.shape[0]
        if proj.shape[1] < n_heads * (2 * dim + vdim):
            raise KernelError(f"scan_inputs: rows of {proj.shape[1]} elements, fewer than the heads need")
        r = rotation
        if r is not None and (r.cos.dtype != torch.float32 or r.cos.shape != r.sin.shape or r.cos.shape[1] != r.rotary_dim // 2 or positions.numel() != n):
            raise KernelError("scan_inputs: rotary tables are float32 [positions, rotary_dim/2], and every token has a position")
        out = torch.empty((n, n_heads * (2 * dim + vdim)), dtype=torch.float32, device=proj.device)
        self._check(self.lib.yk_scan_inputs(
            proj.data_ptr(), proj.stride(0), _code(proj.dtype), n_heads, dim, vdim, _ptr(positions) if r is not None else None,
            None if r is None else r.cos.data_ptr(), None if r is None else r.sin.data_ptr(), 0 if r is None else r.rotary_dim,
            int(bool(r is not None and r.interleaved)), 0 if r is None else r.cos.shape[0], float(k_scale), int(act == "silu"), out.data_ptr(), n,
            self._stream()))
        return out

    # scratch for the sums of a step's chunks (a few hundred chunks at these sizes; more are taken slab by slab)
    DECAY_SLAB_BYTES = 256 << 20

    def fixed_decay_scan(self, proj, n_heads, dim, vdim, state, ctx, decay, k_scale=1.0, rotation=None, act=None, chunks=None, seq_chunk0=None,
                         form: Optional[str] = None):
        """The recurrence S <- a_h S + k v^T, o = S^T q with a constant decay per head (``decay`` float32 [heads]) over each
        request's span, S [slots, heads, dim, vdim] float32 updated in place.  ``proj`` [N, >= heads * (2 * dim + vdim)]: columns
        [q | k | v | ...] as projected; see ``scan_inputs`` for what is made of them first.  Returns o float32 [N, heads * vdim].

        Steps of single tokens take a kernel of their own; spans in bfloat16 the matrix cores, chunk by chunk (``chunks`` and
        ``seq_chunk0``: ``span_chunks`` and ``chunk_starts`` of ``fixed_decay_chunk()`` tokens), where the sizes allow; what is left
        is walked token by token.  ``form`` ("step", "chunks", "walk") forces one of them (tests, measurements)."""
        self._rows(proj, "fixed_decay_scan input")
        if act not in (None, "silu"):
            raise KernelError(f"fixed_decay_scan: activation {act!r} is not offered")
        n = proj.shape[0]
        a = ctx.arrays
        positions, n_seqs = a["positions"], a["seq_qstart"].numel()
        if state.dtype != torch.float32 or not state.is_contiguous() or tuple(state.shape[1:]) != (n_heads, dim, vdim):
            raise KernelError(f"fixed_decay_scan: state {tuple(state.shape)} does not hold {n_heads} matrices of {dim} x {vdim}")
        if decay.dtype != torch.float32 or decay.numel() != n_heads or not decay.is_contiguous() or positions.numel() != n:
            raise KernelError("fixed_decay_scan: the decays are contiguous float32 [heads], and every token has a position")
        if proj.shape[1] < n_heads * (2 * dim + vdim):
            raise KernelError(f"fixed_decay_scan: rows of {proj.shape[1]} elements, fewer than the heads need")
        r = rotation
        if r is not None and (r.cos.dtype != torch.float32 or r.cos.shape != r.sin.shape or r.cos.shape[1] != r.rotary_dim // 2):
            raise KernelError("fixed_decay_scan: rotary tables are float32 [positions, rotary_dim/2]")
        rot, inter, rows = (0, 0, 0) if r is None else (r.rotary_dim, int(bool(r.interleaved)), r.cos.shape[0])
        inputs = (None if r is None else r.cos.data_ptr(), None if r is None else r.sin.data_ptr(), rot, inter, rows, float(k_scale), int(act == "silu"))
        can_step = ctx.max_qlen == 1 and vdim % 4 == 0 and dim <= 4096
        can_chunk = (proj.dtype == torch.bfloat16 and chunks is not None and proj.stride(0) % 8 == 0 and proj.data_ptr() % 16 == 0
                     and self._ask("yk_decay_scan_chunks_ok", dim, vdim, rot, inter) == 1)
        if form is None:
            form = "step" if can_step else ("chunks" if can_chunk else "walk")
        if (form == "step" and not can_step) or (form == "chunks" and not can_chunk):
            raise KernelError(f"fixed_decay_scan: this step cannot take the form {form!r}")
        if form == "walk":
            x = self.scan_inputs(proj, n_heads, dim, vdim, k_scale, rotation, positions, act)
            return self.linear_state_scan(x, n_heads, n_heads, dim, vdim, state, ctx, decay=("fixed", decay))
        out = torch.empty((n, n_heads * vdim), dtype=torch.float32, device=proj.device)
        if form == "step":
            self._check(self.lib.yk_decay_scan_step(
                proj.data_ptr(), proj.stride(0), _code(proj.dtype), n_heads, dim, vdim, state.data_ptr(), a["seq_qstart"].data_ptr(),
                a["state_slots"].data_ptr(), n_seqs, positions.data_ptr(), *inputs, decay.data_ptr(), out.data_ptr(), self._stream()))
            return out
        n_chunks = chunks.shape[0]
        if seq_chunk0 is None or seq_chunk0.numel() != n_seqs + 1 or chunks.shape[1] != 3:
            raise KernelError("fixed_decay_scan: chunks are rows of (request, first token, count), with every request's first row")
        slab = max(1, min(n_chunks, self.DECAY_SLAB_BYTES // (4 * n_heads * dim * vdim)))
        need = int(self.lib.yk_decay_scan_chunks_bytes(n_chunks, slab, n_heads, dim, vdim, int(act == "silu")))
        ws = torch.empty(need, dtype=torch.uint8, device=proj.device)
        self._check(self.lib.yk_decay_scan_chunks(
            proj.data_ptr(), proj.stride(0), n_heads, dim, vdim, state.data_ptr(), a["state_slots"].data_ptr(), n_seqs, chunks.data_ptr(), n_chunks,
            seq_chunk0.data_ptr(), slab, positions.data_ptr(), *inputs, decay.data_ptr(), ws.data_ptr(), need, out.data_ptr(), self._stream()))
        return out

    def gated_head_norm(self, o, weight, eps, gate, gate_col, n_heads, vdim, out_dtype, gate_first: bool = False,
                        gate_act: str = "silu") -> torch.Tensor:
        """Per head, o / sqrt(mean(o^2) + eps) * weight * silu(gate[:, gate_col + h * vdim + .]); ``o`` float32
        [N, heads * vdim], ``weight`` [vdim] shared by the heads, or [heads * vdim], or None.  The "heads" are whatever equal
        parts of a row are normed each by its own root mean square.  ``gate_first``: the gate comes before the
        norm, rms(o * silu(gate)) * weight.  ``gate_act`` "sigmoid": the sigmoid in silu's place.  The gate comes in
        ``out_dtype`` or float32."""
        if gate_act not in ("silu", "sigmoid"):
            raise KernelError(f"gated_head_norm: gate {gate_act!r} is not offered")
        n = o.shape[0]
        self._rows(gate, "gated_head_norm gate")
        if o.dtype != torch.float32 or not o.is_contiguous() or o.shape[1] != n_heads * vdim or (weight is not None and (
                weight.numel() not in (vdim, n_heads * vdim) or not weight.is_contiguous())):
            raise KernelError("gated_head_norm: o is contiguous float32 [N, heads * vdim], the weight [vdim] or [heads * vdim]")
        if gate.dtype not in (out_dtype, torch.float32) or gate.shape[0] != n or gate.shape[1] < gate_col + n_heads * vdim:
            raise KernelError("gated_head_norm: the gate does not fit")
        out = torch.empty((n, n_heads * vdim), dtype=out_dtype, device=o.device)
        self._check(self.lib.yk_gated_head_norm(
            o.data_ptr(), _ptr(weight), _F32 if weight is None else _code(weight.dtype), float(eps), gate.data_ptr(), _code(gate.dtype), gate.stride(0),
            gate_col, n_heads, vdim, out.data_ptr(), _code(out_dtype), n, int(weight is not None and (weight.numel() != vdim or n_heads == 1)),
            int(bool(gate_first)), int(gate_act == "sigmoid"), self._stream()))
        return out

    # ------------------------------------------------- inputs mixed with the token before's, low-rank pairs
    def token_shift_mix(self, x, mu, state, ctx) -> torch.Tensor:
        """[mixes, N, width]: x + (x' - x) * mu[s] for every row of ``mu`` (float32 [mixes, width]), x' the row of the
        request's token before (``state`` [slots, width] for a span's first one; it is left at the span's last row)."""
        self._rows(x, "token_shift_mix input")
        n, width = x.shape
        if not x.is_contiguous() or mu.dtype != torch.float32 or mu.dim() != 2 or mu.shape[1] != width or not mu.is_contiguous():
            raise KernelError("token_shift_mix: contiguous rows, and float32 mixes [mixes, width]")
        if state.dtype != x.dtype or tuple(state.shape[1:]) != (width,) or not state.is_contiguous():
            raise KernelError(f"token_shift_mix: the state {tuple(state.shape)} does not hold a row of {width}")
        a = ctx.arrays
        out = torch.empty((mu.shape[0], n, width), dtype=x.dtype, device=x.device)
        self._check(self.lib.yk_token_shift_mix(
            x.data_ptr(), _code(x.dtype), mu.data_ptr(), mu.shape[0], state.data_ptr(), a["token_seq"].data_ptr(), a["seq_qstart"].data_ptr(),
            a["seq_qlen"].data_ptr(), a["state_slots"].data_ptr(), out.data_ptr(), n, width, self._stream()))
        return out

    def grouped_linear(self, x, w, group_rows: int, out_dtype) -> torch.Tensor:
        """``w``'s rows come in groups of ``group_rows`` (the last may have fewer), each with an input of its own: columns
        g * group_rows .. of the result are x[g] . (group g of w)^T.  ``x`` [groups, N, K].  Few rows of bfloat16 run as one
        launch; otherwise a product a group, each writing its columns."""
        groups, m, k = x.shape
        n = w.shape[0]
        self._rows(w, "grouped_linear weight")
        if w.shape[1] != k or not x.is_contiguous() or group_rows < 1 or -(-n // group_rows) != groups:
            raise KernelError(f"grouped_linear: {groups} inputs of {k} columns against {n} rows in groups of {group_rows}")
        y = torch.empty((m, n), dtype=out_dtype, device=x.device)
        if m == 0:
            return y
        bf = torch.bfloat16
        aligned = x.dtype == bf and w.dtype == bf and k % 8 == 0 and w.stride(0) % 8 == 0 and w.data_ptr() % 16 == 0 and x.data_ptr() % 16 == 0
        if aligned and m <= 32 and group_rows % 64 == 0:
            splits = self._ask("yk_gemm_skinny_splits", m, n, k, 0)
            ws = self._gemm_ws(splits * m * n) if splits > 1 else None
            self._check(self.lib.yk_gemm_mfma_skinny_grouped(
                x.data_ptr(), m * k, group_rows, w.data_ptr(), y.data_ptr(), _code(out_dtype), _ptr(ws), 0 if ws is None else ws.numel(),
                m, n, k, k, w.stride(0), n, self._stream()))
            return y
        size = y.element_size()
        for g in range(groups):
            rows = min(group_rows, n - g * group_rows)
            xg, wg, yp = x[g], w[g * group_rows:], y.data_ptr() + g * group_rows * size
            if aligned and m > SKINNY_MAX_ROWS and rows >= 64 and yp % 16 == 0 and wg.data_ptr() % 16 == 0 and xg.data_ptr() % 16 == 0 and (n * size) % 16 == 0:
                if self._library_workspace is None:
                    self._library_workspace = torch.empty(self.LIBRARY_WORKSPACE_BYTES, dtype=torch.uint8, device=self.device)
                self._check(self.lib.yk_gemm_library(
                    xg.data_ptr(), wg.data_ptr(), yp, _code(out_dtype), m, rows, k, k, w.stride(0), n, self._library_workspace.data_ptr(),
                    self._library_workspace.numel(), None, self._stream()))
            elif aligned and wg.data_ptr() % 16 == 0 and xg.data_ptr() % 16 == 0:
                splits = self._ask("yk_gemm_skinny_splits", m, rows, k, 0)
                ws = self._gemm_ws(splits * m * rows) if splits > 1 else None
                rc = self.lib.yk_gemm_mfma_skinny(
                    xg.data_ptr(), wg.data_ptr(), yp, _code(out_dtype), _ptr(ws), 0 if ws is None else ws.numel(), m, rows, k, k, w.stride(0),
                    n, 0, 0, self._stream())
                if rc < 0:
                    self._check(rc)
            else:
                self._check(self.lib.yk_gemm_fma(xg.data_ptr(), _code(x.dtype), wg.data_ptr(), _code(w.dtype), yp, _code(out_dtype), m, rows, k,
                                                 k, w.stride(0), n, self._stream()))
        return y

    LOW_RANK_ACTS = {None: 0, "tanh": 1}

    def low_rank(self, y, w, act: Optional[str] = None) -> torch.Tensor:
        """float32 act(y) . w^T: the second product of a low-rank pair, ``y`` [N, rank] (a view with a row stride may be given),
        ``w`` [columns, rank].  Few tokens: one launch, the activation and the sums in float32.  Many: the activation's rows,
        rounded, and a product."""
        if act not in self.LOW_RANK_ACTS:
            raise KernelError(f"low_rank: activation {act!r} is not offered")
        self._rows(y, "low_rank input")
        n, rank = y.shape
        if w.dim() != 2 or w.shape[1] != rank or not w.is_contiguous():
            raise KernelError(f"low_rank: the weight {tuple(w.shape)} does not take rows of {rank}")
        code = self.LOW_RANK_ACTS[act]
        if n <= SKINNY_MAX_ROWS and rank <= 1536 and (y.dtype == torch.bfloat16 or w.dtype == torch.float32):
            out = torch.empty((n, w.shape[0]), dtype=torch.float32, device=y.device)
            self._check(self.lib.yk_low_rank(y.data_ptr(), y.stride(0), _code(y.dtype), w.data_ptr(), _code(w.dtype), code, out.data_ptr(), n,
                                             w.shape[0], rank, self._stream()))
            return out
        if code:
            rows = torch.empty((n, rank), dtype=y.dtype, device=y.device)
            self._check(self.lib.yk_act_rows(y.data_ptr(), y.stride(0), _code(y.dtype), code, rows.data_ptr(), n, rank, self._stream()))
            y = rows
        return self.linear(y, w, torch.float32)

    # spans of more than this many tokens are scanned in chunks (cut by the caller)
    RGLRU_CHUNKED_FROM = 32

    def rglru(self, u, y, x, wa_t, ba, wi_t, bi, lam, rate, s_state, conv_state, taps, ctx, wa=None, wi=None,
              chunks=None, seq_chunk0=None) -> torch.Tensor:
        """The real-gated linear recurrence over each request's span.  ``u`` [N, C] the convolved
        branch, ``y`` [N, C] the other branch before its gelu, ``x`` [N, C] the convolution's inputs (its
        state is brought up to date here); gate matrices transposed [blocks, in, out] (and, as ``wa`` /
        ``wi``, in their own layout [blocks, out, in], which the matrix-core form of the gates reads).
        ``chunks`` [n, 3] (request, first token, count) and ``seq_chunk0`` [requests + 1] cut the spans for
        the scan in chunks, which runs when the step's longest span exceeds ``RGLRU_CHUNKED_FROM``.  Returns
        S_t * gelu(y_t) [N, C]; ``s_state`` [slots, C] float32 and ``conv_state`` are left as after the span."""
        n, channels = u.shape
        blocks = wa_t.shape[0]
        bs = channels // blocks
        if tuple(wa_t.shape) != (blocks, bs, bs) or tuple(wi_t.shape) != (blocks, bs, bs) or not wa_t.is_contiguous() or not wi_t.is_contiguous():
            raise KernelError("rglru: gate matrices must be contiguous [blocks, width / blocks, width / blocks]")
        for t in (ba, bi, lam):
            if t.numel() != channels or t.dtype != wa_t.dtype or not t.is_contiguous():
                raise KernelError("rglru: gate biases and decay parameters are [width] in the matrices' dtype")
        if s_state.dtype != torch.float32 or s_state.shape[1] != channels:
            raise KernelError("rglru: the recurrent state is float32 [slots, width]")
        if not u.is_contiguous() or y.stride(1) != 1 or x.stride(1) != 1 or y.dtype != u.dtype or x.dtype != u.dtype:
            raise KernelError("rglru: branches must share a dtype and have unit column stride")
        a = torch.empty((n, channels), dtype=torch.float32, device=u.device)
        b = torch.empty((n, channels), dtype=torch.float32, device=u.device)
        self._check(
            self.lib.yk_rglru_gates(
                u.data_ptr(), _code(u.dtype), wa_t.data_ptr(), ba.data_ptr(), wi_t.data_ptr(), bi.data_ptr(), lam.data_ptr(),
                _code(wa_t.dtype), float(rate), a.data_ptr(), b.data_ptr(), n, channels, blocks,
                _ptr(wa) if wa is not None and wa.is_contiguous() and wa.dtype == wa_t.dtype else None,
                _ptr(wi) if wi is not None and wi.is_contiguous() and wi.dtype == wa_t.dtype else None, self._stream(),
            )
        )
        out = torch.empty((n, channels), dtype=u.dtype, device=u.device)
        arr = ctx.arrays
        if chunks is not None and ctx.max_qlen > self.RGLRU_CHUNKED_FROM:
            pq = torch.empty((chunks.shape[0], 2, channels), dtype=torch.float32, device=u.device)
            self._check(
                self.lib.yk_rglru_scan_chunked(
                    a.data_ptr(), b.data_ptr(), y.data_ptr(), y.stride(0), x.data_ptr(), x.stride(0), _code(u.dtype),
                    s_state.data_ptr(), _ptr(conv_state), arr["seq_qstart"].data_ptr(), arr["seq_qlen"].data_ptr(),
                    arr["state_slots"].data_ptr(), chunks.data_ptr(), chunks.shape[0], seq_chunk0.data_ptr(), pq.data_ptr(),
                    out.data_ptr(), arr["seq_qstart"].numel(), channels, int(taps), self._stream(),
                )
            )
            return out
        self._check(
            self.lib.yk_rglru_scan(
                a.data_ptr(), b.data_ptr(), y.data_ptr(), y.stride(0), x.data_ptr(), x.stride(0), _code(u.dtype),
                s_state.data_ptr(), _ptr(conv_state), arr["seq_qstart"].data_ptr(), arr["seq_qlen"].data_ptr(),
                arr["state_slots"].data_ptr(), out.data_ptr(), arr["seq_qstart"].numel(), channels, int(taps), self._stream(),
            )
        )
        return out

    # --------------------------------------------------------------- mixture of experts
    def moe_experts(self, x, token_ids, table, w_gate_up, w_down, activation, input_per_token: bool = False) -> torch.Tensor:
        """Every token through the experts its id names in ``table`` [vocab, top]: returns float32
        rows [N * top, hidden], row n * top + k the output of token n's k-th expert (uncombined).
        ``w_gate_up`` [experts, 2, ff, hidden] (gate rows, then up rows), ``w_down`` [experts, hidden, ff].
        ``token_ids`` None: ``table`` has a row per token of the step (a router's choice) and ``x`` a row per
        (token, k) already, [N * top, hidden] (what ``moe_router_topk`` returns), or, with ``input_per_token``, a row per
        token that all its experts read.  ``w_gate_up`` [experts, 1, ff, hidden]: experts without a gate, down(act(up x))
        with ``activation`` a plain one (``plain_kind``)."""
        self._rows(x, "expert input")
        vocab, top = table.shape
        if token_ids is None:
            n, hidden = vocab, x.shape[1]
            x_top = top if input_per_token else 1  # x_top: how many pairs share a row of x
            if x.shape[0] != (n if input_per_token else n * top):
                raise KernelError("moe: with a choice per token the input has a row per (token, choice), or a row per token")
        else:
            (n, hidden), x_top = x.shape, top
        experts, two, ff, hid = w_gate_up.shape
        gated = two == 2
        if two not in (1, 2) or hid != hidden or tuple(w_down.shape) != (experts, hidden, ff) or not w_gate_up.is_contiguous() or not w_down.is_contiguous():
            raise KernelError("moe: expert weights must be contiguous [experts, 2 (or 1: no gate), ff, hidden] and [experts, hidden, ff]")
        if table.dtype != torch.int32 or not table.is_contiguous() or (token_ids is not None and (token_ids.dtype != torch.int32 or token_ids.numel() != n)):
            raise KernelError("moe: the table and the token ids are int32, one id per row")
        kind, p0, p1 = self.gated_kind(activation) if gated else (self.plain_kind(activation), 0.0, 0.0)
        pairs = n * top
        dev = x.device
        rows = torch.empty((pairs, hidden), dtype=torch.float32, device=dev)
        if n == 0:
            return rows
        # tiles of 128 or 64 pairs where an expert has that many on average, else of 16
        tile_rows = 128 if pairs >= 96 * experts else (64 if pairs >= 48 * experts else 16)
        max_tiles = self.lib.yk_moe_max_tiles(pairs, experts, tile_rows)
        ints = torch.empty(2 * pairs + 3 * max_tiles + 1, dtype=torch.int32, device=dev)
        order, slot_expert = ints[:pairs], ints[pairs: 2 * pairs]
        tiles, n_tiles = ints[2 * pairs: 2 * pairs + 3 * max_tiles], ints[2 * pairs + 3 * max_tiles:]
        self._check(
            self.lib.yk_moe_route(_ptr(token_ids), table.data_ptr(), vocab, top, experts, n, tile_rows, order.data_ptr(),
                                  slot_expert.data_ptr(), tiles.data_ptr(), n_tiles.data_ptr(), self._stream())
        )
        bf = torch.bfloat16
        if (tile_rows == 128 and x.dtype == bf and w_gate_up.dtype == bf and w_down.dtype == bf and hidden % 8 == 0 and ff % 8 == 0
                and x.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0):
            # many pairs an expert: both products as tiles of 128 x 128 through LDS (the grouped form of
            # ``gemm_tile``), the gated pair by the activation kernel between them
            gu = torch.empty((pairs, two * ff), dtype=bf, device=dev)
            self._check(
                self.lib.yk_gemm_tile_grouped(
                    x.data_ptr(), x.stride(0), order.data_ptr(), x_top, w_gate_up.data_ptr(), two * ff * hidden, hidden, gu.data_ptr(),
                    _BF16, two * ff, None, tiles.data_ptr(), n_tiles.data_ptr(), max_tiles, two * ff, hidden, self._stream(),
                )
            )
            y = self.gated_act(gu, activation, bf) if gated else self.activation(gu, activation, bf)
            self._check(
                self.lib.yk_gemm_tile_grouped(
                    y.data_ptr(), ff, None, 1, w_down.data_ptr(), hidden * ff, ff, rows.data_ptr(), _F32, hidden,
                    order.data_ptr(), tiles.data_ptr(), n_tiles.data_ptr(), max_tiles, hidden, ff, self._stream(),
                )
            )
            return rows
        y = torch.empty((pairs, ff), dtype=x.dtype, device=dev)
        self._check(
            self.lib.yk_moe_gate_up(
                x.data_ptr(), x.stride(0), _code(x.dtype), w_gate_up.data_ptr(), _code(w_gate_up.dtype), order.data_ptr(),
                slot_expert.data_ptr(), tiles.data_ptr(), n_tiles.data_ptr(), tile_rows, max_tiles, pairs, x_top, hidden, ff,
                kind, p0, p1, y.data_ptr(), int(gated), self._stream(),
            )
        )
        self._check(
            self.lib.yk_moe_down(
                y.data_ptr(), _code(y.dtype), w_down.data_ptr(), _code(w_down.dtype), order.data_ptr(), slot_expert.data_ptr(),
                tiles.data_ptr(), n_tiles.data_ptr(), tile_rows, max_tiles, pairs, hidden, ff, rows.data_ptr(), self._stream(),
            )
        )
        return rows

    def moe_router_topk(self, logits, x, top: int, experts: Optional[int] = None, bias=None, scores: str = "sigmoid"):
        """From a router's float32 ``logits`` [N, >= experts] (``experts``: how many of a row's columns are experts; the
        rest is padding): the ``top`` experts with the largest logits of every token
        (int32 [N, top]; among equals the lower number) and the token's row of ``x`` once per chosen expert times the
        expert's score sigmoid(logit) ([N * top, hidden] in x's dtype): the score weighs the expert's input.  ``bias``
        (float32 [experts]) joins the logits before the choice.  ``scores`` "softmax_of_chosen": nothing is copied (``x``
        may be None); the second result is float32 [N, top], the softmax over the chosen logits alone, which weighs the
        experts' outputs."""
        self._rows(logits, "router logits")
        n = logits.shape[0]
        experts = logits.shape[1] if experts is None else int(experts)
        if logits.dtype != torch.float32 or experts > logits.shape[1] or not 1 <= top <= min(experts, 64):
            raise KernelError("moe_router_topk: logits are float32 [N, >= experts], top between 1 and min(experts, 64)")
        if bias is not None and (bias.dtype != torch.float32 or bias.numel() != experts or not bias.is_contiguous()):
            raise KernelError("moe_router_topk: the bias is contiguous float32 [experts]")
        choice = torch.empty((n, top), dtype=torch.int32, device=logits.device)
        if scores == "softmax_of_chosen":
            weights = torch.empty((n, top), dtype=torch.float32, device=logits.device)
            self._check(self.lib.yk_moe_router_topk(logits.data_ptr(), logits.stride(0), experts, int(top), None, 0, _F32, 0, choice.data_ptr(),
                                                    None, n, _ptr(bias), weights.data_ptr(), self._stream()))
            return choice, weights
        if scores != "sigmoid":
            raise KernelError(f"moe_router_topk: scores {scores!r} are not offered")
        self._rows(x, "router input")
        if x.shape[0] != n:
            raise KernelError("moe_router_topk: a row of x per row of logits")
        xs = torch.empty((n * top, x.shape[1]), dtype=x.dtype, device=x.device)
        self._check(self.lib.yk_moe_router_topk(logits.data_ptr(), logits.stride(0), experts, int(top), x.data_ptr(), x.stride(0), _code(x.dtype),
                                                x.shape[1], choice.data_ptr(), xs.data_ptr(), n, _ptr(bias), None, self._stream()))
        return choice, xs

    def moe_router_share(self, logits, top: int, experts: Optional[int] = None, bias=None, correction=None, groups=None):
        """(choice int32 [N, top], weights float32 [N, top]) from a router's float32 ``logits`` [N, >= experts]: scores are their
        sigmoids (``bias`` float32 [experts] joins the logits), the choice is by score + ``correction`` (float32 [experts]); with
        ``groups`` = (count, keep) among the experts of the ``keep`` best of ``count`` equal groups of neighbours, a group's score
        the sum of its two largest; a chosen expert's weight is its score over the sum of the chosen scores + 1e-20.  Among
        equals the lower number wins."""
        self._rows(logits, "router logits")
        n = logits.shape[0]
        experts = logits.shape[1] if experts is None else int(experts)
        if logits.dtype != torch.float32 or experts > logits.shape[1]:
            raise KernelError("moe_router_share: logits are float32 [N, >= experts]")
        for t in (bias, correction):
            if t is not None and (t.dtype != torch.float32 or t.numel() != experts or not t.is_contiguous()):
                raise KernelError("moe_router_share: the bias and the correction are contiguous float32 [experts]")
        count, keep = (0, 0) if groups is None else (int(groups[0]), int(groups[1]))
        choice = torch.empty((n, top), dtype=torch.int32, device=logits.device)
        weights = torch.empty((n, top), dtype=torch.float32, device=logits.device)
        self._check(self.lib.yk_moe_router_share(logits.data_ptr(), logits.stride(0), experts, int(top), _ptr(bias), _ptr(correction), count, keep,
                                                 choice.data_ptr(), weights.data_ptr(), n, self._stream()))
        return choice, weights

    def moe_combine(self, dense, rows, top: int, weight: float = 1.0, row_weights=None) -> torch.Tensor:
        """float32 [N, width]: ``dense`` (a tensor, a ``SplitSum`` or None) + weight * the sum of each token's ``top``
        consecutive rows of ``rows`` (float32 [N * top, width]), each first multiplied by its entry of ``row_weights``
        (float32 [N, top]) where given."""
        if isinstance(dense, SplitAttention):
            dense = dense.merge()
        if row_weights is not None and (row_weights.dtype != torch.float32 or row_weights.numel() != rows.shape[0] or not row_weights.is_contiguous()):
            raise KernelError("moe_combine: the rows' weights are contiguous float32, one per row")
        if rows.dtype != torch.float32 or not rows.is_contiguous() or rows.dim() != 2 or rows.shape[0] % top:
            raise KernelError("moe_combine: the experts' rows are contiguous float32 [N * top, width]")
        n, width = rows.shape[0] // top, rows.shape[1]
        n_splits, round_sum, src = 1, 0, dense
        if isinstance(dense, SplitSum):
            dense.check_live()
            n_splits, round_sum, src = dense.n_splits, dense.round_sum, dense.tensor
        if dense is not None and (tuple(dense.shape) != (n, width) or not src.is_contiguous()):
            raise KernelError(f"moe_combine: the dense part {tuple(dense.shape)} does not match the rows {(n, width)}")
        out = torch.empty((n, width), dtype=torch.float32, device=rows.device)
        self._check(self.lib.yk_moe_combine(_ptr(src), 0 if src is None else _code(src.dtype), n_splits, round_sum, rows.data_ptr(),
                                            int(top), float(weight), out.data_ptr(), n, width, _ptr(row_weights), self._stream()))
        return out

    # ------------------------------------------------------------------- sampling
    def argmax(self, logits: torch.Tensor) -> torch.Tensor:
        if logits.dtype != torch.float32 or not logits.is_contiguous() or logits.dim() != 2:
            raise KernelError("argmax takes contiguous float32 logits [rows, vocab]")
        out = torch.empty(logits.shape[0], dtype=torch.int32, device=logits.device)
        ws = self._ws(64 * logits.shape[0])
        lib = self._library("sampling")
        self._check(lib.yk_argmax(logits.data_ptr(), out.data_ptr(), logits.shape[0], logits.shape[1],
                                  ws.data_ptr(), ws.numel(), self._stream()), lib)
        return out

    def sample(self, logits, temperature, top_k, top_p, seeds, draws, whole_row: bool = False, paths=None) -> torch.Tensor:
        """Per row: temperature (float32; 0 = greedy), top_k (int32; 0 = off), top_p
        (float32), seed and draw number (int32).  Returns int32 token ids.  Rows of a large
        vocabulary are divided among workgroups; ``whole_row`` forces one workgroup a row on
        the path that never narrows the row down to candidates (for tests), and ``paths``
        (int32, one per row) receives which way each divided row went: 0 greedy, 1 a race
        over the row, 3 settled among candidates, 4 left to one workgroup after all."""
        if logits.dtype != torch.float32 or not logits.is_contiguous() or logits.dim() != 2:
            raise KernelError("sample takes contiguous float32 logits [rows, vocab]")
        rows = logits.shape[0]
        for name, t, dt in (("temperature", temperature, torch.float32), ("top_k", top_k, torch.int32),
                            ("top_p", top_p, torch.float32), ("seeds", seeds, torch.int32), ("draws", draws, torch.int32)):
            if t.dtype != dt or t.numel() != rows or not t.is_contiguous():
                raise KernelError(f"sample: {name} must be {dt} with one entry per row")
        if paths is not None and (paths.dtype != torch.int32 or paths.numel() != rows or not paths.is_contiguous()):
            raise KernelError("sample: paths must be int32 with one entry per row")
        out = torch.empty(rows, dtype=torch.int32, device=logits.device)
        lib = self._library("sampling")
        need = 0 if whole_row else int(lib.yk_sample_workspace_bytes(rows, logits.shape[1]))
        ws = self._ws((need + 3) // 4) if need else None
        self._check(
            lib.yk_sample(
                logits.data_ptr(), out.data_ptr(), rows, logits.shape[1], temperature.data_ptr(), top_k.data_ptr(),
                top_p.data_ptr(), seeds.data_ptr(), draws.data_ptr(), int(bool(whole_row)),
                _ptr(ws), 0 if ws is None else ws.numel() * 4, _ptr(paths), self._stream(),
            ),
            lib,
        )
        return out

    def cache_tiled(self, dtype: torch.dtype, head_dim: int, page_size: int) -> bool:
        """Whether pages of this kind are kept in the order the matrix-core attention loads
        them rather than as plain [slot, dim] keys and [dim, slot] values.  The kernels that
        write and read pages decide alike from the same three numbers; code that fills or
        inspects pages by hand (tests) has to ask."""
        return bool(self.lib.yk_cache_tiled(_code(dtype), int(head_dim), int(page_size)))

    # ------------------------------------------------------------------ machine probes
    def probe_stream_read(self, data: torch.Tensor, workgroups: int, sink: torch.Tensor, nontemporal: bool = False) -> None:
        """Reads every byte of ``data`` once with a plain streaming kernel (for timing);
        ``nontemporal`` marks the loads as not to be kept in the caches."""
        lib = self._library("probe")
        self._check(lib.yk_probe_stream_read(data.data_ptr(), data.numel() * data.element_size(), int(workgroups),
                                             int(bool(nontemporal)), sink.data_ptr(), self._stream()), lib)

    def probe_mfma_bf16(self, workgroups: int, iterations: int, sink: torch.Tensor) -> int:
        """Issues a loop of bfloat16 matrix-core instructions from registers; returns its flop count."""
        lib = self._library("probe")
        self._check(lib.yk_probe_mfma_bf16(int(workgroups), int(iterations), sink.data_ptr(), self._stream()), lib)
        return int(workgroups) * 4 * int(iterations) * 4 * 16384
