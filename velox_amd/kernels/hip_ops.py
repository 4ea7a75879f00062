"""Python face of the HIP kernels: shape and dtype checks on the host, then a C call on the current stream.

Every kernel the model calls goes through one method of :class:`HipOps`.  The methods check
what the kernels and their launch grids assume (devices, dtypes, contiguity, alignment, sizes)
before launching, because a kernel that reads out of bounds takes the whole GPU down.  There
is no fallback: without a GPU, without hipcc or without the libraries, loading fails.

Matrix products: a float32 run uses the exact FMA kernel (``gemm.hip``); so does any operand mix
a library has no call for.  bfloat16 x bfloat16 products go to the library behind
``torch.nn.functional.linear`` (hipBLASLt), as the reference uses cuBLAS through ``nn.Linear``
(reference ``src/self_attention.py:48,90``, ``src/mlp.py:13,15``).
"""
from __future__ import annotations

import ctypes
import logging
import os
import tempfile
from typing import Tuple, Dict, Optional

import torch

from ..parts.base import DeferredNorm, NormedSum, ReadyInput, ResidualCopy, ResidualSink, SumOf
from . import build

logger = logging.getLogger(__name__)

_DTYPE_CODE = {torch.float32: 0, torch.bfloat16: 1}
_P = ctypes.c_void_p
_I = ctypes.c_int
_F = ctypes.c_float


class KernelError(RuntimeError):
    pass


def _code(dtype: torch.dtype) -> int:
    if dtype not in _DTYPE_CODE:
        raise KernelError(f"kernels take float32 or bfloat16, got {dtype}")
    return _DTYPE_CODE[dtype]


def _ptr(t: Optional[torch.Tensor]):
    return _P(0) if t is None else _P(t.data_ptr())


class PreparedWeight:
    """A ``[N, K]`` weight together with the copies of it that the decode-sized products read (``HipOps.prepare_weight``).
    The part that owns the weight owns this; it stands wherever the weight stands in ``linear``, ``linear_silu_mul`` and
    ``qkv_rope_write``.  ``copies``: 1 and 2 = ``pack_rows`` of the weight as one matrix or as two stacked ones,
    ``"rotary"`` = the copy in the row order of ``qkv_rope_write``."""

    def __init__(self, weight: torch.Tensor) -> None:
        self.weight = weight
        self.version = weight._version
        self.copies: Dict[object, torch.Tensor] = {}

    @property
    def shape(self):
        return self.weight.shape

    @property
    def dtype(self):
        return self.weight.dtype

    def copy(self, key=1) -> Optional[torch.Tensor]:
        if self.weight._version != self.version:
            raise KernelError("a weight was changed in place after the kernels prepared their copies of it; prepare it again")
        return self.copies.get(key)


def _weight_of(weight) -> Tuple[torch.Tensor, Optional[PreparedWeight]]:
    if isinstance(weight, PreparedWeight):
        return weight.weight, weight
    return weight, None


class HipOps:
    name = "hip-gfx950"
    MAX_TILED_HEAD_DIM = 256  # head sizes above this go to the plain attention kernel
    FEW_PAIRS = 64  # up to this many (token, expert) pairs the experts' plan kernel copies the rows itself

    def __init__(self, device) -> None:
        self.device = torch.device(device)
        if self.device.type != "cuda" or not torch.cuda.is_available():
            raise KernelError("the HIP kernels need a GPU (device 'cuda'); there is no CPU path")
        if self.device.index is None:
            self.device = torch.device("cuda", torch.cuda.current_device())
        arch = torch.cuda.get_device_properties(self.device).gcnArchName.split(":")[0]
        if arch != build.ARCH:
            raise KernelError(f"the kernels are built for {build.ARCH}; this GPU is {arch}")
        self._core = ctypes.CDLL(build.ensure_core())
        self._attention: Dict[Tuple[int, str], ctypes.CDLL] = {}
        self._declare_core()
        self.num_cus = torch.cuda.get_device_properties(self.device).multi_processor_count
        self.use_library_gemm = True
        self.use_skinny_gemm = True
        self.pack_decode_weights = True
        self.fuse_residual_norm = True
        self.use_grouped_mfma = True  # (False: the grouped bfloat16 products take the exact multiply-add tiles, for tests)
        self._mm_out_dtype_ok: Optional[bool] = None
        self._bias_copies: Dict[Tuple[int, int], Tuple[torch.Tensor, torch.Tensor]] = {}
        self._raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)

    # -- loading --------------------------------------------------------------------------------
    def _declare_core(self) -> None:
        c = self._core
        c.velox_embed.argtypes = [_P, _P, _P, _I, _I, _I, _I, _F, _P]
        c.velox_place_tokens.argtypes = [_P, _P, _P, _P, _I, _I, _I, _P]
        c.velox_add_rmsnorm.argtypes = [_P, _P, _P, _P, _P, _I, _I, _F, _I, _I, _I, ctypes.c_longlong, _P, _I, _P]
        c.velox_skinny_qkv_rotary_bf16.argtypes = [_P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P, _I, _F, _F, _I, _P]
        c.velox_silu_mul.argtypes = [_P, _P, _I, _I, _I, _P]
        c.velox_rope_kv_write.argtypes = [_P, _P, _P, _P, _P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P]
        c.velox_rope_kv_write_partial_bf16.argtypes = [_P, _P, _I, _P, _P, _P, _P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P]
        c.velox_rope_kv_write_partial_bf16.restype = _I
        c.velox_gemm_fma.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P]
        c.velox_skinny_gemm_bf16.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P, _I, _F, _F, _I, _I, _P]
        c.velox_skinny_residual_norm_bf16.argtypes = [_P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _P]
        c.velox_skinny_residual_norm_bf16.restype = _I
        c.velox_row_scale_apply.argtypes = [_P, _P, _I, _F, _F, _P, _I, _I, _P]
        c.velox_skinny_gemm_bf16.restype = _I
        c.velox_skinny_gemm_glu_bf16.argtypes = [_P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _F, _F, _I, _P, _P]
        c.velox_skinny_gemm_glu_act_bf16.argtypes = [_P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _F, _F, _I, _P, _I, _P]
        c.velox_skinny_gemm_glu_act_bf16.restype = _I
        c.velox_skinny_gemm_glu_bf16.restype = _I
        c.velox_skinny_glu_rows_bf16.argtypes = [_P, _P, _P, _I, _I, _I, _I, _P]
        c.velox_skinny_glu_rows_bf16.restype = _I
        c.velox_skinny_gemm_splitk_bf16.argtypes = [_P, _P, _P, _I, _I, _I, _I, _I, _P]
        c.velox_skinny_gemm_splitk_bf16.restype = _I
        c.velox_argmax.argtypes = [_P, _P, _P, _I, _I, _I, _P]
        c.velox_sample.argtypes = [_P, _P, _P, _I, _I, _P]
        c.velox_count_tokens.argtypes = [_P, _P, _I, _I, _P]
        c.velox_count_sampled.argtypes = [_P, _P, _P, _I, _I, _P]
        c.velox_penalties_from_counts.argtypes = [_P, _P, _P, _P, _I, _I, _I, _P]
        c.velox_sample_chunked.argtypes = [_P, _P, _P, _I, _I, _I, _P, ctypes.c_longlong, _I, _P]
        c.velox_sample_chunked_scratch_bytes.argtypes = [_I, _I]
        c.velox_sample_chunked_scratch_bytes.restype = ctypes.c_longlong
        c.velox_apply_penalties.argtypes = [_P, _P, _P, _P, _I, _I, _I, _P]
        c.velox_probe_read.argtypes = [_P, ctypes.c_longlong, _P, _I, _P]
        c.velox_probe_read.restype = _I
        c.velox_probe_mfma.argtypes = [_I, _I, _P, _P]
        c.velox_probe_mfma.restype = _I
        c.velox_probe_grid_barrier.argtypes = [_I, _I, _I, _P, _P, _P]
        c.velox_probe_grid_barrier.restype = _I
        c.velox_latent_rotate_write.argtypes = [_P, _I, _P, _I, _I, _I, _I, _I, _I, _I, _P, _P, _P, _I, _I, _P, _F, _P, _P, _P, _I, _I, _I, _I, _P, _P, _P]
        c.velox_head_linear.argtypes = [_P, _I, _I, _I, _P, _P, _I, _I, _I, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P]
        c.velox_plain_attention.argtypes = [_P, _I, _P, _P, _P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _I, _I, _P, _I, _P, _I, _F, _P, _I, _I, _P]
        c.velox_plain_attention.restype = _I
        c.velox_route_top.argtypes = [_P, _P, _P, _I, _I, _I, _I, _I, _P, _I, _I, _F, _P]
        c.velox_routed_plan_elems.argtypes = [_I, _I]
        c.velox_routed_plan_elems.restype = ctypes.c_longlong
        c.velox_routed_plan.argtypes = [_P, _I, _I, _P, _I, _P, _P, _P, _I, _I, _I, _P]
        c.velox_grouped_glu.argtypes = [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _F, _F, _I, _P]
        c.velox_grouped_down.argtypes = [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P]
        c.velox_routed_combine.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _I, _P, _P, _I, _P]
        c.velox_routed_products_bf16.argtypes = [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _F, _F, _I, _P]
        c.velox_routed_combine_norm.argtypes = [_P, _P, _P, _I, _I, _I, _I, _I, _P, _P, _I, _P, _P, _F, _F, _P, _P, _F, _P]
        c.velox_routed_combine_norm.restype = _I
        c.velox_add_sinusoid.argtypes = [_P, _P, _P, _I, _I, _P]
        c.velox_add_cast.argtypes = [_P, _P, _I, _P, ctypes.c_longlong, _P]
        c.velox_norm_add.argtypes = [_P, _P, _I, _P, _P, _I, _I, _F, _F, _I, ctypes.c_longlong, _P]
        c.velox_qk_norm_write.argtypes = [_P, _I, _P, _P, _P, _P, _P, _I, _I, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F, _F, _I, _I, _P]
        c.velox_stream_norm.argtypes = [_P, _P, _I, _F, _P, _I, _F, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _F, _P]
        c.velox_embed_copies.argtypes = [_P, _P, _I, _P, _I, _I, _I, _F, _I, _P]
        c.velox_gated_act_mul.argtypes = [_P, _P, _I, _I, _I, _I, _P]
        c.velox_short_conv.argtypes = [_P, _I, _I, _P, _I, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P, _P]
        c.velox_sum_norm.argtypes = [_P, _P, _P, _I, _I, _F, _P, _P, _F, _P, _I, _P, _I, _I, _I, _P]
        c.velox_softcap.argtypes = [_P, ctypes.c_longlong, _F, _F, _P]
        c.velox_state_space_scan.argtypes = [_P, _I, _I, _P, _I, _I, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P]
        c.velox_state_space_scratch_elems.argtypes = [_I, _I, _I, _I, _I]
        c.velox_state_space_scratch_elems.restype = ctypes.c_longlong
        c.velox_state_space_max_state.argtypes = []
        c.velox_gated_group_norm.argtypes = [_P, _P, _I, _I, _I, _P, _F, _P, _I, _I, _I, _I, _P]
        for fn in (c.velox_sum_norm, c.velox_softcap, c.velox_state_space_scan, c.velox_state_space_max_state, c.velox_gated_group_norm):
            fn.restype = _I
        c.velox_rotate_pad_write.argtypes = [_P, _I, _P, _P, _P, _P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _P]
        c.velox_recurrence_prepare.argtypes = [_P, _I, _I, _I, _I, _I, _I, _I, _F, _P, _I, _I, _I, _I, _I, _P, _P, _F, _P, _I, _I, _I, _P, _P, _P, _I, _P]
        c.velox_linear_scan.argtypes = [_P, _P, _I, _I, _I, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P]
        c.velox_linear_scan_lanes.argtypes = [_I]
        c.velox_gated_head_norm.argtypes = [_P, _P, _F, _P, _I, _I, _I, _I, _P, _I, _I, _I, _I, _I, _P]
        c.velox_removal_prepare.argtypes = [_P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _P, _P, _P, _F, _P, _P, _P, _I, _P]
        c.velox_gated_scan.argtypes = [_P, _I, _I, _P, _P, _F, _P, _P, _P, _P, _P, _I, _I, _P]
        c.velox_gated_scan_scratch_elems.argtypes = [_I, _I, _I]
        c.velox_gated_scan_scratch_elems.restype = ctypes.c_longlong
        c.velox_norm_add_norm.argtypes = [_P, _P, _I, _P, _F, _P, _F, _P, _P, _I, _I, _I, _I, ctypes.c_longlong, _P]
        c.velox_poly_norm.argtypes = [_P, _P, _P, _I, _I, _F, _I, _P]
        c.velox_removal_chunk_scan.argtypes = [_P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _P, _P, _P, _F, _P, _P, _P, _P, _P, _I, _I, _P]
        c.velox_removal_chunk_scan.restype = _I
        c.velox_removal_chunk_scratch_elems.argtypes = [_I, _I, _I, _I, _I, _I]
        c.velox_removal_chunk_scratch_elems.restype = ctypes.c_longlong
        for fn in (c.velox_removal_prepare, c.velox_gated_scan, c.velox_norm_add_norm, c.velox_poly_norm):
            fn.restype = _I
        c.velox_embed_bigram.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _P, _P, _P, _P, _P]
        c.velox_add_dynamic_tanh.argtypes = [_P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, ctypes.c_longlong, _P, _I, _P]
        c.velox_scale.argtypes = [_P, ctypes.c_longlong, _F, _P]
        c.velox_activation.argtypes = [_P, _P, ctypes.c_longlong, _I, _I, _P]
        for fn in (c.velox_embed_bigram, c.velox_add_dynamic_tanh, c.velox_scale, c.velox_activation):
            fn.restype = _I
        for fn in (c.velox_stream_norm, c.velox_embed_copies, c.velox_gated_act_mul, c.velox_short_conv, c.velox_rotate_pad_write, c.velox_recurrence_prepare,
                   c.velox_linear_scan, c.velox_linear_scan_lanes, c.velox_gated_head_norm):
            fn.restype = _I
        c.velox_routed_products_bf16.restype = _I
        for fn in (c.velox_latent_rotate_write, c.velox_head_linear, c.velox_route_top, c.velox_routed_plan, c.velox_grouped_glu, c.velox_grouped_down,
                   c.velox_routed_combine, c.velox_add_sinusoid, c.velox_add_cast, c.velox_norm_add, c.velox_qk_norm_write):
            fn.restype = _I
        for fn in (c.velox_embed, c.velox_place_tokens, c.velox_add_rmsnorm, c.velox_silu_mul, c.velox_rope_kv_write, c.velox_gemm_fma,
                   c.velox_argmax, c.velox_sample, c.velox_sample_chunked, c.velox_apply_penalties, c.velox_count_tokens, c.velox_count_sampled,
                   c.velox_penalties_from_counts):
            fn.restype = _I

    def attention_library(self, head_dim: int, biased: bool = False, kept: bool = False, capped: bool = False, gated: bool = False) -> ctypes.CDLL:
        """The attention kernels for one head size; ``biased``: the build whose scores take a bias by distance; ``kept``: whose
        windows keep the first keys; ``capped``: whose scores are capped; ``gated``: whose outputs are gated."""
        key = (head_dim, build.attention_options(biased, kept, capped, gated))
        lib = self._attention.get(key)
        if lib is None:
            lib = ctypes.CDLL(build.ensure_attention(head_dim, biased=bool(biased), kept=bool(kept), capped=bool(capped), gated=bool(gated)))
            lib.velox_paged_attention.argtypes = [_P, _I, _P, _P, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _I, _P, _I, _P,
                                                  _I, _F, _P, _I, _I, _P]
            lib.velox_attention_options.restype = _I
            lib.velox_paged_attention.restype = _I
            lib.velox_attention_head_dim.restype = _I
            lib.velox_attention_portion_kernel.argtypes = [_I]
            lib.velox_attention_portion_kernel.restype = None
            if lib.velox_attention_head_dim() != head_dim:
                raise KernelError(f"attention library for head_dim={head_dim} reports {lib.velox_attention_head_dim()}")
            wanted = sum(bit for bit, on in zip((1, 2, 4, 8), (biased, kept, capped, gated)) if on)
            if lib.velox_attention_options() != wanted:
                raise KernelError(f"attention library for head_dim={head_dim}: built with the options {lib.velox_attention_options()}, not {wanted}")
            self._attention[key] = lib
        return lib

    def prepare(self, model, dtype) -> None:
        """Lets every part get what it needs of the kernels before the first step (``Part.prepare_kernels``): the weights
        that decode-sized products read are registered, and libraries that are built per size (attention, per head
        size) are built and loaded by the parts that use them."""
        for part in model.all_parts():
            part.prepare_kernels(self)
        if dtype == torch.bfloat16 and self.use_library_gemm and self._mm_out_dtype_ok is None:
            self._decide_float32_out_route()

    def prepare_weight(self, weight: torch.Tensor, stacked: int = 1, rotary_heads: Optional[Tuple[int, int, int]] = None,
                       handle: Optional[PreparedWeight] = None) -> Optional[PreparedWeight]:
        """A second copy of a bfloat16 ``[N, K]`` weight in the order the skinny kernels' lanes read it (see
        ``pack_rows``): decode-sized products then stream contiguous kilobytes.  ``stacked`` = 2 marks ``[Wgate; Wup]``;
        ``rotary_heads = (heads, kv_heads, head_dim)`` marks ``[Wq; Wk; Wv]`` whose product is followed by a rotation of
        whole heads and gets a further copy for ``qkv_rope_write``.  Each copy costs the weight's size again in memory;
        ``pack_decode_weights = False`` turns them off.  Returns what the caller keeps and passes in the weight's place
        (``handle``: an earlier result for the same weight, which is extended), or None when the kernels read this weight
        as it is."""
        if (not self.pack_decode_weights or weight is None or weight.dtype != torch.bfloat16 or weight.dim() != 2
                or weight.shape[1] % 64 != 0 or weight.shape[0] % stacked != 0 or weight.device != self.device):
            return handle
        if handle is None or handle.weight is not weight or handle.version != weight._version:
            handle = PreparedWeight(weight)
        copies = handle.copies
        if stacked not in copies:
            per_matrix = weight.shape[0] // stacked
            whole_tiles = [c for key, c in copies.items() if key in (1, 2)] if per_matrix % 16 == 0 else []
            # with whole tiles every stacking gives the same bytes
            copies[stacked] = whole_tiles[0] if whole_tiles else self.pack_rows(weight, stacked)
        if rotary_heads is not None and "rotary" not in copies:
            heads, kv_heads, head_dim = rotary_heads
            if head_dim % 32 == 0 and weight.shape[0] == (heads + 2 * kv_heads) * head_dim:
                copies["rotary"] = self.pack_rows(weight[self.rotary_row_order(heads, kv_heads, head_dim, weight.device)])
        return handle

    @staticmethod
    def rotary_row_order(heads: int, kv_heads: int, head_dim: int, device) -> torch.Tensor:
        """Row order of ``[Wq; Wk; Wv]`` for ``qkv_rope_write``: inside every query and key head, 16 channels of the low
        half are followed by their 16 partners of the high half; value heads keep their order."""
        half = head_dim // 2
        inside = torch.arange(half, device=device).view(half // 16, 1, 16) + torch.tensor([0, half], device=device).view(1, 2, 1)
        rotary = (torch.arange(heads + kv_heads, device=device).view(-1, 1) * head_dim + inside.reshape(1, -1)).reshape(-1)
        values = torch.arange((heads + kv_heads) * head_dim, (heads + 2 * kv_heads) * head_dim, device=device)
        return torch.cat([rotary, values])

    def library_serves(self, m: int, n: int, k: int) -> bool:
        """Whether ``linear`` hands ``x[m, k] @ w[n, k]^T`` in bfloat16 to the matrix library, and the product is large
        enough for the library's timing of its candidates to mean something (a weight of a few megabytes is timed
        from the caches, which says little about a step that streams it from memory)."""
        if not self.use_library_gemm:
            return False
        if m > 64:
            return True
        return m > 16 and n > 8192 and n * k >= (32 << 20)

    def tuning_file(self) -> Optional[str]:
        """Where timings of the matrix library's kernels are kept between runs by default: beside the built kernel
        libraries, one file per kind of GPU (the file's own header names the library versions it holds for, and
        TunableOp refuses a file made by others)."""
        directory = next((d for d in build.build_dirs() if build._writable(d)), None)
        arch = torch.cuda.get_device_properties(self.device).gcnArchName.split(":")[0]
        return os.path.join(directory, f"tunableop_{arch}.csv") if directory else None

    def tune_library_products(self, shapes, token_counts, seconds_per_shape: float = 0.2, results_file: Optional[str] = None) -> int:
        """Lets PyTorch's TunableOp time the library's candidate kernels for ``x[M, K] @ w[N, K]^T`` at the given
        ``(N, K)`` shapes and ``M`` values, and keeps its choices for later calls.  Tuning stays off afterwards, so
        other shapes keep the library's default choice and never pay for a search.  ``results_file``: what was found is
        kept there, and shapes that an earlier run has timed are not timed again.  Returns the number of products run."""
        tunable = torch.cuda.tunable
        tunable.enable(True)
        if results_file is None:
            # TunableOp writes what it finds to a file: keep that out of the working folder
            results_file = os.path.join(tempfile.gettempdir(), f"velox_amd_tunableop_{os.getuid()}_{os.getpid()}.csv")
        if tunable.get_filename() != results_file:
            tunable.set_filename(results_file)
            if os.path.isfile(results_file) and not tunable.read_file(results_file):
                # made with other versions of the libraries, or half written: start again.  Only a file of the engine's
                # own (beside its kernel libraries, or the temporary one) is removed; a caller's file is left alone and
                # what is found now goes to a new name beside it
                own = results_file == self.tuning_file() or os.path.dirname(results_file) == tempfile.gettempdir()
                if own:
                    os.remove(results_file)
                else:
                    fresh = f"{results_file}.{os.getpid()}"
                    logger.warning("the timings in %s cannot be read by this version of the matrix library; leaving it and writing to %s", results_file, fresh)
                    results_file = fresh
                    tunable.set_filename(results_file)
        tunable.set_max_tuning_duration(int(seconds_per_shape * 1000))
        tunable.tuning_enable(True)
        done = 0
        try:
            for n, k in sorted(set(shapes)):
                # (operands like the real ones: a kernel's time and its clocks depend on the bits it moves)
                weight = torch.randn((n, k), dtype=torch.float32, device=self.device).mul_(0.02).to(torch.bfloat16)
                for m in sorted(set(token_counts)):
                    x = torch.randn((m, k), dtype=torch.float32, device=self.device).to(torch.bfloat16)
                    torch.nn.functional.linear(x, weight)
                    done += 1
                del weight
            torch.cuda.synchronize(self.device)
        finally:
            tunable.tuning_enable(False)
        return done

    # -- helpers --------------------------------------------------------------------------------
    def _stream(self):
        # (the raw handle of the current stream: the same value as torch.cuda.current_stream(device).cuda_stream, without
        # building a Stream object for every kernel call, which costs more host time than the launch itself)
        if self._raw_stream is not None:
            return _P(self._raw_stream(self.device.index))
        return _P(torch.cuda.current_stream(self.device).cuda_stream)

    def _check(self, name: str, t: torch.Tensor, dtype=None, shape=None, align: int = 4) -> None:
        if not isinstance(t, torch.Tensor) or t.device != self.device:
            raise KernelError(f"{name}: expected a tensor on {self.device}, got {getattr(t, 'device', type(t))}")
        if not t.is_contiguous():
            raise KernelError(f"{name}: must be contiguous (shape {tuple(t.shape)}, strides {t.stride()})")
        if dtype is not None and t.dtype != dtype:
            raise KernelError(f"{name}: expected {dtype}, got {t.dtype}")
        if shape is not None and tuple(t.shape) != tuple(shape):
            raise KernelError(f"{name}: expected shape {tuple(shape)}, got {tuple(t.shape)}")
        if t.data_ptr() % align != 0:
            raise KernelError(f"{name}: address must be a multiple of {align}")

    @staticmethod
    def _launched(status: int, what: str) -> None:
        if status != 0:
            raise KernelError(f"{what}: launch failed with HIP error {status}")

    # -- embedding and norms ----------------------------------------------------------------------
    def embed(self, token_ids: torch.Tensor, table: torch.Tensor, scale: float = 1.0, copies: int = 1) -> torch.Tensor:
        """``copies`` > 1: every row is written that many times side by side, ``[T, copies * H]`` (residual streams)."""
        self._check("token_ids", token_ids, torch.int32)
        self._check("table", table)
        if token_ids.dim() != 1 or table.dim() != 2:
            raise KernelError("embed: token_ids must be [T] and the table [V, H]")
        vocab, hidden = table.shape
        if copies != 1:
            if copies < 1:
                raise KernelError(f"embed: copies={copies} must be at least 1")
            out = torch.empty((token_ids.shape[0], copies * hidden), dtype=torch.float32, device=self.device)
            self._launched(self._core.velox_embed_copies(_ptr(token_ids), _ptr(table), _code(table.dtype), _ptr(out), token_ids.shape[0], hidden, vocab,
                                                         float(scale), int(copies), self._stream()), "embed")
            return out
        out = torch.empty((token_ids.shape[0], hidden), dtype=torch.float32, device=self.device)
        status = self._core.velox_embed(_ptr(token_ids), _ptr(table), _ptr(out), token_ids.shape[0], hidden, vocab, _code(table.dtype), float(scale), self._stream())
        self._launched(status, "embed")
        return out

    def place_tokens(self, ids: torch.Tensor, dest: torch.Tensor, source: torch.Tensor, tokens: torch.Tensor, count: int) -> None:
        """``ids[dest[k]] = tokens[source[k]]`` for ``k < count``, all int32 on the device: token ids that the step in flight
        is still sampling, put into this step's rows without a trip to the host."""
        for name, t in (("ids", ids), ("dest", dest), ("source", source), ("tokens", tokens)):
            self._check(name, t, torch.int32)
            if t.dim() != 1:
                raise KernelError(f"place_tokens: {name} must have one dimension")
        if count < 0 or count > dest.numel() or count > source.numel():
            raise KernelError(f"place_tokens: {count} pairs do not fit dest [{dest.numel()}] and source [{source.numel()}]")
        status = self._core.velox_place_tokens(_ptr(ids), _ptr(dest), _ptr(source), _ptr(tokens), int(count), ids.numel(), tokens.numel(), self._stream())
        self._launched(status, "place_tokens")

    def embed_bigram(self, token_ids, table, bigram, scale, buckets, mul_prev, mul_cur, positions, cu_q, slots, state, max_q_len) -> torch.Tensor:
        """``table[ids[t]] * scale + bigram[row(t)]`` in float32, ``row(t) = (previous * mul_prev + ids[t] * mul_cur) mod buckets`` and
        ``buckets`` at position 0; the token before a portion's first one is ``state[slots[b], 0]`` (int32 ``[slots, 1]``), which is
        then set to the portion's last token."""
        self._check("token_ids", token_ids, torch.int32)
        self._check("table", table)
        if token_ids.dim() != 1 or table.dim() != 2:
            raise KernelError("embed_bigram: token_ids must be [T] and the table [V, H]")
        tokens = token_ids.shape[0]
        vocab, hidden = table.shape
        self._check("bigram", bigram, table.dtype, (int(buckets) + 1, hidden))
        self._check("positions", positions, torch.int32, (tokens,))
        self._check("cu_q", cu_q, torch.int32)
        num_seqs = cu_q.shape[0] - 1
        self._check("slots", slots, torch.int32, (num_seqs,))
        self._check("state", state, torch.int32)
        if state.dim() != 2 or state.shape[1] != 1:
            raise KernelError(f"embed_bigram: the state holds one token per slot, [slots, 1]; got {tuple(state.shape)}")
        if not 1 <= max_q_len <= tokens or num_seqs < 1:
            raise KernelError(f"embed_bigram: max_q_len={max_q_len} outside [1, {tokens}]")
        if not 1 <= int(buckets) < 2 ** 31:
            raise KernelError(f"embed_bigram: buckets={buckets} must lie between 1 and 2^31 - 1")
        out = torch.empty((tokens, hidden), dtype=torch.float32, device=self.device)
        # (the multipliers reduced mod buckets, exactly, whatever their size or sign: the kernel's 64-bit sum then cannot overflow)
        status = self._core.velox_embed_bigram(_ptr(token_ids), _ptr(table), _ptr(bigram), _ptr(out), tokens, num_seqs, int(max_q_len), hidden, vocab,
                                               _code(table.dtype), float(scale), int(buckets), int(mul_prev) % int(buckets), int(mul_cur) % int(buckets), _ptr(positions), _ptr(cu_q),
                                               _ptr(slots), _ptr(state), self._stream())
        self._launched(status, "embed_bigram")
        return out

    def add_dynamic_tanh(self, residual, delta, weight, bias, alpha, out_dtype, rows=None):
        """``residual += delta`` (float32, in place; with ``rows`` nothing is changed and only those rows are worked), then
        ``tanh(alpha x) * weight + bias``; ``alpha`` is a float32 tensor of one number on the device.  ``delta`` as for ``add_rmsnorm``."""
        self._check("residual", residual, torch.float32)
        if residual.dim() != 2:
            raise KernelError("add_dynamic_tanh: residual must be [T, H]")
        tokens, hidden = residual.shape
        self._check("weight", weight, torch.float32, (hidden,))
        self._check("bias", bias, torch.float32, (hidden,))
        self._check("alpha", alpha, torch.float32)
        if alpha.numel() != 1:
            raise KernelError("add_dynamic_tanh: alpha is one number")
        partials, partial_stride = 1, 0
        second = None
        if isinstance(delta, SumOf):
            delta, second = delta.first, delta.second
            self._check("second term of the delta", second, None, (tokens, hidden))
        if delta is not None:
            if delta.dim() == 3:
                partials, partial_stride = delta.shape[0], tokens * hidden
                self._check("delta", delta, torch.float32, (partials, tokens, hidden), align=16)
            else:
                self._check("delta", delta, None, (tokens, hidden))
        count = tokens
        if rows is not None:
            self._check("rows", rows, torch.int32)
            count = rows.shape[0]
        out = torch.empty((count, hidden), dtype=out_dtype, device=self.device)
        delta_code = _code(delta.dtype) if delta is not None else _code(out_dtype)
        status = self._core.velox_add_dynamic_tanh(_ptr(residual), _ptr(delta), _ptr(rows), _ptr(weight), _ptr(bias), _ptr(alpha), _ptr(out), count, hidden,
                                                   delta_code, _code(out_dtype), partials, partial_stride, _ptr(second),
                                                   _code(second.dtype) if second is not None else 0, self._stream())
        self._launched(status, "add_dynamic_tanh")
        return out

    def scale_(self, x: torch.Tensor, factor: float) -> torch.Tensor:
        """``x *= factor`` in place, float32."""
        self._check("x", x, torch.float32)
        self._launched(self._core.velox_scale(_ptr(x), x.numel(), float(factor), self._stream()), "scale")
        return x

    _ACTIVATION_CODES = {"relu2": 1}

    def activation(self, x: torch.Tensor, kind: str) -> torch.Tensor:
        """The activation of a unit without a gate branch, float32 arithmetic with one rounding: ``relu2`` = ``relu(x)^2``."""
        if kind not in self._ACTIVATION_CODES:
            raise KernelError(f"activation {kind!r} is not implemented")
        self._check("x", x)
        out = torch.empty_like(x)
        self._launched(self._core.velox_activation(_ptr(x), _ptr(out), x.numel(), self._ACTIVATION_CODES[kind], _code(x.dtype), self._stream()), "activation")
        return out

    def linear_act(self, x, weight, out_dtype: torch.dtype, kind: str) -> torch.Tensor:
        """``act(x @ weight^T)`` for a unit without a gate branch: for decode-sized bfloat16 batches one kernel (the activation
        on the float32 sums is the product's epilogue, so the sums are rounded once), else the product and the
        activation's kernel."""
        if kind not in self._ACTIVATION_CODES:
            raise KernelError(f"activation {kind!r} is not implemented")
        plain, prepared = _weight_of(weight)
        x = self.materialize(x)
        skinny_rows = 16 if plain.shape[0] > 8192 else 32  # (as ``linear`` sends its products)
        if (self.use_skinny_gemm and x.dim() == 2 and x.dtype == torch.bfloat16 and plain.dtype == torch.bfloat16 and out_dtype == torch.bfloat16
                and x.shape[0] <= skinny_rows and x.shape[1] % 64 == 0 and x.shape[1] == plain.shape[1]):
            self._check("x", x, align=16)
            self._check("weight", plain, align=16)
            return self.skinny_gemm(x, plain, None, out_dtype, packed=prepared.copy(1) if prepared is not None else None,
                                    x_packed=self._packed_rows_of(x, x.shape[1]), ungated=kind)
        return self.activation(self.linear(x, weight, None, out_dtype), kind)

    def _norm(self, residual, delta, rows, weight, eps, out_dtype):
        self._check("residual", residual, torch.float32)
        if residual.dim() != 2:
            raise KernelError("add_rmsnorm: residual must be [T, H]")
        tokens, hidden = residual.shape
        self._check("weight", weight, torch.float32, (hidden,))
        partials, partial_stride = 1, 0
        second = None
        if isinstance(delta, SumOf):  # two terms, added to each other first
            delta, second = delta.first, delta.second
            self._check("second term of the delta", second, None, (tokens, hidden))
        if delta is not None:
            if delta.dim() == 3:  # partial sums of a split product, added here
                partials, partial_stride = delta.shape[0], tokens * hidden
                self._check("delta", delta, torch.float32, (partials, tokens, hidden), align=16)
            else:
                self._check("delta", delta, None, (tokens, hidden))
        if rows is not None:
            self._check("rows", rows, torch.int32)
            count = rows.shape[0]
        else:
            count = tokens
        out = torch.empty((count, hidden), dtype=out_dtype, device=self.device)
        delta_code = _code(delta.dtype) if delta is not None else _code(out_dtype)
        status = self._core.velox_add_rmsnorm(_ptr(residual), _ptr(delta), _ptr(rows), _ptr(weight), _ptr(out), count, hidden, float(eps), delta_code, _code(out_dtype), partials, partial_stride,
                                              _ptr(second), _code(second.dtype) if second is not None else 0, self._stream())
        self._launched(status, "add_rmsnorm")
        return out

    def add_rmsnorm(self, residual, delta, weight, eps, out_dtype):
        return self._norm(residual, delta, None, weight, eps, out_dtype)

    def add_rmsnorm_rows(self, residual, delta, rows, weight, eps, out_dtype):
        return self._norm(residual, delta, rows, weight, eps, out_dtype)

    def add_sinusoid(self, hidden: torch.Tensor, positions: torch.Tensor, frequencies: torch.Tensor) -> torch.Tensor:
        """``hidden[t, 2i] += sin(p_t f_i)``, ``hidden[t, 2i + 1] += cos(p_t f_i)`` in place; ``frequencies`` float64 [ceil(H / 2)]."""
        self._check("hidden", hidden, torch.float32)
        if hidden.dim() != 2:
            raise KernelError("add_sinusoid: hidden must be [T, H]")
        tokens, width = hidden.shape
        self._check("positions", positions, torch.int32, (tokens,))
        self._check("frequencies", frequencies, torch.float64, ((width + 1) // 2,), align=8)
        self._launched(self._core.velox_add_sinusoid(_ptr(hidden), _ptr(positions), _ptr(frequencies), tokens, width, self._stream()), "add_sinusoid")
        return hidden

    def add_cast(self, residual: torch.Tensor, delta: Optional[torch.Tensor], out_dtype: torch.dtype) -> torch.Tensor:
        """``residual += delta`` in place (``delta`` may be None) and the residual in ``out_dtype`` (itself when that is float32)."""
        self._check("residual", residual, torch.float32)
        if delta is not None:
            self._check("delta", delta, None, tuple(residual.shape))
        if delta is None and out_dtype == torch.float32:
            return residual
        out = torch.empty_like(residual, dtype=out_dtype) if out_dtype != torch.float32 else None
        self._launched(self._core.velox_add_cast(_ptr(residual), _ptr(delta), _code(delta.dtype) if delta is not None else 0, _ptr(out), residual.numel(),
                                                 self._stream()), "add_cast")
        return residual if out is None else out

    def norm_add(self, residual: torch.Tensor, delta: torch.Tensor, weight: torch.Tensor, eps: float, mult: float, out_dtype: torch.dtype) -> torch.Tensor:
        """``residual += mult * delta * rsqrt(mean(delta^2) + eps) * weight`` in place, float32 throughout; ``delta`` is [T, H]
        or float32 partial sums [S, T, H], added first to last.  Returns the residual in ``out_dtype`` (itself when float32)."""
        self._check("residual", residual, torch.float32)
        if residual.dim() != 2:
            raise KernelError("norm_add: residual must be [T, H]")
        tokens, hidden = residual.shape
        self._check("weight", weight, torch.float32, (hidden,))
        partials, partial_stride = 1, 0
        if delta.dim() == 3:
            partials, partial_stride = delta.shape[0], tokens * hidden
            self._check("delta", delta, torch.float32, (partials, tokens, hidden))
        else:
            self._check("delta", delta, None, (tokens, hidden))
        out = torch.empty((tokens, hidden), dtype=out_dtype, device=self.device) if out_dtype != torch.float32 else None
        self._launched(self._core.velox_norm_add(_ptr(residual), _ptr(delta), _code(delta.dtype), _ptr(weight), _ptr(out), tokens, hidden, float(eps), float(mult),
                                                 partials, partial_stride, self._stream()), "norm_add")
        return residual if out is None else out

    def norm_add_norm(self, residual: torch.Tensor, delta: torch.Tensor, delta_weight: torch.Tensor, delta_eps: float, weight: torch.Tensor, eps: float,
                      out_dtype: torch.dtype, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """``residual += delta * rsqrt(mean(delta^2) + delta_eps) * delta_weight`` in place, then ``residual * rsqrt(mean(residual^2) +
        eps) * weight`` in ``out_dtype``; float32 throughout.  ``delta`` is [T, H] or float32 partial sums [S, T, H], added first to
        last.  ``rows``: nothing is changed and only those rows are worked."""
        self._check("residual", residual, torch.float32)
        if residual.dim() != 2:
            raise KernelError("norm_add_norm: residual must be [T, H]")
        tokens, hidden = residual.shape
        if hidden > 16352:
            raise KernelError(f"norm_add_norm: rows of {hidden} are beyond the kernel (16,352 at most)")
        self._check("delta_weight", delta_weight, torch.float32, (hidden,))
        self._check("weight", weight, torch.float32, (hidden,))
        partials, partial_stride = 1, 0
        if delta.dim() == 3:
            partials, partial_stride = delta.shape[0], tokens * hidden
            self._check("delta", delta, torch.float32, (partials, tokens, hidden))
        else:
            self._check("delta", delta, None, (tokens, hidden))
        count = tokens
        if rows is not None:
            self._check("rows", rows, torch.int32)
            count = rows.shape[0]
        out = torch.empty((count, hidden), dtype=out_dtype, device=self.device)
        self._launched(self._core.velox_norm_add_norm(_ptr(residual), _ptr(delta), _code(delta.dtype), _ptr(delta_weight), float(delta_eps), _ptr(weight), float(eps),
                                                      _ptr(rows), _ptr(out), _code(out_dtype), count, hidden, partials, partial_stride, self._stream()), "norm_add_norm")
        return out

    def _sum_norm(self, what, residual, delta, rows, weight, eps, start, out):
        """``velox_sum_norm`` on ``delta``: None, a tensor, a ``SumOf`` or a ``NormedSum``."""
        self._check("residual", residual, torch.float32)
        if residual.dim() != 2:
            raise KernelError(f"{what}: residual must be [T, H]")
        tokens, hidden = residual.shape
        if hidden > 16320:
            raise KernelError(f"{what}: rows of {hidden} are beyond the kernel (16,320 at most)")
        normed, weights, scales, term_eps, plain = (), (), (), 1.0, ()
        if isinstance(delta, NormedSum):
            normed, weights, scales, term_eps = delta.terms, delta.weights, delta.scales, delta.eps
            plain = (delta.plain,) if delta.plain is not None else ()
        elif isinstance(delta, SumOf):
            plain = (delta.first, delta.second)
        elif delta is not None:
            if not isinstance(delta, torch.Tensor):
                raise KernelError(f"{what}: a {type(delta).__name__} cannot be added here")
            plain = (delta,)
        if len(normed) > 2 or len(normed) != len(weights) or len(normed) != len(scales) or len(plain) > 2:
            raise KernelError(f"{what}: at most two terms with norms of their own and two without")
        described = (ctypes.c_longlong * 20)()
        factors = (ctypes.c_float * 4)()
        for first, terms in ((0, normed), (2, plain)):
            for i, term in enumerate(terms):
                partials, stride = 1, 0
                if term.dim() == 3:
                    partials, stride = term.shape[0], tokens * hidden
                    self._check("partial sums of a term", term, torch.float32, (partials, tokens, hidden))
                else:
                    self._check("term", term, None, (tokens, hidden))
                norm_weight = 0
                if first == 0:
                    self._check("weight of a term's norm", weights[i], torch.float32, (hidden,))
                    norm_weight = weights[i].data_ptr()
                    factors[i] = float(scales[i])
                described[5 * (first + i):5 * (first + i) + 5] = [term.data_ptr(), _code(term.dtype), partials, stride, norm_weight]
        if weight is not None:
            self._check("weight", weight, torch.float32, (hidden,))
        count = tokens
        if rows is not None:
            self._check("rows", rows, torch.int32)
            count = rows.shape[0]
        status = self._core.velox_sum_norm(_ptr(residual), ctypes.cast(described, _P), ctypes.cast(factors, _P), len(normed), len(plain), float(term_eps), _ptr(rows),
                                           _ptr(weight), float(eps), _ptr(start), _code(start.dtype) if start is not None else 0, _ptr(out), _code(out.dtype),
                                           count, hidden, self._stream())
        self._launched(status, what)
        return out

    def normed_sum_norm(self, residual: torch.Tensor, delta: NormedSum, weight: torch.Tensor, eps: float, out_dtype: torch.dtype,
                        rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """``residual += delta`` in place (the terms' own norms and all sums in float32), then ``residual * rsqrt(mean(residual^2) + eps) *
        weight`` in ``out_dtype``.  ``rows``: nothing is changed and only those rows are worked."""
        count = residual.shape[0] if rows is None else rows.shape[0]
        out = torch.empty((count, residual.shape[-1]), dtype=out_dtype, device=self.device)
        return self._sum_norm("normed_sum_norm", residual, delta, rows, weight, eps, None, out)

    def join_rows(self, residual: torch.Tensor, delta, start: torch.Tensor, out_dtype: torch.dtype) -> torch.Tensor:
        """``[residual + delta ; start]`` in ``out_dtype``, [T, 2 H], and the residual is cleared (what is made of the joined rows
        becomes the residual).  ``delta``: None, a tensor (or float32 partial sums), a ``SumOf`` or a ``NormedSum``; ``start`` [T, H]."""
        self._check("start", start, None, tuple(residual.shape))
        out = torch.empty((residual.shape[0], 2 * residual.shape[1]), dtype=out_dtype, device=self.device)
        return self._sum_norm("join_rows", residual, delta, None, None, 1.0, start, out)

    def kept_copy(self, x: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
        """A float32 ``[T, H]`` tensor in ``dtype``, in memory of its own."""
        return torch.mul(x, 1.0) if dtype == torch.float32 else self.add_cast(x, None, dtype)

    def softcap_(self, x: torch.Tensor, cap: float, scale: float = 1.0) -> torch.Tensor:
        """``x = cap * tanh(scale * x / cap)`` in place, float32."""
        self._check("x", x, torch.float32)
        if not cap > 0:
            raise KernelError(f"softcap: the cap must be positive, got {cap}")
        self._launched(self._core.velox_softcap(_ptr(x), x.numel(), float(scale), float(cap), self._stream()), "softcap")
        return x

    def poly_norm(self, x: torch.Tensor, coefficients: torch.Tensor, eps: float) -> torch.Tensor:
        """``a N(x) + b N(x^2) + c N(x^3) + e`` per row, ``N(y) = y * rsqrt(mean(y^2) + eps)``; ``coefficients`` = (a, b, c, e), float32 on the
        device; float32 arithmetic with one rounding."""
        self._check("x", x)
        if x.dim() != 2:
            raise KernelError("poly_norm: rows are [T, F]")
        self._check("coefficients", coefficients, torch.float32, (4,))
        out = torch.empty_like(x)
        self._launched(self._core.velox_poly_norm(_ptr(x), _ptr(out), _ptr(coefficients), x.shape[0], x.shape[1], float(eps), _code(x.dtype), self._stream()), "poly_norm")
        return out

    def qk_norm_write(self, qkv, num_heads, num_kv_heads, dim, vdim, cached_dim, q_norm, k_norm, whole, eps, q_temp, positions, first_values, mix_weight,
                      slot_mapping, k_cache, v_cache, block_size, write_kv=True) -> torch.Tensor:
        """Rows of ``qkv`` hold ``num_heads`` queries and ``num_kv_heads`` keys of ``dim`` channels and ``num_kv_heads`` values
        of ``vdim`` (and possibly columns of others behind them).  Queries and keys pass an RMS norm (``whole``: over all heads at once, weights of that size; else per head
        with one weight of ``dim``), the queries the temperature ``q_temp = (coef, every)``; values are blended with
        ``first_values = (tensor, first column)`` by ``mix_weight`` (one float32 on the device).  Returns the queries as the
        attention kernels read them, ``[T, num_heads * cached_dim]``; keys and values go into the cache at that head size,
        padding channels as zeros."""
        if qkv.dim() != 2:
            raise KernelError("qk_norm_write: rows are [T, width]")
        tokens, width = qkv.shape
        q_size, k_size, v_size = num_heads * dim, num_kv_heads * dim, num_kv_heads * vdim
        self._check("qkv", qkv)
        if width < q_size + k_size + v_size:
            raise KernelError(f"qk_norm_write: rows of {width} elements do not hold {q_size} + {k_size} + {v_size}")
        self._check("positions", positions, torch.int32, (tokens,))
        self._check("q_norm", q_norm, torch.float32, (q_size if whole else dim,))
        self._check("k_norm", k_norm, torch.float32, (k_size if whole else dim,))
        if cached_dim < max(dim, vdim) or block_size <= 0 or block_size & (block_size - 1):
            raise KernelError(f"qk_norm_write: cached_dim={cached_dim} below dim={dim} or vdim={vdim}, or block_size={block_size} no power of two")
        first = first_offset = first_stride = None
        if first_values is not None:
            first, first_offset = first_values
            self._check("first_values", first, qkv.dtype)
            if first.dim() != 2 or first.shape[0] != tokens or first_offset < 0 or first_offset + v_size > first.shape[1]:
                raise KernelError("qk_norm_write: the earlier layer's values do not lie inside the rows given")
            first_stride = first.shape[1]
            self._check("mix_weight", mix_weight, torch.float32, ())
        if write_kv:
            self._check("slot_mapping", slot_mapping, torch.int32, (tokens,))
            pages = k_cache.shape[0]
            self._check("k_cache", k_cache, qkv.dtype, (pages, num_kv_heads, block_size, cached_dim))
            self._check("v_cache", v_cache, qkv.dtype, (pages, num_kv_heads, cached_dim, block_size))
        coef, every = (float(q_temp[0]), int(q_temp[1])) if q_temp is not None else (0.0, 0)
        if q_temp is not None and every < 1:
            raise KernelError("qk_norm_write: q_temp's 'every' must be at least 1")
        queries = torch.empty((tokens, num_heads * cached_dim), dtype=qkv.dtype, device=self.device)
        status = self._core.velox_qk_norm_write(
            _ptr(qkv), width, _ptr(queries), _ptr(q_norm), _ptr(k_norm), _ptr(positions), _ptr(first), int(first_stride or 0), int(first_offset or 0),
            _ptr(mix_weight) if first is not None else _P(0), _ptr(slot_mapping) if write_kv else _P(0), _ptr(k_cache) if write_kv else _P(0),
            _ptr(v_cache) if write_kv else _P(0), tokens, num_heads, num_kv_heads, dim, vdim, cached_dim, block_size.bit_length() - 1, int(bool(whole)),
            int(bool(write_kv)), float(eps), coef, every, _code(qkv.dtype), self._stream())
        self._launched(status, "qk_norm_write")
        return queries

    # -- matrix products --------------------------------------------------------------------------
    @staticmethod
    def _scale_args(deferred: Optional[DeferredNorm]):
        """The four arguments by which a skinny product learns how to scale its result rows."""
        if deferred is None:
            return _P(0), 0, 0.0, 0.0
        return _ptr(deferred.sums), int(deferred.sums.shape[1]), 1.0 / deferred.width, float(deferred.eps)

    def _packed_rows_of(self, x: torch.Tensor, k: int) -> Optional[torch.Tensor]:
        """The copy of decode-sized activations ``x`` [M <= 16, k] in the order the skinny kernels' lanes read them, if the
        kernel that wrote ``x`` left one (it hangs on the tensor object), else None."""
        twin, version = getattr(x, "_velox_packed_rows", (None, None))
        if (twin is None or version != x._version or x.dim() != 2 or x.shape[0] > 16 or x.shape[1] != k or k % 64 != 0
                or twin.numel() != k // 64 * 1024 or twin.dtype != torch.bfloat16):
            return None
        return twin

    def _room_for_packed_rows(self, m: int, n: int) -> Optional[torch.Tensor]:
        """Room for ``[m, n]`` activations in the lanes' order, if the kernels can write and read them like that and it
        pays: the copy always has 16 rows, and what a product's activations cost is their bytes, not the pieces they come in
        (measured on MI355X, 3584 x 18944: 12 rows row-major 28.5 us, 16 rows 30.9 us, the copy 28.4 us at any number)."""
        if not 13 <= m <= 16 or n % 64 != 0 or not self.pack_decode_weights:
            return None
        return torch.empty(n // 64 * 1024, dtype=torch.bfloat16, device=self.device)

    def materialize(self, x):
        """A ``DeferredNorm`` as the plain normalised tensor (one small kernel); anything else is returned as it is."""
        if not isinstance(x, DeferredNorm):
            return x
        m, n = x.x.shape
        out = torch.empty_like(x.x)
        sums, blocks, inv_width, eps = self._scale_args(x)
        self._launched(self._core.velox_row_scale_apply(_ptr(x.x), sums, blocks, inv_width, eps, _ptr(out), m, n, self._stream()), "row_scale_apply")
        return out

    def linear(self, x, weight: torch.Tensor, bias: Optional[torch.Tensor], out_dtype: torch.dtype, partials_ok: bool = False,
               residual_norm: Optional[ResidualSink] = None):
        """``x @ weight^T (+ bias)`` as ``[M, N]`` in ``out_dtype``.  With ``partials_ok`` the result may instead come back as
        float32 partial sums ``[S, M, N]`` that the consumer adds (``add_rmsnorm`` does).  With ``residual_norm`` it may
        come back as a ``DeferredNorm``: the product has then been added to ``residual_norm.residual`` and multiplied
        with the weight of ``residual_norm.norm`` (decode-sized bfloat16 products whose weight is registered).  ``x`` may
        be a ``DeferredNorm``."""
        weight, prepared = _weight_of(weight)
        packed = prepared.copy(1) if prepared is not None else None
        deferred = x if isinstance(x, DeferredNorm) else None
        if deferred is not None:
            x = deferred.x
            if not (self.use_skinny_gemm and packed is not None and x.shape[0] <= 16 and x.shape[1] % 64 == 0 and weight.dtype == torch.bfloat16):
                x, deferred = self.materialize(deferred), None
        self._check("x", x, align=16)
        self._check("weight", weight, align=16)
        if x.dim() != 2 or weight.dim() != 2 or x.shape[1] != weight.shape[1]:
            raise KernelError(f"linear: x {tuple(x.shape)} and weight {tuple(weight.shape)} do not match")
        m, k = x.shape
        n = weight.shape[0]
        if bias is not None:
            self._check("bias", bias, torch.float32, (n,))
        if deferred is not None:
            return self.skinny_gemm(x, weight, bias, out_dtype, packed=packed, row_scale=deferred, x_packed=self._packed_rows_of(x, k))
        if residual_norm is not None and bias is None:
            fused = self._linear_into_residual(x, weight, residual_norm, packed=packed)
            if fused is not None:
                return fused
        if (partials_ok and bias is None and self.use_skinny_gemm and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16
                and 16 < m <= 64 and k % 64 == 0 and n <= 8192 and n % 4 == 0):
            return self.skinny_gemm_splitk(x, weight, packed=packed)
        skinny_rows = 16 if n > 8192 else 32  # measured on MI355X: beyond this the library's kernels stream faster
        if self.use_skinny_gemm and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16 and m <= skinny_rows and k % 64 == 0:
            return self.skinny_gemm(x, weight, bias, out_dtype, packed=packed, x_packed=self._packed_rows_of(x, k))
        if self.use_library_gemm and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16 and bias is not None and out_dtype == torch.bfloat16:
            # the library adds a bias of the product's own dtype to its float32 sums before the one rounding
            return torch.nn.functional.linear(x, weight, self._bias_in_bfloat16(bias))
        if self.use_library_gemm and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16 and bias is None:
            if out_dtype == torch.bfloat16:
                return torch.nn.functional.linear(x, weight)
            if out_dtype == torch.float32:
                if self._mm_out_dtype_ok is None:
                    self._decide_float32_out_route()
                return torch.mm(x, weight.t(), out_dtype=torch.float32)
        return self.gemm_fma(x, weight, bias, out_dtype)

    def _bias_in_bfloat16(self, bias: torch.Tensor) -> torch.Tensor:
        """A bfloat16 copy of a float32 bias vector, made once per vector (keyed by its storage; the float32 vector is kept
        alive beside it, so the key cannot come to mean another tensor)."""
        key = (bias.data_ptr(), bias.numel())
        held = self._bias_copies.get(key)
        if held is None or held[0] is not bias:
            held = (bias, bias.to(torch.bfloat16))
            self._bias_copies[key] = held
        return held[1]

    def _decide_float32_out_route(self) -> None:
        """Decides once how a bfloat16 product with a float32 result and more rows than the skinny kernels take (the
        head over many wanted rows) is computed: by the library with a float32 output, if this PyTorch has that call.
        If it has not, that is an error here, at load time, and not a silent fall to the exact FMA kernel, which is some
        two hundred times slower at such sizes."""
        probe = torch.zeros((32, 64), dtype=torch.bfloat16, device=self.device)
        try:
            torch.mm(probe, probe.t(), out_dtype=torch.float32)
            self._mm_out_dtype_ok = True
        except (RuntimeError, TypeError) as err:
            self._mm_out_dtype_ok = False
            raise KernelError("this PyTorch's matrix library has no bfloat16 product with a float32 result (torch.mm(..., out_dtype=)); "
                              f"logits of many rows at once need it in a bfloat16 run: {err}") from err

    def _linear_into_residual(self, x: torch.Tensor, weight: torch.Tensor, sink: ResidualSink, waves: Optional[int] = None, row_tiles: Optional[int] = None,
                              packed: Optional[torch.Tensor] = None) -> Optional[DeferredNorm]:
        """``sink.residual += x @ weight^T`` with the first half of ``sink.norm`` in the same kernel, if this product
        qualifies (bfloat16, at most 16 rows, registered weight, a norm that can be split); None otherwise."""
        form = sink.norm.deferred_form()
        weight, prepared = _weight_of(weight)
        if prepared is not None and packed is None:
            packed = prepared.copy(1)
        m, k = x.shape
        n = weight.shape[0]
        residual = sink.residual
        if (not self.use_skinny_gemm or not self.fuse_residual_norm or form is None or packed is None or m > 16 or k % 64 != 0 or n > 16 * 512
                or x.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16):
            return None
        norm_weight, eps = form
        self._check("residual", residual, torch.float32, (m, n), align=16)
        self._check("norm weight", norm_weight, torch.float32, (n,))
        blocks = (n + 15) // 16
        if row_tiles is None:
            # one 16-row tile of the weight per workgroup while that is at most one workgroup per compute unit; a wider
            # weight takes two (measured on MI355X at 8 rows: 5120 x 27648 65.8 -> 58.5 us, 3584 x 18944 27.8 -> 41.4)
            # and a narrow one half a tile, which gives every compute unit a workgroup (1536 x 8960: 13.0 -> 10.8 us)
            row_tiles = 2 if blocks > self.num_cus else 0 if 2 * blocks <= self.num_cus else 1
        if row_tiles == 0:
            blocks *= 2  # (half a tile per workgroup: sums of squares per 8 columns)
        out = torch.empty((m, n), dtype=torch.bfloat16, device=self.device)
        sums = torch.empty((16, blocks), dtype=torch.float32, device=self.device)
        x_packed = self._packed_rows_of(x, k)
        out_packed = self._room_for_packed_rows(m, n)
        status = self._core.velox_skinny_residual_norm_bf16(_ptr(x if x_packed is None else x_packed), _ptr(packed), _ptr(residual), _ptr(norm_weight),
                                                            _ptr(out), _ptr(sums), m, n, k, int(waves or 8), int(row_tiles), int(x_packed is not None), _ptr(out_packed),
                                                            self._stream())
        self._launched(status, "skinny_residual_norm")
        if out_packed is not None:
            out._velox_packed_rows = (out_packed, out._version)
        return DeferredNorm(out, sums, n, float(eps), sink.norm)

    @staticmethod
    def pack_rows(weight: torch.Tensor, matrices: int = 1) -> torch.Tensor:
        """``weight`` [N, K] bfloat16 (``matrices`` stacked matrices of N / matrices rows each) in the order the skinny
        kernels' lanes read it: [row tile of 16][block of 64 indices][half h][lane = 16 * g + row][8 elements] holds index
        ``16 g + 8 h + e`` of the block; each matrix is padded with zero rows to whole tiles.  Each of a wave's two loads of
        a block is then one contiguous kilobyte."""
        n_all, k = weight.shape
        n = n_all // matrices
        tiles = (n + 15) // 16
        padded = torch.zeros((matrices, tiles * 16, k), dtype=weight.dtype, device=weight.device)
        padded[:, :n] = weight.view(matrices, n, k)
        # [matrix, tile, row i, block, group g, half h, 8] -> [matrix, tile, block, h, g, i, 8]
        return padded.view(matrices, tiles, 16, k // 64, 4, 2, 8).permute(0, 1, 3, 5, 4, 2, 6).contiguous().view(-1)

    def skinny_gemm(self, x, weight, bias, out_dtype, waves: Optional[int] = None, row_tiles: Optional[int] = None, packed: Optional[torch.Tensor] = None, n: Optional[int] = None,
                    row_scale: Optional[DeferredNorm] = None, x_packed: Optional[torch.Tensor] = None, ungated: Optional[str] = None):
        """Few rows (M <= 64) times a bfloat16 weight: the weight-streaming kernel of the decode step.  ``packed`` is
        ``pack_rows(weight)``, used instead of ``weight`` when given (``n`` = rows of the weight).  ``row_scale``: ``x`` is
        its ``.x`` and the result rows are scaled as it says (M <= 16).  ``ungated``: the activation of a unit without a gate
        branch (``relu2``) on the float32 sums, as the product's epilogue."""
        m, k = x.shape
        n = weight.shape[0] if weight is not None else n
        if packed is not None:
            weight_arg = packed
            if packed.dtype != torch.bfloat16 or packed.numel() != ((n + 15) // 16) * 16 * k:
                raise KernelError("skinny_gemm: the packed weight does not match N and K")
        else:
            weight_arg = weight
        if x.dtype != torch.bfloat16 or weight_arg.dtype != torch.bfloat16 or m > 64 or k % 64 != 0:
            raise KernelError(f"skinny_gemm: needs bfloat16 operands, M <= 64 and K % 64 == 0 (M={m}, K={k})")
        if row_tiles is None:
            # 64 rows per wave quarter the activation traffic, which pays for the row-major weight only
            row_tiles = 4 if (m <= 16 and n >= 64 * 2 * self.num_cus and (packed is None or m > 8)) else 1
        if waves is None and packed is not None and row_tiles == 1 and m <= 16:
            waves = 8
        if waves is None:
            rows_per_block = 16 * row_tiles if m <= 16 else 32
            blocks = (n + rows_per_block - 1) // rows_per_block
            wanted = (8 * self.num_cus + blocks - 1) // blocks  # about eight waves per SIMD lane group across the GPU
            waves = 16 if wanted > 8 else 8 if wanted > 4 else 4
        out = torch.empty((m, n), dtype=out_dtype, device=self.device)
        if row_scale is not None and m > 16:
            raise KernelError("skinny_gemm: rows are scaled only for M <= 16")
        if x_packed is not None and (m > 16 or x_packed.dtype != torch.bfloat16 or x_packed.numel() != k // 64 * 1024):
            raise KernelError("skinny_gemm: the packed activations do not match M and K")
        status = self._core.velox_skinny_gemm_bf16(_ptr(x if x_packed is None else x_packed), _ptr(weight_arg), _ptr(bias), _ptr(out), m, n, k, _code(out_dtype),
                                                   int(waves), int(row_tiles), 1 if packed is not None else 0, *self._scale_args(row_scale),
                                                   int(x_packed is not None), self._ACTIVATION_CODES[ungated] if ungated else 0, self._stream())
        self._launched(status, "skinny_gemm")
        return out

    _GATED_ACTIVATIONS = {"silu": 0, "gelu_tanh": 1, "relu": 2}

    def linear_gated_act(self, x: torch.Tensor, gate_up_weight: torch.Tensor, out_dtype: torch.dtype, activation: str) -> torch.Tensor:
        """``act(x Wgate^T) * (x Wup^T)`` for ``W = [Wgate; Wup]`` and ``activation`` ``"silu"``, ``"gelu_tanh"`` or ``"relu"``: one kernel for
        decode-sized bfloat16 batches (see ``linear_silu_mul``), else the product followed by the activation's kernel."""
        return self.linear_silu_mul(x, gate_up_weight, out_dtype, activation=activation)

    def linear_silu_mul(self, x: torch.Tensor, gate_up_weight: torch.Tensor, out_dtype: torch.dtype, waves: Optional[int] = None, pairs: Optional[int] = None, packed: Optional[torch.Tensor] = None,
                        activation: str = "silu") -> torch.Tensor:
        """``silu(x Wgate^T) * (x Wup^T)`` for ``W = [Wgate; Wup]`` (``activation="gelu_tanh"``: the tanh form of GELU in SiLU's place; ``"relu"``: the rectifier).  Decode-sized bfloat16 batches run as one kernel that
        never writes the [M, 2I] product (up to 16 rows on any weight, 17 .. 64 rows on a registered one); everything else
        is the product followed by the SiLU kernel.  ``waves`` and ``pairs`` override the launch shape the wrapper would
        pick (up to 16 rows: waves per workgroup and gate/up tile pairs per wave; 17 .. 64 rows: ``pairs`` = tile pairs per
        workgroup)."""
        operand = gate_up_weight  # (as given: handed on to ``linear`` when nothing here applies)
        gate_up_weight, prepared = _weight_of(gate_up_weight)
        if packed is None and prepared is not None:
            packed = prepared.copy(2)
        deferred = x if isinstance(x, DeferredNorm) else None
        if deferred is not None:
            x = deferred.x
        m, k = x.shape
        two_n = gate_up_weight.shape[0]
        fused = (self.use_skinny_gemm and x.dtype == torch.bfloat16 and gate_up_weight.dtype == torch.bfloat16 and out_dtype == torch.bfloat16
                 and m <= 16 and k % 64 == 0 and two_n % 2 == 0 and x.dim() == 2 and gate_up_weight.shape[1] == k)
        if activation not in self._GATED_ACTIVATIONS:
            raise KernelError(f"linear_silu_mul: activation {activation!r} is not built ({', '.join(self._GATED_ACTIVATIONS)})")
        if (not fused and activation == "silu" and deferred is None and self.use_skinny_gemm and x.dim() == 2 and 16 < m <= 64 and k % 64 == 0 and two_n % 2 == 0
                and x.dtype == torch.bfloat16 and gate_up_weight.dtype == torch.bfloat16 and out_dtype == torch.bfloat16
                and gate_up_weight.shape[1] == k and packed is not None):
            # 17 .. 64 rows: the kernel that streams the packed weight once with the activation as its epilogue
            n = two_n // 2
            if packed.dtype != torch.bfloat16 or packed.numel() != 2 * ((n + 15) // 16) * 16 * k:
                raise KernelError("linear_silu_mul: the packed weight does not match N and K")
            self._check("x", x, torch.bfloat16, align=16)
            out = torch.empty((m, n), dtype=torch.bfloat16, device=self.device)
            # pairs of tiles per workgroup: a compute unit holds one such workgroup at a time, so the launch takes
            # rounds x pairs; the fewest wins, then the larger workgroup (measured on MI355X at 64 rows: 37888 x 3584
            # with 5 pairs 51 us, the library's product + SiLU kernel 58; 55296 x 5120 with 4 pairs 106 us against 114)
            tiles = (n + 15) // 16
            per_group = min(range(2, 7), key=lambda p: (-(-(-(-tiles // p)) // self.num_cus) * p, -p))
            self._launched(self._core.velox_skinny_glu_rows_bf16(_ptr(x), _ptr(packed), _ptr(out), m, n, k, per_group if pairs is None else int(pairs), self._stream()),
                           "skinny_glu_rows")
            return out
        if not fused:
            product = self.linear(deferred if deferred is not None else x, operand, None, out_dtype)
            return self.silu_mul(product) if activation == "silu" else self.gated_act_mul(product, activation)
        if deferred is not None and packed is None:  # only the kernels of a registered weight scale rows
            x, deferred = self.materialize(deferred), None
        self._check("x", x, align=16)
        self._check("gate_up_weight", gate_up_weight, align=16)
        n = two_n // 2
        if pairs is None:
            pairs = 1  # measured on MI355X: two pairs per wave never paid, packed or not
        if waves is None:
            waves = 8
        out = torch.empty((m, n), dtype=out_dtype, device=self.device)
        x_packed = self._packed_rows_of(x, k)
        out_packed = self._room_for_packed_rows(m, n)
        status = self._core.velox_skinny_gemm_glu_act_bf16(_ptr(x if x_packed is None else x_packed), _ptr(packed if packed is not None else gate_up_weight), _ptr(out),
                                                           m, n, k, int(waves), int(pairs), 1 if packed is not None else 0, *self._scale_args(deferred),
                                                           int(x_packed is not None), _ptr(out_packed), self._GATED_ACTIVATIONS[activation], self._stream())
        self._launched(status, "skinny_gemm_glu")
        if out_packed is not None:
            out._velox_packed_rows = (out_packed, out._version)
        return out

    def skinny_gemm_splitk(self, x, weight, splits: Optional[int] = None, packed: Optional[torch.Tensor] = None) -> torch.Tensor:
        """17 .. 64 rows times a bfloat16 weight with few rows and a long K: float32 partial sums ``[S, M, N]``.
        ``packed``: ``pack_rows(weight)``, read instead of ``weight`` when given."""
        m, k = x.shape
        n = weight.shape[0]
        if x.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16 or m > 64 or k % 64 != 0:
            raise KernelError(f"skinny_gemm_splitk: needs bfloat16 operands, M <= 64 and K % 64 == 0 (M={m}, K={k})")
        self._check("x", x, align=16)
        self._check("weight", weight, align=16)
        if splits is None:
            # one workgroup per compute unit (measured on MI355X: a unit that gets a second one holds the others up)
            blocks = (n + 63) // 64
            splits = max(1, min(self.num_cus // blocks, k // 256, 16))
        per_split = (k // 64 + splits - 1) // splits
        splits = (k // 64 + per_split - 1) // per_split  # no empty slice
        out = torch.empty((splits, m, n), dtype=torch.float32, device=self.device)
        if packed is not None and (packed.dtype != torch.bfloat16 or packed.numel() != ((n + 15) // 16) * 16 * k):
            raise KernelError("skinny_gemm_splitk: the packed weight does not match N and K")
        status = self._core.velox_skinny_gemm_splitk_bf16(_ptr(x), _ptr(weight if packed is None else packed), _ptr(out), m, n, k, splits,
                                                          int(packed is not None), self._stream())
        self._launched(status, "skinny_gemm_splitk")
        return out

    def gemm_fma(self, x, weight, bias, out_dtype):
        m, k = x.shape
        n = weight.shape[0]
        out = torch.empty((m, n), dtype=out_dtype, device=self.device)
        status = self._core.velox_gemm_fma(_ptr(x), _ptr(weight), _ptr(bias), _ptr(out), m, n, k, _code(x.dtype), _code(weight.dtype), _code(out_dtype), self._stream())
        self._launched(status, "gemm_fma")
        return out

    def silu_mul(self, gate_up: torch.Tensor) -> torch.Tensor:
        self._check("gate_up", gate_up)
        if gate_up.dim() != 2 or gate_up.shape[1] % 2 != 0:
            raise KernelError("silu_mul: expected [T, 2 * intermediate]")
        tokens, inter = gate_up.shape[0], gate_up.shape[1] // 2
        out = torch.empty((tokens, inter), dtype=gate_up.dtype, device=self.device)
        status = self._core.velox_silu_mul(_ptr(gate_up), _ptr(out), tokens, inter, _code(gate_up.dtype), self._stream())
        self._launched(status, "silu_mul")
        return out

    # -- residual streams, short convolution, linear recurrences ------------------------------------
    MAX_STREAMS = 8
    MAX_STREAM_WIDTH = 16384
    MAX_CONV_TAPS = 8

    def stream_norm(self, residual, terms, scales, mix, out_weights, in_weights, weight, eps, streams, center, out_dtype, rows=None):
        """``residual`` float32 ``[T, streams * H]``.  With ``terms`` (one or two ``[T, H]`` tensors, ``y = sum_i scales[i] terms[i]``):
        ``x_t <- sum_s mix[s, t] x_s + out_weights[t] y`` for all streams at once (``mix`` None: the identity, ``out_weights``
        None: ones), in place unless ``rows`` picks rows.  Returns ``norm(sum_s in_weights[s] x_s) * weight`` in
        ``out_dtype``, for all rows or for ``rows``; ``center``: a layer norm without bias, else an RMS norm."""
        self._check("residual", residual, torch.float32)
        if residual.dim() != 2 or streams < 1 or residual.shape[1] % streams != 0:
            raise KernelError(f"stream_norm: residual must be [T, streams * H], got {tuple(residual.shape)} for {streams} streams")
        tokens, hidden = residual.shape[0], residual.shape[1] // streams
        if streams > self.MAX_STREAMS or hidden > self.MAX_STREAM_WIDTH:
            raise KernelError(f"stream_norm: at most {self.MAX_STREAMS} streams of at most {self.MAX_STREAM_WIDTH} channels")
        self._check("weight", weight, torch.float32, (hidden,))
        if len(terms) > 2 or len(terms) != len(scales):
            raise KernelError("stream_norm: one or two terms, each with its scale")
        for i, term in enumerate(terms):
            self._check(f"term {i}", term, None, (tokens, hidden))
        for name, t, shape in (("mix", mix, (streams, streams)), ("out_weights", out_weights, (streams,)), ("in_weights", in_weights, (streams,))):
            if t is not None:
                self._check(name, t, torch.float32, shape)
        if rows is not None:
            self._check("rows", rows, torch.int32)
        count = tokens if rows is None else rows.shape[0]
        out = torch.empty((count, hidden), dtype=out_dtype, device=self.device)
        t0 = terms[0] if len(terms) > 0 else None
        t1 = terms[1] if len(terms) > 1 else None
        status = self._core.velox_stream_norm(
            _ptr(residual), _ptr(t0), _code(t0.dtype) if t0 is not None else 0, float(scales[0]) if t0 is not None else 0.0,
            _ptr(t1), _code(t1.dtype) if t1 is not None else 0, float(scales[1]) if t1 is not None else 0.0, len(terms),
            _ptr(mix), _ptr(out_weights), _ptr(in_weights), _ptr(weight), _ptr(rows), _ptr(out), _code(out_dtype), count, hidden, int(streams),
            int(bool(center)), float(eps), self._stream())
        self._launched(status, "stream_norm")
        return out

    def gated_act_mul(self, gate_up: torch.Tensor, activation: str) -> torch.Tensor:
        """``act(gate) * up`` of ``[T, 2 * I]`` (gate first), ``activation`` ``"silu"``, ``"gelu_tanh"`` or ``"relu"``; float32 inside."""
        self._check("gate_up", gate_up)
        kinds = self._GATED_ACTIVATIONS
        if gate_up.dim() != 2 or gate_up.shape[1] % 2 != 0 or activation not in kinds:
            raise KernelError("gated_act_mul: expected [T, 2 * intermediate] and 'silu', 'gelu_tanh' or 'relu'")
        tokens, inter = gate_up.shape[0], gate_up.shape[1] // 2
        out = torch.empty((tokens, inter), dtype=gate_up.dtype, device=self.device)
        for first in range(0, tokens, 65535):
            count = min(65535, tokens - first)
            self._launched(self._core.velox_gated_act_mul(_ptr(gate_up[first:first + count]), _ptr(out[first:first + count]), count, inter,
                                                          _code(gate_up.dtype), kinds[activation], self._stream()), "gated_act_mul")
        return out

    def short_conv(self, x, channels, weight, tail, slots, cu_q, max_q_len, activation="none", update_state=True, first=0, bias=None):
        """The ``channels`` columns of ``x`` [T, >= first + channels] from column ``first`` on through ``y_t = sum_j w[:, j] u_(t - taps + 1 + j)
        (+ bias)`` per sequence (``weight`` float32 [channels, taps], ``bias`` float32 [channels]); the inputs before a portion's start come from ``tail[slot]`` ([taps - 1, channels],
        oldest first, the dtype of ``x``; None: zeros), which is brought up to date unless ``update_state`` is false.
        ``activation``: ``"none"`` or ``"silu"``.  Returns [T, channels] in x's dtype."""
        self._check("x", x)
        if x.dim() != 2 or first < 0 or x.shape[1] < first + channels:
            raise KernelError(f"short_conv: x {tuple(x.shape)} has fewer than {first} + {channels} columns")
        if bias is not None:
            self._check("bias", bias, torch.float32, (channels,))
        if weight.dim() != 2:
            raise KernelError("short_conv: the weights must be [channels, taps]")
        taps = weight.shape[1]
        self._check("weight", weight, torch.float32, (channels, taps))
        if not 1 <= taps <= self.MAX_CONV_TAPS:
            raise KernelError(f"short_conv: 1 to {self.MAX_CONV_TAPS} taps, got {taps}")
        self._check("slots", slots, torch.int32)
        self._check("cu_q", cu_q, torch.int32, (slots.shape[0] + 1,))
        if tail is not None and taps > 1:
            self._check("tail", tail, x.dtype)
            if tail.dim() != 3 or tuple(tail.shape[1:]) != (taps - 1, channels):
                raise KernelError(f"short_conv: the state must be [slots, {taps - 1}, {channels}], got {tuple(tail.shape)}")
        else:
            tail = None
        if activation not in ("none", "silu"):
            raise KernelError(f"short_conv: activation {activation!r}")
        out = torch.empty((x.shape[0], channels), dtype=x.dtype, device=self.device)
        status = self._core.velox_short_conv(_P(x.data_ptr() + first * x.element_size()), x.shape[1], int(channels), _ptr(weight), taps, _ptr(tail), _ptr(slots), _ptr(cu_q), _ptr(out),
                                             slots.shape[0], int(max_q_len), _code(x.dtype), int(activation == "silu"), int(bool(update_state)), _ptr(bias), self._stream())
        self._launched(status, "short_conv")
        return out

    def rotate_pad_write(self, qkv, num_heads, num_kv_heads, dim, vdim, cached_dim, positions, cos, sin, slot_mapping, k_cache, v_cache, block_size, write_kv=True,
                         interleaved=False, post_norm_eps: float = 0.0, values_are_keys: bool = False):
        """Rotates the first ``2 * cos.shape[1]`` channels of every q and k head of ``qkv`` [T, heads * dim + kv_heads * (dim + vdim)]
        (channel i with i + half, or 2i with 2i + 1 when ``interleaved``), writes k and v into the pages at ``cached_dim`` channels a head (zeros in the padding)
        and returns q as [T, heads * cached_dim].  ``post_norm_eps`` > 0: every q and k head is divided by its root mean square
        behind the rotation.  ``values_are_keys``: the rows hold no values ([T, (heads + kv_heads) * dim]); a head's values are its
        keys as they stand in the row."""
        self._check("qkv", qkv)
        tokens = qkv.shape[0]
        if values_are_keys and vdim != dim:
            raise KernelError(f"rotate_pad_write: values that are the keys have their size, not {vdim} beside {dim}")
        width = num_heads * dim + num_kv_heads * (dim + (0 if values_are_keys else vdim))
        if qkv.dim() != 2 or qkv.shape[1] != width:
            raise KernelError(f"rotate_pad_write: qkv must be [T, {width}], got {tuple(qkv.shape)}")
        if dim > cached_dim or vdim > cached_dim:
            raise KernelError("rotate_pad_write: the cached head size must cover dim and vdim")
        self._check("positions", positions, torch.int32, (tokens,))
        half = 0
        if cos is not None:
            half = cos.shape[1]
            self._check("cos", cos, torch.float32)
            self._check("sin", sin, torch.float32, tuple(cos.shape))
            if 2 * half > dim:
                raise KernelError(f"rotate_pad_write: the rotation spans {2 * half} channels of heads of {dim}")
        if write_kv:
            self._check("slot_mapping", slot_mapping, torch.int32, (tokens,))
            self._check("k_cache", k_cache, qkv.dtype)
            self._check("v_cache", v_cache, qkv.dtype)
            if tuple(k_cache.shape[1:]) != (num_kv_heads, block_size, cached_dim) or tuple(v_cache.shape[1:]) != (num_kv_heads, cached_dim, block_size):
                raise KernelError(f"rotate_pad_write: pages of {tuple(k_cache.shape[1:])} / {tuple(v_cache.shape[1:])} do not hold "
                                  f"{num_kv_heads} heads of {cached_dim} over {block_size} tokens")
        q = torch.empty((tokens, num_heads * cached_dim), dtype=qkv.dtype, device=self.device)
        status = self._core.velox_rotate_pad_write(_ptr(qkv), width, _ptr(q), _ptr(positions), _ptr(cos), _ptr(sin), half, _ptr(slot_mapping) if write_kv else _P(0),
                                                   _ptr(k_cache) if write_kv else _P(0), _ptr(v_cache) if write_kv else _P(0), tokens, num_heads, num_kv_heads,
                                                   dim, vdim, cached_dim, int(block_size), int(bool(write_kv)), _code(qkv.dtype), int(bool(interleaved)), float(post_norm_eps),
                                                   int(bool(values_are_keys)), self._stream())
        self._launched(status, "rotate_pad_write")
        return q

    def recurrence_prepare(self, qkv, q_at, k_at, kv_heads, dim, unit, q_scale, decay_source, decay_at, heads, decay_columns, rate, bias, sign,
                           beta_source, beta_at):
        """-> ``qk`` float32 [T, kv_heads, 2, dim] (a head's q, unit vector if ``unit``, times ``q_scale``; then its k), ``decay``
        float32 [T, decay_columns] = ``exp(-rate[h] softplus(sign (z + bias)))``, ``beta`` float32 [T, heads] = ``sigmoid(b)`` or None."""
        self._check("qkv", qkv)
        tokens = qkv.shape[0]
        if qkv.dim() != 2 or max(q_at, k_at) + kv_heads * dim > qkv.shape[1]:
            raise KernelError("recurrence_prepare: q and k do not lie within the rows of qkv")
        self._check("decay_source", decay_source)
        if decay_source.dim() != 2 or decay_source.shape[0] != tokens or decay_at + decay_columns > decay_source.shape[1] or decay_columns % heads != 0:
            raise KernelError("recurrence_prepare: the decay's columns do not lie within its source")
        self._check("rate", rate, torch.float32, (heads,))
        if bias is not None:
            self._check("bias", bias, torch.float32, (decay_columns,))
        beta = None
        if beta_source is not None:
            self._check("beta_source", beta_source)
            if beta_source.dim() != 2 or beta_source.shape[0] != tokens or beta_at + heads > beta_source.shape[1]:
                raise KernelError("recurrence_prepare: beta's columns do not lie within its source")
            beta = torch.empty((tokens, heads), dtype=torch.float32, device=self.device)
        qk = torch.empty((tokens, kv_heads, 2, dim), dtype=torch.float32, device=self.device)
        decay = torch.empty((tokens, decay_columns), dtype=torch.float32, device=self.device)
        status = self._core.velox_recurrence_prepare(
            _ptr(qkv), _code(qkv.dtype), qkv.shape[1], int(q_at), int(k_at), int(kv_heads), int(dim), int(bool(unit)), float(q_scale),
            _ptr(decay_source), _code(decay_source.dtype), decay_source.shape[1], int(decay_at), int(heads), int(decay_columns), _ptr(rate), _ptr(bias), float(sign),
            _ptr(beta_source), _code(beta_source.dtype) if beta_source is not None else 0, beta_source.shape[1] if beta_source is not None else 0, int(beta_at),
            _ptr(qk), _ptr(decay), _ptr(beta), tokens, self._stream())
        self._launched(status, "recurrence_prepare")
        return qk, decay, beta

    def removal_prepare(self, main, r_at, k_at, a_at, low_at, rank, heads, dim, a_bias, w2, w0, decay_scale):
        """What the generalized delta rule reads of a row of ``main`` (read vectors, keys and removal logits of ``heads * dim``
        columns each at ``r_at``, ``k_at``, ``a_at``; the decay map's inner row of ``rank`` columns at ``low_at``), all float32:
        ``vectors`` [T, heads, 3, dim] = r, u, sigmoid(a + a_bias) * u with the unit key u = k / n; ``decay`` [T, heads * dim] =
        ``exp(-decay_scale sigmoid(w0 + w2 tanh(inner)))``; ``lengths`` [T, heads] = n = sqrt(sum(k^2) + 1e-6)."""
        self._check("main", main)
        size = heads * dim
        if main.dim() != 2 or max(r_at, k_at, a_at) + size > main.shape[1] or low_at + rank > main.shape[1] or min(r_at, k_at, a_at, low_at) < 0:
            raise KernelError("removal_prepare: the columns do not lie within the rows")
        if not 1 <= rank <= 8192:
            raise KernelError(f"removal_prepare: an inner size of {rank} is beyond the kernel (8,192 at most)")
        tokens = main.shape[0]
        self._check("a_bias", a_bias, torch.float32, (size,))
        self._check("w0", w0, torch.float32, (size,))
        self._check("w2", w2, main.dtype, (size, rank))
        vectors = torch.empty((tokens, heads, 3, dim), dtype=torch.float32, device=self.device)
        decay = torch.empty((tokens, size), dtype=torch.float32, device=self.device)
        lengths = torch.empty((tokens, heads), dtype=torch.float32, device=self.device)
        self._launched(self._core.velox_removal_prepare(_ptr(main), _code(main.dtype), main.shape[1], int(r_at), int(k_at), int(a_at), int(low_at), int(rank), int(heads),
                                                        int(dim), _ptr(a_bias), _ptr(w2), _ptr(w0), float(decay_scale), _ptr(vectors), _ptr(decay), _ptr(lengths),
                                                        tokens, self._stream()), "removal_prepare")
        return vectors, decay, lengths

    REMOVAL_CHUNK_TOKENS = 32  # portions at least this long go through the chunked kernels where the sizes are theirs

    def removal_scan(self, main, r_at, k_at, v_at, a_at, low_at, rank, heads, dim, vdim, a_bias, w2, w0, decay_scale, state, slots, cu_q, max_q_len,
                     chunked: Optional[bool] = None):
        """The generalized delta rule from the rows of its input product (columns as for ``removal_prepare``, values of ``heads * vdim``
        columns at ``v_at``) and ``state`` [slots, heads, dim, vdim], which is written back; float32 read-outs [T, heads * vdim].  Steps with a
        long portion are worked in chunks of 16 tokens on the matrix cores (heads of a multiple of 16 channels, 128 at most, and
        decays whose product over a chunk keeps away from underflow), all others token by token; ``chunked`` decides it for a
        test."""
        tokens = main.shape[0]
        scratch_elems = 0
        if chunked is not False and max_q_len >= (1 if chunked else self.REMOVAL_CHUNK_TOKENS) and 16 * decay_scale < 13:
            scratch_elems = int(self._core.velox_removal_chunk_scratch_elems(tokens, slots.shape[0], int(heads), int(dim), int(vdim), int(rank)))
        if scratch_elems == 0:
            if chunked:
                raise KernelError(f"removal_scan: heads of {dim} channels with an inner size of {rank} are not the chunked kernels'")
            vectors, decay, lengths = self.removal_prepare(main, r_at, k_at, a_at, low_at, rank, heads, dim, a_bias, w2, w0, decay_scale)
            return self.linear_scan(vectors, main, v_at, decay, lengths, state, slots, cu_q, max_q_len, heads, heads, dim, vdim, "removal")
        self._check("main", main)
        size = heads * dim
        if (main.dim() != 2 or max(r_at, k_at, a_at) + size > main.shape[1] or low_at + rank > main.shape[1] or v_at + heads * vdim > main.shape[1]
                or min(r_at, k_at, v_at, a_at, low_at) < 0):
            raise KernelError("removal_scan: the columns do not lie within the rows")
        self._check("a_bias", a_bias, torch.float32, (size,))
        self._check("w0", w0, torch.float32, (size,))
        self._check("w2", w2, main.dtype, (size, rank))
        self._check("state", state, torch.float32)
        if state.dim() != 4 or tuple(state.shape[1:]) != (heads, dim, vdim):
            raise KernelError(f"removal_scan: the state must be [slots, {heads}, {dim}, {vdim}], got {tuple(state.shape)}")
        self._check("slots", slots, torch.int32)
        self._check("cu_q", cu_q, torch.int32, (slots.shape[0] + 1,))
        if not 1 <= max_q_len <= tokens:
            raise KernelError(f"removal_scan: max_q_len={max_q_len} outside [1, {tokens}]")
        out = torch.empty((tokens, heads * vdim), dtype=torch.float32, device=self.device)
        scratch = torch.empty(scratch_elems, dtype=torch.float32, device=self.device)
        self._launched(self._core.velox_removal_chunk_scan(_ptr(main), _code(main.dtype), main.shape[1], int(r_at), int(k_at), int(v_at), int(a_at), int(low_at), int(rank),
                                                           int(heads), int(dim), int(vdim), _ptr(a_bias), _ptr(w2), _ptr(w0), float(decay_scale), _ptr(scratch), _ptr(state),
                                                           _ptr(slots), _ptr(cu_q), _ptr(out), slots.shape[0], int(max_q_len), self._stream()), "removal_scan")
        return out

    def gated_scan(self, projected, width, gate_bias, input_bias, shift, state, slots, cu_q, max_q_len):
        """``projected`` [T, 3 * width] = z, u, g of every token; per channel and sequence, from ``state[slot]`` ([slots, width] float32, written
        back): ``S <- (1 - z) S + z c`` with ``z = sigmoid(z + gate_bias)``, ``u += input_bias`` and ``c = u + shift`` (u >= 0) or ``sigmoid(u)``.
        Returns ``S * silu(g)``, [T, width] in the rows' dtype."""
        self._check("projected", projected)
        tokens = projected.shape[0]
        if projected.dim() != 2 or projected.shape[1] != 3 * width:
            raise KernelError(f"gated_scan: rows of {3 * width} columns expected, got {tuple(projected.shape)}")
        self._check("gate_bias", gate_bias, torch.float32, (width,))
        self._check("input_bias", input_bias, torch.float32, (width,))
        self._check("state", state, torch.float32)
        if state.dim() != 2 or state.shape[1] != width:
            raise KernelError(f"gated_scan: the state must be [slots, {width}], got {tuple(state.shape)}")
        self._check("slots", slots, torch.int32)
        self._check("cu_q", cu_q, torch.int32, (slots.shape[0] + 1,))
        if not 1 <= max_q_len <= tokens:
            raise KernelError(f"gated_scan: max_q_len={max_q_len} outside [1, {tokens}]")
        out = torch.empty((tokens, width), dtype=projected.dtype, device=self.device)
        elems = int(self._core.velox_gated_scan_scratch_elems(slots.shape[0], int(max_q_len), int(width)))
        scratch = torch.empty(elems, dtype=torch.float32, device=self.device) if elems else None
        self._launched(self._core.velox_gated_scan(_ptr(projected), _code(projected.dtype), int(width), _ptr(gate_bias), _ptr(input_bias), float(shift), _ptr(state),
                                                   _ptr(slots), _ptr(cu_q), _ptr(out), _ptr(scratch), slots.shape[0], int(max_q_len), self._stream()), "gated_scan")
        return out

    def linear_scan_supports(self, dim: int, vdim: int) -> None:
        """Raises if the scan kernel cannot hold a column of a ``dim x vdim`` state in one wave."""
        if self._core.velox_linear_scan_lanes(int(dim)) > 64:
            raise KernelError(f"linear_scan: key heads of {dim} channels are beyond the kernel (512 at most)")

    _SCAN_RULES = {"additive": 0, "delta": 1, "removal": 2}

    def linear_scan(self, qk, v_source, v_at, decay, beta, state, slots, cu_q, max_q_len, heads, kv_heads, dim, vdim, rule):
        """Per sequence and head, token by token from ``state[slot, head]`` ([dim, vdim] float32), which is written back:
        ``S <- g S`` (rows); ``u = beta (v - S^T k)`` (rule ``"delta"``) or ``u = v`` (``"additive"``); ``S <- S + k u^T``; ``o = S^T q``.
        Rule ``"removal"``: ``qk`` holds a third vector ``b`` per head and token, and ``S <- g S - b (k^T S) + k (beta v)^T`` with both
        terms on the old state.  ``decay`` is [T, heads] or [T, heads * dim].  Returns float32 [T, heads * vdim]."""
        if rule not in self._SCAN_RULES:
            raise KernelError(f"linear_scan: rule {rule!r} is not implemented ({', '.join(self._SCAN_RULES)})")
        delta = rule != "additive"
        tokens = qk.shape[0]
        self._check("qk", qk, torch.float32, (tokens, kv_heads, 3 if rule == "removal" else 2, dim), align=16)
        self._check("v_source", v_source)
        if v_source.dim() != 2 or v_source.shape[0] != tokens or v_at + heads * vdim > v_source.shape[1]:
            raise KernelError("linear_scan: the values do not lie within their source")
        self._check("decay", decay, torch.float32, align=16)
        if tuple(decay.shape) not in ((tokens, heads), (tokens, heads * dim)):
            raise KernelError(f"linear_scan: decay must be [T, heads] or [T, heads * dim], got {tuple(decay.shape)}")
        per_channel = tuple(decay.shape) == (tokens, heads * dim)
        if delta:
            if beta is None:
                raise KernelError(f"linear_scan: the {rule} rule needs beta")
            self._check("beta", beta, torch.float32, (tokens, heads))
        self._check("state", state, torch.float32)
        if state.dim() != 4 or tuple(state.shape[1:]) != (heads, dim, vdim):
            raise KernelError(f"linear_scan: the state must be [slots, {heads}, {dim}, {vdim}], got {tuple(state.shape)}")
        self._check("slots", slots, torch.int32)
        self._check("cu_q", cu_q, torch.int32, (slots.shape[0] + 1,))
        self.linear_scan_supports(dim, vdim)
        out = torch.empty((tokens, heads * vdim), dtype=torch.float32, device=self.device)
        status = self._core.velox_linear_scan(_ptr(qk), _ptr(v_source), _code(v_source.dtype), v_source.shape[1], int(v_at), _ptr(decay), int(per_channel),
                                              _ptr(beta) if delta else _P(0), _ptr(state), _ptr(slots), _ptr(cu_q), _ptr(out), slots.shape[0], int(max_q_len), int(heads),
                                              int(kv_heads), int(dim), int(vdim), self._SCAN_RULES[rule], self._stream())
        self._launched(status, "linear_scan")
        return out

    def gated_head_norm(self, read, weight, eps, gate_source, gate_at, gate_kind, heads, vdim, out_dtype):
        """``read`` float32 [T, heads * vdim]: every head divided by its root mean square (``eps`` inside the root), times
        ``weight`` ([vdim], shared by the heads, or [heads * vdim]), times ``silu(z)`` or ``sigmoid(z)`` of the gate's columns;
        [T, heads * vdim] in ``out_dtype``."""
        tokens = read.shape[0]
        self._check("read", read, torch.float32, (tokens, heads * vdim))
        self._check("weight", weight, torch.float32, (weight.numel(),))
        if weight.numel() not in (vdim, heads * vdim):
            raise KernelError(f"gated_head_norm: the weight has {vdim} or {heads * vdim} entries, got {weight.numel()}")
        self._check("gate_source", gate_source)
        if gate_source.dim() != 2 or gate_source.shape[0] != tokens or gate_at + heads * vdim > gate_source.shape[1] or gate_kind not in ("silu", "sigmoid"):
            raise KernelError("gated_head_norm: the gate's columns do not lie within its source, or its kind is unknown")
        out = torch.empty((tokens, heads * vdim), dtype=out_dtype, device=self.device)
        status = self._core.velox_gated_head_norm(_ptr(read), _ptr(weight), float(eps), _ptr(gate_source), _code(gate_source.dtype), gate_source.shape[1],
                                                  int(gate_at), 0 if gate_kind == "silu" else 1, _ptr(out), _code(out_dtype), tokens, int(heads), int(vdim),
                                                  int(weight.numel() != vdim), self._stream())
        self._launched(status, "gated_head_norm")
        return out

    def state_space_supports(self, size: int, vdim: int) -> None:
        """Raises if the kernels cannot hold a head's state of ``size x vdim`` numbers."""
        if size > self._core.velox_state_space_max_state():
            raise KernelError(f"state_space_scan: {size} entries per column of a head's state are beyond the kernel ({self._core.velox_state_space_max_state()} at most)")

    STATE_SPACE_CHUNK_TOKENS = 32  # portions at least this long are worked in chunks

    def state_space_scan(self, xbc, step_source, step_at, dt_bias, rate, skip, state, slots, cu_q, max_q_len, heads, groups, size, vdim,
                         chunked: Optional[bool] = None):
        """Rows of ``xbc`` hold x (``heads * vdim``), B and C (``groups * size`` each), a token's dt stands in ``step_source`` from column ``step_at``
        on.  With ``d = softplus(dt + dt_bias)``, per sequence and head from ``state[slot, head]`` ([size, vdim] float32), which is written
        back: ``S <- exp(-rate d) S + d B x^T``; ``y = S^T C + skip x``.  Float32 [T, heads * vdim].  Steps with a long portion are worked
        in chunks of 64 tokens on the matrix cores, others token by token; ``chunked`` decides it for a test."""
        self._check("xbc", xbc)
        if xbc.dim() != 2 or groups < 1 or heads % groups != 0 or xbc.shape[1] != heads * vdim + 2 * groups * size:
            raise KernelError(f"state_space_scan: rows of {heads} * {vdim} + 2 * {groups} * {size} columns expected, got {tuple(xbc.shape)}")
        tokens = xbc.shape[0]
        self._check("step_source", step_source, xbc.dtype)
        if step_source.dim() != 2 or step_source.shape[0] != tokens or step_at < 0 or step_at + heads > step_source.shape[1]:
            raise KernelError("state_space_scan: the step sizes do not lie within their source")
        for name, t in (("dt_bias", dt_bias), ("rate", rate), ("skip", skip)):
            self._check(name, t, torch.float32, (heads,))
        self._check("state", state, torch.float32)
        if state.dim() != 4 or tuple(state.shape[1:]) != (heads, size, vdim):
            raise KernelError(f"state_space_scan: the state must be [slots, {heads}, {size}, {vdim}], got {tuple(state.shape)}")
        self._check("slots", slots, torch.int32)
        self._check("cu_q", cu_q, torch.int32, (slots.shape[0] + 1,))
        if not 1 <= max_q_len <= tokens:
            raise KernelError(f"state_space_scan: max_q_len={max_q_len} outside [1, {tokens}]")
        self.state_space_supports(size, vdim)
        out = torch.empty((tokens, heads * vdim), dtype=torch.float32, device=self.device)
        scratch = None
        if chunked or (chunked is None and max_q_len >= self.STATE_SPACE_CHUNK_TOKENS):
            elems = int(self._core.velox_state_space_scratch_elems(tokens, slots.shape[0], int(heads), int(size), int(vdim)))
            scratch = torch.empty(elems, dtype=torch.float32, device=self.device)
        self._launched(self._core.velox_state_space_scan(_ptr(xbc), _code(xbc.dtype), xbc.shape[1], _ptr(step_source), step_source.shape[1], int(step_at),
                                                         _ptr(dt_bias), _ptr(rate), _ptr(skip), _ptr(state), _ptr(slots), _ptr(cu_q), _ptr(out), _ptr(scratch),
                                                         tokens, slots.shape[0], int(max_q_len), int(heads), int(groups), int(size), int(vdim), self._stream()),
                       "state_space_scan")
        return out

    def gated_group_norm(self, read, gate_source, gate_at, weight, eps, groups, out_dtype):
        """``y = read * silu(z)`` with ``z`` the columns of ``gate_source`` from ``gate_at`` on; each of ``groups`` equal parts of a row divided by its
        root mean square (``eps`` inside the root), times ``weight``; [T, width] in ``out_dtype``."""
        self._check("read", read, torch.float32)
        if read.dim() != 2 or groups < 1 or read.shape[1] % groups != 0:
            raise KernelError(f"gated_group_norm: rows {tuple(read.shape)} do not fall into {groups} equal parts")
        tokens, width = read.shape
        self._check("weight", weight, torch.float32, (width,))
        self._check("gate_source", gate_source)
        if gate_source.dim() != 2 or gate_source.shape[0] != tokens or gate_at < 0 or gate_at + width > gate_source.shape[1]:
            raise KernelError("gated_group_norm: the gate's columns do not lie within its source")
        out = torch.empty((tokens, width), dtype=out_dtype, device=self.device)
        self._launched(self._core.velox_gated_group_norm(_ptr(read), _ptr(gate_source), _code(gate_source.dtype), gate_source.shape[1], int(gate_at), _ptr(weight),
                                                         float(eps), _ptr(out), _code(out_dtype), tokens, width, int(groups), self._stream()), "gated_group_norm")
        return out

    # -- rotary + cache write ---------------------------------------------------------------------
    def rope_kv_write(self, qkv, num_heads, num_kv_heads, head_dim, positions, cos, sin, slot_mapping, k_cache, v_cache, block_size, write_kv=True, bias=None):
        tokens = qkv.shape[0]
        width = (num_heads + 2 * num_kv_heads) * head_dim
        self._check("qkv", qkv, None, (tokens, width), align=16)
        self._check("positions", positions, torch.int32, (tokens,))
        self._check("slot_mapping", slot_mapping, torch.int32, (tokens,))
        if bias is not None:
            self._check("bias", bias, torch.float32, (width,))
        half = 0
        if cos is not None:
            self._check("cos", cos, torch.float32)
            self._check("sin", sin, torch.float32, tuple(cos.shape))
            half = cos.shape[1]
            if 2 * half > head_dim:
                raise KernelError(f"rotary span {2 * half} exceeds head_dim {head_dim}")
        pages = k_cache.shape[0]
        self._check("k_cache", k_cache, qkv.dtype, (pages, num_kv_heads, block_size, head_dim), align=16)
        self._check("v_cache", v_cache, qkv.dtype, (pages, num_kv_heads, head_dim, block_size), align=16)
        # positions index the tables and slots index the cache: both are built by the batch builder from
        # block tables the cache manager handed out, bounded by max_model_len and the pool size
        status = self._core.velox_rope_kv_write(
            _ptr(qkv), _ptr(bias), _ptr(positions), _ptr(cos), _ptr(sin), half, _ptr(slot_mapping), _ptr(k_cache), _ptr(v_cache),
            tokens, num_heads, num_kv_heads, head_dim, block_size, 1 if write_kv else 0, _code(qkv.dtype), self._stream())
        self._launched(status, "rope_kv_write")

    def rope_kv_write_partial(self, partial, num_heads, num_kv_heads, head_dim, positions, cos, sin, slot_mapping, k_cache, v_cache, block_size,
                              write_kv=True, bias=None) -> torch.Tensor:
        """``rope_kv_write`` on rows that come as float32 partial sums ``[S, M, (heads + 2 kv_heads) * head_dim]`` (bfloat16
        caches): returns bfloat16 ``[M, width]`` whose query columns hold the rotated queries (the others are not written)."""
        if partial.dim() != 3:
            raise KernelError("rope_kv_write_partial: partial sums are [S, M, width]")
        parts, tokens, width = partial.shape
        if width != (num_heads + 2 * num_kv_heads) * head_dim or head_dim % 16 != 0:
            raise KernelError(f"rope_kv_write_partial: rows of {width} elements do not hold {num_heads} + 2 x {num_kv_heads} heads of {head_dim}")
        self._check("partial", partial, torch.float32, (parts, tokens, width), align=16)
        self._check("positions", positions, torch.int32, (tokens,))
        self._check("slot_mapping", slot_mapping, torch.int32, (tokens,))
        if bias is not None:
            self._check("bias", bias, torch.float32, (width,), align=16)
        half = 0
        if cos is not None:
            self._check("cos", cos, torch.float32, align=16)
            self._check("sin", sin, torch.float32, tuple(cos.shape), align=16)
            half = cos.shape[1]
            if 2 * half != head_dim:
                raise KernelError("rope_kv_write_partial: the rotation has to span the whole head")
        pages = k_cache.shape[0]
        self._check("k_cache", k_cache, torch.bfloat16, (pages, num_kv_heads, block_size, head_dim), align=16)
        self._check("v_cache", v_cache, torch.bfloat16, (pages, num_kv_heads, head_dim, block_size), align=16)
        out = torch.empty((tokens, width), dtype=torch.bfloat16, device=self.device)
        status = self._core.velox_rope_kv_write_partial_bf16(
            _ptr(out), _ptr(partial), parts, _ptr(bias), _ptr(positions), _ptr(cos), _ptr(sin), half, _ptr(slot_mapping), _ptr(k_cache), _ptr(v_cache),
            tokens, num_heads, num_kv_heads, head_dim, block_size, 1 if write_kv else 0, self._stream())
        self._launched(status, "rope_kv_write_partial")
        return out

    def qkv_rope_write(self, x, weight, bias, num_heads, num_kv_heads, head_dim, positions, cos, sin, slot_mapping, k_cache, v_cache,
                       block_size, write_kv=True, waves: Optional[int] = None, fused: Optional[bool] = None) -> torch.Tensor:
        """Projects ``x`` with ``weight = [Wq; Wk; Wv]``, adds ``bias``, rotates queries and keys and writes keys and values
        into the cache.  Returns a tensor whose first ``num_heads * head_dim`` columns are the rotated queries (it may be
        wider).  Decode-sized bfloat16 batches run as one kernel when ``weight`` is what ``prepare_weight(w, rotary_heads=...)``
        returned; everything else is the product followed by ``rope_kv_write``."""
        operand = weight
        weight, prepared = _weight_of(weight)
        deferred = x if isinstance(x, DeferredNorm) else None
        if deferred is not None:
            x = deferred.x
        m, k = x.shape
        packed = prepared.copy("rotary") if prepared is not None else None
        can_fuse = (self.use_skinny_gemm and packed is not None and write_kv and x.dtype == torch.bfloat16 and m <= 16 and k % 64 == 0
                    and cos is not None and 2 * cos.shape[1] == head_dim and head_dim % 32 == 0 and k_cache.dtype == torch.bfloat16)
        if fused is None:
            fused = can_fuse
        elif fused and not can_fuse:
            raise KernelError("qkv_rope_write: this call cannot run fused")
        if not fused:
            n = weight.shape[0]
            if (deferred is None and self.use_skinny_gemm and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16 and k_cache.dtype == torch.bfloat16
                    and 16 < m <= 64 and k % 64 == 0 and n <= 8192 and n == (num_heads + 2 * num_kv_heads) * head_dim and head_dim % 16 == 0
                    and (cos is None or 2 * cos.shape[1] == head_dim)):
                # 17 .. 64 rows: the split-K kernel streams the weight faster than the library's choice (measured on
                # MI355X: 15 us against 21 for 4608 x 3584 at 64 rows), and the rotation adds its partial sums
                partial = self.skinny_gemm_splitk(x, weight, packed=prepared.copy(1) if prepared is not None else None)
                return self.rope_kv_write_partial(partial, num_heads, num_kv_heads, head_dim, positions, cos, sin, slot_mapping, k_cache, v_cache,
                                                  block_size, write_kv=write_kv, bias=bias)
            qkv = self.linear(deferred if deferred is not None else x, operand, None, x.dtype)
            self.rope_kv_write(qkv, num_heads, num_kv_heads, head_dim, positions, cos, sin, slot_mapping, k_cache, v_cache, block_size,
                               write_kv=write_kv, bias=bias)
            return qkv
        width = (num_heads + 2 * num_kv_heads) * head_dim
        self._check("x", x, torch.bfloat16, align=16)
        if weight.shape != (width, k):
            raise KernelError(f"qkv_rope_write: weight {tuple(weight.shape)} is not [{width}, {k}]")
        self._check("positions", positions, torch.int32, (m,))
        self._check("slot_mapping", slot_mapping, torch.int32, (m,))
        if bias is not None:
            self._check("bias", bias, torch.float32, (width,), align=16)
        self._check("cos", cos, torch.float32, align=16)
        self._check("sin", sin, torch.float32, tuple(cos.shape), align=16)
        pages = k_cache.shape[0]
        self._check("k_cache", k_cache, torch.bfloat16, (pages, num_kv_heads, block_size, head_dim), align=16)
        self._check("v_cache", v_cache, torch.bfloat16, (pages, num_kv_heads, head_dim, block_size), align=16)
        q = torch.empty((m, num_heads * head_dim), dtype=torch.bfloat16, device=self.device)
        x_packed = self._packed_rows_of(x, k)
        status = self._core.velox_skinny_qkv_rotary_bf16(
            _ptr(x if x_packed is None else x_packed), _ptr(packed), _ptr(bias), _ptr(positions), _ptr(cos), _ptr(sin), _ptr(slot_mapping), _ptr(q), _ptr(k_cache),
            _ptr(v_cache), m, k, num_heads, num_kv_heads, head_dim, block_size, int(waves or 8), *self._scale_args(deferred),
            int(x_packed is not None), self._stream())
        self._launched(status, "skinny_qkv_rotary")
        return q

    # -- attention over a cached latent -----------------------------------------------------------
    def latent_rotate_write(self, projected, num_heads, dim, rot_dim, kv_rank, cached_dim, down_offset, positions, cos, sin, interleaved,
                            norm_weight, eps, slot_mapping, k_cache, v_cache, block_size, q_latent=None):
        """Rows of ``projected`` hold ``num_heads`` queries of ``dim`` plain and ``rot_dim`` rotated channels and, at
        ``down_offset`` (-1: none, nothing is written to the cache), a latent of ``kv_rank`` and a shared key part of
        ``rot_dim`` channels.  Returns the queries the attention kernels read, ``[T, num_heads * cached_dim]``: of every head
        the channels from ``kv_rank`` on are written here (the rotated part, then zeros), the first ``kv_rank`` are left
        for ``head_linear``.  The normed latent and the rotated shared part go into the cache.  ``num_heads`` = 0: no
        queries.  ``q_latent = (offset, rank, weight)``: those columns of every row are RMS-normed with the weight as well;
        then ``(queries, normed [T, rank])`` comes back."""
        if projected.dim() != 2:
            raise KernelError("latent_rotate_write: rows are [T, width]")
        tokens, width = projected.shape
        self._check("projected", projected, None, (tokens, width))
        self._check("positions", positions, torch.int32, (tokens,))
        half = 0
        if cos is not None:
            self._check("cos", cos, torch.float32)
            self._check("sin", sin, torch.float32, tuple(cos.shape))
            half = cos.shape[1]
        if (num_heads < 0 or num_heads * (dim + rot_dim) > width or 2 * half > rot_dim or cached_dim < kv_rank + rot_dim
                or (down_offset >= 0 and down_offset + kv_rank + rot_dim > width)):
            raise KernelError(f"latent_rotate_write: rows of {width} do not hold {num_heads} x ({dim} + {rot_dim}) queries and a latent of {kv_rank} + {rot_dim} at {down_offset}")
        if down_offset >= 0:
            self._check("slot_mapping", slot_mapping, torch.int32, (tokens,))
            self._check("norm_weight", norm_weight, torch.float32, (kv_rank,))
            pages = k_cache.shape[0]
            self._check("k_cache", k_cache, projected.dtype, (pages, 1, block_size, cached_dim))
            self._check("v_cache", v_cache, projected.dtype, (pages, 1, cached_dim, block_size))
        normed, norm2 = None, (0, 0, None)
        if q_latent is not None:
            norm2 = (int(q_latent[0]), int(q_latent[1]), q_latent[2])
            self._check("q_latent weight", norm2[2], torch.float32, (norm2[1],))
            if norm2[0] < 0 or norm2[1] < 1 or norm2[0] + norm2[1] > width:
                raise KernelError(f"latent_rotate_write: columns {norm2[0]} .. {norm2[0] + norm2[1]} lie outside rows of {width}")
            normed = torch.empty((tokens, norm2[1]), dtype=projected.dtype, device=self.device)
        queries = torch.empty((tokens, num_heads * cached_dim), dtype=projected.dtype, device=self.device)
        status = self._core.velox_latent_rotate_write(
            _ptr(projected), width, _ptr(queries), tokens, num_heads, dim, rot_dim, kv_rank, cached_dim, int(down_offset), _ptr(positions), _ptr(cos), _ptr(sin),
            half, int(bool(interleaved)), _ptr(norm_weight) if down_offset >= 0 else _P(0), float(eps), _ptr(slot_mapping) if down_offset >= 0 else _P(0),
            _ptr(k_cache) if down_offset >= 0 else _P(0), _ptr(v_cache) if down_offset >= 0 else _P(0), int(block_size), _code(projected.dtype),
            norm2[0], norm2[1], _ptr(norm2[2]), _ptr(normed), self._stream())
        self._launched(status, "latent_rotate_write")
        return queries if q_latent is None else (queries, normed)

    def latent_write(self, projected, rot_dim, kv_rank, cached_dim, down_offset, positions, cos, sin, interleaved, norm_weight, eps, slot_mapping,
                     k_cache, v_cache, block_size, q_latent=None):
        """The cache write of ``latent_rotate_write`` without any queries (the same kernel): norm of the latent at
        ``down_offset``, rotation of the shared key part, both into the pages.  ``q_latent = (offset, rank, weight)``: those
        columns come back RMS-normed with the weight, ``[T, rank]`` (the queries' own latent, on its way to its second product)."""
        result = self.latent_rotate_write(projected, 0, 0, rot_dim, kv_rank, cached_dim, down_offset, positions, cos, sin, interleaved, norm_weight, eps,
                                          slot_mapping, k_cache, v_cache, block_size, q_latent=q_latent)
        return None if q_latent is None else result[1]

    def head_linear(self, x, x_head_stride, x_offset, maps, out, out_head_stride, out_offset, gate=None, gate_offset=0, gate_per_head=False) -> torch.Tensor:
        """``out[t, g * out_head_stride + out_offset + j] = sum_k x[t, g * x_head_stride + x_offset + k] * maps[g, j, k]``, times
        ``sigmoid(gate[t, gate_offset + g * n + j])`` when ``gate`` is given (``gate_per_head``: ``sigmoid(gate[t, gate_offset + g])``,
        one number for all outputs of a head): one small product per head, the heads at fixed
        strides inside the rows of ``x`` and ``out`` (written in place, other columns untouched)."""
        if x.dim() != 2 or out.dim() != 2 or maps.dim() != 3 or x.shape[0] != out.shape[0]:
            raise KernelError("head_linear: x and out are [T, width], maps is [groups, n, k]")
        groups, n, k = maps.shape
        self._check("x", x)
        self._check("maps", maps, x.dtype)
        self._check("out", out, x.dtype)
        if (min(x_head_stride, x_offset, out_head_stride, out_offset) < 0 or (groups - 1) * x_head_stride + x_offset + k > x.shape[1]
                or (groups - 1) * out_head_stride + out_offset + n > out.shape[1]):
            raise KernelError("head_linear: a head's channels lie outside the rows")
        gate_width = 0
        if gate is not None:
            self._check("gate", gate, x.dtype)
            gate_width = gate.shape[1]
            if gate.dim() != 2 or gate.shape[0] != x.shape[0] or gate_offset < 0 or gate_offset + (groups if gate_per_head else groups * n) > gate_width:
                raise KernelError("head_linear: the gate's columns lie outside its rows")
        status = self._core.velox_head_linear(_ptr(x), x.shape[1], int(x_head_stride), int(x_offset), _ptr(maps), _ptr(out), out.shape[1], int(out_head_stride),
                                              int(out_offset), _ptr(gate), gate_width, int(gate_offset), x.shape[0], groups, n, k, _code(x.dtype), int(bool(gate_per_head)), self._stream())
        self._launched(status, "head_linear")
        return out

    # -- routed experts ---------------------------------------------------------------------------
    def route_top(self, logits: torch.Tensor, top: int, score: str = "sigmoid", renormalize: bool = False, correction: Optional[torch.Tensor] = None,
                  groups: Optional[Tuple[int, int]] = None, norm_floor: float = 0.0):
        """float32 ``logits`` [T, E] -> (int32 choices [T, top], float32 weights [T, top]): the ``top`` largest scores
        (``sigmoid`` or ``softmax`` over all experts), ties to the lower index, divided by their sum when ``renormalize``.
        ``correction`` (float32 [E]) is added to the scores for the choice only: the weights are the scores without it.
        ``groups = (count, keep)``: the experts form ``count`` equal groups of neighbours (64 at most), a group's score is the sum of
        its two largest choice scores, and only experts of the ``keep`` best groups can be chosen.  ``norm_floor`` is added to
        the sum that renormalised weights are divided by."""
        self._check("logits", logits, torch.float32)
        count, keep = (int(groups[0]), int(groups[1])) if groups else (0, 0)
        if groups and (not 1 <= count <= 64 or logits.shape[-1] % count or not 1 <= keep <= count or keep * (logits.shape[-1] // count) < top):
            raise KernelError(f"route_top: groups={groups} do not fit {logits.shape[-1]} experts and top={top}")
        if correction is not None:
            self._check("correction", correction, torch.float32, (logits.shape[-1],))
        if logits.dim() != 2 or not 1 <= top <= logits.shape[1] or score not in ("sigmoid", "softmax"):
            raise KernelError(f"route_top: logits {tuple(logits.shape)}, top={top}, score={score!r}")
        tokens, experts = logits.shape
        choice = torch.empty((tokens, top), dtype=torch.int32, device=self.device)
        weight = torch.empty((tokens, top), dtype=torch.float32, device=self.device)
        self._launched(self._core.velox_route_top(_ptr(logits), _ptr(choice), _ptr(weight), tokens, experts, int(top), int(score == "softmax"),
                                                  int(bool(renormalize)), _ptr(correction), count, keep, float(norm_floor), self._stream()), "route_top")
        return choice, weight

    def routed_plan_elems(self, max_num_tokens: int, top: int, experts: int) -> int:
        """int32 elements of the plan of a step of at most ``max_num_tokens`` tokens."""
        return int(self._core.velox_routed_plan_elems(int(max_num_tokens) * int(top), int(experts)))

    def routed_experts(self, x, choice, weight, gate_up_weight, down_weight, num_experts: int, scale_input: bool, shared, out_dtype, workspace=None,
                       unit: Tuple[float, float, float] = (1.0, float("inf"), 0.0), identity_experts: int = 0, output_norm=None, ungated: Optional[str] = None):
        """``sum_k unit_{choice[t, k]}(weight[t, k] x[t])`` (or the weight on the unit's output), plus ``shared``: the pairs
        are sorted by expert on the device, two grouped products run every expert on its rows, and each token's results
        are added in the order of its choices.  ``gate_up_weight`` [E * 2F, H] (per expert gate rows, then up rows),
        ``down_weight`` [E * H, F].  ``unit = (alpha, limit, shift)``: the middle of a unit is ``g sigmoid(alpha g) (u +
        shift)`` with ``g = min(gate, limit)``, ``u = clamp(up, -limit, limit)``.  ``identity_experts``: choices from
        ``num_experts`` on are experts without tensors whose result is ``weight[t, k] x[t]``; the plan leaves them out and
        the last kernel adds them in their turn.  ``output_norm`` (an ``OutputNormSink``): the last kernel norms the sum in
        float32 and adds it to the sink's residual; what comes back is then a ``ResidualCopy`` of the updated residual, or, when
        the sink names the norm that follows, a ``ReadyInput`` with that norm's result.
        ``ungated`` (``"relu2"``): the units have no gate branch, ``W_down act(W_up x)``; ``gate_up_weight`` is then [E * F, H]."""
        alpha, limit, shift = (float(v) for v in unit)
        if ungated is not None and ungated not in self._ACTIVATION_CODES:
            raise KernelError(f"routed_experts: activation {ungated!r} is not implemented")
        act_code = self._ACTIVATION_CODES[ungated] if ungated is not None else 0
        branches = 1 if ungated is not None else 2
        if not limit > 0 or identity_experts < 0:
            raise KernelError(f"routed_experts: unit={unit}, identity_experts={identity_experts}")
        tokens, hidden = x.shape
        top = choice.shape[1]
        pairs = tokens * top
        inter = gate_up_weight.shape[0] // (branches * num_experts)
        self._check("x", x)
        self._check("choice", choice, torch.int32, (tokens, top))
        self._check("weight", weight, torch.float32, (tokens, top))
        self._check("gate_up_weight", gate_up_weight, x.dtype, (num_experts * branches * inter, hidden))
        self._check("down_weight", down_weight, x.dtype, (num_experts * hidden, inter))
        if shared is not None:
            self._check("shared", shared, out_dtype, (tokens, hidden))
        if out_dtype != x.dtype:
            raise KernelError("routed_experts: the result has the activations' dtype")
        elems = self.routed_plan_elems(tokens, top, num_experts)
        if workspace is not None:
            plan = workspace.get("routed_plan", elems).view(torch.int32)
        else:
            plan = torch.empty(elems, dtype=torch.int32, device=self.device)
        on_matrix_cores = x.dtype == torch.bfloat16 and hidden % 8 == 0 and inter % 8 == 0 and self.use_grouped_mfma
        # tiles of 128 rows for the matrix cores when the experts have that many rows on average (W is then read half as often)
        tile_rows = 128 if on_matrix_cores and pairs >= 128 * num_experts and branches * inter > 128 and hidden > 128 else 64
        # few pairs: the plan's kernel also copies the rows into its order, and the step runs one kernel less
        ordered = torch.empty((pairs, hidden), dtype=x.dtype, device=self.device) if on_matrix_cores else None
        copied_by_plan = on_matrix_cores and pairs <= self.FEW_PAIRS
        self._launched(self._core.velox_routed_plan(_ptr(choice), pairs, num_experts, _ptr(plan), tile_rows, _ptr(x) if copied_by_plan else _P(0),
                                                    _ptr(ordered) if copied_by_plan else _P(0), _ptr(weight), top, hidden, int(bool(scale_input)), self._stream()),
                       "routed_plan")
        act = torch.empty((pairs, inter), dtype=x.dtype, device=self.device)
        y = torch.empty((pairs, hidden), dtype=torch.float32, device=self.device)
        if on_matrix_cores:
            # bfloat16 rows of whole 16-byte pieces: sorted copies of the rows, then both products on the matrix cores
            self._launched(self._core.velox_routed_products_bf16(_P(0) if copied_by_plan else _ptr(x), _ptr(gate_up_weight), _ptr(down_weight), _ptr(ordered), _ptr(act), _ptr(y), _ptr(plan),
                                                                 _ptr(weight), pairs, num_experts, top, inter, hidden, int(bool(scale_input)), tile_rows,
                                                                 alpha, limit, shift, act_code, self._stream()), "routed_products")
            # (a weight on the output is applied by the last kernel: the second product is the same kernel either way)
            return self._routed_combine(y, plan, shared, tokens, top, num_experts, hidden, out_dtype, x if identity_experts else None, weight,
                                        scale_rows=not scale_input, output_norm=output_norm)
        self._launched(self._core.velox_grouped_glu(_ptr(x), _ptr(gate_up_weight), _ptr(act), _ptr(plan), _ptr(weight), pairs, num_experts, top, inter, hidden,
                                                    int(bool(scale_input)), _code(x.dtype), alpha, limit, shift, act_code, self._stream()), "grouped_glu")
        self._launched(self._core.velox_grouped_down(_ptr(act), _ptr(down_weight), _ptr(y), _ptr(plan), _ptr(weight), pairs, num_experts, top, hidden, inter,
                                                     int(not scale_input), _code(x.dtype), self._stream()), "grouped_down")
        return self._routed_combine(y, plan, shared, tokens, top, num_experts, hidden, out_dtype, x if identity_experts else None, weight,
                                    output_norm=output_norm)

    def _routed_combine(self, y, plan, shared, tokens, top, num_experts, hidden, out_dtype, identity_input=None, weight=None, scale_rows=False,
                        output_norm=None):
        if output_norm is not None:
            self._check("residual", output_norm.residual, torch.float32, (tokens, hidden))
            self._check("norm weight", output_norm.weight, torch.float32, (hidden,))
            following = output_norm.following.deferred_form() if output_norm.following is not None else None
            copy = torch.empty((tokens, hidden), dtype=out_dtype, device=self.device) if out_dtype != torch.float32 or following is not None else None
            if following is not None:
                self._check("next norm weight", following[0], torch.float32, (hidden,))
            status = self._core.velox_routed_combine_norm(_ptr(y), _ptr(plan), _ptr(shared), tokens, top, num_experts, hidden, _code(out_dtype),
                                                          _ptr(identity_input), _ptr(weight), int(bool(scale_rows)), _ptr(output_norm.residual),
                                                          _ptr(output_norm.weight), float(output_norm.eps), float(output_norm.mult), _ptr(copy),
                                                          _ptr(following[0]) if following is not None else _P(0), float(following[1]) if following is not None else 0.0,
                                                          self._stream())
            if status == 0 and following is not None:
                return ReadyInput(copy, output_norm.following)
            if status == 0:
                return ResidualCopy(output_norm.residual if copy is None else copy)
            if status != -1:
                self._launched(status, "routed_combine_norm")
            # (a row too long for the fused kernel's registers: the two kernels one after the other)
            out = self._routed_combine(y, plan, shared, tokens, top, num_experts, hidden, out_dtype, identity_input, weight, scale_rows)
            if following is not None:
                self.norm_add(output_norm.residual, out, output_norm.weight, output_norm.eps, output_norm.mult, torch.float32)
                return ReadyInput(self.add_rmsnorm(output_norm.residual, None, following[0], following[1], out_dtype), output_norm.following)
            return ResidualCopy(self.norm_add(output_norm.residual, out, output_norm.weight, output_norm.eps, output_norm.mult, out_dtype))
        out = torch.empty((tokens, hidden), dtype=out_dtype, device=self.device)
        self._launched(self._core.velox_routed_combine(_ptr(y), _ptr(plan), _ptr(shared), _ptr(out), tokens, top, num_experts, hidden, _code(out_dtype),
                                                       _ptr(identity_input), _ptr(weight), int(bool(scale_rows)), self._stream()), "routed_combine")
        return out

    # -- attention ------------------------------------------------------------------------------
    def choose_splits(self, num_seqs: int, num_kv_heads: int, row_tiles: int, max_kv_len: int, all_decode: bool) -> int:
        """Splits of the key range for an all-decode step (reference ``src/decode_attention.py:237-252``: enough
        workgroups to fill the GPU).  Measured on MI355X the streaming kernel runs best with one workgroup per compute
        unit: more of them add partial results to write and merge and gain nothing.  At least 64 keys per split."""
        if not all_decode:
            return 1
        base = num_seqs * num_kv_heads * row_tiles
        splits = max(1, min(self.num_cus // max(base, 1), 32, max_kv_len // 64))
        # Splits and their merge cost about 3 us; a workgroup streams 64 keys in about 0.7 us.  Behind few keys one
        # workgroup per sequence and KV head is quicker (measured on MI355X, one sequence of 256 keys: 7.2 us against 9.4
        # with 4 splits; 512 keys: 9.8 us against 8.0 with 8).
        if max_kv_len * (splits - 1) < 448 * splits:
            splits = 1
        return splits

    def choose_portion_splits(self, num_tokens: int, group: int, num_kv_heads: int, max_kv_len: int) -> int:
        """Splits of the key range for portions of prompts.  Few tokens behind many keys are few workgroups that each walk
        all the keys: with the keys split the step fills the GPU with the large workgroups (measured on MI355X, 512
        tokens behind 8,192 keys: 157 us in one pass, 104 us in four splits and their merge; behind 32,768: 611 and 331).
        At least 1,024 keys per split, and none below 4,096 keys, where one pass is as quick."""
        if max_kv_len < 4096:
            return 1
        blocks = max(1, num_tokens * group // 128 * num_kv_heads)  # workgroups of 128 rows, as the launch counts them
        if blocks >= self.num_cus:
            return 1
        return max(1, min(-(-self.num_cus // blocks), max_kv_len // 1024, 16))

    def attention_scratch_elems(self, num_heads: int, num_kv_heads: int, head_dim: int, max_num_tokens: int, max_num_seqs: int, max_model_len: int) -> Tuple[int, int]:
        """The most float32 elements ``paged_attention`` asks its workspace for (partial outputs, partial log-sums) in
        any step of at most ``max_num_tokens`` tokens and ``max_num_seqs`` sequences behind at most ``max_model_len`` keys,
        with the splits that ``choose_splits`` and ``choose_portion_splits`` pick.  The bound counts TOKENS, not sequences:
        the sequence on the null page that pads a step up to a timed number of rows (one more than ``max_num_seqs``) brings
        tokens within ``max_num_tokens`` like any other and is covered."""
        if head_dim > self.MAX_TILED_HEAD_DIM:
            return 0, 0  # (the plain kernel splits nothing)
        group = num_heads // num_kv_heads
        rows = 0  # splits x the rows the partial results are counted by
        for count in range(1, max_num_seqs + 1):  # single tokens, alone or before portions
            rows = max(rows, count * self.choose_splits(count, num_kv_heads, 1, max_model_len, True))
        for portion in range(1, max_num_tokens + 1):  # portions of prompts, behind up to max_num_seqs - 1 single tokens
            whole = min(max_num_tokens, portion + max_num_seqs - 1)
            rows = max(rows, whole * self.choose_portion_splits(portion, group, num_kv_heads, max_model_len))
        return rows * num_heads * head_dim, rows * num_heads

    def paged_attention(self, qkv, num_heads, num_kv_heads, head_dim, k_cache, v_cache, block_size, block_tables, cu_q, kv_lens,
                        max_q_len, max_kv_len, scale, window, all_decode, workspace, splits: Optional[int] = None, decode_prefix: int = 0,
                        portions_max_kv_len: Optional[int] = None, distance_bias: Optional[torch.Tensor] = None, sinks: Optional[torch.Tensor] = None,
                        keep_first: int = 0, softcap: Optional[float] = None, gate: Optional[Tuple[torch.Tensor, int, int]] = None):
        """Attention of every token of the step over its sequence's keys in the cache.  ``decode_prefix``: how many of the
        first sequences bring exactly one token (the engine puts decoded tokens before portions of prompts).  In a mixed
        step those run through the streaming kernel with their keys split over workgroups, the others through the
        general kernel: a single token behind many keys would otherwise be one workgroup's long walk that the
        whole step waits for.  ``portions_max_kv_len``: the most keys any sequence behind that prefix holds (default: ``max_kv_len``).
        ``distance_bias``: float32 ``[num_heads, L]``, added to the scaled scores: a key ``n`` positions behind the query reads
        column ``min(n, L - 1)`` of its query head's row (the kernels' build for it is loaded by ``attention_library(d, True)``).
        ``sinks``: float32 ``[num_heads]``; ``exp(sinks[h])`` joins the denominator of every softmax of head ``h`` (a sink has no key
        and no value and is not scaled).  ``keep_first`` beside a window: so many first tokens of a sequence are seen whatever the
        window.  ``softcap``: a scaled score ``s`` becomes ``softcap * tanh(s / softcap)`` (before the bias).  ``gate = (source, first column, channels)``:
        head ``h``'s output times ``sigmoid`` of the source's columns, ``channels`` per head (channels beyond are left alone) or one per head
        with ``channels`` = 0.  (Each of the three has a build of the kernels: ``attention_library``.)"""
        tokens = qkv.shape[0]
        keep_first = int(keep_first) if window else 0
        gate_at, gate_stride, gate_channels = 0, 0, 0
        if gate is not None:
            gate, gate_at, gate_channels = gate
            self._check("gate", gate, qkv.dtype)
            gate_stride = gate.shape[1] if gate.dim() == 2 else 0
            if gate.dim() != 2 or gate.shape[0] != tokens or gate_at < 0 or not 0 <= gate_channels <= head_dim or gate_at + num_heads * max(gate_channels, 1) > gate_stride:
                raise KernelError("paged_attention: the gate's columns do not lie within its source")
        if keep_first < 0 or (softcap is not None and not softcap > 0):
            raise KernelError(f"paged_attention: keep_first={keep_first} must not be negative, softcap={softcap} must be positive")

        def gate_rows(first_token: int):
            return _P(0) if gate is None else _P(gate.data_ptr() + (first_token * gate_stride + gate_at) * gate.element_size())
        if sinks is not None:
            self._check("sinks", sinks, torch.float32, (num_heads,))
        width = qkv.shape[1] if qkv.dim() == 2 else -1  # rows may carry keys and values after the queries
        if width not in (num_heads * head_dim, (num_heads + 2 * num_kv_heads) * head_dim):
            raise KernelError(f"paged_attention: rows of {width} elements hold neither the queries nor queries, keys and values")
        self._check("qkv", qkv, None, (tokens, width), align=16)
        num_seqs = kv_lens.shape[0]
        self._check("kv_lens", kv_lens, torch.int32, (num_seqs,))
        self._check("cu_q", cu_q, torch.int32, (num_seqs + 1,))
        self._check("block_tables", block_tables, torch.int32)
        if block_tables.dim() != 2 or block_tables.shape[0] != num_seqs:
            raise KernelError(f"block_tables must be [{num_seqs}, W], got {tuple(block_tables.shape)}")
        if block_size <= 0 or block_size & (block_size - 1):
            raise KernelError(f"block_size must be a power of two, got {block_size}")
        if block_tables.shape[1] * block_size < max_kv_len:
            raise KernelError(f"block tables of width {block_tables.shape[1]} cannot cover {max_kv_len} keys")
        pages = k_cache.shape[0]
        self._check("k_cache", k_cache, qkv.dtype, (pages, num_kv_heads, block_size, head_dim), align=16)
        self._check("v_cache", v_cache, qkv.dtype, (pages, num_kv_heads, head_dim, block_size), align=16)
        if num_heads % num_kv_heads != 0:
            raise KernelError("num_heads must be a multiple of num_kv_heads")
        if not scale > 0:
            raise KernelError(f"paged_attention: the scale must be positive, got {scale}")
        if max_q_len < 1 or max_q_len > tokens:
            raise KernelError(f"max_q_len={max_q_len} outside [1, {tokens}]")
        if not 0 <= decode_prefix <= num_seqs or num_seqs > tokens:
            raise KernelError(f"decode_prefix={decode_prefix} does not fit {num_seqs} sequences with {tokens} tokens")
        out = torch.empty((tokens, num_heads * head_dim), dtype=qkv.dtype, device=self.device)
        bias_len = 0
        if distance_bias is not None:
            self._check("distance_bias", distance_bias, torch.float32)
            if distance_bias.dim() != 2 or distance_bias.shape[0] != num_heads or distance_bias.shape[1] < 1:
                raise KernelError(f"paged_attention: the bias by distance is [{num_heads}, L], got {tuple(distance_bias.shape)}")
            bias_len = int(distance_bias.shape[1])
        if head_dim > self.MAX_TILED_HEAD_DIM:
            # beyond the tiled kernels: one workgroup per token and head, plain float32 arithmetic
            if head_dim > 1024:
                raise KernelError(f"paged_attention: head_dim={head_dim} is beyond every kernel (1,024 at most)")
            status = self._core.velox_plain_attention(_ptr(qkv), width, _ptr(k_cache), _ptr(v_cache), _ptr(block_tables), block_tables.shape[1], _ptr(cu_q),
                                                      _ptr(kv_lens), _ptr(out), num_seqs, tokens, num_heads, num_kv_heads, head_dim,
                                                      block_size.bit_length() - 1, float(scale), int(window or 0), _code(qkv.dtype), _ptr(distance_bias), bias_len,
                                                      _ptr(sinks), keep_first, float(softcap or 0.0), gate_rows(0), gate_stride, int(gate_channels), self._stream())
            self._launched(status, "plain_attention")
            return out
        lib = self.attention_library(head_dim, distance_bias is not None, kept=keep_first > 0, capped=softcap is not None, gated=gate is not None)
        group = num_heads // num_kv_heads

        def launch(first_seq: int, count: int, first_token: int, num_tokens: int, longest: int, decode_only: bool, splits: Optional[int]) -> None:
            # sequences [first_seq, first_seq + count); their tokens are rows [first_token, first_token + num_tokens) of qkv
            # and out.  cu_q holds absolute rows, so the general kernel takes qkv and out whole; the streaming kernel
            # counts rows from its first sequence and takes the slices.
            row_tiles = (longest * group + 63) // 64
            if splits is None:
                # (a window bounds the keys a row block walks, however long the sequence)
                seen = window + keep_first + longest if window else max_kv_len
                splits = self.choose_splits(count, num_kv_heads, row_tiles, min(max_kv_len, seen), decode_only)
                if not decode_only:
                    splits = self.choose_portion_splits(num_tokens, group, num_kv_heads, min(max_kv_len, portions_max_kv_len or max_kv_len, seen))
            if count * splits > 65535:
                raise KernelError(f"{count} sequences x {splits} splits exceed the launch grid")
            part_o = part_lse = None
            if splits > 1:
                if workspace is None:
                    raise KernelError("split attention needs a workspace")
                span = num_tokens if decode_only else tokens  # the rows the kernels count partial results by
                part_o = workspace.get("attention_partial_out", splits * span * num_heads * head_dim)
                part_lse = workspace.get("attention_partial_lse", splits * span * num_heads)
            rows_in, rows_out = (qkv[first_token:first_token + num_tokens], out[first_token:first_token + num_tokens]) if decode_only else (qkv, out)
            status = lib.velox_paged_attention(
                _ptr(rows_in), width, _ptr(k_cache), _ptr(v_cache), _ptr(block_tables[first_seq:]), block_tables.shape[1],
                _ptr(cu_q[first_seq:]), _ptr(kv_lens[first_seq:]), _ptr(rows_out), _ptr(part_o), _ptr(part_lse), count,
                num_tokens if decode_only else tokens, longest, int(max_kv_len), num_heads, num_kv_heads,
                block_size.bit_length() - 1, float(scale), int(window or 0), splits, 0 if decode_only else first_token, _code(qkv.dtype),
                _ptr(distance_bias), bias_len, _ptr(sinks), keep_first, float(softcap or 0.0), gate_rows(first_token if decode_only else 0), gate_stride,
                int(gate_channels), self._stream())
            self._launched(status, "paged_attention")

        if not all_decode and splits is None and 0 < decode_prefix < num_seqs and group <= 16:
            launch(0, decode_prefix, 0, decode_prefix, 1, True, None)
            launch(decode_prefix, num_seqs - decode_prefix, decode_prefix, tokens - decode_prefix, max_q_len, False, None)
        else:
            launch(0, num_seqs, 0, tokens, max_q_len, bool(all_decode), splits)
        return out

    # -- sampling -------------------------------------------------------------------------------
    def argmax(self, logits: torch.Tensor) -> torch.Tensor:
        self._check("logits", logits, torch.float32)
        rows, vocab = logits.shape
        out = torch.empty(rows, dtype=torch.int32, device=self.device)
        # few rows alone would leave most of the GPU idle: the vocabulary is cut into chunks of at least 2048 entries
        chunks = max(1, min(2 * self.num_cus // rows, vocab // 2048, 256))
        partial = torch.empty((rows, chunks, 2), dtype=torch.int32, device=self.device) if chunks > 1 else None
        self._launched(self._core.velox_argmax(_ptr(logits), _ptr(out), _ptr(partial), rows, vocab, chunks, self._stream()), "argmax")
        return out

    def sample(self, logits: torch.Tensor, options: torch.Tensor, with_filter: bool = True, chunks: Optional[int] = None) -> torch.Tensor:
        """One token per row of float32 ``logits`` by the rows' ``options`` (int32 ``[rows, 6]``: see ``sample_kernel``).
        ``with_filter=False`` promises that no row has top-k or top-p (a row that has one all the same comes back as -1 when rows are cut into chunks).  ``chunks``: into how many pieces a row is cut
        (default: one workgroup per row when the rows fill the GPU, else enough pieces to fill it); the tokens do not
        depend on it."""
        self._check("logits", logits, torch.float32)
        rows, vocab = logits.shape
        self._check("options", options, torch.int32, (rows, 6))
        out = torch.empty(rows, dtype=torch.int32, device=self.device)
        if chunks is None:
            # About one workgroup per compute unit: every workgroup of a pass works out the digit before its own from the
            # row's tables again, so more chunks than fill the GPU cost more than they save (64 rows of 152,064 on
            # MI355X: 187 us whole, 86 us in 4 chunks, 148 us in 16; 8 rows: 178 us whole, 46 us in 16 chunks).
            chunks = max(1, min(self.num_cus // rows, vocab // 8192, 32))
        if chunks > 1:
            if chunks > 1024 or rows > 65535:
                raise KernelError(f"sample: {rows} rows x {chunks} chunks exceed the launch grid")
            size = int(self._core.velox_sample_chunked_scratch_bytes(rows, chunks))
            scratch = torch.empty(size, dtype=torch.uint8, device=self.device)
            status = self._core.velox_sample_chunked(_ptr(logits), _ptr(options), _ptr(out), rows, vocab, chunks, _ptr(scratch), size,
                                                     1 if with_filter else 0, self._stream())
            self._launched(status, "sample_chunked")
            return out
        self._launched(self._core.velox_sample(_ptr(logits), _ptr(options), _ptr(out), rows, vocab, self._stream()), "sample")
        return out

    def apply_penalties(self, logits, tokens, lengths, coeffs) -> None:
        self._check("logits", logits, torch.float32)
        rows, vocab = logits.shape
        self._check("tokens", tokens, torch.int32)
        if tokens.dim() != 2 or tokens.shape[0] != rows:
            raise KernelError("apply_penalties: tokens must be [rows, width]")
        self._check("lengths", lengths, torch.int32, (rows,))
        self._check("coeffs", coeffs, torch.float32, (rows, 3))
        status = self._core.velox_apply_penalties(_ptr(logits), _ptr(tokens), _ptr(lengths), _ptr(coeffs), rows, vocab, tokens.shape[1], self._stream())
        self._launched(status, "apply_penalties")

    def count_tokens(self, counts_row: torch.Tensor, tokens: torch.Tensor) -> None:
        """``counts_row[token] += 1`` for every token of int32 ``tokens`` (ids outside the row are skipped)."""
        self._check("counts_row", counts_row, torch.int32)
        self._check("tokens", tokens, torch.int32)
        if counts_row.dim() != 1 or tokens.dim() != 1:
            raise KernelError("count_tokens: a row of counts and a list of tokens are expected")
        self._launched(self._core.velox_count_tokens(_ptr(counts_row), _ptr(tokens), tokens.numel(), counts_row.numel(), self._stream()), "count_tokens")

    def count_sampled(self, counts: torch.Tensor, row_of: torch.Tensor, tokens: torch.Tensor) -> None:
        """``counts[row_of[r], tokens[r]] += 1`` for every batch row ``r`` with ``row_of[r] >= 0``."""
        self._check("counts", counts, torch.int32)
        rows = tokens.numel()
        self._check("row_of", row_of, torch.int32, (rows,))
        self._check("tokens", tokens, torch.int32, (rows,))
        if counts.dim() != 2:
            raise KernelError("count_sampled: counts must be [table rows, vocab]")
        self._launched(self._core.velox_count_sampled(_ptr(counts), _ptr(row_of), _ptr(tokens), rows, counts.shape[1], self._stream()), "count_sampled")

    def apply_penalties_from_counts(self, logits: torch.Tensor, counts: torch.Tensor, row_of: torch.Tensor, coeffs: torch.Tensor) -> None:
        """Penalises float32 ``logits`` [rows, vocab] in place: row ``r`` by the counts of table row ``row_of[r]`` (rows with
        -1 are left alone) and ``coeffs[r] = (repetition, presence, frequency)``.  The host must keep ``row_of`` inside the table."""
        self._check("logits", logits, torch.float32)
        rows, vocab = logits.shape
        self._check("counts", counts, torch.int32)
        if counts.dim() != 2 or counts.shape[1] != vocab:
            raise KernelError(f"apply_penalties_from_counts: counts must be [table rows, {vocab}], got {tuple(counts.shape)}")
        self._check("row_of", row_of, torch.int32, (rows,))
        self._check("coeffs", coeffs, torch.float32, (rows, 3))
        chunks = max(1, min(2 * self.num_cus // rows, (vocab + 2047) // 2048))
        status = self._core.velox_penalties_from_counts(_ptr(logits), _ptr(counts), _ptr(row_of), _ptr(coeffs), rows, vocab, chunks, self._stream())
        self._launched(status, "penalties_from_counts")

    # -- probes ---------------------------------------------------------------------------------
    def _timed(self, launch, repeats: int) -> float:
        """Seconds per call of ``launch`` (the best of ``repeats`` after one untimed call)."""
        launch()
        torch.cuda.synchronize(self.device)
        best = float("inf")
        for _ in range(repeats):
            start, end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            start.record()
            launch()
            end.record()
            end.synchronize()
            best = min(best, start.elapsed_time(end) * 1e-3)
        return best

    def probe_read_bandwidth(self, num_bytes: int = 4 << 30, repeats: int = 5) -> float:
        """GB/s at which a kernel that only reads streams ``num_bytes`` of device memory (far more than the caches hold)."""
        num_bytes -= num_bytes % 16
        data = torch.empty(num_bytes, dtype=torch.uint8, device=self.device).zero_()
        sink = torch.zeros(1, dtype=torch.int32, device=self.device)
        blocks = self.num_cus * 8
        seconds = self._timed(lambda: self._launched(self._core.velox_probe_read(_ptr(data), num_bytes, _ptr(sink), blocks, self._stream()), "probe_read"), repeats)
        return num_bytes / seconds * 1e-9

    def probe_grid_barrier(self, fenced: bool, rounds: int = 2000, repeats: int = 3) -> float:
        """Microseconds per barrier across one workgroup per compute unit inside one kernel: with relaxed agent-scope
        counters only, or (``fenced``) with the release and acquire that ordinary stores and loads around it need."""
        counters = torch.zeros(17 * 32, dtype=torch.int32, device=self.device)
        failed = torch.zeros(1, dtype=torch.int32, device=self.device)

        def launch() -> None:
            counters.zero_()
            self._launched(self._core.velox_probe_grid_barrier(self.num_cus, rounds, int(fenced), _ptr(counters), _ptr(failed), self._stream()), "probe_grid_barrier")

        seconds = self._timed(launch, repeats)
        if int(failed.item()) != 0:
            raise KernelError("probe_grid_barrier: a workgroup gave up waiting for the others")
        return seconds / rounds * 1e6

    def probe_mfma_rate(self, iterations: int = 20000, repeats: int = 5) -> float:
        """TFLOP/s of independent bfloat16 32x32x16 matrix instructions, two workgroups of four waves per compute unit."""
        sink = torch.zeros(1, dtype=torch.float32, device=self.device)
        blocks = self.num_cus * 2
        seconds = self._timed(lambda: self._launched(self._core.velox_probe_mfma(blocks, iterations, _ptr(sink), self._stream()), "probe_mfma"), repeats)
        return blocks * 4 * iterations * 4 * 32768.0 / seconds * 1e-12
