"""`HipOps`: the kernel surface on hand-written HIP kernels for gfx950.

The kernels live in shared libraries built from `distie_amd/csrc` and are called through
ctypes with raw device pointers on torch's current HIP stream, so they take part in
stream order and in graph capture like any other launch. torch is the allocator and the
stream/graph owner; the only library routine on this path is the matrix product for
large bfloat16 operands (the reference leaves its products to a library too).

Constructing `HipOps` without a GPU, without hipcc-built libraries, or for a head size
the kernels refuse, raises: there is no fallback.
"""

from __future__ import annotations

import ctypes
import logging
from typing import Dict, Optional

import numpy as np
import torch

from ..csrc import build
from .interface import BatchMeta, Ops, RouteRule

_log = logging.getLogger(__name__)

_F32, _BF16 = 0, 1
_CODES = {torch.float32: _F32, torch.bfloat16: _BF16}
_P = ctypes.c_void_p
_I = ctypes.c_int
_L = ctypes.c_int64
_F = ctypes.c_float


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)


class KernelError(RuntimeError):
    pass


def _code(t: torch.Tensor) -> int:
    try:
        return _CODES[t.dtype]
    except KeyError:
        raise KernelError(f"kernels take float32 and bfloat16 tensors, not {t.dtype}") from None


def _check(status: int, name: str) -> None:
    if status == 0:
        return
    if status < 0:
        raise KernelError(f"{name}: the kernel refuses these sizes or types")
    raise KernelError(f"{name}: launch failed with HIP error {status}")


def _written(t: torch.Tensor):
    """How often `t` has been written in place, as far as anyone can know: torch's own count (every in-place
    torch operation on the tensor or on a view of it) and the count of this module's kernels that write their
    argument (`_mark_written`)."""
    return (t._version, getattr(t, "_distie_version", 0))


def _mark_written(t: torch.Tensor) -> None:
    t._distie_version = getattr(t, "_distie_version", 0) + 1


class _NotATensorYet:
    """What `HipOps` hands out in place of a tensor. Anything asked of it that only a tensor has raises
    with the way out, instead of an AttributeError far from the cause."""

    def __getattr__(self, name):
        raise KernelError(f"{type(self).__name__} is a result of the HIP kernels that is not a tensor yet (asked for "
                          f".{name}): a part that computes on the values itself calls ops.dense(value) first")


class PartialSums(_NotATensorYet):
    """The result of a matrix product whose reduction was cut into slices: float32
    [slices, rows, columns], to be added in order by whoever reads it. `linear` returns it for
    small batches (a sum across workgroups inside the product would cost more than the product);
    `add_rmsnorm`, `silu_mul` and `rope_kv_write` add the slices while they read, every other
    operation sees the finished sum through `HipOps.dense`."""

    def __init__(self, data: torch.Tensor, dtype: torch.dtype) -> None:
        self.data = data
        self.dtype = dtype                  # the dtype the finished sum would have
        self.shape = data.shape[1:]
        self.device = data.device

    @property
    def slices(self) -> int:
        return self.data.shape[0]


class PendingNorm(_NotATensorYet):
    """rmsnorm(residual) * weight, not computed yet: for steps of few rows the product that reads it computes
    it itself, in front of its own work (`distie_decode_norm_product`); anything else sees the finished
    tensor through `HipOps.dense`. Valid as long as the residual it was made from is unchanged: a write in
    place by torch (also through a view) or by one of this module's kernels between `rmsnorm` and the use is
    found out and raises, instead of a norm of the wrong values."""

    def __init__(self, residual: torch.Tensor, weight: torch.Tensor, eps: float, dtype: torch.dtype) -> None:
        self.residual = residual
        self.weight = weight
        self.eps = float(eps)
        self.dtype = dtype
        self.shape = residual.shape
        self.device = residual.device
        self.version = _written(residual)

    def check(self) -> None:
        if _written(self.residual) != self.version:
            raise KernelError("a normed value was used after the residual stream it was made from had changed")


class PendingProduct(_NotATensorYet):
    """x W^T + bias for few rows of x, not computed yet: if the next thing that happens to it is the sum into
    the residual stream, the product adds itself to the stream in place (`distie_decode_product_residual`) and
    never exists as a tensor; anything else sees the finished tensor through `HipOps.dense`."""

    def __init__(self, x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor]) -> None:
        self.x = x
        self.weight = weight
        self.bias = bias
        self.dtype = x.dtype
        self.shape = torch.Size((x.shape[0], weight.shape[0]))
        self.device = x.device


class NormedSum(_NotATensorYet):
    """scale * sum_i rmsnorm(terms[i]) * weights[i], not computed yet: if what happens to it next is the norm behind
    its sub-layer and the sum into the residual stream, one kernel does all of it (`distie_norm_chain`); anything else
    sees the finished float32 tensor through `HipOps.dense`."""

    def __init__(self, terms, weights, eps: float, scale: float) -> None:
        self.terms, self.weights, self.eps, self.scale = terms, weights, eps, scale
        self.dtype = torch.float32
        self.shape = terms[0].shape
        self.device = terms[0].device


class HipOps(Ops):
    # Steps of up to FUSED_MAX_ROWS rows can run their products with the norm in front and the residual sum behind
    # folded in (six launches a layer instead of eight, no partial sums handed on). On the device that is no
    # gain: a kernel's time here is a chain of trips to memory, and the folded-in norm or the sum across a
    # workgroup's waves adds its trip to the product's own (measured at 8 rows, 1,536 wide: gate+up 18.7 us with
    # the norm against 13.4 + 4.2 us apart; down 13.2 against 8.3 us in 14 slices, since 96 workgroups pull
    # less than 1,344; q/k/v 9.0 against 5.5 + 4.2 us). Where the host bounds a step, two launches fewer a layer
    # count: steps that are launched kernel by kernel take this path, captured steps do not.
    FUSED_MAX_ROWS = 16
    FUSED_IN_CAPTURED_STEPS = False
    # float32 products (and products against weights kept in float32) of up to ROWS_MAX_ROWS rows stream the weights
    # through `gemv_rows` (FMAs on the vector ALU); beyond that the tiled float32 kernel
    ROWS_MAX_ROWS = 64
    # bfloat16 products by rows of x: up to SKINNY_MAX_ROWS the weights are streamed by one wave per block
    # of 16 weight rows, x straight from memory (above that, the library's tiles are faster);
    SKINNY_MAX_ROWS = 16
    # on a packed copy the one-wave kernel is the faster one only up to 8 rows: at 9 to 16 rows every wave reads all
    # 16 rows of x beside its weights, and the kernel that shares x through LDS takes over (decode step at batch 12
    # and 16: 1.5B shape 1.77 -> 1.66 and 1.95 -> 1.81 ms, 7B shape 4.34 -> 3.91 and 4.92 -> 4.14 ms; at batch 8 and
    # below the one-wave kernel is level or ahead)
    ONE_WAVE_MAX_ROWS = 8
    # with a packed copy of the weight, more rows go through the kernel that shares the x tile of a workgroup in
    # LDS, in passes over the weight: up to PACKED_MAX_ROWS in a captured step (measured in the decode step: 9 %
    # faster than the library at 72 rows, 5 % at 96, 4 % slower at 128), and up to PACKED_MAX_ROWS_EAGER in a step
    # that is launched kernel by kernel, which the host bounds at these sizes: the library's products cost it
    # 18 us each and the activation and rotation kernels beside them more launches (a portion of n tokens behind
    # 512, this way and through the library, 1.5B shape: 100: 2.8 and 3.4 ms, 160: 3.1 and 3.4, 200: 3.6 and 3.5,
    # 224: 3.7 and 3.5).
    # A weight of more than PACKED_LARGE_ELEMENTS (64 MB) is not held by the memory-side cache from one pass to the
    # next: a pass takes up to 96 rows, and every further one reads the weight from memory again, which the library
    # does once. Which is faster then goes by the weight's shape (7B shape at 128 rows, the packed kernels in two
    # passes and the library's best kernel by timing, with the same flush of the caches before each: gate+up
    # [37888, 3584] 144 and 115 us, the head [152064, 3584] 535 and 297, down [3584, 18944] 75 and 91):
    #  * K longer than the weight has rows (down): the packed kernels, whose K is cut into slices, up to
    #    PACKED_MAX_ROWS_LARGE rows, captured or not;
    #  * more rows than K (gate+up, the head, a large q/k/v): one pass, PACKED_MAX_ROWS_LARGE_WIDE rows. Once the
    #    library's kernels were timed for a class of row counts (`library_timed_rows`, set by the engine's start with
    #    `tune_products`), the library takes over from 65 rows on (PACKED_MAX_ROWS_LARGE_WIDE_TIMED): untimed, its
    #    choice is good at one row count and poor at the next. 7B shape, decode step at batch 72, 80, 96, 112, 128,
    #    160, 192: 6.4, 6.6, 7.3, 8.1, 8.4, 10.4, 10.9 ms timed; 6.6, 6.8, 8.0, 8.6, 9.6, 11.7, 12.0 untimed; and with
    #    every large weight on the packed kernels up to 192 rows 6.6, 6.8, 8.0, 9.2, 9.7, 11.9, 13.3. At 24 to 64 rows
    #    the timed library is 1-3 % ahead as well (gate+up rounded to bfloat16 before the activation): left as it is.
    # The 1.5B shape's weights are small, its head large: its captured step is the same either way.
    PACKED_MAX_ROWS = 96
    PACKED_MAX_ROWS_LARGE = 192
    PACKED_MAX_ROWS_LARGE_WIDE = 96
    PACKED_MAX_ROWS_LARGE_WIDE_TIMED = 64
    PACKED_MAX_ROWS_EAGER = 192
    PACKED_LARGE_ELEMENTS = 32 << 20
    # or, for a weight of at most this many elements (too few row blocks to occupy the chip that way),
    # through the one-wave kernel once per 16 rows of x
    ROW_GROUPS_MAX_ELEMENTS = 4 << 20
    # the q/k/v product with rotation and cache write in its epilogue exists per 16 rows only; from so many rows on a
    # weight above that size runs on the wide kernel instead, with rotation and cache write as the kernel behind it
    # (7B shape, decode step: 1.5 % slower at 24 rows, the same at 32 and 48, 2.7 % faster at 64)
    WIDE_QKV_MIN_ROWS = 49
    # ... and that kernel takes more than 32 rows in two passes of 32 over a weight of at most this many elements
    # (64 MB: the second pass reads it from the memory-side cache; much larger ones would come from memory twice)
    TWO_PASS_MAX_ELEMENTS = 32 << 20
    # ... and a larger one is read once per pass: as few passes as the kernel's 96 rows a pass allow, of equal size
    # (7B shape: decode step at batch 80 6.8 ms in one pass of 80 rows, 7.7 as 64 + 16; at batch 96 8.1 and 8.3;
    # a portion of 160 tokens 7.4 ms in two passes of 80 and 8.4 in three of 64, 64 and 32)
    WIDE_PASS_MAX_BLOCKS = 6
    # attention over a portion of a prompt: from so many visible keys on, the walk over the keys is cut into so
    # many parts that run side by side (measured at 12 heads of 128, 2,048 new tokens: 3 parts are best up to
    # 4,096 keys, 5 at 8,192, 8 from 16,384 on; the kernel takes up to 16)
    PREFILL_PARTS = ((1024, 3), (8192, 5), (16384, 8))
    PREFILL_WORKGROUPS = 512         # as many workgroups a short portion's attention should have, if its keys allow
    PACKED_KEEPS_FREE = 0.3          # share of the device's memory that packed weight copies leave free
    PREFILL_F32_MIN_TOKENS = 32      # float32 steps with a portion of at least this many tokens go to the tiled float32 kernel
    # decode attention cuts the keys into runs so that about DECODE_WAVES waves are at work, with at most
    # DECODE_MAX_RUNS places for partial results per request and head. The kernel keeps two waves a SIMD (2,048 on
    # the chip); 1,536 is what the step likes best (1.5B shape, batch 32 and 64: 2.07 and 2.77 ms with 1,024, 2.02
    # and 2.71 with 1,536, 2.11 and 2.75 with 2,048; 7B shape, batch 160: 10.85, 10.05, 10.15 ms; batch 1 to 16 the same)
    DECODE_WAVES = 1536
    # where the same number of runs for every request leaves more than a fifth of those waves unused (1,024 pairs
    # of a request and a kv head: one run each), the requests of a decode step share one run length instead: the
    # shortest with which their runs together stay within DECODE_WAVES, so that a long request gets more runs than a
    # short one (256 requests on 4 kv heads, contexts of 1,050 to 3,150 keys: 263 -> 245 us a layer; contexts of one
    # length are cut as before). Everywhere else it is level or behind (32 requests: 30 -> 33 us).
    DECODE_SHARED_BELOW = 0.8
    DECODE_MAX_RUNS = 256
    # attention with mixed heads: from so many tokens a step on a workgroup takes 16 queries instead of 8 (fewer would
    # leave compute units without one)
    MIXED_WIDE_TOKENS = 6144
    # the matrix-core attention kernels take heads up to 256; wider ones (a latent that all heads share) run on the
    # wave-per-token kernel, in either precision
    LARGEST_MATRIX_CORE_HEAD = 256
    LARGEST_HEAD = 1024

    def __init__(self, device="cuda:0", packed_weights=True) -> None:
        """`packed_weights` (True, False, or the roles that get one, as the parts name them in
        `prepare_linear`: "qkv", "attn_out", "gate_up", "down", "head"): keep a second copy of every bfloat16 weight in the order in which the
        matrix cores take it, for products with at most `PACKED_MAX_ROWS_EAGER` rows (decode, short portions). It doubles
        the memory of the weights and makes those products 15-25 % faster, and it is what the fused
        epilogues (activation, rotation and cache write) work on; without it products of up to
        `SKINNY_MAX_ROWS` rows stream the weights as they are stored and larger ones go to the library."""
        self.device = torch.device(device)
        if isinstance(packed_weights, (bool, int)) or packed_weights is None:
            self.packed_weights = bool(packed_weights)
            self.packed_roles = None
        else:
            self.packed_roles = frozenset(packed_weights)
            self.packed_weights = bool(self.packed_roles)
        if self.device.type != "cuda" or not torch.cuda.is_available():
            raise KernelError("HipOps needs an AMD GPU (torch.cuda is not available): there is no CPU path")
        name = torch.cuda.get_device_properties(self.device).gcnArchName
        if not name.startswith("gfx950"):
            raise KernelError(f"the kernels are built for gfx950 (MI355X); this device is {name}")
        self._device_index = self.device.index if self.device.index is not None else torch.cuda.current_device()
        self._compute_units = torch.cuda.get_device_properties(self.device).multi_processor_count
        self._lib = None
        self._tuning = False
        self.library_timed_rows = 0
        self._packed_left_out = 0
        self._ops = ctypes.CDLL(str(build.ensure("ops")))
        self._declare()
        self._attn: Dict[int, ctypes.CDLL] = {}
        self._mixed: Dict[int, ctypes.CDLL] = {}
        # pinned staging buffers for `upload`, used in turn: [host tensor, its numpy view, event of the last copy]
        self._uploads = [[None, None, None] for _ in range(self.UPLOAD_BUFFERS)]
        self._next_upload = 0

    # ------------------------------------------------------------ plumbing
    UPLOAD_BUFFERS = 8

    def upload(self, values: np.ndarray) -> torch.Tensor:
        """Through pinned memory, so that the copy is queued like a kernel: `torch.tensor(..., device=...)` copies
        from pageable memory and returns only when everything queued before it is done, which made the host
        wait for the running step three times per sampled step."""
        values = np.ascontiguousarray(values)
        dtype = torch.from_numpy(np.empty(0, dtype=values.dtype)).dtype
        nbytes = values.nbytes
        if nbytes == 0:
            return torch.empty(values.shape, dtype=dtype, device=self.device)
        slot = self._uploads[self._next_upload]
        self._next_upload = (self._next_upload + 1) % len(self._uploads)
        if slot[2] is not None:
            slot[2].synchronize()                       # the copy made out of this buffer some calls ago is done
        if slot[0] is None or slot[0].numel() < nbytes:
            slot[0] = torch.empty(max(4096, 2 * nbytes), dtype=torch.uint8, pin_memory=True)
            slot[1] = slot[0].numpy()
            slot[2] = torch.cuda.Event()
        slot[1][:nbytes] = values.reshape(-1).view(np.uint8)
        dev = torch.empty(nbytes, dtype=torch.uint8, device=self.device)
        dev.copy_(slot[0][:nbytes], non_blocking=True)
        slot[2].record()
        return dev.view(dtype).view(values.shape)

    def _declare(self) -> None:
        o = self._ops
        o.distie_scatter_i32.argtypes = [_P, _P, _P, _I, _L, _P]
        o.distie_embed.argtypes = [_P, _P, _I, _P, _I, _I, _I, _F, _P]
        o.distie_rmsnorm.argtypes = [_P, _P, _I, _I, _P, _I, _P, _I, _I, _I, _F, _P]
        o.distie_rope_kv_write.argtypes = [_P, _I, _I, _P, _I, _P, _P, _P, _P, _P, _I, _P, _I, _I, _I, _I, _I, _I, _I, _P]
        o.distie_rope_table.argtypes = [_P, _P, _P, _I, _I, _P]
        o.distie_silu_mul.argtypes = [_P, _I, _I, _P, _I, _I, _I, _P]
        o.distie_sum_slices.argtypes = [_P, _I, _L, _P, _I, _P]
        o.distie_gather_rows.argtypes = [_P, _P, _P, _I, _L, _I, _P]
        o.distie_gemm_generic.argtypes = [_P, _I, _P, _I, _P, _P, _I, _I, _I, _I, _P]
        o.distie_gemv_rows.argtypes = [_P, _I, _P, _I, _P, _P, _I, _I, _I, _I, _P]
        o.distie_gemm_skinny_slices.argtypes = [_I, _I, _I]
        o.distie_gemm_skinny_bf16.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _P]
        o.distie_pack_rows.argtypes = [_P, _P, _P, _I, _I, _P]
        o.distie_gemm_packed_bf16.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _I, _F, _F, _F, _P]
        o.distie_gemm_packed_wide_bf16.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _F, _F, _P]
        o.distie_gemm_packed_wide_slices.argtypes = [_I, _I]
        o.distie_gemm_packed_wide_qkv_bf16.argtypes = [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P]
        o.distie_gemm_packed_rotary_bf16.argtypes = [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P]
        o.distie_gemm_packed_each_bf16.argtypes = [_P, _P, _P, _I, _I, _I, _P, _P]
        o.distie_decode_norm_fits.argtypes = [_I]
        o.distie_decode_product_residual.argtypes = [_P, _P, _P, _P, _I, _I, _I, _P]
        o.distie_decode_norm_product.argtypes = [_P, _P, _F, _P, _P, _P, _I, _I, _I, _I, _P, _P, _P, _P,
                                                 _I, _I, _I, _I, _I, _P]
        o.distie_hyper_step.argtypes = [_P, _I, _P, _P, _I, _I, _P, _I, _L, _I, _P, _P, _P, _P, _I, _I, _F, _P, _I, _I, _I, _P]
        o.distie_causal_conv.argtypes = [_P, _I, _L, _P, _I, _I, _P, _P, _I, _L, _I, _P, _P, _P, _P, _I, _I, _P]
        o.distie_conv_state.argtypes = [_P, _I, _L, _I, _P, _P, _P, _I, _I, _I, _P]
        o.distie_conv_rope_kv_write.argtypes = [_P, _I, _L, _P, _I, _I, _P, _P, _I, _F, _P, _P, _P, _I, _P, _P, _P, _P,
                                                _I, _I, _I, _I, _I, _I, _I, _I, _I, _P, _F, _I, _P, _P, _F, _I, _I, _I, _P]
        o.distie_sigmoid_gate.argtypes = [_P, _I, _I, _I, _P, _I, _L, _P, _I, _I, _I, _P]
        o.distie_rmsnorm_gate.argtypes = [_P, _P, _I, _F, _P, _I, _L, _P, _I, _I, _I, _I, _I, _I, _P]
        o.distie_norm_chain.argtypes = [_P, _I, _I, _P, _P, _I, _I, _P, _F, _F, _P, _F, _P, _P, _F, _P, _I, _P, _I, _I, _P]
        o.distie_gated_decay_scan.argtypes = [_P, _I, _L, _P, _P, _L, _P, _P, _I, _P, _P, _P, _P, _I, _I, _I, _I, _F, _F, _P]
        o.distie_gated_decay_scan_chunked.argtypes = [_P, _I, _L, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _F, _F, _P]
        o.distie_lru_gates.argtypes = [_P, _I, _L, _P, _P, _P, _P, _I, _P, _F, _P, _P, _I, _I, _I, _P]
        o.distie_lru_scan.argtypes = [_P, _P, _P, _P, _I, _L, _I, _P, _I, _P, _P, _I, _I, _P]
        o.distie_lru_scan_chunked.argtypes = [_P, _P, _P, _P, _P, _P, _P, _I, _L, _I, _P, _I, _P, _P, _P, _I, _I, _I, _P]
        o.distie_route_topk.argtypes = [_P, _I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _P, _I, _I, _F, _I, _P]
        o.distie_route_glu.argtypes = [_P, _I, _L, _I, _P, _P, _I, _I, _I, _I, _F, _F, _F, _I, _I, _P, _I, _P]
        o.distie_route_topk_glu.argtypes = [_P, _P, _P, _I, _I, _P, _I, _L, _I, _I, _I, _I, _I, _F, _F, _F, _I, _P, _I, _I, _F, _I, _I, _P, _I, _P]
        o.distie_softcap_f32.argtypes = [_P, _L, _F, _P]
        o.distie_route_scale.argtypes = [_P, _I, _L, _P, _P, _I, _I, _I, _I, _P]
        o.distie_scale_f32.argtypes = [_P, _L, _F, _P]
        o.distie_activation.argtypes = [_P, _I, _I, _P, _I, _L, _I, _P]
        o.distie_decay_scan.argtypes = [_P, _I, _L, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P, _I, _I, _F, _P]
        o.distie_decay_scan_chunked.argtypes = [_P, _I, _L, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _I, _F, _P]
        o.distie_delta_scan.argtypes = [_P, _I, _L, _P, _L, _P, _L, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _F, _F, _P]
        o.distie_delta_scan_chunked.argtypes = [_P, _I, _L, _P, _L, _P, _L, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P,
                                                _P, _I, _I, _I, _I, _I, _I, _F, _F, _P]
        o.distie_latent_norm_rope_write.argtypes = [_P, _I, _L, _I, _P, _I, _P, _F, _I, _P, _F, _I, _P, _I, _P, _P, _I, _P,
                                                    _I, _I, _I, _I, _P]
        o.distie_latent_queries.argtypes = [_P, _I, _I, _I, _P, _I, _P, _I, _I, _I, _I, _I, _I, _P, _F, _I, _P]
        o.distie_rope_heads.argtypes = [_P, _I, _I, _I, _P, _I, _I, _I, _I, _I, _P, _F, _I, _P]
        o.distie_heads_linear.argtypes = [_P, _I, _I, _P, _I, _P, _I, _I, _I, _I, _I, _P]
        o.distie_head_gate.argtypes = [_P, _I, _I, _I, _P, _I, _L, _P, _I, _I, _I, _P]
        o.distie_ssm_scan.argtypes = [_P, _I, _L, _P, _L, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P]
        o.distie_ssm_scan_chunked.argtypes = [_P, _I, _L, _P, _L, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I,
                                              _I, _I, _P]
        o.distie_gate_rmsnorm.argtypes = [_P, _P, _I, _F, _P, _I, _L, _P, _I, _I, _I, _I, _I, _P]
        o.distie_glu_mul.argtypes = [_P, _I, _I, _P, _I, _I, _I, _I, _F, _F, _F, _P]
        o.distie_group_chain.argtypes = [_P, _I, _I, _P, _F, _I, _P, _P, _P, _P, _I, _P, _P, _I, _I, _I, _P, _I, _P, _P, _P]
        o.distie_token_shift.argtypes = [_P, _I, _P, _I, _P, _P, _P, _P, _P, _I, _I, _P]
        o.distie_wkv_scan.argtypes = [_P, _P, _P, _P, _I, _L, _P, _I, _L, _I, _P, _P, _P, _P, _P, _F, _P, _I, _P, _P, _I, _I,
                                      _I, _P]
        o.distie_wkv_scan_chunked.argtypes = [_P, _P, _P, _P, _I, _L, _P, _P, _P, _P, _F, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I,
                                              _I, _P]
        o.distie_tanh_f32.argtypes = [_P, _L, _P, _I, _I, _P]
        o.distie_mixed_attention_generic.argtypes = [_P, _I, _L, _P, _P, _I, _P, _P, _P, _I, _P, _P, _I, _I, _I, _I, _I, _F,
                                                     _I, _I, _F, _P, _I, _P, _P, _P]
        o.distie_argmax.argtypes = [_P, _P, _I, _I, _P, _P, _P]
        o.distie_argmax_parts.argtypes = [_I, _I]
        o.distie_sample.argtypes = [_P, _P, _P, _P, _P, _I, _I, _P, _P, _P, _P]

    def tune_library_products(self, on: bool) -> None:
        """While on, every new shape of a large product has the library's candidate kernels timed, and the
        fastest is kept for that shape, and for the other row counts of its class of 32 rows, from then on; shapes
        first met while off take their class's choice, or the library's first. Products of up to `PACKED_MAX_ROWS`
        rows do not go to the library at all (`PACKED_MAX_ROWS_EAGER` outside captured steps; large weights:
        see there). The caller that has had every class up to some number of rows timed says so in
        `library_timed_rows`: up to there large weights with more rows than K leave the packed kernels at 65 rows."""
        self._tuning = bool(on)

    def graphs_supported(self) -> bool:
        """Every kernel launches on torch's current stream and keeps its scratch at fixed
        addresses, so a step can be captured into a HIP graph."""
        return True

    def _stream(self):
        # torch's current stream as a raw handle; the direct getter saves the 4 us a call that building a
        # Stream object costs (a step makes some 200 calls)
        if _raw_stream is not None:
            return _raw_stream(self._device_index)
        return torch.cuda.current_stream(self.device).cuda_stream

    def attention_library(self, head_dim: int) -> ctypes.CDLL:
        lib = self._attn.get(head_dim)
        if lib is None:
            if head_dim % 2 or not 2 <= head_dim <= self.LARGEST_HEAD:
                raise KernelError(f"attention kernels take even head sizes up to {self.LARGEST_HEAD}, not {head_dim}")
            lib = ctypes.CDLL(str(build.ensure(f"attn_d{head_dim}")))
            lib.distie_attention_generic.argtypes = [_P, _I, _L, _P, _P, _I, _P, _P, _P, _I, _P, _P,
                                                     _I, _I, _I, _I, _F, _I, _P, _F, _P, _P]
            lib.distie_attention_prefill_bf16.argtypes = [_P, _L, _P, _P, _P, _P, _P, _I, _P, _P, _I, _I, _I, _I, _I,
                                                          _F, _I, _I, _P, _P, _P, _I, _P, _P]
            lib.distie_attention_prefill_f32.argtypes = lib.distie_attention_prefill_bf16.argtypes
            lib.distie_attention_decode_bf16.argtypes = [_P, _L, _P, _P, _P, _P, _P, _I, _P, _P, _P, _P, _I, _I, _I,
                                                         _I, _F, _I, _I, _I, _I, _P, _P, _P]
            lib.distie_attention_decode_run_len.argtypes = [_P, _I, _I, _I, _P, _P]
            if lib.distie_attention_head_dim() != head_dim:
                raise KernelError("attention library was built for another head size")
            self._attn[head_dim] = lib
        return lib

    def mixed_attention_library(self, head_dim: int) -> ctypes.CDLL:
        lib = self._mixed.get(head_dim)
        if lib is None:
            lib = ctypes.CDLL(str(build.ensure(f"mixattn_d{head_dim}")))
            lib.distie_mixed_fits.argtypes = [_I, _I]
            lib.distie_mixed_attention_bf16.argtypes = [_P, _L, _P, _P, _P, _P, _P, _I, _P, _P, _I, _I, _I, _I, _I, _F, _I, _I,
                                                        _F, _P, _I, _P, _P, _I, _I, _I, _I, _P, _P, _P]
            if lib.distie_mixed_head_dim() != head_dim:
                raise KernelError("the library of attention with mixed heads was built for another head size")
            self._mixed[head_dim] = lib
        return lib

    def _own(self, *tensors) -> None:
        for t in tensors:
            if t is None:
                continue
            if t.device != self.device:
                raise KernelError(f"tensor on {t.device}, kernels run on {self.device}")
            if not t.is_contiguous():
                raise KernelError("kernels take contiguous tensors")

    @staticmethod
    def _check_cache(k_cache, v_cache, kv_heads, block_size, head_dim) -> None:
        if tuple(k_cache.shape[1:]) != (kv_heads, block_size, head_dim) or \
                tuple(v_cache.shape[1:]) != (kv_heads, head_dim, block_size) or k_cache.shape[0] != v_cache.shape[0]:
            raise KernelError("cache is not k [pages, kv_heads, block_size, head_dim], "
                              "v [pages, kv_heads, head_dim, block_size]")

    # ------------------------------------------------------------ operations
    def scatter_int32(self, table, index, value):
        self._own(table, index, value)
        if table.dtype != torch.int32 or index.dtype != torch.int32 or value.dtype != torch.int32 or \
                index.shape != value.shape:
            raise KernelError("scatter_int32 takes int32 tensors, one value for each index")
        _check(self._ops.distie_scatter_i32(table.data_ptr(), index.data_ptr(), value.data_ptr(), index.numel(),
                                            table.numel(), self._stream()), "scatter_i32")
        _mark_written(table)

    def embed(self, ids, table, scale=1.0):
        self._own(ids, table)
        out = torch.empty((ids.shape[0], table.shape[1]), dtype=torch.float32, device=self.device)
        _check(self._ops.distie_embed(ids.data_ptr(), table.data_ptr(), _code(table), out.data_ptr(),
                                      ids.shape[0], table.shape[1], table.shape[0], float(scale), self._stream()), "embed")
        return out

    def _norm_later(self, residual, weight, out_dtype) -> bool:
        """The norm of these rows can be left to the product that reads it."""
        return (self.packed_weights and self._fused(residual.shape[0]) and out_dtype == torch.bfloat16 and
                residual.dtype == torch.float32 and residual.dim() == 2 and
                weight.dtype in _CODES and bool(self._ops.distie_decode_norm_fits(residual.shape[1])))

    def _fused(self, rows: int) -> bool:
        return rows <= self.FUSED_MAX_ROWS and (self.FUSED_IN_CAPTURED_STEPS or not self.captured)

    def rmsnorm(self, x, weight, eps, out_dtype):
        self._own(x, weight)
        if x.dtype != torch.float32:
            raise KernelError("rmsnorm reads the float32 residual stream")
        if self._norm_later(x, weight, out_dtype):
            return PendingNorm(x, weight, eps, out_dtype)
        return self._rmsnorm_now(x, weight, eps, out_dtype)

    def _rmsnorm_now(self, x, weight, eps, out_dtype):
        out = torch.empty(x.shape, dtype=out_dtype, device=self.device)
        _check(self._ops.distie_rmsnorm(x.data_ptr(), None, _F32, 1, weight.data_ptr(), _code(weight),
                                        out.data_ptr(), _CODES[out_dtype], x.shape[0], x.shape[1], eps,
                                        self._stream()), "rmsnorm")
        return out

    def add_rmsnorm(self, residual, delta, weight, eps, out_dtype):
        if isinstance(delta, PendingProduct):
            self._own(residual, weight)
            if residual.dtype != torch.float32 or residual.shape != delta.shape:
                raise KernelError("add_rmsnorm: residual must be float32 and shaped like delta")
            # the product adds itself to the stream; what is left is the norm of the stream
            self._product_into_residual(delta, residual)
            return self.rmsnorm(residual, weight, eps, out_dtype)
        slices = 1
        delta = self.dense(delta) if isinstance(delta, PendingNorm) else delta
        if isinstance(delta, PartialSums):
            slices, delta = delta.slices, delta.data
        self._own(residual, delta, weight)
        if residual.dtype != torch.float32 or residual.shape != delta.shape[-2:]:
            raise KernelError("add_rmsnorm: residual must be float32 and shaped like delta")
        out = torch.empty(residual.shape, dtype=out_dtype, device=self.device)
        _check(self._ops.distie_rmsnorm(residual.data_ptr(), delta.data_ptr(), _code(delta), slices,
                                        weight.data_ptr(), _code(weight), out.data_ptr(), _CODES[out_dtype],
                                        residual.shape[0], residual.shape[1], eps, self._stream()), "add_rmsnorm")
        _mark_written(residual)
        return out

    def _product_into_residual(self, product: PendingProduct, residual: torch.Tensor) -> None:
        x, weight, bias = product.x, product.weight, product.bias
        packed = getattr(weight, "_distie_packed")
        M, K = x.shape
        N = weight.shape[0]
        if packed.numel() != self._packed_elements(N, K, False):
            raise KernelError("linear: the packed copy does not belong to this weight")
        _check(self._ops.distie_decode_product_residual(
            x.data_ptr(), packed.data_ptr(), bias.data_ptr() if bias is not None else None, residual.data_ptr(),
            M, N, K, self._stream()), "decode_product_residual")
        _mark_written(residual)

    def dense(self, x):
        """The finished tensor of a value that an operation here returned in a form of its own (partial sums,
        a norm or a product that was left for later); any other tensor as it is."""
        if isinstance(x, PendingNorm):
            x.check()
            return self._rmsnorm_now(x.residual, x.weight, x.eps, x.dtype)
        if isinstance(x, PendingProduct):
            return self._linear(x.x, x.weight, x.bias, x.dtype, lazy=False)
        if isinstance(x, NormedSum):
            return self._norm_chain(x.terms, x.weights, x.eps, x.scale, None, None, None, None)
        if not isinstance(x, PartialSums):
            return x
        out = torch.empty(tuple(x.shape), dtype=x.dtype, device=self.device)
        _check(self._ops.distie_sum_slices(x.data.data_ptr(), x.slices, out.numel(), out.data_ptr(),
                                           _CODES[x.dtype], self._stream()), "sum_slices")
        return out

    # ---- packed copies of weights: tiles of 16 rows x 32 k in the matrix cores' lane order
    @staticmethod
    def _row_map(N, gated, rotary):
        """Which row of the weight sits at each place of the packed copy's row blocks (-1: zeros)."""
        if gated:
            inter = N // 2
            j = torch.arange(-(-inter // 8) * 8, dtype=torch.int64).view(-1, 8)
            gate = torch.where(j < inter, j, -1)
            up = torch.where(j < inter, j + inter, -1)
            return torch.cat([gate, up], dim=1).reshape(-1)
        if rotary is not None:
            heads, kv_heads, dim = rotary
            lo = torch.arange(dim // 2, dtype=torch.int64).view(-1, 8)                 # [dim/16, 8]
            one = torch.cat([lo, lo + dim // 2], dim=1).reshape(-1)                   # rows of a q or k head
            turned = (torch.arange(heads + kv_heads, dtype=torch.int64)[:, None] * dim + one[None, :]).reshape(-1)
            return torch.cat([turned, torch.arange((heads + kv_heads) * dim, N, dtype=torch.int64)])
        rows = torch.full((-(-N // 16) * 16,), -1, dtype=torch.int64)
        rows[:N] = torch.arange(N)
        return rows

    @staticmethod
    def _packed_elements(N, K, gated):
        row_blocks = -(-(N // 2) // 8) if gated else -(-N // 16)
        return row_blocks * -(-K // 32) * 512

    def prepare_linear(self, weight, gated=False, rotary=None, role=None):
        if self.packed_roles is not None and role not in self.packed_roles:
            return
        if not self.packed_weights or weight.dtype != torch.bfloat16 or weight.dim() != 2 or weight.shape[1] % 8:
            return
        N, K = weight.shape
        name = "_distie_packed"
        if gated:
            if N % 2:
                return
            name = "_distie_gated"
        elif rotary is not None:
            heads, kv_heads, dim = rotary
            if dim % 16 or N != (heads + 2 * kv_heads) * dim:
                rotary = None                 # the fused kernel does not take it: the plain copy serves
            else:
                name = "_distie_rotary"
        if hasattr(weight, name):
            return
        self._own(weight)
        row_map = self._row_map(N, gated, rotary)
        if row_map.numel() % 16 or int(row_map.max()) >= N or int(row_map.min()) < -1 or \
                row_map.numel() // 16 * -(-K // 32) * 512 != self._packed_elements(N, K, gated):
            raise KernelError("prepare_linear: bad row map")
        # The copies are for speed, the cache is needed: a copy that would leave less than PACKED_KEEPS_FREE of the
        # card's memory free is left out (the product then streams the stored layout), said once.
        free, total = torch.cuda.mem_get_info(self.device)
        if free - 2 * self._packed_elements(N, K, gated) < self.PACKED_KEEPS_FREE * total:
            if not self._packed_left_out:
                _log.warning("packed weight copies are left out from here on: less than %.0f %% of the device's "
                             "memory would stay free", 100 * self.PACKED_KEEPS_FREE)
            self._packed_left_out += 1
            return
        row_map = row_map.to(device=self.device, dtype=torch.int32)
        packed = torch.empty(self._packed_elements(N, K, gated), dtype=torch.bfloat16, device=self.device)
        _check(self._ops.distie_pack_rows(weight.data_ptr(), packed.data_ptr(), row_map.data_ptr(),
                                          row_map.numel() // 16, K, self._stream()), "pack_rows")
        torch.cuda.current_stream(self.device).synchronize()      # row_map is freed on return
        # the copy lives and dies with the weight
        setattr(weight, name, (packed, tuple(rotary)) if name == "_distie_rotary" else packed)

    def _norm_product(self, x: PendingNorm, packed, bias, out, mode, N, rotary=None):
        """`out` = the product of rmsnorm(x.residual) with the weight whose packed copy is `packed`, the norm
        computed inside the product."""
        x.check()
        M, K = x.shape
        table = slots = k_cache = v_cache = None
        heads = kv_heads = dim = block_size = write = 0
        if rotary is not None:
            table, slots, k_cache, v_cache, heads, kv_heads, dim, block_size, write = rotary
        ptr = lambda t: t.data_ptr() if t is not None else None
        norm_weight = x.weight
        if norm_weight.dtype != torch.float32:
            # the kernel takes the norm's weights in float32 (a bfloat16 value is one exactly); kept on the tensor
            norm_weight = getattr(x.weight, "_distie_f32", None)
            if norm_weight is None:
                norm_weight = x.weight._distie_f32 = x.weight.float()
        _check(self._ops.distie_decode_norm_product(
            x.residual.data_ptr(), norm_weight.data_ptr(), x.eps, packed.data_ptr(), ptr(bias),
            out.data_ptr(), mode, M, N, K, ptr(table), ptr(slots), ptr(k_cache), ptr(v_cache), heads, kv_heads, dim,
            block_size, write, self._stream()), "decode_norm_product")
        return out

    def linear_silu_mul(self, x, gate_up_weight):
        return self.linear_glu(x, gate_up_weight, "silu")

    def linear_glu(self, x, gate_up_weight, kind):
        """The gated product with the activation in its epilogue, on the GATED copy of the weight (steps of few rows);
        else the product, then `glu_mul`."""
        if kind not in self.ACTIVATIONS:
            raise KernelError(f"linear_glu: no activation named {kind!r}")
        return self._linear_gated(x, gate_up_weight, 1 if kind == "silu" else 1 | ((self.ACTIVATIONS[kind] + 1) << 8),
                                  lambda product: self.glu_mul(product, kind))

    CLAMPED = 5                      # the clamped activation, as the packed products number what stands on the gate

    def linear_clamped_glu(self, x, gate_up_weight, limit, slope, up_shift):
        if not limit > 0:
            raise KernelError("linear_clamped_glu: the limit must be positive")
        return self._linear_gated(self.dense(x), gate_up_weight, 1 | (self.CLAMPED << 8),
                                  lambda product: self.clamped_glu(product, limit, slope, up_shift),
                                  (float(limit), float(slope), float(up_shift)))

    def _linear_gated(self, x, gate_up_weight, gated, apart, clamp=(0.0, 1.0, 0.0)):
        """`gated`: 1, and above the low eight bits what stands on the gate; `apart`: the same on a finished product."""
        packed = getattr(gate_up_weight, "_distie_gated", None)
        if isinstance(x, PendingNorm) and packed is not None and gate_up_weight.shape[1] == x.shape[1]:
            N, K = gate_up_weight.shape
            if packed.numel() != self._packed_elements(N, K, True):
                raise KernelError("linear_silu_mul: the packed copy does not belong to this weight")
            out = torch.empty((x.shape[0], N // 2), dtype=torch.bfloat16, device=self.device)
            return self._norm_product(x, packed, None, out, gated, N)
        x = self.dense(x)
        if packed is None or x.dtype != torch.bfloat16 or x.shape[0] > self._packed_rows(x.shape[0], *gate_up_weight.shape):
            return apart(self.linear(x, gate_up_weight))
        self._own(x)
        M, K = x.shape
        N = gate_up_weight.shape[0]
        if gate_up_weight.shape[1] != K:
            raise KernelError(f"linear: x is [{M}, {K}], weight is {list(gate_up_weight.shape)}")
        if packed.numel() != self._packed_elements(N, K, True):
            raise KernelError("linear_silu_mul: the packed copy does not belong to this weight")
        out = torch.empty((M, N // 2), dtype=x.dtype, device=self.device)
        if M <= self.ONE_WAVE_MAX_ROWS:
            _check(self._ops.distie_gemm_packed_bf16(x.data_ptr(), packed.data_ptr(), None, out.data_ptr(), _code(out),
                                                     M, N, K, gated, *clamp, self._stream()), "gemm_packed_bf16")
        else:
            _check(self._ops.distie_gemm_packed_wide_bf16(
                x.data_ptr(), packed.data_ptr(), None, out.data_ptr(), _code(out), M, N, K, gated,
                self._pass_blocks(M, N * K), *clamp, self._stream()), "gemm_packed_wide_bf16")
        return out

    def linear_rope_kv_write(self, x, weight, bias, meta, group, k_cache, v_cache, inv_freq, num_heads, num_kv_heads,
                             head_dim, write):
        held = getattr(weight, "_distie_rotary", None)
        if isinstance(x, PendingNorm) and held is not None and held[1] == (num_heads, num_kv_heads, head_dim) and \
                inv_freq is not None and 2 * inv_freq.shape[0] == head_dim and k_cache.dtype == torch.bfloat16 and \
                weight.shape[1] == x.shape[1]:
            packed = held[0]
            slots = meta.groups[group].slots
            self._own(bias, k_cache, v_cache, inv_freq, slots)
            M, K = x.shape
            N = weight.shape[0]
            if N != (num_heads + 2 * num_kv_heads) * head_dim:
                raise KernelError(f"linear: weight is {list(weight.shape)} for {num_heads} + 2 x {num_kv_heads} heads")
            if bias is not None and (bias.dtype != torch.float32 or bias.shape[0] != N):
                raise KernelError("linear: bias must be float32 [N]")
            if packed.numel() != self._packed_elements(N, K, False):
                raise KernelError("linear_rope_kv_write: the packed copy does not belong to this weight")
            self._check_cache(k_cache, v_cache, num_kv_heads, meta.block_size, head_dim)
            if M != meta.num_tokens or slots.shape[0] != M:
                raise KernelError("linear_rope_kv_write: rows do not match the batch")
            table = self._rope_table(meta, inv_freq)
            out = torch.empty((M, N), dtype=torch.bfloat16, device=self.device)
            return self._norm_product(x, packed, bias, out, 2, N, rotary=(
                table, slots, k_cache, v_cache, num_heads, num_kv_heads, head_dim, meta.block_size, 1 if write else 0))
        x = self.dense(x)
        fused = held is not None and held[1] == (num_heads, num_kv_heads, head_dim) and \
            x.dtype == torch.bfloat16 and x.shape[0] <= self._packed_rows(x.shape[0], *weight.shape) and \
            inv_freq is not None and 2 * inv_freq.shape[0] == head_dim and k_cache.dtype == torch.bfloat16
        if not fused:
            return self.rope_kv_write(self.linear(x, weight, bias), meta, group, k_cache, v_cache, inv_freq,
                                      num_heads, num_kv_heads, head_dim, write)
        packed = held[0]
        slots = meta.groups[group].slots
        self._own(x, bias, k_cache, v_cache, inv_freq, slots)
        M, K = x.shape
        N = weight.shape[0]
        if weight.shape[1] != K or N != (num_heads + 2 * num_kv_heads) * head_dim:
            raise KernelError(f"linear: x is [{M}, {K}], weight is {list(weight.shape)}")
        if bias is not None and (bias.dtype != torch.float32 or bias.shape[0] != N):
            raise KernelError("linear: bias must be float32 [N]")
        if packed.numel() != self._packed_elements(N, K, False):
            raise KernelError("linear_rope_kv_write: the packed copy does not belong to this weight")
        self._check_cache(k_cache, v_cache, num_kv_heads, meta.block_size, head_dim)
        if M != meta.num_tokens or slots.shape[0] != M:
            raise KernelError("linear_rope_kv_write: rows do not match the batch")
        if M >= self.WIDE_QKV_MIN_ROWS and N * K > self.ROW_GROUPS_MAX_ELEMENTS:
            # more than one group of 16 rows against a weight that fills the chip through the wide kernel: the
            # epilogue kernel would read the weight once per group, so the product runs wide (weights once, K in
            # slices) and the rotation with the cache write behind it adds the slices
            slices = self._ops.distie_gemm_packed_wide_slices(N, K)
            shape, dtype = ((M, N), torch.bfloat16) if slices == 1 else ((slices, M, N), torch.float32)
            product = torch.empty(shape, dtype=dtype, device=self.device)
            _check(self._ops.distie_gemm_packed_wide_qkv_bf16(
                x.data_ptr(), packed.data_ptr(), bias.data_ptr() if bias is not None else None, product.data_ptr(),
                _code(product), M, K, num_heads, num_kv_heads, head_dim, self._pass_blocks(M, N * K), self._stream()),
                "gemm_packed_wide_qkv_bf16")
            if slices > 1:
                product = PartialSums(product, torch.bfloat16)
            return self.rope_kv_write(product, meta, group, k_cache, v_cache, inv_freq, num_heads, num_kv_heads,
                                      head_dim, write)
        table = self._rope_table(meta, inv_freq)
        out = torch.empty((M, N), dtype=torch.bfloat16, device=self.device)
        _check(self._ops.distie_gemm_packed_rotary_bf16(
            x.data_ptr(), packed.data_ptr(), bias.data_ptr() if bias is not None else None, out.data_ptr(),
            table.data_ptr(), slots.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), M, K, num_heads,
            num_kv_heads, head_dim, meta.block_size, 1 if write else 0, self._stream()), "gemm_packed_rotary_bf16")
        return out

    def _packed_rows(self, M: int, N: int, K: int) -> int:
        """Most rows of x that go through the kernels on the packed copy of an [N, K] weight, for a product of M rows."""
        if N * K > self.PACKED_LARGE_ELEMENTS:
            if K > N:
                return self.PACKED_MAX_ROWS_LARGE
            return self.PACKED_MAX_ROWS_LARGE_WIDE_TIMED if M <= self.library_timed_rows else self.PACKED_MAX_ROWS_LARGE_WIDE
        return self.PACKED_MAX_ROWS if self.captured else self.PACKED_MAX_ROWS_EAGER

    def _library(self):
        """The vendor library's products, called directly; loaded at the first large product."""
        if self._lib is None:
            lib = ctypes.CDLL(str(build.ensure("library")))
            lib.distie_lib_init.argtypes = [ctypes.c_int]
            lib.distie_lib_init.restype = ctypes.c_int
            lib.distie_lib_linear.argtypes = [_P, _P, _P, _P, ctypes.c_int, ctypes.c_int, ctypes.c_int, ctypes.c_int,
                                              ctypes.c_int, ctypes.c_int64, ctypes.c_int, _P]
            lib.distie_lib_linear.restype = ctypes.c_int
            lib.distie_lib_counts.argtypes = [ctypes.POINTER(ctypes.c_long), ctypes.POINTER(ctypes.c_long)]
            lib.distie_lib_counts.restype = None
            lib.distie_lib_more_counts.argtypes = [ctypes.POINTER(ctypes.c_long)] * 3
            lib.distie_lib_more_counts.restype = None
            with torch.cuda.device(self.device):
                _check(lib.distie_lib_init(self._device_index), "lib_init")
            self._lib = lib
        return self._lib

    def library_plans(self):
        """(shapes the library has a plan for, shapes whose kernel was chosen by timing)"""
        made, timed = ctypes.c_long(0), ctypes.c_long(0)
        self._library().distie_lib_counts(ctypes.byref(made), ctypes.byref(timed))
        return made.value, timed.value

    def library_counts(self) -> dict:
        """`held`: shapes the library holds a plan for now; `asked`: how often it was asked to rank its kernels
        (row counts of one class of 32 share a choice); `refused`: timed candidates dropped because their
        result differed from that of the library's first choice."""
        held, asked, refused = ctypes.c_long(0), ctypes.c_long(0), ctypes.c_long(0)
        self._library().distie_lib_more_counts(ctypes.byref(held), ctypes.byref(asked), ctypes.byref(refused))
        return {"held": held.value, "asked": asked.value, "refused": refused.value}

    LIBRARY_UNSUPPORTED = -3

    def _library_linear(self, x, weight, bias, out_dtype):
        """x [M, K] . weight [N, K]^T (+ float32 bias) by the library, float32 sums, into a new [M, N] of `out_dtype`.
        x and weight are both bfloat16, or both float32 (then every product is a float32 product). None if the
        library has no kernel for the product as asked."""
        M, K = x.shape
        N = weight.shape[0]
        if x.stride(1) != 1 or x.stride(0) != K:
            x = x.contiguous()
        if weight.stride(1) != 1 or weight.stride(0) != K:
            weight = weight.contiguous()
        out = torch.empty((M, N), dtype=out_dtype, device=self.device)
        lib = self._library()
        code, size, w_size = _CODES[out_dtype], out.element_size(), weight.element_size()
        # The library's large bfloat16 kernels work on tiles of 256 x 256, one a compute unit at a time: a product
        # with a few tiles more than a whole number of rounds pays a full round for them (at 2,048 rows 16,384
        # columns take 82 us and 17,920 take 116). The last columns as a product of their own cost less (20 us
        # for 1,536), written into the same output.
        tail = self._library_tail(M, N) if out_dtype == torch.bfloat16 else 0
        for lo, hi in (((0, N - tail), (N - tail, N)) if tail else ((0, N),)):
            rc = lib.distie_lib_linear(
                x.data_ptr(), weight.data_ptr() + lo * K * w_size, bias.data_ptr() + lo * 4 if bias is not None else None,
                out.data_ptr() + lo * size, _code(x), code, M, hi - lo, K, N, 1 if self._tuning else 0, self._stream())
            if rc == self.LIBRARY_UNSUPPORTED:
                return None
            _check(rc, "lib_linear")
        return out

    LIBRARY_TILE = 256

    def _library_tail(self, M: int, N: int) -> int:
        """How many of the last columns of a large library product to run as a product of their own: those
        beyond the last whole round of tiles over the compute units, if they are few (at most a quarter of a
        round) and there is at least one whole round before them; else 0."""
        tile = self.LIBRARY_TILE
        row_tiles = -(-M // tile)
        if row_tiles > self._compute_units:
            return 0
        round_columns = self._compute_units // row_tiles * tile
        tail = N % round_columns
        if N < round_columns or tail == 0 or tail > round_columns // 4 or tail % 8:
            return 0
        return tail

    def _pass_blocks(self, rows: int, elements: int) -> int:
        """Blocks of 16 rows of x per pass of the wide product over a weight of `elements` (0: one pass)."""
        if elements > self.TWO_PASS_MAX_ELEMENTS:
            if rows <= 64:
                return 0
            blocks = -(-rows // 16)
            passes = -(-blocks // self.WIDE_PASS_MAX_BLOCKS)
            return -(-blocks // passes)
        # (a single pass takes at most 64 rows; beyond 128 rows passes of 48 were 5 % faster than of 32 or 64)
        return 0 if rows <= 32 else (2 if rows <= 128 else 3)

    def _rope_table(self, meta, inv_freq):
        """Cosines and sines of the step's positions, float32 [T, pairs, 2]: computed by the first layer
        that asks, used by all."""
        pairs = inv_freq.shape[0]
        key = ("rope", inv_freq.data_ptr(), pairs)
        table = meta.scratch.get(key)
        if table is None:
            table = torch.empty((meta.num_tokens, pairs, 2), dtype=torch.float32, device=self.device)
            _check(self._ops.distie_rope_table(meta.positions.data_ptr(), inv_freq.data_ptr(), table.data_ptr(),
                                               meta.num_tokens, pairs, self._stream()), "rope_table")
            meta.scratch[key] = table
        return table

    def _linear(self, x, weight, bias, out_dtype, partial_ok=False, lazy=False):
        packed = getattr(weight, "_distie_packed", None)
        if isinstance(x, PendingNorm) and out_dtype == torch.float32 and bias is None and packed is not None and \
                weight.shape[1] == x.shape[1] and weight.dtype == torch.bfloat16:
            # the head behind the final norm
            N, K = weight.shape
            if packed.numel() != self._packed_elements(N, K, False):
                raise KernelError("linear: the packed copy does not belong to this weight")
            out = torch.empty((x.shape[0], N), dtype=torch.float32, device=self.device)
            return self._norm_product(x, packed, None, out, 0, N)
        x = self.dense(x)
        self._own(x, weight, bias)
        M, K = x.shape
        N = weight.shape[0]
        if weight.shape[1] != K:
            raise KernelError(f"linear: x is [{M}, {K}], weight is {list(weight.shape)}")
        if bias is not None and (bias.dtype != torch.float32 or bias.shape[0] != N):
            raise KernelError("linear: bias must be float32 [N]")
        both_bf16 = x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16
        packed = packed if both_bf16 else None
        if lazy and packed is not None and self._fused(M) and K % 8 == 0 and out_dtype == torch.bfloat16:
            return PendingProduct(x, weight, bias)
        if packed is not None and self.ONE_WAVE_MAX_ROWS < M <= self._packed_rows(M, N, K) and K % 8 == 0 and \
                N * K > self.ROW_GROUPS_MAX_ELEMENTS:
            if packed.numel() != self._packed_elements(N, K, False):
                raise KernelError("linear: the packed copy does not belong to this weight")
            slices = self._ops.distie_gemm_packed_wide_slices(N, K)
            if slices == 1:
                out = torch.empty((M, N), dtype=out_dtype, device=self.device)
            else:
                out = torch.empty((slices, M, N), dtype=torch.float32, device=self.device)
            _check(self._ops.distie_gemm_packed_wide_bf16(
                x.data_ptr(), packed.data_ptr(), bias.data_ptr() if bias is not None else None, out.data_ptr(),
                _code(out), M, N, K, 0, self._pass_blocks(M, N * K), 0.0, 1.0, 0.0, self._stream()),
                "gemm_packed_wide_bf16")
            if slices == 1:
                return out
            return PartialSums(out, out_dtype) if partial_ok else self.dense(PartialSums(out, out_dtype))
        if both_bf16 and K % 8 == 0 and (M <= self.SKINNY_MAX_ROWS or (packed is not None and M <= self._packed_rows(M, N, K))):
            if packed is not None:
                if packed.numel() != self._packed_elements(N, K, False):
                    raise KernelError("linear: the packed copy does not belong to this weight")
            slices = self._ops.distie_gemm_skinny_slices(M, N, K)       # the same cut for both kernels
            if slices == 1:
                out = torch.empty((M, N), dtype=out_dtype, device=self.device)
            else:
                out = torch.empty((slices, M, N), dtype=torch.float32, device=self.device)
            if packed is not None:
                _check(self._ops.distie_gemm_packed_bf16(
                    x.data_ptr(), packed.data_ptr(), bias.data_ptr() if bias is not None else None, out.data_ptr(),
                    _code(out), M, N, K, 0, 0.0, 1.0, 0.0, self._stream()), "gemm_packed_bf16")
            else:
                _check(self._ops.distie_gemm_skinny_bf16(
                    x.data_ptr(), weight.data_ptr(), bias.data_ptr() if bias is not None else None, out.data_ptr(),
                    _code(out), M, N, K, self._stream()), "gemm_skinny_bf16")
            if slices == 1:
                return out
            return PartialSums(out, out_dtype) if partial_ok else self.dense(PartialSums(out, out_dtype))
        if both_bf16:
            # large bfloat16 product: the library's matrix-core kernels
            out = self._library_linear(x, weight, bias, out_dtype)
            if out is None:
                # no kernel of the library's for this product as asked for: through torch, which knows more ways
                out = torch.mm(x, weight.t(), out_dtype=torch.float32)
                out = out if bias is None else out + bias
                out = out if out_dtype == torch.float32 else out.to(out_dtype)
            return out
        both_f32 = x.dtype == torch.float32 and weight.dtype == torch.float32 and out_dtype == torch.float32
        if both_f32 and M > self.ROWS_MAX_ROWS:
            # large float32 product: the library's float32 kernels (float32 products and sums); else the generic one
            out = self._library_linear(x, weight, bias, out_dtype)
            if out is not None:
                return out
        out = torch.empty((M, N), dtype=out_dtype, device=self.device)
        if M <= self.ROWS_MAX_ROWS and K % 8 == 0:
            # few rows in float32 (or against a weight kept in float32): the weights are streamed, FMAs only
            _check(self._ops.distie_gemv_rows(
                x.data_ptr(), _code(x), weight.data_ptr(), _code(weight), bias.data_ptr() if bias is not None else None,
                out.data_ptr(), _CODES[out_dtype], M, N, K, self._stream()), "gemv_rows")
            return out
        _check(self._ops.distie_gemm_generic(
            x.data_ptr(), _code(x), weight.data_ptr(), _code(weight), bias.data_ptr() if bias is not None else None,
            out.data_ptr(), _CODES[out_dtype], M, N, K, self._stream()), "gemm_generic")
        return out

    def linear(self, x, weight, bias=None):
        """May return `PartialSums` (see there)."""
        return self._linear(x, weight, bias, x.dtype, partial_ok=True, lazy=True)

    def linear_dense(self, x, weight, bias=None):
        """Steps of up to ONE_WAVE_MAX_ROWS rows: the packed product with the whole K in one workgroup, which writes the
        finished values (cut into slices, a kernel that adds them up would have to follow)."""
        x = self.dense(x)
        packed = getattr(weight, "_distie_packed", None)
        M, K = x.shape
        N = weight.shape[0]
        if packed is None or x.dtype != torch.bfloat16 or M > self.ONE_WAVE_MAX_ROWS or K % 8 or weight.shape[1] != K:
            return self.dense(self.linear(x, weight, bias))
        self._own(x, bias)
        if bias is not None and (bias.dtype != torch.float32 or bias.shape[0] != N):
            raise KernelError("linear: bias must be float32 [N]")
        if packed.numel() != self._packed_elements(N, K, False):
            raise KernelError("linear: the packed copy does not belong to this weight")
        out = torch.empty((M, N), dtype=x.dtype, device=self.device)
        _check(self._ops.distie_gemm_packed_bf16(
            x.data_ptr(), packed.data_ptr(), bias.data_ptr() if bias is not None else None, out.data_ptr(), _code(out), M, N, K,
            2, 0.0, 1.0, 0.0, self._stream()), "gemm_packed_bf16")
        return out

    def linear_f32out(self, x, weight, bias=None, scale=1.0, partial=False):
        if partial and scale == 1.0:
            return self._linear(x, weight, bias, torch.float32, partial_ok=True)
        out = self._linear(x, weight, bias, torch.float32)
        if scale != 1.0:
            _check(self._ops.distie_scale_f32(out.data_ptr(), out.numel(), float(scale), self._stream()), "scale_f32")
        return out

    def rope_kv_write(self, qkv, meta: BatchMeta, group, k_cache, v_cache, inv_freq, num_heads, num_kv_heads,
                      head_dim, write):
        if isinstance(qkv, (PendingNorm, PendingProduct)):
            qkv = self.dense(qkv)
        slices, source = 1, qkv
        if isinstance(qkv, PartialSums):
            slices, source = qkv.slices, qkv.data
            out = torch.empty(tuple(qkv.shape), dtype=qkv.dtype, device=self.device)
        else:
            out = qkv
        self._own(source, k_cache, v_cache, inv_freq)
        T = out.shape[0]
        if out.shape[1] != (num_heads + 2 * num_kv_heads) * head_dim:
            raise KernelError("rope_kv_write: qkv width does not match the head counts")
        self._check_cache(k_cache, v_cache, num_kv_heads, meta.block_size, head_dim)
        if T != meta.num_tokens:
            raise KernelError("rope_kv_write: qkv rows do not match the batch")
        pairs = 0 if inv_freq is None else inv_freq.shape[0]
        slots = meta.groups[group].slots
        table = self._rope_table(meta, inv_freq) if pairs else None
        _check(self._ops.distie_rope_kv_write(
            source.data_ptr(), _code(source), slices, out.data_ptr(), _code(out),
            table.data_ptr() if table is not None else None, meta.positions.data_ptr(),
            slots.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), _code(k_cache),
            inv_freq.data_ptr() if inv_freq is not None else None, pairs, T, num_heads, num_kv_heads, head_dim,
            meta.block_size, 1 if write else 0, self._stream()), "rope_kv_write")
        _mark_written(out)
        return out

    def paged_attention(self, qkv, meta: BatchMeta, group, k_cache, v_cache, num_heads, num_kv_heads, head_dim,
                        scale, window, extras=None):
        """The matrix-core kernels and the tiled float32 kernel compute attention with plain scores (a sink in the
        denominator they take, and chunks instead of a window); a step whose `extras` bend the scores goes to the
        wave-per-token kernel, which takes slopes and a cap as well (any types and sizes)."""
        if not scale > 0:
            raise KernelError(f"paged_attention: the scale of the scores must be positive, not {scale}")
        qkv = self.dense(qkv)
        self._own(qkv, k_cache, v_cache)
        T = qkv.shape[0]
        table = meta.groups[group].block_table
        self._check_cache(k_cache, v_cache, num_kv_heads, meta.block_size, head_dim)
        rows = meta.table_rows
        if T != meta.num_tokens or (rows is None and table.shape[0] != meta.num_requests) or \
                (rows is not None and rows.shape[0] != meta.num_requests):
            raise KernelError("paged_attention: tensors do not match the batch")
        rows_ptr = rows.data_ptr() if rows is not None else None
        out = torch.empty((T, num_heads * head_dim), dtype=qkv.dtype, device=self.device)
        plain = extras is None or not extras.bends_scores
        slopes, cap = (None, 0.0) if plain else (extras.head_slopes, float(extras.score_cap or 0.0))
        sinks = extras.sinks if extras is not None else None
        for name, vector in (("head_slopes", slopes), ("sinks", sinks)):
            if vector is not None:
                self._own(vector)
                if vector.dtype != torch.float32 or tuple(vector.shape) != (num_heads,):
                    raise KernelError(f"paged_attention: {name} must be float32 [num_heads]")
        sinks_ptr = sinks.data_ptr() if sinks is not None else None
        chunk = extras.chunk if extras is not None else 0
        if chunk and (window or extras.mixes_heads):
            raise KernelError("paged_attention: chunks do not go with a window or with mixed heads")
        reach = -int(chunk) if chunk else int(window or 0)       # as the kernels take it: a window, or minus the chunks' size
        if extras is not None and extras.mixes_heads:
            self._mixed_attention(qkv, meta, table, rows_ptr, k_cache, v_cache, out, num_heads, num_kv_heads, head_dim, scale,
                                  window, extras)
            return out
        lib = self.attention_library(head_dim)
        bf16 = qkv.dtype == torch.bfloat16 and k_cache.dtype == torch.bfloat16
        if plain and bf16 and meta.block_size % 16 == 0 and head_dim % 16 == 0 and head_dim <= self.LARGEST_MATRIX_CORE_HEAD:
            # how the step is launched, and its buffers for partial results, are the same for every layer
            # with these sizes: worked out once per step (the layers run one after the other, so they can
            # share the buffers)
            key = ("attention", reach, num_heads, num_kv_heads, head_dim, meta.max_kv, meta.all_decode,
                   meta.singles_bound, self.PREFILL_PARTS, self.PREFILL_WORKGROUPS, self.DECODE_WAVES, self.DECODE_MAX_RUNS,
                   self.DECODE_SHARED_BELOW)
            plan = meta.scratch.get(key)
            if plan is None or plan["cu_q"] is not meta.host_cu_q:
                plan = meta.scratch[key] = self._attention_plan(lib, meta, T, num_heads, num_kv_heads, head_dim, abs(reach))
            if plan["decode"]:
                _check(lib.distie_attention_decode_bf16(
                    qkv.data_ptr(), qkv.shape[1], k_cache.data_ptr(), v_cache.data_ptr(), meta.kv_len.data_ptr(),
                    meta.cu_q.data_ptr(), table.data_ptr(), table.shape[1], rows_ptr, out.data_ptr(),
                    plan["decode_o"].data_ptr(), plan["decode_ml"].data_ptr(), meta.num_requests, num_heads,
                    num_kv_heads, meta.block_size, float(scale), reach, plan["split_len"],
                    plan["max_splits"], 1 if meta.all_decode else 0,
                    plan["run_len"].data_ptr() if plan["run_len"] is not None else None, sinks_ptr, self._stream()),
                    "attention_decode_bf16")
            if plan["prefill"]:
                parts = plan["parts"]
                _check(lib.distie_attention_prefill_bf16(
                    qkv.data_ptr(), qkv.shape[1], k_cache.data_ptr(), v_cache.data_ptr(), meta.positions.data_ptr(),
                    meta.cu_q.data_ptr(), table.data_ptr(), table.shape[1], rows_ptr, out.data_ptr(), T, meta.num_requests,
                    num_heads, num_kv_heads, meta.block_size, float(scale), reach,
                    2 if plan["decode"] else 1, meta.token_request.data_ptr(),
                    plan["prefill_o"].data_ptr() if parts > 1 else None,
                    plan["prefill_ml"].data_ptr() if parts > 1 else None, parts, sinks_ptr, self._stream()),
                    "attention_prefill_bf16")
            return out
        f32 = qkv.dtype == torch.float32 and k_cache.dtype == torch.float32
        if plain and f32 and meta.max_q >= self.PREFILL_F32_MIN_TOKENS and meta.block_size % 16 == 0 and \
                qkv.shape[1] % 4 == 0 and lib.distie_attention_prefill_f32_fits():
            # portions of prompts in float32: the tiled kernel on float32 matrix products takes the whole step
            key = ("attention_f32", reach, num_heads, head_dim, meta.max_kv, self.PREFILL_PARTS,
                   self.PREFILL_WORKGROUPS)
            plan = meta.scratch.get(key)
            if plan is None:
                plan = meta.scratch[key] = self._prefill_parts(meta, T, num_heads, head_dim, abs(reach))
            parts = plan["parts"]
            _check(lib.distie_attention_prefill_f32(
                qkv.data_ptr(), qkv.shape[1], k_cache.data_ptr(), v_cache.data_ptr(), meta.positions.data_ptr(),
                meta.cu_q.data_ptr(), table.data_ptr(), table.shape[1], rows_ptr, out.data_ptr(), T, meta.num_requests,
                num_heads, num_kv_heads, meta.block_size, float(scale), reach, 1,
                meta.token_request.data_ptr(), plan["prefill_o"].data_ptr() if parts > 1 else None,
                plan["prefill_ml"].data_ptr() if parts > 1 else None, parts, sinks_ptr, self._stream()),
                "attention_prefill_f32")
            return out
        _check(lib.distie_attention_generic(
            qkv.data_ptr(), _code(qkv), qkv.shape[1], k_cache.data_ptr(), v_cache.data_ptr(), _code(k_cache),
            meta.positions.data_ptr(), meta.token_request.data_ptr(), table.data_ptr(), table.shape[1], rows_ptr,
            out.data_ptr(), T, num_heads, num_kv_heads, meta.block_size, float(scale), reach,
            slopes.data_ptr() if slopes is not None else None, cap, sinks_ptr, self._stream()), "attention_generic")
        return out

    def _mixed_attention(self, q, meta: BatchMeta, table, rows_ptr, k_cache, v_cache, out, num_heads, num_kv_heads, head_dim,
                         scale, window, extras) -> None:
        """Attention for layers whose heads see each other's scores (csrc/mixed_attention.hip)."""
        if extras.head_slopes is not None:
            raise KernelError("paged_attention: slopes do not go with mixed heads")
        bias, mix = extras.distance_bias, extras.head_mix
        for name, t, rows in (("distance_bias", bias, num_heads), ("head_mix", mix, num_heads)):
            if t is not None:
                self._own(t)
                if t.dtype != torch.float32 or t.dim() != 2 or t.shape[0] != rows:
                    raise KernelError(f"paged_attention: {name} must be float32 with a row a head")
        if mix is not None and mix.shape[1] != num_heads:
            raise KernelError("paged_attention: head_mix must be [num_heads, num_heads]")
        if q.shape[1] != num_heads * head_dim:
            raise KernelError("paged_attention: mixed heads take q alone")
        ptr = lambda t: t.data_ptr() if t is not None else None
        keep = int(extras.keep_first) if window else 0
        if q.dtype == torch.bfloat16 and k_cache.dtype == torch.bfloat16 and meta.block_size % 16 == 0 and \
                head_dim % 32 == 0 and head_dim <= self.LARGEST_MATRIX_CORE_HEAD:
            lib = self.mixed_attention_library(head_dim)
            queries = lib.distie_mixed_fits(num_heads, num_kv_heads)
            if queries:
                key = ("mixed_attention", int(window or 0), keep, num_heads, head_dim, meta.max_kv, meta.all_decode,
                       meta.singles_bound)
                plan = meta.scratch.get(key)
                if plan is None or plan["cu_q"] is not meta.host_cu_q:
                    plan = meta.scratch[key] = self._mixed_plan(lib, meta, num_heads, head_dim, window, keep)
                if queries == 16 and q.shape[0] < self.MIXED_WIDE_TOKENS:
                    queries = 8
                _check(lib.distie_mixed_attention_bf16(
                    q.data_ptr(), q.shape[1], k_cache.data_ptr(), v_cache.data_ptr(), meta.positions.data_ptr(),
                    meta.cu_q.data_ptr(), table.data_ptr(), table.shape[1], rows_ptr, out.data_ptr(), q.shape[0],
                    meta.num_requests, num_heads, num_kv_heads, meta.block_size, float(scale), int(window or 0), keep,
                    float(extras.score_cap or 0.0), ptr(bias), bias.shape[1] if bias is not None else 0, ptr(mix),
                    ptr(extras.sinks), 1 if plan["prefill"] else 0, queries, (2 if meta.all_decode else 1) if plan["decode"] else 0, plan["splits"],
                    ptr(plan["partial_o"]), ptr(plan["partial_ml"]), self._stream()), "mixed_attention_bf16")
                return
        if not self._ops.distie_mixed_attention_fits(num_heads, head_dim):
            raise KernelError(f"paged_attention: {num_heads} mixed heads of {head_dim} do not fit the LDS of a compute unit")
        _check(self._ops.distie_mixed_attention_generic(
            q.data_ptr(), _code(q), q.shape[1], k_cache.data_ptr(), v_cache.data_ptr(), _code(k_cache),
            meta.positions.data_ptr(), meta.token_request.data_ptr(), table.data_ptr(), table.shape[1], rows_ptr,
            out.data_ptr(), q.shape[0], num_heads, num_kv_heads, head_dim, meta.block_size, float(scale), int(window or 0),
            keep, float(extras.score_cap or 0.0), ptr(bias), bias.shape[1] if bias is not None else 0, ptr(mix),
            ptr(extras.sinks), self._stream()), "mixed_attention_generic")

    def _mixed_plan(self, lib, meta: BatchMeta, num_heads, head_dim, window, keep) -> dict:
        """Which of the mixed heads' kernels a step needs, and the buffers for partial results of single tokens (one
        for every run of keys a token may see): the same for every layer with these sizes."""
        singles = meta.num_requests if meta.all_decode else 0
        if not meta.all_decode and meta.singles_bound is not None:
            singles = meta.singles_bound
        elif not meta.all_decode and meta.host_cu_q is not None:
            singles = int((meta.host_cu_q[1:] - meta.host_cu_q[:-1] == 1).sum())
        run = lib.distie_mixed_decode_keys()
        plan = {"cu_q": meta.host_cu_q, "decode": singles > 0, "splits": 0, "partial_o": None, "partial_ml": None,
                "prefill": singles < meta.num_requests or (meta.singles_bound is not None and not meta.all_decode)}
        if plan["decode"]:
            splits = -(-meta.max_kv // run)
            if window:
                splits = min(splits, -(-keep // run) + (int(window) + run - 2) // run + 1)
            plan["splits"] = max(1, splits)
            shape = (meta.num_requests, plan["splits"], num_heads)
            plan["partial_o"] = torch.empty((*shape, head_dim), dtype=torch.float32, device=self.device)
            plan["partial_ml"] = torch.empty((*shape, 2), dtype=torch.float32, device=self.device)
        return plan

    def _attention_plan(self, lib, meta: BatchMeta, T, num_heads, num_kv_heads, head_dim, window) -> dict:
        group = num_heads // num_kv_heads
        singles = meta.num_requests if meta.all_decode else 0
        if not meta.all_decode and meta.singles_bound is not None:
            # a captured step of portions and single tokens: which requests bring one token is known on the device
            # only; both kernels are launched for as many as there may be, and each leaves the other's requests alone
            singles = meta.singles_bound
        elif not meta.all_decode and meta.host_cu_q is not None:
            singles = int((meta.host_cu_q[1:] - meta.host_cu_q[:-1] == 1).sum())
        plan = {"cu_q": meta.host_cu_q, "decode": singles > 0 and group <= lib.distie_attention_decode_columns()}
        if plan["decode"]:
            # requests that bring one token: keys are cut into runs, one wave each, so that the chip is
            # filled even when few requests decode. The kernel cuts every request's visible keys (counted
            # from a 64-key boundary) into at most `max_splits` runs by the request's own length; the length
            # of the longest request's runs is passed along as a hint for the first lookups of pages.
            visible = min(meta.max_kv, int(window) + 63) if window else meta.max_kv
            max_splits = max(1, min(self.DECODE_MAX_RUNS, self.DECODE_WAVES // (singles * num_kv_heads),
                                    -(-visible // 64)))
            plan["split_len"] = -(-visible // (64 * max_splits)) * 64
            # every request with one token, no window, waves left over: one run length for all of them, so that a
            # long request gets more runs than a short one (up to twice what every request would get)
            plan["run_len"] = None
            pairs = singles * num_kv_heads
            if meta.all_decode and not window and max_splits * pairs <= self.DECODE_SHARED_BELOW * self.DECODE_WAVES:
                splits = max_splits
                max_splits = max(1, min(self.DECODE_MAX_RUNS, 2 * splits, -(-visible // 64)))
                plan["run_len"] = torch.empty(1, dtype=torch.int32, device=self.device)
                _check(lib.distie_attention_decode_run_len(meta.kv_len.data_ptr(), meta.num_requests,
                                                           max(1, self.DECODE_WAVES // num_kv_heads), max_splits,
                                                           plan["run_len"].data_ptr(), self._stream()),
                       "attention_decode_run_len")
            plan["max_splits"] = max_splits
            plan["decode_o"] = torch.empty((meta.num_requests, num_heads, max_splits, head_dim), dtype=torch.float32,
                                           device=self.device)
            plan["decode_ml"] = torch.empty((meta.num_requests, num_heads, max_splits, 2), dtype=torch.float32,
                                            device=self.device)
        plan["prefill"] = singles < meta.num_requests or not plan["decode"] or \
            (meta.singles_bound is not None and not meta.all_decode)
        if plan["prefill"]:
            plan.update(self._prefill_parts(meta, T, num_heads, head_dim, window))
        return plan

    def _prefill_parts(self, meta: BatchMeta, T, num_heads, head_dim, window) -> dict:
        """Into how many parts the tiled kernel cuts its walk over the keys, and the buffers between it and the
        merge. Portions of prompts (and single tokens too, if no other kernel took them): long walks over the
        keys are cut into parts that run side by side."""
        visible = min(meta.max_kv, int(window) + 128) if window else meta.max_kv
        parts = 1
        for keys, cut in self.PREFILL_PARTS:
            if visible >= keys:
                parts = cut
        # few new tokens make few workgroups (one per 128 tokens of a request and head), each walking all
        # the keys alone: more parts then, down to 128 keys a part
        tiles = -(-T // 128) + meta.num_requests
        wanted = -(-self.PREFILL_WORKGROUPS // (tiles * num_heads))
        parts = max(parts, min(wanted, visible // 128, 16))
        plan = {"parts": parts}
        if parts > 1:
            plan["prefill_o"] = torch.empty((parts, T, num_heads, head_dim), dtype=torch.float32, device=self.device)
            plan["prefill_ml"] = torch.empty((parts, T, num_heads, 2), dtype=torch.float32, device=self.device)
        return plan

    # ---- residual streams, convolutions over time, decayed states, gates (csrc/sequence.hip)
    def _rows_view(self, t: torch.Tensor, width: int):
        """(pointer, row stride) of a [T, width] tensor or column view whose rows are contiguous."""
        if t.device != self.device or t.dim() != 2 or t.shape[1] != width or (t.shape[1] > 1 and t.stride(1) != 1):
            raise KernelError("kernels take row views with contiguous columns on their own device")
        return t.data_ptr(), t.stride(0)

    NORM_KINDS = {"none": 0, "layer": 1, "rms": 2}
    # a step in which some request brings at least so many rows runs the decayed state in chunks of rows that are
    # worked side by side (three kernels) instead of row after row (one)
    SCAN_CHUNKED_MIN_ROWS = 16
    LRU_CHUNKED_MIN_ROWS = 128       # the same for the scan of a channel-wise recurrence (chunks of 64 rows, two kernels)
    ACTIVATIONS = {"relu2": 0, "silu": 1, "gelu_tanh": 2, "relu": 3}

    def hyper_step(self, streams, *, init=None, delta=None, gate=None, mix=None, write=None, read=None,
                   norm_weight=None, norm="none", eps=0.0, out_dtype=None):
        if norm not in self.NORM_KINDS:
            raise KernelError(f"no norm named {norm!r}")
        if init is not None:
            if streams is not None or mix is None and write is None and read is None:
                raise KernelError("hyper_step: `init` makes the streams; it needs their number from mix, write or read")
            self._own(init)
            count = (read if read is not None else write).shape[0]
            if init.dtype != torch.float32 or init.dim() != 2:
                raise KernelError("hyper_step: init must be float32 [T, C]")
            streams = torch.empty((init.shape[0], count, init.shape[1]), dtype=torch.float32, device=self.device)
        self._own(streams, mix, write, read, norm_weight)
        if streams.dtype != torch.float32 or streams.dim() != 3:
            raise KernelError("hyper_step: streams must be float32 [T, S, C]")
        T, S, C = streams.shape
        for name, t, shape in (("mix", mix, (S, S)), ("write", write, (S,)), ("read", read, (S,))):
            if t is not None and (t.dtype != torch.float32 or tuple(t.shape) != shape):
                raise KernelError(f"hyper_step: {name} must be float32 {list(shape)}")
        if init is not None and tuple(init.shape) != (T, C):
            raise KernelError("hyper_step: init does not match the streams")
        slices, y, y_code, g_ptr, g_code, g_ld, g_slices = 1, None, _F32, None, _F32, 0, 1
        if delta is not None:
            if mix is None or write is None:
                raise KernelError("hyper_step: a delta needs mix and write weights")
            if isinstance(delta, (PendingNorm, PendingProduct)):
                delta = self.dense(delta)
            if isinstance(delta, PartialSums):
                slices, delta = delta.slices, delta.data
            self._own(delta)
            if tuple(delta.shape[-2:]) != (T, C):
                raise KernelError("hyper_step: delta must be [T, C]")
            y, y_code = delta.data_ptr(), _code(delta)
            if gate is not None:
                if isinstance(gate, (PendingNorm, PendingProduct)):
                    gate = self.dense(gate)
                if isinstance(gate, PartialSums):
                    g_slices, gate = gate.slices, gate.data
                    self._own(gate)
                    if tuple(gate.shape[-2:]) != (T, C):
                        raise KernelError("hyper_step: the gate must be [T, C]")
                    g_ptr, g_ld = gate.data_ptr(), C
                else:
                    g_ptr, g_ld = self._rows_view(gate, C)
                g_code = _code(gate)
        h = None
        if read is not None:
            if norm != "none" and (norm_weight is None or tuple(norm_weight.shape) != (C,)):
                raise KernelError("hyper_step: the norm needs a weight [C]")
            h = torch.empty((T, C), dtype=out_dtype or torch.float32, device=self.device)
        ptr = lambda t: t.data_ptr() if t is not None else None
        _check(self._ops.distie_hyper_step(
            streams.data_ptr(), S, ptr(init), y, y_code, slices, g_ptr, g_code, g_ld, g_slices, ptr(mix), ptr(write), ptr(read),
            ptr(norm_weight), _code(norm_weight) if norm_weight is not None else _F32, self.NORM_KINDS[norm], float(eps),
            ptr(h), _code(h) if h is not None else _F32, T, C, self._stream()), "hyper_step")
        _mark_written(streams)
        return streams, h

    def causal_conv(self, x, weight, state, meta, residual=False, bias=None, act=None):
        if act is not None and act not in self.ACTIVATIONS:
            raise KernelError(f"causal_conv: no activation named {act!r}")
        x = self.dense(x)
        self._own(weight, state, bias)
        T, N = x.shape
        x_ptr, ldx = self._rows_view(x, N)
        taps = weight.shape[1]
        if tuple(weight.shape) != (N, taps) or T != meta.num_tokens:
            raise KernelError("causal_conv: weight must be [channels of x, taps], x the step's rows")
        if bias is not None and (bias.dtype != torch.float32 or tuple(bias.shape) != (N,)):
            raise KernelError("causal_conv: bias must be float32 [channels]")
        self._check_conv_state(state, taps, N)
        out = torch.empty((T, N), dtype=x.dtype, device=self.device)
        _check(self._ops.distie_causal_conv(
            x_ptr, _code(x), ldx, weight.data_ptr(), _code(weight), taps, state.data_ptr() if taps > 1 else None,
            out.data_ptr(), _code(out), N, (1 if residual else 0) | (0 if act is None else (self.ACTIVATIONS[act] + 1) << 1),
            bias.data_ptr() if bias is not None else None,
            meta.cu_q.data_ptr(), meta.token_request.data_ptr(), meta.state_slots.data_ptr(), T, N, self._stream()),
            "causal_conv")
        if taps > 1 and not meta.all_decode:
            # requests that bring one row moved their state on in the kernel above; the others here, once all
            # rows of the step have read the old one
            _check(self._ops.distie_conv_state(x_ptr, _code(x), ldx, taps, state.data_ptr(), meta.cu_q.data_ptr(),
                                               meta.state_slots.data_ptr(), meta.num_requests, N, 1, self._stream()),
                   "conv_state")
        if taps > 1:
            _mark_written(state)
        return out

    def _check_conv_state(self, state, taps, channels) -> None:
        if taps > 1 and (state is None or state.dtype != torch.float32 or tuple(state.shape[1:]) != (taps - 1, channels)):
            raise KernelError(f"the state of a convolution of {taps} taps over {channels} channels is float32 "
                              f"[slots, {taps - 1}, {channels}]")

    def conv_rope_kv_write(self, product, conv_weight, state, meta, group, k_cache, v_cache, inv_freq, magnitude,
                           num_heads, num_kv_heads, dim, value_dim, padded_dim, has_kv, write, q_temp=None, qk_norm=None,
                           keys_are_values=False, neighbours=False):
        # without a filter the kernel adds up a product's partial sums itself while it reads them
        slices, q_dtype = 1, None
        if isinstance(product, PartialSums) and conv_weight is None:
            slices, q_dtype, product = product.slices, product.dtype, product.data.view(-1, product.data.shape[-1])
        else:
            product = self.dense(product)
            q_dtype = product.dtype
        q_norm = k_norm = None
        norm_eps = 0.0
        if qk_norm is not None:
            q_norm, k_norm, norm_eps = qk_norm
            self._own(q_norm, k_norm)
            for weight in (q_norm, k_norm):
                if weight is not None and (weight.dtype != torch.float32 or tuple(weight.shape) != (dim,)):
                    raise KernelError("conv_rope_kv_write: the norms' weights of q and k are float32 [dim]")
            if q_norm is None or (has_kv and k_norm is None):
                raise KernelError("conv_rope_kv_write: a norm on the heads needs a weight for q, and for k where there are keys")
        self._own(product, conv_weight, state, k_cache, v_cache, inv_freq)
        T, W = product.shape[0] // slices, product.shape[1]
        if keys_are_values and (not has_kv or conv_weight is not None or value_dim != dim):
            raise KernelError("conv_rope_kv_write: values that are the keys go with keys, one head size and no filter")
        channels = num_heads * dim + (num_kv_heads * (dim if keys_are_values else dim + value_dim) if has_kv else 0)
        taps = 0 if conv_weight is None else conv_weight.shape[1]
        if T != meta.num_tokens or W < channels:
            raise KernelError("conv_rope_kv_write: the product does not match the batch or the head counts")
        if conv_weight is not None and tuple(conv_weight.shape) != (channels, taps):
            raise KernelError(f"conv_rope_kv_write: the filters must be [{channels}, taps]")
        self._check_conv_state(state, taps, channels)
        write = bool(write and has_kv)
        if write:
            self._check_cache(k_cache, v_cache, num_kv_heads, meta.block_size, padded_dim)
            if k_cache.dtype != v_cache.dtype:
                raise KernelError("conv_rope_kv_write: keys and values are cached in one dtype")
        pairs = 0 if inv_freq is None else inv_freq.shape[0]
        table = self._rope_table(meta, inv_freq) if pairs else None
        q = torch.empty((T, num_heads * padded_dim), dtype=q_dtype, device=self.device)
        ptr = lambda t: t.data_ptr() if t is not None else None
        _check(self._ops.distie_conv_rope_kv_write(
            product.data_ptr(), _code(product), W, ptr(conv_weight), _code(conv_weight) if conv_weight is not None else _F32,
            taps, ptr(state) if taps > 1 else None, ptr(table), pairs, float(magnitude), q.data_ptr(),
            ptr(k_cache) if write else None, ptr(v_cache) if write else None, _code(k_cache) if write else _code(product),
            meta.groups[group].slots.data_ptr() if write else None, meta.cu_q.data_ptr(), meta.token_request.data_ptr(),
            meta.state_slots.data_ptr(), T, num_heads, num_kv_heads, dim, value_dim, padded_dim, meta.block_size,
            2 if keys_are_values else (1 if has_kv else 0), 1 if write else 0, meta.positions.data_ptr(), float(q_temp[0]) if q_temp else 0.0,
            int(q_temp[1]) if q_temp else 0, ptr(q_norm), ptr(k_norm) if has_kv else None, float(norm_eps),
            slices, _CODES[q_dtype], 1 if neighbours else 0, self._stream()), "conv_rope_kv_write")
        if taps > 1:
            if not meta.all_decode:
                # (requests that bring one row had their state moved on by the kernel above)
                _check(self._ops.distie_conv_state(product.data_ptr(), _code(product), W, taps, state.data_ptr(),
                                                   meta.cu_q.data_ptr(), meta.state_slots.data_ptr(), meta.num_requests,
                                                   channels, 1, self._stream()), "conv_state")
            _mark_written(state)
        return q

    def sigmoid_gate(self, x, num_heads, head_stride, width, gates, per_head=False):
        x = self.dense(x)
        self._own(x)
        T = x.shape[0]
        if x.shape[1] != num_heads * head_stride or width > head_stride:
            raise KernelError("sigmoid_gate: x must be [T, heads * head_stride]")
        if per_head:
            if gates is None:
                raise KernelError("sigmoid_gate: a gate for each head needs the gates")
            g_ptr, g_ld = self._rows_view(gates, num_heads)
            out = torch.empty((T, num_heads * width), dtype=x.dtype, device=self.device)
            _check(self._ops.distie_head_gate(x.data_ptr(), _code(x), head_stride, width, g_ptr, _code(gates), g_ld,
                                              out.data_ptr(), _code(out), T, num_heads * width, self._stream()), "head_gate")
            return out
        g_ptr, g_ld = self._rows_view(gates, num_heads * width) if gates is not None else (None, 0)
        out = torch.empty((T, num_heads * width), dtype=x.dtype, device=self.device)
        _check(self._ops.distie_sigmoid_gate(x.data_ptr(), _code(x), head_stride, width, g_ptr,
                                             _code(gates) if gates is not None else _code(x), g_ld,
                                             out.data_ptr(), _code(out), T, num_heads * width, self._stream()),
               "sigmoid_gate")
        return out

    def _scan_chunks(self, meta, rows, num_heads, dim, value_dim):
        """Which rows of the step form a chunk of a state's scan, worked out from the step's row counts (known on the
        host outside captured steps): (number of chunks, the table {request, first row, rows, 0} with the first chunk
        of every request behind it, scratch for a state a chunk)."""
        table_key = ("scan_chunk_table", rows)
        held = meta.scratch.get(table_key)
        if held is None:
            cu = np.asarray(meta.host_cu_q, dtype=np.int64)
            table, first = [], [0]
            for b in range(meta.num_requests):
                for at in range(int(cu[b]), int(cu[b + 1]), rows):
                    table.append((b, at, min(rows, int(cu[b + 1]) - at), 0))
                first.append(len(table))
            packed = self.upload(np.concatenate([np.asarray(table, dtype=np.int32).reshape(-1),
                                                 np.asarray(first, dtype=np.int32)]))
            held = meta.scratch[table_key] = (len(table), packed)
        count, packed = held
        key = ("scan_chunks", rows, num_heads, dim, value_dim)
        scratch = meta.scratch.get(key)
        if scratch is None:
            scratch = meta.scratch[key] = torch.empty((count, num_heads, dim, value_dim), dtype=torch.float32,
                                                      device=self.device)
        return count, packed, scratch

    def decay_scan(self, product, state, decay, meta, num_heads, dim, value_dim, act="silu", k_scale=1.0, inv_freq=None,
                   neighbours=False):
        if act not in ("silu", None) or (act is not None and (inv_freq is not None or k_scale != 1.0)):
            raise KernelError("decay_scan: silu on q, k and v, or no activation with a rotation and a scale of k")
        product = self.dense(product)
        self._own(product, state, decay)
        T, W = product.shape
        if T != meta.num_tokens or W < num_heads * (2 * dim + value_dim):
            raise KernelError("decay_scan: the product does not match the batch or the head counts")
        if state.dtype != torch.float32 or tuple(state.shape[1:]) != (num_heads, dim, value_dim):
            raise KernelError("decay_scan: the state is float32 [slots, heads, dim, value_dim]")
        if decay.dtype != torch.float32 or tuple(decay.shape) != (num_heads,):
            raise KernelError("decay_scan: decay must be float32 [heads]")
        if dim > self._ops.distie_decay_scan_max_dim():
            raise KernelError(f"decay_scan: heads of up to {self._ops.distie_decay_scan_max_dim()} dimensions")
        pairs = 0 if inv_freq is None else inv_freq.shape[0]
        if 2 * pairs > dim:
            raise KernelError("decay_scan: the rotation turns more dimensions than a head has")
        table = self._rope_table(meta, inv_freq) if pairs else None
        turn = (1 if act else 0, table.data_ptr() if pairs else None, pairs, 1 if neighbours else 0, float(k_scale))
        out = torch.empty((T, num_heads * value_dim), dtype=torch.float32, device=self.device)
        if not self.captured and meta.host_cu_q is not None and meta.max_q >= self.SCAN_CHUNKED_MIN_ROWS and \
                dim <= self._ops.distie_decay_scan_chunked_max_dim():
            # portions of prompts: chunks of rows side by side instead of one row after the other. Which rows form
            # a chunk is worked out here from the step's row counts (known on the host outside captured steps).
            count, packed, scratch = self._scan_chunks(meta, self._ops.distie_decay_scan_chunk_rows(), num_heads, dim,
                                                       value_dim)
            _check(self._ops.distie_decay_scan_chunked(
                product.data_ptr(), _code(product), W, state.data_ptr(), decay.data_ptr(), out.data_ptr(),
                scratch.data_ptr(), packed.data_ptr(), packed.data_ptr() + 16 * count, meta.state_slots.data_ptr(),
                count, meta.num_requests, num_heads, dim, value_dim, *turn, self._stream()), "decay_scan_chunked")
            _mark_written(state)
            return out
        _check(self._ops.distie_decay_scan(product.data_ptr(), _code(product), W, state.data_ptr(), decay.data_ptr(),
                                           out.data_ptr(), meta.cu_q.data_ptr(), meta.state_slots.data_ptr(),
                                           meta.num_requests, num_heads, dim, value_dim, *turn, self._stream()),
               "decay_scan")
        _mark_written(state)
        return out

    def rmsnorm_gate(self, x, weight, eps, gates, out_dtype, group=None, gate="sigmoid", gate_first=False):
        self._own(x, weight)
        if gate not in ("sigmoid", "silu"):
            raise KernelError(f"rmsnorm_gate: no gate named {gate!r}")
        if gate_first:
            # the gate in front of the norm, every column with a weight of its own
            if gates is None:
                raise KernelError("rmsnorm_gate: no gate to put in front of the norm")
            if x.dtype != torch.float32 or x.dim() != 2 or tuple(weight.shape) != (x.shape[1],) or \
                    (group is not None and (group < 1 or x.shape[1] % group)):
                raise KernelError("rmsnorm_gate: x must be float32 [T, N], weight [N], N a multiple of the group")
            T, N = x.shape
            size = group or N
            g_ptr, g_ld = self._rows_view(gates, N)
            out = torch.empty((T, N), dtype=out_dtype, device=self.device)
            _check(self._ops.distie_gate_rmsnorm(x.data_ptr(), weight.data_ptr(), _code(weight), float(eps), g_ptr,
                                                 _code(gates), g_ld, out.data_ptr(), _code(out), T, size, N // size,
                                                 1 if gate == "silu" else 0, self._stream()), "gate_rmsnorm")
            return out
        if x.dtype != torch.float32 or x.dim() != 2 or (group is not None and (group < 1 or x.shape[1] % group)) or \
                tuple(weight.shape) not in ((group or x.shape[1],), (x.shape[1],)):
            raise KernelError("rmsnorm_gate: x must be float32 [T, N], weight [N] (or [group], N a multiple of it)")
        T, N = x.shape
        g_ptr, g_ld, g_code = None, 0, _F32
        if gates is not None:
            g_ptr, g_ld = self._rows_view(gates, N)
            g_code = _code(gates)
        out = torch.empty((T, N), dtype=out_dtype, device=self.device)
        size = group or N
        _check(self._ops.distie_rmsnorm_gate(x.data_ptr(), weight.data_ptr(), _code(weight), float(eps), g_ptr, g_code,
                                             g_ld, out.data_ptr(), _code(out), T, size, N // size,
                                             1 if gate == "silu" else 0, 1 if weight.shape[0] != size else 0,
                                             self._stream()), "rmsnorm_gate")
        return out

    # ---- norms behind sub-layers, mixers side by side, gated states, routers (csrc/recurrent.hip)
    def _term(self, value):
        """(tensor, slices) of a sub-layer's result as the norm kernels read it."""
        if isinstance(value, (NormedSum, PendingNorm, PendingProduct)):
            value = self.dense(value)
        if isinstance(value, PartialSums):
            self._own(value.data)
            return value.data, value.slices
        self._own(value)
        return value, 1

    def _norm_chain(self, terms, weights, term_eps, scale, post, residual, pre, out_dtype):
        held = [self._term(t) for t in terms]
        T, C = held[0][0].shape[-2:]
        for tensor, _ in held:
            if tuple(tensor.shape[-2:]) != (T, C):
                raise KernelError("norm chain: the terms must all be [T, C]")
        vectors = list(weights or []) + [v[0] for v in (post, pre) if v is not None]
        self._own(*vectors)
        for w in vectors:
            if w.dtype != torch.float32 or tuple(w.shape) != (C,):
                raise KernelError("norm chain: norm weights are float32 [C]")
        if residual is not None:
            self._own(residual)
            if residual.dtype != torch.float32 or tuple(residual.shape) != (T, C):
                raise KernelError("norm chain: the residual is float32 [T, C]")
        out = y = None
        if residual is None:
            y = torch.empty((T, C), dtype=torch.float32, device=self.device)
        elif out_dtype is not None:
            # with a norm in front of the next sub-layer (`pre`), or the new residual as it is, in `out_dtype`
            out = torch.empty((T, C), dtype=out_dtype, device=self.device)
        (t0, s0), (t1, s1) = held[0], (held[1] if len(held) > 1 else (None, 1))
        ptr = lambda t: t.data_ptr() if t is not None else None
        _check(self._ops.distie_norm_chain(
            t0.data_ptr(), _code(t0), s0, ptr(weights[0]) if weights else None, ptr(t1), _code(t1) if t1 is not None else _F32,
            s1, ptr(weights[1]) if weights and len(weights) > 1 else None, float(term_eps), float(scale),
            ptr(post[0]) if post else None, float(post[1]) if post else 0.0, ptr(residual),
            ptr(pre[0]) if pre else None, float(pre[1]) if pre else 0.0, ptr(out), _code(out) if out is not None else _F32,
            ptr(y), T, C, self._stream()), "norm_chain")
        if residual is not None:
            _mark_written(residual)
        return out if residual is not None else y

    def normed_sum(self, terms, weights, eps, scale):
        if not 1 <= len(terms) <= 2 or len(weights) != len(terms):
            raise KernelError("normed_sum takes one or two terms, a weight for each")
        return NormedSum(list(terms), [self._f32(w) for w in weights], float(eps), float(scale))

    @staticmethod
    def _f32(weight):
        """A norm's weight as float32 (a bfloat16 value is one exactly); kept on the tensor."""
        if weight.dtype == torch.float32:
            return weight
        held = getattr(weight, "_distie_f32", None)
        if held is None:
            held = weight._distie_f32 = weight.float()
        return held

    def add_normed(self, residual, delta, weight, eps):
        self.add_normed_rmsnorm(residual, delta, weight, eps, None, 0.0, None)

    def add_normed_rmsnorm(self, residual, delta, post_weight, post_eps, weight, eps, out_dtype):
        post = (self._f32(post_weight), post_eps)
        pre = (self._f32(weight), eps) if weight is not None else None
        if isinstance(delta, NormedSum):
            return self._norm_chain(delta.terms, delta.weights, delta.eps, delta.scale, post, residual, pre, out_dtype)
        return self._norm_chain([delta], None, 0.0, 1.0, post, residual, pre, out_dtype)

    def read_residual(self, residual, out_dtype):
        self._own(residual)
        if residual.dtype != torch.float32 or residual.dim() != 2:
            raise KernelError("read_residual reads the float32 residual stream")
        if out_dtype == torch.float32:
            return residual
        out = torch.empty(residual.shape, dtype=out_dtype, device=self.device)
        _check(self._ops.distie_sum_slices(residual.data_ptr(), 1, out.numel(), out.data_ptr(), _CODES[out_dtype],
                                           self._stream()), "sum_slices")
        return out

    def add_normed_read(self, residual, delta, post_weight, post_eps, out_dtype):
        if out_dtype == torch.float32:
            self.add_normed(residual, delta, post_weight, post_eps)
            return residual
        post = (self._f32(post_weight), post_eps)
        if isinstance(delta, NormedSum):
            return self._norm_chain(delta.terms, delta.weights, delta.eps, delta.scale, post, residual, None, out_dtype)
        return self._norm_chain([delta], None, 0.0, 1.0, post, residual, None, out_dtype)

    def gated_decay_scan(self, product, decay_logits, state, meta, num_heads, dim, value_dim, q_scale, tau, decay_low=None):
        product = self.dense(product)
        self._own(product, decay_logits, state)
        T, W = product.shape
        if T != meta.num_tokens or W < num_heads * (2 * dim + value_dim):
            raise KernelError("gated_decay_scan: the product does not match the batch or the head counts")
        if state.dtype != torch.float32 or tuple(state.shape[1:]) != (num_heads, dim, value_dim):
            raise KernelError("gated_decay_scan: the state is float32 [slots, heads, dim, value_dim]")
        chunked = not self.captured and meta.host_cu_q is not None and meta.max_q >= self.SCAN_CHUNKED_MIN_ROWS and \
            dim % 4 == 0 and value_dim % 4 == 0 and dim <= self._ops.distie_gated_decay_scan_chunked_max_dim()
        low_ptr, low_ld, up, up_bias, rank = None, 0, None, None, 0
        if decay_logits is None:
            if decay_low is None:
                raise KernelError("gated_decay_scan: neither the decay's logits nor what they are made from")
            low, up, up_bias = decay_low
            rank = up.shape[1]
            if tuple(up.shape) != (num_heads * dim, rank) or low.shape[0] != T or low.dtype != product.dtype or \
                    up_bias.dtype != torch.float32 or tuple(up_bias.shape) != (num_heads * dim,):
                raise KernelError("gated_decay_scan: low [T, rank] of the product's dtype, up [heads * dim, rank], "
                                  "bias float32 [heads * dim]")
            if chunked or rank > self._ops.distie_gated_decay_scan_max_rank():
                # portions of prompts (and wide projections): the logits as a product of their own
                decay_logits = self.decay_logits_of(decay_low)
            else:
                low_ptr, low_ld = self._rows_view(low, rank)
                up = self._f32(up)
                self._own(up, up_bias)
        if decay_logits is not None and (decay_logits.dtype != torch.float32 or
                                         tuple(decay_logits.shape) != (T, num_heads * dim)):
            raise KernelError("gated_decay_scan: the decay's logits are float32 [T, heads * dim]")
        out = torch.empty((T, num_heads * value_dim), dtype=torch.float32, device=self.device)
        if chunked:
            # portions of prompts: chunks of rows side by side instead of one row after the other
            count, packed, scratch = self._scan_chunks(meta, self._ops.distie_gated_decay_scan_chunk_rows(), num_heads,
                                                       dim, value_dim)
            totals = torch.empty((count, num_heads, dim), dtype=torch.float32, device=self.device)
            _check(self._ops.distie_gated_decay_scan_chunked(
                product.data_ptr(), _code(product), W, decay_logits.data_ptr(), state.data_ptr(), out.data_ptr(),
                scratch.data_ptr(), totals.data_ptr(), packed.data_ptr(), packed.data_ptr() + 16 * count,
                meta.state_slots.data_ptr(), count, meta.num_requests, num_heads, dim, value_dim, float(q_scale),
                float(tau), self._stream()), "gated_decay_scan_chunked")
            _mark_written(state)
            return out
        _check(self._ops.distie_gated_decay_scan(
            product.data_ptr(), _code(product), W, decay_logits.data_ptr() if decay_logits is not None else None,
            low_ptr, low_ld, up.data_ptr() if low_ptr is not None else None,
            up_bias.data_ptr() if low_ptr is not None else None, rank if low_ptr is not None else 0, state.data_ptr(),
            out.data_ptr(), meta.cu_q.data_ptr(), meta.state_slots.data_ptr(), meta.num_requests, num_heads, dim,
            value_dim, float(q_scale), float(tau), self._stream()), "gated_decay_scan")
        _mark_written(state)
        return out

    # ---- time mixing with a token shift, norms in groups, averages over the depth (csrc/time_mixing.hip, csrc/depth.hip)
    def token_shift(self, x, mu, state, meta):
        x = self.dense(x)
        self._own(x, mu, state)
        T, C = x.shape
        if T != meta.num_tokens or mu.dtype != torch.float32 or mu.dim() != 2 or mu.shape[1] != C:
            raise KernelError("token_shift: x are the step's rows, mu float32 [mixes, C]")
        if state.dtype != torch.float32 or tuple(state.shape[1:]) != (C,):
            raise KernelError("token_shift: the state is float32 [slots, C]")
        out = torch.empty((mu.shape[0], T, C), dtype=x.dtype, device=self.device)
        _check(self._ops.distie_token_shift(x.data_ptr(), _code(x), mu.data_ptr(), mu.shape[0], state.data_ptr(),
                                            out.data_ptr(), meta.cu_q.data_ptr(), None if meta.all_decode else meta.token_request.data_ptr(),
                                            meta.state_slots.data_ptr(), T, C, self._stream()), "token_shift")
        _mark_written(state)
        return out

    EACH_MAX_ROWS = 32        # up to so many rows several products with inputs of their own run as one launch

    def prepare_linear_each(self, weights):
        """One packed copy for all, kept on the first weight: the weights one behind the other, each rounded up to whole
        row blocks (the projections of few rows); beside it nothing, as more rows go to the library."""
        first = weights[0]
        if (self.packed_roles is not None and "qkv" not in self.packed_roles) or not self.packed_weights or \
                any(w.dtype != torch.bfloat16 or w.dim() != 2 or w.shape[1] != first.shape[1] for w in weights) or \
                first.shape[1] % 8 or len(weights) > 8 or hasattr(first, "_distie_each"):
            return
        K = first.shape[1]
        blocks = [-(-w.shape[0] // 16) for w in weights]
        free, total = torch.cuda.mem_get_info(self.device)
        if free - 2 * sum(blocks) * -(-K // 32) * 512 < self.PACKED_KEEPS_FREE * total:
            self._packed_left_out += 1
            return
        packed = torch.empty(sum(blocks) * -(-K // 32) * 512, dtype=torch.bfloat16, device=self.device)
        at, maps = 0, []
        for w, count in zip(weights, blocks):
            self._own(w)
            row_map = self._row_map(w.shape[0], False, None).to(device=self.device, dtype=torch.int32)
            maps.append(row_map)
            size = count * -(-K // 32) * 512
            _check(self._ops.distie_pack_rows(w.data_ptr(), packed[at:at + size].data_ptr(), row_map.data_ptr(), count, K,
                                              self._stream()), "pack_rows")
            at += size
        torch.cuda.current_stream(self.device).synchronize()      # the row maps are freed on return
        first._distie_each = (packed, np.cumsum(np.asarray(blocks, dtype=np.int32)).astype(np.int32))

    def linear_each(self, xs, weights, unrounded=()):
        held = getattr(weights[0], "_distie_each", None)
        if held is None or xs.dtype != torch.bfloat16 or xs.shape[1] > self.EACH_MAX_ROWS:
            return super().linear_each(xs, weights, unrounded)
        self._own(xs)
        packed, ends = held
        count, M, K = xs.shape
        if count != len(weights) or any(w.shape[1] != K for w in weights) or \
                [int(e) for e in np.diff(ends, prepend=0)] != [-(-w.shape[0] // 16) for w in weights] or \
                packed.numel() != int(ends[-1]) * -(-K // 32) * 512:
            raise KernelError("linear_each: an input [rows, K] for every weight [N, K], the weights it was prepared for")
        out = torch.empty((M, 16 * int(ends[-1])), dtype=torch.float32, device=self.device)
        _check(self._ops.distie_gemm_packed_each_bf16(xs.data_ptr(), packed.data_ptr(), out.data_ptr(), M, K, count,
                                                      ends.ctypes.data, self._stream()), "gemm_packed_each_bf16")
        starts = [0] + [16 * int(e) for e in ends[:-1]]
        return [out[:, at:at + w.shape[0]] for at, w in zip(starts, weights)]

    def wkv_decay_logits(self, low, up, up_bias):
        low = low if low.dtype == torch.float32 else low.float()
        ptr, ld = self._rows_view(low, up.shape[1])
        bent = torch.empty(low.shape, dtype=torch.float32, device=self.device)
        _check(self._ops.distie_tanh_f32(ptr, ld, bent.data_ptr(), low.shape[0], low.shape[1], self._stream()), "tanh_f32")
        return self.linear_f32out(bent, up, up_bias)

    def wkv_mix(self, r, k, v, gates, low, up, up_bias, bonus, state, meta, num_heads, dim, norm_weight, eps, out_dtype):
        N, T, rank = num_heads * dim, r.shape[0], up.shape[1]
        self._own(up, up_bias, bonus, state, norm_weight)
        views = [self._rows_view(t, N) for t in (r, k, v, gates)]
        ld = views[0][1]
        if T != meta.num_tokens or any(t.dtype != r.dtype or t.shape[0] != T for t in (k, v, gates)) or \
                any(view[1] != ld for view in views) or low.shape[0] != T:
            raise KernelError("wkv_mix: r, k, v and gates are the step's rows, of one dtype and row stride")
        for name, t, shape in (("up", up, (N, rank)), ("up_bias", up_bias, (N,)), ("bonus", bonus, (N,)),
                               ("norm_weight", norm_weight, (N,))):
            if t.dtype != torch.float32 or tuple(t.shape) != shape:
                raise KernelError(f"wkv_mix: {name} must be float32 {list(shape)}")
        if state.dtype != torch.float32 or tuple(state.shape[1:]) != (num_heads, dim, dim):
            raise KernelError("wkv_mix: the state is float32 [slots, heads, dim, dim]")
        if dim > self._ops.distie_wkv_scan_max_dim() or rank > self._ops.distie_wkv_scan_max_rank():
            raise KernelError(f"wkv_mix: heads of up to {self._ops.distie_wkv_scan_max_dim()} and decays through up to "
                              f"{self._ops.distie_wkv_scan_max_rank()} dimensions")
        low_ptr, low_ld = self._rows_view(low, rank)
        out = torch.empty((T, N), dtype=out_dtype, device=self.device)
        if not self.captured and meta.host_cu_q is not None and meta.max_q >= self.SCAN_CHUNKED_MIN_ROWS and \
                dim <= self._ops.distie_wkv_chunked_max_dim():
            # portions of prompts: chunks of rows side by side instead of one row after the other
            z = self.wkv_decay_logits(low, up, up_bias)
            count, packed, scratch = self._scan_chunks(meta, self._ops.distie_wkv_chunk_rows(), num_heads, dim, dim)
            totals = torch.empty((count, num_heads, dim), dtype=torch.float32, device=self.device)
            _check(self._ops.distie_wkv_scan_chunked(
                views[0][0], views[1][0], views[2][0], views[3][0], _code(r), ld, z.data_ptr(), bonus.data_ptr(),
                state.data_ptr(), norm_weight.data_ptr(), float(eps), out.data_ptr(), _code(out), scratch.data_ptr(),
                totals.data_ptr(), packed.data_ptr(), packed.data_ptr() + 16 * count, meta.state_slots.data_ptr(), count,
                meta.num_requests, num_heads, dim, self._stream()), "wkv_scan_chunked")
            _mark_written(state)
            return out
        _check(self._ops.distie_wkv_scan(
            views[0][0], views[1][0], views[2][0], views[3][0], _code(r), ld, low_ptr, _code(low), low_ld, rank, up.data_ptr(),
            up_bias.data_ptr(), bonus.data_ptr(), state.data_ptr(), norm_weight.data_ptr(), float(eps), out.data_ptr(),
            _code(out), None if meta.all_decode else meta.cu_q.data_ptr(), meta.state_slots.data_ptr(), meta.num_requests,
            num_heads, dim, self._stream()), "wkv_scan")
        _mark_written(state)
        return out

    def group_rmsnorm(self, x, weight, eps, groups, out_dtype):
        return self._group_chain(x, weight, eps, groups, None, None, None, out_dtype)

    def _group_chain(self, delta, weight, eps, groups, residual, into, history, out_dtype, shift=None):
        delta, slices = self._term(delta)
        T, C = delta.shape[-2:]
        self._own(weight, residual, into)
        if weight.dtype != torch.float32 or tuple(weight.shape) != (C,) or groups < 1 or C % groups:
            raise KernelError("norm in groups: weight float32 [C], C a multiple of the groups")
        for t in (residual, into):
            if t is not None and (t.dtype != torch.float32 or tuple(t.shape) != (T, C)):
                raise KernelError("norm in groups: the residual is float32 [T, C]")
        first = rest = weights = None
        index = 0
        if history is not None:
            first, rest, index, weights = history
            self._own(first, rest, weights)
            if first.dtype != torch.float32 or rest.dtype != torch.float32 or tuple(first.shape) != (T, C) or \
                    rest.dim() != 3 or tuple(rest.shape[1:]) != (T, C) or not 0 <= index < rest.shape[0] or \
                    weights.dtype != torch.float32 or tuple(weights.shape) != (index + 2,):
                raise KernelError("average over the depth: X_0 float32 [T, C], the others [layers, T, C], a weight for each")
        mu = state = slots = None
        if shift is not None:
            mu, state, slots = shift
            self._own(mu, state, slots)
            if mu.dtype != torch.float32 or mu.dim() != 2 or mu.shape[1] != C or slots.shape[0] != T or \
                    state.dtype != torch.float32 or tuple(state.shape[1:]) != (C,):
                raise KernelError("norm in groups with a token shift: mu float32 [mixes, C], the state float32 [slots, C], a row "
                                  "a request")
        out = None
        if out_dtype is not None:
            out = torch.empty((T, C) if mu is None else (mu.shape[0], T, C), dtype=out_dtype, device=self.device)
        ptr = lambda t: t.data_ptr() if t is not None else None
        _check(self._ops.distie_group_chain(
            delta.data_ptr(), _code(delta), slices, weight.data_ptr(), float(eps), int(groups), ptr(residual), ptr(into),
            ptr(first), ptr(rest), int(index), ptr(weights), ptr(out), _code(out) if out is not None else _F32, T, C, ptr(mu),
            mu.shape[0] if mu is not None else 0, ptr(state), ptr(slots), self._stream()), "group_chain")
        if state is not None:
            _mark_written(state)
        if into is not None:
            _mark_written(into)
        return out

    def add_group_normed(self, residual, delta, weight, eps, groups, out_dtype, in_place=True, history=None):
        into = residual if in_place else torch.empty_like(residual)
        read = self._group_chain(delta, weight, eps, groups, residual, into, history,
                                 None if out_dtype == torch.float32 else out_dtype)
        return into, into if out_dtype == torch.float32 else read

    def add_group_normed_shift(self, residual, delta, weight, eps, groups, out_dtype, in_place, history, mu, state, meta):
        if not meta.all_decode:
            return super().add_group_normed_shift(residual, delta, weight, eps, groups, out_dtype, in_place, history, mu, state,
                                                  meta)
        # a row a request: the block that owns a row shifts it too
        into = residual if in_place else torch.empty_like(residual)
        return into, self._group_chain(delta, weight, eps, groups, residual, into, history, out_dtype,
                                       (mu, state, meta.state_slots))

    def lru_gates(self, u, recur_weight, recur_bias, input_weight, input_bias, lam, rate):
        u = self.dense(u)
        self._own(recur_weight, recur_bias, input_weight, input_bias, lam)
        T, R = u.shape
        u_ptr, ldu = self._rows_view(u, R)
        blocks = recur_weight.shape[0]
        n = R // max(blocks, 1)
        if recur_weight.dim() != 3 or tuple(recur_weight.shape) != (blocks, n, n) or blocks * n != R or \
                input_weight.shape != recur_weight.shape or input_weight.dtype != recur_weight.dtype:
            raise KernelError("lru_gates: the gates' weights are [blocks, R / blocks, R / blocks], of one dtype")
        for t in (recur_bias, input_bias, lam):
            if t.dtype != torch.float32 or t.numel() != R:
                raise KernelError("lru_gates: biases and lam are float32 with R elements")
        a = torch.empty((T, R), dtype=torch.float32, device=self.device)
        x = torch.empty((T, R), dtype=torch.float32, device=self.device)
        _check(self._ops.distie_lru_gates(u_ptr, _code(u), ldu, recur_weight.data_ptr(), recur_bias.data_ptr(),
                                          input_weight.data_ptr(), input_bias.data_ptr(), _code(recur_weight),
                                          lam.data_ptr(), float(rate), a.data_ptr(), x.data_ptr(), T, R, blocks,
                                          self._stream()), "lru_gates")
        return a, x

    def lru_scan(self, a, x, state, meta, mul, mul_act, out_dtype):
        self._own(a, x, state)
        T, R = a.shape
        if a.dtype != torch.float32 or x.dtype != torch.float32 or x.shape != a.shape or T != meta.num_tokens:
            raise KernelError("lru_scan: a and x are float32 [T, R], the step's rows")
        if state.dtype != torch.float32 or tuple(state.shape[1:]) != (R,):
            raise KernelError("lru_scan: the state is float32 [slots, R]")
        kind = -1
        if mul_act is not None:
            if mul_act not in self.ACTIVATIONS:
                raise KernelError(f"no activation named {mul_act!r}")
            kind = self.ACTIVATIONS[mul_act]
        m_ptr, m_ld, m_code = None, 0, _F32
        if mul is not None:
            m_ptr, m_ld = self._rows_view(mul, R)
            m_code = _code(mul)
        out = torch.empty((T, R), dtype=out_dtype, device=self.device)
        if not self.captured and meta.host_cu_q is not None and meta.max_q >= self.LRU_CHUNKED_MIN_ROWS:
            # portions of prompts: chunks of rows side by side, each scanned twice (alone, then from what stands before it)
            count, packed, sums = self._scan_chunks(meta, self._ops.distie_lru_scan_chunk_rows(), 1, 1, R)
            factors = torch.empty((count, R), dtype=torch.float32, device=self.device)
            init = torch.empty((meta.num_requests, R), dtype=torch.float32, device=self.device)
            _check(self._ops.distie_lru_scan_chunked(
                a.data_ptr(), x.data_ptr(), state.data_ptr(), factors.data_ptr(), sums.data_ptr(), init.data_ptr(), m_ptr,
                m_code, m_ld, kind, out.data_ptr(), _code(out), packed.data_ptr(), packed.data_ptr() + 16 * count,
                meta.state_slots.data_ptr(), count, meta.num_requests, R, self._stream()), "lru_scan_chunked")
            _mark_written(state)
            return out
        _check(self._ops.distie_lru_scan(a.data_ptr(), x.data_ptr(), state.data_ptr(), m_ptr, m_code, m_ld, kind,
                                         out.data_ptr(), _code(out), meta.cu_q.data_ptr(), meta.state_slots.data_ptr(),
                                         meta.num_requests, R, self._stream()), "lru_scan")
        _mark_written(state)
        return out

    SCORINGS = {"softmax": 0, "sigmoid": 1, "softmax_all": 2, "sigmoid_share": 3}
    NO_RULE = RouteRule()

    def _route_rule(self, rule, scoring, experts):
        """The rule's numbers as the kernels take them: (correction, groups, kept, scale, shared)."""
        rule = rule or self.NO_RULE
        if scoring != "sigmoid_share" and (rule.correction is not None or rule.groups != 1 or rule.scale != 1.0):
            raise KernelError("a router's correction, groups and scale go with the scoring sigmoid_share")
        self._own(rule.correction)
        if rule.correction is not None and (rule.correction.dtype != torch.float32 or tuple(rule.correction.shape) != (experts,)):
            raise KernelError("a router's correction is float32 [experts]")
        return (rule.correction.data_ptr() if rule.correction is not None else None, int(rule.groups), int(rule.kept),
                float(rule.scale), 1 if rule.shared else 0)

    def route_topk(self, x, weight, bias, top, scoring="softmax", rule=None):
        if scoring not in self.SCORINGS:
            raise KernelError(f"route_topk: no scoring named {scoring!r}")
        x = self.dense(x)
        self._own(x, weight, bias)
        T, C = x.shape
        rows = weight.shape[0]
        shared = 1 if rule is not None and rule.shared else 0
        E = rows - shared
        if tuple(weight.shape) != (rows, C) or (bias is not None and (bias.dtype != torch.float32 or tuple(bias.shape) != (rows,))):
            raise KernelError("route_topk: weight [experts (+ 1 with a shared one), C], bias float32 with a number a row")
        numbers = self._route_rule(rule, scoring, E)
        experts = torch.empty((T, top), dtype=torch.int32, device=self.device)
        gates = torch.empty((T, top + shared), dtype=torch.float32, device=self.device)
        _check(self._ops.distie_route_topk(x.data_ptr(), _code(x), weight.data_ptr(), _code(weight),
                                           bias.data_ptr() if bias is not None else None, experts.data_ptr(),
                                           gates.data_ptr(), T, C, E, int(top), self.SCORINGS[scoring], *numbers,
                                           self._stream()), "route_topk")
        return experts, gates

    def route_glu(self, gate_up, experts, gates, num_experts, width, limit, slope, up_shift, on_input, shared_width=0):
        if isinstance(gate_up, (PendingNorm, PendingProduct)):
            gate_up = self.dense(gate_up)
        slices, source, dtype, ld = 1, gate_up, gate_up.dtype, gate_up.shape[1]
        if isinstance(gate_up, PartialSums):
            slices, source = gate_up.slices, gate_up.data
        elif gate_up.dim() == 2 and gate_up.stride(1) == 1 and gate_up.stride(0) > gate_up.shape[1]:
            # rows that lie further apart than they are wide (`linear_spread`): the kernel takes the row stride
            ld = gate_up.stride(0)
            if gate_up.device != self.device:
                raise KernelError(f"tensor on {gate_up.device}, kernels run on {self.device}")
            source = None
        self._own(source, experts, gates)
        source = gate_up if source is None else source
        T, top = experts.shape
        total = num_experts * width + shared_width
        if experts.dtype != torch.int32 or gates.dtype != torch.float32 or \
                tuple(gates.shape) != (T, top + (1 if shared_width else 0)) or \
                gate_up.shape[0] != T or gate_up.shape[1] != 2 * total:
            raise KernelError("route_glu: experts int32 and gates float32 [T, top] (one more with a shared expert), gate_up "
                              "[T, 2 * (experts * width + shared_width)]")
        if limit is not None and not limit > 0:
            raise KernelError("route_glu: the limit must be positive")
        out = torch.empty((T, total), dtype=dtype, device=self.device)
        _check(self._ops.distie_route_glu(source.data_ptr(), _code(source), ld, slices, experts.data_ptr(),
                                          gates.data_ptr(), T, top, num_experts, width, float(limit or 0.0), float(slope),
                                          float(up_shift), 1 if on_input else 0, int(shared_width), out.data_ptr(),
                                          _code(out), self._stream()), "route_glu")
        return out

    FUSED_ROUTE_ROWS = 64       # up to so many rows every block works out its row's choice itself

    def route_experts_glu(self, x, router_weight, router_bias, top, scoring, gate_up, num_experts, width, limit, slope,
                          up_shift, on_input, rule=None, shared_width=0):
        if scoring not in self.SCORINGS:
            raise KernelError(f"route_experts_glu: no scoring named {scoring!r}")
        x = self.dense(x)
        T, C = x.shape
        if T > self.FUSED_ROUTE_ROWS or x.dtype != torch.bfloat16 or router_weight.dtype != torch.bfloat16 or C % 8 or \
                x.data_ptr() % 16 or router_weight.data_ptr() % 16 or not x.is_contiguous():
            return super().route_experts_glu(x, router_weight, router_bias, top, scoring, gate_up, num_experts, width,
                                             limit, slope, up_shift, on_input, rule, shared_width)
        if isinstance(gate_up, (PendingNorm, PendingProduct)):
            gate_up = self.dense(gate_up)
        slices, source, dtype = 1, gate_up, gate_up.dtype
        if isinstance(gate_up, PartialSums):
            slices, source = gate_up.slices, gate_up.data
        self._own(x, router_weight, router_bias, source)
        numbers = self._route_rule(rule, scoring, num_experts)
        rows, total = num_experts + numbers[-1], num_experts * width + shared_width
        if tuple(router_weight.shape) != (rows, C) or not 1 <= top <= num_experts or gate_up.shape[0] != T or \
                gate_up.shape[1] != 2 * total or (shared_width and not numbers[-1]) or \
                (router_bias is not None and (router_bias.dtype != torch.float32 or tuple(router_bias.shape) != (rows,))):
            raise KernelError("route_experts_glu: x [T, C], router [E, C], bias float32 [E], gate_up [T, 2 * E * width]")
        if limit is not None and not limit > 0:
            raise KernelError("route_experts_glu: the limit must be positive")
        out = torch.empty((T, total), dtype=dtype, device=self.device)
        _check(self._ops.distie_route_topk_glu(
            x.data_ptr(), router_weight.data_ptr(), router_bias.data_ptr() if router_bias is not None else None, C,
            self.SCORINGS[scoring], source.data_ptr(), _code(source), gate_up.shape[1], slices, T, int(top),
            num_experts, width, float(limit or 0.0), float(slope), float(up_shift), 1 if on_input else 0, *numbers,
            int(shared_width), out.data_ptr(), _code(out), self._stream()), "route_topk_glu")
        return out

    def softcap(self, x, cap):
        self._own(x)
        if x.dtype != torch.float32:
            raise KernelError("softcap works on float32 values")
        _check(self._ops.distie_softcap_f32(x.data_ptr(), x.numel(), float(cap), self._stream()), "softcap_f32")
        _mark_written(x)
        return x

    def route_scale(self, hidden, experts, gates, num_experts, width):
        hidden = self.dense(hidden)
        self._own(hidden, experts, gates)
        T, top = experts.shape
        if experts.dtype != torch.int32 or gates.dtype != torch.float32 or gates.shape != experts.shape or \
                hidden.shape[0] != T or hidden.shape[1] < num_experts * width:
            raise KernelError("route_scale: experts int32 and gates float32 [T, top], hidden [T, >= experts * width]")
        _check(self._ops.distie_route_scale(hidden.data_ptr(), _code(hidden), hidden.shape[1], experts.data_ptr(),
                                            gates.data_ptr(), T, top, num_experts, width, self._stream()), "route_scale")
        _mark_written(hidden)
        return hidden

    def activation(self, x, kind):
        if kind not in self.ACTIVATIONS:
            raise KernelError(f"no activation named {kind!r}")
        if isinstance(x, (PendingNorm, PendingProduct)):
            x = self.dense(x)
        slices, source, dtype = 1, x, x.dtype
        if isinstance(x, PartialSums):
            slices, source = x.slices, x.data
        self._own(source)
        out = torch.empty(tuple(x.shape), dtype=dtype, device=self.device)
        _check(self._ops.distie_activation(source.data_ptr(), _code(source), slices, out.data_ptr(), _code(out), out.numel(),
                                           self.ACTIVATIONS[kind], self._stream()), "activation")
        return out

    # ---- the gated delta rule (csrc/delta.hip)
    def delta_scan(self, qkv, beta, decay, a_log, dt_bias, state, meta, num_heads, num_kv_heads, dim, value_dim, q_scale,
                   unit_eps):
        qkv = self.dense(qkv)
        H, G, D, E = num_heads, num_kv_heads, dim, value_dim
        q_ptr, ld = self._rows_view(qkv, qkv.shape[1])
        b_ptr, ldb = self._rows_view(beta, H)
        d_ptr, ldd = self._rows_view(decay, H)
        self._own(a_log, dt_bias, state)
        T = qkv.shape[0]
        if T != meta.num_tokens or qkv.shape[1] < 2 * G * D + H * E or H % G or beta.shape[0] != T or decay.shape[0] != T or \
                beta.dtype != qkv.dtype or decay.dtype != qkv.dtype:
            raise KernelError("delta_scan: q, k, v and the logits do not match the batch or the head counts")
        if D > self._ops.distie_delta_scan_max_dim():
            raise KernelError(f"delta_scan: keys of up to {self._ops.distie_delta_scan_max_dim()} dimensions a head")
        if state.dtype != torch.float32 or tuple(state.shape[1:]) != (H, D, E):
            raise KernelError("delta_scan: the state is float32 [slots, heads, dim, value_dim]")
        for vector in (a_log, dt_bias):
            if vector.dtype != torch.float32 or tuple(vector.shape) != (H,):
                raise KernelError("delta_scan: a_log and dt_bias are float32 [heads]")
        out = torch.empty((T, H * E), dtype=torch.float32, device=self.device)
        if not self.captured and meta.host_cu_q is not None and meta.max_q >= self.SCAN_CHUNKED_MIN_ROWS:
            # portions of prompts: chunks of rows, the triangular systems of all chunks side by side
            rows = self._ops.distie_delta_scan_chunk_rows()
            DP, EP = self._ops.distie_delta_scan_padded_dim(D), -(-E // 16) * 16
            count, packed, states = self._scan_chunks(meta, rows, H, DP, EP)
            key = ("delta_scratch", count, H, DP, EP)
            held = meta.scratch.get(key)
            if held is None:
                held = meta.scratch[key] = [torch.empty((count, H, *shape), dtype=torch.float32, device=self.device)
                                            for shape in ((rows, DP), (rows, EP), (rows, EP), (DP, rows), (rows, rows), (rows,),
                                                          ())]
            _check(self._ops.distie_delta_scan_chunked(
                q_ptr, _code(qkv), ld, b_ptr, ldb, d_ptr, ldd, a_log.data_ptr(), dt_bias.data_ptr(), state.data_ptr(),
                out.data_ptr(), *(t.data_ptr() for t in held), states.data_ptr(), packed.data_ptr(),
                packed.data_ptr() + 16 * count, meta.state_slots.data_ptr(), count, meta.num_requests, H, G, D, E,
                float(q_scale), float(unit_eps), self._stream()), "delta_scan_chunked")
            _mark_written(state)
            return out
        _check(self._ops.distie_delta_scan(
            q_ptr, _code(qkv), ld, b_ptr, ldb, d_ptr, ldd, a_log.data_ptr(), dt_bias.data_ptr(), state.data_ptr(),
            out.data_ptr(), meta.cu_q.data_ptr(), meta.state_slots.data_ptr(), meta.num_requests, H, G, D, E, float(q_scale),
            float(unit_eps), self._stream()), "delta_scan")
        _mark_written(state)
        return out

    # ---- a state with one decay a head and token, attention over a shared latent (csrc/ssm.hip, csrc/latent.hip)
    SSM_CHUNKED_MIN_ROWS = 32        # a step with a portion of so many rows scans the state-space state in chunks

    def ssm_scan_captures(self, state_size):
        return state_size <= self._ops.distie_ssm_scan_max_state()

    def ssm_scan(self, xbc, dt, dt_bias, a_log, skip, state, meta, num_heads, value_dim, state_size, groups):
        xbc = self.dense(xbc)
        H, P, N, G = num_heads, value_dim, state_size, groups
        width = H * P + 2 * G * N
        x_ptr, ld = self._rows_view(xbc, xbc.shape[1])
        d_ptr, ldd = self._rows_view(dt, H)
        self._own(dt_bias, a_log, skip, state)
        T = xbc.shape[0]
        if T != meta.num_tokens or xbc.shape[1] < width or dt.dtype != xbc.dtype or H % G:
            raise KernelError("ssm_scan: x, B and C do not match the batch or the head counts")
        if state.dtype != torch.float32 or tuple(state.shape[1:]) != (H, N, P):
            raise KernelError("ssm_scan: the state is float32 [slots, heads, state_size, value_dim]")
        for vector in (dt_bias, a_log, skip):
            if vector.dtype != torch.float32 or tuple(vector.shape) != (H,):
                raise KernelError("ssm_scan: dt_bias, a_log and skip are float32 [heads]")
        out = torch.empty((T, H * P), dtype=torch.float32, device=self.device)
        wide = N > self._ops.distie_ssm_scan_max_state()      # more rows a head than the row-by-row kernel keeps
        if not self.captured and meta.host_cu_q is not None and (meta.max_q >= self.SSM_CHUNKED_MIN_ROWS or wide):
            count, packed, scratch = self._scan_chunks(meta, self._ops.distie_ssm_scan_chunk_rows(), H, N, P)
            key = ("ssm_totals", count, H, G)
            held = meta.scratch.get(key)
            if held is None:
                rows = self._ops.distie_ssm_scan_chunk_rows()
                held = meta.scratch[key] = (torch.empty((count, H), dtype=torch.float32, device=self.device),
                                            torch.empty((count, G, rows, rows), dtype=torch.float32, device=self.device))
            totals, pairs = held
            _check(self._ops.distie_ssm_scan_chunked(
                x_ptr, _code(xbc), ld, d_ptr, ldd, dt_bias.data_ptr(), a_log.data_ptr(), skip.data_ptr(),
                state.data_ptr(), out.data_ptr(), scratch.data_ptr(), totals.data_ptr(), pairs.data_ptr(), packed.data_ptr(),
                packed.data_ptr() + 16 * count, meta.state_slots.data_ptr(), count, meta.num_requests, H, P, N, G,
                self._stream()), "ssm_scan_chunked")
            _mark_written(state)
            return out
        if wide:
            raise KernelError(f"ssm_scan: a state of {N} rows a head is beyond the row-by-row kernel, which is all a "
                              f"captured step can use")
        _check(self._ops.distie_ssm_scan(x_ptr, _code(xbc), ld, d_ptr, ldd, dt_bias.data_ptr(), a_log.data_ptr(),
                                         skip.data_ptr(), state.data_ptr(), out.data_ptr(), meta.cu_q.data_ptr(),
                                         meta.state_slots.data_ptr(), meta.num_requests, H, P, N, G, self._stream()),
               "ssm_scan")
        _mark_written(state)
        return out

    def latent_norm_rope_write(self, down, q_rank, q_weight, kv_rank, kv_weight, eps, rot_dim, inv_freq, magnitude,
                               neighbours, meta, group, k_cache, v_cache, write, out_dtype):
        slices = 1
        if isinstance(down, PartialSums) and down.dtype == torch.float32 and \
                down.shape[1] <= self._ops.distie_latent_norm_max_width():
            slices, down = down.slices, down.data.view(-1, down.data.shape[-1])        # added up while they are read
        else:
            down = self.dense(down)
        self._own(down, q_weight, kv_weight, k_cache, v_cache, inv_freq)
        T, W = down.shape[0] // slices, down.shape[1]
        if slices == 1 and W > self._ops.distie_latent_norm_max_width():
            raise KernelError("latent_norm_rope_write: the down-projection is wider than the kernel's row")
        if down.dtype != torch.float32 or W < q_rank + kv_rank + rot_dim or T != meta.num_tokens:
            raise KernelError("latent_norm_rope_write: the down-projection is float32 [T, q_rank + kv_rank + rot_dim]")
        for weight, size in ((q_weight, q_rank), (kv_weight, kv_rank)):
            if size and (weight is None or weight.dtype != torch.float32 or tuple(weight.shape) != (size,)):
                raise KernelError("latent_norm_rope_write: the norms' weights are float32 [rank]")
        padded = k_cache.shape[-1]
        if write:
            self._check_cache(k_cache, v_cache, 1, meta.block_size, padded)
            if k_cache.dtype != v_cache.dtype or padded < kv_rank + rot_dim:
                raise KernelError("latent_norm_rope_write: one key/value head of at least kv_rank + rot_dim, in one dtype")
        pairs = 0 if inv_freq is None else inv_freq.shape[0]
        if pairs and 2 * pairs != rot_dim:
            raise KernelError("latent_norm_rope_write: the rotation turns all of the rotated part")
        table = self._rope_table(meta, inv_freq) if pairs else None
        latent = torch.empty((T, q_rank), dtype=out_dtype, device=self.device) if q_rank else None
        ptr = lambda t: t.data_ptr() if t is not None else None
        _check(self._ops.distie_latent_norm_rope_write(
            down.data_ptr(), slices, W, q_rank, ptr(q_weight), kv_rank, kv_weight.data_ptr(), float(eps), rot_dim, ptr(table),
            float(magnitude), 1 if neighbours else 0, ptr(latent), _CODES[out_dtype], k_cache.data_ptr(),
            v_cache.data_ptr(), _code(k_cache), meta.groups[group].slots.data_ptr(), T, meta.block_size, padded,
            1 if write else 0, self._stream()), "latent_norm_rope_write")
        return latent

    def latent_queries(self, q, key_up, num_heads, dim, rot_dim, padded_dim, inv_freq, magnitude, neighbours, meta):
        """One launch on the matrix cores for bfloat16 steps (the product's partial sums added up while they are read);
        else the product by head, then the rotation."""
        kv_rank = key_up.shape[1]
        slices, source, dtype = 1, q, getattr(q, "dtype", None)
        if isinstance(q, PartialSums):
            slices, source = q.slices, q.data
        fused = dtype == torch.bfloat16 and key_up.dtype == torch.bfloat16 and inv_freq is not None and \
            isinstance(source, torch.Tensor) and 2 * inv_freq.shape[0] == rot_dim and dim % 8 == 0 and \
            (dim + rot_dim) % 8 == 0 and tuple(key_up.shape) == (num_heads, kv_rank, dim) and \
            tuple(q.shape) == (meta.num_tokens, num_heads * (dim + rot_dim)) and padded_dim >= kv_rank + rot_dim
        if not fused:
            return super().latent_queries(self.dense(q), key_up, num_heads, dim, rot_dim, padded_dim, inv_freq, magnitude,
                                          neighbours, meta)
        self._own(source, key_up, inv_freq)
        T = meta.num_tokens
        table = self._rope_table(meta, inv_freq)
        out = torch.empty((T, num_heads * padded_dim), dtype=torch.bfloat16, device=self.device)
        _check(self._ops.distie_latent_queries(
            source.data_ptr(), _code(source), slices, dim + rot_dim, key_up.data_ptr(), _code(key_up), out.data_ptr(),
            padded_dim, T, num_heads, kv_rank, dim, rot_dim // 2, table.data_ptr(), float(magnitude),
            1 if neighbours else 0, self._stream()), "latent_queries")
        return out

    def heads_linear(self, x, weight, in_stride, out_stride, out=None):
        x = self.dense(x)
        self._own(x, weight, out)
        if weight.dim() != 3:
            raise KernelError("heads_linear: the weight is [heads, N, K]")
        H, N, K = weight.shape
        T = x.shape[0]
        if x.shape[1] != H * in_stride or K > in_stride or N > out_stride:
            raise KernelError("heads_linear: x is [T, heads * in_stride] with in_stride >= K, out_stride >= N")
        if out is None:
            make = torch.empty if N == out_stride else torch.zeros
            out = make((T, H * out_stride), dtype=x.dtype, device=self.device)
        elif out.dtype != x.dtype or tuple(out.shape) != (T, H * out_stride):
            raise KernelError("heads_linear: out is [T, heads * out_stride] of x's dtype")
        _check(self._ops.distie_heads_linear(x.data_ptr(), _code(x), in_stride, weight.data_ptr(), _code(weight),
                                             out.data_ptr(), out_stride, T, H, N, K, self._stream()), "heads_linear")
        return out

    def rope_heads(self, x, in_stride, in_offset, out, out_stride, out_offset, num_heads, inv_freq, magnitude,
                   neighbours, meta):
        x = self.dense(x)
        self._own(x, out, inv_freq)
        T = x.shape[0]
        if x.dtype != out.dtype or x.shape[1] != num_heads * in_stride or tuple(out.shape) != (T, num_heads * out_stride) \
                or T != meta.num_tokens:
            raise KernelError("rope_heads: x [T, heads * in_stride] and out [T, heads * out_stride] of one dtype")
        table = self._rope_table(meta, inv_freq)
        _check(self._ops.distie_rope_heads(x.data_ptr(), _code(x), in_stride, in_offset, out.data_ptr(), out_stride,
                                           out_offset, T, num_heads, inv_freq.shape[0], table.data_ptr(),
                                           float(magnitude), 1 if neighbours else 0, self._stream()), "rope_heads")
        return out

    def glu_mul(self, gate_up, kind):
        if kind == "silu":
            return self.silu_mul(gate_up)
        if kind not in self.ACTIVATIONS:
            raise KernelError(f"glu_mul: no activation named {kind!r}")
        return self._glu_mul(gate_up, self.ACTIVATIONS[kind])

    def clamped_glu(self, gate_up, limit, slope, up_shift):
        if not limit > 0:
            raise KernelError("clamped_glu: the limit must be positive")
        return self._glu_mul(gate_up, len(self.ACTIVATIONS), (float(limit), float(slope), float(up_shift)))

    def _glu_mul(self, gate_up, kind, clamp=(0.0, 1.0, 0.0)):
        if isinstance(gate_up, (PendingNorm, PendingProduct)):
            gate_up = self.dense(gate_up)
        slices, source, dtype = 1, gate_up, gate_up.dtype
        if isinstance(gate_up, PartialSums):
            slices, source = gate_up.slices, gate_up.data
        self._own(source)
        rows, two = gate_up.shape
        out = torch.empty((rows, two // 2), dtype=dtype, device=self.device)
        _check(self._ops.distie_glu_mul(source.data_ptr(), _code(source), slices, out.data_ptr(), _code(out), rows,
                                        two // 2, kind, *clamp, self._stream()), "glu_mul")
        return out

    def silu_mul(self, gate_up):
        if isinstance(gate_up, (PendingNorm, PendingProduct)):
            gate_up = self.dense(gate_up)
        slices, source, dtype = 1, gate_up, gate_up.dtype
        if isinstance(gate_up, PartialSums):
            slices, source = gate_up.slices, gate_up.data
        self._own(source)
        rows, two = gate_up.shape
        out = torch.empty((rows, two // 2), dtype=dtype, device=self.device)
        _check(self._ops.distie_silu_mul(source.data_ptr(), _code(source), slices, out.data_ptr(), _code(out),
                                         rows, two // 2, self._stream()), "silu_mul")
        return out

    def gather_rows(self, x, rows):
        x = self.dense(x)
        self._own(x, rows)
        out = torch.empty((rows.shape[0], x.shape[1]), dtype=x.dtype, device=self.device)
        _check(self._ops.distie_gather_rows(x.data_ptr(), rows.data_ptr(), out.data_ptr(), rows.shape[0],
                                            x.shape[1] * x.element_size(), x.shape[0], self._stream()), "gather_rows")
        return out

    def argmax(self, logits):
        self._own(logits)
        if logits.dtype != torch.float32:
            raise KernelError("argmax reads float32 logits")
        rows, vocab = logits.shape
        out = torch.empty(rows, dtype=torch.int32, device=self.device)
        parts = self._ops.distie_argmax_parts(rows, vocab)
        values = indexes = None
        if parts > 1:
            values = torch.empty(rows * parts, dtype=torch.float32, device=self.device)
            indexes = torch.empty(rows * parts, dtype=torch.int32, device=self.device)
        _check(self._ops.distie_argmax(logits.data_ptr(), out.data_ptr(), rows, vocab,
                                       values.data_ptr() if parts > 1 else None,
                                       indexes.data_ptr() if parts > 1 else None, self._stream()), "argmax")
        return out

    def sample(self, logits, temperature, seeds, counters):
        self._own(logits, temperature, seeds, counters)
        if logits.dtype != torch.float32 or temperature.dtype != torch.float32 or \
                seeds.dtype != torch.int64 or counters.dtype != torch.int64:
            raise KernelError("sample: logits/temperature float32, seeds/counters int64")
        rows, vocab = logits.shape
        out = torch.empty(rows, dtype=torch.int32, device=self.device)
        parts = self._ops.distie_argmax_parts(rows, vocab)
        values = indexes = sums = None
        if parts > 1:
            values = torch.empty(rows * parts, dtype=torch.float32, device=self.device)
            indexes = torch.empty(rows * parts, dtype=torch.int32, device=self.device)
            sums = torch.empty(rows * parts, dtype=torch.float32, device=self.device)
        _check(self._ops.distie_sample(logits.data_ptr(), temperature.data_ptr(), seeds.data_ptr(),
                                       counters.data_ptr(), out.data_ptr(), rows, vocab,
                                       values.data_ptr() if parts > 1 else None,
                                       indexes.data_ptr() if parts > 1 else None,
                                       sums.data_ptr() if parts > 1 else None, self._stream()), "sample")
        return out
