"""The engine's device ops: thin, checked wrappers over the HIP library.

Each method validates shapes, types and contiguity on the host (a kernel that
reads past a buffer can take the whole GPU down), then launches on torch's
current stream through ``ctypes``. There is no other implementation: if the
library cannot be built or loaded, construction fails. Tensors are torch
tensors on the GPU; outputs are allocated with torch's caching allocator.

Matrix products: float32 goes to the library's own fused-multiply-add kernel
(true 32-bit). bfloat16 with up to 64 rows (128 for the gated product and for
products cut along K) goes to the library's MFMA kernels, which stream the
weights; bfloat16 with more rows goes to the vendor BLAS through
``torch.matmul``, as the reference leaves its products to cuBLAS
(qwen3_runtime/models/qwen3.py:76-77,134-135).
"""

from __future__ import annotations

import ctypes
import math
from ctypes import POINTER, Structure, byref, c_float, c_int, c_long, c_void_p

import numpy as np
import torch

from . import build

F32, BF16 = 0, 1
_CODE = {torch.float32: F32, torch.bfloat16: BF16}


class OpsError(RuntimeError):
    pass


class _QkArgs(Structure):
    _fields_ = [
        ("q_in", c_void_p), ("q_stride", c_long),
        ("k_in", c_void_p), ("k_stride", c_long),
        ("v_in", c_void_p), ("v_stride", c_long),
        ("q_weight", c_void_p), ("k_weight", c_void_p), ("inv_freq", c_void_p),
        ("positions", c_void_p), ("slots", c_void_p),
        ("q_out", c_void_p), ("k_out", c_void_p), ("v_out", c_void_p),
        ("k_cache", c_void_p), ("v_cache", c_void_p),
        ("num_tokens", c_int), ("nq", c_int), ("nkv", c_int), ("nv", c_int),
        ("head_dim", c_int), ("page_size", c_int), ("eps", c_float), ("rope", c_void_p),
        ("value_dim", c_int), ("rot_pairs", c_int), ("v_rope", c_void_p),
    ]


class _AttnArgs(Structure):
    _fields_ = [
        ("q", c_void_p), ("out", c_void_p), ("k_cache", c_void_p), ("v_cache", c_void_p),
        ("positions", c_void_p), ("seq_of_token", c_void_p), ("block_table", c_void_p),
        ("table_width", c_int), ("num_tokens", c_int), ("nq", c_int), ("nkv", c_int),
        ("head_dim", c_int), ("page_size", c_int), ("window", c_int), ("scale", c_float),
        ("chunk", c_int), ("softcap", c_float), ("value_dim", c_int), ("gate", c_void_p), ("gate_stride", c_long),
        ("keep_first", c_int), ("sink", c_int), ("turn", c_void_p),
    ]


class _MixNormArgs(Structure):
    _fields_ = [
        ("x_in", c_void_p), ("x_out", c_void_p), ("y", c_void_p), ("mix", c_void_p), ("out_w", c_void_p),
        ("read", c_void_p), ("weight", c_void_p), ("bias", c_void_p), ("rows", c_void_p), ("out", c_void_p),
        ("num_out", c_int), ("hidden", c_int), ("streams", c_int), ("s_in", c_int), ("planes", c_int),
        ("y_dtype", c_int), ("out_dtype", c_int), ("plane_stride", c_long), ("eps", c_float),
    ]


class _AttnTileArgs(Structure):
    _fields_ = [
        ("q", c_void_p), ("out", c_void_p), ("k_cache", c_void_p), ("v_cache", c_void_p),
        ("cu_q", c_void_p), ("kv_lens", c_void_p), ("block_table", c_void_p),
        ("tile_seq", c_void_p), ("tile_row0", c_void_p), ("part_o", c_void_p), ("part_lse", c_void_p),
        ("table_width", c_int), ("num_tiles", c_int), ("nq", c_int), ("nkv", c_int),
        ("page_size", c_int), ("window", c_int), ("num_splits", c_int), ("waves", c_int),
        ("scale_log2", c_float), ("row_tiles", c_int), ("use_lds", c_int),
        ("merge_tokens", c_void_p), ("num_merge_tokens", c_int),
        ("qkv", c_void_p), ("qkv_stride", c_long), ("q_weight", c_void_p), ("k_weight", c_void_p),
        ("rope", c_void_p), ("slots", c_void_p), ("eps", c_float), ("split_blocks", c_int),
        ("max_items", c_int), ("items", c_void_p),
        ("chunk", c_int), ("cap_in", c_float), ("cap_out", c_float),
        ("gate", c_void_p), ("gate_stride", c_long), ("keep_first", c_int), ("sink", c_int),
        ("rope_pairs", c_int), ("turn", c_void_p),
    ]


class _ConvArgs(Structure):
    _fields_ = [
        ("x", c_void_p), ("x_stride", c_long), ("taps", c_void_p), ("tail", c_void_p),
        ("cu_q", c_void_p), ("seq_of_token", c_void_p), ("state_slots", c_void_p), ("out", c_void_p),
        ("num_tokens", c_int), ("channels", c_int), ("num_taps", c_int), ("nseg", c_int),
        ("seg_first", c_int * 4), ("seg_heads", c_int * 4), ("seg_width", c_int * 4), ("seg_mode", c_int * 4),
        ("total_heads", c_int), ("unit_eps", c_float), ("fuse_tail", c_int), ("bias", c_void_p),
        ("out_code", c_int), ("no_activation", c_int),
    ]


class _RotateArgs(Structure):
    _fields_ = [
        ("x", c_void_p), ("x_row", c_long), ("in_stride", c_int), ("in_offset", c_int),
        ("out", c_void_p), ("out_row", c_long), ("out_stride", c_int), ("out_offset", c_int),
        ("heads", c_int), ("width", c_int), ("pairs", c_int),
        ("positions", c_void_p), ("freq", c_void_p), ("scale_from_head", c_int), ("scale", c_float),
        ("neighbours", c_int), ("magnitude", c_float),
    ]


class _JointNormArgs(Structure):
    _fields_ = [
        ("qk", c_void_p), ("row", c_long), ("bias", c_void_p), ("q_weight", c_void_p), ("k_weight", c_void_p),
        ("positions", c_void_p), ("q_out", c_void_p), ("slots", c_void_p), ("k_cache", c_void_p), ("v_cache", c_void_p),
        ("page_size", c_int), ("nq", c_int), ("nkv", c_int), ("d", c_int), ("values_are_keys", c_int),
        ("eps", c_float), ("temp_coef", c_float), ("temp_every", c_int), ("num_tokens", c_int), ("group_values", c_int), ("wide", c_int),
    ]


class _RetentionArgs(Structure):
    _fields_ = [
        ("qkv", c_void_p), ("channels", c_int), ("q_first", c_int), ("k_first", c_int), ("v_first", c_int),
        ("decay", c_void_p), ("state", c_void_p), ("out", c_void_p), ("cu_q", c_void_p), ("state_slots", c_void_p),
        ("heads", c_int), ("dim", c_int), ("vdim", c_int), ("share", c_int),
        ("step", c_void_p), ("step_stride", c_long), ("step_code", c_int),
        ("step_bias", c_void_p), ("a_log", c_void_p), ("skip", c_void_p), ("qkv_code", c_int), ("seq_ids", c_void_p),
        ("gates", c_void_p), ("last_out", c_void_p),
    ]


class _SpaceArgs(Structure):
    _fields_ = [
        ("xbc", c_void_p), ("channels", c_int), ("x_first", c_int), ("b_first", c_int), ("c_first", c_int), ("step", c_void_p), ("step_stride", c_long), ("step_code", c_int),
        ("step_bias", c_void_p), ("a_log", c_void_p), ("skip", c_void_p), ("state", c_void_p), ("out", c_void_p),
        ("cu_q", c_void_p), ("state_slots", c_void_p), ("seq_ids", c_void_p),
        ("heads", c_int), ("groups", c_int), ("n", c_int), ("p", c_int), ("gates", c_void_p), ("last_out", c_void_p),
    ]


class _RuleArgs(Structure):
    _fields_ = [
        ("qkv", c_void_p), ("channels", c_int), ("q_first", c_int), ("k_first", c_int), ("v_first", c_int),
        ("b", c_void_p), ("b_stride", c_long), ("b_code", c_int),
        ("a", c_void_p), ("a_stride", c_long), ("a_code", c_int),
        ("a_log", c_void_p), ("dt_bias", c_void_p), ("state", c_void_p), ("out", c_void_p),
        ("cu_q", c_void_p), ("state_slots", c_void_p),
        ("heads", c_int), ("kv_heads", c_int), ("dim", c_int), ("vdim", c_int), ("per_channel", c_int),
    ]


ACTIVATIONS = {"swiglu": 0, "clamped": 1, "relu2": 2}  # relu2 has no gate


def _planes(y, t, h, name):
    """(pointer, dtype code, planes) of a sub-layer output: a matrix [T, H], or float32 planes [P, T, H]."""
    if y.dim() == 3:
        _need(y, name, torch.float32, (y.shape[0], t, h))
        return _ptr(y), F32, y.shape[0]
    _need(y, name, shape=(t, h))
    return _ptr(y), _CODE[y.dtype], 1


class _SampleArgs(Structure):
    _fields_ = [
        ("logits", c_void_p), ("work", c_void_p), ("counts", c_void_p), ("slot", c_void_p),
        ("fparams", c_void_p), ("iparams", c_void_p), ("seeds", c_void_p),
        ("out_token", c_void_p), ("out_logprob", c_void_p), ("rows", c_int), ("vocab", c_int),
        ("write_work", c_int), ("partials", c_void_p), ("parts", c_int),
    ]


def _load(name: str) -> ctypes.CDLL:
    path = build.build_library(name)
    try:
        lib = ctypes.CDLL(str(path))
    except OSError as exc:
        raise OpsError(f"cannot load {path}: {exc}") from exc
    if hasattr(lib, "qrt_last_error"):  # a library from outside need not link runtime.hip
        lib.qrt_last_error.restype = ctypes.c_char_p
    return lib


_core: ctypes.CDLL | None = None
_attn: dict[tuple[int, int], ctypes.CDLL] = {}


def core_library() -> ctypes.CDLL:
    global _core
    if _core is None:
        _core = _load("core")
    return _core


def attention_library(head_dim: int, value_dim: int | None = None) -> ctypes.CDLL:
    """The MFMA attention kernels of one size of keys and (None: the same) of values."""
    key = (head_dim, value_dim or head_dim)
    if key not in _attn:
        _attn[key] = _load(f"attn_bf16_d{head_dim}" + ("" if key[1] == head_dim else f"v{key[1]}"))
    return _attn[key]


_extra: dict[str, ctypes.CDLL] = {}


def load_library(name: str) -> ctypes.CDLL:
    """A library registered with ``ops.build.register_library``, built if need be, as a
    ``ctypes.CDLL``; its entry points take raw device pointers and ``current_stream()``."""
    if name not in _extra:
        _extra[name] = _load(name)
    return _extra[name]


def _ptr(t: torch.Tensor | None):
    return None if t is None else c_void_p(t.data_ptr())


def _addr(t: torch.Tensor | None):
    """Address for a structure field (ctypes takes an int or None there)."""
    return None if t is None else t.data_ptr()


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)
_raw_device = getattr(torch._C, "_cuda_getDevice", None)


def _stream() -> c_void_p:
    """torch's current stream on the current device. The two calls behind the public
    ``torch.cuda.current_stream()`` are used directly where this torch has them: the public one
    builds a Stream object and cost 9 us a launch, a quarter of a short prompt step's host time."""
    if _raw_stream is not None and _raw_device is not None:
        return c_void_p(_raw_stream(_raw_device()))
    return c_void_p(torch.cuda.current_stream().cuda_stream)


current_stream = _stream


def _need(t: torch.Tensor, name: str, dtype=None, shape=None) -> torch.Tensor:
    if not t.is_cuda:
        raise OpsError(f"{name} must be on the GPU, it is on {t.device}")
    if not t.is_contiguous():
        raise OpsError(f"{name} must be contiguous, strides are {t.stride()} for shape {tuple(t.shape)}")
    if dtype is not None and t.dtype != dtype:
        raise OpsError(f"{name} must be {dtype}, it is {t.dtype}")
    if shape is not None and tuple(t.shape) != tuple(shape):
        raise OpsError(f"{name} must have shape {tuple(shape)}, it has {tuple(t.shape)}")
    return t


check_tensor = _need  # for parts that call a library of their own


class HipOps:
    # bfloat16 products with more rows than this go to the vendor BLAS
    own_max_rows = 64
    # the same for the two forms in which a block fetches fewer activations than weights: the
    # gated product, and the product cut along K whose planes the residual's norm adds
    own_max_rows_shared = 128
    # Rows from which a product takes the kernel that shares the activations through LDS
    # instead of the few-row kernel (both stream the weights as stored, through LDS by direct
    # loads). Measured at the 4B shapes on the matrices of 36 layers in turn: cut along K the
    # sharing kernel is faster from 9 rows on, gated from 12 rows on. (Timed on one weight
    # matrix over and over, the sharing kernel looks 15 to 40 % faster than the few-row kernel
    # down to one row, because a matrix of up to some 100 MB then stays in the memory-side
    # cache; in a step it is 5 % slower at 8 rows, and a decode step with it from one row on
    # lost 3 % at batch 8 and 9 % at batch 1.)
    shared_from_rows = {"whole": 17, "gated": 12, "planes": 9}
    # steps of single tokens: norm, rotation, cache write and attention in one kernel
    fuse_decode = True
    # tiles of 16 rows per wave in the attention kernel for long portions (1 or 2)
    prefill_row_tiles = 2
    # long portions: keys and values go through LDS, shared by the four waves of a block
    prefill_through_lds = True
    # ... in blocks of eight waves, two groups that take the blocks of keys in turn: 1 never, 2 always,
    # None where the longest tile's chain of rounds would otherwise set the kernel's time
    prefill_key_groups = None

    def __init__(self):
        self.lib = core_library()

    def _check(self, lib, code: int) -> None:
        if code != 0:
            raise OpsError(lib.qrt_last_error().decode())

    # ---- embedding, norms, activations ---------------------------------------
    def embed(self, ids, table, scale=1.0):
        _need(ids, "ids", torch.int32)
        _need(table, "embedding table")
        t, (v, h) = ids.numel(), table.shape
        out = torch.empty((t, h), dtype=torch.float32, device=table.device)
        self._check(self.lib, self.lib.qrt_embed(_ptr(ids), _ptr(table), _CODE[table.dtype], _ptr(out),
                                                 c_int(t), c_int(v), c_int(h), c_float(scale), _stream()))
        return out

    def embed_pairs(self, ctx, ids, table, pairs, mul_prev, mul_cur, last):
        """Rows of ``table`` plus rows of ``pairs`` [buckets + 1, H], which (previous token * mul_prev + token *
        mul_cur) mod buckets picks, the last one for a sequence's first token; float32 [T, H]. ``last`` int32
        [slots, 1] holds each request's last token and is brought up to date."""
        t, (_, h) = ids.numel(), table.shape
        _need(ids, "ids", torch.int32, (ctx.num_tokens,))
        _need(table, "embedding table")
        _need(pairs, "table of pairs", shape=(pairs.shape[0], h))
        _need(last, "last tokens", torch.int32, (last.shape[0], 1))
        _need(ctx.positions, "positions", torch.int32, (t,))
        _need(ctx.seq_of_token, "seq_of_token", torch.int32, (t,))
        _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,))
        _need(ctx.state_slots, "state_slots", torch.int32, (ctx.num_seqs,))
        out = torch.empty((t, h), dtype=torch.float32, device=table.device)
        self._check(self.lib, self.lib.qrt_embed_pairs(
            _ptr(ids), _ptr(ctx.positions), _ptr(ctx.seq_of_token), _ptr(ctx.cu_q), _ptr(ctx.state_slots), _ptr(table),
            _CODE[table.dtype], _ptr(pairs), _CODE[pairs.dtype], _ptr(last), _ptr(out), c_int(t), c_int(h),
            c_int(pairs.shape[0] - 1), c_long(mul_prev), c_long(mul_cur), _stream()))
        return out

    def scale(self, x, factor):
        """``x *= factor`` in place, float32."""
        _need(x, "x", torch.float32)
        self._check(self.lib, self.lib.qrt_scale(_ptr(x), c_float(factor), c_long(x.numel()), _stream()))
        return x

    def softcap(self, x, limit):
        """``x = limit * tanh(x / limit)`` in place, float32."""
        _need(x, "x", torch.float32)
        self._check(self.lib, self.lib.qrt_softcap(_ptr(x), c_float(limit), c_long(x.numel()), _stream()))
        return x

    def unary_act(self, x, kind):
        """An activation without a gate, element by element: ``relu2`` is ``max(x, 0)^2``."""
        _need(x, "x")
        out = torch.empty_like(x)
        self._check(self.lib, self.lib.qrt_unary_act(_ptr(x), _ptr(out), _CODE[x.dtype], c_long(x.numel()),
                                                     c_int({"relu2": 0}[kind]), _stream()))
        return out

    def new_rows(self, t, width, dtype, device):
        return torch.empty((t, width), dtype=dtype, device=device)

    def add_rmsnorm(self, residual, delta, weight, eps, out_dtype, rows=None, delta_scale=1.0, delta_norm=None):
        """``residual += delta_scale * delta`` in place (``delta`` a matrix or float32 planes), then the
        rows' RMS norm; with ``rows`` only those, and ``residual`` is left alone. ``delta_norm`` =
        (weight, eps): ``delta`` joins the stream as ``delta / rms(delta) * weight``."""
        if delta_norm is not None:
            return self._norm_add_rmsnorm(residual, delta, delta_norm[0], delta_norm[1], weight, eps, out_dtype, rows)
        t, h = residual.shape
        _need(residual, "residual", torch.float32)
        _need(weight, "norm weight", torch.float32, (h,))
        planes, plane_stride = 1, 0
        if delta is not None:
            if delta.dim() == 3:  # the parts of a product whose K was cut: added here, in order
                planes, plane_stride = delta.shape[0], t * h
                _need(delta, "delta", shape=(planes, t, h))
            else:
                _need(delta, "delta", shape=(t, h))
        n_out = t
        if rows is not None:
            _need(rows, "rows", torch.int32)
            n_out = rows.numel()
        out = torch.empty((n_out, h), dtype=out_dtype, device=residual.device)
        self._check(self.lib, self.lib.qrt_add_rmsnorm(
            _ptr(residual), _ptr(delta), _CODE[delta.dtype] if delta is not None else F32, _ptr(weight),
            _ptr(rows), _ptr(out), _CODE[out_dtype], c_int(n_out), c_int(h), c_float(eps), c_int(planes),
            c_long(plane_stride), c_float(delta_scale), _stream()))
        return out

    def _norm_add_rmsnorm(self, residual, y, w_after, eps_after, weight, eps, out_dtype, rows):
        t, h = residual.shape
        _need(residual, "residual", torch.float32)
        _need(weight, "norm weight", torch.float32, (h,))
        _need(w_after, "weight of the norm behind the sub-layer", torch.float32, (h,))
        py, cy, ny = _planes(y, t, h, "sub-layer output")
        n_out = t
        if rows is not None:
            _need(rows, "rows", torch.int32)
            n_out = rows.numel()
        out = torch.empty((n_out, h), dtype=out_dtype, device=residual.device)
        self._check(self.lib, self.lib.qrt_norm_add_rmsnorm(
            _ptr(residual), py, c_int(cy), c_int(ny), c_long(t * h), _ptr(w_after), c_float(eps_after), _ptr(weight),
            c_float(eps), _ptr(rows), _ptr(out), _CODE[out_dtype], c_int(n_out), c_int(h), _stream()))
        return out

    def scaled_add_rmsnorm(self, residual, parts, weight, eps, out_dtype, rows=None, vector=None):
        """``residual += sum_i scale_i * y_i (+ vector)`` in place, element by element (``parts``: up to four
        (y, scale), ``y`` a matrix or float32 planes, ``scale`` float32 [H]; ``vector`` float32 [H]), then the rows' RMS norm;
        with ``rows`` only those, and ``residual`` is left alone."""
        t, h = residual.shape
        _need(residual, "residual", torch.float32)
        _need(weight, "norm weight", torch.float32, (h,))
        n = len(parts)
        if not (0 if vector is not None else 1) <= n <= 4:
            raise OpsError(f"a sum of {n} scaled outputs (1 to 4)")
        if vector is not None:
            _need(vector, "vector", torch.float32, (h,))
        ptrs, codes, counts, scales = (c_void_p * n)(), (c_int * n)(), (c_int * n)(), (c_void_p * n)()
        for i, (y, scale) in enumerate(parts):
            py, codes[i], counts[i] = _planes(y, t, h, "sub-layer output")
            ptrs[i] = py.value if hasattr(py, "value") else py
            scales[i] = _need(scale, "vector of a sub-layer's output", torch.float32, (h,)).data_ptr()
        n_out = t
        if rows is not None:
            _need(rows, "rows", torch.int32)
            n_out = rows.numel()
        out = torch.empty((n_out, h), dtype=out_dtype, device=residual.device)
        self._check(self.lib, self.lib.qrt_scaled_add_rmsnorm(
            _ptr(residual), ptrs, codes, counts, scales, c_int(n), _ptr(vector), c_long(t * h), _ptr(weight), c_float(eps), _ptr(rows),
            _ptr(out), _CODE[out_dtype], c_int(n_out), c_int(h), _stream()))
        return out

    # ---- norms in groups of the row ---------------------------------------------------
    def group_norm_update(self, residual, y, after, norm, groups, out_dtype, rows=None):
        """``residual += y`` in place (``y`` a matrix or float32 planes, or None: nothing is pending), ``y``
        first RMS-normed in ``groups`` equal parts of the row if ``after`` = (weight, eps) is given; returns
        the rows of the sum in ``out_dtype``, normed likewise by ``norm`` = (weight, eps), or (None) as they
        are. With ``rows`` only those, and ``residual`` is left alone."""
        t, h = residual.shape
        _need(residual, "residual", torch.float32)
        if groups < 1 or h % groups:
            raise OpsError(f"a norm of {h} elements in {groups} equal parts")
        py, cy, ny = (None, F32, 1) if y is None else _planes(y, t, h, "sub-layer output")
        wa, ea = (None, 0.0) if after is None else after
        wn, en = (None, 0.0) if norm is None else norm
        for name, w in (("weight of the norm behind the sub-layer", wa), ("norm weight", wn)):
            if w is not None:
                _need(w, name, torch.float32, (h,))
        n_out = t
        if rows is not None:
            _need(rows, "rows", torch.int32)
            n_out = rows.numel()
        out = torch.empty((n_out, h), dtype=out_dtype, device=residual.device)
        self._check(self.lib, self.lib.qrt_group_norm_update(
            _ptr(residual), py, c_int(cy), c_int(ny), c_long(t * h), _ptr(wa), c_float(ea), _ptr(wn), c_float(en), _ptr(rows),
            _ptr(out), _CODE[out_dtype], c_int(n_out), c_int(h), c_int(groups), _stream()))
        return out

    def gated_group_norm(self, o, gate, weight, eps, groups, out_dtype):
        """``v = o * silu(gate)`` over all heads of a token, then the RMS norm of ``v`` in ``groups`` equal parts
        times ``weight``; ``gate`` may be columns of a wider matrix. [T, heads * vdim]."""
        t, heads, vdim = o.shape
        width = heads * vdim
        _need(o, "read-out", torch.float32)
        _need(weight, "read-out norm weight", torch.float32, (width,))
        if not gate.is_cuda or tuple(gate.shape) != (t, width) or gate.stride(1) != 1 or gate.dtype not in _CODE:
            raise OpsError(f"gate {tuple(gate.shape)} {gate.dtype} does not fit {t} tokens of {width} channels")
        if groups < 1 or width % groups:
            raise OpsError(f"a norm of {width} elements in {groups} equal parts")
        out = torch.empty((t, width), dtype=out_dtype, device=o.device)
        self._check(self.lib, self.lib.qrt_gated_group_norm(
            _ptr(o), c_void_p(gate.data_ptr()), c_long(gate.stride(0)), _CODE[gate.dtype], _ptr(weight), c_float(eps), _ptr(out),
            _CODE[out_dtype], c_int(t), c_int(width), c_int(groups), _stream()))
        return out

    # ---- attention through a latent, retention ------------------------------------------
    def rmsnorm_columns(self, y, first, width, weight, eps):
        """The RMS norm of columns ``first .. first + width`` of ``y`` [T, W], [T, width] in ``y``'s type."""
        t, w = y.shape
        _need(y, "y")
        _need(weight, "norm weight", torch.float32, (width,))
        if not 0 <= first <= first + width <= w:
            raise OpsError(f"columns {first}..{first + width} of {w}")
        out = torch.empty((t, width), dtype=y.dtype, device=y.device)
        self._check(self.lib, self.lib.qrt_rmsnorm_columns(_ptr(y), c_long(w), c_int(first), c_int(width), _ptr(weight),
                                                           c_float(eps), _ptr(out), _CODE[y.dtype], c_int(t), _stream()))
        return out

    def latent_store(self, y, first, rank, rot_dim, weight, eps, positions, freq, cache, neighbours=False, magnitude=1.0):
        """Columns ``first .. first + rank`` of ``y`` RMS-normed (the latent ``c``) and the ``rot_dim``
        columns behind them rotated (rotate-half over the first ``2 len(freq)``; ``neighbours``: element
        2i against 2i + 1; cosines and sines times ``magnitude``) go into the cache of
        one key/value head: the key row ``[c | k_rot]``, the value row ``[c | 0]``."""
        if cache is None:
            return
        t, w = y.shape
        width = rank + rot_dim
        _need(y, "y")
        _need(weight, "latent norm weight", torch.float32, (rank,))
        pairs = 0 if freq is None else freq.numel()
        if pairs:
            _need(freq, "freq", torch.float32, (pairs,))
        _need(positions, "positions", torch.int32, (t,))
        pages = self._check_cache(cache, 1, width, y.dtype)
        _need(cache.group.slots, "slots", torch.int32, (t,))
        if not 0 <= first <= first + width <= w or 2 * pairs > rot_dim:
            raise OpsError(f"latent_store: columns {first}..{first + width} of {w}, {pairs} pairs in {rot_dim}")
        self._check(self.lib, self.lib.qrt_latent_store(
            _ptr(y), c_long(w), c_int(first), c_int(rank), c_int(rot_dim), _ptr(weight), c_float(eps), _ptr(positions),
            _ptr(freq), c_int(pairs), _ptr(cache.group.slots), _ptr(cache.k), _ptr(cache.v), c_int(cache.group.page_size),
            c_long(pages), _CODE[y.dtype], c_int(t), c_int(bool(neighbours)), c_float(magnitude), _stream()))

    def rotate_half(self, x, in_stride, in_offset, out, out_stride, out_offset, heads, width, positions, freq,
                    scale_from_head=None, scale=1.0, neighbours=False, magnitude=1.0):
        """For every token and head copy ``width`` elements from ``x[t, h * in_stride + in_offset ...]`` to
        ``out[t, h * out_stride + out_offset ...]``, the first ``2 len(freq)`` of them turned (element i
        against element i + len(freq), by ``position * freq[i]``); heads from ``scale_from_head`` on are
        multiplied by ``scale``. ``neighbours``: element 2i turns against element 2i + 1 instead; cosines and
        sines are multiplied by ``magnitude``. ``out`` may be float32 for a bfloat16 ``x``."""
        t = x.shape[0]
        _need(x, "x")
        _need(out, "out", shape=(t, out.shape[1]))
        pairs = 0 if freq is None else freq.numel()
        a = _RotateArgs()
        a.x, a.x_row, a.in_stride, a.in_offset = x.data_ptr(), x.shape[1], in_stride, in_offset
        a.out, a.out_row, a.out_stride, a.out_offset = out.data_ptr(), out.shape[1], out_stride, out_offset
        a.heads, a.width, a.pairs = heads, width, pairs
        if pairs:
            a.freq = _need(freq, "freq", torch.float32, (pairs,)).data_ptr()
            a.positions = _need(positions, "positions", torch.int32, (t,)).data_ptr()
        a.scale_from_head, a.scale = heads if scale_from_head is None else scale_from_head, scale
        a.neighbours, a.magnitude = int(bool(neighbours)), magnitude
        self._check(self.lib, self.lib.qrt_rotate_half(byref(a), _CODE[x.dtype], _CODE[out.dtype], c_int(t), _stream()))
        return out

    # bfloat16 steps with more tokens than this take the per-head products to the vendor library
    heads_linear_own_max_rows = 16

    def heads_linear(self, x, in_stride, in_offset, w, out, out_stride, out_offset):
        """A product per head on strided rows: ``out[t, h * out_stride + out_offset + n] =
        sum_k w[h, n, k] x[t, h * in_stride + in_offset + k]``; ``w`` [heads, N, K]."""
        t = x.shape[0]
        heads, n, k = w.shape
        _need(x, "x")
        _need(w, "weights", x.dtype)
        _need(out, "out", x.dtype, (t, out.shape[1]))
        if (heads * in_stride > x.shape[1] or in_offset + k > in_stride or heads * out_stride > out.shape[1]
                or out_offset + n > out_stride):
            raise OpsError(f"heads_linear: {heads} heads of {in_stride} in rows of {x.shape[1]}, of {out_stride} in rows of {out.shape[1]}")
        if x.dtype == torch.bfloat16 and t > self.heads_linear_own_max_rows:
            src = x.view(t, -1)[:, : heads * in_stride].view(t, heads, in_stride)[:, :, in_offset: in_offset + k]
            res = torch.bmm(src.transpose(0, 1), w.transpose(1, 2))  # [heads, T, N]
            out.view(t, -1)[:, : heads * out_stride].view(t, heads, out_stride)[:, :, out_offset: out_offset + n] = \
                res.transpose(0, 1)
            return out
        self._check(self.lib, self.lib.qrt_heads_linear(
            _ptr(x), c_long(x.shape[1]), c_int(in_stride), c_int(in_offset), _ptr(w), c_int(heads), c_int(n), c_int(k),
            _ptr(out), c_long(out.shape[1]), c_int(out_stride), c_int(out_offset), _CODE[x.dtype], c_int(t), _stream()))
        return out

    def retention_prepare(self, y, heads, dim, vdim, positions, freq, k_scale):
        """float32 [T, 2 heads dim + heads vdim] from the first columns of a product ``y``: queries and
        keys with their first ``2 len(freq)`` elements a head turned (rotate-half), keys then times
        ``k_scale``, values as they are."""
        t, w = y.shape
        c = 2 * heads * dim + heads * vdim
        if c > w:
            raise OpsError(f"retention_prepare: {c} channels in {w} columns")
        out = torch.empty((t, c), dtype=torch.float32, device=y.device)
        self.rotate_half(y, dim, 0, out, dim, 0, 2 * heads, dim, positions, freq, scale_from_head=heads, scale=k_scale)
        # the values: a copy into float32 behind them
        a = _RotateArgs()
        _need(y, "y")
        a.x, a.x_row, a.in_stride, a.in_offset = y.data_ptr() + 2 * heads * dim * y.element_size(), w, vdim, 0
        a.out, a.out_row, a.out_stride, a.out_offset = out.data_ptr() + 2 * heads * dim * 4, c, vdim, 0
        a.heads, a.width, a.pairs, a.scale_from_head, a.scale = heads, vdim, 0, heads, 1.0
        a.magnitude = 1.0
        self._check(self.lib, self.lib.qrt_rotate_half(byref(a), _CODE[y.dtype], F32, c_int(t), _stream()))
        return out

    def retention_rule(self, ctx, qkv, decay, state, heads, dim, vdim):
        """``S <- decay S + k v^T; o = S^T q`` over each sequence's tokens from its slot's state (float32
        [slots, heads, vdim, dim], updated in place); ``qkv`` float32 [T, C] as ``retention_prepare``
        leaves it. Returns the read-outs, float32 [T, heads, vdim]."""
        t = ctx.num_tokens
        c = 2 * heads * dim + heads * vdim
        _need(qkv, "q | k | v", torch.float32, (t, c))
        _need(state, "state", torch.float32, (state.shape[0], heads, vdim, dim))
        _need(decay, "decay", torch.float32, (heads,))
        a = _RetentionArgs()
        a.qkv, a.channels, a.q_first, a.k_first, a.v_first = qkv.data_ptr(), c, 0, heads * dim, 2 * heads * dim
        a.decay, a.state = decay.data_ptr(), state.data_ptr()
        out = torch.empty((t, heads, vdim), dtype=torch.float32, device=qkv.device)
        a.out = out.data_ptr()
        a.cu_q = _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,)).data_ptr()
        a.state_slots = _need(ctx.state_slots, "state_slots", torch.int32, (ctx.num_seqs,)).data_ptr()
        a.heads, a.dim, a.vdim = heads, dim, vdim
        self._check(self.lib, self.lib.qrt_retention(byref(a), c_int(t), c_int(ctx.num_seqs), c_int(state.shape[0]), _stream()))
        return out

    def state_space(self, ctx, xbc, step, step_bias, a_log, skip, state, heads, groups, n, vdim):
        """Per sequence and head from the slot's state (float32 [slots, heads, vdim, n], updated in place):
        ``D = softplus(step + step_bias); S <- exp(-exp(a_log) D) S + (D x) B^T; y = S C + skip x``. ``xbc``
        [T, heads * vdim | groups * n | groups * n] (x, B, C; head h uses group h // (heads / groups)),
        float32 or bfloat16; ``step`` [T, heads] may be columns of a wider matrix. Returns y, float32 [T, heads,
        vdim]. Float32 inputs, short spans and odd sizes go token by token; long spans of bfloat16
        inputs chunk by chunk, in a launch of their own beside the short ones of the same step."""
        t = ctx.num_tokens
        c = heads * vdim + 2 * groups * n
        _need(xbc, "x | B | C", shape=(t, c))
        _need(state, "state", torch.float32, (state.shape[0], heads, vdim, n))
        if not step.is_cuda or tuple(step.shape) != (t, heads) or step.stride(1) != 1 or step.dtype not in _CODE:
            raise OpsError(f"step logits: {tuple(step.shape)} {step.dtype} with strides {step.stride()} for {t} tokens of {heads}")
        if heads % groups:
            raise OpsError(f"{heads} heads in {groups} groups")
        consts = {name: _need(w, name, torch.float32, (heads,)).data_ptr()
                  for name, w in (("step_bias", step_bias), ("a_log", a_log), ("skip", skip))}
        cu_q = _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,)).data_ptr()
        slots = _need(ctx.state_slots, "state_slots", torch.int32, (ctx.num_seqs,)).data_ptr()
        out = torch.empty((t, heads, vdim), dtype=torch.float32, device=xbc.device)
        chunked, short, num_chunked, short_tokens = self._space_split(ctx, xbc, n, vdim)
        if num_chunked:
            b = _SpaceArgs()
            b.xbc, b.channels, b.step, b.step_stride, b.step_code = xbc.data_ptr(), c, step.data_ptr(), step.stride(0), _CODE[step.dtype]
            b.state, b.out, b.cu_q, b.state_slots, b.seq_ids = state.data_ptr(), out.data_ptr(), cu_q, slots, _addr(chunked)
            b.heads, b.groups, b.n, b.p = heads, groups, n, vdim
            b.x_first, b.b_first, b.c_first = 0, heads * vdim, heads * vdim + groups * n
            for name, ptr in consts.items():
                setattr(b, name, ptr)
            self._check(self.lib, self.lib.qrt_state_space_chunks(byref(b), c_int(num_chunked), _stream()))
        if num_chunked < ctx.num_seqs:
            a = _RetentionArgs()
            a.qkv, a.qkv_code, a.channels = xbc.data_ptr(), _CODE[xbc.dtype], c
            a.v_first, a.k_first, a.q_first = 0, heads * vdim, heads * vdim + groups * n
            a.step, a.step_stride, a.step_code = step.data_ptr(), step.stride(0), _CODE[step.dtype]
            for name, ptr in consts.items():
                setattr(a, name, ptr)
            a.state, a.out, a.cu_q, a.state_slots, a.seq_ids = state.data_ptr(), out.data_ptr(), cu_q, slots, _addr(short)
            a.heads, a.dim, a.vdim, a.share = heads, n, vdim, heads // groups
            self._check(self.lib, self.lib.qrt_retention(byref(a), c_int(short_tokens), c_int(ctx.num_seqs - num_chunked),
                                                         c_int(state.shape[0]), _stream()))
        return out

    # ---- matrix memory -----------------------------------------------------------------
    def memory_gates(self, ctx, logits, bias, cap, top, heads):
        """From the logits [T, heads input | heads forget] (float32; + ``bias``, softly held to ``cap``) and the
        running maxima ``top`` [slots, heads] (brought up to date): float32 [T, 3, heads], the logarithms of
        what a token keeps of the memory and of what its write weighs, and its running maximum."""
        t = ctx.num_tokens
        _need(logits, "gate logits", torch.float32, (t, 2 * heads))
        _need(bias, "gate biases", torch.float32, (2 * heads,))
        _need(top, "running maxima", torch.float32, (top.shape[0], heads))
        _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,))
        _need(ctx.state_slots, "state_slots", torch.int32, (ctx.num_seqs,))
        out = torch.empty((t, 3, heads), dtype=torch.float32, device=logits.device)
        self._check(self.lib, self.lib.qrt_memory_gates(_ptr(logits), _ptr(bias), c_float(cap), _ptr(top), _ptr(out), _ptr(ctx.cu_q),
                                                        _ptr(ctx.state_slots), c_int(heads), c_int(t), c_int(ctx.num_seqs),
                                                        c_int(ctx.max_q_len), _stream()))
        return out

    def matrix_memory(self, ctx, y, gates, state, heads, dim, vdim):
        """``S <- keep S + write k [v | 1]^T; o = S^T q`` over each sequence's tokens from its slot's state (float32
        [slots, heads, vdim + 1, dim], updated in place). ``y`` [T, W]: its first columns are q | k | v; ``gates``
        as ``memory_gates`` leaves them. Returns (o float32 [T, heads, vdim], the last column's [T, heads]). Float32
        inputs, short spans and odd sizes go token by token; long spans of bfloat16 inputs chunk by chunk, in
        a launch of their own beside the short ones of the same step."""
        t, w = y.shape
        c = 2 * heads * dim + heads * vdim
        _need(y, "q | k | v", shape=(ctx.num_tokens, w))
        if c > w:
            raise OpsError(f"matrix_memory: {c} channels in {w} columns")
        _need(state, "state", torch.float32, (state.shape[0], heads, vdim + 1, dim))
        _need(gates, "gates", torch.float32, (t, 3, heads))
        out = torch.empty((t, heads, vdim), dtype=torch.float32, device=y.device)
        last = torch.empty((t, heads), dtype=torch.float32, device=y.device)
        cu_q = _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,)).data_ptr()
        slots = _need(ctx.state_slots, "state_slots", torch.int32, (ctx.num_seqs,)).data_ptr()
        chunked, short, num_chunked, short_tokens = self._space_split(ctx, y, dim, vdim)
        if num_chunked:
            b = _SpaceArgs()
            b.xbc, b.channels, b.x_first, b.b_first, b.c_first = y.data_ptr(), w, 2 * heads * dim, heads * dim, 0
            b.gates, b.last_out, b.state, b.out = gates.data_ptr(), last.data_ptr(), state.data_ptr(), out.data_ptr()
            b.cu_q, b.state_slots, b.seq_ids = cu_q, slots, _addr(chunked)
            b.heads, b.groups, b.n, b.p = heads, heads, dim, vdim
            self._check(self.lib, self.lib.qrt_state_space_chunks(byref(b), c_int(num_chunked), _stream()))
        if num_chunked < ctx.num_seqs:
            a = _RetentionArgs()
            a.qkv, a.qkv_code, a.channels, a.q_first, a.k_first, a.v_first = y.data_ptr(), _CODE[y.dtype], w, 0, heads * dim, 2 * heads * dim
            a.gates, a.last_out, a.state, a.out = gates.data_ptr(), last.data_ptr(), state.data_ptr(), out.data_ptr()
            a.cu_q, a.state_slots, a.seq_ids = cu_q, slots, _addr(short)
            a.heads, a.dim, a.vdim = heads, dim, vdim
            self._check(self.lib, self.lib.qrt_retention(byref(a), c_int(short_tokens), c_int(ctx.num_seqs - num_chunked),
                                                         c_int(state.shape[0]), _stream()))
        return out, last

    def memory_out(self, read, norm_read, gates, weight, out_gate, eps, q_scale, out_dtype):
        """Per head ``o = s read / (max(|s norm_read|, exp(-m)) + 1e-6)`` (s = ``q_scale``), divided by its root mean
        square, times ``weight`` (of all heads) and sigmoid(``out_gate``), columns of a wider matrix; [T, heads * vdim]."""
        t, heads, vdim = read.shape
        _need(read, "read-out", torch.float32)
        _need(norm_read, "normaliser's read-out", torch.float32, (t, heads))
        _need(gates, "gates", torch.float32, (t, 3, heads))
        _need(weight, "read-out norm weight", torch.float32, (heads * vdim,))
        if not out_gate.is_cuda or tuple(out_gate.shape) != (t, heads * vdim) or out_gate.stride(1) != 1 or out_gate.dtype not in _CODE:
            raise OpsError(f"gate {tuple(out_gate.shape)} {out_gate.dtype} does not fit {t} tokens of {heads} heads of {vdim}")
        out = torch.empty((t, heads * vdim), dtype=out_dtype, device=read.device)
        self._check(self.lib, self.lib.qrt_memory_out(
            _ptr(read), _ptr(norm_read), _ptr(gates), _ptr(weight), c_void_p(out_gate.data_ptr()), c_long(out_gate.stride(0)),
            _CODE[out_gate.dtype], _ptr(out), _CODE[out_dtype], c_int(t), c_int(heads), c_int(vdim), c_float(eps), c_float(q_scale),
            _stream()))
        return out

    # spans of at least this many tokens run chunk by chunk
    space_chunk_min_tokens = 16

    def _space_split(self, ctx, xbc, n, vdim):
        """(ids of the sequences that run chunk by chunk or None for all, ids of the others or None for
        all, how many of the first, tokens of the others): the same for every layer of the step."""
        if xbc.dtype != torch.bfloat16 or n > 256 or n % 8 or vdim % 8 or ctx.max_q_len < self.space_chunk_min_tokens:
            return None, None, 0, ctx.num_tokens
        plan = ctx.scratch.get("space_split")
        if plan is None:
            is_long = [q >= self.space_chunk_min_tokens for q in ctx.q_lens_host]
            if all(is_long):
                plan = (None, None, ctx.num_seqs, 0)
            else:
                ids = lambda keep: torch.tensor([s for s, x in enumerate(is_long) if x == keep], dtype=torch.int32, device=xbc.device)  # noqa: E731
                plan = (ids(True), ids(False), sum(is_long), sum(q for q, x in zip(ctx.q_lens_host, is_long) if not x))
            ctx.scratch["space_split"] = plan
        return plan

    # ---- steps between sub-layers that are neither a product nor a plain norm -----------
    def norm_mean(self, ya, wa, yb, wb, eps):
        """``(rmsnorm(ya) * wa + rmsnorm(yb) * wb) / 2`` over the rows, float32 [T, H]; either input a
        matrix or float32 planes whose sum it is."""
        t, h = ya.shape[-2:]
        pa, ca, na = _planes(ya, t, h, "left output")
        pb, cb, nb = _planes(yb, t, h, "right output")
        _need(wa, "left weight", torch.float32, (h,))
        _need(wb, "right weight", torch.float32, (h,))
        out = torch.empty((t, h), dtype=torch.float32, device=wa.device)
        self._check(self.lib, self.lib.qrt_norm_mean(pa, c_int(ca), c_int(na), pb, c_int(cb), c_int(nb), _ptr(wa), _ptr(wb),
                                                     _ptr(out), c_int(t), c_int(h), c_float(eps), _stream()))
        return out

    def add_concat(self, residual, delta, delta_scale, origin, out_dtype):
        """``[residual + delta_scale * delta | origin]``, [T, 2H] in ``out_dtype``."""
        t, h = residual.shape
        _need(residual, "residual", torch.float32)
        _need(origin, "origin", torch.float32, (t, h))
        pd, cd, nd = (None, F32, 1) if delta is None else _planes(delta, t, h, "delta")
        out = torch.empty((t, 2 * h), dtype=out_dtype, device=residual.device)
        self._check(self.lib, self.lib.qrt_add_concat(_ptr(residual), pd, c_int(cd), c_int(nd), c_float(delta_scale),
                                                      _ptr(origin), _ptr(out), _CODE[out_dtype], c_int(t), c_int(h), _stream()))
        return out

    def accumulate(self, acc, y):
        """``acc += y`` (float32 [T, H]; ``y`` a matrix or planes); returns ``acc``."""
        t, h = acc.shape
        _need(acc, "sum", torch.float32)
        py, cy, ny = _planes(y, t, h, "addend")
        self._check(self.lib, self.lib.qrt_accumulate(_ptr(acc), py, c_int(cy), c_int(ny), c_long(t * h), _stream()))
        return acc

    def gated_act(self, gate_up, activation="swiglu", limit=0.0, scale=None, order=None, row_scale=None):
        """The gated activation of [T, 2I] (gate columns first): ``swiglu``, or ``clamped``, row t of it times
        ``row_scale[t]`` (float32). With ``scale`` (float32 [T]) both halves of row t are first multiplied by ``scale[order[t]]`` (``order`` None: ``scale[t]``)."""
        if scale is not None:
            _need(scale, "row scales", torch.float32)
            if order is not None:
                _need(order, "order", torch.int32, (gate_up.shape[0],))
            if scale.numel() != gate_up.shape[0]:
                raise OpsError(f"{scale.numel()} row scales for {gate_up.shape[0]} rows")
        if row_scale is not None:
            _need(row_scale, "row factors", torch.float32, (gate_up.shape[0],))
        _need(gate_up, "gate_up")
        t, two_i = gate_up.shape
        if two_i % 2:
            raise OpsError(f"gate_up has odd width {two_i}")
        out = torch.empty((t, two_i // 2), dtype=gate_up.dtype, device=gate_up.device)
        self._check(self.lib, self.lib.qrt_gated_act(_ptr(gate_up), _ptr(out), _CODE[gate_up.dtype], c_int(t),
                                                     c_int(two_i // 2), c_int(ACTIVATIONS[activation]), c_float(limit),
                                                     _ptr(scale), _ptr(order), _ptr(row_scale), _stream()))
        return out

    def bias_rotate_pairs(self, x, bias, positions, freq, rot_heads, head_dim):
        """In place on a product's output [T, W]: add ``bias`` [W] (float32; None: none), then turn
        the first ``2 * len(freq)`` elements of each of the first ``rot_heads`` heads of ``head_dim``
        columns, in interleaved pairs, by ``positions * freq`` (``freq`` None: no rotation)."""
        t, w = x.shape
        _need(x, "x")
        if bias is not None:
            _need(bias, "bias", torch.float32, (w,))
        pairs = 0
        if freq is not None:
            pairs = freq.numel()
            _need(freq, "freq", torch.float32, (pairs,))
            _need(positions, "positions", torch.int32, (t,))
        self._check(self.lib, self.lib.qrt_bias_rotate_pairs(_ptr(x), c_long(x.stride(0)), c_int(w), _CODE[x.dtype], _ptr(bias),
                                                             _ptr(positions) if freq is not None else None, _ptr(freq),
                                                             c_int(rot_heads), c_int(head_dim), c_int(pairs), c_int(t), _stream()))
        return x

    # ---- gated delta rule ---------------------------------------------------------------
    def delta_conv(self, ctx, y, channels, taps, tail, segments, unit_eps, first=0, bias=None, out_dtype=torch.float32,
                   activation="silu"):
        """``channels`` columns of ``y`` [T, W], from column ``first`` on, through their causal convolutions
        (``taps`` float32 [C, K]; ``bias`` float32 [C] or None is added) and silu (``activation`` None: without), then per head as ``segments`` say, each (heads, width,
        mode): 0 as it is, 1 scaled to a unit vector, 2 that times width^(-1/2). [T, C] in ``out_dtype``.
        ``tail`` [slots, C, K-1] float32 holds each request's last inputs and is brought up to date."""
        t, w = y.shape
        _need(y, "projections")
        k = taps.shape[1]
        _need(taps, "taps", torch.float32, (channels, k))
        slots = tail.shape[0]
        _need(tail, "convolution tail", torch.float32, (slots, channels, max(k - 1, 1)))
        if t != ctx.num_tokens or first < 0 or first + channels > w or not 1 <= len(segments) <= 4:
            raise OpsError(f"delta_conv: {t} rows for {ctx.num_tokens} tokens, {channels} channels in {w} columns")
        a = _ConvArgs()
        a.x, a.x_stride, a.taps, a.tail = y.data_ptr() + first * y.element_size(), y.stride(0), taps.data_ptr(), tail.data_ptr()
        if bias is not None:
            a.bias = _need(bias, "convolution bias", torch.float32, (channels,)).data_ptr()
        a.cu_q = _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,)).data_ptr()
        a.seq_of_token = _need(ctx.seq_of_token, "seq_of_token", torch.int32, (t,)).data_ptr()
        a.state_slots = _need(ctx.state_slots, "state_slots", torch.int32, (ctx.num_seqs,)).data_ptr()
        out = torch.empty((t, channels), dtype=out_dtype, device=y.device)
        a.out_code = _CODE[out_dtype]
        if activation not in ("silu", None):
            raise OpsError(f"delta_conv: unknown activation {activation!r}")
        a.no_activation = int(activation is None)
        a.out, a.num_tokens, a.channels, a.num_taps, a.nseg, a.unit_eps = out.data_ptr(), t, channels, k, len(segments), unit_eps
        at = 0
        for i, (heads, width, mode) in enumerate(segments):
            a.seg_first[i], a.seg_heads[i], a.seg_width[i], a.seg_mode[i] = at, heads, width, mode
            at += heads * width
        if at != channels:
            raise OpsError(f"delta_conv: segments cover {at} of {channels} channels")
        self._check(self.lib, self.lib.qrt_delta_conv(byref(a), _CODE[y.dtype], c_int(ctx.num_seqs), c_int(slots),
                                                      c_int(ctx.max_q_len), _stream()))
        return out

    def delta_rule(self, ctx, qkv, beta, a_logits, a_log, dt_bias, state, heads, kv_heads, dim, vdim, per_channel):
        """The recurrence over each sequence's tokens from its slot's state (float32
        [slots, heads, vdim, dim], updated in place). ``qkv`` float32 [T, C] as ``delta_conv`` leaves
        it; ``beta`` [T, heads] and ``a_logits`` [T, heads] (or [T, heads * dim], ``per_channel``)
        may be columns of wider matrices. Returns the read-outs, float32 [T, heads, vdim]."""
        t = ctx.num_tokens
        c = 2 * kv_heads * dim + heads * vdim
        _need(qkv, "convolved q | k | v", torch.float32, (t, c))
        _need(state, "state", torch.float32, (state.shape[0], heads, vdim, dim))
        per = heads * dim if per_channel else heads
        for name, m, width in (("beta", beta, heads), ("decay logits", a_logits, per)):
            if not m.is_cuda or tuple(m.shape) != (t, width) or m.stride(1) != 1 or m.dtype not in _CODE:
                raise OpsError(f"{name}: {tuple(m.shape)} {m.dtype} with strides {m.stride()} for {t} tokens of {width}")
        _need(a_log, "A_log", torch.float32, (heads,))
        _need(dt_bias, "dt_bias", torch.float32, (per,))
        a = _RuleArgs()
        a.qkv, a.channels, a.q_first, a.k_first, a.v_first = qkv.data_ptr(), c, 0, kv_heads * dim, 2 * kv_heads * dim
        a.b, a.b_stride, a.b_code = beta.data_ptr(), beta.stride(0), _CODE[beta.dtype]
        a.a, a.a_stride, a.a_code = a_logits.data_ptr(), a_logits.stride(0), _CODE[a_logits.dtype]
        a.a_log, a.dt_bias, a.state = a_log.data_ptr(), dt_bias.data_ptr(), state.data_ptr()
        out = torch.empty((t, heads, vdim), dtype=torch.float32, device=qkv.device)
        a.out = out.data_ptr()
        a.cu_q = _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,)).data_ptr()
        a.state_slots = _need(ctx.state_slots, "state_slots", torch.int32, (ctx.num_seqs,)).data_ptr()
        a.heads, a.kv_heads, a.dim, a.vdim, a.per_channel = heads, kv_heads, dim, vdim, int(bool(per_channel))
        self._check(self.lib, self.lib.qrt_delta_rule(byref(a), c_int(t), c_int(ctx.num_seqs), c_int(ctx.max_q_len), _stream()))
        return out

    def delta_out(self, o, weight, gate, eps, gate_kind, out_dtype):
        """Per head: ``o / rms(o) * weight * act(gate)``, act silu or sigmoid; [T, heads * vdim]."""
        t, heads, vdim = o.shape
        _need(o, "read-out", torch.float32)
        _need(weight, "read-out norm weight", torch.float32, (vdim,))
        if not gate.is_cuda or tuple(gate.shape) != (t, heads * vdim) or gate.stride(1) != 1 or gate.dtype not in _CODE:
            raise OpsError(f"gate {tuple(gate.shape)} {gate.dtype} does not fit {t} tokens of {heads} heads of {vdim}")
        out = torch.empty((t, heads * vdim), dtype=out_dtype, device=o.device)
        self._check(self.lib, self.lib.qrt_delta_out(_ptr(o), _ptr(weight), c_void_p(gate.data_ptr()), c_long(gate.stride(0)),
                                                     _CODE[gate.dtype], _ptr(out), _CODE[out_dtype], c_int(t), c_int(heads),
                                                     c_int(vdim), c_float(eps), c_int({"silu": 0, "sigmoid": 1}[gate_kind]), _stream()))
        return out

    def mix_norm(self, streams, update, read, weight, bias, eps, out_dtype, rows=None):
        """The step between two sub-layers over residual streams ``[T, S, H]`` (or one stream
        ``[T, H]``), float32, in one kernel: apply the pending ``update`` in place (a
        ``StreamUpdate``: ``new[:, t] = sum_s mix[s, t] old[:, s] + out[t] y``; a plain tensor or
        planes: added, one stream only; None: nothing), form ``sum_t read[t] new[:, t]`` and
        normalise it: layer norm with ``bias``, RMS norm without. With ``rows`` only those rows are
        normalised and nothing is written back."""
        one = streams.dim() == 2
        t, s, h = (streams.shape[0], 1, streams.shape[1]) if one else streams.shape
        _need(streams, "residual streams", torch.float32)
        _need(weight, "norm weight", torch.float32, (h,))
        a = _MixNormArgs()
        a.x_in, a.streams, a.s_in, a.hidden, a.eps = streams.data_ptr(), s, s, h, eps
        a.weight, a.bias = weight.data_ptr(), _addr(None if bias is None else _need(bias, "norm bias", torch.float32, (h,)))
        if update is not None:
            y = update.y if hasattr(update, "y") else update
            if hasattr(update, "y"):
                a.mix = _need(update.mix, "stream mix", torch.float32, (s, s)).data_ptr()
                a.out_w = _need(update.out, "stream out", torch.float32, (s,)).data_ptr()
            elif s != 1:
                raise OpsError("several residual streams take a StreamUpdate, not a plain delta")
            if y.dim() == 3:
                a.planes, a.plane_stride = y.shape[0], t * h
                _need(y, "pending output", shape=(y.shape[0], t, h))
            else:
                a.planes = 1
                _need(y, "pending output", shape=(t, h))
            a.y, a.y_dtype = y.data_ptr(), _CODE[y.dtype]
        if read is not None:
            a.read = _need(read, "stream read", torch.float32, (s,)).data_ptr()
        n_out = t
        if rows is not None:
            a.rows = _need(rows, "rows", torch.int32).data_ptr()
            n_out = rows.numel()
        elif update is not None:
            a.x_out = streams.data_ptr()
        out = torch.empty((n_out, h), dtype=out_dtype, device=streams.device)
        a.out, a.out_dtype, a.num_out = out.data_ptr(), _CODE[out_dtype], n_out
        self._check(self.lib, self.lib.qrt_mix_norm(byref(a), _stream()))
        return out

    # ---- routed experts --------------------------------------------------------------
    def route_top(self, x, router, router_bias, top, scoring="softmax_top", groups=1, keep=None, group_score="top2",
                  correction=None, renormalise=False, weight_scale=1.0, gate_row=False):
        """Router logits ``x W^T + b`` in float32, the ``top`` largest per token and the softmax
        over those alone: (int32 [T, top], float32 [T, top]). ``scoring="sigmoid"``: the choice goes
        by ``sigmoid`` of the logits, which are also the weights, as they are; ``"softmax_all"``: by the
        softmax over all experts' logits, likewise. ``groups``, ``keep``: only experts of the ``keep``
        best of ``groups`` equal groups of neighbours can be chosen, a group's score being the sum of
        its two largest entries (``group_score="top2"``) or its largest (``"max"``). With scores over all
        experts: ``correction`` [E] is added to them for the choice alone, ``renormalise`` divides the
        chosen scores by their sum (+ 1e-20), ``weight_scale`` multiplies the weights at the end.
        ``gate_row``: the router's last row is no expert; the sigmoid of its product is returned as well,
        float32 [T]."""
        t, h = x.shape
        _need(x, "x")
        n = router.shape[0] - int(bool(gate_row))
        _need(router, "router", torch.float32, (n + int(bool(gate_row)), h))
        gate = torch.empty((t,), dtype=torch.float32, device=x.device) if gate_row else None
        if correction is not None:
            _need(correction, "correction of the choice", torch.float32, (n,))
        if router_bias is not None:
            _need(router_bias, "router bias", torch.float32, (n,))
        index = torch.empty((t, top), dtype=torch.int32, device=x.device)
        weight = torch.empty((t, top), dtype=torch.float32, device=x.device)
        self._check(self.lib, self.lib.qrt_route_top(_ptr(x), _CODE[x.dtype], _ptr(router), _ptr(router_bias),
                                                     _ptr(index), _ptr(weight), c_int(t), c_int(h), c_int(n),
                                                     c_int(top), c_int({"softmax_top": 0, "sigmoid": 1, "softmax_all": 2}[scoring]),
                                                     c_int(groups), c_int(groups if keep is None else keep),
                                                     c_int(group_score == "max"), _ptr(correction),
                                                     c_int(bool(renormalise)), c_float(weight_scale), _ptr(gate), _stream()))
        return (index, weight, gate) if gate_row else (index, weight)

    def moe_swiglu(self, x, gate_up, down, index, weight, activation="swiglu", limit=0.0, out=None, weight_on_input=False):
        """``sum_j weight[t, j] * down[e] (silu(gate[e] x) * (up[e] x))`` with ``e = index[t, j]``;
        ``gate_up`` [E, 2I, H] (gate rows first), ``down`` [E, H, I]. float32 [T, H]. ``activation="relu2"``:
        experts without a gate, ``down[e] relu(up[e] x)^2``, and ``gate_up`` is the up rows alone, [E, I, H].
        ``weight_on_input`` (gated experts): a weight scales its expert's input, ``sum_j expert_j(weight[t, j] x)``:
        it multiplies the first products in float32 in front of the activation, and nothing after it."""
        if weight_on_input and activation == "relu2":
            raise OpsError("weights on the experts' input go with gated experts")
        t, h = x.shape
        n, rows_e, _ = gate_up.shape
        inter = rows_e if activation == "relu2" else rows_e // 2
        top = index.shape[1]
        _need(x, "x")
        _need(gate_up, "expert gate/up", x.dtype, (n, rows_e, h))
        _need(down, "expert down", x.dtype, (n, h, inter))
        _need(index, "expert index", torch.int32, (t, top))
        _need(weight, "expert weight", torch.float32, (t, top))
        if out is None:
            out = torch.empty((t, h), dtype=torch.float32, device=x.device)
        else:  # the caller's own float32 rows (a plane of a sum that the next norm adds up)
            _need(out, "experts' output", torch.float32, (t, h))
        if t == 0:
            return out
        pairs = t * top
        if (pairs >= self.moe_grouped_min_pairs and pairs >= self.moe_grouped_pairs_per_expert * n
                and not torch.cuda.is_current_stream_capturing()):
            return self._moe_grouped(x, gate_up, down, index, weight, out, activation, limit, weight_on_input)
        kind = (c_int(ACTIVATIONS[activation]), c_float(limit))
        act = torch.empty((t * top, inter), dtype=x.dtype, device=x.device)
        vec = 16 // x.element_size()
        if pairs >= self.moe_by_expert_pairs_per_expert * n and h % vec == 0 and inter % vec == 0:
            # several tokens an expert: each expert's rows are read once, by blocks that own them
            order = torch.empty(pairs, dtype=torch.int32, device=x.device)
            place = torch.empty(pairs, dtype=torch.int32, device=x.device)
            offsets = torch.empty(n + 1, dtype=torch.int32, device=x.device)
            y = torch.empty((pairs, h), dtype=x.dtype, device=x.device)
            self._check(self.lib, self.lib.qrt_moe_group(_ptr(index), _ptr(order), _ptr(place), _ptr(offsets),
                                                         c_int(pairs), c_int(n), _stream()))
            self._check(self.lib, self.lib.qrt_moe_by_expert(_ptr(x), _ptr(gate_up), _ptr(down), _ptr(order), _ptr(offsets),
                                                             _ptr(act), _ptr(y), _CODE[x.dtype], c_int(h), c_int(inter),
                                                             c_int(n), c_int(top), *kind, _ptr(weight) if weight_on_input else None,
                                                            _stream()))
            self._check(self.lib, self.lib.qrt_moe_combine(_ptr(y), _ptr(place), _ptr(index), _ptr(offsets), c_int(0),
                                                           None if weight_on_input else _ptr(weight), _ptr(out),
                                                           _CODE[x.dtype], c_int(t), c_int(h), c_int(top), _stream()))
            return out
        self._check(self.lib, self.lib.qrt_moe_pairs(_ptr(x), _ptr(gate_up), _ptr(down), _ptr(index), _ptr(weight),
                                                     _ptr(act), _ptr(out), _CODE[x.dtype], c_int(t), c_int(h),
                                                     c_int(inter), c_int(n), c_int(top), *kind, c_int(bool(weight_on_input)),
                                                     _stream()))
        return out

    # Steps of many tokens run the experts one by one, each on the rows of its own tokens, with
    # the engine's matrix products (an expert's matrices are then read once, not once per pair):
    # from this many pairs on, and from this many pairs per expert on. It reads the experts'
    # row counts on the host, so a step that is being captured into a graph never takes it.
    moe_grouped_min_pairs = 64
    moe_grouped_pairs_per_expert = 4
    # Steps that may not wait for the device (captured ones) and steps too small for that: from
    # this many pairs per expert on, the experts' rows are read once per expert by a kernel that
    # walks the expert's tokens; below it, once per pair (fewer launches, and pairs rarely meet).
    moe_by_expert_pairs_per_expert = 1

    def _moe_grouped(self, x, gate_up, down, index, weight, out, activation="swiglu", limit=0.0, weight_on_input=False):
        t, h = x.shape
        n, top = gate_up.shape[0], index.shape[1]
        pairs = t * top
        dev = x.device
        order = torch.empty(pairs, dtype=torch.int32, device=dev)
        place = torch.empty(pairs, dtype=torch.int32, device=dev)
        offsets = torch.empty(n + 1, dtype=torch.int32, device=dev)
        self._check(self.lib, self.lib.qrt_moe_group(_ptr(index), _ptr(order), _ptr(place), _ptr(offsets),
                                                     c_int(pairs), c_int(n), _stream()))
        bounds = offsets.cpu().tolist()  # the one wait of the step's host for the device
        # The experts' rows lie one expert after the other (``padded`` = 0). The kernels also know a
        # layout in which every expert has a stretch of equal length, made for one batched library
        # product over all experts; that product is not used: the one run of it at the sizes of a
        # real model ended in a fault of the device whose cause has not been found.
        padded = 0
        xs = torch.empty((pairs, h), dtype=x.dtype, device=dev)
        self._check(self.lib, self.lib.qrt_moe_gather(_ptr(x), _ptr(order), _ptr(index), _ptr(offsets), c_int(padded),
                                                      _ptr(xs), _CODE[x.dtype], c_int(pairs), c_int(h), c_int(top),
                                                      _stream()))
        y = torch.empty((pairs, h), dtype=x.dtype, device=dev)
        busy = [(e, bounds[e], bounds[e + 1]) for e in range(n) if bounds[e + 1] > bounds[e]]
        # weights on the input: each row's own, found through the order of the rows, in front of the activation
        scaled = {"scale": weight.view(-1), "order": order} if weight_on_input else {}
        if x.dtype == torch.bfloat16:
            # what bounds this form is the host's time per launch, so an expert costs two of them:
            # its products go straight into its rows of one buffer each (the library's for more
            # rows than the engine's own kernels take), and one activation kernel serves all experts
            both = torch.empty((pairs, gate_up.shape[1]), dtype=x.dtype, device=dev)
            for e, a, b in busy:
                if b - a > self.own_max_rows:
                    torch.mm(xs[a:b], gate_up[e].t(), out=both[a:b])
                else:
                    both[a:b] = self.linear(xs[a:b], gate_up[e])
            act = self.unary_act(both, activation) if activation == "relu2" else \
                self.gated_act(both, activation, limit, **scaled)
            for e, a, b in busy:
                if b - a > self.own_max_rows:
                    torch.mm(act[a:b], down[e].t(), out=y[a:b])
                else:
                    y[a:b] = self.linear(act[a:b], down[e])
        else:
            for e, a, b in busy:
                if activation == "relu2":
                    act = self.unary_act(self.linear(xs[a:b], gate_up[e]), activation)
                elif weight_on_input:
                    act = self.gated_act(self.linear(xs[a:b], gate_up[e]), activation, limit,
                                         weight.view(-1)[order[a:b].long()].contiguous())
                else:
                    act = self.gated_linear(xs[a:b], gate_up[e], activation, limit)
                y[a:b] = self.linear(act, down[e])
        self._check(self.lib, self.lib.qrt_moe_combine(_ptr(y), _ptr(place), _ptr(index), _ptr(offsets), c_int(padded),
                                                       None if weight_on_input else _ptr(weight), _ptr(out),
                                                       _CODE[x.dtype], c_int(t), c_int(h), c_int(top), _stream()))
        return out

    def sigmoid_gate(self, out, gate):
        """``out *= sigmoid(gate)`` in place; ``gate`` may be columns of a wider matrix."""
        t, w = out.shape
        _need(out, "attention output")
        if gate.dtype != out.dtype or tuple(gate.shape) != (t, w) or gate.stride(1) != 1:
            raise OpsError(f"gate {tuple(gate.shape)} {gate.dtype} does not fit output {tuple(out.shape)} {out.dtype}")
        self._check(self.lib, self.lib.qrt_sigmoid_gate(_ptr(out), c_void_p(gate.data_ptr()), c_long(gate.stride(0)),
                                                        _CODE[out.dtype], c_int(t), c_int(w), _stream()))
        return out

    def swiglu(self, gate_up, scale=None, order=None):
        return self.gated_act(gate_up, scale=scale, order=order)

    # ---- matrix products -------------------------------------------------------
    def linear(self, x, w, out_f32=False):
        _need(x, "x")
        _need(w, "weight")
        m, k = x.shape
        n, kw = w.shape
        if k != kw:
            raise OpsError(f"linear: x is {tuple(x.shape)}, weight is {tuple(w.shape)}")
        if w.dtype == torch.float32:
            # true 32-bit product; a float32 weight met by bfloat16 activations keeps its precision
            xin = x if x.dtype == torch.float32 else x.float()
            out = torch.empty((m, n), dtype=torch.float32, device=x.device)
            self._check(self.lib, self.lib.qrt_gemm_f32(_ptr(xin), _ptr(w), _ptr(out), c_int(m), c_int(n),
                                                        c_int(k), _stream()))
            return out if (out_f32 or x.dtype == torch.float32) else out.to(x.dtype)
        if x.dtype != torch.bfloat16 or w.dtype != torch.bfloat16:
            raise OpsError(f"linear: no product of {x.dtype} activations with {w.dtype} weights")
        kernel = self._own_kernel(m, n, k, "whole")
        if kernel is None:
            # many rows: the vendor library; both accumulate in float32
            if out_f32:
                return torch.mm(x, w.t(), out_dtype=torch.float32)
            return self._library_product(x, w)
        out = torch.empty((m, n), dtype=torch.float32 if out_f32 else torch.bfloat16, device=x.device)
        self._check(self.lib, self.lib.qrt_gemm_bf16(
            _ptr(x), _ptr(w), _ptr(out), F32 if out_f32 else BF16,
            c_int(m), c_int(n), c_int(k), c_int(0), c_int(kernel), c_int(1), _stream()))
        return out

    # rows from which a library product is made in two column chunks; False: never
    library_split_min_rows = 256

    def _library_product(self, x, w):
        """``x @ w.T`` by the vendor library, in one call or in two over column chunks of the result.

        The library's kernels work on tiles of the result (256 x 256 for these shapes), and a
        result whose tiles do not fill the 256 compute units a whole number of times leaves
        them idle in the last round: 2,048 x 19,456 is 608 tiles, 2.4 rounds (0.93 PFLOP/s, where
        2,048 x 24,576, three whole rounds, runs at 1.45). A first chunk of columns that fills
        whole rounds and a second call for the rest is faster wherever such a cut exists: over the
        products of the 1.7B to 32B sizes at 256 to 8,192 rows the two calls took 0.69 to 0.99 of
        the one call's time (0.80 for the case above), 1.02 at worst. The cut depends on the
        shape alone, so equal inputs give equal bits in every process (the two ways use other
        library kernels, which round differently)."""
        m, k = x.shape
        n = w.shape[0]
        split = self.library_split(m, n)
        if not split:
            return torch.matmul(x, w.t())
        out = torch.empty((m, n), dtype=x.dtype, device=x.device)
        torch.mm(x, w[:split].t(), out=out[:, :split])
        torch.mm(x, w[split:].t(), out=out[:, split:])
        return out

    def library_split(self, m: int, n: int) -> int:
        """Columns of the first chunk (0: one call): the most whose 256 x 256 tiles fill the
        compute units a whole number of times, if that leaves a second chunk."""
        if not self.library_split_min_rows or m < self.library_split_min_rows:
            return 0
        row_tiles = -(-m // 256)
        per_round = 256 * max(1, 256 // row_tiles)  # columns whose tiles fill the compute units once
        split = (n // per_round) * per_round
        return split if 0 < split < n else 0

    def _own_kernel(self, m: int, n: int, k: int, form: str) -> int | None:
        """Which of the library's kernels multiplies ``m`` rows by a weight [n, k]: 0 the few-row
        kernel (up to 16 rows), 1 the kernel that shares the activations through LDS (K a
        multiple of 64 and at least 128, n a multiple of 16), None the vendor library. Both read
        the weight as stored. ``form``: "whole", "gated", or "planes" (cut along K). Measured at
        the 4B shapes against the vendor library: 28 to 32 % less time over the four products of
        a layer at 32 and 64 rows; at 128 rows 71 us against 116 for the gated product and the
        two cut along K."""
        limit = self.own_max_rows if form == "whole" else self.own_max_rows_shared
        if (k % 64 == 0 and k >= 128 and n % 16 == 0 and n <= 1 << 20
                and self.shared_from_rows[form] <= m <= limit):
            return 1
        if m <= min(16, limit):
            return 0
        return None

    def linear_for_residual(self, x, w):
        """``linear(x, w)`` for a result that is only ever added to the residual stream.

        May return the result in planes ``[P, T, N]`` float32 whose sum it is (``add_rmsnorm``
        adds them): a product with few rows and few weight rows then cuts K over several blocks
        per row tile, which fills the chip (160 row tiles for 256 compute units at the 4B size)."""
        m, k = x.shape
        n = w.shape[0]
        kernel, parts = None, 1
        if x.dtype == torch.bfloat16 and w.dtype == torch.bfloat16 and k % 64 == 0:
            kernel = self._own_kernel(m, n, k, "planes")
            if kernel is not None:
                parts = self.choose_k_parts(n, k, m, kernel == 1)
        if parts == 1:
            return self.linear(x, w)
        _need(x, "x", torch.bfloat16)
        _need(w, "weight", torch.bfloat16, (n, k))
        out = torch.empty((parts, m, n), dtype=torch.float32, device=x.device)
        self._check(self.lib, self.lib.qrt_gemm_bf16(
            _ptr(x), _ptr(w), _ptr(out), F32, c_int(m), c_int(n), c_int(k), c_int(0),
            c_int(kernel), c_int(parts), _stream()))
        return out

    def linear_planes_with_spare(self, x, w):
        """``linear_for_residual(x, w)`` as float32 planes ``[P + 1, T, N]`` of which the last is left
        for the caller to fill with one more addend of the same sum (so that the sum costs no
        kernel of its own); None where the product does not run in the engine's own kernels."""
        m, k = x.shape
        n = w.shape[0]
        if not (x.dtype == torch.bfloat16 and w.dtype == torch.bfloat16 and k % 64 == 0):
            return None
        kernel = self._own_kernel(m, n, k, "planes")
        if kernel is None:
            return None
        parts = self.choose_k_parts(n, k, m, kernel == 1)
        if parts == 1 and m > self.own_max_rows:  # above that many rows only products cut along K have a kernel
            return None
        _need(x, "x", torch.bfloat16)
        _need(w, "weight", torch.bfloat16, (n, k))
        out = torch.empty((parts + 1, m, n), dtype=torch.float32, device=x.device)
        self._check(self.lib, self.lib.qrt_gemm_bf16(
            _ptr(x), _ptr(w), _ptr(out), F32, c_int(m), c_int(n), c_int(k), c_int(0),
            c_int(kernel), c_int(parts), _stream()))
        return out

    @staticmethod
    def choose_k_parts(n: int, k: int, m: int = 1, shared: bool | None = None) -> int:
        """The few-row kernel: cut K when there are fewer row tiles than about two per compute
        unit and K is long. The kernel that shares activations (``shared``; by default from 17
        rows on): a block takes up to eight row tiles, and K is cut until there are about as
        many blocks as compute units, each part keeping 12 k-steps or more."""
        tiles = n // 16
        if shared is None:
            shared = m > 16
        if not shared:
            if tiles >= 384 or k < 2048:
                return 1
            # four parts up to 8,192 columns and eight beyond, in a number of planes the residual's
            # norm knows when compiling (timed on the matrices of 36 layers in turn at the 4B, 8B
            # and 32B sizes: the attention's output product 6.2, 7.6 and 17.6 us in four parts
            # against 6.8, 8.9 and 18.3 in eight; the down projection 10.6 and 40.6 us in eight
            # against 12.0 and 43.6 in four at the 4B and 32B sizes, level at the 8B size)
            return 4 if k <= 8192 else 8
        blocks = (tiles + 7) // 8
        return max(1, min(8, 256 // blocks, (k // 32) // 12))


    def gated_linear(self, x, w_gate_up, activation="swiglu", limit=0.0, row_scale=None):
        """``gated_act(linear(x, w_gate_up), ...)`` with ``w_gate_up`` [2I, K], gate rows first. With few
        rows in bfloat16 one kernel forms both halves and applies the activation in its epilogue,
        so the [T, 2I] intermediate never reaches memory."""
        m, k = x.shape
        two_i, kw = w_gate_up.shape
        if k != kw or two_i % 2:
            raise OpsError(f"gated_linear: x is {tuple(x.shape)}, weight is {tuple(w_gate_up.shape)}")
        if x.dtype == torch.bfloat16 and w_gate_up.dtype == torch.bfloat16 and k % 32 == 0:
            _need(x, "x")
            _need(w_gate_up, "weight")
            kernel = self._own_kernel(m, two_i // 2, k, "gated")
            if kernel is not None:
                out = torch.empty((m, two_i // 2), dtype=torch.bfloat16, device=x.device)
                if row_scale is not None:
                    _need(row_scale, "row factors", torch.float32, (m,))
                self._check(self.lib, self.lib.qrt_gated_gemm_bf16(
                    _ptr(x), _ptr(w_gate_up), _ptr(out), BF16, c_int(m), c_int(two_i // 2), c_int(k), c_int(kernel),
                    c_int(ACTIVATIONS[activation]), c_float(limit), _ptr(row_scale), _stream()))
                return out
        return self.gated_act(self.linear(x, w_gate_up), activation, limit, row_scale=row_scale)

    # ---- q/k norm, rotation, cache write ----------------------------------------
    def _qk(self, args: _QkArgs, dtype, num_pages=0):
        self._check(self.lib, self.lib.qrt_qk_norm_rope_store(byref(args), _CODE[dtype], c_long(num_pages), _stream()))

    # tokens from which the step's cosines and sines are computed once (rope_table) and looked up by
    # every layer, instead of being computed in every layer's kernel
    rope_table_from_tokens = 256

    def qk_norm_rope_store(self, qkv, nq, nkv, d, q_w, k_w, eps, inv_freq, positions, cache, ctx=None,
                           angles_key=None, value_dim=None, extra=0, value_turn=None):
        """Per-head RMSNorm of queries and keys, rotation of their first ``2 len(inv_freq)`` elements (first
        half of those against second half), and the write of keys and values into
        the cache, in one pass over ``qkv``; returns the queries. ``value_turn`` (frequencies, a name for them
        as ``angles_key``): the values turn too, over all their elements, before they are stored. With the step's context given,
        the angles of a long step come from ``rope_table`` (``angles_key`` as there). Values may
        have ``value_dim`` elements a head; ``extra`` columns behind them are left alone."""
        t, width = qkv.shape
        dv = d if value_dim is None else int(value_dim)
        _need(qkv, "qkv", shape=(t, (nq + nkv) * d + nkv * dv + extra))
        for name, w in (("q_norm", q_w), ("k_norm", k_w)):
            if w is not None:
                _need(w, name, torch.float32, (d,))
        if inv_freq is not None:
            pairs = inv_freq.numel()
            _need(inv_freq, "inv_freq", torch.float32, (pairs,))
            if not 1 <= pairs <= d // 2:
                raise OpsError(f"{pairs} pairs turn in heads of {d}")
            _need(positions, "positions", torch.int32, (t,))
        q = torch.empty((t, nq * d), dtype=qkv.dtype, device=qkv.device)
        es = qkv.element_size()
        a = _QkArgs()
        a.q_in, a.q_stride = qkv.data_ptr(), width
        a.k_in, a.k_stride = qkv.data_ptr() + nq * d * es, width
        a.v_in, a.v_stride = qkv.data_ptr() + (nq + nkv) * d * es, width
        a.q_weight, a.k_weight, a.inv_freq = _addr(q_w), _addr(k_w), _addr(inv_freq)
        a.positions = _addr(positions) if inv_freq is not None else None
        if inv_freq is not None and ctx is not None and t >= self.rope_table_from_tokens and t == ctx.num_tokens \
                and positions is ctx.positions:
            a.rope = self.rope_table(ctx, inv_freq, angles_key).data_ptr()
        a.q_out = q.data_ptr()
        a.num_tokens, a.nq, a.nkv, a.nv, a.head_dim, a.eps = t, nq, nkv, nkv, d, eps
        a.value_dim = dv
        if inv_freq is not None:
            a.rot_pairs = pairs
        if value_turn is not None and cache is not None:
            if ctx is None or value_turn[0].numel() * 2 != dv:
                raise OpsError(f"turned values of {dv} take the step's context and {dv // 2} frequencies")
            a.v_rope = self.rope_table(ctx, *value_turn).data_ptr()
        pages = 0
        if cache is not None:
            pages = self._check_cache(cache, nkv, d, qkv.dtype, dv)
            _need(cache.group.slots, "slots", torch.int32, (t,))
            a.slots, a.k_cache, a.v_cache = _addr(cache.group.slots), _addr(cache.k), _addr(cache.v)
            a.page_size = cache.group.page_size
        else:
            a.nkv = a.nv = 0  # keys and values go nowhere: only queries are needed
        self._qk(a, qkv.dtype, pages)
        return q

    def qk_joint_norm_store(self, qk, nq, nkv, d, bias, q_w, k_w, eps, positions, q_temp, values_are_keys, cache):
        """From the columns q | k (| v) of one product: biases (float32 over those columns, or None),
        the RMS norm of all ``nq * d`` query elements of a token at once with weights of that size and
        likewise of its ``nkv * d`` key elements, the queries times the temperature of their position
        (``q_temp`` = (coef, every): ``1 + coef ln(floor((p + 1) / every) + 1)``; None: 1), and the write
        of normed keys and raw values into the cache, the values being the biased keys themselves
        (``values_are_keys``) or the v columns. Returns the queries [T, nq * d]."""
        t, width = qk.shape
        cols = (nq + (1 if values_are_keys else 2) * nkv) * d
        _need(qk, "qk")
        if width < cols:
            raise OpsError(f"qk_joint_norm_store: rows of {width} for {cols} columns")
        a = _JointNormArgs()
        a.qk, a.row = qk.data_ptr(), width
        if bias is not None:
            if bias.numel() < cols:
                raise OpsError(f"qk_joint_norm_store: {bias.numel()} biases for {cols} columns")
            a.bias = _need(bias, "bias", torch.float32).data_ptr()
        a.q_weight = _need(q_w, "q_norm", torch.float32, (nq * d,)).data_ptr()
        a.k_weight = _need(k_w, "k_norm", torch.float32, (nkv * d,)).data_ptr()
        a.positions = _need(positions, "positions", torch.int32, (t,)).data_ptr()
        q = torch.empty((t, nq * d), dtype=qk.dtype, device=qk.device)
        a.q_out, a.nq, a.nkv, a.d, a.values_are_keys, a.eps = q.data_ptr(), nq, nkv, d, int(bool(values_are_keys)), eps
        if q_temp is not None:
            a.temp_coef, a.temp_every = float(q_temp[0]), int(q_temp[1])
        pages = 0
        if cache is not None:
            pages = self._check_cache(cache, nkv, d, qk.dtype)
            a.slots = _need(cache.group.slots, "slots", torch.int32, (t,)).data_ptr()
            a.k_cache, a.v_cache, a.page_size = cache.k.data_ptr(), cache.v.data_ptr(), cache.group.page_size
        self._check(self.lib, self.lib.qrt_qk_joint_norm_store(byref(a), _CODE[qk.dtype], c_int(t), c_long(pages), _stream()))
        return q

    def qk_norm_split(self, qkv, nq, nkv, d, q_w, k_w, eps):
        t, width = qkv.shape
        _need(qkv, "qkv", shape=(t, (nq + 2 * nkv) * d))
        q = torch.empty((t, nq, d), dtype=qkv.dtype, device=qkv.device)
        k = torch.empty((t, nkv, d), dtype=qkv.dtype, device=qkv.device)
        v = torch.empty((t, nkv, d), dtype=qkv.dtype, device=qkv.device)
        es = qkv.element_size()
        a = _QkArgs()
        a.q_in, a.q_stride = qkv.data_ptr(), width
        a.k_in, a.k_stride = qkv.data_ptr() + nq * d * es, width
        a.v_in, a.v_stride = qkv.data_ptr() + (nq + nkv) * d * es, width
        a.q_weight, a.k_weight = _addr(q_w), _addr(k_w)
        a.q_out, a.k_out, a.v_out = q.data_ptr(), k.data_ptr(), v.data_ptr()
        a.num_tokens, a.nq, a.nkv, a.nv, a.head_dim, a.eps = t, nq, nkv, nkv, d, eps
        self._qk(a, qkv.dtype)
        return q, k, v

    def rope_neox(self, q, k, positions, inv_freq):
        t, nq, d = q.shape
        nkv = k.shape[1]
        _need(q, "q")
        _need(k, "k", q.dtype, (t, nkv, d))
        _need(inv_freq, "inv_freq", torch.float32, (d // 2,))
        _need(positions, "positions", torch.int32, (t,))
        q_out, k_out = torch.empty_like(q), torch.empty_like(k)
        a = _QkArgs()
        a.q_in, a.q_stride = q.data_ptr(), nq * d
        a.k_in, a.k_stride = k.data_ptr(), nkv * d
        a.inv_freq, a.positions = _addr(inv_freq), _addr(positions)
        a.q_out, a.k_out = q_out.data_ptr(), k_out.data_ptr()
        a.num_tokens, a.nq, a.nkv, a.nv, a.head_dim = t, nq, nkv, 0, d
        self._qk(a, q.dtype)
        return q_out, k_out

    def kv_store(self, k, v, cache):
        t, nkv, d = k.shape
        _need(k, "k")
        _need(v, "v", k.dtype, (t, nkv, d))
        pages = self._check_cache(cache, nkv, d, k.dtype)
        _need(cache.group.slots, "slots", torch.int32, (t,))
        a = _QkArgs()
        a.k_in, a.k_stride = k.data_ptr(), nkv * d
        a.v_in, a.v_stride = v.data_ptr(), nkv * d
        a.slots, a.k_cache, a.v_cache = _addr(cache.group.slots), _addr(cache.k), _addr(cache.v)
        a.num_tokens, a.nq, a.nkv, a.nv, a.head_dim = t, 0, nkv, nkv, d
        a.page_size = cache.group.page_size
        self._qk(a, k.dtype, pages)

    @staticmethod
    def _check_cache(cache, nkv, d, dtype, dv=None) -> int:
        ps = cache.group.page_size
        pages = cache.k.shape[0]
        _need(cache.k, "key cache", dtype, (pages, nkv, ps, d))
        _need(cache.v, "value cache", dtype, (pages, nkv, d if dv is None else dv, ps))
        return pages

    # ---- attention ---------------------------------------------------------------
    # ---- decoding: norm, rotation, cache write and attention in one kernel -------------
    def rope_table(self, ctx, inv_freq, angles_key=None):
        """Cosines and sines of the step's rotation angles, float32 [T, 2 * len(inv_freq)]
        (cosines first): computed once per pass and looked up by every layer that rotates inside
        its attention kernel. ``angles_key`` names the angles (layers with equal keys share the
        table); without it the tensor ``inv_freq`` itself does."""
        key = ("rope_table", angles_key if angles_key is not None else inv_freq.data_ptr())
        table = ctx.per_pass.get(key)
        if table is None:
            half = inv_freq.numel()
            _need(inv_freq, "inv_freq", torch.float32, (half,))
            _need(ctx.positions, "positions", torch.int32, (ctx.num_tokens,))
            table = torch.empty((ctx.num_tokens, 2 * half), dtype=torch.float32, device=inv_freq.device)
            self._check(self.lib, self.lib.qrt_rope_table(_ptr(ctx.positions), _ptr(inv_freq), _ptr(table),
                                                          c_int(ctx.num_tokens), c_int(half), _stream()))
            ctx.per_pass[key] = table
        return table

    def fuses_decode_attention(self, ctx, qkv, nq, nkv, d, cache, value_dim=None, chunk=None, softcap=None,
                               gate=None, keep_first=0, sink=False, rot_pairs=None, value_turn=None) -> bool:
        """Whether ``decode_attention`` serves this step: one token per sequence, bfloat16, a head
        size that keeps a rotation pair in one lane (a multiple of 64, up to 256; ``rot_pairs``, the pairs
        of a head that turn, a multiple of 32; values of a multiple of 16, up to 256), at most 16
        query heads per key head, and a layer that writes its own cache."""
        dv = d if value_dim is None else value_dim
        if dv % 16 or dv > 256 or (rot_pairs is not None and rot_pairs % 32) or qkv.shape[1] % 8:
            return False
        return (self.fuse_decode and qkv.dtype == torch.bfloat16 and ctx.max_q_len == 1
                and ctx.num_tokens == ctx.num_seqs and d % 64 == 0 and d <= 256 and nq // nkv <= 16
                and cache is not None and cache.writes and cache.group.page_size % 8 == 0
                and cache.k.dtype == torch.bfloat16)

    def decode_attention(self, qkv, cache, ctx, nq, nkv, d, scale, window, q_w, k_w, eps, inv_freq,
                         angles_key=None, chunk=None, softcap=None, gate=None, value_dim=None, keep_first=0, sink=False,
                         value_turn=None):
        """``paged_attention(qk_norm_rope_store(qkv, ...))`` for a step of single tokens, in one
        kernel: each block forms its queries from ``qkv`` (RMSNorm per head, NeoX rotation by the
        step's angle table), attends over the cached keys before the token, adds the token's own
        key and value from registers and stores them into the cache for later steps. Saves the
        kernel between the product and the attention, and the round trip of the queries."""
        t, width = qkv.shape
        dv = d if value_dim is None else int(value_dim)
        extra = 0 if gate is None else gate.shape[1]  # the gate's columns, behind q | k | v
        _need(qkv, "qkv", torch.bfloat16, (t, (nq + nkv) * d + nkv * dv + extra))
        self._check_cache(cache, nkv, d, qkv.dtype, dv)
        for name, w in (("q_norm", q_w), ("k_norm", k_w)):
            if w is not None:
                _need(w, name, torch.float32, (d,))
        _need(cache.group.slots, "slots", torch.int32, (t,))
        table = _need(cache.group.block_table, "block table", torch.int32)
        if table.shape[0] != ctx.num_seqs:
            raise OpsError(f"block table has {table.shape[0]} rows for {ctx.num_seqs} sequences")
        ps = cache.group.page_size
        if table.shape[1] < (ctx.max_kv_len + ps - 1) // ps:
            raise OpsError(f"block table is {table.shape[1]} pages wide, the longest sequence needs more")
        if not scale > 0:
            raise OpsError(f"the bfloat16 attention kernels take a positive score scale, not {scale}")
        own = {"qkv": qkv, "q_weight": q_w, "k_weight": k_w, "eps": eps,
               "rope": None if inv_freq is None else self.rope_table(ctx, inv_freq, angles_key),
               "rope_pairs": 0 if inv_freq is None else inv_freq.numel()}
        out = torch.empty((t, nq * dv), dtype=qkv.dtype, device=qkv.device)
        self._launch_attention(None, out, cache, ctx, nq, nkv, d, scale, window or 0, None, True, own,
                               chunk=chunk or 0, softcap=softcap or 0.0, gate=gate, keep_first=keep_first, sink=sink,
                               turn=self._turn_table(ctx, value_turn, dv), dv=dv)
        return out

    def _turn_table(self, ctx, value_turn, dv):
        """The step's angles of turned values of ``dv`` elements (None: values are not turned)."""
        if value_turn is None:
            return None
        if value_turn[0].numel() * 2 != dv:
            raise OpsError(f"{value_turn[0].numel()} frequencies for turned values of {dv}")
        return self.rope_table(ctx, *value_turn)

    def paged_attention(self, q, cache, ctx, nq, nkv, d, scale, window, chunk=None, softcap=None, value_dim=None,
                        gate=None, keep_first=0, sink=False, value_turn=None):
        """Attention of every query over its sequence's cache. ``value_turn`` (frequencies, a name for
        them): the cached values are turned by their positions, and each head's output is turned back by
        the query's. Beyond the plain form: a mask of
        chunks instead of a window (``chunk``), a tanh cap on the scaled scores (``softcap``),
        values of ``value_dim`` elements, and a ``gate`` [T, nq * value_dim] (columns of a wider
        matrix will do) whose sigmoid multiplies the output."""
        t = ctx.num_tokens
        dv = d if value_dim is None else int(value_dim)
        _need(q, "q", shape=(t, nq * d))
        self._check_cache(cache, nkv, d, q.dtype, dv)
        if gate is not None and (gate.dtype != q.dtype or tuple(gate.shape) != (t, nq * dv) or gate.stride(1) != 1):
            raise OpsError(f"gate {tuple(gate.shape)} {gate.dtype} does not fit {t} tokens of {nq} heads of {dv}")
        table = _need(cache.group.block_table, "block table", torch.int32)
        if table.shape[0] != ctx.num_seqs:
            raise OpsError(f"block table has {table.shape[0]} rows for {ctx.num_seqs} sequences")
        ps = cache.group.page_size
        need_pages = (ctx.max_kv_len + ps - 1) // ps
        if table.shape[1] < need_pages:
            raise OpsError(f"block table is {table.shape[1]} pages wide, the longest sequence needs {need_pages}")
        out = torch.empty((t, nq * dv), dtype=q.dtype, device=q.device)
        if keep_first and not window:
            raise OpsError("first keys are kept in sight beside a window")
        if q.dtype == torch.bfloat16 and d % 16 == 0 and d <= 512 and dv % 16 == 0 and dv <= 512 and ps % 8 == 0:
            self._attention_mfma(q, out, cache, ctx, nq, nkv, d, scale, window or 0, chunk or 0, softcap or 0.0, gate,
                                 keep_first=int(keep_first), sink=bool(sink), turn=self._turn_table(ctx, value_turn, dv), dv=dv)
        else:
            a = _AttnArgs()
            a.q, a.out, a.k_cache, a.v_cache = q.data_ptr(), out.data_ptr(), cache.k.data_ptr(), cache.v.data_ptr()
            a.positions = _need(ctx.positions, "positions", torch.int32, (t,)).data_ptr()
            a.seq_of_token = _need(ctx.seq_of_token, "seq_of_token", torch.int32, (t,)).data_ptr()
            a.block_table, a.table_width = table.data_ptr(), table.shape[1]
            a.num_tokens, a.nq, a.nkv, a.head_dim, a.page_size = t, nq, nkv, d, ps
            a.window, a.scale = window or 0, scale
            a.chunk, a.softcap, a.value_dim = chunk or 0, softcap or 0.0, dv
            if gate is not None:
                a.gate, a.gate_stride = gate.data_ptr(), gate.stride(0)
            a.keep_first, a.sink = int(keep_first), int(bool(sink))
            a.turn = _addr(self._turn_table(ctx, value_turn, dv))
            self._check(self.lib, self.lib.qrt_attention_f32(byref(a), _CODE[q.dtype], _stream()))
        return out

    resident_blocks = 512  # blocks of the prompt kernels the chip holds at once: 2 on each of 256 CUs

    @staticmethod
    def plan_tiles(q_lens, kv_lens, group_size: int, rows_per_tile: int, nkv: int = 1, resident: int = 0,
                   seq_ids=None):
        """Work list of the MFMA attention kernels: (sequence, first row) per tile of rows.

        Tiles that see the most keys come first: blocks that start late are then the short ones,
        and the chip stays full until the end although causal tiles differ in length. When all
        blocks (tiles x ``nkv`` key heads) fit on the chip at once (``resident``), nothing starts
        late: each CU then holds block i and block i + resident / 2 of the launch order from start
        to end, so the second half of the list is turned round and long tiles share a CU with
        short ones."""
        items = []
        for i, (n, kv) in enumerate(zip(q_lens, kv_lens)):
            s = i if seq_ids is None else seq_ids[i]  # the lists may cover some of the step's sequences
            first = kv - n
            for r in range(0, n * group_size, rows_per_tile):
                last_tok = min(n * group_size, r + rows_per_tile) - 1
                items.append((-(first + last_tok // group_size), s, r))
        items.sort()
        half = resident // (2 * max(nkv, 1))
        if resident and half < len(items) <= 2 * half:
            items = items[:half] + items[half:][::-1]
        seqs = [s for _, s, _ in items]
        row0 = [r for _, _, r in items]
        return np.asarray(seqs + row0, dtype=np.int32), len(seqs)

    def choose_key_groups(self, q_lens, kv_lens, group_size: int, nkv: int, window: int, forced_splits=None) -> int:
        """Long portions through LDS: blocks of four waves, two to a compute unit (1), or blocks of
        eight waves whose two halves take the blocks of keys in turn (2). A tile of 128 rows walks
        its keys in rounds of 32, one after the other, and a lone block's round takes 0.78 of what
        it takes beside a second block: where the tile with the most rounds has about as many as a
        compute unit gets from all tiles together, that chain sets the kernel's time, and halving
        it pays although the eight waves, which meet at one barrier, walk a round more slowly than
        two blocks of four. Measured at head size 128 with 32 query heads on 8 key heads (two
        groups against one): a 2,048-token prompt 63 against 69 us; prompts of 1,024 tokens with
        0 and 1,976 tokens before them 83 against 98; portions of 700, 900 and 448 tokens with
        0, 400 and 4,552 before them 104 against 145; 2,048 tokens with 1,024 before them level;
        with 2,048 before them 148 against 142. Where the keys are cut over blocks anyway (few
        tiles), they are not cut again."""
        if self.prefill_key_groups is not None:
            return self.prefill_key_groups
        rounds = longest = tiles = 0
        for n, kv in zip(q_lens, kv_lens):
            first = kv - n
            for r in range(0, n * group_size, 128):
                hi = first + (min(n * group_size, r + 128) - 1) // group_size
                lo = max(0, first + r // group_size - window + 1) if window else 0
                t = (hi >> 5) - (lo >> 5) + 1
                rounds += t
                longest = max(longest, t)
                tiles += 1
        splits = forced_splits or self.choose_splits(tiles, nkv, max(kv_lens))
        if splits > 1:
            return 1
        return 2 if longest > self.key_groups_ratio * rounds * nkv / 256 else 1

    # see choose_key_groups: the longest tile's rounds over the mean rounds of a compute unit
    key_groups_ratio = 0.9

    @staticmethod
    def choose_splits(num_tiles: int, nkv: int, max_kv: int, head_dim: int = 0) -> int:
        """Portions: how many ways to split the keys so that few long sequences still fill the chip.
        Heads wider than 256 (one block of waves a compute unit, and no decode kernel of their own, so
        that decoded tokens come here too): parts of 64 keys and more, 256 blocks in all."""
        work = num_tiles * nkv
        if head_dim > 256:
            return 1 if max_kv <= 128 or work >= 256 else max(1, min((max_kv + 63) // 64, (256 + work - 1) // work, 64))
        if max_kv <= 512 or work >= 512:
            return 1
        return max(1, min((max_kv + 255) // 256, (1024 + work - 1) // work, 64))

    @staticmethod
    def choose_decode_splits(num_tiles: int, nkv: int, max_kv: int) -> int:
        """Decoding: blocks of four waves, two to a compute unit. The parts are chosen by a small
        model of the launch's time that the measurements fit: the busiest compute unit gets
        ceil(blocks / 256) blocks, each a part of a sequence's keys plus a fixed cost (some 2.5 us:
        0.06 of a walk over 2,100 keys), so the time goes as ceil(work * parts / 256) *
        (1 / parts + cost). Counts of blocks that leave some units one block more than others are
        what it avoids: 12 sequences of 2,100 keys on 8 key heads 32 us in 3 parts (288 blocks), 27
        in 2; 24 sequences 49 us in 2 parts, 42 in 4; 40 sequences 78 us in 1 part, 65 in 4. At
        least 8 key blocks of 32 a part (4 each measured 2 % slower over a batch-1 decode step at
        2,048 keys), at most 64 parts (what the merge kernel reads with every load in flight)."""
        work = num_tiles * nkv
        blocks = (max_kv + 31) // 32
        cost = 0.06 * 2100 / max(max_kv, 1)
        best, best_time = 1, None
        for parts in range(1, max(1, min(blocks // 8, 64)) + 1):
            time = -(-work * parts // 256) * (1.0 / parts + cost)
            if best_time is None or time < best_time * 0.999:
                best, best_time = parts, time
        return best

    # decoding over unequal lengths: from this ratio of the longest to the mean length on, pieces
    decode_piece_ratio = 1.35

    def decode_in_pieces(self, kv_lens) -> bool:
        """Whether a decode launch over sequences of these lengths cuts their keys into pieces
        of one length (as many per sequence as it has) instead of every sequence into equally
        many parts. Measured on 8 to 128 sequences with lengths drawn evenly around 1,024 to
        8,192: the pieces win from a longest length of 1.3 to 1.4 times the mean on (0.80 to 0.9
        of the time at 1.6 to 1.9), lose 5 to 12 % below it, and lose at any spread while the
        longest context is under some 2,000 keys (the merge of the parts then weighs too much)."""
        n, total = len(kv_lens), sum(kv_lens)
        return n >= 2 and max(kv_lens) * n > self.decode_piece_ratio * total and max(kv_lens) >= 2048

    def choose_decode_piece(self, kv_lens, nkv: int):
        """Keys per piece for such a launch (a multiple of 32), or None. Equal parts of every
        sequence make blocks whose work is the sequence's length: with 56 sequences of 300 keys
        and 8 of 8,000 the launch takes 231 us where the two kinds alone take 18 and 48, and more
        parts do not help, because the blocks reach the compute units in launch order, round
        robin, and heavy blocks a fixed stride apart land on the same few. Pieces of one length,
        whole ones first in the list: about 1,536 blocks in all, no piece under 512 keys (a block
        costs some 8 us before its first key arrives) and no sequence in more than 32 (the merge
        reads every piece's part, up to 64 with all its loads in flight at once: 8 sequences of
        1,000 to 30,000 keys 91 us in pieces of 1,024, 96 in pieces of 512, 126 in pieces of 4,096)."""
        if not self.decode_in_pieces(kv_lens):
            return None
        piece = max(512, -(-sum(kv_lens) * nkv // 1536), -(-max(kv_lens) // 32))
        return -(-piece // 32) * 32

    # mixed steps: sequences with few rows leave the prompt kernel when their context is this long
    split_launch_min_kv = 1024

    def _attention_mfma(self, q, out, cache, ctx, nq, nkv, d, scale, window, chunk=0, softcap=0.0, gate=None,
                        keep_first=0, sink=False, turn=None, dv=None):
        """Which kernel for which sequences. Steps of decoded tokens only: the decode kernel.
        Other steps: the prompt kernels; but sequences of at most 16 rows with a long context
        (decoded tokens beside a prompt portion) would each walk all their keys in one block
        there, and hold the step up, so they go to the decode kernel in a launch of their own,
        which cuts their keys over many blocks."""
        if not scale > 0:
            raise OpsError(f"the bfloat16 attention kernels take a positive score scale, not {scale}")
        g = nq // nkv
        seqs = range(ctx.num_seqs)
        dv = dv or d
        widest = max(d, dv)
        more = {"keep_first": keep_first, "sink": sink, "turn": turn, "dv": dv}
        if ctx.max_q_len * g <= 16 and widest <= 256:
            return self._launch_attention(q, out, cache, ctx, nq, nkv, d, scale, window, None, True, chunk=chunk, softcap=softcap, gate=gate, **more)
        small = [s for s in seqs if ctx.q_lens_host[s] * g <= 16]
        if (widest <= 256 and small and len(small) < ctx.num_seqs
                and max(ctx.kv_lens_host[s] for s in small) >= self.split_launch_min_kv):
            small_set = set(small)
            big = [s for s in seqs if s not in small_set]
            self._launch_attention(q, out, cache, ctx, nq, nkv, d, scale, window, small, True, chunk=chunk, softcap=softcap, gate=gate, **more)
            self._launch_attention(q, out, cache, ctx, nq, nkv, d, scale, window, big, False, chunk=chunk, softcap=softcap, gate=gate, **more)
            return
        self._launch_attention(q, out, cache, ctx, nq, nkv, d, scale, window, None, False, chunk=chunk, softcap=softcap, gate=gate, **more)

    def _launch_attention(self, q, out, cache, ctx, nq, nkv, d, scale, window, subset, decode, own=None,
                          chunk=0, softcap=0.0, gate=None, keep_first=0, sink=False, turn=None, dv=None):
        """One launch over the sequences in ``subset`` (None: all of the step's). ``own``: the
        decode kernel takes the tokens' queries, own keys and own values from the q/k/v product
        (``decode_attention``); ``q`` is then None. ``chunk``: a mask of chunks in place of a
        window; ``softcap``: the cap on the scaled scores; ``gate`` [T, nq * dv] (columns of a wider
        matrix will do): its sigmoid multiplies the output where the kernels write it. ``dv``: the size
        of a value (None: ``d``)."""
        dv = dv or d
        widest = max(d, dv)
        lib = attention_library(d, dv)
        # how far back a query can see at most: what the choices below (key splits, pieces) go by
        reach = window or chunk
        g = nq // nkv
        if subset is None:  # the step's own maxima: under a graph they are those of its bucket
            q_lens, kv_lens = ctx.q_lens_host, ctx.kv_lens_host
            max_rows, max_kv = ctx.max_q_len * g, ctx.max_kv_len
        else:
            q_lens = [ctx.q_lens_host[s] for s in subset]
            kv_lens = [ctx.kv_lens_host[s] for s in subset]
            max_rows, max_kv = max(q_lens) * g, max(kv_lens)
        seen_kv = min(max_kv, reach) if reach else max_kv  # keys that the splits divide
        waves = 1 if max_rows <= 16 else (2 if max_rows <= 32 else 4)
        # long portions: several row tiles per wave, so that loaded keys and values serve more rows
        # (heads wider than 256 fill a lane's registers with one tile)
        row_tiles = 1 if max_rows <= 64 or widest > 256 else (self.prefill_row_tiles if widest <= 128 else min(2, self.prefill_row_tiles))
        # the list depends on the rows a tile holds (head geometry and kernel choice): layers of
        # another geometry in the same step get a list of their own
        key = ("attn_plan", g, nkv, widest, waves, row_tiles, decode, None if subset is None else tuple(subset), reach)
        plan = ctx.scratch.get(key)
        if plan is None:  # the same for every layer of the step
            dev = out.device
            if decode:
                tiles = None if subset is None else torch.tensor(subset, dtype=torch.int32, device=dev)
                n_tiles = len(q_lens)
            else:
                lds = waves == 4 and row_tiles >= 2 and self.prefill_through_lds
                groups = self.choose_key_groups(q_lens, kv_lens, g, nkv, reach,
                                                ctx.scratch.get("attn_splits")) if lds else 0
                host, n_tiles = self.plan_tiles(q_lens, kv_lens, g, 16 * waves * row_tiles, nkv,
                                                self.resident_blocks if waves == 4 and row_tiles >= 2 and groups < 2
                                                else 0, subset)
                tiles = torch.from_numpy(host).to(dev)
            tokens = None
            if subset is not None:  # the tokens of these sequences: where a merge of key splits may write
                cu = np.concatenate([[0], np.cumsum(ctx.q_lens_host)])
                tokens = torch.from_numpy(np.concatenate([np.arange(cu[s], cu[s + 1]) for s in subset])
                                          .astype(np.int32)).to(dev)
            plan = (tiles, n_tiles, tokens, 0 if decode else groups)
            ctx.scratch[key] = plan
        tiles, n_tiles, tokens, groups = plan
        splits = ctx.scratch.get("attn_splits") or (
            self.choose_decode_splits(n_tiles, nkv, seen_kv) if decode else self.choose_splits(n_tiles, nkv, seen_kv, widest))
        a = _AttnTileArgs()
        a.chunk = chunk
        # beside a window the sequence's first keys stay in sight; a sink: one more term in the softmax's sum
        a.keep_first, a.sink = int(keep_first), int(bool(sink))
        a.turn = _addr(turn)  # float32 [T, dv]: angles by which the outputs are turned back
        if softcap:
            a.cap_in, a.cap_out = scale / softcap, softcap / scale
        if gate is not None:
            if gate.dtype != torch.bfloat16 or tuple(gate.shape) != (ctx.num_tokens, nq * dv) or gate.stride(1) != 1:
                raise OpsError(f"gate {tuple(gate.shape)} {gate.dtype} does not fit {ctx.num_tokens} tokens of {nq} heads of {dv}")
            a.gate, a.gate_stride = gate.data_ptr(), gate.stride(0)
        piece = None
        if decode and n_tiles <= 1024:
            piece = ctx.scratch.get("attn_piece")  # keys per piece, a multiple of 32: asked for outright
            if piece is None and "attn_splits" not in ctx.scratch:
                # the lengths as they are; a capture sees its bucket's instead and is told them beside
                lens = ctx.scratch.get("attn_lens") or kv_lens
                piece = self.choose_decode_piece([min(n, reach) for n in lens] if reach else lens, nkv)
        if piece:
            a.split_blocks = piece // 32
            # 32-key blocks a sequence of this launch can have: all its keys, or those of its
            # window, which may begin and end inside a block
            span = (max_kv + 31) // 32 if not reach else (min(max_kv, reach + 32) + 31) // 32 + 1
            splits = max(1, -(-span // a.split_blocks))
            if n_tiles * splits > 65535:
                piece, a.split_blocks = None, 0
                splits = self.choose_decode_splits(n_tiles, nkv, seen_kv)
        a.out, a.k_cache, a.v_cache = out.data_ptr(), cache.k.data_ptr(), cache.v.data_ptr()
        if own is None:
            a.q = q.data_ptr()
        else:  # the token's own query, key and value come from the product that made them
            a.qkv, a.qkv_stride = own["qkv"].data_ptr(), own["qkv"].shape[1]
            a.q_weight, a.k_weight, a.rope = _addr(own["q_weight"]), _addr(own["k_weight"]), _addr(own["rope"])
            a.rope_pairs = own["rope_pairs"]
            a.slots, a.eps = cache.group.slots.data_ptr(), own["eps"]
        a.cu_q = _need(ctx.cu_q, "cu_q", torch.int32, (ctx.num_seqs + 1,)).data_ptr()
        a.kv_lens = _need(ctx.kv_lens, "kv_lens", torch.int32, (ctx.num_seqs,)).data_ptr()
        a.block_table, a.table_width = cache.group.block_table.data_ptr(), cache.group.block_table.shape[1]
        if tiles is not None:
            a.tile_seq = tiles.data_ptr()
            if not decode:
                a.tile_row0 = tiles.data_ptr() + 4 * n_tiles
        if tokens is not None:
            a.merge_tokens, a.num_merge_tokens = tokens.data_ptr(), tokens.numel()
        a.num_tiles, a.nq, a.nkv, a.page_size, a.window = n_tiles, nq, nkv, cache.group.page_size, window
        a.num_splits, a.waves, a.row_tiles = splits, waves, row_tiles
        a.use_lds = groups
        a.scale_log2 = scale * math.log2(math.e)
        if splits > 1:
            part_o = torch.empty((ctx.num_tokens * nq * splits, dv), dtype=torch.float32, device=out.device)
            part_lse = torch.empty((ctx.num_tokens * nq * splits,), dtype=torch.float32, device=out.device)
            a.part_o, a.part_lse = part_o.data_ptr(), part_lse.data_ptr()
        if piece:
            # the list of (sequence, piece): from the step's lengths on the device, once per pass
            a.max_items = n_tiles * splits
            list_key = ("attn_items", key, window, chunk, own is not None, piece, a.max_items)
            items = ctx.per_pass.get(list_key)
            if items is None:
                items = torch.empty((a.max_items, 2), dtype=torch.int32, device=out.device)
                a.items = items.data_ptr()
                self._check(lib, lib.qrt_attention_work_list(byref(a), c_int(own is not None), _stream()))
                ctx.per_pass[list_key] = items
            a.items = items.data_ptr()
        if decode:
            self._check(lib, lib.qrt_attention_bf16_decode(byref(a), c_int(ctx.num_tokens * nq), _stream()))
        else:
            self._check(lib, lib.qrt_attention_bf16(byref(a), c_int(ctx.num_tokens * nq), _stream()))

    # ---- sampling ------------------------------------------------------------------
    def argmax(self, logits):
        _need(logits, "logits", torch.float32)
        r, v = logits.shape
        out = torch.empty((r,), dtype=torch.int32, device=logits.device)
        self._check(self.lib, self.lib.qrt_argmax(_ptr(logits), _ptr(out), c_int(r), c_int(v), _stream()))
        return out

    def sample(self, logits, slot, fparams, iparams, seeds, counts=None, keep_processed=False):
        """One token per row of ``logits``. Options are read from the row's state slot:
        ``fparams[slot]`` = temperature, top_p, min_p, repetition, presence, frequency;
        ``iparams[slot]`` = top_k; ``seeds[slot]`` = seed, index of the next draw (advanced
        here). Returns (token int32 [R], logprob float32 [R], processed logits [R, V], buffer); the
        first two are the rows of the int32 buffer [2, R], so that one copy brings both to the host."""
        _need(logits, "logits", torch.float32)
        r, v = logits.shape
        _need(slot, "slot", torch.int32, (r,))
        n = fparams.shape[0]
        _need(fparams, "fparams", torch.float32, (n, 8))
        _need(iparams, "iparams", torch.int32, (n, 2))
        _need(seeds, "seeds", torch.int64, (n, 2))
        if counts is not None:
            _need(counts, "counts", torch.int32, (n, v))
        work = torch.empty_like(logits)
        # ids and log-probabilities side by side, so that one copy brings both to the host
        both = torch.empty((2, r), dtype=torch.int32, device=logits.device)
        tok, lp = both[0], both[1].view(torch.float32)
        a = _SampleArgs()
        a.logits, a.work, a.counts, a.slot = logits.data_ptr(), work.data_ptr(), _addr(counts), slot.data_ptr()
        a.fparams, a.iparams, a.seeds = fparams.data_ptr(), iparams.data_ptr(), seeds.data_ptr()
        a.out_token, a.out_logprob, a.rows, a.vocab = tok.data_ptr(), lp.data_ptr(), r, v
        a.write_work = 1 if keep_processed else 0  # greedy rows skip the write unless asked
        # few rows: the first pass over each row is spread over blocks (about 256 in all)
        parts = min(64, 256 // r, v // 2048) if r <= 64 else 0
        if parts >= 2:
            partials = torch.empty((r, parts, 4), dtype=torch.float32, device=logits.device)
            a.partials, a.parts = partials.data_ptr(), parts
        self._check(self.lib, self.lib.qrt_sample(byref(a), _stream()))
        return tok, lp, work, both

    def count_tokens(self, counts, slots, tokens):
        _need(counts, "counts", torch.int32)
        _need(slots, "slots", torch.int32)
        _need(tokens, "tokens", torch.int32, tuple(slots.shape))
        self._check(self.lib, self.lib.qrt_count_tokens(_ptr(counts), _ptr(slots), _ptr(tokens),
                                                        c_int(slots.numel()), c_int(counts.shape[1]), _stream()))

    def add_bias(self, logits, rows, tokens, values):
        _need(logits, "logits", torch.float32)
        n = rows.numel()
        _need(rows, "rows", torch.int32)
        _need(tokens, "tokens", torch.int32, (n,))
        _need(values, "values", torch.float32, (n,))
        self._check(self.lib, self.lib.qrt_add_bias(_ptr(logits), _ptr(rows), _ptr(tokens), _ptr(values),
                                                    c_int(n), c_int(logits.shape[1]), _stream()))
