"""Python face of the HIP kernels: checks operands on the host, then launches
on the current stream.  Tensors are torch tensors on the GPU (torch is the
allocator and the stream owner; the arithmetic is in `*.hip`).  There is no
CPU path: without a GPU or without the compiled libraries these raise.
"""
from __future__ import annotations

import ctypes
from typing import Optional

import torch

from ..parts.base import Injected, PartialSums, Prenormed, ScaledSum
from . import build
from .tuning import ProductTuning
from .limits import (MAX_DELTA_HEAD_DIM, MAX_GLA_HEAD_DIM, MAX_HEAD_DIM, MAX_SSD_DIM, MAX_SUMMED_NORM_WIDTH,
                     MAX_WKV_HEAD_DIM)

F32, BF16 = 0, 1
_P = ctypes.c_void_p
_I = ctypes.c_int
_L = ctypes.c_int64
_F = ctypes.c_float


class KernelError(RuntimeError):
    pass


def dtype_code(dtype: torch.dtype) -> int:
    if dtype == torch.float32:
        return F32
    if dtype == torch.bfloat16:
        return BF16
    raise KernelError(f"kernels take float32 or bfloat16 tensors, not {dtype}")


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _need(cond: bool, msg: str) -> None:
    if not cond:
        raise KernelError(msg)


def _dev(t: torch.Tensor, name: str, dtype=None) -> None:
    # (on every operand of every launch: the messages are made only when they are needed)
    if not t.is_cuda:
        raise KernelError(f"{name} must live on the GPU")
    if not t.is_contiguous():
        raise KernelError(f"{name} must be contiguous")
    if dtype is not None and t.dtype != dtype:
        raise KernelError(f"{name} must be {dtype}, is {t.dtype}")


def _rows(t: torch.Tensor, name: str, dtype=None) -> None:
    """A matrix whose rows may lie apart (some columns of a wider one): elements of a row are neighbours."""
    if not t.is_cuda:
        raise KernelError(f"{name} must live on the GPU")
    if t.dim() != 2 or (t.shape[1] > 1 and t.stride(1) != 1):
        raise KernelError(f"{name} must be a matrix with contiguous rows")
    if dtype is not None and t.dtype != dtype:
        raise KernelError(f"{name} must be {dtype}, is {t.dtype}")


# the current stream's handle without the Stream object around it (a launch is a few microseconds
# of Python as it is; torch.cuda.current_stream() alone costs as much again)
_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)


_raw_device = getattr(torch._C, "_cuda_getDevice", None)


def _stream_handle() -> int:
    if _raw_stream is not None and _raw_device is not None:
        return _raw_stream(_raw_device())
    return torch.cuda.current_stream().cuda_stream


class HipOps:
    """The operations a model part may call.  One instance per process is enough."""

    MAX_HEAD_DIM = MAX_HEAD_DIM

    def __init__(self, tuning: Optional[ProductTuning] = None):
        if not torch.cuda.is_available():
            raise KernelError("litellmengine_amd needs a GPU: its kernels have no CPU form")
        self._fn = {}
        self.tuning = tuning or ProductTuning()  # which kernel takes a product (never what it gives)

    # -- plumbing ---------------------------------------------------------
    def _get(self, lib: str, name: str, argtypes):
        key = (lib, name)
        fn = self._fn.get(key)
        if fn is None:
            fn = getattr(build.load_library(lib), name)
            fn.argtypes = argtypes
            fn.restype = ctypes.c_int
            self._fn[key] = fn
        return fn

    def _run(self, lib: str, name: str, argtypes, *args):
        fn = self._get(lib, name, argtypes)
        code = fn(*args, _stream_handle())
        if code != 0:
            msg = build.load_library(lib).lle_error_string(code).decode()
            raise KernelError(f"{name} failed to launch: {msg} (hip error {code})")

    # -- embedding -----------------------------------------------------------
    def embedding(self, ids: torch.Tensor, table: torch.Tensor, feedback=None, token_seq=None,
                  seq_slots=None, scale: float = 1.0) -> torch.Tensor:
        """ids int32 [N], table [V, H] -> float32 [N, H] (the residual stream), times `scale`.  With `feedback`
        (int32, indexed by request slot), `token_seq` [N] and `seq_slots`: an id below zero is
        replaced by feedback[seq_slots[token_seq[n]]], the token that argmax(..., scatter=...) left there."""
        _dev(ids, "ids", torch.int32)
        _dev(table, "embedding table")
        _need(ids.dim() == 1 and table.dim() == 2, "embedding wants ids [N] and a table [V, H]")
        N, H = ids.shape[0], table.shape[1]
        if feedback is not None:
            for t, name in ((feedback, "feedback"), (token_seq, "token_seq"), (seq_slots, "seq_slots")):
                _need(t is not None, "feedback, token_seq and seq_slots come together")
                _dev(t, name, torch.int32)
            _need(token_seq.shape == (N,), "token_seq must be [N]")
        out = torch.empty((N, H), dtype=torch.float32, device=table.device)
        self._run("elementwise", "lle_embedding_scaled", [_P, _P, _P, _I, _I, _I, _P, _P, _P, _F, _P],
                  _ptr(ids), _ptr(table), _ptr(out), N, H, dtype_code(table.dtype), _ptr(feedback),
                  _ptr(token_seq) if feedback is not None else None, _ptr(seq_slots) if feedback is not None else None,
                  float(scale))
        return out

    def embedding_rmsnorm(self, ids, table, weight, eps: float, feedback=None, token_seq=None, seq_slots=None):
        """embedding() and the RMSNorm of its rows in one launch: (float32 [N, H] residual stream,
        [N, H] normed rows in the table's type)."""
        _dev(ids, "ids", torch.int32)
        _dev(table, "embedding table")
        _dev(weight, "norm weight")
        _need(ids.dim() == 1 and table.dim() == 2, "embedding wants ids [N] and a table [V, H]")
        N, H = ids.shape[0], table.shape[1]
        _need(weight.shape == (H,), f"norm weight must be [{H}], is {list(weight.shape)}")
        if feedback is not None:
            for t, name in ((feedback, "feedback"), (token_seq, "token_seq"), (seq_slots, "seq_slots")):
                _need(t is not None, "feedback, token_seq and seq_slots come together")
                _dev(t, name, torch.int32)
            _need(token_seq.shape == (N,), "token_seq must be [N]")
        hidden = torch.empty((N, H), dtype=torch.float32, device=table.device)
        out = torch.empty((N, H), dtype=table.dtype, device=table.device)
        self._run("norm", "lle_embedding_rmsnorm", [_P, _P, _P, _P, _I, _P, _I, _I, _F, _I, _P, _P, _P, _P],
                  _ptr(ids), _ptr(table), _ptr(hidden), _ptr(weight), dtype_code(weight.dtype), _ptr(out), N, H,
                  float(eps), dtype_code(table.dtype), _ptr(feedback),
                  _ptr(token_seq) if feedback is not None else None, _ptr(seq_slots) if feedback is not None else None)
        return hidden, out

    def embedding_norm(self, ids, table, scale: float, positions, pos_table, weight, eps: float, next_weight, next_eps: float,
                       out_dtype, feedback=None, token_seq=None, seq_slots=None):
        """The first rows of the residual stream where they are more than the embedding's: float32 [N, H]
        h[n] = RMSNorm(table[ids[n]] * scale + pos_table[positions[n]]) * weight (`pos_table` None: no position vectors;
        `weight` None: without that norm), and RMSNorm(h) * next_weight in `out_dtype` from the same launch (None where
        `next_weight` is None).  The caller has checked ids and positions."""
        _dev(ids, "ids", torch.int32)
        _dev(table, "embedding table")
        _need(ids.dim() == 1 and table.dim() == 2, "embedding wants ids [N] and a table [V, H]")
        N, H = ids.shape[0], table.shape[1]
        if pos_table is not None:
            _dev(pos_table, "position table")
            _dev(positions, "positions", torch.int32)
            _need(pos_table.dim() == 2 and pos_table.shape[1] == H and pos_table.shape[0] > 0, f"the position table must be [P, {H}]")
            _need(positions.shape == (N,), "positions must be [N]")
        for t, name in ((weight, "norm weight"), (next_weight, "next norm weight")):
            if t is not None:
                _dev(t, name)
                _need(t.shape == (H,), f"{name} must be [{H}]")
        if feedback is not None:
            for t, name in ((feedback, "feedback"), (token_seq, "token_seq"), (seq_slots, "seq_slots")):
                _need(t is not None, "feedback, token_seq and seq_slots come together")
                _dev(t, name, torch.int32)
            _need(token_seq.shape == (N,), "token_seq must be [N]")
        hidden = torch.empty((N, H), dtype=torch.float32, device=table.device)
        out = torch.empty((N, H), dtype=out_dtype, device=table.device) if next_weight is not None else None
        code = lambda t: F32 if t is None else dtype_code(t.dtype)
        self._run("norm", "lle_embedding_norm",
                  [_P, _P, _I, _F, _P, _P, _P, _P, _I, _I, _P, _P, _I, _F, _P, _P, _I, _F, _P, _I, _I, _I, _P],
                  _ptr(ids), _ptr(table), dtype_code(table.dtype), float(scale), _ptr(feedback),
                  _ptr(token_seq) if feedback is not None else None, _ptr(seq_slots) if feedback is not None else None,
                  _ptr(pos_table), code(pos_table), pos_table.shape[0] if pos_table is not None else 0,
                  _ptr(positions) if pos_table is not None else None, _ptr(weight), code(weight), float(eps), _ptr(hidden),
                  _ptr(next_weight), code(next_weight), float(next_eps), _ptr(out), N, H, dtype_code(out_dtype))
        return hidden, out

    # -- norms ---------------------------------------------------------------
    def add_rmsnorm(self, hidden, delta, weight, eps: float, out_dtype, rows=None) -> torch.Tensor:
        """hidden float32 [N, H] (+ delta [N, H] of out_dtype, or float32 partial sums
        [slices, N, H], bare or as PartialSums, that are added in slice order) -> norm * weight, out_dtype.
        Without `rows` the sum is written back to `hidden` and every row is normed;
        with `rows` (int32 [R]) only those rows are read and nothing is written back."""
        _dev(hidden, "hidden", torch.float32)
        _dev(weight, "norm weight")
        N, H = hidden.shape
        _need(weight.shape == (H,), f"norm weight must be [{H}], is {list(weight.shape)}")
        if isinstance(delta, PartialSums):
            delta = delta.sums
        sums = delta is not None and delta.dim() == 3  # partial sums of a product taken in slices of K
        if sums:
            _dev(delta, "partial sums", torch.float32)
            _need(delta.shape[1:] == hidden.shape and H % 4 == 0 and H <= MAX_SUMMED_NORM_WIDTH,
                  f"partial sums {list(delta.shape)} do not fit the residual stream {list(hidden.shape)}")
        elif delta is not None:
            _dev(delta, "delta", out_dtype)
            _need(delta.shape == hidden.shape, "delta must have the shape of hidden")
        if rows is not None:
            _dev(rows, "rows", torch.int32)
            R = rows.shape[0]
        else:
            R = N
        out = torch.empty((R, H), dtype=out_dtype, device=hidden.device)
        if sums:
            self._run("norm", "lle_add_rmsnorm_sums", [_P, _P, _I, _L, _P, _P, _I, _P, _I, _I, _F, _I, _P],
                      _ptr(hidden), _ptr(delta), delta.shape[0], delta.stride(0), _ptr(rows), _ptr(weight),
                      dtype_code(weight.dtype), _ptr(out), R, H, float(eps), dtype_code(out_dtype))
            return out
        self._run("norm", "lle_add_rmsnorm", [_P, _P, _P, _P, _I, _P, _I, _I, _F, _I, _P],
                  _ptr(hidden), _ptr(delta), _ptr(rows), _ptr(weight), dtype_code(weight.dtype), _ptr(out),
                  R, H, float(eps), dtype_code(out_dtype))
        return out

    def rmsnorm(self, x, weight, eps: float, out_dtype=None) -> torch.Tensor:
        """x [R, H] -> x * rsqrt(mean(x^2) + eps) * weight, same type (`out_dtype` bfloat16 for float32 rows: the
        result in bfloat16 from the same launch)."""
        _dev(x, "x")
        _dev(weight, "norm weight")
        R, H = x.shape
        _need(weight.shape == (H,), f"norm weight must be [{H}], is {list(weight.shape)}")
        if out_dtype is not None and out_dtype != x.dtype:
            _need(x.dtype == torch.float32 and out_dtype == torch.bfloat16, "a norm hands float32 rows on as they are or in bfloat16")
            out = torch.empty((R, H), dtype=out_dtype, device=x.device)
            self._run("norm", "lle_rmsnorm_f32_to_bf16", [_P, _P, _I, _P, _I, _I, _F, _P],
                      _ptr(x), _ptr(weight), dtype_code(weight.dtype), _ptr(out), R, H, float(eps))
            return out
        out = torch.empty_like(x)
        self._run("norm", "lle_rmsnorm", [_P, _P, _I, _P, _I, _I, _F, _I, _P],
                  _ptr(x), _ptr(weight), dtype_code(weight.dtype), _ptr(out), R, H, float(eps), dtype_code(x.dtype))
        return out

    # -- matrix products -------------------------------------------------------
    def can_fold_norm(self, rows: int, width: int, dtype) -> bool:
        """Whether an RMSNorm over `width` of a step of `rows` tokens can be done by the
        products before and after it (the weight-streaming kernel's few-rows forms)."""
        most = 32 if width <= self.tuning.skinny_small_width else self.tuning.skinny_max_rows
        return dtype == torch.bfloat16 and 0 < rows <= most and width % 8 == 0 and not self.force_library_gemm

    def norm_sum_parts(self, width: int) -> int:
        """Into how many column ranges the product before a folded norm over `width` splits the
        sums of squares (one per tile of its launch; the kernel library decides the tiles)."""
        fn = getattr(build.load_library("gemm"), "lle_gemm_skinny_resid_parts")
        fn.argtypes, fn.restype = [_I], _I
        return int(fn(int(width)))

    def _linear_folded(self, x, weight, fold, gated: bool, out_dtype=torch.bfloat16):
        """The forms of the weight-streaming product around a folded norm: `x` a Prenormed
        (its row factors are applied to the result), `fold` a NormFold (the result goes
        into the residual stream and comes back as the next Prenormed)."""
        pre = x if isinstance(x, Prenormed) else None
        xin = pre.xw if pre is not None else x
        _dev(xin, "x", torch.bfloat16)
        _dev(weight, "weight", torch.bfloat16)
        M, K = xin.shape
        N = weight.shape[0]
        _need(weight.shape[1] == K, f"weight [{N}, {weight.shape[1]}] does not fit x [{M}, {K}]")
        _need(K % 8 == 0, f"the weight-streaming product needs a multiple of 8 columns, not {K}")
        _need(pre is None or fold is None, "a product takes a Prenormed or makes one, not both")
        if pre is not None:
            _need(self.can_fold_norm(M, K, xin.dtype), f"a norm over {K} cannot be folded for {M} rows")
            _dev(pre.sums, "sums", torch.float32)
            parts = pre.sums.shape[1]
            _need(pre.sums.shape == (16 if M <= 16 else 32, parts) and pre.xw.shape[1] == K,
                  "sums of squares do not fit")
            _need(not gated or N % 2 == 0, "a gated weight has an even number of rows")
            _need(out_dtype == torch.bfloat16 or (out_dtype == torch.float32 and not gated),
                  "the product after a folded norm writes bfloat16, or float32 where it is not gated")
            out = torch.empty((M, N // 2 if gated else N), dtype=out_dtype, device=xin.device)
            self._run("gemm", "lle_gemm_skinny_scaled_bf16", [_P, _P, _P, _P, _I, _F, _I, _I, _I, _I, _I, _P],
                      _ptr(xin), _ptr(weight), _ptr(out), _ptr(pre.sums), parts, float(pre.eps), M, N, K, int(gated),
                      dtype_code(out_dtype))
            return out
        _dev(fold.hidden, "hidden", torch.float32)
        _dev(fold.weight, "norm weight")
        _need(not gated and fold.hidden.shape == (M, N) and fold.weight.shape == (N,),
              f"residual stream {list(fold.hidden.shape)} does not fit a product [{M}, {N}]")
        _need(self.can_fold_norm(M, N, xin.dtype), f"a norm over {N} cannot be folded for {M} rows")
        xw = torch.empty((M, N), dtype=torch.bfloat16, device=xin.device)
        sums = torch.empty((16 if M <= 16 else 32, self.norm_sum_parts(N)), dtype=torch.float32, device=xin.device)
        self._run("gemm", "lle_gemm_skinny_resid_bf16", [_P, _P, _P, _P, _I, _P, _P, _I, _I, _I, _P],
                  _ptr(xin), _ptr(weight), _ptr(fold.hidden), _ptr(fold.weight), dtype_code(fold.weight.dtype),
                  _ptr(xw), _ptr(sums), M, N, K)
        return Prenormed(xw, sums, fold.eps)

    def linear(self, x, weight, out_dtype=None, fold=None, sums_ok=False):
        """x [M, K] . weight [N, K]^T -> [M, N].  With `sums_ok` the caller takes the result also as
        PartialSums (float32 [slices, M, N], what add_rmsnorm adds into the residual stream).  float32 operands take a true 32-bit
        product: few rows the weight-streaming kernel, more rows a tiled kernel, both
        with the float32 matrix instruction; the plain-FMA kernel where K is no multiple of 4.  bfloat16 operands: few rows take the
        weight-streaming matrix-core kernel, more rows the library product; both
        accumulate in 32-bit and write either result type.  `x` a Prenormed or `fold`
        a NormFold: see _linear_folded."""
        if fold is not None or isinstance(x, Prenormed):
            _need(out_dtype in (None, torch.bfloat16) or (fold is None and out_dtype == torch.float32),
                  "a product that makes a folded norm's input writes bfloat16")
            return self._linear_folded(x, weight, fold, gated=False, out_dtype=out_dtype or torch.bfloat16)
        _dev(x, "x")
        _dev(weight, "weight", x.dtype)
        M, K = x.shape
        N = weight.shape[0]
        _need(weight.shape[1] == K, f"weight [{N}, {weight.shape[1]}] does not fit x [{M}, {K}]")
        out_dtype = out_dtype or x.dtype
        if x.dtype == torch.bfloat16:
            if sums_ok and out_dtype == torch.bfloat16:
                slices = self.slices_for(M, N, K)
                if slices:
                    return PartialSums(self.linear_slices(x, weight, slices))
                slices = self.library_slices_for(M, N, K)
                if slices:
                    # one batched library product over the slices of K, partial sums left in 32-bit
                    xs = x.view(M, slices, K // slices).permute(1, 0, 2)
                    ws = weight.view(N, slices, K // slices).permute(1, 2, 0)
                    return PartialSums(torch.bmm(xs, ws, out_dtype=torch.float32))
            t = self.tuning
            skinny = K % 8 == 0 and not self.force_library_gemm and (
                M <= t.skinny_max_rows
                or (M <= 32 and K <= t.skinny_small_width and N * K <= t.skinny_small_weight)
                # 17 to 32 rows against a weight with many rows for every CU: the streaming kernel with two
                # tiles of X rows in its registers (K a multiple of 1024 up to 4096)
                or (M <= 32 and K % 1024 == 0 and K <= 4096 and N >= t.stream_32_rows_min_share * self.compute_units()))
            if skinny:
                out = torch.empty((M, N), dtype=out_dtype, device=x.device)
                self._run("gemm", "lle_gemm_skinny_bf16", [_P, _P, _P, _I, _I, _I, _I, _P],
                          _ptr(x), _ptr(weight), _ptr(out), M, N, K, dtype_code(out_dtype))
                return out
            # the library product accumulates in 32-bit and can leave the result so
            return torch.mm(x, weight.t()) if out_dtype == torch.bfloat16 else torch.mm(x, weight.t(), out_dtype=out_dtype)
        _need(out_dtype == torch.float32, "a float32 product has a float32 result")
        out = torch.empty((M, N), dtype=out_dtype, device=x.device)
        if M <= self.tuning.skinny_f32_max_rows and K % 4 == 0 and not self.force_library_gemm:
            # few rows: W streamed once, float32 matrix instruction
            self._run("gemm", "lle_gemm_skinny_f32", [_P, _P, _P, _I, _I, _I, _P], _ptr(x), _ptr(weight), _ptr(out),
                      M, N, K)
            return out
        if K % 4 == 0 and not self.force_simt_gemm:
            # many rows: 64 x 64 tiles through the float32 matrix instruction
            self._run("gemm", "lle_gemm_nt_mfma_f32", [_P, _P, _P, _I, _I, _I, _L, _L, _L, _P],
                      _ptr(x), _ptr(weight), _ptr(out), M, N, K, K, K, N)
            return out
        self._run("gemm", "lle_gemm_nt_simt", [_P, _P, _P, _I, _I, _I, _L, _L, _L, _I, _I, _P],
                  _ptr(x), _ptr(weight), _ptr(out), M, N, K, K, K, N, dtype_code(x.dtype), dtype_code(out_dtype))
        return out

    SLICED_MIN_ROWS, SLICED_MAX_ROWS = 17, 128  # (lle_gemm_mid_slices_max_rows)
    SLICED_UNIT = 1024  # columns of K that a slice is a multiple of (lle_gemm_mid_slices_unit)

    def slices_for(self, M: int, N: int, K: int) -> int:
        """In how many slices of K the product of 17 to 128 rows with a weight [N, K] is taken
        (see linear_slices), or 0 where the library product stays.  Weights with rows enough for
        every CU need no slices.  For the others the slice count is the one that a small model of
        the kernel's time likes best (rounds of N / 64 x slices workgroups over the CUs, each
        taking in its W and X at what a CU takes in, plus the way of the partial sums to the norm
        and back), and it is used where the workgroups fill the CUs in whole rounds (at least
        0.85 of them: o_proj, down_proj of the 8B sizes), or where K is at least twice N and the
        weight is not small: there the library's tiles are too few for the CUs and it does not
        split K (measured at 64 rows: down_proj of the 32B sizes, 5120 x 25600, in 5 slices 76 us
        against the library's 158; of the 14B sizes, 5120 x 17408, in 17 slices 70 against 132)."""
        if not (self.SLICED_MIN_ROWS <= M <= self.SLICED_MAX_ROWS) or N % 64 != 0 or self.force_library_gemm:
            return 0
        if N > MAX_SUMMED_NORM_WIDTH:  # the only reader of the partial sums (add_rmsnorm) takes no wider rows
            return 0
        units, t = self.compute_units(), self.tuning
        groups = N // 64
        if groups > units // 2 or K % self.SLICED_UNIT != 0:  # (rows enough for the library's own tiles)
            return 0
        parts = K // self.SLICED_UNIT
        rows = 32 if M <= 32 else 64 if M <= 64 else 96 if M <= 96 else 128  # the kernel's tiles of X
        best, best_time, best_fill = 0, 0.0, 0.0
        for slices in range(1, min(parts, 32) + 1):
            if parts % slices != 0:
                continue
            rounds = -(-groups * slices // units)
            taken_in = (64 + rows) * (K // slices) * 2  # bytes of W and X through a CU
            seconds = (rounds * (t.sliced_round_seconds + taken_in / t.cu_intake_bytes_per_s)
                       + slices * M * N * 8 / t.partial_sums_bytes_per_s)
            if best == 0 or seconds < best_time:
                best, best_time, best_fill = slices, seconds, groups * slices / (rounds * units)
        if best_fill >= t.sliced_min_fill or (K >= 2 * N and N * K >= t.sliced_long_k_min_weight):
            return best
        return 0

    def library_slices_for(self, M: int, N: int, K: int) -> int:
        """In how many slices of K the LIBRARY takes a product of more than 128 rows whose result is a
        delta of the residual stream, or 0 for the whole product.  The library cuts the result into
        tiles of up to 256 x 256 and does not split K: a weight with few rows and a long K
        (down_proj) leaves CUs without a tile or gets small tiles.  Slices are tiles as well (one
        batched product), up to 4 while the CUs have room for them; the residual add + norm then
        reads float32 partial sums, which costs part of the gain.  Measured at 4096 x 12288 against
        the whole product, both with the norm: 512 rows 90 -> 65 us (4 slices), 1024 rows 126 -> 106
        (4), 2048 rows 214 -> 205 (2), 4096 rows slower (not taken); square weights (o_proj) gain nothing."""
        if M <= self.SLICED_MAX_ROWS or self.force_library_gemm or K < 2 * N:
            return 0
        if N > MAX_SUMMED_NORM_WIDTH or N % 4 != 0:
            return 0
        tiles = -(-M // 256) * -(-N // 256)
        slices = min(self.tuning.library_max_slices, self.compute_units() // tiles)
        while slices > 1 and K % (8 * slices) != 0:
            slices -= 1
        return slices if slices > 1 else 0

    def linear_slices(self, x, weight, slices: int) -> torch.Tensor:
        """x [M, K] . weight [N, K]^T as float32 partial sums over `slices` equal parts of K:
        [slices, M, N], to be added up by the reader in slice order (M <= 128)."""
        _dev(x, "x", torch.bfloat16)
        _dev(weight, "weight", torch.bfloat16)
        M, K = x.shape
        N = weight.shape[0]
        _need(weight.shape[1] == K, f"weight [{N}, {weight.shape[1]}] does not fit x [{M}, {K}]")
        _need(0 < M <= self.SLICED_MAX_ROWS and N % 64 == 0 and slices > 0 and K % (self.SLICED_UNIT * slices) == 0,
              f"no product in {slices} slices for [{M}, {K}] x [{N}, {K}]")
        out = torch.empty((slices, M, N), dtype=torch.float32, device=x.device)
        self._run("gemm", "lle_gemm_mid_slices_bf16", [_P, _P, _P, _I, _I, _I, _I, _P], _ptr(x), _ptr(weight), _ptr(out),
                  M, N, K, slices)
        return out

    # (which of these kernels takes a product is decided by the numbers in self.tuning)
    force_library_gemm = False
    force_simt_gemm = False  # tests flip this to reach the plain-FMA kernel at sizes the matrix instruction takes

    # -- attention ---------------------------------------------------------------
    def rope_table(self, positions, inv_freq) -> torch.Tensor:
        """cos and sin of float(position) * inv_freq for every token: float32 [N, len(inv_freq), 2].
        Made once per step; every head of every layer with this rotation reads it."""
        _dev(positions, "positions", torch.int32)
        _dev(inv_freq, "inv_freq", torch.float32)
        N, half = positions.shape[0], inv_freq.shape[0]
        out = torch.empty((N, half, 2), dtype=torch.float32, device=positions.device)
        self._run("rope_kv", "lle_rope_table", [_P, _P, _P, _I, _I, _P], _ptr(positions), _ptr(inv_freq), _ptr(out),
                  N, half)
        return out

    def qk_norm_rope_write(self, qkv, slots, q_weight, k_weight, cos_sin, rotary_dim: int, eps: float, kv_layer,
                           num_q_heads: int, num_kv_heads: int, head_dim: int, write_kv: bool = True) -> torch.Tensor:
        """qkv [N, (nq + 2 nkv) d] -> q [N, nq, d] normed and rotated; K (normed, rotated)
        and V go to the pages `kv_layer` [pages, 2, nkv, page_size, d] at `slots` [N].
        `cos_sin` is rope_table()'s [N, rotary_dim / 2, 2] (None when rotary_dim is 0)."""
        _dev(qkv, "qkv")
        _dev(slots, "slots", torch.int32)
        _dev(kv_layer, "kv_layer", qkv.dtype)
        nq, nkv, d = num_q_heads, num_kv_heads, head_dim
        N = qkv.shape[0]
        _need(qkv.shape == (N, (nq + 2 * nkv) * d), "qkv has the wrong width")
        _need(slots.shape == (N,), "slots must be [N]")
        _need(kv_layer.dim() == 5 and kv_layer.shape[1] == 2 and kv_layer.shape[2] == nkv
              and kv_layer.shape[4] == d, "kv_layer must be [pages, 2, nkv, page_size, d]")
        _need(0 <= rotary_dim <= d and rotary_dim % 2 == 0, "rotary_dim must be even and <= head_dim")
        wd = F32
        for w, name in ((q_weight, "q_norm weight"), (k_weight, "k_norm weight")):
            if w is not None:
                _dev(w, name)
                _need(w.shape == (d,), f"{name} must be [{d}]")
                wd = dtype_code(w.dtype)
        if q_weight is not None and k_weight is not None:
            _need(q_weight.dtype == k_weight.dtype, "q_norm and k_norm weights must share a type")
        if rotary_dim > 0:
            _dev(cos_sin, "cos_sin", torch.float32)
            _need(cos_sin.shape == (N, rotary_dim // 2, 2), "cos_sin must be [N, rotary_dim / 2, 2]")
        page_size = kv_layer.shape[3]
        q_out = torch.empty((N, nq, d), dtype=qkv.dtype, device=qkv.device)
        self._run("rope_kv", "lle_qk_norm_rope_write",
                  [_P, _P, _P, _P, _I, _P, _I, _F, _P, _P, _I, _I, _I, _I, _I, _L, _I, _I, _P],
                  _ptr(qkv), _ptr(slots), _ptr(q_weight), _ptr(k_weight), wd,
                  _ptr(cos_sin) if rotary_dim > 0 else None, rotary_dim, float(eps), _ptr(q_out), _ptr(kv_layer),
                  N, nq, nkv, d, page_size, kv_layer.stride(0), 1 if write_kv else 0, dtype_code(qkv.dtype))
        return q_out

    def paged_attention(self, q, kv_layer, block_table, seq_slots, cu_tokens, kv_lens, token_seq,
                        window: Optional[int], scale: float, min_q_len: int = 0, max_q_len: int = 0,
                        max_kv_len: int = 0, sinks=None, keep_first: int = 0, softcap: Optional[float] = None) -> torch.Tensor:
        """q [N, nq, d] against the pages -> [N, nq * d].  `softcap`: the scores pass through
        softcap * tanh(score / softcap) (None: not).  `keep_first`: beside a window the first so many keys stay
        in sight too.  `sinks` (float32 [nq], or None): every head's
        softmax has one more place, with that score and no value: p_j = exp(s_j) / (exp(sink) + sum exp(s_j)).
        `min_q_len`, `max_q_len`
        and `max_kv_len` are host-side bounds of this batch; they choose the kernels
        and the number of key splits, never the result.  bfloat16 with head_dim a
        multiple of 32 and a page size a multiple of 16 runs on the matrix cores;
        everything else takes the generic kernel."""
        _dev(q, "q")
        _dev(kv_layer, "kv_layer", q.dtype)
        for t, name in ((block_table, "block_table"), (seq_slots, "seq_slots"), (cu_tokens, "cu_tokens"),
                        (kv_lens, "kv_lens"), (token_seq, "token_seq")):
            _dev(t, name, torch.int32)
        N, nq, d = q.shape
        nkv, page_size = kv_layer.shape[2], kv_layer.shape[3]
        _need(kv_layer.shape[4] == d and kv_layer.shape[1] == 2, "kv_layer must be [pages, 2, nkv, page_size, d]")
        _need(nq % nkv == 0, "q heads must be a multiple of kv heads")
        _need(d <= self.MAX_HEAD_DIM, f"head_dim {d} is larger than the attention kernels take ({self.MAX_HEAD_DIM})")
        _need(token_seq.shape == (N,), "token_seq must be [N]")
        S = seq_slots.shape[0]
        _need(cu_tokens.shape == (S + 1,) and kv_lens.shape == (S,), "cu_tokens [S + 1], kv_lens [S]")
        _need(block_table.dim() == 2, "block_table must be [slots, pages]")
        if sinks is not None:
            _dev(sinks, "sinks", torch.float32)
            _need(sinks.shape == (nq,), "sinks must be [nq]")
        out = torch.empty((N, nq * d), dtype=q.dtype, device=q.device)
        win = int(window) if window else 0
        keep = int(keep_first) if win else 0
        _need(keep >= 0, "keep_first must not be negative")
        cap = float(softcap) if softcap else 0.0
        _need(cap >= 0.0, "a cap must be positive")
        both = keep > 0 and cap > 0.0  # (only the generic kernel knows kept keys and capped scores together)
        mfma = (q.dtype == torch.bfloat16 and d % 32 == 0 and page_size % 16 == 0 and max_q_len > 0
                and max_kv_len > 0 and S <= 65535 and not both and not self.force_generic_attention)
        group = nq // nkv
        if (q.dtype == torch.float32 and d % 16 == 0 and page_size % 16 == 0 and max_q_len > 0 and max_kv_len > 0
                and S <= 65535 and not both and not self.force_generic_attention):
            # float32 on the matrix cores (float32 operands, products and sums)
            rows = max_q_len * group
            row_blocks = 1 if rows <= 16 else -(-rows // 64)
            ns = self.f32_attention_splits(S, nkv, row_blocks, max_q_len, max_kv_len, win)
            ws_o = ws_ml = None
            if ns > 1:
                ws_o = torch.empty((N * nq * ns * d,), dtype=torch.float32, device=q.device)
                ws_ml = torch.empty((N * nq * ns * 2,), dtype=torch.float32, device=q.device)
            self._run("attention", "lle_paged_attention_mfma_f32",
                      [_P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _L, _I, _I, _I, _F, _I, _I, _P, _F, _P],
                      _ptr(q), _ptr(kv_layer), _ptr(block_table), _ptr(seq_slots), _ptr(cu_tokens), _ptr(kv_lens),
                      _ptr(out), _ptr(ws_o), _ptr(ws_ml), N, S, nq, nkv, d, page_size, kv_layer.stride(0),
                      block_table.shape[1], win, keep, float(scale), row_blocks, ns, _ptr(sinks), cap)
            return out
        if not mfma:
            self._run("attention", "lle_paged_attention_generic",
                      [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _L, _I, _I, _I, _F, _I, _P, _F, _P],
                      _ptr(q), _ptr(kv_layer), _ptr(block_table), _ptr(seq_slots), _ptr(cu_tokens), _ptr(kv_lens),
                      _ptr(token_seq), _ptr(out), N, nq, nkv, d, page_size, kv_layer.stride(0), block_table.shape[1],
                      win, keep, float(scale), dtype_code(q.dtype), _ptr(sinks), cap)
            return out
        min_q_len = min_q_len or 1
        run_decode = min_q_len * group <= 16
        run_prefill = max_q_len * group > 16
        ns_decode = self.decode_splits(S, nkv, max_kv_len, win) if run_decode else 1
        ns_prefill = self.prefill_splits(S, nkv, group, d, max_q_len, max_kv_len, win) if run_prefill else 1
        row_tiles = (self.prefill_form(S, nkv, group, d, max_q_len, max_kv_len, win, ns_prefill, q.device)
                     if run_prefill else 0)
        ns = max(ns_decode, ns_prefill)
        ws_o = ws_ml = None
        if ns > 1:
            ws_o = torch.empty((N * nq * ns * d,), dtype=torch.float32, device=q.device)
            ws_ml = torch.empty((N * nq * ns * 2,), dtype=torch.float32, device=q.device)
        self._run("attention", "lle_paged_attention_mfma",
                  [_P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _L, _I, _I, _F, _I, _I, _I, _I, _I, _I,
                   _P, _I, _F, _P],
                  _ptr(q), _ptr(kv_layer), _ptr(block_table), _ptr(seq_slots), _ptr(cu_tokens), _ptr(kv_lens),
                  _ptr(token_seq), _ptr(out), _ptr(ws_o), _ptr(ws_ml), N, S, nq, nkv, d, page_size,
                  kv_layer.stride(0), block_table.shape[1], win, float(scale), int(run_decode), ns_decode,
                  int(run_prefill), ns_prefill, max_q_len, row_tiles, _ptr(sinks), keep, cap)
        return out

    def can_fuse_rope_attention(self, dtype, head_dim: int, rotary_dim: int, page_size: int, group: int,
                                max_q_len: int, max_kv_len: int, num_seqs: int) -> bool:
        """Whether qk_norm_rope_attention takes this step: bfloat16, a rotation over the whole head
        of a multiple of 64 elements, and only requests of at most 16 / group tokens (decode steps)."""
        return (dtype == torch.bfloat16 and head_dim % 64 == 0 and head_dim <= self.MAX_HEAD_DIM
                and rotary_dim == head_dim and page_size % 16 == 0 and 0 < max_q_len and max_q_len * group <= 16
                and max_kv_len > 0 and num_seqs <= 65535 and not self.force_generic_attention
                and not self.force_separate_rope)

    def qk_norm_rope_attention(self, qkv, slots, q_weight, k_weight, cos_sin, eps: float, kv_layer, nq: int,
                               nkv: int, d: int, write_kv: bool, block_table, seq_slots, cu_tokens, kv_lens,
                               token_seq, window: Optional[int], scale: float, max_kv_len: int) -> torch.Tensor:
        """qk_norm_rope_write and paged_attention of a decode step in one launch (see
        can_fuse_rope_attention): the workgroup whose keys include a new token's position writes
        its K and V, every workgroup norms and rotates the q rows it multiplies."""
        _dev(qkv, "qkv", torch.bfloat16)
        _dev(kv_layer, "kv_layer", torch.bfloat16)
        _dev(cos_sin, "cos_sin", torch.float32)
        for t, name in ((slots, "slots"), (block_table, "block_table"), (seq_slots, "seq_slots"),
                        (cu_tokens, "cu_tokens"), (kv_lens, "kv_lens"), (token_seq, "token_seq")):
            _dev(t, name, torch.int32)
        N = qkv.shape[0]
        page_size = kv_layer.shape[3]
        _need(qkv.shape[1] == (nq + 2 * nkv) * d, "qkv must be [N, (nq + 2 nkv) * d]")
        _need(tuple(kv_layer.shape[1:]) == (2, nkv, page_size, d), "kv_layer must be [pages, 2, nkv, page_size, d]")
        _need(slots.shape == (N,) and token_seq.shape == (N,), "slots and token_seq must be [N]")
        _need(cos_sin.shape == (N, d // 2, 2), f"cos_sin must be [{N}, {d // 2}, 2]")
        _need((q_weight is None) == (k_weight is None), "q and k norm weights come together")
        wcode = 0
        if q_weight is not None:
            _dev(q_weight, "q_weight")
            _dev(k_weight, "k_weight", q_weight.dtype)
            _need(q_weight.shape == (d,) and k_weight.shape == (d,), f"q/k norm weights must be [{d}]")
            wcode = dtype_code(q_weight.dtype)
        S = seq_slots.shape[0]
        _need(cu_tokens.shape == (S + 1,) and kv_lens.shape == (S,), "cu_tokens [S + 1], kv_lens [S]")
        _need(nq % nkv == 0 and d % 64 == 0 and page_size % 16 == 0 and S <= 65535,
              "the fused decode attention does not take these sizes")
        win = int(window) if window else 0
        ns = self.decode_splits(S, nkv, max_kv_len, win)
        out = torch.empty((N, nq * d), dtype=torch.bfloat16, device=qkv.device)
        ws_o = ws_ml = None
        if ns > 1:
            ws_o = torch.empty((N * nq * ns * d,), dtype=torch.float32, device=qkv.device)
            ws_ml = torch.empty((N * nq * ns * 2,), dtype=torch.float32, device=qkv.device)
        self._run("attention", "lle_qk_norm_rope_attention_decode",
                  [_P, _P, _P, _P, _I, _P, _F, _I, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _L, _I, _I,
                   _F, _I, _P],
                  _ptr(qkv), _ptr(slots), _ptr(q_weight), _ptr(k_weight), wcode, _ptr(cos_sin), float(eps),
                  int(bool(write_kv)), _ptr(kv_layer), _ptr(block_table), _ptr(seq_slots), _ptr(cu_tokens),
                  _ptr(kv_lens), _ptr(token_seq), _ptr(out), _ptr(ws_o), _ptr(ws_ml), N, S, nq, nkv, d, page_size,
                  kv_layer.stride(0), block_table.shape[1], win, float(scale), ns)
        return out

    force_generic_attention = False  # tests flip this to compare the two families of kernels
    force_prefill_form = 0           # tests set 1, 2 or 3 to reach every shape of the prompt-portion workgroups
    force_separate_rope = False      # tests flip this to compare the fused decode step with its two halves
    # measured on MI355X: about one workgroup per CU and at least 8 32-key steps (two per
    # wavefront) per split are best; more splits cost more in partial results than they gain
    DECODE_MIN_STEPS_PER_SPLIT = 8
    DECODE_MIN_STEPS_TO_SPLIT = 32

    PREFILL_MIN_STEPS_PER_SPLIT = 8

    def prefill_splits(self, num_seqs: int, num_kv_heads: int, group: int, head_dim: int, max_q_len: int,
                       max_kv_len: int, window: int) -> int:
        """Key splits of the prompt-portion kernel: 1 unless the portions are short and come after a
        long past, when their row blocks alone leave most of the chip idle.  Only the keys that
        every row sees count (the past; a prompt from an empty cache is never split: measured
        twice as slow at 512 tokens).  A split keeps at least 8 steps of 32 keys while the row
        blocks fill less than half the CUs and 32 otherwise, the splits fill the CUs once, and
        twice where every split still keeps 32 steps, at least two row blocks share the keys of a
        head and the row blocks alone fill at most half the CUs (measured: 128 tokens after 1 k keys 26 -> 20 us with 4 splits, 512 tokens after 16 k
        keys 289 -> 149 us with 4, 512 tokens after 1 k keys best unsplit; row blocks that fill the
        CUs by themselves are never split: 2048 tokens after 2048 keys 115 us unsplit, 151 in two;
        four requests of 32 tokens after 16 k keys 57 us in 8 splits, one workgroup a CU, 70 in 16)."""
        units = self.compute_units()
        rows_per_block = 128 if head_dim <= 128 else 64
        blocks = ((max_q_len * group + rows_per_block - 1) // rows_per_block) * num_kv_heads * max(1, num_seqs)
        past = max_kv_len - max_q_len
        if window:
            past = min(past, window)
        steps = max(0, past) // 32
        by_work = max(1, steps // (self.PREFILL_MIN_STEPS_PER_SPLIT if 2 * blocks < units else 32))
        by_fill = max(1, units // blocks)
        splits = min(by_work, by_fill)
        shared_keys = max_q_len * group >= 2 * rows_per_block  # else the keys' way from memory bounds the launch
        if splits == by_fill and 2 * blocks <= units and shared_keys and steps // (2 * splits) >= 32:
            splits *= 2
        return int(min(splits, 64))

    _compute_units: dict = {}

    def compute_units(self, device=None) -> int:
        """CUs of `device` (the current one if not given), asked once per device."""
        key = device.index if device is not None and device.index is not None else torch.cuda.current_device()
        if key not in self._compute_units:
            self._compute_units[key] = torch.cuda.get_device_properties(key).multi_processor_count
        return self._compute_units[key]

    def prefill_form(self, num_seqs: int, num_kv_heads: int, group: int, head_dim: int, max_q_len: int,
                     max_kv_len: int, window: int, nsplit: int, device) -> int:
        """The shape of the prompt-portion kernel's workgroups:
          1: four wavefronts of one 16-row tile each (64 rows a workgroup),
          2: four wavefronts of two tiles each (128 rows; every operand read from LDS serves both tiles),
          3: eight wavefronts of one tile each (128 rows; four wavefronts a SIMD; heads of 128 only).
        The low form when its workgroups all fit the chip at once (a short portion; at heads of 128
        at most one workgroup a CU, or one prompt from an empty cache); else the tall ones, which share a pass over the keys between more
        rows: form 3 at heads of 128, form 2 below.  Measured on MI355X at heads of 128 (forms 1 / 2 / 3): 2048 tokens from an empty cache
        60 / 65 / 57 us, 2048 tokens after 2048 keys 148 / 128 / 118 us, 49 tokens after 2048 keys
        17 / 21 / 19 us."""
        if head_dim > 128:
            return 1
        if self.force_prefill_form:
            return self.force_prefill_form if head_dim == 128 or self.force_prefill_form < 3 else 2
        resident = 2 * self.compute_units(device)
        rows = max_q_len * group
        low = -(-rows // 64) * num_kv_heads * max(1, num_seqs) * max(1, nsplit)
        if head_dim == 128:
            # (measured: a launch of at most one low workgroup a CU is about 1 us, up to 10 %, faster in
            # the low form, whatever its past and however many requests; so is one prompt from an empty
            # cache while the low form fits the chip at once; else form 3 wins by 5-15 %)
            units = resident // 2
            return 1 if low <= units or (low <= resident and max_kv_len <= max_q_len and num_seqs <= 1) else 3
        return 1 if low <= resident else 2

    def f32_attention_splits(self, num_seqs: int, num_kv_heads: int, row_blocks: int, max_q_len: int,
                             max_kv_len: int, window: int) -> int:
        """Key splits of the float32 matrix-core kernel: enough workgroups for one round of the CUs
        (measured: more cost 10 % at batch 8 and at 512-token portions), at least 4 of its 16-key
        steps each (measured at 512 keys: batch 1 in 2 / 8 splits 20 / 12 us, batch 8 in 2 / 4 splits
        22 / 18 us)."""
        span = min(max_kv_len, window + max_q_len) if window else max_kv_len
        steps = (span + 15) // 16
        by_work = max(1, steps // 4)
        by_fill = max(1, self.compute_units() // max(1, num_seqs * num_kv_heads * row_blocks))
        return int(min(by_work, by_fill, 64))

    def decode_splits(self, num_seqs: int, num_kv_heads: int, max_kv_len: int, window: int) -> int:
        """Key splits of the decode kernel: enough workgroups to fill the chip, but
        at least DECODE_MIN_STEPS_PER_SPLIT 32-key steps each, and none below DECODE_MIN_STEPS_TO_SPLIT steps: the merge
        that splits need is a launch of its own and costs what those steps take (measured at 512 keys:
        batch 16 unsplit 12.1 us, in two 14.2; batch 1 the same either way)."""
        span = min(max_kv_len, window + 32) if window else max_kv_len
        steps = (span + 31) // 32 + (1 if window else 0)
        by_work = max(1, steps // self.DECODE_MIN_STEPS_PER_SPLIT) if steps >= self.DECODE_MIN_STEPS_TO_SPLIT else 1
        by_fill = max(1, self.compute_units() // max(1, num_seqs * num_kv_heads))
        return int(min(by_work, by_fill, 64))

    def add_bias(self, x, bias) -> torch.Tensor:
        """x [M, N] += bias [N], in place (the sum in 32-bit); returns x."""
        _dev(x, "x")
        _dev(bias, "bias")
        _need(x.dim() == 2 and bias.shape == (x.shape[1],), f"bias {list(bias.shape)} does not fit x {list(x.shape)}")
        self._run("elementwise", "lle_add_bias", [_P, _P, _I, _I, _I, _I, _P], _ptr(x), _ptr(bias), x.shape[0],
                  x.shape[1], dtype_code(x.dtype), dtype_code(bias.dtype))
        return x

    # -- feed-forward --------------------------------------------------------------
    def silu_mul(self, gate_up) -> torch.Tensor:
        """gate_up [N, 2 I] (gate columns first) -> silu(gate) * up, [N, I]."""
        _dev(gate_up, "gate_up")
        N, two_i = gate_up.shape
        _need(two_i % 2 == 0, "gate_up must have an even width")
        out = torch.empty((N, two_i // 2), dtype=gate_up.dtype, device=gate_up.device)
        self._run("elementwise", "lle_silu_mul", [_P, _P, _I, _I, _I, _P],
                  _ptr(gate_up), _ptr(out), N, two_i // 2, dtype_code(gate_up.dtype))
        return out

    def gate_up_silu(self, x, weight) -> torch.Tensor:
        """x [M, K], weight [2 I, K] (gate rows, then up rows) -> silu(x gate^T) * (x up^T), [M, I].
        Few bfloat16 rows run as ONE weight-streaming launch with the activation in its
        epilogue; otherwise the product and silu_mul."""
        if isinstance(x, Prenormed):
            return self._linear_folded(x, weight, None, gated=True)
        _dev(x, "x")
        _dev(weight, "weight", x.dtype)
        M, K = x.shape
        N2 = weight.shape[0]
        _need(weight.shape[1] == K and N2 % 2 == 0, f"weight {list(weight.shape)} does not fit x [{M}, {K}]")
        few = M <= self.tuning.skinny_max_rows or (M <= 32 and N2 * K <= self.tuning.skinny_small_weight)
        if x.dtype == torch.bfloat16 and few and K % 8 == 0 and not self.force_library_gemm:
            out = torch.empty((M, N2 // 2), dtype=x.dtype, device=x.device)
            self._run("gemm", "lle_gemm_skinny_gated_bf16", [_P, _P, _P, _I, _I, _I, _P],
                      _ptr(x), _ptr(weight), _ptr(out), M, N2, K)
            return out
        return self.silu_mul(self.linear(x, weight))

    def gate_up_clamped(self, x, weight, bias, limit: float) -> torch.Tensor:
        """x [M, K], weight [2 I, K] (gate rows, then up rows), bias [2 I] or None -> [M, I]: with g = min(x gate^T + b,
        limit) and u = clamp(x up^T + b, -limit, limit) the result is g sigmoid(1.702 g) (u + 1).  Few bfloat16 rows run as
        ONE weight-streaming launch with the activation in its epilogue; otherwise the product and bias_act."""
        _dev(x, "x")
        _dev(weight, "weight", x.dtype)
        M, K = x.shape
        N2 = weight.shape[0]
        _need(weight.shape[1] == K and N2 % 2 == 0, f"weight {list(weight.shape)} does not fit x [{M}, {K}]")
        if bias is not None:
            _dev(bias, "bias", x.dtype)
            _need(bias.shape == (N2,), "bias must cover the whole weight")
        few = M <= self.tuning.skinny_max_rows or (M <= 32 and N2 * K <= self.tuning.skinny_small_weight)
        if x.dtype == torch.bfloat16 and few and K % 8 == 0 and not self.force_library_gemm:
            _need(limit > 0.0, "a clamped activation has a positive limit")
            out = torch.empty((M, N2 // 2), dtype=x.dtype, device=x.device)
            self._run("gemm", "lle_gemm_skinny_clamped_bf16", [_P, _P, _P, _F, _P, _I, _I, _I, _P],
                      _ptr(x), _ptr(weight), _ptr(bias), float(limit), _ptr(out), M, N2, K)
            return out
        return self.bias_act(self.linear(x, weight), "clamp", True, bias=bias, limit=limit)

    # -- arrangements that norm a sublayer's output ------------------------------------
    def cast(self, x, dtype) -> torch.Tensor:
        """x in `dtype` (x itself where it has that type already)."""
        if x.dtype == dtype:
            return x
        _dev(x, "x")
        out = torch.empty(x.shape, dtype=dtype, device=x.device)
        self._run("elementwise", "lle_cast", [_P, _P, _L, _I, _I, _P], _ptr(x), _ptr(out), x.numel(),
                  dtype_code(x.dtype), dtype_code(dtype))
        return out

    def scale_(self, x, factor: float) -> torch.Tensor:
        """float32 x *= factor, in place."""
        _dev(x, "x", torch.float32)
        self._run("elementwise", "lle_scale", [_P, _L, _F, _P], _ptr(x), x.numel(), float(factor))
        return x

    def rmsnorm_add(self, hidden, y, weight, eps: float, out_dtype, extra=None) -> torch.Tensor:
        """hidden float32 [N, H] += RMSNorm(y [+ extra]) * weight, in place and in 32-bit; returns the new
        rows in `out_dtype` (`hidden` itself for float32).  `y`, `extra`: [N, H], float32 or bfloat16 each."""
        _dev(hidden, "hidden", torch.float32)
        _dev(weight, "norm weight")
        N, H = hidden.shape
        _need(weight.shape == (H,), f"norm weight must be [{H}], is {list(weight.shape)}")
        for t, name in ((y, "y"), (extra, "extra")):
            if t is not None:
                _dev(t, name)
                _need(t.shape == hidden.shape, f"{name} must have the shape of hidden")
        out = None if out_dtype == torch.float32 else torch.empty((N, H), dtype=out_dtype, device=hidden.device)
        self._run("norm", "lle_rmsnorm_add", [_P, _P, _I, _P, _I, _P, _I, _P, _I, _I, _F, _I, _P],
                  _ptr(hidden), _ptr(y), dtype_code(y.dtype), _ptr(extra), dtype_code(extra.dtype) if extra is not None else 0,
                  _ptr(weight), dtype_code(weight.dtype), _ptr(out), N, H, float(eps), dtype_code(out_dtype))
        return hidden if out is None else out

    # -- gated recurrence -------------------------------------------------------------
    MINGRU_PIECE = 16  # tokens of one request that one thread walks before the walk is cut into pieces

    def mingru_scan(self, zxg, z_bias, x_bias, state, seq_slots, cu_tokens, out_dtype, max_q_len: int = 0):
        """zxg [N, 3 W] (update-gate, candidate and output-gate inputs side by side; float32 or bfloat16),
        biases float32 [W], state float32 [slots + 1, W] (read and advanced per request) -> [N, W] in
        `out_dtype`: S <- (1 - z) S + z c per token, out = S * silu(gate).  `max_q_len` (a host-side
        bound of the longest request of the step) only decides into how many pieces a walk is cut."""
        _dev(zxg, "zxg")
        _dev(z_bias, "z_bias", torch.float32)
        _dev(x_bias, "x_bias", torch.float32)
        _dev(state, "state", torch.float32)
        _dev(seq_slots, "seq_slots", torch.int32)
        _dev(cu_tokens, "cu_tokens", torch.int32)
        W = z_bias.shape[0]
        N, S = zxg.shape[0], seq_slots.shape[0]
        _need(zxg.shape == (N, 3 * W) and x_bias.shape == (W,), "zxg must be [N, 3 W] and the biases [W]")
        _need(state.dim() == 2 and state.shape[1] == W, "state must be [slots, W]")
        _need(cu_tokens.shape == (S + 1,), "cu_tokens must be [S + 1]")
        out = torch.empty((N, W), dtype=out_dtype, device=zxg.device)
        pieces = max(1, min(1024, -(-max(1, max_q_len) // self.MINGRU_PIECE)))
        part = torch.empty((S * pieces * 3 * W,), dtype=torch.float32, device=zxg.device) if pieces > 1 else None
        self._run("recurrent", "lle_mingru_scan", [_P, _I, _P, _P, _P, _P, _P, _P, _I, _P, _I, _I, _I, _P],
                  _ptr(zxg), dtype_code(zxg.dtype), _ptr(z_bias), _ptr(x_bias), _ptr(state), _ptr(seq_slots),
                  _ptr(cu_tokens), _ptr(out), dtype_code(out_dtype), _ptr(part), S, W, pieces)
        return out

    # -- latent attention -------------------------------------------------------------
    def latent_kv_write(self, dkv, norm_w, eps: float, cos_sin, rot_dims: int, slots, pages, page_size: int,
                        rank: int, rot: int) -> None:
        """dkv [N, rank + rot] -> the pages: c = RMSNorm(first rank) * norm_w and the rest with its first
        `rot_dims` elements rotated in neighbouring pairs by cos_sin [N, rot_dims / 2, 2].  A page
        (one row of `pages`) is the latents [page_size][rank], the same transposed [rank][page_size],
        then the rotated parts [page_size][rot]; slots[n] < 0 writes nothing."""
        _dev(dkv, "dkv")
        _dev(norm_w, "latent norm weight")
        _dev(slots, "slots", torch.int32)
        N = dkv.shape[0]
        _need(dkv.shape == (N, rank + rot) and norm_w.shape == (rank,) and slots.shape == (N,), "dkv [N, rank + rot]")
        _need(pages.is_cuda and pages.dtype == dkv.dtype and pages.dim() == 2 and pages.stride(1) == 1
              and pages.shape[1] >= page_size * (2 * rank + rot), "pages must be [pages, page_size * (2 rank + rot)]")
        if rot_dims:
            _dev(cos_sin, "cos_sin", torch.float32)
            _need(cos_sin.shape == (N, rot_dims // 2, 2), "cos_sin must be [N, rot_dims / 2, 2]")
        self._run("latent", "lle_latent_kv_write", [_P, _P, _I, _F, _P, _I, _P, _P, _L, _I, _I, _I, _I, _I, _P],
                  _ptr(dkv), _ptr(norm_w), dtype_code(norm_w.dtype), float(eps), _ptr(cos_sin) if rot_dims else None,
                  int(rot_dims), _ptr(slots), _ptr(pages), pages.stride(0), int(page_size), N, rank, rot,
                  dtype_code(dkv.dtype))

    def latent_q_rope(self, q, cos_sin, rot_dims: int, heads: int, dim: int, rot: int) -> torch.Tensor:
        """q [N, heads * (dim + rot)] -> the last `rot` elements of every head, rotated, float32 [N, heads, rot]."""
        _dev(q, "q")
        N = q.shape[0]
        _need(q.shape == (N, heads * (dim + rot)), "q must be [N, heads * (dim + rot)]")
        if rot_dims:
            _dev(cos_sin, "cos_sin", torch.float32)
            _need(cos_sin.shape == (N, rot_dims // 2, 2), "cos_sin must be [N, rot_dims / 2, 2]")
        out = torch.empty((N, heads, rot), dtype=torch.float32, device=q.device)
        self._run("latent", "lle_latent_q_rope", [_P, _P, _I, _P, _I, _I, _I, _I, _I, _P],
                  _ptr(q), _ptr(cos_sin) if rot_dims else None, int(rot_dims), _ptr(out), N, heads, dim, rot,
                  dtype_code(q.dtype))
        return out

    def heads_linear(self, x, heads: int, col0: int, K: int, weight, out_dtype) -> torch.Tensor:
        """x [N, heads * xw] (or [N, heads, xw]) and weight [heads, out, K]: for every head the columns
        col0 .. col0 + K of its part times weight[h]^T -> [N, heads, out].  bfloat16: one batched
        library product (32-bit accumulation, either result type); float32: the true 32-bit kernels, head by head."""
        _dev(x, "x")
        _dev(weight, "weight", x.dtype)
        N = x.shape[0]
        x3 = x.view(N, heads, -1)
        xw, O = x3.shape[2], weight.shape[1]
        _need(weight.shape == (heads, O, K) and 0 <= col0 and col0 + K <= xw, "weight must be [heads, out, K]")
        if x.dtype == torch.bfloat16:
            a = x3[:, :, col0 : col0 + K].transpose(0, 1)  # [heads, N, K]
            b = weight.transpose(1, 2)  # [heads, K, out]
            y = torch.bmm(a, b) if out_dtype == torch.bfloat16 else torch.bmm(a, b, out_dtype=out_dtype)
            return y.transpose(0, 1)  # [N, heads, out], strided
        _need(out_dtype == torch.float32, "a float32 product has a float32 result")
        out = torch.empty((N, heads, O), dtype=torch.float32, device=x.device)
        quick = K % 4 == 0 and xw % 4 == 0 and col0 % 4 == 0 and not self.force_simt_gemm
        for h in range(heads):
            a_ptr = x.data_ptr() + 4 * (h * xw + col0)
            b_ptr = weight.data_ptr() + 4 * h * O * K
            c_ptr = out.data_ptr() + 4 * h * O
            if quick:
                self._run("gemm", "lle_gemm_nt_mfma_f32", [_P, _P, _P, _I, _I, _I, _L, _L, _L, _P],
                          a_ptr, b_ptr, c_ptr, N, O, K, heads * xw, K, heads * O)
            else:
                self._run("gemm", "lle_gemm_nt_simt", [_P, _P, _P, _I, _I, _I, _L, _L, _L, _I, _I, _P],
                          a_ptr, b_ptr, c_ptr, N, O, K, heads * xw, K, heads * O, F32, F32)
        return out

    LATENT_GROUPS_PER_CU = 1
    force_generic_latent = False  # tests flip this to compare the two kernels
    last_latent_kernel = None  # (which kernel, key ranges) of the last latent_attention call: for tests

    def latent_query_dtype(self, cache_dtype, page_size: int, rank: int, rot: int):
        """The type in which latent_attention wants q_lat: the cache's where the matrix-core kernel takes the
        sizes (bfloat16, rank a multiple of 16 up to 512, rot a multiple of 8 up to 64, pages of a multiple of
        16 tokens), float32 otherwise."""
        mfma = (cache_dtype == torch.bfloat16 and rank % 16 == 0 and rank <= 512 and rot % 8 == 0 and rot <= 64
                and page_size % 16 == 0 and not self.force_generic_latent)
        return torch.bfloat16 if mfma else torch.float32

    def latent_row_tiles(self, heads: int, max_q_len: int) -> int:
        """16-row tiles per workgroup of the matrix-core kernel: two for prompt portions (a step's operands then
        serve 32 rows: measured at rank 512, 2048 tokens, 388 -> 325 us at 16 heads and 758 -> 629 us at 32), one for
        decoded tokens (two cost a wavefront a SIMD and 2 us of 22 at 32 heads)."""
        return self.force_latent_row_tiles or (2 if max_q_len >= 4 and max_q_len * heads >= 64 else 1)

    force_latent_row_tiles = 0  # tests set 1 or 2

    def latent_splits(self, num_seqs: int, heads: int, max_q_len: int, max_kv_len: int, window: int) -> int:
        """Key ranges per 16-row tile of the matrix-core kernel: enough workgroups (of four wavefronts) for
        LATENT_GROUPS_PER_CU on every CU, at least two 64-key steps each, at most 64."""
        tiles = max(1, num_seqs) * -(-max(1, max_q_len) * heads // (16 * self.latent_row_tiles(heads, max_q_len)))
        span = min(max_kv_len, window + max_q_len) if window else max_kv_len
        steps = -(-max(1, span) // 64)
        return int(max(1, min(-(-self.LATENT_GROUPS_PER_CU * self.compute_units() // tiles), steps // 2, 64)))

    def latent_attention(self, q_lat, q_rot, pages, page_size: int, rank: int, rot: int, block_table, seq_slots,
                         cu_tokens, kv_lens, token_seq, sink, window: Optional[int], scale: float, max_q_len: int,
                         max_kv_len: int, out_dtype) -> torch.Tensor:
        """All heads of every token against the cached latents: q_lat [N, H, rank] (float32 or the
        cache's type; any strides over N and H), q_rot float32 [N, H, rot], sink float32 [H] (None: an ordinary
        softmax, nothing but the keys in its sum) ->
        sum_j p_j c_j, [N, H, rank] in the cache's type.  `max_q_len` and `max_kv_len` are host-side
        bounds; they choose kernels, never results."""
        _dev(q_rot, "q_rot", torch.float32)
        if sink is not None:
            _dev(sink, "sink", torch.float32)
        for t, name in ((block_table, "block_table"), (seq_slots, "seq_slots"), (cu_tokens, "cu_tokens"),
                        (kv_lens, "kv_lens"), (token_seq, "token_seq")):
            _dev(t, name, torch.int32)
        N, H, _ = q_lat.shape
        S = seq_slots.shape[0]
        _need(q_lat.is_cuda and q_lat.shape == (N, H, rank) and q_lat.stride(2) == 1, "q_lat must be [N, H, rank]")
        _need(q_lat.dtype in (torch.float32, pages.dtype), "q_lat is float32 or of the cache's type")
        _need(q_rot.shape == (N, H, rot) and (sink is None or sink.shape == (H,)), "q_rot [N, H, rot], sink [H]")
        _need(pages.is_cuda and pages.dim() == 2 and pages.stride(1) == 1 and pages.dtype == out_dtype
              and pages.shape[1] >= page_size * (2 * rank + rot), "pages must be [pages, page_size * (2 rank + rot)]")
        _need(token_seq.shape == (N,) and cu_tokens.shape == (S + 1,) and kv_lens.shape == (S,), "the step's arrays")
        _need(block_table.dim() == 2, "block_table must be [slots, pages]")
        _need(rank <= 1024, f"a latent of {rank} elements is wider than the attention kernels take (1024)")
        out = torch.empty((N, H, rank), dtype=out_dtype, device=pages.device)
        win = int(window) if window else 0
        if (q_lat.dtype == torch.bfloat16 and self.latent_query_dtype(pages.dtype, page_size, rank, rot) == torch.bfloat16
                and q_lat.stride(0) % 8 == 0 and q_lat.stride(1) % 8 == 0 and pages.stride(0) % 8 == 0
                and max_q_len > 0 and max_kv_len > 0):
            ns = self.latent_splits(S, H, max_q_len, max_kv_len, win)
            rt = self.latent_row_tiles(H, max_q_len)
            self.last_latent_kernel = ("matrix cores", ns)
            ws_o = ws_ml = None
            if ns > 1:
                ws_o = torch.empty((N * H * ns * rank,), dtype=torch.float32, device=pages.device)
                ws_ml = torch.empty((N * H * ns * 2,), dtype=torch.float32, device=pages.device)
            self._run("latent", "lle_latent_attention_mfma",
                      [_P, _L, _L, _P, _P, _L, _I, _I, _I, _P, _I, _P, _P, _P, _P, _I, _F, _P, _P, _P, _I, _I, _I, _I, _I, _I,
                       _P],
                      _ptr(q_lat), q_lat.stride(0), q_lat.stride(1), _ptr(q_rot), _ptr(pages), pages.stride(0),
                      int(page_size), rank, rot, _ptr(block_table), block_table.shape[1], _ptr(seq_slots),
                      _ptr(cu_tokens), _ptr(kv_lens), _ptr(sink), win, float(scale), _ptr(out), _ptr(ws_o), _ptr(ws_ml),
                      N, S, H, -(-max_q_len * H // (16 * rt)), ns, rt)
            return out
        self.last_latent_kernel = ("generic", 1)
        self._run("latent", "lle_latent_attention_generic",
                  [_P, _I, _L, _L, _P, _P, _L, _I, _I, _I, _P, _I, _P, _P, _P, _P, _P, _I, _F, _P, _I, _I, _I, _P],
                  _ptr(q_lat), dtype_code(q_lat.dtype), q_lat.stride(0), q_lat.stride(1), _ptr(q_rot), _ptr(pages),
                  pages.stride(0), int(page_size), rank, rot, _ptr(block_table), block_table.shape[1], _ptr(seq_slots),
                  _ptr(cu_tokens), _ptr(kv_lens), _ptr(token_seq), _ptr(sink), int(window) if window else 0,
                  float(scale), _ptr(out), N, H, dtype_code(out_dtype))
        return out

    # -- routed feed-forward ----------------------------------------------------------
    def moe_route(self, logits, bias, top: int, score: str = "softmax_chosen", experts: Optional[int] = None):
        """float32 logits [N, >= E] (+ bias [E], or None) -> (int32 ids [N, top] of the largest among the first
        E = `experts` columns (default: all), the lower index first among equals; float32 gains [N, top]).
        `score`: "softmax_chosen": the softmax over the chosen alone; "sigmoid": the sigmoid of every chosen
        value, as it is."""
        _dev(logits, "router logits", torch.float32)
        N, cols = logits.shape
        E = cols if experts is None else int(experts)
        _need(0 < E <= cols and 0 < top <= min(E, 32), "a router picks between 1 and 32 of its experts")
        _need(score in ("softmax_chosen", "sigmoid"), f"unknown router score {score!r}")
        if bias is not None:
            _dev(bias, "router bias", torch.float32)
            _need(bias.shape == (E,), "the router's bias must be [E]")
        ids = torch.empty((N, top), dtype=torch.int32, device=logits.device)
        gains = torch.empty((N, top), dtype=torch.float32, device=logits.device)
        self._run("moe", "lle_moe_route", [_P, _P, _P, _P, _I, _I, _I, _I, _I, _P], _ptr(logits), _ptr(bias), _ptr(ids),
                  _ptr(gains), N, E, top, cols, 1 if score == "sigmoid" else 0)
        return ids, gains

    def moe_route_grouped(self, logits, correction, top: int, groups: int = 1, keep: int = 1, score: str = "softmax",
                          group_top: int = 1):
        """float32 logits [N, E] -> (int32 ids [N, top], float32 gains [N, top]).  Scores are the softmax over
        all E (`score` "sigmoid": every logit's own sigmoid); the choice is made on score + correction [E] (None:
        on the scores), among the experts of the `keep` of `groups` equal groups of neighbours whose `group_top`
        largest choice scores add up to most (the lower index wins a tie); gains are the chosen scores, without
        the correction, divided by their sum (+ 1e-20)."""
        _dev(logits, "router logits", torch.float32)
        N, E = logits.shape
        if correction is not None:
            _dev(correction, "router correction", torch.float32)
            _need(correction.shape == (E,), "the router's correction must be [E]")
        _need(score in ("softmax", "sigmoid") and group_top >= 1, f"unknown router score {score!r}")
        _need(0 < top <= min(E, 32), "a router picks between 1 and 32 of its experts")
        _need(groups > 0 and E % groups == 0 and 0 < keep <= groups and top <= keep * (E // groups),
              "the experts form equal groups, and the kept groups hold at least `top` experts")
        _need(2 * E + groups <= 4096, "the router's kernel keeps its scores in LDS: at most about 2000 experts")
        ids = torch.empty((N, top), dtype=torch.int32, device=logits.device)
        gains = torch.empty((N, top), dtype=torch.float32, device=logits.device)
        self._run("moe", "lle_moe_route_grouped", [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P], _ptr(logits),
                  _ptr(correction), _ptr(ids), _ptr(gains), N, E, top, int(groups), int(keep),
                  1 if score == "sigmoid" else 0, int(group_top))
        return ids, gains

    MOE_TILED_MIN_PAIRS = 129  # (token, choice) pairs from which the sorted, tiled kernels take a bfloat16 step

    EXPERT_FORMS = {"gated_silu": 0, "relu2": 1, "gated_clamp": 2}

    def moe_experts(self, x, ids, gains, gate_up, down, form: str = "gated_silu", gain_on_input: bool = False,
                    limit: float = 0.0) -> torch.Tensor:
        """x [N, K]; ids, gains [N, top]; gate_up [E, 2 F, K] (gate rows, then up rows); down [E, H, F] ->
        float32 [N, H]: sum_k gains[n, k] * down[e] (silu(gate[e] x) * (up[e] x)), e = ids[n, k].  An id from E on
        names an identity expert, whose result is x itself (then H = K).
        `form` "relu2": experts without a gate, down[e] relu(up[e] x)^2, `gate_up` is up [E, F, K].
        `form` "gated_clamp": g = min(gate[e] x, limit), u = clamp(up[e] x, -limit, limit), down[e] (g sigmoid(1.702 g) (u + 1)).
        `gain_on_input`: the result is sum_k expert_e(gains[n, k] * x) instead; the gain is applied to the first
        products' results, in 32-bit, before the activation.
        Few pairs, or float32: every pair streams its expert's rows.  Many bfloat16 pairs: sorted by expert
        on the device, then tiles of 128 pairs of one expert on the matrix cores."""
        _dev(x, "x")
        _dev(ids, "ids", torch.int32)
        _dev(gains, "gains", torch.float32)
        _dev(gate_up, "gate_up", x.dtype)
        _dev(down, "down", x.dtype)
        N, K = x.shape
        top = ids.shape[1]
        _need(form in self.EXPERT_FORMS, f"unknown expert form {form!r}")
        _need(form != "gated_clamp" or limit > 0.0, "clamped experts need a positive limit")
        plain = form == "relu2"
        E, F2, _ = gate_up.shape
        H = down.shape[1]
        F = F2 if plain else F2 // 2
        _need(ids.shape == (N, top) and gains.shape == (N, top), "ids and gains must be [N, top]")
        _need(gate_up.shape == (E, F2, K) and (plain or F2 % 2 == 0) and down.shape == (E, H, F), "expert weights do not fit")
        act = torch.empty((N * top, F), dtype=x.dtype, device=x.device)
        out = torch.empty((N, H), dtype=torch.float32, device=x.device)
        code, on_input = self.EXPERT_FORMS[form], (1 if gain_on_input else 0)
        if (x.dtype == torch.bfloat16 and N * top >= self.MOE_TILED_MIN_PAIRS and E <= 256 and K % 8 == 0 and F % 8 == 0
                and H % 4 == 0):
            plan = torch.empty((4 * E + 1,), dtype=torch.int32, device=x.device)
            order = torch.empty((2, N * top), dtype=torch.int32, device=x.device)
            y = torch.empty((N * top, H), dtype=torch.float32, device=x.device)
            self._run("moe", "lle_moe_experts_tiled",
                      [_P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _P],
                      _ptr(x), _ptr(ids), _ptr(gains), _ptr(gate_up), _ptr(down), _ptr(plan), order[0].data_ptr(),
                      order[1].data_ptr(), _ptr(act), _ptr(y), _ptr(out), N, top, E, F, K, H, code, on_input, float(limit))
            return out
        self._run("moe", "lle_moe_experts", [_P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F, _P],
                  _ptr(x), _ptr(ids), _ptr(gains), _ptr(gate_up), _ptr(down), _ptr(act), _ptr(out), N, top, E, F,
                  K, H, dtype_code(x.dtype), code, on_input, float(limit))
        return out

    # -- projections normed as a whole, sinks' attention gates -------------------------------
    def proj_norm_rope_write(self, qkv, bias, slots, q_weight, k_weight, cos_sin, rotary_dim: int, eps: float, kv_layer,
                             num_q_heads: int, num_kv_heads: int, dim: int, vdim: int, has_kv: bool = True,
                             write_kv: bool = True, per_head: bool = False) -> torch.Tensor:
        """A row of qkv holds q [nq dim], then (`has_kv`) k [nkv dim] and v [nkv vdim], then columns that are
        left alone; `bias` (or None) covers the whole row.  q and k are divided by the root mean square of their
        whole projection (`per_head`: every head by its own), times q_weight [nq dim] / k_weight [nkv dim] (None:
        times one), then the first `rotary_dim` elements of
        every head are rotated (half-split) by cos_sin [N, rotary_dim / 2, 2].  Returns q [N, nq, D] with
        D = kv_layer.shape[4] >= max(dim, vdim), zeros past dim; K and V^T go to the pages `kv_layer`
        [pages, 2, nkv, page_size, D] at `slots` [N] with zeros past dim and vdim."""
        _dev(qkv, "qkv")
        _dev(slots, "slots", torch.int32)
        _dev(kv_layer, "kv_layer", qkv.dtype)
        nq, nkv = num_q_heads, num_kv_heads
        N, cols = qkv.shape
        need = nq * dim + (nkv * (dim + vdim) if has_kv else 0)
        _need(cols >= need, "qkv has too few columns")
        _need(slots.shape == (N,), "slots must be [N]")
        _need(kv_layer.dim() == 5 and kv_layer.shape[1] == 2 and kv_layer.shape[2] == nkv, "kv_layer must be [pages, 2, nkv, page_size, D]")
        D, page_size = kv_layer.shape[4], kv_layer.shape[3]
        _need(D >= max(dim, vdim), "the cache's heads are smaller than the model's")
        _need(0 <= rotary_dim <= dim and rotary_dim % 2 == 0, "rotary_dim must be even and <= dim")
        if bias is not None:
            _dev(bias, "bias", qkv.dtype)
            _need(bias.shape == (cols,), "bias must cover the whole row")
        if q_weight is not None:
            _dev(q_weight, "q norm weight")
            _need(q_weight.shape == (nq * dim,), f"q norm weight must be [{nq * dim}]")
        if has_kv and k_weight is not None:
            _need(q_weight is not None, "both norms have weights, or neither")
            _dev(k_weight, "k norm weight", q_weight.dtype)
            _need(k_weight.shape == (nkv * dim,), f"k norm weight must be [{nkv * dim}]")
        _need(not per_head or nq + nkv <= 512, "heads normed one by one: at most 512 query and key heads together")
        if rotary_dim > 0:
            _dev(cos_sin, "cos_sin", torch.float32)
            _need(cos_sin.shape == (N, rotary_dim // 2, 2), "cos_sin must be [N, rotary_dim / 2, 2]")
        q_out = torch.empty((N, nq, D), dtype=qkv.dtype, device=qkv.device)
        self._run("rope_kv", "lle_proj_norm_rope_write",
                  [_P, _I, _P, _P, _P, _P, _I, _P, _I, _F, _P, _P, _I, _I, _I, _I, _I, _I, _I, _L, _I, _I, _I, _I, _P],
                  _ptr(qkv), cols, _ptr(bias), _ptr(slots), _ptr(q_weight), _ptr(k_weight) if has_kv else None,
                  dtype_code(q_weight.dtype) if q_weight is not None else F32, _ptr(cos_sin) if rotary_dim > 0 else None,
                  rotary_dim, float(eps), _ptr(q_out), _ptr(kv_layer), N, nq, nkv, dim, vdim, D, page_size,
                  kv_layer.stride(0), 1 if has_kv else 0, 1 if write_kv else 0, 1 if per_head else 0,
                  dtype_code(qkv.dtype))
        return q_out

    def head_gate(self, a, gates, col0: int, heads: int, vdim: int) -> torch.Tensor:
        """a [N, heads * D], D >= vdim -> [N, heads * vdim]: head h's first vdim elements times
        sigmoid(gates[n, col0 + h])."""
        _dev(a, "a")
        _dev(gates, "gates", a.dtype)
        N = a.shape[0]
        _need(a.dim() == 2 and a.shape[1] % heads == 0 and a.shape[1] // heads >= vdim, "a must be [N, heads * D], D >= vdim")
        _need(gates.dim() == 2 and gates.shape[0] == N and 0 <= col0 and col0 + heads <= gates.shape[1], "gates [N, >= col0 + heads]")
        out = torch.empty((N, heads * vdim), dtype=a.dtype, device=a.device)
        self._run("elementwise", "lle_head_gate", [_P, _P, _I, _I, _P, _I, _I, _I, _I, _I, _P], _ptr(a), _ptr(gates),
                  gates.shape[1], int(col0), _ptr(out), N, heads, a.shape[1] // heads, vdim, dtype_code(a.dtype))
        return out

    def tanh_(self, x) -> torch.Tensor:
        """x = tanh(x), in place."""
        _dev(x, "x")
        self._run("elementwise", "lle_tanh", [_P, _L, _I, _P], _ptr(x), x.numel(), dtype_code(x.dtype))
        return x

    def scaled_add_rmsnorm(self, hidden, a, b, mult: float, weight, eps: float, out_dtype, rows=None,
                           mult_b: Optional[float] = None) -> torch.Tensor:
        """hidden float32 [N, H] += mult * a + mult_b * b in 32-bit and in place (`b` may be None; a, b [N, H],
        float32 or bfloat16 each; `mult_b` None: mult), then RMSNorm(hidden) * weight in `out_dtype`.  With `rows` (int32 [R]) only
        those rows are read, row rows[r] gives row r of the result, and `hidden` is left alone."""
        _dev(hidden, "hidden", torch.float32)
        _dev(weight, "norm weight")
        N, H = hidden.shape
        _need(weight.shape == (H,), f"norm weight must be [{H}]")
        for t, name in ((a, "a"), (b, "b")):
            if t is not None:
                _dev(t, name)
                _need(t.shape == hidden.shape, f"{name} must have the shape of hidden")
        R = N
        if rows is not None:
            _dev(rows, "rows", torch.int32)
            R = rows.shape[0]
        out = torch.empty((R, H), dtype=out_dtype, device=hidden.device)
        self._run("norm", "lle_scaled_add_rmsnorm", [_P, _P, _I, _P, _I, _F, _F, _P, _P, _I, _P, _I, _I, _F, _I, _P],
                  _ptr(hidden), _ptr(a), dtype_code(a.dtype), _ptr(b), dtype_code(b.dtype) if b is not None else 0,
                  float(mult), float(mult if mult_b is None else mult_b), _ptr(rows), _ptr(weight), dtype_code(weight.dtype), _ptr(out), R, H, float(eps),
                  dtype_code(out_dtype))
        return out

    # -- recurrence with a matrix state ------------------------------------------------------
    def shift_mix(self, x, state, prev_offset: int, mu, token_seq, cu_tokens, seq_slots) -> torch.Tensor:
        """x [N, W] -> [M, N, W]: out[m, n] = x[n] + (prev - x[n]) * mu[m], prev = x[n - 1], or for the first
        token of a request's portion state[slot, prev_offset : prev_offset + W] (float32; what the step before
        left there).  mu float32 [M, W]."""
        _dev(x, "x")
        _rows(state, "state", torch.float32)
        _dev(mu, "mu", torch.float32)
        for t, name in ((token_seq, "token_seq"), (cu_tokens, "cu_tokens"), (seq_slots, "seq_slots")):
            _dev(t, name, torch.int32)
        N, W = x.shape
        M = mu.shape[0]
        _need(mu.shape == (M, W) and state.dim() == 2 and prev_offset + W <= state.shape[1], "mu [M, W]; the state row holds W saved elements")
        out = torch.empty((M, N, W), dtype=x.dtype, device=x.device)
        self._run("wkv", "lle_shift_mix", [_P, _P, _L, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _P], _ptr(x), _ptr(state),
                  state.stride(0), int(prev_offset), _ptr(mu), _ptr(token_seq), _ptr(cu_tokens), _ptr(seq_slots), _ptr(out),
                  N, W, M, dtype_code(x.dtype))
        return out

    WKV_PIECE = 64  # tokens of one request that are walked in a row before the walk is cut into pieces
    WKV_MAX_DIM = MAX_WKV_HEAD_DIM

    def wkv_scan(self, r, k, v, wraw, w0, u, g, norm_w, eps: float, x, state, heads: int, dim: int, seq_slots,
                 cu_tokens, out_dtype, max_q_len: int = 0) -> torch.Tensor:
        """Per head, with the matrix state S [dim, dim] of the request (float32, `state[slot, : heads dim dim]`):
            o_t = (S + diag(u) k_t v_t^T)^T r_t;   S <- diag(exp(-exp(wraw_t + w0))) S + k_t v_t^T
        and the result [N, heads * dim] in `out_dtype` is o_t / rms(o_t) (per head, eps inside the root)
        * norm_w * silu(g_t).  r, k, v, wraw float32 [N, heads * dim]; w0, u float32 [heads * dim]; g, x in
        `out_dtype`.  The last row of every request's x [N, W] is saved behind the matrix state.
        `max_q_len` (a host-side bound) only decides into how many pieces a walk is cut."""
        HD = heads * dim
        for t, name in ((r, "r"), (k, "k"), (v, "v"), (wraw, "wraw"), (w0, "w0"), (u, "u")):
            _dev(t, name, torch.float32)
        _rows(state, "state", torch.float32)
        _dev(g, "g", out_dtype)
        _dev(x, "x", out_dtype)
        _dev(norm_w, "norm weight")
        _dev(seq_slots, "seq_slots", torch.int32)
        _dev(cu_tokens, "cu_tokens", torch.int32)
        N, W = x.shape
        S = seq_slots.shape[0]
        _need(0 < dim <= self.WKV_MAX_DIM, f"a head of the recurrence holds at most {self.WKV_MAX_DIM} channels")
        for t in (r, k, v, wraw, g):
            _need(t.shape == (N, HD), "r, k, v, wraw and g must be [N, heads * dim]")
        _need(w0.shape == (HD,) and u.shape == (HD,) and norm_w.shape == (HD,), "w0, u and the norm weight must be [heads * dim]")
        _need(state.dim() == 2 and state.shape[1] >= HD * dim + W, "a state row holds heads * dim * dim + W floats")
        _need(cu_tokens.shape == (S + 1,), "cu_tokens must be [S + 1]")
        out = torch.empty((N, HD), dtype=out_dtype, device=x.device)
        piece = self.WKV_PIECE
        pieces = -(-max_q_len // piece) if max_q_len > 2 * piece else 1
        part = None
        if pieces > 1:
            part = torch.empty((S * pieces * heads * (dim * dim + dim),), dtype=torch.float32, device=x.device)
        else:
            piece = 1 << 30
        self._run("wkv", "lle_wkv_scan",
                  [_P, _P, _P, _P, _P, _P, _P, _P, _I, _F, _P, _P, _L, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _P],
                  _ptr(r), _ptr(k), _ptr(v), _ptr(wraw), _ptr(w0), _ptr(u), _ptr(g), _ptr(norm_w),
                  dtype_code(norm_w.dtype), float(eps), _ptr(x), _ptr(state), state.stride(0), HD * dim, _ptr(seq_slots),
                  _ptr(cu_tokens), _ptr(out), S, heads, dim, W, pieces, piece, _ptr(part), dtype_code(out_dtype))
        return out

    # -- what enters the stream between two blocks ------------------------------------------------
    def inject_rmsnorm(self, hidden, delta, vector, again, weight, eps: float, out_dtype, rows=None) -> torch.Tensor:
        """hidden float32 [N, H] += delta + vector + the embedding's rows, in 32-bit and in place, then
        RMSNorm(hidden) * weight in `out_dtype`.  `delta`: [N, H] in either type, PartialSums, a ScaledSum with a
        factor of one, or None (any other delta is added up first); `vector` float32 [H] or None; `again` a
        parts.base.EmbeddedRows or None.  With `rows` (int32 [R]) only those rows are read, row rows[r] gives row r of
        the result, and `hidden` is left alone."""
        _dev(hidden, "hidden", torch.float32)
        _dev(weight, "norm weight")
        N, H = hidden.shape
        _need(weight.shape == (H,), f"norm weight must be [{H}]")
        a, b, slices, stride = delta, None, 1, 0
        if isinstance(delta, PartialSums):
            a = delta.sums
            slices, stride = a.shape[0], a.stride(0)
            _dev(a, "partial sums", torch.float32)
            _need(a.dim() == 3 and a.shape[1:] == hidden.shape, "partial sums must be [slices, N, H]")
        elif isinstance(delta, ScaledSum):
            a, b = delta.a, delta.b
            if delta.mult != 1.0 or (delta.b is not None and delta.mult_b not in (None, 1.0)):
                a, b = delta.total(), None
        elif isinstance(delta, Injected):
            a = delta.total()
        if a is not None and not isinstance(delta, PartialSums):
            for t, name in ((a, "delta"), (b, "delta's second summand")):
                if t is not None:
                    _dev(t, name)
                    _need(t.shape == hidden.shape, f"{name} must have the shape of hidden")
        if vector is not None:
            _dev(vector, "vector", torch.float32)
            _need(vector.shape == (H,), f"vector must be [{H}]")
        ids = table = feedback = token_seq = seq_slots = None
        scale = 1.0
        if again is not None:
            ids, table, scale = again.ids, again.table, float(again.scale)
            feedback, token_seq, seq_slots = again.feedback, again.token_seq, again.seq_slots
            _dev(ids, "ids", torch.int32)
            _dev(table, "embedding table")
            _need(ids.shape == (N,) and table.dim() == 2 and table.shape[1] == H, "the embedding's rows must fit hidden")
            if feedback is not None:
                for t, name in ((feedback, "feedback"), (token_seq, "token_seq"), (seq_slots, "seq_slots")):
                    _need(t is not None, "feedback, token_seq and seq_slots come together")
                    _dev(t, name, torch.int32)
                _need(token_seq.shape == (N,), "token_seq must be [N]")
        R = N
        if rows is not None:
            _dev(rows, "rows", torch.int32)
            R = rows.shape[0]
        out = torch.empty((R, H), dtype=out_dtype, device=hidden.device)
        code = lambda t: 0 if t is None else dtype_code(t.dtype)
        self._run("norm", "lle_inject_rmsnorm",
                  [_P, _P, _I, _I, _L, _P, _I, _P, _P, _P, _I, _F, _P, _P, _P, _P, _P, _I, _P, _I, _I, _F, _I, _P],
                  _ptr(hidden), _ptr(a), code(a), slices, stride, _ptr(b), code(b), _ptr(vector), _ptr(ids), _ptr(table),
                  code(table), scale, _ptr(feedback), _ptr(token_seq) if feedback is not None else None,
                  _ptr(seq_slots) if feedback is not None else None, _ptr(rows), _ptr(weight), dtype_code(weight.dtype),
                  _ptr(out), R, H, float(eps), dtype_code(out_dtype))
        return out

    # -- attention gated element by element, heads' weights mixed ----------------------------------
    def pair_rope_write(self, u, bias, slots, cos_sin, v_cos_sin, kv_layer, num_q_heads: int, num_kv_heads: int, dim: int,
                        vdim: int, write_kv: bool = True) -> torch.Tensor:
        """A row of u holds q [nq dim], k [nkv dim], v [nkv vdim], then columns that are left alone; `bias` (or None)
        covers those three.  The first elements of every q and k head turn in neighbouring pairs by cos_sin
        [N, rot / 2, 2] (None: not), whole values by v_cos_sin [N, vdim / 2, 2] (None: not).  Returns q [N, nq, D] with
        D = kv_layer.shape[4] >= max(dim, vdim), zeros past dim; K and V^T go to the pages `kv_layer`
        [pages, 2, nkv, page_size, D] at `slots` [N] with zeros past dim and vdim."""
        _dev(u, "u")
        _dev(slots, "slots", torch.int32)
        _dev(kv_layer, "kv_layer", u.dtype)
        nq, nkv = num_q_heads, num_kv_heads
        N, cols = u.shape
        used = nq * dim + nkv * (dim + vdim)
        _need(cols >= used, "u has too few columns")
        _need(slots.shape == (N,), "slots must be [N]")
        _need(kv_layer.dim() == 5 and kv_layer.shape[1] == 2 and kv_layer.shape[2] == nkv, "kv_layer must be [pages, 2, nkv, page_size, D]")
        D, page_size = kv_layer.shape[4], kv_layer.shape[3]
        _need(D >= max(dim, vdim) and D % 2 == 0, "the cache's heads are smaller than the model's, or odd")
        if bias is not None:
            _dev(bias, "bias", u.dtype)
            _need(bias.shape == (used,), "bias must cover q, k and v")
        rot = 0
        for t, name, most in ((cos_sin, "cos_sin", dim), (v_cos_sin, "v_cos_sin", vdim)):
            if t is not None:
                _dev(t, name, torch.float32)
                _need(t.dim() == 3 and t.shape[0] == N and t.shape[2] == 2 and 2 * t.shape[1] <= most, f"{name} must be [N, pairs, 2]")
        if cos_sin is not None:
            rot = 2 * cos_sin.shape[1]
        _need(v_cos_sin is None or 2 * v_cos_sin.shape[1] == vdim, "v_cos_sin must cover the whole value")
        q_out = torch.empty((N, nq, D), dtype=u.dtype, device=u.device)
        self._run("rope_kv", "lle_pair_rope_write",
                  [_P, _I, _P, _P, _P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _L, _I, _I, _P],
                  _ptr(u), cols, _ptr(bias), _ptr(slots), _ptr(cos_sin), rot, _ptr(v_cos_sin), _ptr(q_out), _ptr(kv_layer), N,
                  nq, nkv, dim, vdim, D, page_size, kv_layer.stride(0), 1 if write_kv else 0, dtype_code(u.dtype))
        return q_out

    def turn_back_gate(self, a, u, gate_col: int, heads: int, vdim: int, v_cos_sin, out_scale: float = 1.0) -> torch.Tensor:
        """a [N, heads * D], D >= vdim -> [N, heads * vdim]: every head's first vdim elements, turned back in
        neighbouring pairs by v_cos_sin [N, vdim / 2, 2] (None: not), times sigmoid(u[n, gate_col + ...]) element by
        element, times out_scale."""
        _dev(a, "a")
        _dev(u, "u", a.dtype)
        N = a.shape[0]
        _need(a.dim() == 2 and a.shape[1] % heads == 0 and a.shape[1] // heads >= vdim, "a must be [N, heads * D], D >= vdim")
        _need(u.dim() == 2 and u.shape[0] == N and 0 <= gate_col and gate_col + heads * vdim <= u.shape[1], "u [N, >= gate_col + heads * vdim]")
        if v_cos_sin is not None:
            _dev(v_cos_sin, "v_cos_sin", torch.float32)
            _need(v_cos_sin.shape == (N, vdim // 2, 2) and vdim % 2 == 0, "v_cos_sin must cover the whole value")
        out = torch.empty((N, heads * vdim), dtype=a.dtype, device=a.device)
        self._run("rope_kv", "lle_turn_back_gate", [_P, _P, _I, _I, _P, _P, _I, _I, _I, _I, _F, _I, _P], _ptr(a), _ptr(u),
                  u.shape[1], int(gate_col), _ptr(v_cos_sin), _ptr(out), N, heads, a.shape[1] // heads, vdim, float(out_scale),
                  dtype_code(a.dtype))
        return out

    def talking_attention(self, q, kv_layer, block_table, seq_slots, cu_tokens, kv_lens, token_seq, chunk: Optional[int],
                          scale: float, slopes, talk, min_q_len: int = 0, max_q_len: int = 0,
                          max_kv_len: int = 0) -> torch.Tensor:
        """q [N, H, D] against the pages -> [N, H * D].  Position p sees the keys p // chunk * chunk .. p (chunk None:
        all from 0 on); scores (q . k) * scale - slopes[h] * (p - j) (slopes float32 [H] or None), softmax, then the
        heads' weights mixed, w_h <- sum_g talk[h, g] w_g (talk float32 [H, H]), head h on its own key/value head's
        values.  `min_q_len`, `max_q_len` and `max_kv_len` are host-side bounds of this batch; they choose the
        kernels, never the result."""
        _dev(q, "q")
        _dev(kv_layer, "kv_layer", q.dtype)
        for t, name in ((block_table, "block_table"), (seq_slots, "seq_slots"), (cu_tokens, "cu_tokens"),
                        (kv_lens, "kv_lens"), (token_seq, "token_seq")):
            _dev(t, name, torch.int32)
        N, H, D = q.shape
        G, P = kv_layer.shape[2], kv_layer.shape[3]
        _need(kv_layer.dim() == 5 and kv_layer.shape[4] == D and kv_layer.shape[1] == 2, "kv_layer must be [pages, 2, G, page_size, D]")
        _need(H % G == 0, "query heads must be a multiple of key/value heads")
        _need(token_seq.shape == (N,), "token_seq must be [N]")
        S = seq_slots.shape[0]
        _need(cu_tokens.shape == (S + 1,) and kv_lens.shape == (S,), "cu_tokens [S + 1], kv_lens [S]")
        _need(block_table.dim() == 2, "block_table must be [slots, pages]")
        _need(chunk is None or chunk > 0, "a chunk must be positive")
        _dev(talk, "talk", torch.float32)
        _need(talk.shape == (H, H), "talk must be [H, H]")
        if slopes is not None:
            _dev(slopes, "slopes", torch.float32)
            _need(slopes.shape == (H,), "slopes must be [H]")
        out = torch.empty((N, H * D), dtype=q.dtype, device=q.device)
        run_decode, run_prefill = min_q_len <= 1, max_q_len > 1
        if (q.dtype == torch.bfloat16 and D % 32 == 0 and D <= 128 and P % 16 == 0 and max_q_len > 0 and max_kv_len > 0
                and S <= 65535 and (H <= 32 if run_prefill else H <= 128) and not self.force_generic_attention):
            K = splits = 0
            ws_s = ws_ml = None
            if run_decode:
                seen = min(chunk, max_kv_len) if chunk else max_kv_len  # keys that a query sees at most
                K = -(-(seen + 15) // 16) * 16
                # a wavefront should have a tile of 16 keys or two, and the workgroups fill the CUs once or twice
                splits = int(max(1, min(-(-K // 64), 2 * self.compute_units() // max(1, S * G))))
                ws_s = torch.empty((S * H * K,), dtype=torch.float32, device=q.device)
                ws_ml = torch.empty((S * H * (K // 16) * 2,), dtype=torch.float32, device=q.device)
            ws_sums = torch.empty((N * H,), dtype=torch.float32, device=q.device) if run_prefill else None
            # one output head a wavefront: twice the workgroups, which make all scores again; where the tiles leave CUs idle
            out_heads = 1 if -(-max_q_len // 16) * S * 2 <= self.compute_units() else 2
            self._run("talking", "lle_talking_mfma",
                      [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _L, _I, _I, _F, _P, _P, _I, _I, _I, _P, _P, _I, _I, _I,
                       _P, _P],
                      _ptr(q), _ptr(kv_layer), _ptr(block_table), _ptr(seq_slots), _ptr(cu_tokens), _ptr(kv_lens),
                      _ptr(token_seq), _ptr(out), S, H, G, D, P, kv_layer.stride(0), block_table.shape[1], int(chunk or 0),
                      float(scale), _ptr(slopes), _ptr(talk), int(run_decode), splits, K, _ptr(ws_s), _ptr(ws_ml),
                      int(run_prefill), max_q_len, out_heads, _ptr(ws_sums))
            return out
        self._run("talking", "lle_talking_generic",
                  [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _L, _I, _I, _F, _P, _P, _I, _P],
                  _ptr(q), _ptr(kv_layer), _ptr(block_table), _ptr(seq_slots), _ptr(cu_tokens), _ptr(kv_lens), _ptr(token_seq),
                  _ptr(out), N, H, G, D, P, kv_layer.stride(0), block_table.shape[1], int(chunk or 0), float(scale),
                  _ptr(slopes), _ptr(talk), dtype_code(q.dtype))
        return out

    # -- gated linear attention -----------------------------------------------------------------------
    GLA_PIECE = 64  # tokens of one request that are walked in a row before the walk is cut into pieces

    def gla_decay(self, low, a2, bias, tau: float) -> torch.Tensor:
        """sigmoid(low @ a2 + bias)^(1 / tau), all float32: low [N, R], a2 [R, C], bias [C] -> [N, C]."""
        for t, name in ((low, "low"), (a2, "a2"), (bias, "bias")):
            _dev(t, name, torch.float32)
        N, R = low.shape
        C = bias.shape[0]
        _need(a2.shape == (R, C), "a2 must be [R, C]")
        out = torch.empty((N, C), dtype=torch.float32, device=low.device)
        self._run("gla", "lle_gla_decay", [_P, _P, _P, _P, _I, _I, _I, _F, _P], _ptr(low), _ptr(a2), _ptr(bias), _ptr(out), N, R,
                  C, float(tau))
        return out

    def gla_scan(self, u, decay, q_scale: float, norm_w, eps: float, state, heads: int, dim: int, vdim: int, seq_slots,
                 cu_tokens, max_q_len: int = 0) -> torch.Tensor:
        """Per head, with the matrix state S [dim, vdim] of the request (float32, `state[slot, : heads dim vdim]`):
            S <- diag(decay_t) S + k_t v_t^T;   o_t = S^T (q_scale q_t)
        and the result [N, heads * vdim] is o_t / rms(o_t) (per head, eps inside the root) * norm_w [vdim] * silu(g_t).
        A row of u holds q [heads dim], k [heads dim], v [heads vdim], g [heads vdim]; decay float32 [N, heads * dim].
        `max_q_len` (a host-side bound) only decides into how many pieces a walk is cut."""
        _dev(u, "u")
        _dev(decay, "decay", torch.float32)
        _dev(norm_w, "norm weight", torch.float32)
        _rows(state, "state", torch.float32)
        _dev(seq_slots, "seq_slots", torch.int32)
        _dev(cu_tokens, "cu_tokens", torch.int32)
        N, cols = u.shape
        S = seq_slots.shape[0]
        _need(0 < dim <= MAX_GLA_HEAD_DIM and 0 < vdim <= MAX_GLA_HEAD_DIM, f"a head of the recurrence holds at most {MAX_GLA_HEAD_DIM} channels")
        _need(cols >= 2 * heads * (dim + vdim), "u has too few columns")
        _need(decay.shape == (N, heads * dim), "decay must be [N, heads * dim]")
        _need(norm_w.shape == (vdim,), "the norm weight must be [vdim]")
        _need(state.dim() == 2 and state.shape[1] >= heads * dim * vdim, "a state row holds heads * dim * vdim floats")
        _need(cu_tokens.shape == (S + 1,), "cu_tokens must be [S + 1]")
        out = torch.empty((N, heads * vdim), dtype=u.dtype, device=u.device)
        piece = self.GLA_PIECE
        pieces = -(-max_q_len // piece) if max_q_len > 2 * piece else 1
        part = None
        if pieces > 1:
            part = torch.empty((S * pieces * heads * (dim * vdim + dim),), dtype=torch.float32, device=u.device)
        else:
            piece = 1 << 30
        self._run("gla", "lle_gla_scan",
                  [_P, _I, _P, _F, _P, _F, _P, _L, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _P],
                  _ptr(u), cols, _ptr(decay), float(q_scale), _ptr(norm_w), float(eps), _ptr(state), state.stride(0),
                  _ptr(seq_slots), _ptr(cu_tokens), _ptr(out), S, heads, dim, vdim, pieces, piece, _ptr(part),
                  dtype_code(u.dtype))
        return out

    # -- activations, caps, chained norms ---------------------------------------------------------
    ACT_CODES = {"silu": 0, "relu": 1, "relu2": 2, "gelu_tanh": 3, "clamp": 4}

    def bias_act(self, z, kind: str, gated: bool, bias=None, row_gate=None, limit: float = 0.0) -> torch.Tensor:
        """gated: z [N, 2 F] (gate columns first) -> act(gate + b) * (up + b), [N, F]; else z [N, F] -> act(z + b).
        `kind`: silu, relu, relu2 (the square of relu), gelu_tanh (gelu in its tanh form), or, gated only, clamp: with
        g = min(gate + b, limit) and u = clamp(up + b, -limit, limit) the result is g sigmoid(1.702 g) (u + 1); `bias` (or None) covers z's row; `row_gate` = (t, col), t
        float32 [N, any]: row n is multiplied by sigmoid(t[n, col]).  Everything in 32-bit."""
        _dev(z, "z")
        _need(kind in self.ACT_CODES, f"unknown activation {kind!r}")
        N, cols = z.shape
        _need(not gated or cols % 2 == 0, "a gated input has an even width")
        _need(kind != "clamp" or (gated and limit > 0.0), "a clamped activation is gated and has a positive limit")
        F = cols // 2 if gated else cols
        if bias is not None:
            _dev(bias, "bias", z.dtype)
            _need(bias.shape == (cols,), "bias must cover the whole row")
        gate_t, stride, col = None, 0, 0
        if row_gate is not None:
            gate_t, col = row_gate
            _dev(gate_t, "row gate", torch.float32)
            _need(gate_t.dim() == 2 and gate_t.shape[0] == N and 0 <= col < gate_t.shape[1], "row gate [N, > col]")
            stride = gate_t.shape[1]
        out = torch.empty((N, F), dtype=z.dtype, device=z.device)
        self._run("elementwise", "lle_bias_act", [_P, _P, _P, _I, _I, _P, _I, _I, _I, _I, _F, _I, _P], _ptr(z), _ptr(bias),
                  _ptr(gate_t), stride, int(col), _ptr(out), N, F, 1 if gated else 0, self.ACT_CODES[kind],
                  float(limit), dtype_code(z.dtype))
        return out

    def softcap_(self, x, cap: float) -> torch.Tensor:
        """float32 x = cap * tanh(x / cap), in place."""
        _dev(x, "x", torch.float32)
        _need(cap > 0.0, "a cap must be positive")
        self._run("elementwise", "lle_softcap", [_P, _L, _F, _P], _ptr(x), x.numel(), float(cap))
        return x

    def rmsnorm_add_rmsnorm(self, hidden, y, weight, eps: float, next_weight, next_eps: float, out_dtype,
                            extra=None) -> torch.Tensor:
        """hidden float32 [N, H] += RMSNorm(y [+ extra]) * weight, in place and in 32-bit; returns
        RMSNorm(the new hidden) * next_weight in `out_dtype`: the norm after one sublayer and the norm before
        the next in one launch.  `y`, `extra`: [N, H], float32 or bfloat16 each."""
        _dev(hidden, "hidden", torch.float32)
        _dev(weight, "norm weight")
        _dev(next_weight, "next norm weight", weight.dtype)
        N, H = hidden.shape
        _need(weight.shape == (H,) and next_weight.shape == (H,), f"norm weights must be [{H}]")
        for t, name in ((y, "y"), (extra, "extra")):
            if t is not None:
                _dev(t, name)
                _need(t.shape == hidden.shape, f"{name} must have the shape of hidden")
        out = torch.empty((N, H), dtype=out_dtype, device=hidden.device)
        self._run("norm", "lle_rmsnorm_add_rmsnorm", [_P, _P, _I, _P, _I, _P, _P, _I, _P, _I, _I, _F, _F, _I, _P],
                  _ptr(hidden), _ptr(y), dtype_code(y.dtype), _ptr(extra), dtype_code(extra.dtype) if extra is not None else 0,
                  _ptr(weight), _ptr(next_weight), dtype_code(weight.dtype), _ptr(out), N, H, float(eps), float(next_eps),
                  dtype_code(out_dtype))
        return out

    # -- attention behind a short convolution --------------------------------------------------------
    def conv_norm_rope_write(self, u, taps, state, token_seq, cu_tokens, seq_slots, slots, q_weight, k_weight, cos_sin,
                             rotary_dim: int, eps: float, kv_layer, num_q_heads: int, num_kv_heads: int, dim: int,
                             vdim: int, write_kv: bool = True) -> torch.Tensor:
        """A row of u holds q [nq dim], k [nkv dim], v [nkv vdim] of one token.  Every channel is convolved over
        time with its J taps (float32 [cols, J]; the last tap meets the token itself), reading the rows of the
        same request ahead of it in this step and, before those, the request's state row (float32
        [slots + 1, (J - 1) cols], the last J - 1 rows of u that earlier steps brought, oldest first; None for
        J = 1).  Then every head of q and k is divided by its root mean square times q_weight / k_weight
        (float32 [dim], one for all heads), the first `rotary_dim` elements of every head are rotated (half-split)
        by cos_sin [N, rotary_dim / 2, 2].  Returns q [N, nq, D], D = kv_layer.shape[4] >= max(dim, vdim), zeros
        past dim; K and V^T go to the pages at `slots` with zeros past dim and vdim.  The state is left as it
        is: conv_state_update advances it."""
        _dev(u, "u")
        _dev(taps, "taps", torch.float32)
        _dev(slots, "slots", torch.int32)
        _dev(kv_layer, "kv_layer", u.dtype)
        for t, name in ((token_seq, "token_seq"), (cu_tokens, "cu_tokens"), (seq_slots, "seq_slots")):
            _dev(t, name, torch.int32)
        nq, nkv = num_q_heads, num_kv_heads
        N, cols = u.shape
        J = taps.shape[1]
        S = seq_slots.shape[0]
        _need(cols == (nq + nkv) * dim + nkv * vdim, "a row of u holds q, k and v")
        _need(taps.shape == (cols, J) and J >= 1, "taps must be [cols, J]")
        _need(slots.shape == (N,) and token_seq.shape == (N,) and cu_tokens.shape == (S + 1,), "slots, token_seq [N]; cu_tokens [S + 1]")
        _need(kv_layer.dim() == 5 and kv_layer.shape[1] == 2 and kv_layer.shape[2] == nkv, "kv_layer must be [pages, 2, nkv, page_size, D]")
        D, page_size = kv_layer.shape[4], kv_layer.shape[3]
        _need(D >= max(dim, vdim), "the cache's heads are smaller than the model's")
        _need(0 <= rotary_dim <= dim and rotary_dim % 2 == 0, "rotary_dim must be even and <= dim")
        if J > 1:
            _need(state is not None, "a convolution of several taps needs the requests' state rows")
            _rows(state, "state", torch.float32)
            _need(state.shape[1] >= (J - 1) * cols, "a state row holds J - 1 rows of u")
        _dev(q_weight, "q norm weight", torch.float32)
        _dev(k_weight, "k norm weight", torch.float32)
        _need(q_weight.shape == (dim,) and k_weight.shape == (dim,), f"the heads' norm weights must be [{dim}]")
        if rotary_dim > 0:
            _dev(cos_sin, "cos_sin", torch.float32)
            _need(cos_sin.shape == (N, rotary_dim // 2, 2), "cos_sin must be [N, rotary_dim / 2, 2]")
        q_out = torch.empty((N, nq, D), dtype=u.dtype, device=u.device)
        self._run("rope_kv", "lle_conv_norm_rope_write",
                  [_P, _I, _P, _I, _P, _L, _P, _P, _P, _P, _P, _P, _P, _I, _F, _P, _P, _I, _I, _I, _I, _I, _I, _I, _L, _I, _I, _P],
                  _ptr(u), cols, _ptr(taps), J, _ptr(state) if J > 1 else None, state.stride(0) if J > 1 else 0,
                  _ptr(token_seq), _ptr(cu_tokens), _ptr(seq_slots), _ptr(slots), _ptr(q_weight), _ptr(k_weight),
                  _ptr(cos_sin) if rotary_dim > 0 else None, rotary_dim, float(eps), _ptr(q_out), _ptr(kv_layer), N, nq, nkv,
                  dim, vdim, D, page_size, kv_layer.stride(0), 1 if write_kv else 0, dtype_code(u.dtype))
        return q_out

    def conv_state_update(self, u, state, kept: int, cu_tokens, seq_slots) -> None:
        """state row of every request of the step <- the last `kept` rows of (the `kept` rows it held, then the
        request's rows of u in this step); state float32 [slots + 1, >= kept * cols], u [N, cols]."""
        _dev(u, "u")
        _rows(state, "state", torch.float32)
        _dev(cu_tokens, "cu_tokens", torch.int32)
        _dev(seq_slots, "seq_slots", torch.int32)
        N, cols = u.shape
        S = seq_slots.shape[0]
        _need(kept > 0 and state.shape[1] >= kept * cols and cu_tokens.shape == (S + 1,), "a state row holds `kept` rows of u")
        self._run("rope_kv", "lle_conv_state_update", [_P, _I, _P, _L, _I, _P, _P, _I, _I, _P], _ptr(u), cols, _ptr(state),
                  state.stride(0), int(kept), _ptr(cu_tokens), _ptr(seq_slots), S, dtype_code(u.dtype))

    # -- the gated delta rule --------------------------------------------------------------
    DELTA_MAX_DIM = MAX_DELTA_HEAD_DIM
    DELTA_MAX_ADVANCE = 8  # (lle_delta_conv_max_advance)

    def delta_conv(self, u, taps, state, token_seq, cu_tokens, seq_slots, kv_heads: int, dim: int, heads: int, vdim: int,
                   unit_eps: float, q_scale: float, advance: bool = False):
        """A row of u holds q [G dim], k [G dim], v [H vdim] of one token (G = kv_heads, H = heads).  Every channel is
        convolved over time with its J taps (float32 [cols, J]; the last tap meets the token itself), reading the
        rows of the same request ahead of it in this step and, before those, the request's state row (float32
        [slots + 1, >= (J - 1) cols], the last J - 1 rows of u that earlier steps brought, oldest first; None for
        J = 1), then passes silu; every head of q and k becomes x / sqrt(sum x^2 + unit_eps), q times q_scale.
        Returns float32 q [N, G dim], k [N, G dim], v [N, H vdim].  The state is left as it is (conv_state_update
        advances it), or with `advance` moves on in the same launch (see can_advance_conv)."""
        _dev(u, "u")
        _dev(taps, "taps", torch.float32)
        for t, name in ((token_seq, "token_seq"), (cu_tokens, "cu_tokens"), (seq_slots, "seq_slots")):
            _dev(t, name, torch.int32)
        N, cols = u.shape
        J = taps.shape[1]
        S = seq_slots.shape[0]
        G, H = int(kv_heads), int(heads)
        _need(cols == 2 * G * dim + H * vdim, "a row of u holds q, k and v")
        _need(taps.shape == (cols, J) and J >= 1, "taps must be [cols, J]")
        _need(token_seq.shape == (N,) and cu_tokens.shape == (S + 1,), "token_seq [N]; cu_tokens [S + 1]")
        _need(0 < dim <= self.DELTA_MAX_DIM and 0 < vdim <= self.DELTA_MAX_DIM,
              f"a head of the delta rule holds at most {self.DELTA_MAX_DIM} channels")
        if J > 1:
            _need(state is not None, "a convolution of several taps needs the requests' state rows")
            _rows(state, "state", torch.float32)
            _need(state.shape[1] >= (J - 1) * cols, "a state row holds J - 1 rows of u")
        q = torch.empty((N, G * dim), dtype=torch.float32, device=u.device)
        k = torch.empty((N, G * dim), dtype=torch.float32, device=u.device)
        v = torch.empty((N, H * vdim), dtype=torch.float32, device=u.device)
        _need(not advance or (1 < J <= self.DELTA_MAX_ADVANCE and N == S), "the state moves on in this launch for single tokens")
        self._run("delta", "lle_delta_conv", [_P, _I, _P, _I, _P, _L, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _F, _F, _I, _I, _P],
                  _ptr(u), cols, _ptr(taps), J, _ptr(state) if J > 1 else None, state.stride(0) if J > 1 else 0,
                  _ptr(token_seq), _ptr(cu_tokens), _ptr(seq_slots), _ptr(q), _ptr(k), _ptr(v), N, G, dim, H, vdim,
                  float(unit_eps), float(q_scale), int(advance), dtype_code(u.dtype))
        return q, k, v

    def can_advance_conv(self, taps: int, max_q_len: int) -> bool:
        """Whether delta_conv can move the kept rows on itself: a step of single tokens, few taps."""
        return max_q_len == 1 and 1 < taps <= self.DELTA_MAX_ADVANCE

    def low_rank_gates(self, low, a_col: int, a2, a_log, dt_bias, dim: int, g_col: int = 0, g2=None):
        """low float32 [N, cols], a2 float32 [CA, RA], a_log float32 [CA / dim], dt_bias float32 [CA] ->
        decay float32 [N, CA]: exp(-exp(a_log[c // dim]) softplus(low[:, a_col : a_col + RA] @ a2[c] + dt_bias[c])); and with
        g2 [CG, RG] gate float32 [N, CG] = low[:, g_col : g_col + RG] @ g2^T (else None).  RA and RG are multiples of 16 (pad
        weights and columns with zeros), columns start at multiples of 4."""
        for t, name in ((low, "low"), (a2, "a2"), (a_log, "a_log"), (dt_bias, "dt_bias")):
            _dev(t, name, torch.float32)
        N, cols = low.shape
        CA, RA = a2.shape
        CG, RG = (0, 0) if g2 is None else g2.shape
        if g2 is not None:
            _dev(g2, "g2", torch.float32)
        _need(CA % dim == 0 and a_log.shape == (CA // dim,) and dt_bias.shape == (CA,), "a2 [heads * dim, R], a_log [heads], dt_bias [heads * dim]")
        _need(RA % 16 == 0 and RG % 16 == 0 and cols % 4 == 0 and a_col % 4 == 0 and g_col % 4 == 0, "ranks are multiples of 16, columns start at multiples of 4")
        _need(0 <= a_col and a_col + RA <= cols and 0 <= g_col and g_col + RG <= cols, "low has too few columns")
        decay = torch.empty((N, CA), dtype=torch.float32, device=low.device)
        gate = torch.empty((N, CG), dtype=torch.float32, device=low.device) if g2 is not None else None
        self._run("delta", "lle_low_rank_gates", [_P, _I, _I, _I, _P, _I, _I, _P, _I, _I, _P, _P, _I, _P, _P, _I, _P],
                  _ptr(low), cols, int(a_col), int(g_col), _ptr(a2), RA, CA, _ptr(g2), RG, CG, _ptr(a_log), _ptr(dt_bias), int(dim),
                  _ptr(decay), _ptr(gate), N)
        return decay, gate

    DELTA_GATES_AHEAD = 64  # tokens of a step from which decays and betas are made by a launch of their own

    def delta_scan(self, q, k, v, ba, a_log, dt_bias, state, heads: int, kv_heads: int, dim: int, vdim: int, seq_slots,
                   cu_tokens, decay=None) -> torch.Tensor:
        """Per head h, with the matrix state S [dim, vdim] of the request (float32; `state[slot]` holds the heads'
        states transposed, [heads][vdim][dim]) and the q, k of head h // (heads // kv_heads), token by token:
            beta = sigmoid(ba[t, h]);  g = exp(-exp(a_log[h]) softplus(ba[t, heads + h] + dt_bias[h]))
            S <- g S;  w = beta (v_t - S^T k_t);  S <- S + k_t w^T;  o_t = S^T q_t
        q, k float32 [N, kv_heads dim]; v float32 [N, heads vdim]; ba float32 [N, 2 heads]; a_log, dt_bias float32
        [heads].  With `decay` (float32 [N, heads dim], one of every key channel) S <- diag(decay_t) S instead; ba
        [N, >= heads] then begins with beta's inputs, and a_log and dt_bias are not used (None).
        Returns o float32 [N, heads vdim]; the states are advanced in place."""
        for t, name in ((q, "q"), (k, "k"), (v, "v"), (ba, "ba")) + (((a_log, "a_log"), (dt_bias, "dt_bias")) if decay is None
                                                                      else ((decay, "decay"),)):
            _dev(t, name, torch.float32)
        _rows(state, "state", torch.float32)
        _dev(seq_slots, "seq_slots", torch.int32)
        _dev(cu_tokens, "cu_tokens", torch.int32)
        N = v.shape[0]
        S = seq_slots.shape[0]
        H, G = int(heads), int(kv_heads)
        _need(G > 0 and H % G == 0, "the value heads are a multiple of the query/key heads")
        _need(0 < dim <= self.DELTA_MAX_DIM, f"a head of the delta rule holds at most {self.DELTA_MAX_DIM} key channels")
        _need(q.shape == (N, G * dim) and k.shape == (N, G * dim) and v.shape == (N, H * vdim),
              "q, k [N, kv_heads dim]; v [N, heads vdim]")
        if decay is None:
            _need(ba.shape == (N, 2 * H), "ba must be [N, 2 heads]")
            _need(a_log.shape == (H,) and dt_bias.shape == (H,), "a_log and dt_bias must be [heads]")
        else:
            _need(ba.dim() == 2 and ba.shape[0] == N and ba.shape[1] >= H and decay.shape == (N, H * dim),
                  "ba [N, >= heads]; decay [N, heads dim]")
        _need(state.shape[1] >= H * vdim * dim, "a state row holds heads * vdim * dim floats")
        _need(cu_tokens.shape == (S + 1,), "cu_tokens must be [S + 1]")
        out = torch.empty((N, H * vdim), dtype=torch.float32, device=v.device)
        # steps with portions: the exponentials of decay and beta leave the walk (a step of single tokens keeps them there:
        # one launch less).  The number of tokens is known on the host and fixed inside a graph.
        gates = torch.empty((N, 2 * H), dtype=torch.float32, device=v.device) if decay is None and N >= max(self.DELTA_GATES_AHEAD, 2 * S) else None
        self._run("delta", "lle_delta_scan", [_P, _P, _P, _P, _I, _P, _P, _P, _P, _L, _P, _P, _P, _I, _I, _I, _I, _I, _P, _I, _P],
                  _ptr(q), _ptr(k), _ptr(v), _ptr(ba), ba.shape[1], _ptr(decay), _ptr(a_log), _ptr(dt_bias), _ptr(state), state.stride(0),
                  _ptr(seq_slots), _ptr(cu_tokens), _ptr(out), S, H, G, dim, vdim, _ptr(gates), N)
        return out

    def delta_out_norm(self, o, gate, norm_w, eps: float, heads: int, vdim: int, act: str = "silu", out_dtype=None) -> torch.Tensor:
        """o float32 [N, heads vdim], gate [N, heads vdim] in the activation type (or float32, with `out_dtype` saying
        the activation type) -> every head of o divided by its root mean square (eps inside the root) times norm_w [vdim]
        times act(gate), act silu or sigmoid."""
        _dev(o, "o", torch.float32)
        _dev(gate, "gate")
        _dev(norm_w, "norm weight")
        _need(act in ("silu", "sigmoid"), f"a gate's activation is silu or sigmoid, not {act!r}")
        N = o.shape[0]
        _need(o.shape == (N, heads * vdim) and gate.shape == o.shape and norm_w.shape == (vdim,),
              "o and gate [N, heads vdim]; norm weight [vdim]")
        out = torch.empty(o.shape, dtype=out_dtype or gate.dtype, device=o.device)
        _need(gate.dtype in (torch.float32, out.dtype), "the gate is float32 or of the result's type")
        self._run("delta", "lle_delta_out_norm", [_P, _P, _I, _I, _P, _I, _F, _P, _I, _I, _I, _I, _P], _ptr(o), _ptr(gate),
                  dtype_code(gate.dtype), 1 if act == "sigmoid" else 0, _ptr(norm_w), dtype_code(norm_w.dtype), float(eps),
                  _ptr(out), N, int(heads), int(vdim), dtype_code(out.dtype))
        return out

    # -- the state-space recurrence of Mamba-2 ----------------------------------------------------
    SSD_MAX_DIM = MAX_SSD_DIM
    SSD_CHUNK = 64  # tokens of a chunk (lle_ssd_chunk)
    SSD_WALK = 32  # most tokens of a request that are walked one by one (lle_ssd_walk)

    def ssd_conv(self, u, col0: int, taps, bias, state, token_seq, cu_tokens, seq_slots, single: bool = False, x=None,
                 dt_w=None):
        """The columns col0 .. col0 + C - 1 of u [N, cols] convolved over time channel by channel with J taps (float32
        [C, J]; the last tap meets the token itself) + bias (float32 [C] or None), then silu -> float32 [N, C].  Tokens
        ahead of the step come from the request's state row (float32 [slots + 1, >= (J - 1) C]: the last J - 1 inputs of
        earlier steps, oldest first; None for J = 1), which moves on by the step's tokens.  `single`: every request of the
        step has one token (the row then moves on in the same launch).  With x [N, K] and dt_w [H, K] the result is (that,
        x dt_w^T float32 [N, H]): in the same launch for single tokens and up to 8 taps, else a product of its own."""
        if x is not None and not (single and taps.shape[1] <= 8):
            return self.ssd_conv(u, col0, taps, bias, state, token_seq, cu_tokens, seq_slots, single), self.linear(x, dt_w, torch.float32)
        _dev(u, "u")
        _dev(taps, "taps", torch.float32)
        for t, name in ((token_seq, "token_seq"), (cu_tokens, "cu_tokens"), (seq_slots, "seq_slots")):
            _dev(t, name, torch.int32)
        N, cols = u.shape
        C, J = taps.shape
        S = seq_slots.shape[0]
        _need(0 <= col0 and col0 + C <= cols and J >= 1, "u has too few columns")
        _need(token_seq.shape == (N,) and cu_tokens.shape == (S + 1,), "token_seq [N]; cu_tokens [S + 1]")
        if bias is not None:
            _dev(bias, "bias", torch.float32)
            _need(bias.shape == (C,), "the convolution's bias must be [C]")
        if J > 1:
            _need(state is not None, "a convolution of several taps needs the requests' state rows")
            _rows(state, "state", torch.float32)
            _need(state.shape[1] >= (J - 1) * C, "a state row holds J - 1 inputs")
        out = torch.empty((N, C), dtype=torch.float32, device=u.device)
        dt, K, H = None, 0, 0
        if x is not None:
            _dev(x, "x", u.dtype)
            _dev(dt_w, "dt_w", u.dtype)
            K, H = x.shape[1], dt_w.shape[0]
            _need(x.shape[0] == N and dt_w.shape == (H, K), "x must be [N, K], dt_w [H, K]")
            dt = torch.empty((N, H), dtype=torch.float32, device=u.device)
        self._run("ssd", "lle_ssd_conv",
                  [_P, _I, _I, _P, _I, _P, _P, _L, _P, _P, _P, _P, _I, _I, _I, _I, _P, _P, _P, _I, _I, _I, _P],
                  _ptr(u), cols, int(col0), _ptr(taps), J, _ptr(bias), _ptr(state) if J > 1 else None,
                  state.stride(0) if J > 1 else 0, _ptr(token_seq), _ptr(cu_tokens), _ptr(seq_slots), _ptr(out), N, S, C,
                  1 if single else 0, _ptr(x), _ptr(dt_w), _ptr(dt), K, H, dtype_code(u.dtype))
        return out if x is None else (out, dt)

    def ssd_heads_a_group(self, heads: int, groups: int, chunks: int) -> int:
        """Heads of a group that one workgroup of the chunks' second pass takes (they share C . B): as many as leave
        two workgroups for every CU."""
        most, share = max(1, heads * chunks // (2 * self.compute_units())), heads // groups
        return max(k for k in range(1, share + 1) if share % k == 0 and (k <= most or k == 1))

    def ssd_scan(self, c, dt_in, dt_bias, a_log, D, state, heads: int, groups: int, vdim: int, n: int, seq_slots, cu_tokens,
                 min_q_len: int = 0, max_q_len: int = 0) -> torch.Tensor:
        """Per head h, with the matrix state S [n, vdim] of the request (float32; `state[slot]` begins with the heads'
        states transposed, [heads][vdim][n]) and the B, C of group h // (heads // groups), token by token:
            dt = softplus(dt_in[t, h] + dt_bias[h]);  S <- exp(-exp(a_log[h]) dt) S + dt B_t x_t^T;  y_t = S^T C_t + D[h] x_t
        A row of c (float32) holds x [heads vdim], B [groups n], C [groups n]; dt_in float32 [N, >= heads].  Returns y float32
        [N, heads vdim]; the states are advanced in place.  `min_q_len` and `max_q_len` are host-side bounds of the
        requests' tokens in this step (0: not known); they choose kernels, never results."""
        for t, name in ((c, "c"), (dt_in, "dt_in"), (dt_bias, "dt_bias"), (a_log, "a_log"), (D, "D")):
            _dev(t, name, torch.float32)
        _rows(state, "state", torch.float32)
        _dev(seq_slots, "seq_slots", torch.int32)
        _dev(cu_tokens, "cu_tokens", torch.int32)
        N, CC = c.shape
        S = seq_slots.shape[0]
        H, G = int(heads), int(groups)
        _need(G > 0 and H % G == 0, "the heads are a multiple of the groups")
        _need(0 < vdim <= self.SSD_MAX_DIM and 0 < n <= self.SSD_MAX_DIM, f"a head of the recurrence holds at most {self.SSD_MAX_DIM} channels")
        _need(CC == H * vdim + 2 * G * n, "a row of c holds x, B and C")
        _need(dt_in.dim() == 2 and dt_in.shape[0] == N and dt_in.shape[1] >= H, "dt_in must be [N, >= heads]")
        _need(dt_bias.shape == (H,) and a_log.shape == (H,) and D.shape == (H,), "dt_bias, a_log and D must be [heads]")
        _need(state.shape[1] >= H * vdim * n and cu_tokens.shape == (S + 1,), "a state row holds heads * vdim * n floats")
        longest = min(max_q_len or N, N)
        pieces = -(-longest // self.SSD_CHUNK) if longest > self.SSD_WALK else 0
        y = torch.empty((N, H * vdim), dtype=torch.float32, device=c.device)
        part = part_decay = None
        together = 1
        if pieces:
            slots = N // self.SSD_CHUNK + S
            part = torch.empty((slots * H * vdim * n,), dtype=torch.float32, device=c.device)
            part_decay = torch.empty((slots * H,), dtype=torch.float32, device=c.device)
            together = self.ssd_heads_a_group(H, G, -(-N // self.SSD_CHUNK))
        self._run("ssd", "lle_ssd_scan",
                  [_P, _I, _P, _I, _P, _P, _P, _P, _L, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P, _P, _P],
                  _ptr(c), CC, _ptr(dt_in), dt_in.shape[1], _ptr(dt_bias), _ptr(a_log), _ptr(D), _ptr(state), state.stride(0),
                  _ptr(seq_slots), _ptr(cu_tokens), _ptr(y), S, H, G, int(vdim), int(n),
                  1 if (min_q_len or 1) <= self.SSD_WALK else 0, pieces, together, _ptr(part), _ptr(part_decay))
        return y

    def ssd_gate_norm(self, y, u, z_col: int, norm_w, eps: float, groups: int) -> torch.Tensor:
        """y float32 [N, inner], z = u[:, z_col : z_col + inner] -> y * silu(z), every one of `groups` equal parts of a row
        divided by its own root mean square (eps inside the root), times norm_w (float32 [inner]), in u's type."""
        _dev(y, "y", torch.float32)
        _dev(u, "u")
        _dev(norm_w, "norm weight", torch.float32)
        N, inner = y.shape
        _need(u.shape[0] == N and 0 <= z_col and z_col + inner <= u.shape[1], "u has too few columns")
        _need(norm_w.shape == (inner,) and groups > 0 and inner % groups == 0, "the norm weight must be [inner], cut into equal parts")
        out = torch.empty((N, inner), dtype=u.dtype, device=u.device)
        self._run("ssd", "lle_ssd_gate_norm", [_P, _P, _I, _I, _P, _F, _P, _I, _I, _I, _I, _P], _ptr(y), _ptr(u), u.shape[1],
                  int(z_col), _ptr(norm_w), float(eps), _ptr(out), N, inner, int(groups), dtype_code(u.dtype))
        return out

    # -- picking tokens --------------------------------------------------------------
    def argmax(self, logits, scatter=None) -> torch.Tensor:
        """float32 [R, V] -> int32 [R], first maximum wins.  `scatter` = (dst int32, index int32 [R]):
        the pick of row r is also written to dst[index[r]] (the host has made sure that index is in range)."""
        _dev(logits, "logits", torch.float32)
        R, V = logits.shape
        out = torch.empty((R,), dtype=torch.int32, device=logits.device)
        chunks = max(1, min(64, V // 2048))  # enough workgroups to stream a long row from all CUs
        part_val = torch.empty((R * chunks,), dtype=torch.float32, device=logits.device)
        part_idx = torch.empty((R * chunks,), dtype=torch.int32, device=logits.device)
        dst = index = None
        if scatter is not None:
            dst, index = scatter
            _dev(dst, "scatter destination", torch.int32)
            _dev(index, "scatter index", torch.int32)
            _need(index.shape == (R,), "one scatter index for every row")
        self._run("sampling", "lle_argmax_rows_scatter", [_P, _P, _P, _P, _I, _I, _I, _P, _P, _P],
                  _ptr(logits), _ptr(out), _ptr(part_val), _ptr(part_idx), R, V, chunks, _ptr(dst), _ptr(index))
        return out

    def sample(self, logits, temperature, uniform) -> torch.Tensor:
        """float32 logits [R, V], temperature [R] (<= 0: greedy), uniform [R] in [0, 1) -> int32 [R]."""
        _dev(logits, "logits", torch.float32)
        _dev(temperature, "temperature", torch.float32)
        _dev(uniform, "uniform", torch.float32)
        R, V = logits.shape
        _need(temperature.shape == (R,) and uniform.shape == (R,), "temperature and uniform must be [R]")
        out = torch.empty((R,), dtype=torch.int32, device=logits.device)
        self._run("sampling", "lle_sample_rows", [_P, _P, _P, _P, _I, _I, _P],
                  _ptr(logits), _ptr(temperature), _ptr(uniform), _ptr(out), R, V)
        return out


    # -- measured peaks (the benchmark's rooflines) ---------------------------------------------
    def probe_read_stream(self, data: torch.Tensor, blocks: int) -> None:
        """Launch a kernel that only reads `data` (any type, a multiple of 16 bytes), `blocks` workgroups."""
        _dev(data, "data")
        nbytes = data.numel() * data.element_size()
        _need(nbytes % 16 == 0 and nbytes > 0, "the read probe takes a multiple of 16 bytes")
        self._run("probe", "lle_probe_read_stream", [_P, _L, _I, _P, _P], _ptr(data), nbytes, int(blocks), None)

    def probe_mfma(self, dtype, blocks: int, iters: int) -> float:
        """Launch a kernel of nothing but matrix instructions on registers; returns its flops."""
        self._run("probe", "lle_probe_mfma", [_I, _I, _I, _P, _P], dtype_code(dtype), int(blocks), int(iters), None)
        per_instruction = 2.0 * 16 * 16 * (32 if dtype == torch.bfloat16 else 4)
        return per_instruction * 16 * iters * 4 * blocks


_default: Optional[HipOps] = None


def default_ops() -> HipOps:
    global _default
    if _default is None:
        _default = HipOps()
    return _default
