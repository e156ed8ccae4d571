"""The entry points of libdecdec_mixers.so as functions on torch tensors.  They raise if the library is missing; there is
no fallback.  Storage dtype float32 or bfloat16; the residual stream and recurrent states are float32 in both."""
from __future__ import annotations

import ctypes

import torch

from . import _lib
from .ext import _check, _ptr, _stream

GATE_SIGMOID, GATE_SILU = 0, 1
ACT_XIELU, ACT_GELU_TANH = 0, 1
_CODE = {torch.float32: 0, torch.bfloat16: 2}
_opt = lambda t: None if t is None else t.data_ptr()


def _dt(dtype: torch.dtype) -> int:
    _check(dtype in _CODE, "these layers run in float32 or bfloat16")
    return _CODE[dtype]


def _on_gpu(*ts):
    for t in ts:
        _check(t is None or t.is_cuda, "tensors must be CUDA tensors")


def gemv(weight: torch.Tensor, x: torch.Tensor, out: torch.Tensor, act=None, act_rows: int = 0, kind: int = ACT_XIELU,
         scale: float = 1.0) -> None:
    """out = scale * weight @ x for one token; the first act_rows results pass the activation `kind` (xIELU: with the two
    numbers of `act`)."""
    _on_gpu(weight, x, out, act)
    N, K = weight.shape
    _check(weight.is_contiguous() and x.is_contiguous() and out.is_contiguous() and x.numel() == K and out.numel() == N
           and x.dtype == out.dtype == weight.dtype, "weight [N, K], x with K and out with N elements of one dtype")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_gemv(_ptr(weight), _ptr(x), _ptr(out), _opt(act), act_rows, kind, float(scale),
                                                         _dt(weight.dtype), N, K, _stream()))


def _tanh_norm(norm, dim: int, dtype) -> "_lib.TanhNorm":
    """(alpha, weight, bias) of a dynamic tanh."""
    alpha, weight, bias = norm
    _on_gpu(alpha, weight, bias)
    _check(alpha.numel() == 1 and weight.numel() == bias.numel() == dim and alpha.dtype == weight.dtype == bias.dtype == dtype and
           weight.is_contiguous() and bias.is_contiguous(), "alpha [], weight and bias [dim] of the storage dtype")
    return _lib.TanhNorm(alpha.data_ptr(), weight.data_ptr(), bias.data_ptr())


def embed(table: torch.Tensor, tokens: torch.Tensor, x: torch.Tensor, x_e, norm=None) -> None:
    """x = table[tokens] in float32; x_e the same in the table's dtype, through the dynamic tanh `norm` if given."""
    _on_gpu(table, tokens, x, x_e)
    _check(tokens.dtype == torch.int64 and tokens.is_contiguous() and table.is_contiguous() and x.is_contiguous() and
           x.dtype == torch.float32 and x.numel() == tokens.numel() * table.shape[1], "int64 tokens and a float32 row for each")
    _check(x_e is None or (x_e.dtype == table.dtype and x_e.is_contiguous() and x_e.numel() == x.numel()), "x_e like x, of the table's dtype")
    n = None if norm is None else ctypes.byref(_tanh_norm(norm, table.shape[1], table.dtype))
    _lib.check_mixers(_lib.load_mixers().decdec_mix_embed(_ptr(table), _ptr(tokens), _ptr(x), _opt(x_e), n, _dt(table.dtype),
                                                          tokens.numel(), table.shape[0], table.shape[1], _stream()))


def residual_tanh(x: torch.Tensor, y, norm, out: torch.Tensor) -> None:
    """Rows of x [rows, dim] (float32, updated): x += y (None: nothing to add); out = tanh(alpha x) * weight + bias."""
    _on_gpu(x, y, out)
    rows, dim = x.shape
    _check(x.dtype == torch.float32 and x.is_contiguous() and out.is_contiguous() and out.shape == x.shape and
           (y is None or (y.is_contiguous() and y.shape == x.shape and y.dtype == out.dtype)), "x float32, y and out [rows, dim]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_residual_tanh(_ptr(x), _opt(y), ctypes.byref(_tanh_norm(norm, dim, out.dtype)), _ptr(out),
                                                                  _dt(out.dtype), rows, dim, _stream()))


def gated_residual(x: torch.Tensor, y: torch.Tensor, gate, gate_ld: int, bias, weight: torch.Tensor, x_e, eps: float,
                   final_weight=None, final_out=None) -> None:
    """Rows of x [rows, dim] (float32, updated): x += rms_norm(y * sigmoid(gate + bias)) * weight.  `gate` starts at its
    first element of row 0, rows gate_ld apart."""
    _on_gpu(x, y, gate, bias, weight, x_e, final_weight, final_out)
    rows, dim = x.shape
    _check(x.dtype == torch.float32 and x.is_contiguous() and y.is_contiguous() and y.shape == x.shape and weight.numel() == dim,
           "x, y [rows, dim] and weight [dim]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_gated_residual(
        _ptr(x), _ptr(y), _opt(gate), gate_ld, _opt(bias), _ptr(weight), _opt(x_e), _opt(final_weight), _opt(final_out),
        _dt(y.dtype), rows, dim, float(eps), _stream()))


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor, eps: float) -> None:
    _on_gpu(x, weight, out)
    rows, dim = x.shape
    _check(x.dtype == torch.float32 and x.is_contiguous() and out.is_contiguous() and out.shape == x.shape and weight.numel() == dim,
           "x float32, out [rows, dim] and weight [dim]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_rmsnorm(_ptr(x), _ptr(weight), _ptr(out), _dt(out.dtype), rows, dim, float(eps), _stream()))


def activation(rows_in: torch.Tensor, n: int, act, out: torch.Tensor, kind: int = ACT_XIELU) -> None:
    """First n columns of rows_in [rows, ld] through the activation into out [rows, n] (which may be rows_in itself where ld
    is n); xIELU takes the two numbers of `act`."""
    _on_gpu(rows_in, act, out)
    rows, ld = rows_in.shape
    _check(rows_in.is_contiguous() and out.is_contiguous() and tuple(out.shape) == (rows, n) and rows_in.dtype == out.dtype, "out must be [rows, n]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_activation(_ptr(rows_in), ld, _opt(act), kind, _ptr(out), _dt(out.dtype), rows, n, _stream()))


def _row_stride(t: torch.Tensor) -> int:
    _check(t.stride(1) == 1, "rows must be contiguous")
    return t.stride(0) if t.shape[0] > 1 else t.shape[1]


def group_norm_gate(o: torch.Tensor, gate: torch.Tensor, ld: int, weight: torch.Tensor, out: torch.Tensor, groups: int,
                    eps: float, kind: int, scale: float = 1.0) -> None:
    """o float32 [rows, groups * n]: RMS norm per group of n, times weight [n], times the gate function of `gate` (whose
    rows are ld apart), times scale.  `out` may be some columns of a wider array."""
    _on_gpu(o, gate, weight, out)
    rows, width = o.shape
    _check(o.dtype == torch.float32 and o.is_contiguous() and out.shape == o.shape and
           weight.numel() * groups == width, "o and out [rows, groups * n], weight [n]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_group_norm_gate(
        _ptr(o), _ptr(gate), ld, _ptr(weight), _ptr(out), _row_stride(out), _dt(out.dtype), rows, groups, width // groups, float(eps),
        kind, float(scale), _stream()))


# ---- recurrences -------------------------------------------------------------------------------------------
def recurrence_step_fuses(dim: int, vdim: int) -> bool:
    return bool(_lib.load_mixers().decdec_mix_recurrence_step_fuses(dim, vdim))


def recurrence_step(p: "_lib.Recurrence", dtype, o=None, out=None, norm_weight=None, eps: float = 0.0, kind: int = GATE_SILU) -> None:
    _lib.check_mixers(_lib.load_mixers().decdec_mix_recurrence_step(ctypes.byref(p), _opt(o), _opt(out), _opt(norm_weight),
                                                                    float(eps), kind, _dt(dtype), _stream()))


def recurrence_workspace(p: "_lib.Recurrence", rows: int) -> int:
    return int(_lib.load_mixers().decdec_mix_recurrence_workspace(ctypes.byref(p), rows))


def recurrence_rows(p: "_lib.Recurrence", dtype, o: torch.Tensor, workspace: torch.Tensor, rows: int) -> None:
    _check(o.dtype == torch.float32 and o.is_contiguous() and o.numel() == rows * p.heads * p.vdim, "o float32 [rows, heads * vdim]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_recurrence_rows(ctypes.byref(p), _ptr(o), _ptr(workspace),
                                                                    workspace.numel() * workspace.element_size(), _dt(dtype), rows, _stream()))


# ---- grouped attention -------------------------------------------------------------------------------------
def grouped_append(p: "_lib.Grouped", dtype, q_out: torch.Tensor, rows: int) -> None:
    _check(q_out.dtype == dtype and q_out.is_contiguous() and q_out.numel() == rows * p.heads * p.dim, "q_out [rows, heads, dim]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_grouped_append(ctypes.byref(p), _ptr(q_out), _dt(dtype), rows, _stream()))


def grouped_attention(p: "_lib.Grouped", dtype, q: torch.Tensor, out: torch.Tensor, start: int, rows: int) -> None:
    """`out` [rows, heads * vdim] may be some columns of a wider array."""
    _on_gpu(q, out)
    _check(q.dtype == out.dtype == dtype and q.is_contiguous() and q.numel() == rows * p.heads * p.dim and
           tuple(out.shape) == (rows, p.heads * p.vdim), "q [rows, heads, dim], out [rows, heads * vdim]")
    p.out_ld = _row_stride(out)
    _lib.check_mixers(_lib.load_mixers().decdec_mix_grouped_attention(ctypes.byref(p), _ptr(q), _ptr(out), _dt(dtype), start, rows, _stream()))


def grouped_step_workspace(p: "_lib.Grouped") -> int:
    return int(_lib.load_mixers().decdec_mix_grouped_step_workspace(ctypes.byref(p)))


def grouped_step(p: "_lib.Grouped", dtype, out: torch.Tensor, workspace: torch.Tensor) -> None:
    _check(out.dtype == dtype and out.is_contiguous() and out.numel() == p.heads * p.vdim, "out [heads * vdim]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_grouped_step(ctypes.byref(p), _ptr(out), _ptr(workspace),
                                                                 workspace.numel() * workspace.element_size(), _dt(dtype), _stream()))


# ---- latent attention --------------------------------------------------------------------------------------
def latent_append(p: "_lib.Latent", dtype, q_out: torch.Tensor, rows: int) -> None:
    _check(q_out.dtype == dtype and q_out.is_contiguous() and q_out.numel() == rows * p.heads * (p.dim + p.rot), "q_out [rows, heads, dim + rot]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_latent_append(ctypes.byref(p), _ptr(q_out), _dt(dtype), rows, _stream()))


def latent_attention(p: "_lib.Latent", dtype, q: torch.Tensor, k: torch.Tensor, vt: torch.Tensor, out: torch.Tensor, start: int,
                     rows: int) -> None:
    """k [keys, heads * dim], vt [heads * vdim, keys rounded up to 64]."""
    _on_gpu(q, k, vt, out)
    _check(q.dtype == k.dtype == vt.dtype == out.dtype == dtype and k.is_contiguous() and vt.is_contiguous() and out.is_contiguous(),
           "operands must be contiguous and share a dtype")
    _check(k.shape[0] >= start + rows and k.shape[1] == p.heads * p.dim and vt.shape[0] == p.heads * p.vdim and
           out.numel() == rows * p.heads * p.vdim, "operand shape mismatch")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_latent_attention(ctypes.byref(p), _ptr(q), _ptr(k), _ptr(vt), vt.shape[1], _ptr(out),
                                                                     _dt(dtype), start, rows, _stream()))


def latent_step_workspace(p: "_lib.Latent") -> int:
    return int(_lib.load_mixers().decdec_mix_latent_step_workspace(ctypes.byref(p)))


def latent_step(p: "_lib.Latent", dtype, out: torch.Tensor, workspace: torch.Tensor) -> None:
    _check(out.dtype == dtype and out.is_contiguous() and out.numel() == p.heads * p.vdim, "out [heads * vdim]")
    _lib.check_mixers(_lib.load_mixers().decdec_mix_latent_step(ctypes.byref(p), _ptr(out), _ptr(workspace),
                                                                workspace.numel() * workspace.element_size(), _dt(dtype), _stream()))
