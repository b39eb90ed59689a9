"""Python faces of the HIP kernels.

Every function checks on the host that shapes, element types, strides and devices are what the
kernel and its launch grid assume, and only then passes raw device pointers and the current HIP
stream through ctypes.  A kernel that cannot take a size says so here with a clear error; there
is no CPU fallback, and a missing or unbuildable library raises at the first call.
"""

from __future__ import annotations

import ctypes
import logging
from ctypes import c_float, c_int, c_long, c_longlong, c_ulonglong, c_void_p

import numpy as np
import torch

from . import build

log = logging.getLogger("paged_llm_amd")
_warned_plain_attention: list = []       # (said once per process)
F32, BF16 = 0, 1
_DTYPE_CODE = {torch.float32: F32, torch.bfloat16: BF16}
MAX_HEAD_DIM_GENERIC = 256


class KernelError(RuntimeError):
    pass


def dtype_code(dtype: torch.dtype) -> int:
    try:
        return _DTYPE_CODE[dtype]
    except KeyError:
        raise KernelError(f"kernels take float32 or bfloat16, not {dtype}") from None


_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)
_raw_device = getattr(torch._C, "_cuda_getDevice", None)


def _stream():
    """The current HIP stream of the current device, as what ctypes passes for a pointer."""
    if _raw_stream is not None and _raw_device is not None:
        return _raw_stream(_raw_device())
    return torch.cuda.current_stream().cuda_stream


def _ptr(t: torch.Tensor | None):
    return None if t is None else t.data_ptr()


def _check(code: int, what: str) -> None:
    if code != 0:
        raise KernelError(f"{what}: kernel launch failed with code {code}")


def _need(cond: bool, msg: str) -> None:
    if not cond:
        raise KernelError(msg)


def _on_gpu(*tensors: torch.Tensor | None) -> None:
    for t in tensors:
        if t is not None and not t.is_cuda:
            raise KernelError("kernel operands must live on the GPU (there is no CPU path)")


_SIGNATURES = {
    "pllm_embed_gather": [c_int, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_void_p],
    "pllm_rmsnorm": [c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_int, c_int, c_void_p, c_int, c_long,
                     c_void_p],
    "pllm_gate_mul": [c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p],
    "pllm_add_bias": [c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_void_p],
    "pllm_rope_scatter": [c_int, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p,
                          c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p],
    "pllm_copy_pages": [c_int, c_void_p, c_void_p, c_void_p, c_int, c_long, c_void_p],
    "pllm_gemm_nt": [c_int, c_int, c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_int, c_int, c_int, c_void_p],
    "pllm_paged_attention_generic": [c_int, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_int,
                                     c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_float, c_int,
                                     c_float, c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p],
    "pllm_sample": [c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_ulonglong, c_void_p,
                    c_void_p, c_void_p],
    "pllm_sample_workspace_bytes": [c_int, c_int],
    "pllm_argmax": [c_void_p, c_int, c_int, c_void_p, c_void_p],
}
_FUNCS: dict = {}


def _fn(source: str, name: str, defines: dict | None = None, signature: list | None = None):
    key = (source, name, tuple(sorted(defines.items()))) if defines else (source, name)
    f = _FUNCS.get(key)
    if f is None:
        lib = build.load_library(source, defines)
        f = getattr(lib, name)
        f.argtypes = signature if signature is not None else _SIGNATURES[name]
        f.restype = c_int
        _FUNCS[key] = f
    return f


# ------------------------------------------------------------------------------------------- rows
def embed_gather(ids: torch.Tensor, table: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
    """out[t] = table[ids[t]]; ids int32 [T] (range already checked by the caller)."""
    _on_gpu(ids, table)
    _need(ids.dtype == torch.int32 and ids.dim() == 1 and ids.is_contiguous(), "ids must be contiguous int32 [T]")
    _need(table.dim() == 2 and table.is_contiguous(), "embedding table must be contiguous [vocab, hidden]")
    T, (V, H) = ids.numel(), table.shape
    if out is None:
        out = torch.empty((T, H), dtype=table.dtype, device=table.device)
    _need(out.shape == (T, H) and out.dtype == table.dtype and out.is_contiguous(), "bad output for embed_gather")
    _check(_fn("elementwise.hip", "pllm_embed_gather")(dtype_code(table.dtype), _ptr(ids), _ptr(table), _ptr(out),
                                                        T, H, V, _stream()), "embed_gather")
    return out


def rmsnorm(x: torch.Tensor, weight: torch.Tensor, eps: float, delta: torch.Tensor | None = None,
            row_index: torch.Tensor | None = None, write_residual: bool = True) -> torch.Tensor:
    """RMS norm of the rows of x (after adding delta, when given).

    With ``delta`` the sum ``x + delta`` (float add, rounded to the element type) is the new
    residual; it is written back into ``x`` unless ``write_residual`` is False.  ``row_index``
    (int32) selects which rows are normed; the output then has one row per index.
    ``delta`` may also be a float tensor [ranges, rows, hidden]: the partial sums of a product whose inner dimension
    was cut into ranges (``stream_linear`` with SL_PARTIAL); they are added in order, in float, with x.
    """
    _on_gpu(x, weight, delta, row_index)
    _need(x.dim() == 2 and x.is_contiguous(), "x must be contiguous [rows, hidden]")
    H = x.shape[1]
    _need(weight.dtype == torch.float32 and weight.shape == (H,) and weight.is_contiguous(),
          f"norm weight must be float32 [{H}], got {weight.dtype} {tuple(weight.shape)}")
    _need((H + 16) * 4 <= min(_max_lds_bytes(x.device), 160 * 1024),
          f"rmsnorm kernel stages one row in LDS as floats: hidden size {H} is above its limit")
    parts = None
    if delta is not None and delta.dim() == 3:
        parts, delta = delta, None
        _need(parts.dtype == torch.float32 and tuple(parts.shape[1:]) == tuple(x.shape) and parts.is_contiguous(),
              f"partial sums must be contiguous float32 [ranges, {x.shape[0]}, {H}]")
    if delta is not None:
        _need(delta.shape == x.shape and delta.dtype == x.dtype and delta.is_contiguous(), "delta must match x")
    if row_index is not None:
        _need(row_index.dtype == torch.int32 and row_index.dim() == 1 and row_index.is_contiguous(),
              "row_index must be contiguous int32")
        rows = row_index.numel()
    else:
        rows = x.shape[0]
    out = torch.empty((rows, H), dtype=x.dtype, device=x.device)
    x_out = x if ((delta is not None or parts is not None) and write_residual) else None
    _check(_fn("elementwise.hip", "pllm_rmsnorm")(dtype_code(x.dtype), _ptr(x), _ptr(delta), _ptr(row_index), _ptr(weight),
                                                   c_float(eps), _ptr(out), _ptr(x_out), rows, H, _ptr(parts),
                                                   0 if parts is None else parts.shape[0], 0 if parts is None else x.numel(),
                                                   _stream()), "rmsnorm")
    return out


ACTIVATIONS = {"silu": 0, "gelu_tanh": 1}      # the gate's activation in a gated product (PLLM_ACT_* in common.h)


def activation_code(name: str) -> int:
    _need(name in ACTIVATIONS, f"gate activation {name!r}: one of {sorted(ACTIVATIONS)}")
    return ACTIVATIONS[name]


# of single elements, without a gate (PLLM_ROW_ACT_* in common.h); "xielu" has two parameters, "relu2" is max(z, 0)^2
ROW_ACTIVATIONS = {**ACTIVATIONS, "gelu": 2, "xielu": 3, "tanh": 4, None: 5, "relu2": 6}


def row_activation_code(name: str | None) -> int:
    _need(name in ROW_ACTIVATIONS, f"activation {name!r}: one of {tuple(ROW_ACTIVATIONS)}")
    return ROW_ACTIVATIONS[name]


def activate_rows(rows: torch.Tensor, activation: str | None, params: tuple = (0.0, 0.0), out_dtype: torch.dtype | None = None) -> torch.Tensor:
    """act(rows) element by element in float, contiguous [T, cols] of ``out_dtype`` (default: the rows' type); rows a view with unit
    inner stride, either element type.  ``params``: the two numbers of "xielu" (see ``row_activation`` in common.h)."""
    _on_gpu(rows)
    _need(rows.dim() == 2 and rows.stride(1) == 1, "activate_rows: [T, cols] with unit inner stride")
    out = torch.empty(rows.shape, dtype=out_dtype or rows.dtype, device=rows.device)
    sig = [c_int, c_int, c_void_p, c_long, c_void_p, c_long, c_int, c_int, c_int, c_float, c_float, c_void_p]
    _check(_fn("float_stream.hip", "pllm_activate_rows", signature=sig)(
        dtype_code(rows.dtype), dtype_code(out.dtype), _ptr(rows), rows.stride(0), _ptr(out), out.stride(0), rows.shape[0], rows.shape[1],
        row_activation_code(activation), c_float(params[0]), c_float(params[1]), _stream()), "activate_rows")
    return out


def cap_rows(x: torch.Tensor, cap: float) -> torch.Tensor:
    """x = cap tanh(x / cap) in place, contiguous float32 (logits with a cap); returns x."""
    _on_gpu(x)
    _need(x.dtype == torch.float32 and x.is_contiguous() and cap > 0.0, "cap_rows takes contiguous float32 rows and a positive cap")
    _check(_fn("float_stream.hip", "pllm_cap_rows", signature=[c_void_p, c_float, c_long, c_void_p])(_ptr(x), c_float(cap), x.numel(), _stream()),
           "cap_rows")
    return x


def gate_mul(gate_up: torch.Tensor, activation: str = "silu") -> torch.Tensor:
    """[T, 2I] -> act(first half) * second half, [T, I]."""
    _on_gpu(gate_up)
    _need(gate_up.dim() == 2 and gate_up.is_contiguous() and gate_up.shape[1] % 2 == 0, "gate_up must be contiguous [T, 2I]")
    T, I = gate_up.shape[0], gate_up.shape[1] // 2
    out = torch.empty((T, I), dtype=gate_up.dtype, device=gate_up.device)
    _check(_fn("elementwise.hip", "pllm_gate_mul")(dtype_code(gate_up.dtype), activation_code(activation), _ptr(gate_up), _ptr(out), T, I,
                                                   _stream()), "gate_mul")
    return out


def silu_mul(gate_up: torch.Tensor) -> torch.Tensor:
    return gate_mul(gate_up, "silu")


def add_bias(sums: torch.Tensor, bias: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """float sums [T, N] + float bias [N], rounded once to ``dtype``."""
    _on_gpu(sums, bias)
    _need(sums.dtype == torch.float32 and sums.dim() == 2 and sums.stride(1) == 1, "add_bias: float rows with unit inner stride")
    _need(bias.dtype == torch.float32 and bias.shape == (sums.shape[1],) and bias.is_contiguous(), f"bias: float32 [{sums.shape[1]}]")
    out = torch.empty(sums.shape, dtype=dtype, device=sums.device)
    _check(_fn("elementwise.hip", "pllm_add_bias")(dtype_code(dtype), _ptr(sums), sums.stride(0), _ptr(bias), _ptr(out), out.stride(0),
                                                   sums.shape[0], sums.shape[1], _stream()), "add_bias")
    return out


def rope_scatter(qkv: torch.Tensor, positions: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor,
                 num_heads: int, num_kv_heads: int, head_dim: int, slot_mapping: torch.Tensor | None,
                 k_pages: torch.Tensor | None, v_pages: torch.Tensor | None, block_size: int,
                 rotary_dim: int | None = None, interleaved: bool = False) -> None:
    """Rotate q (in place) and k by the tables' angles at ``positions``; write k and v into pages.

    qkv: [T, >= (num_heads + 2 kv_heads) * d] rows (only q columns are needed when nothing is
    written).  k_pages [P, kv, bs, d], v_pages [P, kv, d, bs].  ``rotary_dim`` (default: the whole
    head) is how many leading elements of a head turn; ``interleaved`` pairs (2i, 2i + 1) instead of
    (i, i + rotary_dim / 2).  The caller guarantees positions < cos.shape[0] and slots < P * bs
    (checked on the host where the batch is built).
    """
    write_kv = k_pages is not None
    _on_gpu(qkv, positions, cos, sin, slot_mapping, k_pages, v_pages)
    T = qkv.shape[0]
    _need(qkv.dim() == 2 and qkv.stride(1) == 1, "qkv must be [T, width] with unit inner stride")
    need_cols = (num_heads + (2 * num_kv_heads if write_kv else 0)) * head_dim
    _need(qkv.shape[1] >= need_cols, f"qkv rows hold {qkv.shape[1]} values, need {need_cols}")
    rotary_dim = head_dim if rotary_dim is None else int(rotary_dim)
    _need(0 <= rotary_dim <= head_dim and rotary_dim % 2 == 0,
          f"rotary pairing needs an even width of at most the head size {head_dim}, got {rotary_dim}")
    _need(positions.dtype == torch.int32 and positions.shape == (T,) and positions.is_contiguous(), "positions: int32 [T]")
    half = rotary_dim // 2
    _need((cos is None) == (sin is None), "cos and sin tables come together")
    for t in (cos, sin):
        if t is None:
            continue
        _need(t.dtype == torch.float32 and t.dim() == 2 and t.shape[1] == half and t.is_contiguous(),
              f"rotary tables must be float32 [positions, {half}]")
    if write_kv:
        _need(slot_mapping is not None and slot_mapping.dtype == torch.int32 and slot_mapping.shape == (T,)
              and slot_mapping.is_contiguous(), "slot_mapping: int32 [T]")
        P = k_pages.shape[0]
        _need(tuple(k_pages.shape) == (P, num_kv_heads, block_size, head_dim) and k_pages.is_contiguous()
              and k_pages.dtype == qkv.dtype, "k_pages must be contiguous [pages, kv_heads, block_size, head_dim]")
        _need(tuple(v_pages.shape) == (P, num_kv_heads, head_dim, block_size) and v_pages.is_contiguous()
              and v_pages.dtype == qkv.dtype, "v_pages must be contiguous [pages, kv_heads, head_dim, block_size]")
    _check(_fn("elementwise.hip", "pllm_rope_scatter")(
        dtype_code(qkv.dtype), _ptr(qkv), qkv.stride(0), _ptr(positions), _ptr(cos), _ptr(sin), _ptr(slot_mapping),
        _ptr(k_pages), _ptr(v_pages), T, num_heads, num_kv_heads, head_dim, block_size, 1 if write_kv else 0,
        rotary_dim, 1 if interleaved else 0, _stream()), "rope_scatter")


def copy_pages(pages: torch.Tensor, src: torch.Tensor, dst: torch.Tensor) -> None:
    """pages[dst[i]] = pages[src[i]] (whole pages of one tensor of a layer's cache, of any element type: the
    bytes are copied in units of two or four)."""
    _on_gpu(pages, src, dst)
    _need(pages.is_contiguous() and pages.dim() >= 2, "pages must be contiguous [pages, ...]")
    _need(src.dtype == torch.int32 and dst.dtype == torch.int32 and src.shape == dst.shape and src.dim() == 1,
          "src and dst must be int32 vectors of one length")
    page_bytes = pages[0].numel() * pages.element_size()
    _need(page_bytes % 2 == 0 and pages.data_ptr() % 4 == 0, "a page must be an even number of bytes")
    unit, code = (4, F32) if page_bytes % 4 == 0 else (2, BF16)
    _check(_fn("elementwise.hip", "pllm_copy_pages")(code, _ptr(pages), _ptr(src), _ptr(dst),
                                                      src.numel(), page_bytes // unit, _stream()), "copy_pages")


# ------------------------------------------------------------------------------------------- products
def gemm_generic(a: torch.Tensor, w: torch.Tensor, out_dtype: torch.dtype | None = None) -> torch.Tensor:
    """a [M, K] times w [N, K] transposed, float accumulation in ascending k, any sizes."""
    _on_gpu(a, w)
    _need(a.dim() == 2 and w.dim() == 2 and a.shape[1] == w.shape[1], f"gemm shapes {tuple(a.shape)} x {tuple(w.shape)}^T")
    _need(a.stride(1) == 1 and w.stride(1) == 1, "gemm operands need unit inner stride")
    _need(a.dtype == w.dtype, "gemm operands must share their element type")
    out_dtype = out_dtype or a.dtype
    M, K = a.shape
    N = w.shape[0]
    out = torch.empty((M, N), dtype=out_dtype, device=a.device)
    _check(_fn("gemm_generic.hip", "pllm_gemm_nt")(dtype_code(a.dtype), dtype_code(out_dtype), _ptr(a), a.stride(0),
                                                    _ptr(w), w.stride(0), _ptr(out), N, M, N, K, _stream()), "gemm_generic")
    return out


# ------------------------------------------------------------------------------------------- attention
def _check_attention_args(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads, head_dim):
    _on_gpu(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k)
    _need(q.dim() == 2 and q.stride(1) == 1 and q.shape[1] >= num_heads * head_dim, "q must be [T, >= heads * d]")
    P, kvh, bs, d = k_pages.shape
    _need(kvh == num_kv_heads and d == head_dim and k_pages.is_contiguous(), "k_pages: contiguous [pages, kv_heads, bs, d]")
    _need(tuple(v_pages.shape) == (P, kvh, d, bs) and v_pages.is_contiguous(), "v_pages: contiguous [pages, kv_heads, d, bs]")
    _need(k_pages.dtype == q.dtype and v_pages.dtype == q.dtype, "q, k_pages and v_pages must share their element type")
    _need(num_heads % num_kv_heads == 0, "heads must be a multiple of kv heads")
    _need(block_tables.dtype == torch.int32 and block_tables.dim() == 2 and block_tables.stride(1) == 1, "block_tables: int32 [S, B]")
    S = block_tables.shape[0]
    _need(cu_seqlens_q.dtype == torch.int32 and cu_seqlens_q.numel() >= S + 1 and cu_seqlens_q.is_contiguous(), "cu_seqlens_q: int32 [S+1]")
    _need(seq_lens_k.dtype == torch.int32 and seq_lens_k.numel() >= S and seq_lens_k.is_contiguous(), "seq_lens_k: int32 [S]")
    return S, bs


class ScoreTerms:
    """Further terms of an attention score, for mixers that have them (None everywhere else).  With x the scaled
    product of a query at position i and a key at position n of head h:

        score = cap(x) + slopes[h] * (n - i),     cap(x) = c * tanh(x / c) for ``cap`` = c > 0, x for 0,

    and ``sinks[h]``: a logit that takes part in the softmax's sum and in nothing else.  ``slopes`` and ``sinks``
    are float32 [heads] on the device or None."""

    __slots__ = ("cap", "slopes", "sinks")

    def __init__(self, cap: float = 0.0, slopes: torch.Tensor | None = None, sinks: torch.Tensor | None = None):
        self.cap, self.slopes, self.sinks = float(cap), slopes, sinks

    def any(self) -> bool:
        return self.cap > 0.0 or self.slopes is not None or self.sinks is not None

    def compiled_as(self) -> int:
        """The form of the matrix-core kernels that serves these terms: 0 without any, 1 with all of them, 2 with sinks alone."""
        return 1 if self.cap > 0.0 or self.slopes is not None else 2 if self.sinks is not None else 0

    def checked(self, num_heads: int, device) -> "ScoreTerms":
        _need(self.cap >= 0.0 and self.cap == self.cap, f"a cap of the scores is positive, or 0 for none; got {self.cap}")
        for name, t in (("slopes", self.slopes), ("sinks", self.sinks)):
            if t is not None:
                _on_gpu(t)
                _need(t.dtype == torch.float32 and t.shape == (num_heads,) and t.is_contiguous() and t.device == device,
                      f"{name}: float32 [{num_heads}] beside the queries, got {tuple(t.shape)} {t.dtype} on {t.device}")
        return self


class KeyWeights:
    """How the visible keys of a query are chosen and weighed where that differs from a causal window under a softmax
    (None everywhere else):

    * ``keep_first`` k > 0: the sequence's first k positions stay visible to every later query whatever the window
      (query i sees key j when j <= i and (i - j < window or j < k)); the kept keys are at their own positions;
    * ``sigmoid``: no softmax; a visible key weighs sigmoid(score + ``head_bias[h]``) (float32 [heads] on the device, or
      None for no bias) and the weights are not normalised over the keys."""

    __slots__ = ("keep_first", "sigmoid", "head_bias")

    def __init__(self, keep_first: int = 0, sigmoid: bool = False, head_bias: torch.Tensor | None = None):
        self.keep_first, self.sigmoid, self.head_bias = int(keep_first), bool(sigmoid), head_bias

    def any(self) -> bool:
        return self.keep_first > 0 or self.sigmoid

    def checked(self, num_heads: int, window: int, device) -> "KeyWeights":
        _need(self.keep_first >= 0, f"kept first positions: a count >= 0, got {self.keep_first}")
        _need(self.keep_first == 0 or window >= 0, "first positions are kept beside a sliding window, not beside blocks")
        _need(self.head_bias is None or self.sigmoid, "a bias per head belongs to sigmoid weights")
        if self.head_bias is not None:
            t = self.head_bias
            _on_gpu(t)
            _need(t.dtype == torch.float32 and t.shape == (num_heads,) and t.is_contiguous() and t.device == device,
                  f"head_bias: float32 [{num_heads}] beside the queries")
        return self


def _terms_args(terms: "ScoreTerms | None", num_heads: int, device) -> tuple:
    if terms is None:
        return c_float(0.0), None, None
    terms.checked(num_heads, device)
    return c_float(terms.cap), _ptr(terms.slopes), _ptr(terms.sinks)


def paged_attention_generic(q: torch.Tensor, k_pages: torch.Tensor, v_pages: torch.Tensor, block_tables: torch.Tensor,
                            cu_seqlens_q: torch.Tensor, seq_lens_k: torch.Tensor, num_heads: int, num_kv_heads: int,
                            head_dim: int, scale: float, window: int = 0, out: torch.Tensor | None = None,
                            terms: ScoreTerms | None = None, weights: KeyWeights | None = None) -> torch.Tensor:
    """Causal attention over paged keys and values; one wavefront per (token, head), all in float.

    The caller guarantees (and the step function checks on the host) that every table entry
    below ceil(seq_len / block_size) is a valid page and that cu_seqlens_q ends at q.shape[0].
    """
    S, bs = _check_attention_args(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads, head_dim)
    _need(0 < head_dim <= MAX_HEAD_DIM_GENERIC, f"attention kernel takes head sizes up to {MAX_HEAD_DIM_GENERIC}, got {head_dim}")
    _need(num_heads <= 65535, "too many heads for one launch")
    if weights is not None:
        weights.checked(num_heads, int(window or 0), q.device)
    T = q.shape[0]
    if out is None:
        out = torch.empty((T, num_heads * head_dim), dtype=q.dtype, device=q.device)
    _need(out.shape == (T, num_heads * head_dim) and out.stride(1) == 1 and out.dtype == q.dtype, "bad attention output")
    _check(_fn("attention_generic.hip", "pllm_paged_attention_generic")(
        dtype_code(q.dtype), _ptr(q), q.stride(0), _ptr(k_pages), _ptr(v_pages), _ptr(out), out.stride(0),
        _ptr(block_tables), block_tables.stride(0), _ptr(cu_seqlens_q), _ptr(seq_lens_k), S, T, num_heads, num_kv_heads,
        head_dim, bs, c_float(scale), int(window or 0), *_terms_args(terms, num_heads, q.device),
        *((weights.keep_first, int(weights.sigmoid), _ptr(weights.head_bias)) if weights is not None else (0, 0, None)), _stream()),
        "paged_attention_generic")
    return out


# ------------------------------------------------------------------------------------------- sampling
def argmax(logits: torch.Tensor) -> torch.Tensor:
    _on_gpu(logits)
    _need(logits.dtype == torch.float32 and logits.dim() == 2 and logits.is_contiguous(), "logits: contiguous float32 [n, vocab]")
    n, V = logits.shape
    out = torch.empty((n,), dtype=torch.int32, device=logits.device)
    _check(_fn("sampling.hip", "pllm_argmax")(_ptr(logits), n, V, _ptr(out), _stream()), "argmax")
    return out


_sample_workspace: dict = {}


SAMPLE_CANDIDATES_TOP_K, SAMPLE_CANDIDATES_MASS_VOCAB = 64, 65536


def sample_candidates_apply(temperature: float, top_k: int, top_p: float, vocab: int) -> bool:
    """Whether a row with these settings may go by its candidates (the kernel's own rule, for callers that know the
    settings on the host and can spare the launch that picks candidates when no row uses them)."""
    if temperature < 1e-5:
        return False
    if 0 < top_k <= SAMPLE_CANDIDATES_TOP_K:
        return top_k < vocab
    return top_p < 1.0 and vocab >= SAMPLE_CANDIDATES_MASS_VOCAB


def rows_sampled_by_candidates(rows: int, vocab: int, device) -> list:
    """For the last ``sample`` call of this shape on the device: which rows went by their candidates (a look into the
    call's workspace, for tests and measurements)."""
    f = _fn("sampling.hip", "pllm_sample_workspace_bytes")
    f.restype = c_long
    need = int(f(rows, vocab))
    workspace = _sample_workspace.get(str(torch.device(device)))
    if not need or workspace is None:
        return [False] * rows
    chunks = need // 4 // (3 + 2 * 192) // rows
    counts = workspace[: rows * chunks * 4].view(torch.int32).view(rows, chunks)
    return (counts >= 0).all(dim=1).tolist()


def sample(logits: torch.Tensor, temperature: torch.Tensor, top_k: torch.Tensor, top_p: torch.Tensor,
           request_key: torch.Tensor, step: torch.Tensor, seed: int, candidates: bool = True) -> torch.Tensor:
    """One token per row: greedy where temperature < 1e-5, else a draw under top-k / top-p.  ``candidates``: few rows
    of a long vocabulary whose top_k is small are first cut into chunks that hand on their largest logits, and the
    search and the draw run over those (a row's token depends on its own settings only either way; False walks every
    row whole)."""
    _on_gpu(logits, temperature, top_k, top_p, request_key, step)
    _need(logits.dtype == torch.float32 and logits.dim() == 2 and logits.is_contiguous(), "logits: contiguous float32 [n, vocab]")
    n, V = logits.shape
    for t, dt, nm in ((temperature, torch.float32, "temperature"), (top_k, torch.int32, "top_k"), (top_p, torch.float32, "top_p"),
                      (request_key, torch.int64, "request_key"), (step, torch.int32, "step")):
        _need(t.dtype == dt and t.shape == (n,) and t.is_contiguous(), f"{nm}: {dt} [{n}]")
    out = torch.empty((n,), dtype=torch.int32, device=logits.device)
    workspace = None
    if candidates:
        f = _fn("sampling.hip", "pllm_sample_workspace_bytes")
        f.restype = c_long
        need = int(f(n, V))
        if need:
            workspace = _sample_workspace.get(str(logits.device))
            if workspace is None or workspace.numel() < need:
                workspace = _sample_workspace[str(logits.device)] = torch.empty(max(need, 1 << 20), dtype=torch.uint8, device=logits.device)
    _check(_fn("sampling.hip", "pllm_sample")(_ptr(logits), n, V, _ptr(temperature), _ptr(top_k), _ptr(top_p),
                                               _ptr(request_key), _ptr(step), c_ulonglong(seed & (2**64 - 1)), _ptr(out),
                                               _ptr(workspace), _stream()), "sample")
    return out


# ------------------------------------------------------------------------------------------- fused decode products
EPI_BF16, EPI_F32, EPI_GATED, EPI_ROPE_KV, EPI_ACT = 0, 1, 2, 3, 4
DECODE_MAX_ROWS = 16          # rows of the fused form with a sum or norm in front
DECODE_WIDE_MAX_ROWS = 64     # rows of the form for plain rows
_DECODE_SIG = [c_int, c_void_p, c_int, c_void_p, c_int, c_void_p, c_float, c_void_p, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p,
               c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int,
               c_int, c_float, c_float, c_void_p]
_lds_limit: dict = {}


def _max_lds_bytes(device) -> int:
    key = str(device)
    if key not in _lds_limit:
        f = _fn("decode_linear.hip", "pllm_max_lds_bytes", signature=[])
        f.restype = c_long
        with torch.cuda.device(device):
            _lds_limit[key] = int(f())
    return _lds_limit[key]


def decode_linear_takes(rows: int, K: int, x: torch.Tensor, w: torch.Tensor, staged: bool = True) -> bool:
    """Whether the fused decode product takes these operands (else the caller runs the parts apart).
    ``staged``: a residual sum or a norm runs in front, so the rows must fit into LDS; plain rows are read
    straight from memory, may be of any length, and there may be up to 64 of them."""
    if not (x.dtype == torch.bfloat16 and w.dtype == torch.bfloat16 and 0 < rows <= (DECODE_MAX_ROWS if staged else DECODE_WIDE_MAX_ROWS) and K % 8 == 0):
        return False
    if not (x.stride(1) == 1 and w.stride(1) == 1 and x.stride(0) % 8 == 0 and w.stride(0) % 8 == 0
            and x.data_ptr() % 16 == 0 and w.data_ptr() % 16 == 0):
        return False
    if not staged:
        return True
    f = _fn("decode_linear.hip", "pllm_decode_linear_lds_bytes", signature=[c_int, c_int, c_int])
    f.restype = c_long
    return int(f(rows, K, 8)) <= _max_lds_bytes(x.device)


def decode_linear_pays(rows: int, N: int, K: int, epi: int, staged: bool) -> bool:
    """Whether the fused decode product is the faster choice for plain rows (measured against the library's
    product; by sizes only).  Every unit of 16 weight rows rereads all rows from the cache: beyond 8 rows
    that is as much as it streams of weights, and the library wins for long rows (K = 5632, 14336); beyond
    16 rows it wins for all but small matrices (q/k/v and output projections of 2048-wide models), where
    the fused kernel still fills the chip better; beyond 32 rows only the saved rotary kernel pays, and matrices of
    at most 2048 rows, whose units leave half of the GPU free for a second line of workgroups.  The gate/up
    product of a 2048-wide model is the exception: with K <= 2048 a wavefront keeps its share of the rows in
    registers for all units of its workgroup, and with the SiLU kernel saved the fused form wins up to 48 rows
    (11264 x 2048: 15.3 against 17.2 us at 32 rows, 18.0 against 18.8 at 48, 20.2 against 18.7 at 64)."""
    if staged or rows <= 8:
        return True
    if rows <= 16:
        return K <= 4096
    if epi == EPI_GATED and K <= 2048 and rows <= 48:
        return True
    small = N * K <= (1 << 23)
    if small and N <= 2048:
        return True          # (at most 128 units: two lines of workgroups with half the rows each, 7.9 against 9.0 us at 64 rows)
    return small and (rows <= 32 or epi == EPI_ROPE_KV)


def decode_linear(x: torch.Tensor, w: torch.Tensor, epi: int = EPI_BF16, delta: torch.Tensor | None = None,
                  norm_weight: torch.Tensor | None = None, eps: float = 0.0, x_out: torch.Tensor | None = None,
                  row_index: torch.Tensor | None = None, rope: dict | None = None, tiled=None,
                  activation: str = "silu", act_params: tuple = (0.0, 0.0)) -> torch.Tensor:
    """rows = x[row_index] (+ delta) -> optional RMS norm -> rows W^T -> epilogue, in one kernel.
    ``tiled``: the matrix's ``TiledWeight`` with the pairing that goes with ``epi`` (at most 16 rows): the weights are then
    streamed from that copy, in contiguous pieces, wherever the kernel works in units of 16 weight rows.

    epi EPI_BF16 / EPI_F32: [M, N] out.  EPI_ACT: act(out) [M, N] (``activation`` one of ``ROW_ACTIVATIONS`` with ``act_params``).  EPI_GATED: w = [gate; up], out = act(gate) * up [M, N/2] (``activation``).
    EPI_ROPE_KV: w = [q; k; v] rows; q is rotated and returned [M, heads * d]; k (rotated) and v go
    into the cache pages; ``rope`` = dict(positions, cos, sin, slots, k_pages, v_pages, num_heads,
    num_kv_heads, head_dim, block_size).  ``x_out`` receives x + delta (the new residual).
    """
    _on_gpu(x, w, delta, norm_weight, x_out, row_index)
    M = row_index.numel() if row_index is not None else x.shape[0]
    K = x.shape[1]
    _need(x.dim() == 2 and w.dim() == 2 and w.shape[1] == K, f"decode_linear shapes {tuple(x.shape)} x {tuple(w.shape)}^T")
    staged = delta is not None or norm_weight is not None
    _need(decode_linear_takes(M, K, x, w, staged),
          "decode_linear takes bfloat16, K a multiple of 8, 1..64 plain rows, or with a sum or norm in front 1..16 rows that fit LDS")
    if delta is not None:
        _need(delta.shape == x.shape and delta.dtype == x.dtype and delta.stride(1) == 1 and delta.stride(0) % 8 == 0
              and delta.data_ptr() % 16 == 0, "delta must match x")
    if x_out is not None:
        _need(delta is not None and x_out.shape == x.shape and x_out.dtype == x.dtype and x_out.stride(1) == 1
              and x_out.stride(0) % 8 == 0 and x_out.data_ptr() != x.data_ptr(), "x_out must be a separate buffer like x")
    if norm_weight is not None:
        _need(norm_weight.dtype == torch.float32 and norm_weight.shape == (K,) and norm_weight.is_contiguous(), "norm weight: float32 [K]")
    if row_index is not None:
        _need(row_index.dtype == torch.int32 and row_index.dim() == 1 and row_index.is_contiguous(), "row_index: int32")
    N = w.shape[0]
    r = rope or {}
    if tiled is not None:
        _need(M <= DECODE_MAX_ROWS and tiled.in_features == K and tiled.pairing == {EPI_GATED: "gated", EPI_ROPE_KV: "rotary"}.get(epi, "plain")
              and tiled.out_features * (2 if epi == EPI_GATED else 1) == N and tiled.tiles.is_contiguous()
              and (epi != EPI_ROPE_KV or tiled.head_dim == r.get("head_dim")),
              "the tiled copy does not belong to this matrix and epilogue")
    if epi == EPI_GATED:
        _need(N % 2 == 0, "gated product needs [gate; up] rows")
        N //= 2
        out = torch.empty((M, N), dtype=torch.bfloat16, device=x.device)
    elif epi == EPI_ROPE_KV:
        nh, nkv, d, bs = r["num_heads"], r["num_kv_heads"], r["head_dim"], r["block_size"]
        _need(d % 16 == 0 and N == (nh + 2 * nkv) * d, "fused rotary epilogue needs head sizes in multiples of 16 and [q; k; v] rows")
        kp, vp = r["k_pages"], r["v_pages"]
        P = kp.shape[0]
        _need(tuple(kp.shape) == (P, nkv, bs, d) and tuple(vp.shape) == (P, nkv, d, bs) and kp.is_contiguous() and vp.is_contiguous()
              and kp.dtype == torch.bfloat16 and vp.dtype == torch.bfloat16, "bad cache pages")
        for name in ("positions", "slots"):
            t = r[name]
            _need(t.dtype == torch.int32 and t.shape == (M,) and t.is_contiguous(), f"{name}: int32 [{M}]")
        if r.get("cos") is not None:
            for t in (r["cos"], r["sin"]):
                _need(t.dtype == torch.float32 and t.dim() == 2 and t.shape[1] == d // 2 and t.is_contiguous(), "rotary tables")
        out = torch.empty((M, nh * d), dtype=torch.bfloat16, device=x.device)
    else:
        out = torch.empty((M, N), dtype=torch.float32 if epi == EPI_F32 else torch.bfloat16, device=x.device)
    f = _fn("decode_linear.hip", "pllm_decode_linear", signature=_DECODE_SIG)
    _check(f(epi, _ptr(x), x.stride(0), _ptr(delta), delta.stride(0) if delta is not None else 0, _ptr(norm_weight), c_float(eps),
             _ptr(x_out), x_out.stride(0) if x_out is not None else 0, _ptr(row_index), _ptr(w), w.stride(0),
             None if tiled is None else _ptr(tiled.tiles), _ptr(out),
             out.stride(0), M, N, K, _ptr(r.get("positions")), _ptr(r.get("cos")), _ptr(r.get("sin")), _ptr(r.get("slots")),
             _ptr(r.get("k_pages")), _ptr(r.get("v_pages")), int(r.get("num_heads", 0)), int(r.get("num_kv_heads", 0)),
             int(r.get("head_dim", 0)), int(r.get("block_size", 0)), row_activation_code(activation) if epi == EPI_ACT else activation_code(activation),
             c_float(act_params[0]), c_float(act_params[1]), _stream()), "decode_linear")
    return out


# ------------------------------------------------------------------------------------------- products of 17 to a few hundred rows
SL_BF16, SL_F32, SL_GATED, SL_PARTIAL, SL_ROPE_KV, SL_ACT = 0, 1, 2, 3, 4, 5
STREAM_TILE_ROWS, STREAM_TILE_K = 16, 32
_STREAM_SIG = [c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p,
               c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_float, c_float, c_void_p]


class TiledWeight:
    """A weight matrix [N, K] in the order the streaming product kernel reads it: blocks of 16 rows, each block's tiles of
    16 rows x 32 columns one after the other along K, a tile being 1 KB in the order of the matrix instruction's operand
    (lane g * 16 + r: row r, columns 8 g .. 8 g + 7); zero rows pad the blocks to a multiple of 24.  ``pairing`` says
    which rows share a block: "plain" (16 successive rows), "gated" (8 gate rows and the up rows of the same outputs), or
    "rotary" (8 elements of the lower half of a head and their partners in the upper half, ``head_dim`` apart by half)."""

    def __init__(self, tiles: torch.Tensor, out_features: int, in_features: int, pairing: str, head_dim: int = 0):
        self.tiles, self.out_features, self.in_features, self.pairing, self.head_dim = tiles, out_features, in_features, pairing, head_dim

    @property
    def blocks(self) -> int:
        return self.tiles.shape[0]


def stream_linear_takes(w: torch.Tensor) -> bool:
    return w.dtype == torch.bfloat16 and w.dim() == 2 and w.shape[1] % STREAM_TILE_K == 0 and w.is_cuda


def tile_weight(w: torch.Tensor, pairing: str = "plain", head_dim: int = 0) -> TiledWeight:
    """The tiled copy of ``w`` [N, K] (bfloat16, K a multiple of 32).  "gated": w = [gate rows; up rows].  "rotary":
    w = [q; k; v] rows of heads of ``head_dim`` (a multiple of 16) elements."""
    _need(stream_linear_takes(w), "tiled weights: bfloat16 [N, K] on the GPU with K a multiple of 32")
    N, K = w.shape
    out_features = N
    if pairing == "gated":
        _need(N % 2 == 0, "a gated matrix holds gate rows and as many up rows")
        half = N // 2
        units = -(-half // 8)
        j = torch.arange(units * 8, device=w.device).view(units, 8).clamp_(max=half - 1)
        w = w.index_select(0, torch.cat([j, j + half], dim=1).reshape(-1))           # per block: 8 gate rows, their 8 up rows
        out_features = half
    elif pairing == "rotary":
        _need(head_dim > 0 and head_dim % 16 == 0 and N % head_dim == 0, "rotary pairing: whole heads of a multiple of 16 elements")
        heads, half = N // head_dim, head_dim // 2
        lower = (torch.arange(heads, device=w.device).view(heads, 1, 1) * head_dim
                 + torch.arange(half // 8, device=w.device).view(1, half // 8, 1) * 8 + torch.arange(8, device=w.device).view(1, 1, 8))
        w = w.index_select(0, torch.cat([lower, lower + half], dim=2).reshape(-1))    # per block: 8 lower elements, their partners
    else:
        _need(pairing == "plain", f"unknown pairing {pairing!r}")
    blocks = -(-w.shape[0] // 16)
    blocks_padded = -(-blocks // 24) * 24                                 # (whole workgroups of 1, 2, 3, 4 or 8 blocks)
    if blocks_padded * 16 != w.shape[0]:
        w = torch.cat([w, torch.zeros((blocks_padded * 16 - w.shape[0], K), dtype=w.dtype, device=w.device)])
    tiles = w.view(blocks_padded, 16, K // 32, 4, 8).permute(0, 2, 3, 1, 4).contiguous()       # [block, k step, g, r, 8]
    return TiledWeight(tiles, out_features, K, pairing, head_dim)


def _whole_ranges(stages: int, splits: int) -> int:
    """The largest number of ranges up to ``splits`` such that ranges of ceil(stages / ranges) stages leave none empty."""
    while splits > 1 and -(-stages // splits) * (splits - 1) >= stages:
        splits -= 1
    return splits


def stream_linear_plan(M: int, N: int, K: int, compute_units: int, partial: bool = True) -> tuple[int, int]:
    """(blocks of 16 weight rows per workgroup, ranges of K) for a product of M rows with N weight rows: by sizes only.
    What counts is that the workgroups are about as many as the compute units, in one round, and that each reads as few
    input rows as possible (every workgroup reads all rows of its range of K).  With partial sums allowed: two blocks
    and as many ranges of K as give every compute unit a workgroup (2048 x 5632 at 64 rows: 8.6 us in 4 ranges, 11.2 in 2,
    10.9 in 8); four blocks where K is long and the rows few (4096 x 14336 at 64 rows: 28.5 us against 30.6).  In one
    range: a block per workgroup while that fits one round (2048 x 2048: 6.7 us against 9.1 with two), else two."""
    blocks = -(-N // 16)
    row_blocks = -(-M // 128)
    stages = -(-K // 256)
    if not partial:
        return (1 if blocks * row_blocks <= compute_units else 2), 1
    nt = 4 if (K >= 8192 and M <= 64) else 2
    workgroups = -(-blocks // nt) * row_blocks
    splits = 1
    if workgroups < compute_units:
        splits = _whole_ranges(stages, max(1, min(compute_units // workgroups, stages // 2, 8)))
    return nt, splits


def gated_blocks_per_workgroup(out_features: int, compute_units: int) -> int:
    """Blocks of 16 weight rows (8 gate rows and their up rows) a workgroup of the gated product takes: three while
    that gives every block a workgroup in one round (5632 outputs: 235 workgroups, 14.7 us at 64 rows against 16.0
    with four and 19.4 with two), else four (14336 outputs: 56.9 us against 64.9 with three)."""
    units = -(-out_features // 8)
    return 3 if -(-units // 3) <= compute_units else 4


def stream_linear(x: torch.Tensor, w: TiledWeight, epi: int = SL_BF16, nt: int | None = None, splits: int | None = None,
                  rope: dict | None = None, activation: str = "silu", act_params: tuple = (0.0, 0.0)) -> torch.Tensor:
    """x [M, K] bfloat16 times the tiled weights.  SL_BF16 / SL_F32: [M, N]; SL_ACT: act of it (one of ``ROW_ACTIVATIONS`` with ``act_params``); SL_GATED: act(gate) * up [M, N / 2];
    SL_PARTIAL: float [splits, M, N], the sums over ``splits`` ranges of K, to be added in that order; SL_ROPE_KV: q rotated
    [M, heads * d], k (rotated) and v written to their pages (``rope`` as for ``decode_linear``)."""
    _on_gpu(x, w.tiles)
    M, K = x.shape
    _need(x.dtype == torch.bfloat16 and x.dim() == 2 and x.stride(1) == 1 and x.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0,
          "stream_linear: bfloat16 rows that start on 16-byte boundaries")
    _need(K == w.in_features and w.tiles.is_contiguous() and tuple(w.tiles.shape[1:]) == (K // 32, 4, 16, 8) and w.blocks % 24 == 0,
          f"stream_linear: rows of {K} values against tiled weights of {w.in_features}")
    _need({SL_GATED: "gated", SL_ROPE_KV: "rotary"}.get(epi, "plain") == w.pairing,
          f"epilogue {epi} against weights tiled with the {w.pairing} pairing")
    N = w.out_features
    if epi == SL_GATED:
        plan_nt, plan_splits = gated_blocks_per_workgroup(N, _num_compute_units(x.device)), 1
    else:
        plan_nt, plan_splits = stream_linear_plan(M, N, K, _num_compute_units(x.device), partial=epi == SL_PARTIAL)
    nt = nt or plan_nt
    splits = plan_splits if splits is None else splits
    _need(splits == 1 or epi == SL_PARTIAL, "ranges of K give partial sums")
    r = rope or {}
    if epi == SL_PARTIAL:
        out = torch.empty((splits, M, N), dtype=torch.float32, device=x.device)
    elif epi == SL_ROPE_KV:
        nh, nkv, d, bs = r["num_heads"], r["num_kv_heads"], r["head_dim"], r["block_size"]
        _need(d == w.head_dim and N == (nh + 2 * nkv) * d, "the weights were tiled for other heads")
        kp, vp = r["k_pages"], r["v_pages"]
        P = kp.shape[0]
        _need(tuple(kp.shape) == (P, nkv, bs, d) and tuple(vp.shape) == (P, nkv, d, bs) and kp.is_contiguous() and vp.is_contiguous()
              and kp.dtype == torch.bfloat16 and vp.dtype == torch.bfloat16, "bad cache pages")
        for name in ("positions", "slots"):
            t = r[name]
            _need(t.dtype == torch.int32 and t.shape == (M,) and t.is_contiguous(), f"{name}: int32 [{M}]")
        if r.get("cos") is not None:
            for t in (r["cos"], r["sin"]):
                _need(t.dtype == torch.float32 and t.dim() == 2 and t.shape[1] == d // 2 and t.is_contiguous() and t.data_ptr() % 16 == 0,
                      "rotary tables")
        out = torch.empty((M, nh * d), dtype=torch.bfloat16, device=x.device)
    else:
        out = torch.empty((M, N), dtype=torch.float32 if epi == SL_F32 else torch.bfloat16, device=x.device)
    f = _fn("stream_linear.hip", "pllm_stream_linear", signature=_STREAM_SIG)
    _check(f(epi, _ptr(x), x.stride(0), _ptr(w.tiles), _ptr(out), out.stride(-2), M, N, K, w.blocks, nt, splits,
             _ptr(r.get("positions")), _ptr(r.get("cos")), _ptr(r.get("sin")), _ptr(r.get("slots")), _ptr(r.get("k_pages")),
             _ptr(r.get("v_pages")), int(r.get("num_heads", 0)), int(r.get("num_kv_heads", 0)), int(r.get("head_dim", 0)),
             int(r.get("block_size", 0)), row_activation_code(activation) if epi == SL_ACT else activation_code(activation),
             c_float(act_params[0]), c_float(act_params[1]), _stream()), "stream_linear")
    return out


_TILE_SIG = [c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p,
             c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_void_p]
TILE_BLOCK_ROWS = 160           # input rows of one workgroup of the tiled kernel, at most


def tile_linear_plan(M: int, N: int, K: int, compute_units: int) -> int:
    """Ranges of K for the tiled product of M rows with N weight rows: as many as give every compute unit a workgroup
    (tiles of up to 160 rows x 128 weight rows), each at least four stages of 64 columns long."""
    workgroups = -(-N // 128) * -(-M // TILE_BLOCK_ROWS)
    stages = -(-K // 64)
    if workgroups >= compute_units:
        return 1
    return _whole_ranges(stages, max(1, min(compute_units // workgroups, stages // 4, 16)))


def tile_linear_shape(M: int, weight_rows: int, compute_units: int) -> tuple[int, int, int]:
    """(rows per block of input rows, weight rows per tile, workgroups) that the tiled kernel takes for a product in one
    range of K: the shape with the most workgroups in one round of the compute units (chosen in the library)."""
    f = _fn("stream_linear.hip", "pllm_tile_linear_shape", signature=[c_int, c_int, c_int, c_void_p, c_void_p])
    rows, tile = c_int(0), c_int(0)
    wgs = f(int(M), int(weight_rows), int(compute_units), ctypes.byref(rows), ctypes.byref(tile))
    _need(wgs > 0, f"tile_linear_shape({M}, {weight_rows}, {compute_units})")
    return rows.value, tile.value, wgs


def tile_linear(x: torch.Tensor, w: TiledWeight, epi: int = SL_BF16, splits: int | None = None, rope: dict | None = None,
                activation: str = "silu") -> torch.Tensor:
    """As ``stream_linear``, for a few hundred rows: tiles of up to 160 rows x 128 weight rows per workgroup, both
    operands through LDS."""
    _on_gpu(x, w.tiles)
    M, K = x.shape
    _need(x.dtype == torch.bfloat16 and x.dim() == 2 and x.stride(1) == 1 and x.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0,
          "tile_linear: bfloat16 rows that start on 16-byte boundaries")
    _need(K == w.in_features and w.tiles.is_contiguous() and tuple(w.tiles.shape[1:]) == (K // 32, 4, 16, 8) and w.blocks % 24 == 0,
          f"tile_linear: rows of {K} values against tiled weights of {w.in_features}")
    _need({SL_GATED: "gated", SL_ROPE_KV: "rotary"}.get(epi, "plain") == w.pairing,
          f"epilogue {epi} against weights tiled with the {w.pairing} pairing")
    N = w.out_features
    if splits is None:
        splits = tile_linear_plan(M, N * (2 if epi == SL_GATED else 1), K, _num_compute_units(x.device)) if epi == SL_PARTIAL else 1
    _need(splits == 1 or epi == SL_PARTIAL, "ranges of K give partial sums")
    r = rope or {}
    if epi == SL_PARTIAL:
        out = torch.empty((splits, M, N), dtype=torch.float32, device=x.device)
    elif epi == SL_ROPE_KV:
        nh, nkv, d, bs = r["num_heads"], r["num_kv_heads"], r["head_dim"], r["block_size"]
        _need(d == w.head_dim and N == (nh + 2 * nkv) * d, "the weights were tiled for other heads")
        kp, vp = r["k_pages"], r["v_pages"]
        P = kp.shape[0]
        _need(tuple(kp.shape) == (P, nkv, bs, d) and tuple(vp.shape) == (P, nkv, d, bs) and kp.is_contiguous() and vp.is_contiguous()
              and kp.dtype == torch.bfloat16 and vp.dtype == torch.bfloat16, "bad cache pages")
        for name in ("positions", "slots"):
            t = r[name]
            _need(t.dtype == torch.int32 and t.shape == (M,) and t.is_contiguous(), f"{name}: int32 [{M}]")
        if r.get("cos") is not None:
            for t in (r["cos"], r["sin"]):
                _need(t.dtype == torch.float32 and t.dim() == 2 and t.shape[1] == d // 2 and t.is_contiguous() and t.data_ptr() % 16 == 0,
                      "rotary tables")
        out = torch.empty((M, nh * d), dtype=torch.bfloat16, device=x.device)
    else:
        out = torch.empty((M, N), dtype=torch.float32 if epi == SL_F32 else torch.bfloat16, device=x.device)
    f = _fn("stream_linear.hip", "pllm_tile_linear", signature=_TILE_SIG)
    _check(f(epi, _ptr(x), x.stride(0), _ptr(w.tiles), _ptr(out), out.stride(-2), M, N, K, w.blocks, splits,
             _ptr(r.get("positions")), _ptr(r.get("cos")), _ptr(r.get("sin")), _ptr(r.get("slots")), _ptr(r.get("k_pages")),
             _ptr(r.get("v_pages")), int(r.get("num_heads", 0)), int(r.get("num_kv_heads", 0)), int(r.get("head_dim", 0)),
             int(r.get("block_size", 0)), activation_code(activation), _stream()), "tile_linear")
    return out


# ------------------------------------------------------------------------------------------- choices
def gemm_bf16(a: torch.Tensor, w: torch.Tensor, out_dtype: torch.dtype | None = None) -> torch.Tensor:
    """a [M, K] times w [N, K]^T for more rows than the fused decode kernel takes (prompt portions, large
    decode batches): the vendor's matrix-product library, as the reference's engine uses a library for
    its products (nn.Linear, pagedllm/model/llama.py:141-144).  Float accumulation; the result is bfloat16
    or, for logits, float32 straight from the accumulators."""
    _on_gpu(a, w)
    _need(a.dtype == torch.bfloat16 and w.dtype == torch.bfloat16 and a.dim() == 2 and w.dim() == 2 and a.shape[1] == w.shape[1],
          f"gemm_bf16 takes bfloat16 [M, K] x [N, K]^T, got {tuple(a.shape)} {a.dtype} x {tuple(w.shape)} {w.dtype}")
    if out_dtype == torch.float32:
        return torch.mm(a, w.t(), out_dtype=torch.float32)
    _need(out_dtype in (None, torch.bfloat16), "output is bfloat16 or float32")
    return torch.mm(a, w.t())


_ATTN_SIG = [c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int,
             c_int, c_int, c_int, c_float, c_int, c_int, c_int, c_void_p, c_int, c_int, c_void_p, c_int, c_void_p]
_ATTN_TERMS_SIG = _ATTN_SIG[:-1] + [c_int, c_float, c_void_p, c_void_p, c_void_p]
_attn_scratch: dict = {}
_attn_scratch_retired: list = []      # outgrown buffers stay allocated: captured graphs still hold their addresses
_attn_checked: set = set()


def mfma_attention_takes(dtype: torch.dtype, num_heads: int, num_kv_heads: int, head_dim: int, block_size: int) -> bool:
    return (dtype == torch.bfloat16 and head_dim % 16 == 0 and 16 <= head_dim <= 256 and block_size >= 16
            and block_size & (block_size - 1) == 0 and num_heads % num_kv_heads == 0 and num_heads // num_kv_heads <= 64)


def attention_decode_registers(head_dim: int, waves: int) -> int:
    """Vector registers per lane of the compiled decode attention kernel (16 columns, ``waves`` wavefronts)."""
    return int(_fn("attention_mfma.hip", "pllm_attention_decode_registers", {"HEAD_DIM": head_dim}, [c_int])(waves))


def attention_decode_spill_bytes(head_dim: int, waves: int) -> int:
    """Bytes per lane that the same kernel keeps outside registers; 0 unless registers were spilled."""
    return int(_fn("attention_mfma.hip", "pllm_attention_decode_spill_bytes", {"HEAD_DIM": head_dim}, [c_int])(waves))


def _merge_lds_bytes(column_blocks: int, waves: int, head_dim: int) -> int:
    """LDS of the attention kernel's several-wavefront variant (as merge_lds_bytes in attention_mfma.hip):
    maximum and weight per column and wavefront, and every wavefront's partial output."""
    return (2 * waves * column_blocks * 16 + waves * column_blocks * (head_dim // 16) * 4 * 64) * 4


def attention_plan(num_seqs: int, num_kv_heads: int, max_q_len: int, max_k_len: int, group: int, head_dim: int,
                   lds_limit: int, compute_units: int = 256) -> tuple[int, int, int]:
    """(wavefronts per work item, partition_size, num_partitions) for a step.

    Prompt portions have many query tiles: one wavefront per tile walks all its keys (1, 0, 1).
    Decoding has one tile per (sequence, kv head), far too few to fill the GPU: the keys are cut
    into aligned partitions, one workgroup each (merged by a second kernel), and inside a
    workgroup the wavefronts share the partition's blocks of 64 keys (merged in LDS)."""
    cols = max_q_len * group
    if cols > 64 or max_k_len <= 64:
        return 1, 0, 1
    ncb = 1 if cols <= 16 else (2 if cols <= 32 else 4)
    # Heads above 128 elements: a block of 64 keys and values takes more registers than eight wavefronts of a workgroup have
    # (64 sequences x 1 kv head x 2048 keys, in partitions of 512: at head size 144 29.0 us with four wavefronts, 39.3 with
    # eight; at 256 63 and 107 us).
    max_waves = 8 if head_dim <= 128 else 4
    while max_waves >= 4 and _merge_lds_bytes(ncb, max_waves, head_dim) > lds_limit:
        max_waves //= 2
    if max_waves < 4:
        return 1, 0, 1
    # Partitions only as far as they fill the GPU in one round: a workgroup of eight wavefronts has a compute unit to
    # itself, so work items x partitions stay at or under the number of compute units (48 sequences x 4 kv heads x 2048
    # keys at head size 64: 28.1 us in one piece on 192 compute units, 37.0 us in two partitions, which make 384
    # workgroups and two rounds; 24 sequences: 18.8 us in two partitions against 21.9 in four and 24.5 in one), and
    # fewer, longer work items are faster than many short ones plus a larger merge.
    items = num_seqs * num_kv_heads
    want_parts = max(1, compute_units // items)
    size = 256                                        # at least four blocks of 64 keys per workgroup
    while (max_k_len + size - 1) // size > want_parts:
        size *= 2
    parts = (max_k_len + size - 1) // size
    waves = max_waves
    while waves > 4 and (waves // 2) * 64 >= min(size, max_k_len):
        waves //= 2
    # Small heads (two blocks of keys under way per wavefront) and more work items than compute units: two
    # workgroups of four wavefronts on a compute unit stream faster than eight-wavefront workgroups in two rounds
    # (96 sequences x 4 kv heads x 2048 keys at head size 64: 48.7 against 57.5 us; 64 sequences x 8 kv heads: a decode
    # step of Llama-3.2-1B shapes 2.68 against 2.74 ms).  At head size 128 eight wavefronts stay ahead (40 sequences x 8
    # kv heads: 86.7 against 106.3 us).
    if head_dim <= 64 and parts == 1 and items > compute_units:
        waves = 4
    return (waves, size, parts) if parts > 1 else (waves, 0, 1)


def paged_attention_mfma(q: torch.Tensor, k_pages: torch.Tensor, v_pages: torch.Tensor, block_tables: torch.Tensor,
                         cu_seqlens_q: torch.Tensor, seq_lens_k: torch.Tensor, num_heads: int, num_kv_heads: int,
                         head_dim: int, scale: float, window: int, max_q_len: int, partition_size: int = 0,
                         num_partitions: int = 1, waves: int = 1, column_blocks: int = 0,
                         out: torch.Tensor | None = None, work_list: torch.Tensor | None = None,
                         terms: ScoreTerms | None = None, single_prompt: bool = False) -> torch.Tensor:
    """Causal attention over paged keys/values on the matrix cores (bfloat16).  ``max_q_len`` bounds
    the queries of any sequence of the batch; ``partition_size`` > 0 splits the keys of every
    work item into aligned partitions that a second kernel merges (best a multiple of 128 for prompt portions, whose
    workgroups walk the keys in steps of up to 128); ``waves`` > 1 shares the keys
    of a work item between the wavefronts of one workgroup (few queries per sequence only).  ``work_list``
    (prompt portions): int32 [n, 2] pairs of (sequence, tile of 128 query columns), the order in which the
    kernel's workgroups take them (``prompt_work_list``).  ``terms``: further terms of the scores (``ScoreTerms``);
    with any of them the kernels come from a library of their own, compiled with those terms in the score loop.
    ``single_prompt``: all queries but a few belong to one sequence (a hint for the prompt kernel's form)."""
    S, bs = _check_attention_args(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads, head_dim)
    _need(mfma_attention_takes(q.dtype, num_heads, num_kv_heads, head_dim, bs),
          f"MFMA attention takes bfloat16, head sizes 16..256 in steps of 16, pages of >= 16 positions and groups of <= 64 "
          f"heads; got {q.dtype}, head size {head_dim}, page {bs}, {num_heads}/{num_kv_heads} heads")
    _need(q.stride(0) % 8 == 0 and q.data_ptr() % 16 == 0, "q rows must start on 16-byte boundaries")
    T = q.shape[0]
    if out is None:
        out = torch.empty((T, num_heads * head_dim), dtype=q.dtype, device=q.device)
    _need(out.shape == (T, num_heads * head_dim) and out.stride(1) == 1 and out.dtype == q.dtype and out.stride(0) % 4 == 0,
          "bad attention output")
    _need(max_q_len >= 1 and partition_size % 64 == 0 and waves in (1, 4, 8), "bad launch parameters")
    ncb = min(column_blocks or 4, 1 if max_q_len * (num_heads // num_kv_heads) <= 16 else (2 if max_q_len * (num_heads // num_kv_heads) <= 32 else 4))
    _need(column_blocks in (0, 1, 2, 4), "column_blocks is 0 (automatic), 1, 2 or 4")
    _need(waves == 1 or _merge_lds_bytes(ncb, waves, head_dim) <= _max_lds_bytes(q.device),
          "the merge buffers of that many wavefronts do not fit LDS")
    if work_list is not None:
        _on_gpu(work_list)
        _need(work_list.dtype == torch.int32 and work_list.dim() == 2 and work_list.shape[1] == 2 and work_list.is_contiguous()
              and 0 < work_list.shape[0] <= 65535, "work_list: int32 [n, 2], n in 1..65535")
    ws = None
    if partition_size > 0:
        floats = T * num_heads * num_partitions * (head_dim + 2)
        key = str(q.device)
        ws = _attn_scratch.get(key)
        if ws is None or ws.numel() < floats:
            if ws is not None:
                _attn_scratch_retired.append(ws)
            ws = torch.empty(max(floats, 1 << 22), dtype=torch.float32, device=q.device)
            _attn_scratch[key] = ws
    with_terms = terms.checked(num_heads, q.device).compiled_as() if terms is not None else 0
    defines = {"HEAD_DIM": head_dim, "SCORE_TERMS": with_terms} if with_terms else {"HEAD_DIM": head_dim}
    if (head_dim, with_terms) not in _attn_checked:   # the library on disk is the one compiled for this head size
        built = _fn("attention_mfma.hip", "pllm_attention_mfma_head_dim", defines, [])()
        _need(built == head_dim, f"attention library for head size {head_dim} reports head size {built}")
        has_terms = _fn("attention_mfma.hip", "pllm_attention_mfma_score_terms", defines, [])()
        _need(has_terms == with_terms, f"attention library for head size {head_dim}: further score terms compiled in: {has_terms}")
        _attn_checked.add((head_dim, with_terms))
    args = (_ptr(q), q.stride(0), _ptr(k_pages), _ptr(v_pages), _ptr(out), out.stride(0), _ptr(block_tables),
            block_tables.stride(0), _ptr(cu_seqlens_q), _ptr(seq_lens_k), S, T, int(max_q_len), num_heads, num_kv_heads, bs,
            c_float(scale), int(window or 0), int(partition_size), int(num_partitions), _ptr(ws), int(waves), int(column_blocks),
            _ptr(work_list), 0 if work_list is None else work_list.shape[0])
    if with_terms or single_prompt:
        f = _fn("attention_mfma.hip", "pllm_paged_attention_mfma_terms", defines, _ATTN_TERMS_SIG)
        _check(f(*args, int(bool(single_prompt)), *_terms_args(terms, num_heads, q.device), _stream()), "paged_attention_mfma")
    else:
        f = _fn("attention_mfma.hip", "pllm_paged_attention_mfma", defines, _ATTN_SIG)
        _check(f(*args, _stream()), "paged_attention_mfma")
    return out


PROMPT_TILE_COLUMNS = 128   # query columns (queries x heads per kv head) of one workgroup of the prompt kernel
_upload_buffers: dict = {}


def _upload_ints(values: np.ndarray, device) -> torch.Tensor:
    """int32 values to the device without stalling the host: through a pinned buffer (allocated once per
    device) and a copy on the current stream.  A copy from pageable memory would hold the host until the
    stream has caught up, and the kernels of the layers before could then no longer be issued ahead."""
    key = str(device)
    pinned, copied = _upload_buffers.get(key, (None, None))
    if pinned is None or pinned.numel() < values.size:
        pinned, copied = torch.empty(max(values.size, 1 << 14), dtype=torch.int32, pin_memory=True), torch.cuda.Event()
        _upload_buffers[key] = (pinned, copied)
    else:
        copied.synchronize()                                   # the last upload has left the buffer
    staged = pinned[:values.size].view(values.shape)
    staged.copy_(torch.from_numpy(np.ascontiguousarray(values, dtype=np.int32)))
    out = torch.empty(values.shape, dtype=torch.int32, device=device)
    out.copy_(staged, non_blocking=True)
    copied.record()
    return out


def prompt_tiles(q_lens: list, k_lens: list, first_seq: int, group: int, capacity: int | None = None) -> np.ndarray | None:
    """Host side of the prompt kernel's work list for the sequences from ``first_seq`` on: int32 [n, 2] pairs
    (sequence counted from ``first_seq``, tile of PROMPT_TILE_COLUMNS query columns), the tiles that see the most
    keys first.  Without ``capacity``: None when the sequences are all alike (the kernel's own grid then does the
    same).  With ``capacity``: always a list, of exactly that many pairs, the unused ones (-1, -1)."""
    counts = [-(-n * group // PROMPT_TILE_COLUMNS) for n in q_lens[first_seq:]]
    if capacity is None and len(set(counts)) == 1 and len(set(k_lens[first_seq:])) == 1:
        return None
    seqs, tiles, keys = [], [], []
    for i, n in enumerate(counts):
        s = first_seq + i
        t = np.arange(n, dtype=np.int64)
        seqs.append(np.full(n, i, dtype=np.int64))
        tiles.append(t)
        keys.append(k_lens[s] - q_lens[s] + (t + 1) * PROMPT_TILE_COLUMNS // group)
    seqs, tiles, keys = np.concatenate(seqs), np.concatenate(tiles), np.concatenate(keys)
    order = np.argsort(-keys, kind="stable")
    pairs = np.stack([seqs[order], tiles[order]], axis=1).astype(np.int32)
    if capacity is not None:
        _need(pairs.shape[0] <= capacity, f"{pairs.shape[0]} prompt tiles for a list of {capacity}")
        pairs = np.concatenate([pairs, np.full((capacity - pairs.shape[0], 2), -1, dtype=np.int32)])
    return pairs


def prompt_tiles_capacity(num_sequences: int, tokens: int, group: int) -> int:
    """Most pairs ``prompt_tiles`` can give for ``num_sequences`` sequences that share ``tokens`` tokens."""
    return -(-tokens * group // PROMPT_TILE_COLUMNS) + num_sequences


def prompt_work_list(ctx, first_seq: int, group: int) -> torch.Tensor | None:
    """The prompt kernel's work for the sequences from ``first_seq`` on (``prompt_tiles``) on the device.
    Workgroups take the pairs in order, so long pieces start first and none is launched for a tile that a shorter
    sequence does not have (with one long and many short sequences most of a rectangular grid is empty, and
    handing out empty workgroups was measured at 80 us for 3,800 of them).  Built from the host lengths once per
    step and kept in the context; None when the sequences are all alike and the kernel's own grid does the same."""
    cache = getattr(ctx, "launch_cache", None)
    key = ("prompt_tiles", first_seq, group)
    if cache is not None and key in cache:
        return cache[key]
    pairs = prompt_tiles(ctx.q_lens, ctx.k_lens, first_seq, group)
    work = None
    if pairs is not None and 0 < pairs.shape[0] <= 65535:
        work = _upload_ints(pairs, ctx.device)
    if cache is not None:
        cache[key] = work
    return work


_compute_units: dict = {}


def _num_compute_units(device) -> int:
    key = str(device)
    if key not in _compute_units:
        _compute_units[key] = torch.cuda.get_device_properties(device).multi_processor_count
    return _compute_units[key]


PROMPT_PARTITION_MIN_KEYS = 512   # a partition of the prompt kernel holds at least this many keys (four steps of 128)


def prompt_partitions(num_tiles: int, num_kv_heads: int, max_k_len: int, compute_units: int) -> tuple[int, int]:
    """(partition_size, num_partitions) for a launch of the prompt kernel with ``num_tiles`` tiles of query columns
    (all sequences together) whose longest context is ``max_k_len``; (0, 1): no partitions.

    A workgroup walks its tile's keys one step of 128 after the other (about 1.9 us a step at head size 64), so a
    prompt portion of a few hundred tokens behind a long context is a few dozen workgroups that run for a long time
    on a GPU of 256 compute units: 256 tokens at context 2048 took 30 us.  The keys are then cut into as many
    aligned partitions as it takes to give every compute unit a workgroup, each at least PROMPT_PARTITION_MIN_KEYS
    long, and a second kernel merges the partitions (about 5 us)."""
    workgroups = max(1, num_tiles * num_kv_heads)
    parts = min(compute_units // workgroups, max_k_len // PROMPT_PARTITION_MIN_KEYS)
    if parts < 2:
        return 0, 1
    size = -(-max_k_len // parts)
    size = (size + 127) // 128 * 128
    return size, -(-max_k_len // size)


FEW_QUERY_COLUMNS = 64      # queries x heads per kv head that one tile of the decode kernel holds
SPLIT_FROM_CONTEXT_TIMES_HEAD = 160_000   # context x head size of a few-query sequence from which two launches pay


def paged_attention(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads, head_dim,
                    scale, window, ctx, terms: ScoreTerms | None = None, weights: KeyWeights | None = None) -> torch.Tensor:
    """Attention of one step's queries over the paged cache: the MFMA kernels for bfloat16 where they
    take the shape, else the plain kernel.  ``ctx`` gives host-side lengths for launch decisions.

    A step that holds decoded tokens beside prompt portions is one launch of the prompt kernel, in which a decoded
    token is a tile of its own that one workgroup walks through its whole context; when such a context is long
    (13 us per 1024 keys at head size 64, 34 us at 128) the step is launched in two parts instead, if the sequences
    with few queries come first in the batch (the step function orders them so): those go to the kernel that cuts
    their keys into partitions, the portions to the prompt kernel (a portion of 512 tokens beside 7 decoded tokens
    at context 8192: 109 us in one launch, 36 us in two; at context 1024: 19 us and 24 us)."""
    bs = k_pages.shape[2]
    if weights is not None and weights.sigmoid and mfma_attention_takes(q.dtype, num_heads, num_kv_heads, head_dim, bs) and q.stride(0) % 8 == 0:
        return sigmoid_attention(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads, head_dim, scale,
                                 window, weights, terms, ctx.max_q_len)
    if weights is not None and weights.any():
        return paged_attention_generic(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads, head_dim,
                                       scale, window, terms=terms, weights=weights)
    if mfma_attention_takes(q.dtype, num_heads, num_kv_heads, head_dim, bs) and q.stride(0) % 8 == 0:
        group = num_heads // num_kv_heads
        lds = _max_lds_bytes(q.device)
        layout = getattr(ctx, "graph_layout", None)
        if ctx.capturing and layout is not None:
            # A step with prompt portions that is replayed from a graph: the launches depend on the layout's counts
            # and the context bound only.  The single-token rows go to the kernel that cuts their keys into
            # partitions, the portions to the prompt kernel with the work list the step function has put there.
            few = layout.num_single_rows
            work = ctx.launch_cache.get(("prompt_tiles", few, group))
            _need(work is not None, "a replayed step with prompt portions needs the prompt kernel's work list in the context")
            work = work.view(-1, 2)
            out = torch.empty((q.shape[0], num_heads * head_dim), dtype=q.dtype, device=q.device)
            if few:
                waves, size, parts = attention_plan(few, num_kv_heads, 1, ctx.max_k_len, group, head_dim, lds, _num_compute_units(q.device))
                paged_attention_mfma(q[:few], k_pages, v_pages, block_tables[:few], cu_seqlens_q[:few + 1], seq_lens_k[:few],
                                     num_heads, num_kv_heads, head_dim, scale, window, 1, size, parts, waves,
                                     2 if waves == 1 else 0, out=out[:few], terms=terms)
            prompt_q = max(layout.portion_tokens, FEW_QUERY_COLUMNS // group + 1)     # enough columns for the prompt kernel's form
            psize, pparts = prompt_partitions(work.shape[0], num_kv_heads, layout.portion_context, _num_compute_units(q.device))
            paged_attention_mfma(q, k_pages, v_pages, block_tables[few:], cu_seqlens_q[few:], seq_lens_k[few:], num_heads,
                                 num_kv_heads, head_dim, scale, window, prompt_q, psize, pparts, 1, 2, out=out, work_list=work, terms=terms,
                                 single_prompt=layout.num_portions == 2)      # (one portion and the padding sequence)
            return out
        q_lens, k_lens = ctx.q_lens, ctx.k_lens
        few = 0
        while few < len(q_lens) and q_lens[few] * group <= FEW_QUERY_COLUMNS:
            few += 1
        if (0 < few < len(q_lens) and max(k_lens[:few]) * head_dim >= SPLIT_FROM_CONTEXT_TIMES_HEAD and not ctx.capturing
                and all(n * group > FEW_QUERY_COLUMNS for n in q_lens[few:])):
            rows = sum(q_lens[:few])
            out = torch.empty((q.shape[0], num_heads * head_dim), dtype=q.dtype, device=q.device)
            max_q, max_k = max(q_lens[:few]), max(k_lens[:few])
            waves, size, parts = attention_plan(few, num_kv_heads, max_q, max_k, group, head_dim, lds, _num_compute_units(q.device))
            paged_attention_mfma(q[:rows], k_pages, v_pages, block_tables[:few], cu_seqlens_q[:few + 1], seq_lens_k[:few],
                                 num_heads, num_kv_heads, head_dim, scale, window, max_q, size, parts, waves,
                                 2 if waves == 1 else 0, out=out[:rows], terms=terms)
            # the portions: rows, cu_seqlens_q and the output stay absolute, the per-sequence arrays start at `few`
            psize, pparts = prompt_partitions(sum(-(-n * group // PROMPT_TILE_COLUMNS) for n in q_lens[few:]), num_kv_heads,
                                              max(k_lens[few:]), _num_compute_units(q.device))
            paged_attention_mfma(q, k_pages, v_pages, block_tables[few:], cu_seqlens_q[few:], seq_lens_k[few:], num_heads,
                                 num_kv_heads, head_dim, scale, window, max(q_lens[few:]), psize, pparts, 1, 2, out=out,
                                 work_list=prompt_work_list(ctx, few, group), terms=terms)
            return out
        waves, size, parts = attention_plan(ctx.num_seqs, num_kv_heads, ctx.max_q_len, ctx.max_k_len, group, head_dim, lds,
                                            _num_compute_units(q.device))
        # Prompt portions: 32 columns per wavefront leave registers for two wavefronts per SIMD
        # (measured faster than 64 columns at one).
        prompt = waves == 1 and ctx.max_q_len * group > FEW_QUERY_COLUMNS and not ctx.capturing
        if prompt:
            size, parts = prompt_partitions(sum(-(-n * group // PROMPT_TILE_COLUMNS) for n in q_lens), num_kv_heads, ctx.max_k_len,
                                            _num_compute_units(q.device))
        return paged_attention_mfma(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads,
                                    head_dim, scale, window, ctx.max_q_len, size, parts, waves, 2 if waves == 1 else 0,
                                    work_list=prompt_work_list(ctx, 0, group) if prompt else None, terms=terms)
    if q.dtype == torch.bfloat16 and not _warned_plain_attention:
        _warned_plain_attention.append(True)
        log.warning("bfloat16 attention with pages of %d positions, head size %d, %d/%d heads runs on the plain kernel (one "
                    "wavefront per token and head): the matrix-core kernels take pages of at least 16 positions, head sizes "
                    "16..256 in steps of 16 and groups of at most 64 heads", bs, head_dim, num_heads, num_kv_heads)
    return paged_attention_generic(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads,
                                   num_kv_heads, head_dim, scale, window, terms=terms)


def sigmoid_attention_plan(columns: int, head_dim: int, work_items: int = 1) -> tuple:
    """(tiles of 16 columns per workgroup, wavefronts that share them and deal the key blocks, whether the next block is asked for
    ahead) for a launch whose sequences have up to ``columns`` (query, head) pairs per kv head; ``work_items``: sequences times
    kv heads.  Measured at head size 64, 32 heads on 4 key heads, a window of 1,024: a prompt of 2,048 tokens 85 us with one
    wavefront per 32 columns (90 with two, 100 with four; 101 with tiles of 16 columns; asking for the next block ahead costs
    registers and gains nothing: 102 to 125); a prompt of 512 tokens 29 / 23 / 17.5 us with one / two / four wavefronts (too few
    workgroups to fill the GPU otherwise); one decoded token at context 2,048: 14 us with eight wavefronts, 22 with four."""
    if columns <= 16:
        return (1, 8 if head_dim <= 128 else 4, False)              # decoding: one tile, the keys split over the wavefronts
    ncb = 2 if head_dim <= 64 else 1
    workgroups = -(-columns // (16 * ncb)) * max(1, work_items)
    waves = 4 if workgroups <= 768 else (2 if workgroups <= 1536 else 1)
    while waves > 1 and waves * ncb * head_dim * 64 > 64 * 1024:            # (the wavefronts' outputs meet in LDS: 64 bytes a wavefront, column tile and channel)
        waves //= 2
    return (ncb, waves, False)


def sigmoid_attention(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads: int, num_kv_heads: int, head_dim: int,
                      scale: float, window: int, weights: KeyWeights, terms: ScoreTerms | None, max_q_len: int,
                      plan: tuple | None = None) -> torch.Tensor:
    """Attention without a softmax on the matrix cores (bfloat16): a visible key weighs sigmoid(cap(scale q . k) + head_bias),
    not normalised; visible are the last ``window`` positions (0: all) and the sequence's first ``weights.keep_first``.
    ``max_q_len`` bounds the queries of one sequence of the step (the launch covers that many per sequence)."""
    S, bs = _check_attention_args(q, k_pages, v_pages, block_tables, cu_seqlens_q, seq_lens_k, num_heads, num_kv_heads, head_dim)
    weights.checked(num_heads, int(window or 0), q.device)
    _need(q.dtype == torch.bfloat16 and window >= 0 and max_q_len > 0, "sigmoid attention on the matrix cores: bfloat16, a window or none")
    _need(terms is None or (terms.slopes is None and terms.sinks is None), "sigmoid weights take a cap of the scores and no other term")
    T = q.shape[0]
    out = torch.empty((T, num_heads * head_dim), dtype=q.dtype, device=q.device)
    ncb, waves, two = plan or sigmoid_attention_plan(max_q_len * (num_heads // num_kv_heads), head_dim, S * num_kv_heads)
    sig = [c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_float,
           c_int, c_int, c_float, c_void_p, c_int, c_int, c_int, c_void_p]
    _check(_fn("attention_sigmoid.hip", "pllm_sigmoid_attention", {"HEAD_DIM": head_dim}, signature=sig)(
        _ptr(q), q.stride(0), _ptr(k_pages), _ptr(v_pages), _ptr(out), out.stride(0), _ptr(block_tables), block_tables.stride(0),
        _ptr(cu_seqlens_q), _ptr(seq_lens_k), S, int(max_q_len), num_heads, num_kv_heads, bs, c_float(scale), int(window or 0),
        weights.keep_first, c_float(terms.cap if terms is not None else 0.0), _ptr(weights.head_bias), ncb, waves, int(two), _stream()),
        "sigmoid_attention")
    return out


# ------------------------------------------------------------------------------------------- a residual stream kept in float
def embed_scaled(ids: torch.Tensor, table: torch.Tensor, scale: float, want_rows: bool = True, kept: torch.Tensor | None = None):
    """(x, rows): x[t] = float(table[ids[t]]) * scale as float32 [T, hidden], and the same rounded to the table's type
    (None for a float32 table, whose x already is the rows, or when ``want_rows`` is False).  ``kept`` (contiguous float32
    [T, hidden]) receives a second copy of x."""
    _on_gpu(ids, table, kept)
    _need(ids.dtype == torch.int32 and ids.dim() == 1 and ids.is_contiguous(), "ids must be contiguous int32 [T]")
    _need(table.dim() == 2 and table.is_contiguous(), "embedding table must be contiguous [vocab, hidden]")
    T, (V, H) = ids.numel(), table.shape
    x = torch.empty((T, H), dtype=torch.float32, device=table.device)
    rows = torch.empty((T, H), dtype=table.dtype, device=table.device) if want_rows and table.dtype != torch.float32 else None
    _need(kept is None or (kept.dtype == torch.float32 and kept.shape == (T, H) and kept.is_contiguous()), f"kept: contiguous float32 [{T}, {H}]")
    sig = [c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_float, c_void_p]
    _check(_fn("float_stream.hip", "pllm_embed_scaled", signature=sig)(dtype_code(table.dtype), _ptr(ids), _ptr(table), _ptr(x), _ptr(rows), _ptr(kept),
                                                                      T, H, V, c_float(scale), _stream()), "embed_scaled")
    return x, rows


def embed_bigram(ids: torch.Tensor, table: torch.Tensor, pairs: torch.Tensor, scale: float, buckets: int, mul_prev: int, mul_cur: int,
                 state: torch.Tensor, state_slots: torch.Tensor, seq_starts: torch.Tensor, cu_seqlens: torch.Tensor, num_seqs: int,
                 pair_rows: torch.Tensor, move_state: bool = True) -> torch.Tensor:
    """float32 [T, hidden]: x[t] = float(table[ids[t]]) * scale + float(pairs[row(t)]) with row(t) = (token before * mul_prev +
    ids[t] * mul_cur) mod buckets, or ``buckets`` for a sequence's first token.  The token before a step's first token of a
    sequence is ``state[slot, 0]`` (int32 [slots, 1]; none when seq_starts == 0), where every sequence leaves its last token
    of this step.  ``pair_rows`` int32 [T] receives the rows; with ``move_state`` False it is read instead (a second
    gather of the same step) and the state stays as it is."""
    _on_gpu(ids, table, pairs, state, state_slots, seq_starts, cu_seqlens, pair_rows)
    _need(ids.dtype == torch.int32 and ids.dim() == 1 and ids.is_contiguous(), "ids must be contiguous int32 [T]")
    T, (V, H) = ids.numel(), table.shape
    _need(table.dim() == 2 and table.is_contiguous(), "embedding table must be contiguous [vocab, hidden]")
    _need(pairs.shape == (buckets + 1, H) and pairs.is_contiguous() and pairs.dtype == table.dtype, f"bigram table: [{buckets + 1}, {H}] of the token table's type")
    _need(state.dtype == torch.int32 and state.dim() == 2 and state.is_contiguous(), "the last tokens' state is contiguous int32 [slots, 1]")
    for t, n, what in ((state_slots, num_seqs, "state_slots"), (seq_starts, num_seqs, "seq_starts"), (cu_seqlens, num_seqs + 1, "cu_seqlens")):
        _need(t.dtype == torch.int32 and t.dim() == 1 and t.is_contiguous() and t.numel() == n, f"{what} must be contiguous int32 [{n}]")
    _need(pair_rows.dtype == torch.int32 and pair_rows.numel() == T and pair_rows.is_contiguous(), "pair_rows: int32 [T]")
    _need(0 < buckets and abs(mul_prev) < 2 ** 31 and abs(mul_cur) < 2 ** 31, "bigram hash: buckets > 0 and 32-bit multipliers")
    x = torch.empty((T, H), dtype=torch.float32, device=table.device)
    sig = [c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_long, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int,
           c_int, c_int, c_int, c_float, c_int, c_void_p]
    _check(_fn("float_stream.hip", "pllm_embed_bigram", signature=sig)(
        dtype_code(table.dtype), _ptr(ids), _ptr(cu_seqlens), _ptr(seq_starts), _ptr(state_slots), _ptr(state), state.stride(0), _ptr(pair_rows),
        _ptr(table), _ptr(pairs), _ptr(x), T, num_seqs, H, V, buckets, mul_prev, mul_cur, c_float(scale), int(bool(move_state)), _stream()),
        "embed_bigram")
    return x


def layernorm_sum_takes(hidden: int, top: int) -> bool:
    return bool(_fn("float_stream.hip", "pllm_layernorm_sum_takes", signature=[c_int, c_int])(hidden, top))


def _layernorm_of_sum(branch: "ChoiceSum", weight, bias, eps, stream_rows, out_dtype) -> torch.Tensor | None:
    """The layer norm of a sum of experts' rows that the norm's kernel forms itself, added to the stream."""
    rows, H = stream_rows.shape
    e, h, rp, wt = branch.checked(rows, H)
    _on_gpu(weight, bias, stream_rows)
    for t, what in ((weight, "weight"), (bias, "bias")):
        _need(t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous(), f"layer norm {what} must be float32 [{H}]")
    _need(stream_rows.dtype == torch.float32 and stream_rows.is_contiguous(), f"the stream must be contiguous float32 [{rows}, {H}]")
    out = torch.empty((rows, H), dtype=out_dtype, device=stream_rows.device) if out_dtype is not None else None
    sig = [c_int, c_int, c_void_p, c_void_p, c_long, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_int, c_int, c_void_p]
    _check(_fn("float_stream.hip", "pllm_layernorm_sum", signature=sig)(
        dtype_code(out_dtype or torch.float32), dtype_code(h.dtype), _ptr(e), _ptr(h), h.stride(0), _ptr(rp), _ptr(wt), wt.shape[1],
        _ptr(weight), _ptr(bias), c_float(eps), _ptr(stream_rows), _ptr(out), rows, H, _stream()), "layernorm_sum")
    return out


def layernorm(v: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, eps: float, stream_rows: torch.Tensor | None = None,
              row_index: torch.Tensor | None = None, out_dtype: torch.dtype | None = None) -> torch.Tensor | None:
    """y = (v - mean) / sqrt(var + eps) * weight + bias over each row of ``v`` (float32 or bfloat16), in float.

    With ``stream_rows`` (float32, as many rows as are normed): stream_rows += y in place, and the return value is the
    new stream rounded to ``out_dtype`` (None when ``out_dtype`` is None).  Without it the return value is y in
    ``out_dtype``.  ``row_index`` (int32) picks the rows of ``v`` that are normed.  With a stream ``v`` may be a ``ChoiceSum``
    (a weighted sum of experts' rows), which the kernel forms itself where it takes the sizes."""
    if isinstance(v, ChoiceSum):
        _need(stream_rows is not None and row_index is None, "a sum of experts' rows is a branch that enters the stream")
        if v.plain and layernorm_sum_takes(stream_rows.shape[1], v.weights.shape[1]):
            return _layernorm_of_sum(v, weight, bias, eps, stream_rows, out_dtype)
        v = v.rows()
    _on_gpu(v, weight, bias, stream_rows, row_index)
    _need(v.dim() == 2 and v.is_contiguous(), "layernorm input must be contiguous [rows, hidden]")
    H = v.shape[1]
    for t, what in ((weight, "weight"), (bias, "bias")):
        _need(t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous(), f"layer norm {what} must be float32 [{H}]")
    _need((H + 16) * 4 <= min(_max_lds_bytes(v.device), 160 * 1024), f"the layer norm kernel stages one row in LDS: hidden size {H} is above its limit")
    rows = v.shape[0]
    if row_index is not None:
        _need(row_index.dtype == torch.int32 and row_index.dim() == 1 and row_index.is_contiguous(), "row_index must be contiguous int32")
        rows = row_index.numel()
    if stream_rows is not None:
        _need(stream_rows.dtype == torch.float32 and stream_rows.shape == (rows, H) and stream_rows.is_contiguous(),
              f"the stream must be contiguous float32 [{rows}, {H}]")
    else:
        _need(out_dtype is not None, "layernorm without a stream returns rows: say their type")
    out = torch.empty((rows, H), dtype=out_dtype, device=v.device) if out_dtype is not None else None
    sig = [c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_int, c_int, c_void_p]
    _check(_fn("float_stream.hip", "pllm_layernorm", signature=sig)(
        dtype_code(v.dtype), dtype_code(out_dtype or torch.float32), _ptr(v), _ptr(row_index), _ptr(weight), _ptr(bias), c_float(eps),
        _ptr(stream_rows), _ptr(out), rows, H, _stream()), "layernorm")
    return out


def round_rows(x: torch.Tensor) -> torch.Tensor:
    """float32 rows rounded to bfloat16 (the operand of a bfloat16 product read from a float stream)."""
    _on_gpu(x)
    _need(x.dtype == torch.float32 and x.is_contiguous(), "round_rows takes contiguous float32 rows")
    out = torch.empty(x.shape, dtype=torch.bfloat16, device=x.device)
    _check(_fn("float_stream.hip", "pllm_round_rows", signature=[c_void_p, c_void_p, c_long, c_void_p])(_ptr(x), _ptr(out), x.numel(), _stream()),
           "round_rows")
    return out


# ------------------------------------------------------------------------------------------- per-head products
class HeadMatrices:
    """One matrix per head, [heads, N, K] as a checkpoint stores them, in the order ``gemm_heads`` reads: float32 as they are (the plain
    kernel takes rows of K), bfloat16 with N innermost, [heads, K, N] contiguous.  (The vendor's batched bfloat16 product has
    faulted on this hardware with a transposed view as its right operand: it is only ever given a contiguous one.)"""

    __slots__ = ("data", "heads", "out_features", "in_features")

    def __init__(self, w: torch.Tensor):
        _need(w.dim() == 3 and w.dtype in _DTYPE_CODE, "head matrices: [heads, N, K], float32 or bfloat16")
        self.heads, self.out_features, self.in_features = w.shape
        self.data = (w.transpose(1, 2) if w.dtype == torch.bfloat16 else w).contiguous()


def gemm_heads(a: torch.Tensor, w: HeadMatrices, out: torch.Tensor | None = None) -> torch.Tensor:
    """out[t, h, :] = w[h] a[t, h, :] for a [T, heads, K] (a view into wider rows is fine: unit inner stride, any row and
    head strides) and w one [N, K] matrix per head; float accumulation.  Returns [T, heads, N], contiguous
    unless ``out`` (a view of the same freedom) is given."""
    _on_gpu(a, w.data, out)
    _need(a.dim() == 3 and a.shape[1] == w.heads and a.shape[2] == w.in_features and a.dtype == w.data.dtype,
          f"gemm_heads shapes {tuple(a.shape)} {a.dtype} x {w.heads} of [{w.out_features}, {w.in_features}] {w.data.dtype}")
    _need(a.stride(2) == 1, "gemm_heads: unit inner stride of the rows")
    T, heads, K = a.shape
    N = w.out_features
    if out is None:
        out = torch.empty((T, heads, N), dtype=a.dtype, device=a.device)
    _need(out.shape == (T, heads, N) and out.stride(2) == 1 and out.dtype == a.dtype, "bad output for gemm_heads")
    if a.dtype == torch.bfloat16:
        # bfloat16: the vendor's batched product (as the other bfloat16 products of more than a few rows), straight into
        # the output's rows through views with the heads in front
        torch.bmm(a.transpose(0, 1), w.data, out=out.transpose(0, 1))
        return out
    sig = [c_int, c_int, c_void_p, c_int, c_long, c_void_p, c_int, c_long, c_void_p, c_int, c_long, c_int, c_int, c_int, c_int, c_void_p]
    _check(_fn("gemm_generic.hip", "pllm_gemm_nt_batched", signature=sig)(
        dtype_code(a.dtype), dtype_code(out.dtype), _ptr(a), a.stride(0), a.stride(1), _ptr(w.data), K, N * K, _ptr(out), out.stride(0), out.stride(1),
        T, N, K, heads, _stream()), "gemm_heads")
    return out


# ------------------------------------------------------------------------------------------- state of fixed size per request
MAX_CONV_TAPS = 16


def _check_sequences(state: torch.Tensor, state_slots, seq_starts, cu_seqlens, num_seqs: int) -> None:
    _need(state.dtype == torch.float32 and state.dim() == 2 and state.is_contiguous(), "a state tensor is contiguous float32 [slots, size]")
    for t, n, what in ((state_slots, num_seqs, "state_slots"), (seq_starts, num_seqs, "seq_starts"), (cu_seqlens, num_seqs + 1, "cu_seqlens")):
        _need(t.dtype == torch.int32 and t.dim() == 1 and t.is_contiguous() and t.numel() == n, f"{what} must be contiguous int32 [{n}]")


def causal_conv(rows: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor | None, state: torch.Tensor, state_offset: int,
                state_slots: torch.Tensor, seq_starts: torch.Tensor, cu_seqlens: torch.Tensor, num_seqs: int, max_q_len: int,
                activation: str | None = "silu") -> torch.Tensor:
    """Causal convolution per channel over each sequence's rows, then SiLU: rows [T, channels] (a view with unit inner
    stride), weight float32 [channels, taps] (its last column meets the current token), bias float32 [channels].  The
    last taps - 1 inputs of every sequence are read from and left in ``state[slot, state_offset : state_offset +
    channels * (taps - 1)]``; a sequence with seq_starts == 0 starts from zeros.  The host guarantees slots < state.shape[0]."""
    _on_gpu(rows, weight, bias, state, state_slots, seq_starts, cu_seqlens)
    _need(rows.dim() == 2 and rows.stride(1) == 1, "causal_conv rows: [T, channels] with unit inner stride")
    T, C = rows.shape
    taps = weight.shape[1]
    _need(weight.dtype == torch.float32 and weight.shape == (C, taps) and weight.is_contiguous() and 1 <= taps <= MAX_CONV_TAPS,
          f"conv weight: float32 [{C}, taps <= {MAX_CONV_TAPS}]")
    _need(bias is None or (bias.dtype == torch.float32 and bias.shape == (C,) and bias.is_contiguous()), f"conv bias: float32 [{C}]")
    _need(activation in (None, "silu"), "causal_conv applies SiLU or nothing")
    _check_sequences(state, state_slots, seq_starts, cu_seqlens, num_seqs)
    _need(0 <= state_offset and state_offset + C * (taps - 1) <= state.shape[1], "the convolution's inputs do not fit the state slot")
    out = torch.empty((T, C), dtype=rows.dtype, device=rows.device)
    sig = [c_int, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_long, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int,
           c_int, c_int, c_void_p]
    _check(_fn("recurrent.hip", "pllm_causal_conv", signature=sig)(
        dtype_code(rows.dtype), _ptr(rows), rows.stride(0), _ptr(weight), _ptr(bias), state.data_ptr() + 4 * state_offset, state.stride(0),
        _ptr(state_slots), _ptr(seq_starts), _ptr(cu_seqlens), _ptr(out), C, C, taps, 1 if activation else 0, num_seqs, max_q_len, _stream()),
        "causal_conv")
    return out


def rotary_to_float(rows: torch.Tensor, positions: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor, heads: int, head_dim: int,
                    rot_dims: int, interleaved: bool, scale: float = 1.0, second_at: int | None = None, scale2: float = 1.0) -> torch.Tensor:
    """float32 [T, heads, head_dim]: the heads of ``rows`` [T, >= heads * head_dim] (unit inner stride) with their first
    ``rot_dims`` elements turned by the tables' angles at ``positions``, times ``scale``.  With ``second_at``: float32
    [2, T, heads, head_dim], the second set of heads being the one that starts ``second_at`` columns further in the rows,
    times ``scale2`` (queries and keys of one product's rows in one launch)."""
    _on_gpu(rows, positions, cos, sin)
    sets = 1 if second_at is None else 2
    _need(rows.dim() == 2 and rows.stride(1) == 1 and rows.shape[1] >= (second_at or 0) + heads * head_dim, "rotary_to_float rows: [T, >= heads * head_dim]")
    T = rows.shape[0]
    _need(positions.dtype == torch.int32 and positions.numel() == T and positions.is_contiguous(), "positions: int32 [T]")
    _need(rot_dims % 2 == 0 and 0 <= rot_dims <= head_dim, f"rotated width {rot_dims} of a head of {head_dim}")
    for t in (cos, sin):
        _need(t.dtype == torch.float32 and t.dim() == 2 and t.shape[1] == rot_dims // 2 and t.is_contiguous(),
              f"rotary tables: float32 [positions, {rot_dims // 2}]")
    out = torch.empty((sets, T, heads, head_dim), dtype=torch.float32, device=rows.device)
    sig = [c_int, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_float, c_int, c_int, c_long,
           c_float, c_void_p]
    _check(_fn("recurrent.hip", "pllm_rotary_to_float", signature=sig)(
        dtype_code(rows.dtype), _ptr(rows), rows.stride(0), _ptr(positions), _ptr(cos), _ptr(sin), _ptr(out), T, heads, head_dim, rot_dims,
        1 if interleaved else 0, c_float(scale), sets, second_at or 0, T * heads * head_dim, c_float(scale2), _stream()), "rotary_to_float")
    return out if sets == 2 else out[0]


def step_sizes(raw: torch.Tensor, bias: torch.Tensor, a_log: torch.Tensor) -> tuple:
    """(dt, decay), float32 [T, heads]: dt = softplus(raw + bias), decay = exp(-exp(a_log) * dt); raw [T, heads] a view."""
    _on_gpu(raw, bias, a_log)
    _need(raw.dim() == 2 and raw.stride(1) == 1, "step_sizes raw: [T, heads] with unit inner stride")
    T, H = raw.shape
    for t in (bias, a_log):
        _need(t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous(), f"step_sizes: float32 [{H}] per-head constants")
    dt = torch.empty((T, H), dtype=torch.float32, device=raw.device)
    decay = torch.empty((T, H), dtype=torch.float32, device=raw.device)
    sig = [c_int, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p]
    _check(_fn("recurrent.hip", "pllm_step_sizes", signature=sig)(dtype_code(raw.dtype), _ptr(raw), raw.stride(0), _ptr(bias), _ptr(a_log),
                                                                  _ptr(dt), _ptr(decay), T, H, _stream()), "step_sizes")
    return dt, decay


RECURRENCE_CHUNKS_FROM = 128      # tokens of the longest sequence of a step from which its recurrences run in chunks


def recurrence_chunk(max_q_len: int, num_tokens: int) -> int:
    """Tokens per chunk for a step's recurrences (0: every sequence token by token in one workgroup per head).  Chunks
    spread a long portion over the GPU at the price of a workspace of one state per chunk, so they grow with the step."""
    if max_q_len < RECURRENCE_CHUNKS_FROM:
        return 0
    # (short steps: more, shorter chunks, or most of the GPU stays idle.  Measured at width 2,048, a prompt of 256 / 512 /
    #  1,024 / 2,048 tokens in ms: chunks of 16: 2.39 / 3.09 / 4.73 / 8.46; of 32: 2.54 / 3.09 / 4.34 / 7.29; of 64: 3.11 /
    #  3.55 / 4.65 / 6.92; of 128: 4.60 / 4.81 / 5.71 / 7.80)
    for limit, chunk in ((384, 16), (1536, 32), (4096, 64), (16384, 128)):
        if num_tokens <= limit:
            return chunk
    return 256


def linear_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, state: torch.Tensor, state_offset: int,
                      state_slots: torch.Tensor, seq_starts: torch.Tensor, cu_seqlens: torch.Tensor, num_seqs: int,
                      vscale: torch.Tensor | None = None, skip: torch.Tensor | None = None, max_q_len: int = 0,
                      step_sizes: tuple | None = None, normaliser: bool = False, row_decay: torch.Tensor | None = None) -> torch.Tensor:
    """Per head:  S_t = decay_t S_(t-1) + k_t (vscale_t v_t)^T,   y_t = S_t^T q_t + skip v_t,   S [N, P] float32 at
    ``state[slot, state_offset + head * N * P :]``; a sequence with seq_starts == 0 starts from S = 0.

    q, k [T, key_heads, N] (views of one element type and one row stride, unit inner stride, heads side by side; head h
    uses key head h // (heads / key_heads)), v [T, heads, P] likewise, decay float32 [T, heads] or [heads] (one number
    per head for all tokens), vscale float32 [T, heads] or None, skip float32 [heads] or None.  Returns y float32 [T, heads * P].
    ``step_sizes`` = (raw [T, heads] view with unit inner stride, bias float32 [heads], a_log float32 [heads]) in place of
    ``decay`` (None) and ``vscale``: the kernel makes vscale_t = softplus(raw_t + bias) and decay_t = exp(-exp(a_log) vscale_t) itself.
    ``normaliser``: S has one more column, P + 1, whose value is 1 at every token (it holds n_t = decay_t n_(t-1) + vscale_t k_t);
    the state then takes heads * N * (P + 1) floats and y is [T, heads * (P + 1)] with n_t . q_t in every head's last column.
    ``row_decay`` float32 [T, heads, N] (a view, heads side by side, unit inner stride) in place of ``decay`` (None): a decay per
    row of S, S_t = diag(row_decay_t) S_(t-1) + k_t (vscale_t v_t)^T (every head then has its own keys).
    ``max_q_len``: a bound on the tokens of one sequence in this step (0: unknown); from ``RECURRENCE_CHUNKS_FROM`` on the
    sequences are cut into chunks that run side by side (a chunk's own contribution from a zero state, the states carried
    from chunk to chunk, the outputs from each chunk's true starting state), which rounds differently than token by token."""
    _on_gpu(q, k, v, decay, state, state_slots, seq_starts, cu_seqlens, vscale, skip)
    _need(q.dim() == 3 and q.shape == k.shape and q.dtype == k.dtype and q.stride() == k.stride() and q.stride(2) == 1
          and q.stride(1) == q.shape[2], "recurrence q, k: [T, key_heads, N] views of one layout with the heads side by side")
    _need(v.dim() == 3 and v.stride(2) == 1 and v.stride(1) == v.shape[2] and v.shape[0] == q.shape[0], "recurrence v: [T, heads, P], heads side by side")
    T, KH, N = q.shape
    H, v_cols = v.shape[1], v.shape[2]
    P = v_cols + 1 if normaliser else v_cols
    _need(H % KH == 0 and 1 <= N <= 1024, f"{H} heads over {KH} key heads, N = {N} (at most 1024)")
    raw = raw_bias = a_log = None
    if step_sizes is not None:
        raw, raw_bias, a_log = step_sizes
        _on_gpu(raw, raw_bias, a_log)
        _need(decay is None and vscale is None, "step sizes take the place of decay and vscale")
        _need(raw.shape == (T, H) and raw.stride(1) == 1, f"raw step sizes: [{T}, {H}] with unit inner stride")
        for t in (raw_bias, a_log):
            _need(t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous(), f"step sizes: float32 [{H}] per-head constants")
    elif row_decay is not None:
        _on_gpu(row_decay)
        _need(decay is None and KH == H, "a decay per row takes the place of the decay per head, and every head has its own keys")
        _need(row_decay.dtype == torch.float32 and tuple(row_decay.shape) == (T, H, N) and row_decay.stride(2) == 1 and row_decay.stride(1) == N,
              f"row_decay: float32 [{T}, {H}, {N}] with the heads side by side")
    else:
        _need(decay.dtype == torch.float32 and decay.is_contiguous() and tuple(decay.shape) in ((T, H), (H,)), f"decay: float32 [{T}, {H}] or [{H}]")
    _need(vscale is None or (vscale.dtype == torch.float32 and vscale.shape == (T, H) and vscale.is_contiguous()), f"vscale: float32 [{T}, {H}]")
    _need(skip is None or (skip.dtype == torch.float32 and skip.shape == (H,) and skip.is_contiguous()), f"skip: float32 [{H}]")
    _check_sequences(state, state_slots, seq_starts, cu_seqlens, num_seqs)
    _need(0 <= state_offset and state_offset + H * N * P <= state.shape[1], "the recurrence's state does not fit the state slot")
    out = torch.empty((T, H * P), dtype=torch.float32, device=v.device)
    chunk = recurrence_chunk(max_q_len, T)
    max_chunks = T // chunk + num_seqs if chunk else 0
    ws_state = torch.empty((max_chunks, H * N * P), dtype=torch.float32, device=v.device) if chunk else None
    ws_decay = torch.empty((max_chunks, H * (N if row_decay is not None else 1)), dtype=torch.float32, device=v.device) if chunk else None
    sig = [c_void_p, c_void_p, c_int, c_int, c_void_p, c_int, c_int, c_void_p, c_int, c_void_p, c_int, c_void_p, c_void_p,
           c_void_p, c_int, c_int, c_void_p, c_void_p,
           c_void_p, c_long, c_void_p, c_void_p,
           c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p]
    _check(_fn("recurrent.hip", "pllm_linear_recurrence", signature=sig)(
        _ptr(q), _ptr(k), dtype_code(q.dtype), q.stride(0), _ptr(v), dtype_code(v.dtype), v.stride(0), _ptr(decay),
        H if decay is not None and decay.dim() == 2 else 0, _ptr(row_decay), row_decay.stride(0) if row_decay is not None else 0,
        _ptr(vscale), _ptr(skip),
        _ptr(raw), dtype_code(raw.dtype) if raw is not None else 0, raw.stride(0) if raw is not None else 0, _ptr(raw_bias), _ptr(a_log),
        state.data_ptr() + 4 * state_offset, state.stride(0), _ptr(state_slots), _ptr(seq_starts), _ptr(cu_seqlens),
        _ptr(out), num_seqs, H, KH, N, P, v_cols, chunk, max_chunks, _ptr(ws_state), _ptr(ws_decay), _stream()), "linear_recurrence")
    return out


SCAN_STATE_MAX = 512              # state elements per channel that the selective scan takes


def scan_state_size(n: int) -> int:
    """The number of state elements per channel that the selective scan holds for a state of n: 8, 16 or a multiple of 32
    (what is padded has A = B = C = 0 and stays zero)."""
    return 8 if n <= 8 else 16 if n <= 16 else -(-n // 32) * 32


def scan_chunk(max_q_len: int, num_tokens: int, channels: int) -> int:
    """Tokens per chunk of the selective scan (0: every sequence token by token)."""
    if max_q_len < SCAN_CHUNKS_FROM:
        return 0
    for limit, chunk in ((1024, 16), (4096, 32), (16384, 64)):
        if num_tokens <= limit:
            return chunk
    return 128


SCAN_CHUNKS_FROM = 128            # tokens of the longest sequence of a step from which its scans run in chunks


def selective_scan(x: torch.Tensor, raw_dt: torch.Tensor, dt_bias: torch.Tensor, bc: torch.Tensor, a2: torch.Tensor, skip: torch.Tensor,
                   z: torch.Tensor, state: torch.Tensor, state_slots: torch.Tensor, seq_starts: torch.Tensor, cu_seqlens: torch.Tensor,
                   num_seqs: int, max_q_len: int = 0) -> torch.Tensor:
    """s_c <- e^(dt_c A_c) * s_c + (dt_c x_c) B for the N states of channel c,  y_c = <s_c, C> + skip_c x_c,  out = y silu(z), with
    dt = softplus(raw_dt + dt_bias).  x, z [T, channels] (views of one type, unit inner stride), raw_dt contiguous float32
    [T, channels], bc [T, 2 N] of x's type (a view: B, then C; rows on 4-byte boundaries), a2 float32 [N, channels] = A log2(e) transposed, N as
    ``scan_state_size`` gives it; S float32 [N, channels] in front of ``state[slot]``; a sequence with seq_starts == 0 starts
    from S = 0.  Returns [T, channels] in x's type.  From ``SCAN_CHUNKS_FROM`` tokens of one sequence on (``max_q_len``) the
    sequences run in chunks side by side, which rounds differently than token by token."""
    _on_gpu(x, raw_dt, dt_bias, bc, a2, skip, z, state, state_slots, seq_starts, cu_seqlens)
    T, C = x.shape
    N = a2.shape[0]
    _need(x.stride(1) == 1 and z.shape == (T, C) and z.stride(1) == 1 and z.dtype == x.dtype, "selective_scan x, z: [T, channels] of one type, unit inner stride")
    _need(raw_dt.dtype == torch.float32 and raw_dt.shape == (T, C) and raw_dt.is_contiguous(), f"raw_dt: contiguous float32 [{T}, {C}]")
    _need(scan_state_size(N) == N and N <= SCAN_STATE_MAX, f"a state of {N} per channel: 8, 16 or a multiple of 32 up to {SCAN_STATE_MAX}")
    _need(bc.dtype == x.dtype and bc.shape == (T, 2 * N) and bc.stride(1) == 1 and bc.data_ptr() % 4 == 0 and bc.stride(0) * bc.element_size() % 4 == 0,
          f"bc: [{T}, {2 * N}] of x's type with unit inner stride, rows on 4-byte boundaries")
    _need(a2.dtype == torch.float32 and a2.shape == (N, C) and a2.is_contiguous(), f"a2: float32 [{N}, {C}]")
    for t, what in ((dt_bias, "dt_bias"), (skip, "skip")):
        _need(t.dtype == torch.float32 and t.shape == (C,) and t.is_contiguous(), f"{what}: float32 [{C}]")
    _check_sequences(state, state_slots, seq_starts, cu_seqlens, num_seqs)
    _need(N * C <= state.shape[1], "the scan's state does not fit the state slot")
    out = torch.empty((T, C), dtype=x.dtype, device=x.device)
    chunk = scan_chunk(max_q_len, T, C)
    max_chunks = T // chunk + num_seqs if chunk else 0
    ws_state = torch.empty((max_chunks, N * C), dtype=torch.float32, device=x.device) if chunk else None
    ws_steps = torch.empty((max_chunks, C), dtype=torch.float32, device=x.device) if chunk else None
    dt = torch.empty((T, C), dtype=torch.float32, device=x.device) if chunk else None
    if chunk and bc.dtype != torch.float32:
        bc = activate_rows(bc, None, out_dtype=torch.float32)          # (the same numbers: the passes over chunks read them as float)
    sig = [c_int, c_void_p, c_long, c_void_p, c_void_p, c_void_p, c_void_p, c_long, c_void_p, c_void_p, c_void_p, c_long, c_void_p, c_long,
           c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p]
    _check(_fn("selective_scan.hip", "pllm_selective_scan", signature=sig)(
        dtype_code(x.dtype), _ptr(x), x.stride(0), _ptr(raw_dt), _ptr(dt), _ptr(dt_bias), _ptr(bc), bc.stride(0), _ptr(a2), _ptr(skip), _ptr(z),
        z.stride(0), _ptr(state), state.stride(0), _ptr(state_slots), _ptr(seq_starts), _ptr(cu_seqlens), _ptr(out), num_seqs, C, N, chunk,
        max_chunks, _ptr(ws_state), _ptr(ws_steps), _stream()), "selective_scan")
    return out


DELTA_MAX_DIM = 256               # size of a head that the delta memory takes
DELTA_CHUNK = 32                  # tokens that its kernels for long portions work off as matrices
DELTA_CHUNK_MAX_DIM = 128         # ... for heads up to this size
DELTA_CHUNKS_FROM = 48            # tokens of the longest sequence of a step from which those kernels run


def delta_rule(rows: torch.Tensor, columns: dict, raw_w: torch.Tensor, w0: torch.Tensor, bias_a: torch.Tensor, weight: torch.Tensor, eps: float,
               heads: int, dim: int, state: torch.Tensor, state_slots: torch.Tensor, seq_starts: torch.Tensor, cu_seqlens: torch.Tensor,
               num_seqs: int, max_q_len: int = 0) -> torch.Tensor:
    """A matrix memory per head: u = k / sqrt(sum(k^2) + 1e-6), w = exp(-exp(-1/2) sigmoid(raw_w + w0)), a = sigmoid(raw_a +
    bias_a), z = S^T u, S <- w . S - (a . u) z^T + k v^T (w . S: row by row), o = S^T r; then per head o / sqrt(mean(o^2) + eps) *
    weight * sigmoid(gate).  ``rows`` [T, ...] holds r, k, v, raw_a and the gate, heads * dim columns each, from the columns
    ``columns`` = {"r", "k", "v", "a", "g"} on (unit inner stride); raw_w float32 [T, heads * dim]; w0, bias_a, weight float32
    [heads * dim].  S float32 [heads, dim, dim] in front of ``state[slot]``; a sequence with seq_starts == 0 starts from
    S = 0.  Returns [T, heads * dim] in the rows' type.  From ``DELTA_CHUNKS_FROM`` tokens of one sequence on (``max_q_len``) the
    sequences are worked off in chunks of ``DELTA_CHUNK`` tokens as matrix products in float, which round differently than
    token by token."""
    _on_gpu(rows, raw_w, w0, bias_a, weight, state, state_slots, seq_starts, cu_seqlens)
    T, C = rows.shape[0], heads * dim
    _need(rows.dim() == 2 and rows.stride(1) == 1 and all(0 <= columns[n] and columns[n] + C <= rows.shape[1] for n in "rkvag"),
          f"delta_rule rows: five parts of {C} columns with unit inner stride")
    _need(0 < dim <= DELTA_MAX_DIM, f"heads of {dim}: at most {DELTA_MAX_DIM}")
    _need(raw_w.dtype == torch.float32 and raw_w.shape == (T, C) and raw_w.stride(1) == 1, f"raw_w: float32 [{T}, {C}]")
    for t, what in ((w0, "w0"), (bias_a, "bias_a"), (weight, "weight")):
        _need(t.dtype == torch.float32 and t.shape == (C,) and t.is_contiguous(), f"{what}: float32 [{C}]")
    _check_sequences(state, state_slots, seq_starts, cu_seqlens, num_seqs)
    _need(heads * dim * dim <= state.shape[1], "the memory does not fit the state slot")
    if max_q_len >= DELTA_CHUNKS_FROM and dim <= DELTA_CHUNK_MAX_DIM:
        max_chunks = T // DELTA_CHUNK + num_seqs
        per_chunk = _fn("delta_rule.hip", "pllm_delta_chunk_floats", signature=[c_int, c_int])(heads, dim)
        ws = torch.empty(max_chunks * per_chunk, dtype=torch.float32, device=rows.device)
        y = torch.empty((T, C), dtype=torch.float32, device=rows.device)
        sig = [c_int, c_void_p, c_long, c_int, c_int, c_int, c_int, c_void_p, c_long, c_void_p, c_void_p, c_void_p, c_long, c_void_p, c_void_p,
               c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_void_p, c_void_p]
        _check(_fn("delta_rule.hip", "pllm_delta_rule_chunks", signature=sig)(
            dtype_code(rows.dtype), _ptr(rows), rows.stride(0), columns["r"], columns["k"], columns["v"], columns["a"], _ptr(raw_w), raw_w.stride(0),
            _ptr(w0), _ptr(bias_a), _ptr(state), state.stride(0), _ptr(state_slots), _ptr(seq_starts), _ptr(cu_seqlens), _ptr(y), num_seqs, heads,
            dim, max_chunks, _ptr(ws), _stream()), "delta_rule_chunks")
        return gated_group_norm(y, rows[:, columns["g"]:columns["g"] + C], weight, dim, False, eps, gate_activation="sigmoid")
    out = torch.empty((T, C), dtype=rows.dtype, device=rows.device)
    sig = [c_int, c_void_p, c_long, c_int, c_int, c_int, c_int, c_int, c_void_p, c_long, c_void_p, c_void_p, c_void_p, c_float, c_void_p,
           c_long, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_void_p]
    _check(_fn("delta_rule.hip", "pllm_delta_rule", signature=sig)(
        dtype_code(rows.dtype), _ptr(rows), rows.stride(0), columns["r"], columns["k"], columns["v"], columns["a"], columns["g"], _ptr(raw_w),
        raw_w.stride(0), _ptr(w0), _ptr(bias_a), _ptr(weight), c_float(eps), _ptr(state), state.stride(0), _ptr(state_slots), _ptr(seq_starts),
        _ptr(cu_seqlens), _ptr(out), num_seqs, heads, dim, _stream()), "delta_rule")
    return out


GATE_ACTIVATIONS = {"silu": 0, "sigmoid": 1, None: 2}


def gated_group_norm(y: torch.Tensor, gate: torch.Tensor | None, weight: torch.Tensor | None, group: int, gate_first: bool, eps: float,
                     gate_activation: str | None = "silu", out_dtype: torch.dtype | None = None) -> torch.Tensor:
    """Behind a recurrence: y float32 [T, inner], gate [T, inner] (a view, unit inner stride) in the compute type, which is
    also the result's.  ``gate_first``: u = y act(gate), u / sqrt(mean(u^2) + eps) * weight over groups of ``group``
    channels; else y / sqrt(mean(y^2) + eps) * act(gate) (* weight when given).  act(z) is z sigmoid(z) ("silu"), sigmoid(z)
    ("sigmoid"), or 1 (``gate_activation`` None: ``gate`` is None too, and ``out_dtype`` names the result's type)."""
    _on_gpu(y, gate, weight)
    _need(y.dtype == torch.float32 and y.dim() == 2 and y.is_contiguous(), "gated_group_norm y: contiguous float32 [T, inner]")
    T, inner = y.shape
    _need(gate_activation in GATE_ACTIVATIONS, f"gate_activation: one of {tuple(GATE_ACTIVATIONS)}")
    if gate is None:
        _need(gate_activation is None and out_dtype is not None, "without a gate: no gate activation, and the result's type is named")
        return _group_norm_launch(y, None, 0, out_dtype, weight, group, gate_first, eps, 2)
    _need(gate_activation is not None, "a gate has an activation")
    _need(gate.shape == (T, inner) and gate.stride(1) == 1, f"gate: [{T}, {inner}] with unit inner stride")
    return _group_norm_launch(y, gate, gate.stride(0), gate.dtype, weight, group, gate_first, eps, GATE_ACTIVATIONS[gate_activation])


def _group_norm_launch(y, gate, gate_stride, dtype, weight, group, gate_first, eps, act):
    T, inner = y.shape
    _need(group > 0 and inner % group == 0, f"{inner} channels in groups of {group}")
    _need(weight is None or (weight.dtype == torch.float32 and weight.shape == (inner,) and weight.is_contiguous()), f"weight: float32 [{inner}]")
    out = torch.empty((T, inner), dtype=dtype, device=y.device)
    sig = [c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_float, c_void_p]
    _check(_fn("recurrent.hip", "pllm_gated_group_norm", signature=sig)(
        dtype_code(dtype), _ptr(y), _ptr(gate), gate_stride, _ptr(weight), _ptr(out), T, inner, group, 1 if gate_first else 0, act,
        c_float(eps), _stream()), "gated_group_norm")
    return out


def silu_to_float(rows: torch.Tensor, cols: int) -> torch.Tensor:
    """float32 [T, cols]: silu of the first ``cols`` columns of ``rows`` (a view with unit inner stride, either element type):
    activated operands of a recurrence, which stay in float from here on."""
    _on_gpu(rows)
    _need(rows.dim() == 2 and rows.stride(1) == 1 and 0 < cols <= rows.shape[1], f"silu_to_float rows: [T, >= {cols}] with unit inner stride")
    out = torch.empty((rows.shape[0], cols), dtype=torch.float32, device=rows.device)
    _check(_fn("recurrent.hip", "pllm_silu_to_float", signature=[c_void_p, c_int, c_int, c_void_p, c_int, c_int, c_void_p])(
        _ptr(rows), dtype_code(rows.dtype), rows.stride(0), _ptr(out), rows.shape[0], cols, _stream()), "silu_to_float")
    return out


def bounded_forget_gates(rows: torch.Tensor, bias: torch.Tensor | None, lower: torch.Tensor | None, channels: int) -> torch.Tensor:
    """float32 [3, T, channels] = (q, k, f) from ``rows`` [T, >= 2 channels] laid out [raw_q | raw_f | ...] (a view, either element
    type): q = silu(raw_q), f = lower + (1 - lower) sigmoid(raw_f + bias), k = 1 - f; ``bias`` and ``lower`` float32 [channels]."""
    _on_gpu(rows, bias, lower)
    _need(rows.dim() == 2 and rows.stride(1) == 1 and rows.shape[1] >= 2 * channels > 0, f"forget gates' rows: [T, >= {2 * channels}]")
    for t, what in ((bias, "bias"), (lower, "lower")):
        _need(t is None or (t.dtype == torch.float32 and t.shape == (channels,) and t.is_contiguous()), f"{what}: float32 [{channels}]")
    out = torch.empty((3, rows.shape[0], channels), dtype=torch.float32, device=rows.device)
    _check(_fn("recurrent.hip", "pllm_bounded_forget_gates", signature=[c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p])(
        _ptr(rows), dtype_code(rows.dtype), rows.stride(0), _ptr(bias), _ptr(lower), _ptr(out), rows.shape[0], channels, _stream()),
        "bounded_forget_gates")
    return out


def mlstm_gates(raw_i: torch.Tensor, raw_f: torch.Tensor, bias_i: torch.Tensor | None, bias_f: torch.Tensor | None, cap: float,
                state: torch.Tensor, m_at: int, state_slots: torch.Tensor, seq_starts: torch.Tensor, cu_seqlens: torch.Tensor,
                num_seqs: int) -> tuple:
    """Log-domain gates of a matrix memory under a running maximum, per sequence and head, in float:
    i = cap tanh((raw_i + bias_i) / cap), f = logsigmoid(cap tanh((raw_f + bias_f) / cap)) (cap 0: no cap),
    m_t = max(f_t + m_(t-1), i_t) with m = 0 in front of a sequence's first token (``seq_starts`` == 0) and else what
    ``state[slot, m_at + head]`` holds, where the last m is left.  Returns (decay, take, m), float32 [T, heads]:
    exp(f_t + m_(t-1) - m_t), exp(i_t - m_t), m_t.  raw_i, raw_f: [T, heads] views of one type and row stride."""
    _on_gpu(raw_i, raw_f, bias_i, bias_f, state, state_slots, seq_starts, cu_seqlens)
    _need(raw_i.dim() == 2 and raw_i.shape == raw_f.shape and raw_i.stride() == raw_f.stride() and raw_i.stride(1) == 1
          and raw_i.dtype == raw_f.dtype, "mlstm_gates: raw_i and raw_f are [T, heads] views of one layout")
    T, H = raw_i.shape
    for t in (bias_i, bias_f):
        _need(t is None or (t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous()), f"gate biases: float32 [{H}]")
    _check_sequences(state, state_slots, seq_starts, cu_seqlens, num_seqs)
    _need(0 <= m_at and m_at + H <= state.shape[1], "the running maxima do not fit the state slot")
    decay, take, m = (torch.empty((T, H), dtype=torch.float32, device=raw_i.device) for _ in range(3))
    sig = [c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p, c_float, c_void_p, c_long, c_int, c_void_p, c_void_p, c_void_p,
           c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p]
    _check(_fn("recurrent.hip", "pllm_mlstm_gates", signature=sig)(
        _ptr(raw_i), _ptr(raw_f), dtype_code(raw_i.dtype), raw_i.stride(0), _ptr(bias_i), _ptr(bias_f), c_float(cap), _ptr(state),
        state.stride(0), m_at, _ptr(state_slots), _ptr(seq_starts), _ptr(cu_seqlens), _ptr(decay), _ptr(take), _ptr(m), num_seqs, H,
        _stream()), "mlstm_gates")
    return decay, take, m


def mlstm_output(y: torch.Tensor, m: torch.Tensor, gate: torch.Tensor, weight: torch.Tensor | None, heads: int, P: int, qscale: float,
                 eps: float, out_dtype: torch.dtype) -> torch.Tensor:
    """Behind ``linear_recurrence(..., normaliser=True)``: y float32 [T, heads * (P + 1)], m float32 [T, heads], gate
    [T, heads * P] (a view, unit inner stride).  Per head o = y[:P] qscale / (max(|y[P] qscale|, exp(-m)) + 1e-6), then
    o / sqrt(mean(o^2) + eps) * weight * sigmoid(gate), as ``out_dtype`` [T, heads * P]."""
    _on_gpu(y, m, gate, weight)
    T = y.shape[0]
    _need(y.dtype == torch.float32 and y.shape == (T, heads * (P + 1)) and y.is_contiguous(), f"mlstm_output y: float32 [T, {heads * (P + 1)}]")
    _need(m.dtype == torch.float32 and m.shape == (T, heads) and m.is_contiguous(), f"m: float32 [{T}, {heads}]")
    _need(gate.shape == (T, heads * P) and gate.stride(1) == 1, f"gate: [{T}, {heads * P}] with unit inner stride")
    _need(weight is None or (weight.dtype == torch.float32 and weight.shape == (heads * P,) and weight.is_contiguous()), f"weight: float32 [{heads * P}]")
    out = torch.empty((T, heads * P), dtype=out_dtype, device=y.device)
    sig = [c_int, c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_float, c_float, c_void_p]
    _check(_fn("recurrent.hip", "pllm_mlstm_output", signature=sig)(
        dtype_code(out_dtype), _ptr(y), _ptr(m), _ptr(gate), dtype_code(gate.dtype), gate.stride(0), _ptr(weight), _ptr(out), T, heads, P,
        c_float(qscale), c_float(eps), _stream()), "mlstm_output")
    return out


# ------------------------------------------------------------------------------------------- attention over a latent
MAX_LATENT_RANK, MAX_LATENT_ROT = 1024, 256


def latent_prepare(rows: torch.Tensor, down_at: int, positions: torch.Tensor, cos: torch.Tensor | None, sin: torch.Tensor | None, norm_weight: torch.Tensor,
                   eps: float, slots: torch.Tensor | None, k_pages: torch.Tensor, v_pages: torch.Tensor | None, q_out: torch.Tensor,
                   heads: int, plain: int, rot: int, rank: int, interleaved: bool, q_latent: tuple | None = None) -> torch.Tensor | None:
    """From ``rows`` [T, heads x (plain | rot) | rank | rot] (the down-projection at column ``down_at``): the latent
    c = rms_norm(rows[down_at : down_at + rank]) * norm_weight and the key part behind it, turned by the tables' angles at
    ``positions``, go to the token's slot of ``k_pages`` [pages, 1, block, width] as the row [c | key part | 0], and c
    also to ``v_pages`` [pages, 1, width, block] (transposed inside the page) when given; no write for slot -1 or when
    ``slots`` is None.  Every head's rotated rot part goes to ``q_out`` [T, heads, width] at columns rank .. rank + rot,
    zeros behind it (columns 0 .. rank are left alone: the query's latent-space part belongs there).  ``rot`` 0: a latent
    without a rotated part (no tables then; the rows need not hold the queries).  ``rows`` are of the pages' type or float32
    (the sums of the product that made them).  ``q_latent`` = (column, q_rank, weight float32 [q_rank]): the rows also hold
    a latent of the queries at that column; its RMS norm (the same eps) times the weight is returned in the pages' type,
    [T, q_rank], the operand of the product that expands it into the heads' queries."""
    _on_gpu(rows, positions, cos, sin, norm_weight, slots, k_pages, v_pages, q_out)
    _need(rows.dim() == 2 and rows.stride(1) == 1 and rows.shape[1] >= down_at + rank + rot and (rot == 0 or down_at >= heads * (plain + rot)),
          "latent_prepare rows: [T, heads * (plain + rot) + rank + rot]")
    _need(rows.dtype in (k_pages.dtype, torch.float32), "latent_prepare rows: of the pages' type, or float32")
    T = rows.shape[0]
    _need(rot >= 0 and rot % 2 == 0 and rank > 0, f"rot {rot} (even), rank {rank}")
    _need(positions.dtype == torch.int32 and positions.numel() == T and positions.is_contiguous(), "positions: int32 [T]")
    for t in (cos, sin) if rot else ():
        _need(t is not None and t.dtype == torch.float32 and t.dim() == 2 and t.shape[1] == rot // 2 and t.is_contiguous(),
              f"rotary tables: float32 [positions, {rot // 2}]")
    _need(norm_weight.dtype == torch.float32 and norm_weight.shape == (rank,) and norm_weight.is_contiguous(), f"latent norm weight: float32 [{rank}]")
    _need(slots is None or (slots.dtype == torch.int32 and slots.numel() == T and slots.is_contiguous()), "slots: int32 [T]")
    _need(k_pages.dim() == 4 and k_pages.shape[1] == 1 and k_pages.is_contiguous(), "k_pages: [pages, 1, block, width]")
    pages, _, bs, width = k_pages.shape
    _need(width >= rank + rot, f"pages of width {width} for a latent of {rank} + {rot}")
    _need(v_pages is None or (v_pages.shape == (pages, 1, width, bs) and v_pages.is_contiguous() and v_pages.dtype == k_pages.dtype),
          f"v_pages: [{pages}, 1, {width}, {bs}]")
    _need(q_out.shape == (T, heads, width) and q_out.is_contiguous() and q_out.dtype == k_pages.dtype, f"q_out: contiguous [{T}, {heads}, {width}]")
    q_at = q_rank = 0
    q_w = cq = None
    if q_latent is not None:
        q_at, q_rank, q_w = q_latent
        _on_gpu(q_w)
        _need(q_rank > 0 and 0 <= q_at and q_at + q_rank <= rows.shape[1] and q_w.dtype == torch.float32 and q_w.shape == (q_rank,) and q_w.is_contiguous(),
              f"the queries' latent: {q_rank} columns at {q_at} with a float32 weight")
        cq = torch.empty((T, q_rank), dtype=k_pages.dtype, device=rows.device)
    sig = [c_int, c_int, c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int,
           c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p]
    _check(_fn("latent_attention.hip", "pllm_latent_prepare", signature=sig)(
        dtype_code(k_pages.dtype), dtype_code(rows.dtype), _ptr(rows), rows.stride(0), down_at, _ptr(positions), _ptr(cos) if rot else None, _ptr(sin) if rot else None, _ptr(norm_weight), c_float(eps),
        _ptr(slots), _ptr(k_pages), _ptr(v_pages), _ptr(q_out), T, heads, plain, rot, rank, width, bs, 1 if interleaved else 0,
        q_at, q_rank, _ptr(q_w), _ptr(cq), _stream()), "latent_prepare")
    return cq


def latent_attention(q: torch.Tensor, rank: int, rot: int, k_pages: torch.Tensor, block_tables: torch.Tensor, cu_seqlens_q: torch.Tensor,
                     seq_lens_k: torch.Tensor, scale: float, window: int, sinks: torch.Tensor | None = None) -> torch.Tensor:
    """softmax(q . key_n * scale) over the visible keys n (causal; the last ``window`` positions when window > 0), times
    c_n, the first ``rank`` elements of key row n: [T, heads, rank].  q [T, heads, width] contiguous rows [qa | q_rot | 0],
    k_pages [pages, 1, block, width] rows [c | key part | 0].  ``sinks`` (float32 [heads]): a logit per head that takes part in the
    softmax's sum and in nothing else.  For latents wider than the paged attention kernels take."""
    ScoreTerms(0.0, None, sinks).checked(q.shape[1], q.device)
    _on_gpu(q, k_pages, block_tables, cu_seqlens_q, seq_lens_k)
    _need(q.dim() == 3 and q.is_contiguous() and k_pages.dtype == q.dtype, "latent_attention: contiguous q [T, heads, width] of the pages' type")
    T, heads, width = q.shape
    _need(rank <= MAX_LATENT_RANK and rot <= MAX_LATENT_ROT and rank + rot <= width, f"latent sizes up to {MAX_LATENT_RANK} + {MAX_LATENT_ROT}")
    _need(k_pages.dim() == 4 and k_pages.shape[1] == 1 and k_pages.shape[3] == width and k_pages.is_contiguous(), f"k_pages: [pages, 1, block, {width}]")
    S = seq_lens_k.numel()
    _need(block_tables.dtype == torch.int32 and block_tables.dim() == 2 and block_tables.shape[0] == S and block_tables.stride(1) == 1,
          "block_tables: int32 [S, pages per sequence]")
    _need(cu_seqlens_q.dtype == torch.int32 and cu_seqlens_q.numel() == S + 1 and seq_lens_k.dtype == torch.int32, "lengths: int32")
    out = torch.empty((T, heads, rank), dtype=q.dtype, device=q.device)
    sig = [c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_float,
           c_int, c_void_p, c_void_p]
    _check(_fn("latent_attention.hip", "pllm_latent_attention", signature=sig)(
        dtype_code(q.dtype), _ptr(q), _ptr(k_pages), _ptr(out), _ptr(block_tables), block_tables.stride(0), _ptr(cu_seqlens_q),
        _ptr(seq_lens_k), S, T, heads, rank, rot, width, k_pages.shape[2], c_float(scale), window, _ptr(sinks), _stream()), "latent_attention")
    return out


# ------------------------------------------------------------------------------------------- norms on both sides of a branch
SANDWICH_HELD_MAX = 4096      # rows that the norm-add-norm kernel holds in registers


class ChoiceSum:
    """The result of routed experts before its last step: per token the sum, over its choices in order, of weight times
    the pair's row of ``expert_out`` (float32 [pairs, width]) or, where ``row_of_pair`` is -1, the token's own row of
    ``h``.  ``rows()`` forms it (``moe_combine``); ``rms_sandwich`` takes it as a branch and forms it in its own kernel."""

    def __init__(self, expert_out: torch.Tensor, h: torch.Tensor, row_of_pair: torch.Tensor, weights: torch.Tensor,
                 weights_inside: bool = False, shared: torch.Tensor | None = None, shared_gate: torch.Tensor | None = None):
        self.expert_out, self.h, self.row_of_pair, self.weights = expert_out, h, row_of_pair, weights
        # (as ``moe_combine`` takes them: weights that went into the experts' inputs, a feed-forward that every token passes)
        self.weights_inside, self.shared, self.shared_gate = bool(weights_inside), shared, shared_gate

    @property
    def plain(self) -> bool:
        """Whether the sum is the weighted sum of the choices and nothing else."""
        return not self.weights_inside and self.shared is None

    def rows(self) -> torch.Tensor:
        return moe_combine(self.expert_out, self.h, self.row_of_pair, self.weights, self.weights_inside, self.shared, self.shared_gate)

    def checked(self, rows: int, width: int):
        e, h, rp, wt = self.expert_out, self.h, self.row_of_pair, self.weights
        _on_gpu(e, h, rp, wt)
        _need(wt.dtype == torch.float32 and wt.dim() == 2 and wt.shape[0] == rows and wt.is_contiguous(), "weights: float32 [rows, top]")
        top = wt.shape[1]
        _need(e.dtype == torch.float32 and e.shape == (rows * top, width) and e.is_contiguous(), f"expert outputs: float32 [{rows * top}, {width}]")
        _need(h.dim() == 2 and h.shape == (rows, width) and h.stride(1) == 1 and h.dtype in (torch.float32, torch.bfloat16), "the tokens' rows: [rows, width]")
        _need(rp.dtype == torch.int32 and rp.numel() == rows * top and rp.is_contiguous(), "row_of_pair: int32 [rows * top]")
        return e, h, rp, wt


class WeightedPair:
    """A branch that is the weighted sum of two, first_scale * first + second_scale * second (contiguous float32 rows of one
    shape: two mixers side by side), which the kernel that adds the branch to the stream forms where it reads it
    (``rms_sandwich``).  ``rows()`` forms it for any other reader."""

    __slots__ = ("first", "first_scale", "second", "second_scale")

    def __init__(self, first: torch.Tensor, first_scale: float, second: torch.Tensor, second_scale: float):
        self.first, self.first_scale, self.second, self.second_scale = first, float(first_scale), second, float(second_scale)

    def rows(self) -> torch.Tensor:
        return scaled_sum(self.first, self.first_scale, self.second, self.second_scale)


class DepthSum:
    """A weighted sum over the depth of the model that takes a layer's result r: history[n - 1] = r, and the stream becomes
    sum over j < n - 1 of weights[j] history[j] + weights[n - 1] r.  ``history`` float32 [>= n, T, hidden] (contiguous; planes
    0 .. n - 2 filled: the embedding's output and the results of the layers before), ``weights`` float32 [n]."""

    def __init__(self, history: torch.Tensor, weights: torch.Tensor):
        self.history, self.weights = history, weights

    def checked(self, rows: int, width: int):
        h, w = self.history, self.weights
        _on_gpu(h, w)
        _need(w.dtype == torch.float32 and w.dim() == 1 and w.numel() >= 2 and w.is_contiguous(), "depth weights: float32 [n >= 2]")
        _need(h.dtype == torch.float32 and h.dim() == 3 and h.shape[0] >= w.numel() and tuple(h.shape[1:]) == (rows, width) and h.is_contiguous(),
              f"the history is contiguous float32 [>= {w.numel()}, {rows}, {width}]")
        return h, w, w.numel() - 1


def depth_sum(stream: torch.Tensor, depth: DepthSum) -> None:
    """The sum over the depth on its own: the stream (float32 [rows, hidden]) is the layer's result, and becomes the sum."""
    _on_gpu(stream)
    _need(stream.dtype == torch.float32 and stream.dim() == 2 and stream.is_contiguous(), "the stream is contiguous float32 [rows, hidden]")
    h, w, count = depth.checked(*stream.shape)
    _check(_fn("float_stream.hip", "pllm_depth_sum", signature=[c_void_p, c_void_p, c_long, c_void_p, c_int, c_long, c_void_p])(
        _ptr(stream), _ptr(h), h.stride(0), _ptr(w), count, stream.numel(), _stream()), "depth_sum")


def _rms_depth(stream, branch, depth: DepthSum, w_branch, mult, eps, w_next, out, out_dtype, bias):
    rows, H = stream.shape
    if H > SANDWICH_HELD_MAX or (isinstance(branch, ChoiceSum) and not branch.plain) or isinstance(branch, WeightedPair):
        # (rows too long for the kernel that holds them in registers, or a branch with further terms: one kernel after the other)
        rms_sandwich(stream, branch, w_branch, mult, eps, bias=bias)
        depth_sum(stream, depth)
        return rms_sandwich(stream, None, None, 0.0, eps, w_next=w_next, out=out, out_dtype=out_dtype) if out is not None or out_dtype is not None else None
    _on_gpu(stream, None if isinstance(branch, ChoiceSum) else branch, w_branch, w_next, out, bias)
    _need(stream.dtype == torch.float32 and stream.is_contiguous(), "the stream is contiguous float32 [rows, hidden]")
    for t, what in ((w_branch, "w_branch"), (w_next, "w_next"), (bias, "bias")):
        _need(t is None or (t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous()), f"{what} must be float32 [{H}]")
    hist, dw, count = depth.checked(rows, H)
    if out is None and out_dtype is not None:
        out = torch.empty((rows, H), dtype=out_dtype, device=stream.device)
    _need(out is None or (out.dim() == 2 and out.shape == (rows, H) and out.stride(1) == 1), f"the rows' output is [{rows}, {H}] with unit inner stride")
    e = h = rp = wt = None
    if isinstance(branch, ChoiceSum):
        e, h, rp, wt = branch.checked(rows, H)
        branch = None
    else:
        _need(branch.dtype == torch.float32 and branch.shape == stream.shape and branch.is_contiguous(), "a branch is contiguous float32 rows like the stream")
    sig = [c_int, c_int, c_void_p, c_void_p, c_void_p, c_long, c_void_p, c_void_p, c_int, c_void_p, c_long, c_void_p, c_int, c_void_p, c_void_p,
           c_float, c_void_p, c_void_p, c_float, c_void_p, c_long, c_int, c_int, c_void_p]
    _check(_fn("float_stream.hip", "pllm_rms_depth", signature=sig)(
        dtype_code(out.dtype) if out is not None else F32, dtype_code(h.dtype) if h is not None else F32, _ptr(branch), _ptr(e), _ptr(h),
        h.stride(0) if h is not None else 0, _ptr(rp), _ptr(wt), wt.shape[1] if wt is not None else 0, _ptr(hist), hist.stride(0), _ptr(dw), count,
        _ptr(bias), _ptr(w_branch), c_float(mult), _ptr(stream), _ptr(w_next), c_float(eps), _ptr(out), out.stride(0) if out is not None else 0,
        rows, H, _stream()), "rms_depth")
    return out


def rms_sandwich(stream: torch.Tensor, branch: torch.Tensor | None, w_branch: torch.Tensor | None, mult: float, eps: float,
                 w_next: torch.Tensor | None = None, out: torch.Tensor | None = None, out_dtype: torch.dtype | None = None,
                 bias: torch.Tensor | None = None, row_index: torch.Tensor | None = None, depth: DepthSum | None = None) -> torch.Tensor | None:
    """RMS norms around a float32 residual stream, all in float.  With ``branch`` (float32 rows like the stream, or a
    ``ChoiceSum``: a weighted sum of experts' rows that the kernel forms itself):
    stream += mult * rms_norm(branch + bias) * w_branch, in place (``w_branch`` None with float32 rows: stream += mult *
    (branch + bias), the branch as it is: the sum of a pre-norm block).  Then, when ``out`` or ``out_dtype`` is given, the
    rows of the stream as it is now are returned in that type: normed and times ``w_next``, or as they are when
    ``w_next`` is None.  ``out`` may be a view with a row stride of its own (unit inner stride).  Without a branch
    ``row_index`` (int32) picks the rows of the stream; nothing is written to the stream then.  ``depth``: between the branch's
    sum and the rows a ``DepthSum`` takes the stream."""
    if depth is not None:
        _need(branch is not None and row_index is None, "a sum over the depth stands behind a branch, and no rows are picked")
        return _rms_depth(stream, branch, depth, w_branch, mult, eps, w_next, out, out_dtype, bias)
    if isinstance(branch, WeightedPair):
        return _rms_sandwich_pair(stream, branch, w_branch, mult, eps, w_next, out, out_dtype, bias, row_index)
    _on_gpu(stream, None if isinstance(branch, ChoiceSum) else branch, w_branch, w_next, out, bias, row_index)
    _need(stream.dtype == torch.float32 and stream.dim() == 2 and stream.is_contiguous(), "the stream is contiguous float32 [rows, hidden]")
    rows, H = stream.shape
    _need((H + 16) * 4 <= min(_max_lds_bytes(stream.device), 160 * 1024), f"the norm kernel stages one row in LDS: hidden size {H} is above its limit")
    for t, what in ((w_branch, "w_branch"), (w_next, "w_next"), (bias, "bias")):
        _need(t is None or (t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous()), f"{what} must be float32 [{H}]")
    if isinstance(branch, ChoiceSum):
        if H > SANDWICH_HELD_MAX or not branch.plain:
            branch = branch.rows()                          # (rows too long for the kernel that holds them in registers, or a sum with further terms)
        else:
            _need(row_index is None and w_branch is not None, "a branch comes with its norm's weight, and no rows are picked")
            if out is None and out_dtype is not None:
                out = torch.empty((rows, H), dtype=out_dtype, device=stream.device)
            if out is not None:
                _need(out.dim() == 2 and out.shape == (rows, H) and out.stride(1) == 1, f"the rows' output is [{rows}, {H}] with unit inner stride")
            e, h, rp, wt = branch.checked(rows, H)
            _check(_fn("float_stream.hip", "pllm_rms_sandwich_sum",
                       signature=[c_int, c_int, c_void_p, c_void_p, c_long, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_float, c_void_p, c_void_p,
                                  c_float, c_void_p, c_long, c_int, c_int, c_void_p])(
                dtype_code(out.dtype) if out is not None else F32, dtype_code(h.dtype), _ptr(e), _ptr(h), h.stride(0), _ptr(rp), _ptr(wt), wt.shape[1],
                _ptr(bias), _ptr(w_branch), c_float(mult), _ptr(stream), _ptr(w_next), c_float(eps), _ptr(out),
                out.stride(0) if out is not None else 0, rows, H, _stream()), "rms_sandwich_sum")
            return out
    if branch is not None:
        _need(branch.dtype == torch.float32 and branch.shape == stream.shape and branch.is_contiguous(),
              "a branch is contiguous float32 rows like the stream (with its norm's weight, or none: it is added as it is)")
        _need(row_index is None, "rows are picked only where no branch is added")
    if row_index is not None:
        _need(row_index.dtype == torch.int32 and row_index.dim() == 1 and row_index.is_contiguous(), "row_index must be contiguous int32")
        rows = row_index.numel()
    if out is None and out_dtype is not None:
        out = torch.empty((rows, H), dtype=out_dtype, device=stream.device)
    if out is not None:
        _need(out.dim() == 2 and out.shape == (rows, H) and out.stride(1) == 1, f"the rows' output is [{rows}, {H}] with unit inner stride")
    _check(_fn("float_stream.hip", "pllm_rms_sandwich",
               signature=[c_int, c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_long, c_int, c_int, c_void_p])(
        dtype_code(out.dtype) if out is not None else F32, _ptr(branch), _ptr(bias), _ptr(w_branch), c_float(mult), _ptr(stream), _ptr(row_index),
        _ptr(w_next), c_float(eps), _ptr(out), out.stride(0) if out is not None else 0, rows, H, _stream()), "rms_sandwich")
    return out


def scaled_sum(a: torch.Tensor, sa: float, b: torch.Tensor, sb: float) -> torch.Tensor:
    """sa * a + sb * b in float, element by element; a and b contiguous, of one shape and type (float32 or the compute type)."""
    _on_gpu(a, b)
    _need(a.shape == b.shape and a.dtype == b.dtype and a.is_contiguous() and b.is_contiguous(), "scaled_sum: two contiguous tensors of one shape and type")
    out = torch.empty_like(a)
    _check(_fn("float_stream.hip", "pllm_scaled_sum", signature=[c_int, c_void_p, c_float, c_void_p, c_float, c_void_p, c_long, c_void_p])(
        dtype_code(a.dtype), _ptr(a), c_float(sa), _ptr(b), c_float(sb), _ptr(out), a.numel(), _stream()), "scaled_sum")
    return out


def _rms_sandwich_pair(stream, pair: WeightedPair, w_branch, mult, eps, w_next, out, out_dtype, bias, row_index):
    _on_gpu(stream, pair.first, pair.second, w_branch, w_next, out, bias)
    _need(stream.dtype == torch.float32 and stream.dim() == 2 and stream.is_contiguous(), "the stream is contiguous float32 [rows, hidden]")
    rows, H = stream.shape
    _need((H + 16) * 4 <= min(_max_lds_bytes(stream.device), 160 * 1024), f"the norm kernel stages one row in LDS: hidden size {H} is above its limit")
    _need(row_index is None, "rows are picked only where no branch is added")
    for t in (pair.first, pair.second):
        _need(t.dtype == torch.float32 and t.shape == stream.shape and t.is_contiguous(), "a pair's branches are contiguous float32 rows like the stream")
    for t, what in ((w_branch, "w_branch"), (w_next, "w_next"), (bias, "bias")):
        _need(t is None or (t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous()), f"{what} must be float32 [{H}]")
    if out is None and out_dtype is not None:
        out = torch.empty((rows, H), dtype=out_dtype, device=stream.device)
    if out is not None:
        _need(out.dim() == 2 and out.shape == (rows, H) and out.stride(1) == 1, f"the rows' output is [{rows}, {H}] with unit inner stride")
    sig = [c_int, c_void_p, c_float, c_void_p, c_float, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_float, c_void_p, c_long, c_int, c_int, c_void_p]
    _check(_fn("float_stream.hip", "pllm_rms_sandwich_pair", signature=sig)(
        dtype_code(out.dtype) if out is not None else F32, _ptr(pair.first), c_float(pair.first_scale), _ptr(pair.second), c_float(pair.second_scale),
        _ptr(bias), _ptr(w_branch), c_float(mult), _ptr(stream), _ptr(w_next), c_float(eps), _ptr(out), out.stride(0) if out is not None else 0,
        rows, H, _stream()), "rms_sandwich_pair")
    return out


def place_rows(x: torch.Tensor, out: torch.Tensor) -> None:
    """out[:, :] = x converted to out's type; x contiguous float32 [rows, hidden], out a view [rows, hidden] of wider rows."""
    _on_gpu(x, out)
    _need(x.dtype == torch.float32 and x.dim() == 2 and x.is_contiguous(), "place_rows takes contiguous float32 rows")
    _need(out.shape == x.shape and out.stride(1) == 1, "place_rows writes rows of the same shape with unit inner stride")
    _check(_fn("float_stream.hip", "pllm_place_rows", signature=[c_int, c_void_p, c_void_p, c_long, c_int, c_int, c_void_p])(
        dtype_code(out.dtype), _ptr(x), _ptr(out), out.stride(0), x.shape[0], x.shape[1], _stream()), "place_rows")


def dynamic_tanh(stream: torch.Tensor, alpha: float, weight: torch.Tensor | None, bias: torch.Tensor | None, branch=None,
                 row_index: torch.Tensor | None = None, out_dtype: torch.dtype | None = None) -> torch.Tensor | None:
    """Around a float32 residual stream [rows, hidden]: with ``branch`` (float32 rows like the stream, or a ``ChoiceSum``: a
    weighted sum of experts' rows that the kernel forms itself) stream += branch in place; then, when ``out_dtype`` is given, the rows tanh(alpha * stream) * weight + bias of the stream as it is now are
    returned in that type (``row_index``, int32, picks rows when no branch is added)."""
    if isinstance(branch, WeightedPair):
        branch = branch.rows()
    _on_gpu(stream, weight, bias, None if isinstance(branch, ChoiceSum) else branch, row_index)
    _need(stream.dtype == torch.float32 and stream.dim() == 2 and stream.is_contiguous(), "the stream is contiguous float32 [rows, hidden]")
    rows, H = stream.shape
    if isinstance(branch, ChoiceSum):
        # the experts' weighted sum (with what rides on it) is formed by the kernel that adds it to the stream
        _need(row_index is None, "no rows are picked where a branch is added")
        e, h, rp, wt = branch.checked(rows, H)
        shared, gate = branch.shared, branch.shared_gate
        _on_gpu(shared, gate)
        _need(shared is None or (shared.dtype == torch.float32 and shared.shape == (rows, H) and shared.is_contiguous()), f"shared: float32 [{rows}, {H}]")
        _need(gate is None or (shared is not None and gate.dtype == torch.float32 and gate.numel() == rows), f"shared_gate: float32 [{rows}]")
        out = None
        if out_dtype is not None:
            for t, what in ((weight, "weight"), (bias, "bias")):
                _need(t is not None and t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous(), f"{what} must be float32 [{H}]")
            out = torch.empty((rows, H), dtype=out_dtype, device=stream.device)
        sig = [c_int, c_int, c_void_p, c_void_p, c_long, c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_float, c_void_p,
               c_void_p, c_void_p, c_long, c_int, c_int, c_void_p]
        _check(_fn("float_stream.hip", "pllm_dyt_sum", signature=sig)(
            dtype_code(out_dtype or torch.float32), dtype_code(h.dtype), _ptr(e), _ptr(h), h.stride(0), _ptr(rp), _ptr(wt), wt.shape[1],
            int(branch.weights_inside), _ptr(shared), _ptr(gate), gate.stride(0) if gate is not None else 0, _ptr(stream), c_float(alpha),
            _ptr(weight), _ptr(bias), _ptr(out), H, rows, H, _stream()), "dynamic_tanh_sum")
        return out
    if branch is not None:
        _need(branch.dtype == torch.float32 and branch.shape == stream.shape and branch.is_contiguous() and row_index is None,
              "a branch is contiguous float32 rows like the stream, and no rows are picked then")
    if row_index is not None:
        _need(row_index.dtype == torch.int32 and row_index.dim() == 1 and row_index.is_contiguous(), "row_index must be contiguous int32")
        rows = row_index.numel()
    out = None
    if out_dtype is not None:
        for t, what in ((weight, "weight"), (bias, "bias")):
            _need(t is not None and t.dtype == torch.float32 and t.shape == (H,) and t.is_contiguous(), f"{what} must be float32 [{H}]")
        out = torch.empty((rows, H), dtype=out_dtype, device=stream.device)
    _check(_fn("float_stream.hip", "pllm_dyt", signature=[c_int, c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_void_p, c_long,
                                                         c_int, c_int, c_void_p])(
        dtype_code(out_dtype or torch.float32), _ptr(branch), _ptr(stream), _ptr(row_index), c_float(alpha), _ptr(weight), _ptr(bias), _ptr(out),
        H, rows, H, _stream()), "dynamic_tanh")
    return out


def stream_add(stream: torch.Tensor, branch) -> None:
    """stream += branch in place: contiguous float32 [rows, hidden], the branch also a ``ChoiceSum`` (a residual sum that nobody
    norms in the same kernel)."""
    dynamic_tanh(stream, 0.0, None, None, branch)


# ------------------------------------------------------------------------------------------- attention with normed queries and keys
MAX_PREPARED_HEAD = 256
VALUE_MODES = {"projected": 0, "normed": 1, "keys": 2}


def attn_prepare(proj: torch.Tensor, bias: torch.Tensor | None, conv_w: torch.Tensor | None, state: torch.Tensor | None,
                 state_slots, seq_starts, cu_seqlens, num_seqs: int, positions: torch.Tensor, cos: torch.Tensor | None,
                 sin: torch.Tensor | None, rot: int, interleaved: bool, eps: float, heads: int, kv_heads: int, d: int, dv: int, D: int,
                 dtype: torch.dtype, slot_mapping: torch.Tensor | None, k_pages: torch.Tensor | None, v_pages: torch.Tensor | None,
                 qk_norm: bool = True, values: str = "projected", norm_weights: tuple | None = None, norm_first: bool = False) -> torch.Tensor:
    """``values``: "projected" (the product's value columns as they are), "normed" (each value head divided by its root mean
    square, ``eps`` inside the root, no weight) or "keys" (the product has no value columns: a value head is its key head
    as projected, with the bias, before the rotation; dv == d).
    From the float32 sums ``proj`` [T, >= channels] of a q/k/v product (channels = heads d + kv_heads d + kv_heads dv):
    + ``bias``; a causal convolution over time per channel with ``conv_w`` float32 [channels, taps], whose inputs of
    earlier steps lie in ``state[slot]`` as [taps - 1, channels] and are left there for the next step; rotary encoding
    of the first ``rot`` elements of every q and k head; q and k heads divided by their root mean square (``eps``
    inside the root; not with ``qk_norm`` False), behind the rotation or, with ``norm_first``, in front of it, and times ``norm_weights``
    = (of q, of k), float32 [d] each, shared by all heads, when given; returns q as [T, heads * D] in ``dtype`` (heads padded with zeros to D) and writes k into
    ``k_pages`` [pages, kv_heads, block, D] and v into ``v_pages`` [pages, kv_heads, D, block] at ``slot_mapping``."""
    _on_gpu(proj, bias, conv_w, state, positions, cos, sin, slot_mapping, k_pages, v_pages)
    _need(values in VALUE_MODES, f"values: one of {tuple(VALUE_MODES)}, got {values!r}")
    _need(values != "keys" or d == dv, "values that are the keys have the keys' size")
    q_w, k_w = norm_weights if norm_weights is not None else (None, None)
    _on_gpu(q_w, k_w)
    for t in (q_w, k_w):
        _need(t is None or (qk_norm and t.dtype == torch.float32 and t.shape == (d,) and t.is_contiguous()), f"weights of the q/k norm: float32 [{d}]")
    channels = (heads + kv_heads) * d + (0 if values == "keys" else kv_heads * dv)
    _need(proj.dtype == torch.float32 and proj.dim() == 2 and proj.stride(1) == 1 and proj.shape[1] >= channels, f"proj: float32 [T, >= {channels}]")
    T = proj.shape[0]
    _need(0 < d <= D and 0 < dv <= D and D <= MAX_PREPARED_HEAD, f"head sizes {d}, {dv} padded to {D} (at most {MAX_PREPARED_HEAD})")
    _need(rot % 2 == 0 and 0 <= rot <= d, f"rotated width {rot} of a head of {d}")
    _need(positions.dtype == torch.int32 and positions.numel() == T and positions.is_contiguous(), "positions: int32 [T]")
    if rot:
        for t in (cos, sin):
            _need(t is not None and t.dtype == torch.float32 and t.dim() == 2 and t.shape[1] == rot // 2 and t.is_contiguous(),
                  f"rotary tables: float32 [positions, {rot // 2}]")
    _need(bias is None or (bias.dtype == torch.float32 and bias.numel() == channels and bias.is_contiguous()), f"bias: float32 [{channels}]")
    taps = 1
    if conv_w is not None:
        taps = conv_w.shape[1]
        _need(conv_w.dtype == torch.float32 and conv_w.shape == (channels, taps) and conv_w.is_contiguous() and 1 <= taps <= MAX_CONV_TAPS,
              f"conv weight: float32 [{channels}, taps <= {MAX_CONV_TAPS}]")
    if taps > 1:
        _need(state is not None, "a convolution over time needs the requests' state")
        _check_sequences(state, state_slots, seq_starts, cu_seqlens, num_seqs)
        _need(state.shape[1] >= channels * (taps - 1), "the convolution's inputs do not fit the state slot")
    write = slot_mapping is not None
    bs = 0
    if write:
        _need(k_pages is not None and v_pages is not None and k_pages.dim() == 4 and k_pages.is_contiguous() and v_pages.is_contiguous()
              and k_pages.dtype == dtype and v_pages.dtype == dtype, "pages: contiguous, of the queries' type")
        P, kvh, bs, dd = k_pages.shape
        _need(kvh == kv_heads and dd == D and tuple(v_pages.shape) == (P, kvh, D, bs), "pages: k [pages, kv_heads, block, D], v [pages, kv_heads, D, block]")
        _need(slot_mapping.dtype == torch.int32 and slot_mapping.numel() == T and slot_mapping.is_contiguous(), "slot_mapping: int32 [T]")
    q = torch.empty((T, heads * D), dtype=dtype, device=proj.device)
    sig = [c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_void_p, c_long, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_void_p,
           c_int, c_int, c_float, c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p,
           c_int, c_int, c_void_p]
    _check(_fn("attention_prepare.hip", "pllm_attn_prepare", signature=sig)(
        dtype_code(dtype), _ptr(proj), proj.stride(0), _ptr(bias), _ptr(conv_w), taps, _ptr(state) if taps > 1 else None,
        state.stride(0) if taps > 1 else 0, _ptr(state_slots) if taps > 1 else None, _ptr(seq_starts) if taps > 1 else None,
        _ptr(cu_seqlens) if taps > 1 else None, num_seqs, _ptr(positions), _ptr(cos) if rot else None, _ptr(sin) if rot else None, rot,
        int(bool(interleaved)), c_float(eps), int(bool(qk_norm)), int(bool(norm_first)), _ptr(q_w), _ptr(k_w), VALUE_MODES[values], heads, kv_heads, d, dv, D, _ptr(q), _ptr(slot_mapping) if write else None,
        _ptr(k_pages) if write else None, _ptr(v_pages) if write else None, bs, T, _stream()), "attn_prepare")
    return q


def gate_heads(o: torch.Tensor, gate: torch.Tensor | None, heads: int, dv: int, D: int) -> torch.Tensor:
    """[T, heads * dv]: the first ``dv`` elements of every head of ``o`` [T, heads * D], times sigmoid(gate[t, head]) when
    ``gate`` (float32 [T, heads], a view with unit inner stride) is given."""
    _on_gpu(o, gate)
    _need(o.dim() == 2 and o.stride(1) == 1 and o.shape[1] >= heads * D and 0 < dv <= D, "gate_heads: o [T, heads * D]")
    T = o.shape[0]
    _need(gate is None or (gate.dtype == torch.float32 and gate.shape == (T, heads) and gate.stride(1) == 1), f"gate: float32 [{T}, {heads}]")
    out = torch.empty((T, heads * dv), dtype=o.dtype, device=o.device)
    _check(_fn("attention_prepare.hip", "pllm_gate_heads", signature=[c_int, c_void_p, c_int, c_void_p, c_int, c_void_p, c_int, c_int, c_int, c_int, c_void_p])(
        dtype_code(o.dtype), _ptr(o), o.stride(0), _ptr(gate), gate.stride(0) if gate is not None else 0, _ptr(out), T, heads, dv, D, _stream()),
        "gate_heads")
    return out


# ------------------------------------------------------------------------------------------- routed experts
MOE_TILE_ROWS = 16
MOE_MID_TILE_ROWS = 64
MOE_MAX_TILE_ROWS = 128
MOE_MAX_EXPERTS = 1024


MOE_SCORINGS = {"softmax": 0, "sigmoid": 1, "softmax_chosen": 2}
MOE_GROUP_MARKS = {"largest": 1, "two_largest": 2}
MOE_FORMS = {"down": 0, "gated": 1, "plain": 2}


def moe_route(h: torch.Tensor, router_w: torch.Tensor, correction: torch.Tensor | None, groups: int, keep: int, top: int,
              scoring: str = "softmax", extra: int = 0, group_mark: str = "largest") -> tuple:
    """(ids int32 [T, top], weights float32 [T, top]): router outputs h router_w^T in float, scores by a softmax over all of
    them or (``scoring`` "sigmoid") a sigmoid of each, the ``top`` largest of score + correction among the experts of the
    ``keep`` best of ``groups`` groups of neighbours (a group's mark: its largest corrected score, or with ``group_mark`` "two_largest" the sum of its two largest), weights = the chosen
    experts' scores.  ``scoring`` "softmax_chosen": output + correction is what the choice looks at, and the weights are the softmax
    over the chosen experts' output + correction alone.  The last ``extra`` rows of ``router_w`` are no experts: their outputs come back as they are, as a
    third result float32 [T, extra] (further products of the same rows that ride along)."""
    _on_gpu(h, router_w, correction)
    _need(h.dim() == 2 and h.stride(1) == 1, "moe_route rows: [T, width] with unit inner stride")
    T, W = h.shape
    n_all = router_w.shape[0]
    n = n_all - extra
    _need(group_mark in MOE_GROUP_MARKS, f"group_mark {group_mark!r}: one of {tuple(MOE_GROUP_MARKS)}")
    _need(scoring in MOE_SCORINGS and 0 <= extra < n_all, f"scoring {scoring!r} (one of {sorted(MOE_SCORINGS)}), {extra} extra rows of {n_all}")
    _need(router_w.dtype == torch.float32 and router_w.shape == (n_all, W) and router_w.is_contiguous(), f"router: float32 [n, {W}]")
    _need(correction is None or (correction.dtype == torch.float32 and correction.shape == (n,) and correction.is_contiguous()), f"correction: float32 [{n}]")
    _need(groups > 0 and n % groups == 0 and 0 < keep <= groups and 0 < top <= (n // groups) * keep,
          f"{n} router outputs in {groups} groups, {keep} kept, {top} chosen")
    ids = torch.empty((T, top), dtype=torch.int32, device=h.device)
    weights = torch.empty((T, top), dtype=torch.float32, device=h.device)
    extras = torch.empty((T, extra), dtype=torch.float32, device=h.device) if extra else None
    _check(_fn("moe.hip", "pllm_moe_route", signature=[c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int,
                                                        c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p])(
        dtype_code(h.dtype), _ptr(h), h.stride(0), _ptr(router_w), _ptr(correction), T, W, n_all, extra, MOE_SCORINGS[scoring], groups, keep, MOE_GROUP_MARKS[group_mark], top,
        _ptr(ids), _ptr(weights), _ptr(extras), _stream()), "moe_route")
    return (ids, weights, extras) if extra else (ids, weights)


def moe_tile_rows(pairs: int, experts: int, dtype: torch.dtype, *inner_sizes: int) -> int:
    """Rows of a tile of the experts' products for a step of ``pairs`` (token, choice) pairs: where the matrix-core
    kernels run (bfloat16, every product's inner size a multiple of 8) 128 if an expert gets 32 pairs or more on average, 64
    where tiles of 128 would leave compute units idle (small experts) unless an expert gets 128; else 16.  (Both products at width
    2,048, 30 gated experts of 1,408, 512 tokens with 4 choices: 240 us with tiles of 128, 408 with 64, 465 with 16; 16 experts of
    1,024 at width 1,024, 256 tokens: 73, 66 and 83.)  It depends on the step's number of tokens only, so a replayed step keeps its choice."""
    if dtype == torch.bfloat16 and all(k % 8 == 0 for k in inner_sizes):
        if pairs >= 128 * experts:
            return MOE_MAX_TILE_ROWS
        if pairs >= 32 * experts:
            return MOE_MAX_TILE_ROWS if experts * max(inner_sizes[:2]) // 128 >= 160 else MOE_MID_TILE_ROWS
    return MOE_TILE_ROWS


def moe_align(ids: torch.Tensor, experts: int, tile_rows: int = MOE_TILE_ROWS) -> tuple:
    """The (token, choice) pairs of ``ids`` [T, top] whose expert is below ``experts``, sorted by expert:
    (sorted_pair int32 [pairs], row_of_pair int32 [pairs] (-1: an expert without weights), tiles int32 [max_tiles, 3]
    of (expert, first row, rows) with at most ``tile_rows`` rows each, rows 0 past the last tile)."""
    _on_gpu(ids)
    _need(ids.dtype == torch.int32 and ids.dim() == 2 and ids.is_contiguous(), "ids: contiguous int32 [T, top]")
    _need(0 < experts <= MOE_MAX_EXPERTS, f"1 to {MOE_MAX_EXPERTS} experts")
    _need(tile_rows in (MOE_TILE_ROWS, MOE_MID_TILE_ROWS, MOE_MAX_TILE_ROWS), f"tiles of {MOE_TILE_ROWS}, {MOE_MID_TILE_ROWS} or {MOE_MAX_TILE_ROWS} rows")
    pairs = ids.numel()
    max_tiles = -(-pairs // tile_rows) + experts
    sorted_pair = torch.empty(pairs, dtype=torch.int32, device=ids.device)
    row_of_pair = torch.empty(pairs, dtype=torch.int32, device=ids.device)
    tiles = torch.empty((max_tiles, 3), dtype=torch.int32, device=ids.device)
    _check(_fn("moe.hip", "pllm_moe_align", signature=[c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p])(
        _ptr(ids), pairs, experts, _ptr(sorted_pair), _ptr(row_of_pair), _ptr(tiles), max_tiles, tile_rows, _stream()), "moe_align")
    return sorted_pair, row_of_pair, tiles


def moe_expert_gemm(rows_in: torch.Tensor, w: torch.Tensor, tiles: torch.Tensor, sorted_pair: torch.Tensor, top: int, gated: bool,
                    activation: str = "silu", tile_rows: int = MOE_TILE_ROWS, pair_scale: torch.Tensor | None = None, plain: bool = False) -> torch.Tensor:
    """The experts' products over the sorted pairs.  ``gated``: rows_in [T, K] are the tokens' rows, w [experts, 2 N, K]
    holds [gate; up] per expert, the result [pairs, N] in the rows' type is act(gate . a) * (up . a) for the pair's token;
    ``plain``: the same rows, w [experts, N, K], the result act(w . a) (one of ``ROW_ACTIVATIONS`` without parameters).
    Neither: rows_in [pairs, K] are rows in sorted order, w [experts, N, K], and the result is float32 [pairs, N].
    ``pair_scale`` (an expert's first product only; float32, one number per pair in the order of the ids): the pair's input row counts as
    multiplied by it (the factor goes onto the float sums of the expert's first products)."""
    _need(not (gated and plain), "an expert's first product is gated or plain")
    form, first = "gated" if gated else "plain" if plain else "down", gated or plain
    _on_gpu(rows_in, w, tiles, sorted_pair, pair_scale)
    _need(rows_in.dim() == 2 and rows_in.stride(1) == 1 and w.dim() == 3 and w.is_contiguous() and w.dtype == rows_in.dtype
          and w.shape[2] == rows_in.shape[1], f"moe_expert_gemm shapes {tuple(rows_in.shape)} x {tuple(w.shape)}")
    _need(tiles.dtype == torch.int32 and tiles.dim() == 2 and tiles.shape[1] == 3 and tiles.is_contiguous(), "tiles: int32 [n, 3]")
    pairs = sorted_pair.numel()
    _need(sorted_pair.dtype == torch.int32 and sorted_pair.is_contiguous() and tiles.shape[0] >= -(-pairs // tile_rows), "sorted pairs and their tiles")
    _need(tile_rows == MOE_TILE_ROWS or (tile_rows in (MOE_MID_TILE_ROWS, MOE_MAX_TILE_ROWS) and rows_in.dtype == torch.bfloat16 and rows_in.shape[1] % 8 == 0
                                         and rows_in.stride(0) % 8 == 0), "tiles of more than 16 rows are the matrix-core kernels'")
    K = rows_in.shape[1]
    N = w.shape[1] // 2 if gated else w.shape[1]
    _need(first or rows_in.shape[0] == pairs, "the down product takes one row per pair")
    _need(not first or ((w.shape[1] % 2 == 0 or not gated) and rows_in.shape[0] * top == pairs), "an expert's first product takes the tokens' rows")
    _need(activation != "xielu", "an activation with parameters is not for experts")
    _need(pair_scale is None or (first and pair_scale.dtype == torch.float32 and pair_scale.numel() == pairs and pair_scale.is_contiguous()),
          f"pair_scale: float32 [{pairs}], for an expert's first product")
    out = torch.empty((pairs, N), dtype=rows_in.dtype if first else torch.float32, device=rows_in.device)
    _check(_fn("moe.hip", "pllm_moe_expert_gemm", signature=[c_int, c_int, c_void_p, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p, c_int, c_int, c_int, c_int,
                                                              c_void_p, c_int, c_int, c_void_p, c_void_p])(
        dtype_code(rows_in.dtype), MOE_FORMS[form], _ptr(rows_in), rows_in.stride(0), _ptr(w), _ptr(tiles), tiles.shape[0], tile_rows, _ptr(sorted_pair), pairs, top, N, K,
        _ptr(out), out.stride(0), row_activation_code(activation) if plain else activation_code(activation), _ptr(pair_scale), _stream()), "moe_expert_gemm")
    return out


def moe_combine(expert_out: torch.Tensor, h: torch.Tensor, row_of_pair: torch.Tensor, weights: torch.Tensor, weights_inside: bool = False,
                shared: torch.Tensor | None = None, shared_gate: torch.Tensor | None = None) -> torch.Tensor:
    """float32 [T, width]: sum over a token's choices, in their order, of weight * (the pair's row of ``expert_out``
    [pairs, width] float32, or the token's own row of ``h`` where row_of_pair is -1).  ``weights_inside``: the experts' rows
    count once (their weight went into their input; a pass-through row still takes its weight).  ``shared`` (float32
    [T, width]) is added, times sigmoid(shared_gate[t]) when ``shared_gate`` (float32 [T] or [T, 1], any row stride) is given."""
    _on_gpu(expert_out, h, row_of_pair, weights, shared, shared_gate)
    T, top = weights.shape
    W = h.shape[1]
    _need(expert_out.dtype == torch.float32 and expert_out.shape == (T * top, W) and expert_out.is_contiguous(), f"expert outputs: float32 [{T * top}, {W}]")
    _need(h.dim() == 2 and h.shape[0] == T and h.stride(1) == 1, "moe_combine rows: [T, width]")
    _need(row_of_pair.dtype == torch.int32 and row_of_pair.numel() == T * top and row_of_pair.is_contiguous(), "row_of_pair: int32 [T * top]")
    _need(weights.dtype == torch.float32 and weights.is_contiguous(), "weights: float32 [T, top]")
    _need(shared is None or (shared.dtype == torch.float32 and shared.shape == (T, W) and shared.is_contiguous()), f"shared: float32 [{T}, {W}]")
    gate_ld = 0
    if shared_gate is not None:
        _need(shared is not None and shared_gate.dtype == torch.float32 and shared_gate.numel() == T, f"shared_gate: float32 [{T}]")
        gate_ld = shared_gate.stride(0)
    out = torch.empty((T, W), dtype=torch.float32, device=h.device)
    _check(_fn("moe.hip", "pllm_moe_combine", signature=[c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_int,
                                                          c_int, c_int, c_int, c_void_p, c_void_p])(
        dtype_code(h.dtype), _ptr(expert_out), _ptr(h), h.stride(0), _ptr(row_of_pair), _ptr(weights), int(bool(weights_inside)), _ptr(shared),
        _ptr(shared_gate), gate_ld, T, top, W, _ptr(out), _stream()), "moe_combine")
    return out
