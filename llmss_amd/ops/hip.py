"""Validated launchers for the gfx950 kernels in ``llmss_amd/csrc`` (module ``llmss_amd._C``).

Every wrapper checks dtype, device, contiguity/strides and the shape relations the kernel grid
assumes *before* launching, so a malformed call raises here instead of faulting the GPU.
Kernels run on the caller's current HIP stream (``torch.cuda.current_stream()``), which makes
them capturable into HIP graphs together with RCCL collectives.
"""
from __future__ import annotations

import math
import os
import threading
import weakref
from typing import Optional

import torch

from . import reference as _ref
from .reference import PairPending

_C = None
_ERR = None


def lib():
    """The native module; raises loudly if it is missing (no silent eager fallback on GPU)."""
    global _C, _ERR
    if _C is None:
        try:
            from .. import _native
            _C = _native()
        except Exception as e:  # pragma: no cover - exercised only on broken installs
            _ERR = e
            raise RuntimeError(
                "llmss_amd._C is not available: run `python -m llmss_amd._build` (hipcc --offload-arch=gfx950)"
            ) from e
    return _C


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _ptr(t: Optional[torch.Tensor]) -> int:
    return 0 if t is None else t.data_ptr()


def _check(cond: bool, msg: str):
    if not cond:
        raise ValueError(msg)


def _bf16_rows(t: torch.Tensor, name: str, cols: Optional[int] = None):
    _check(t.is_cuda, f"{name} must be on the GPU")
    # kernels launch on the CURRENT device's stream: a tensor of another device would be addressed
    # through the wrong GPU's page tables
    _check(t.device.index == torch.cuda.current_device(),
           f"{name} is on {t.device} but the current device is cuda:{torch.cuda.current_device()}")
    _check(t.dtype == torch.bfloat16, f"{name} must be bfloat16, got {t.dtype}")
    _check(t.dim() == 2, f"{name} must be 2-D")
    _check(t.stride(1) == 1, f"{name} rows must be contiguous")
    _check(t.data_ptr() % 16 == 0 and (t.stride(0) * 2) % 16 == 0, f"{name} must be 16-byte aligned")
    if cols is not None:
        _check(t.shape[1] == cols, f"{name} has {t.shape[1]} columns, expected {cols}")


# ------------------------------------------------------------------------------------- norm
def _fp8_twin(y):
    """Scratch for the per-token fp8 twin of add_norm's output ``y`` [T, H], registered for its W8A8 consumer."""
    T, H = y.shape
    q, s = _PRESCRATCH.get(T, H, y.device)
    _PREQ.clear()  # one live twin at a time: the previous one's consumer has run (same stream, program order)
    _PREQ[id(y)] = (weakref.ref(y), q, s)
    return q, s


def add_norm(x, weight, bias, eps, rms, residual=None, out=None, residual_out=None, fp8_out=False):
    """``fp8_out``: also write the per-token fp8-e4m3 twin of the output (== quant_fp8_rows of it) for the W8A8
    GEMM that consumes it next, which then skips its own quantisation launch."""
    if isinstance(x, PartialSum):
        return add_norm_partial(x, weight, bias, eps, rms, residual, out, fp8_out=fp8_out)
    xcw = 0
    if x.dim() == 3:  # column-chunked [C, T, CW] (DecoderLM._reduce_cols): row t is x[:, t, :] concatenated
        _check(x.is_contiguous() and x.dtype == torch.bfloat16 and x.shape[2] % 8 == 0, "chunked x [C, T, CW]")
        C, T, xcw = x.shape
        H = C * xcw
    else:
        T, H = x.shape
        _bf16_rows(x, "x")
    _check(H % 8 == 0, "hidden must be a multiple of 8")
    _check(weight.is_contiguous() and weight.numel() == H and weight.dtype == torch.bfloat16, "norm weight")
    if bias is not None:
        _check(bias.is_contiguous() and bias.numel() == H and bias.dtype == torch.bfloat16, "norm bias")
    y = out if out is not None else torch.empty(T, H, dtype=x.dtype, device=x.device)
    _bf16_rows(y, "out", H)
    if residual is not None:
        _check(residual.is_contiguous() and residual.shape == (T, H) and residual.dtype == torch.bfloat16, "residual")
        ro = residual_out if residual_out is not None else residual
        _check(ro.is_contiguous() and ro.shape == (T, H), "residual_out")
    else:
        ro = None
    if residual is None and xcw:  # checked before the launch: an invalid call queues no GPU work
        raise ValueError("a column-chunked add_norm input needs a residual (its residual output is row-major)")
    q8, s8 = _fp8_twin(y) if fp8_out else (None, None)
    lib().add_norm(x.data_ptr(), x.stride(0) if not xcw else xcw, _ptr(residual), _ptr(ro), weight.data_ptr(),
                   _ptr(bias), y.data_ptr(), y.stride(0), T, H, float(eps), bool(rms), _stream(), _ptr(q8), _ptr(s8),
                   xcw)
    return y, (ro if residual is not None else x)


# ------------------------------------------------------------------------------------ embed
def embed(ids, wte, positions=None, wpe=None, out=None):
    T = ids.numel()
    V, H = wte.shape
    _check(ids.dtype == torch.int64 and ids.is_contiguous() and ids.is_cuda, "ids must be contiguous int64 cuda")
    _bf16_rows(wte, "wte")
    _check(wte.is_contiguous(), "wte contiguous")
    if wpe is not None:
        _check(positions is not None and positions.dtype == torch.int64 and positions.numel() == T, "positions")
        _check(wpe.is_contiguous() and wpe.shape[1] == H and wpe.dtype == torch.bfloat16, "wpe")
    y = out if out is not None else torch.empty(T, H, dtype=wte.dtype, device=wte.device)
    lib().embed(ids.data_ptr(), _ptr(positions), wte.data_ptr(), _ptr(wpe), y.data_ptr(), T, H, V, _stream())
    return y


# ------------------------------------------------------------------------------ rope + cache
def rope_cache(qkv, positions, cos, sin, k_cache, v_cache, slots, nh, nkv, D, rot, style, do_rope=True):
    """Rotate q/k in place and write k/v to the paged cache; returns the bf16 qkv tensor.

    ``qkv`` may be a :class:`PartialSum` (split-K slabs of the QKV GEMM): the kernel then sums the
    slabs (+ bias) itself and writes the finished rows into a fresh bf16 qkv tensor.
    """
    part = qkv if isinstance(qkv, PartialSum) else None
    if part is not None:
        _check(part.N == (nh + 2 * nkv) * D, "partial qkv width")
        qkv = torch.empty(part.M, part.N, dtype=torch.bfloat16, device=part.device)
    T = qkv.shape[0]
    _bf16_rows(qkv, "qkv")
    _check(qkv.shape[1] >= (nh + 2 * nkv) * D, "qkv too narrow")
    _check(D % 8 == 0 and rot <= D and (not do_rope or rot % 8 == 0), "head_dim / rotary_dim (multiple of 8)")
    _check(positions.dtype == torch.int64 and positions.numel() == T and positions.is_contiguous(), "positions")
    if do_rope and rot > 0:
        _check(cos.dtype == torch.float32 and cos.is_contiguous() and cos.shape[1] == rot // 2, "cos table")
        _check(sin.shape == cos.shape and sin.is_contiguous(), "sin table")
    kv8 = k_cache is not None and k_cache.dtype == torch.uint8
    if k_cache is not None:
        _kv_cache_check(k_cache, v_cache, nkv, D)
        _check(slots is not None and slots.dtype == torch.int64 and slots.numel() == T, "slots")
        bs = k_cache.shape[2]
    else:
        bs = 1
    lib().rope_cache(qkv.data_ptr(), qkv.stride(0), positions.data_ptr(), _ptr(cos) if do_rope else 0,
                     _ptr(sin) if do_rope else 0, _ptr(k_cache), _ptr(v_cache),
                     _ptr(slots) if k_cache is not None else 0, T, nh, nkv, D, rot,
                     bs, nh * D, (nh + nkv) * D, 1 if style == "gptj" else 0, bool(do_rope and rot > 0),
                     part.buf.data_ptr() if part else 0, part.S if part else 0, part.M * part.N if part else 0,
                     _ptr(part.bias) if part else 0, _stream(), kv8)
    return qkv


def _kv_cache_check(k_cache, v_cache, nkv, D):
    """bf16 [nb, nkv, bs, D] caches, or fp8 rows [nb, nkv, bs, D + 16] uint8 (ops/reference.py kv_rows_quant)."""
    kv8 = k_cache.dtype == torch.uint8
    _check(k_cache.is_cuda and k_cache.dtype in (torch.bfloat16, torch.uint8) and k_cache.is_contiguous()
           and k_cache.dim() == 4, "k_cache bf16 / uint8 (fp8 rows) [nb, nkv, bs, row]")
    _check(k_cache.shape[1] == nkv and k_cache.shape[3] == (D + _ref.KV8_TAIL if kv8 else D),
           f"k_cache shape [nb, nkv, bs, {'D + 16' if kv8 else 'D'}]")
    _check(v_cache.shape == k_cache.shape and v_cache.dtype == k_cache.dtype and v_cache.is_contiguous(), "v_cache")
    if kv8:
        _check(D % 16 == 0 and 256 % (D // 8) == 0, "fp8 KV cache needs head_dim 64/128/256")
    return kv8


# -------------------------------------------------------------------------------- attention
def attn_prefill(qkv, cu_seqlens, max_seqlen, nh, nkv, D, scale, out=None):
    T = qkv.shape[0]
    _bf16_rows(qkv, "qkv")
    _check(qkv.shape[1] >= (nh + 2 * nkv) * D, "qkv too narrow")
    _check(D in (64, 128, 256), "prefill attention supports head_dim 64/128/256")
    _check(cu_seqlens.dtype == torch.int32 and cu_seqlens.is_contiguous() and cu_seqlens.is_cuda, "cu_seqlens int32")
    B = cu_seqlens.numel() - 1
    y = out if out is not None else torch.empty(T, nh * D, dtype=qkv.dtype, device=qkv.device)
    _bf16_rows(y, "out")
    _check(qkv.stride(0) % 8 == 0 and qkv.data_ptr() % 16 == 0, "qkv rows 16-B aligned")
    lib().attn_prefill(qkv.data_ptr(), qkv.stride(0), T, cu_seqlens.data_ptr(), y.data_ptr(), y.stride(0), B,
                       int(max_seqlen), nh, nkv, D, nh * D, (nh + nkv) * D, float(scale), _stream())
    return y


def extend_fp8_twin_ok(nh: int, nkv: int) -> bool:
    """Can attn_extend write the per-token fp8 twin of its output in the same launch (every head of a row in
    one workgroup: one kv head, a power-of-two query group <= 16)?"""
    G = nh // nkv
    return nkv == 1 and G <= 16 and G & (G - 1) == 0


def attn_extend(q, k_cache, v_cache, block_tables, cu_q, ctx_lens, max_qlen, nh, nkv, D, scale, out=None,
                fp8_out=False, window=0, key_split=None):
    """``key_split`` = (nsplit, keys per split, a multiple of 64): single-token rows only (cu_q = 0, 1, .., B) - the
    visible keys of each row are cut over nsplit workgroups whose partials a reduce kernel joins.
    Chunked-prefill attention: q rows [T, >= nh*D] (query heads first, as in the QKV output) of B
    sequences (``cu_q`` [B+1] int32), each attending its whole paged context ``ctx_lens`` [B] int32 (the
    chunk's own K/V already written to the cache) causally; ``window`` > 0 limits a position to itself and the
    ``window - 1`` positions before it. ``fp8_out`` (only where extend_fp8_twin_ok):
    also write the output's per-token fp8 twin for the W8A8 o-projection, which then skips its quantisation
    launch."""
    T = q.shape[0]
    _bf16_rows(q, "q")
    _check(q.shape[1] >= nh * D, "q too narrow")
    _check(D in (64, 128, 256), "extend attention supports head_dim 64/128/256")
    kv8 = _kv_cache_check(k_cache, v_cache, nkv, D)
    _check(nh % nkv == 0, "nh % nkv")
    B = cu_q.numel() - 1
    for t, nm in ((cu_q, "cu_q"), (ctx_lens, "ctx_lens"), (block_tables, "block_tables")):
        _check(t.dtype == torch.int32 and t.is_contiguous() and t.is_cuda, f"{nm} must be contiguous int32 cuda")
    _check(ctx_lens.numel() == B and block_tables.dim() == 2 and block_tables.shape[0] >= B, "batch sizes")
    bs = k_cache.shape[2]
    _check(block_tables.shape[1] * bs >= 1, "block table width")
    y = out if out is not None else torch.empty(T, nh * D, dtype=q.dtype, device=q.device)
    _bf16_rows(y, "out")
    _check(y.shape[0] >= T and y.shape[1] >= nh * D, "out shape")
    q8 = s8 = None
    if fp8_out:
        _check(extend_fp8_twin_ok(nh, nkv) and y.shape == (T, nh * D), "fp8 twin: one kv head, group <= 16, dense out")
        q8, s8 = _fp8_twin(y)
    nsplit, split_keys, po, pml = 1, 0, None, None
    if key_split is not None and key_split[0] > 1:
        nsplit, split_keys = int(key_split[0]), int(key_split[1])
        _check(max_qlen == 1 and T == B and split_keys % 64 == 0 and not fp8_out, "key split: single-token rows")
        po, pml = _DECODE_WS.get(T, nh, nsplit, D, q.device)
    lib().attn_extend(q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), block_tables.data_ptr(),
                      block_tables.shape[1], cu_q.data_ptr(), ctx_lens.data_ptr(), y.data_ptr(), y.stride(0), B,
                      int(max_qlen), nh, nkv, D, bs, float(scale), _stream(), kv8, _ptr(q8), _ptr(s8), int(window),
                      nsplit, split_keys, _ptr(po), _ptr(pml))
    return y


def ce_loss_rows(logits, labels, vocab=None):
    """Per-row cross-entropy ``logsumexp(logits[t, :V]) - logits[t, label[t]]`` (0 where label < 0);
    ``logits`` [T, >= V] bf16 or fp32 rows, ``labels`` [T] int64."""
    T = logits.shape[0]
    V = int(vocab or logits.shape[1])
    _check(logits.is_cuda and logits.dim() == 2 and logits.stride(1) == 1, "logits [T, V] rows on the GPU")
    _check(logits.device.index == torch.cuda.current_device(), "logits on the current device")
    _check(logits.dtype in (torch.bfloat16, torch.float32), "logits must be bf16 or fp32")
    _check(logits.stride(0) % 8 == 0 and logits.data_ptr() % 16 == 0, "logits rows 16-B aligned")
    _check(V <= logits.shape[1], "vocab exceeds the row width")
    _check(labels.dtype == torch.int64 and labels.is_cuda and labels.numel() == T and labels.is_contiguous(),
           "labels [T] int64")
    loss = torch.empty(T, dtype=torch.float32, device=logits.device)
    lib().ce_loss(logits.data_ptr(), logits.stride(0), logits.dtype == torch.float32, labels.data_ptr(), T, V,
                  loss.data_ptr(), _stream())
    return loss


class DecodeWorkspace:
    """Split-K partial buffers for decode attention (allocated once; graph-capture safe)."""

    def __init__(self):
        self.po = None
        self.pml = None

    def get(self, B, nh, nsplit, D, device):
        need = B * nh * nsplit
        if (self.po is None or self.po.numel() < need * D or self.pml.numel() < need * 2
                or self.po.device != _dev(device)):
            if torch.cuda.is_current_stream_capturing():
                raise RuntimeError("decode workspace must be allocated before graph capture")
            n_o = max(need * D, 0 if self.po is None else 2 * self.po.numel())  # geometric: few retired buffers
            n_ml = max(need * 2, 0 if self.pml is None else 2 * self.pml.numel())
            _retire(self.po, self.pml)
            self.po = torch.empty(n_o, dtype=torch.float32, device=device)
            self.pml = torch.empty(n_ml, dtype=torch.float32, device=device)
        return self.po, self.pml


class _Slotted:
    """One instance of a scratch / workspace class per workspace slot (``workspace_slot``): kernels of chains
    that may run concurrently on different streams never share a buffer."""

    def __init__(self, cls):
        self._items = [cls() for _ in range(4)]

    def __getattr__(self, name):
        return getattr(self._items[getattr(_SLOT, "k", 0)], name)


_SLOT = threading.local()  # per host thread, like the native slot (csrc/gemm.hip gemm_set_slot)

# Scratch buffers outgrown by a later (eager) call are kept, never freed: a decode graph captured earlier still
# writes to the old addresses on every replay, and a freed block would go back to the caching allocator and be
# handed to live tensors (the native counters do the same, csrc/gemm.hip sk_counters).
_RETIRED: list = []


def _retire(*ts):
    _RETIRED.extend(t for t in ts if t is not None)


def _dev(device) -> torch.device:
    """``device`` as tensors report it ("cuda" -> "cuda:<current>"): a scratch buffer is reused only on its own device,
    and an unindexed name must not look like another device (every call would grow the buffer again)."""
    d = torch.device(device)
    if d.type == "cuda" and d.index is None:
        d = torch.device("cuda", torch.cuda.current_device())
    return d


class workspace_slot:
    """``with workspace_slot(k):`` ops issued inside use workspace slot k (GEMM workspace / combine counters,
    decode-attention partials, fp8 scratch) - for a chain that runs concurrently with slot 0's on another
    stream. Host-side state at launch (and capture) time."""

    def __init__(self, k: int):
        self.k = int(k) & 3

    def __enter__(self):
        self.prev = getattr(_SLOT, "k", 0)
        _SLOT.k = self.k
        lib().gemm_set_slot(self.k)
        return self

    def __exit__(self, *exc):
        _SLOT.k = self.prev
        lib().gemm_set_slot(self.prev)
        return False


_DECODE_WS = _Slotted(DecodeWorkspace)


def decode_splits(B: int, nkv: int, max_ctx: int, block_size: int) -> tuple:
    """(num_splits, partition_size): ~8 workgroups per CU (2048), partitions >= 256 tokens.

    Measured (bench/attn_bench.py): with few (sequence, kv-head) pairs - GQA / TP-sharded kv heads -
    each workgroup otherwise walks the whole context serially and the KV stream drops to 2-3 TB/s."""
    wgs = max(1, B * nkv)
    want = max(1, math.ceil(2048 / wgs))
    nsplit = max(1, min(want, math.ceil(max_ctx / 256)))
    psize = math.ceil(max_ctx / nsplit)
    psize = math.ceil(psize / block_size) * block_size
    nsplit = math.ceil(max_ctx / psize)
    return nsplit, psize


def attn_decode(q, k_cache, v_cache, block_tables, ctx_lens, nh, nkv, D, scale, max_ctx, out=None, splits=None):
    B = q.shape[0]
    _check(q.is_cuda and q.dtype == torch.bfloat16 and q.stride(-1) == 1 and q.dim() == 2, "q [B, >=nh*D]")
    _check(q.shape[1] >= nh * D, "q too narrow")
    _check(D in (64, 128, 256), "decode attention supports head_dim 64/128/256")
    kv8 = _kv_cache_check(k_cache, v_cache, nkv, D)
    _check(block_tables.dtype == torch.int32 and block_tables.dim() == 2 and block_tables.shape[0] >= B
           and block_tables.stride(1) == 1, "block_tables int32 [B, maxb]")
    _check(ctx_lens.dtype == torch.int32 and ctx_lens.numel() >= B and ctx_lens.is_contiguous(), "ctx_lens int32")
    bs = k_cache.shape[2]
    _check(block_tables.shape[1] * bs >= max_ctx, "block table too short for max_ctx")
    nsplit, psize = splits if splits is not None else decode_splits(B, nkv, max_ctx, bs)
    _check(nsplit * psize >= max_ctx, "splits do not cover max_ctx")
    y = out if out is not None else torch.empty(B, nh * D, dtype=q.dtype, device=q.device)
    po, pml = _DECODE_WS.get(B, nh, nsplit, D, q.device) if nsplit > 1 else (None, None)
    lib().attn_decode(q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), block_tables.data_ptr(),
                      block_tables.stride(0), ctx_lens.data_ptr(), y.data_ptr(), y.stride(0), _ptr(po), _ptr(pml),
                      B, nh, nkv, D, bs, nsplit, psize, float(scale), _stream(), kv8)
    return y


# ------------------------------------------------------------------------------------- GEMM
class GemmWorkspace:
    def __init__(self):
        self.buf = None

    def get(self, nbytes, device):
        if self.buf is None or self.buf.numel() * 4 < nbytes or self.buf.device != _dev(device):
            if torch.cuda.is_current_stream_capturing():
                raise RuntimeError("gemm workspace must be allocated before graph capture")
            _retire(self.buf)
            self.buf = torch.empty((max(nbytes, 1 << 20) + 3) // 4, dtype=torch.float32, device=device)
        return self.buf


_GEMM_WS = _Slotted(GemmWorkspace)


def reserve_workspace(device, gemm_bytes: int = 64 << 20, decode_rows: int = 0, nh: int = 0, D: int = 128,
                      nsplit: int = 1):
    _GEMM_WS.get(gemm_bytes, device)
    lib().gemm_reserve_streamk(1 << 16)  # per-tile counters of the in-launch split-K combines
    if decode_rows and nsplit > 1:
        _DECODE_WS.get(decode_rows, nh, nsplit, D, device)


_ACT = {"none": 0, None: 0, "gelu_tanh": 1, "gelu": 2, "relu": 3, "relu2": 5}


class PartialSum:
    """fp32 split-K partial slabs [S, M, N] of a GEMM left in the GEMM workspace; consumed (summed +
    bias) by the next add_norm. Valid only until the next GEMM on the stream."""

    __slots__ = ("buf", "S", "M", "N", "bias", "dtype", "device")

    def __init__(self, buf, S, M, N, bias, device):
        self.buf, self.S, self.M, self.N, self.bias, self.device = buf, S, M, N, bias, device
        self.dtype = torch.bfloat16

    @property
    def shape(self):
        return (self.M, self.N)

    @property
    def is_cuda(self):
        return True


_FP8_PREFILL_M = 128  # untuned fp8 calls above this M run W8A8 (compute-bound); below, W8A16 weight streaming

# nt_hint flag of a W8A8 plan (the tuned table's fp8 entries or an explicit hint): tile = (nt >> 8) & 15
# (1 128x128, 2 64x128, 3 64x64, 4 256x256, 7-15 the gemm_mid tiles), ring depth = (nt >> 12) & 15, split-K = the
# plan's split; W8A8_ILV: the gemm_mid tiles' software-pipelined k-loop (the bf16 plans' interleave bit 512 << 8)
W8A8_FLAG = 1 << 20
W8A8_ILV = 512 << 8


class _QuantScratch:
    """Per-token fp8 activations + scales for W8A8 calls: one buffer reused by every call on the stream (each
    GEMM consumes it before the next quantisation), grown only outside graph capture, so a captured decode
    step quantises into the same addresses on every replay."""

    def __init__(self):
        self.q = None
        self.s = None

    def get(self, M, K, device):
        if self.q is None or self.q.numel() < M * K or self.s.numel() < M or self.q.device != _dev(device):
            if torch.cuda.is_current_stream_capturing():
                raise RuntimeError(f"fp8 activation scratch for [{M}, {K}] must be allocated before graph capture")
            nq = max(M * K, 0 if self.q is None else 2 * self.q.numel())  # geometric: few retired buffers
            ns = max(M, 0 if self.s is None else 2 * self.s.numel())
            _retire(self.q, self.s)
            self.q = torch.empty(nq, dtype=torch.uint8, device=device)
            self.s = torch.empty(ns, dtype=torch.float32, device=device)
        return self.q[:M * K].view(M, K), self.s[:M]


_QSCRATCH = _Slotted(_QuantScratch)


class MxAct:
    """MX-fp8 activations (OCP MX): e4m3 bytes ``q`` [M, K] and one e8m0 scale per row and 32 columns ``s``
    [M, K / 32]. What a W8A8 gate/up GEMM writes for its down projection (``linear(..., mx_out=True)``), consumed by
    ``linear`` like a bf16 input."""

    __slots__ = ("q", "s")

    def __init__(self, q, s):
        self.q, self.s = q, s

    @property
    def shape(self):
        return self.q.shape

    @property
    def is_cuda(self):
        return self.q.is_cuda


class _MxScratch:
    """The MX-fp8 SwiGLU output (one per stream slot, reused by every layer: the down projection consumes it before
    the next gate/up writes it), grown only outside graph capture."""

    def __init__(self):
        self.q = self.s = None

    def get(self, M, K, device):
        if self.q is None or self.q.numel() < M * K or self.q.device != _dev(device):
            if torch.cuda.is_current_stream_capturing():
                raise RuntimeError(f"MX-fp8 activation scratch for [{M}, {K}] must be allocated before graph capture")
            n = max(M * K, 0 if self.q is None else 2 * self.q.numel())  # geometric: few retired buffers
            _retire(self.q, self.s)
            self.q = torch.empty(n, dtype=torch.uint8, device=device)
            self.s = torch.empty(n // 32, dtype=torch.uint8, device=device)
        return self.q[:M * K].view(M, K), self.s[:M * K // 32].view(M, K // 32)


_MXSCRATCH = _Slotted(_MxScratch)
MID_TILE_BN = {7: 48, 8: 128, 9: 128, 10: 256, 11: 128, 12: 256, 13: 192, 14: 32, 15: 96}  # gemm_mid tile -> BN


def _w8a8_mid_plan(M, N, K, glu):
    """The tuned W8A8 plan of this shape when it runs a gemm_mid tile (the MX-capable kernels), else None."""
    tuned = lib().gemm_tuned_get(M, N, K, bool(glu), 1)
    if tuned is None or not tuned[0] & W8A8_FLAG or ((tuned[0] >> 8) & 15) not in MID_TILE_BN:
        return None
    return tuned


def mx_mlp_ok(M: int, up, down) -> bool:
    """The gate/up SwiGLU GEMM can write its output as MX-fp8 for the down projection (no bf16
    intermediate, no per-token quantisation launch): both run tuned W8A8 gemm_mid plans at M rows, the gate/up plan is
    unsplit with whole 32-output blocks per tile (BN % 64 == 0)."""
    if up.w_scale is None or down.w_scale is None or not up.glu or up.N % 128 or down.K % 128 or up.N // 2 != down.K:
        return False
    pu, pd = _w8a8_mid_plan(M, up.N, up.K, True), _w8a8_mid_plan(M, down.N, down.K, False)
    return bool(pu and pd and pu[1] == 1 and MID_TILE_BN[(pu[0] >> 8) & 15] % 64 == 0)


def linear_w8a8(x, wq, w_scale, bias=None, act="none", glu=False, out=None, tile=0, depth=0, split=0,
                partial_ok=False, ilv=False, mx_out=False):
    """Y = (fp8(x) . wq^T) * x_scale[m] * w_scale[n] on the MX-fp8 MFMA (2x the bf16 matrix rate). The
    activations are quantised per token into a reusable scratch (graph-capturable). ``partial_ok``: a split
    plan may return its fp32 slabs as a :class:`PartialSum` for the consumer (rope_cache / add_norm).
    ``x`` may be an :class:`MxAct` (per-32 block scales, gemm_mid tiles); ``mx_out`` (SwiGLU, gemm_mid tile with
    BN % 64 == 0, no split) returns the output as an :class:`MxAct` instead of bf16."""
    mx_in = isinstance(x, MxAct)
    M, K = x.shape
    N = wq.shape[0]
    if mx_in:
        _check(x.q.dtype == torch.uint8 and x.q.is_contiguous() and x.s.is_contiguous() and x.s.numel() == M * K // 32,
               "MX activations: q [M, K] uint8, s [M, K / 32] uint8")
    else:
        _bf16_rows(x, "x")
    _check(wq.dtype == torch.uint8 and wq.is_contiguous() and K % 16 == 0 and wq.shape[1] == K, "fp8 weight")
    _check(w_scale.dtype == torch.float32 and w_scale.numel() == N, "w_scale [N] fp32")
    if glu:
        _check(N % 32 == 0, "glu needs N % 32 == 0")
    if bias is not None:
        _check(bias.dtype == torch.bfloat16 and bias.is_contiguous() and bias.numel() == N, "bias [N] bf16")
    dev = x.q.device if mx_in else x.device
    xs = None
    if mx_in:
        xq = x.q
    else:
        pre = _prequant_of(x)
        if pre is not None:  # add_norm already wrote this tensor's per-token fp8 twin
            xq, xs = pre
        else:
            xq, xs = _QSCRATCH.get(M, K, dev)
            lib().quant_fp8_rows_ld(x.data_ptr(), x.stride(0), xq.data_ptr(), xs.data_ptr(), M, K, _stream())
    nout = N // 2 if glu else N
    ws = _GEMM_WS.get(64 << 20, dev)
    if mx_out:
        _check(glu and out is None and not partial_ok, "MX-fp8 output: SwiGLU, no out buffer, no partial output")
        mq, ms = _MXSCRATCH.get(M, nout, dev)
        lib().gemm_f8f8(xq.data_ptr(), K, _ptr(xs), wq.data_ptr(), K, w_scale.data_ptr(), _ptr(bias), 0, nout, M, N,
                        K, _ACT[act], True, int(tile), int(depth), int(split), ws.data_ptr(), ws.numel() * 4,
                        _stream(), False, bool(ilv), mq.data_ptr(), ms.data_ptr(), 0)
        return MxAct(mq, ms)
    slabs = 0
    if partial_ok and out is None and not glu and act in ("none", None):
        slabs = lib().gemm_f8f8_partial_slabs(M, N, K, bool(glu), 0, int(tile), int(split), ws.numel() * 4)
    y = None if slabs else (out if out is not None else torch.empty(M, nout, dtype=torch.bfloat16, device=dev))
    if y is not None:
        _bf16_rows(y, "out", nout)
    S = lib().gemm_f8f8(xq.data_ptr(), K, _ptr(xs), wq.data_ptr(), K, w_scale.data_ptr(), _ptr(bias), _ptr(y),
                        y.stride(0) if y is not None else nout, M, N, K, _ACT[act], bool(glu), int(tile), int(depth),
                        int(split), ws.data_ptr(), ws.numel() * 4, _stream(), y is None, bool(ilv), 0, 0,
                        x.s.data_ptr() if mx_in else 0)
    if y is None:
        if S <= 1:
            raise RuntimeError("internal: partial W8A8 GEMM did not produce partial slabs")
        return PartialSum(ws, S, M, N, bias, dev)
    return y


# per-token fp8 twins written by add_norm(..., fp8_out=True) for the W8A8 GEMM that consumes the same tensor
# next (its own quantisation launch is then skipped): id(tensor) -> (weakref, q, s). The weakref makes a
# freed (and possibly address-reused) tensor miss; entries die with their tensor.
_PREQ = {}


class _PreQScratch:
    """Separate from _QSCRATCH: between add_norm and its consumer another W8A8 call may quantise into that."""

    def __init__(self):
        self.q = self.s = None

    def get(self, M, K, device):
        if self.q is None or self.q.numel() < M * K or self.s.numel() < M or self.q.device != _dev(device):
            if torch.cuda.is_current_stream_capturing():
                raise RuntimeError(f"fp8 norm-output scratch for [{M}, {K}] must be allocated before graph capture")
            _retire(self.q, self.s)
            nq = max(M * K, 0 if self.q is None else 2 * self.q.numel())  # geometric: few retired buffers
            ns = max(M, 0 if self.s is None else 2 * self.s.numel())
            self.q = torch.empty(nq, dtype=torch.uint8, device=device)
            self.s = torch.empty(ns, dtype=torch.float32, device=device)
        return self.q[:M * K].view(M, K), self.s[:M]


_PRESCRATCH = _Slotted(_PreQScratch)


def _prequant_of(x):
    e = _PREQ.get(id(x))
    if e is None or e[0]() is not x:
        return None
    return e[1], e[2]


def dequant_fp8_rows(q, scale, out=None):
    N, K = q.shape
    _check(q.dtype == torch.uint8 and q.is_contiguous() and K % 8 == 0, "fp8 weight [N, K] uint8, K % 8 == 0")
    _check(scale.dtype == torch.float32 and scale.numel() == N and scale.is_contiguous(), "scale [N] fp32")
    w = out if out is not None else torch.empty(N, K, dtype=torch.bfloat16, device=q.device)
    lib().dequant_fp8_rows(q.data_ptr(), scale.data_ptr(), w.data_ptr(), N, K, _stream())
    return w


def linear(x, w, bias=None, act="none", glu=False, w_scale=None, out=None, nt_hint=0, split_hint=0,
           partial_ok=False, mx_out=False):
    """``x`` bf16 [M, K], or an :class:`MxAct` for an fp8 weight with a W8A8 gemm_mid plan; ``mx_out``: return an
    fp8 SwiGLU output as :class:`MxAct` (its plan must allow it: :func:`mx_mlp_ok`)."""
    M, K = x.shape
    if isinstance(x, MxAct) or mx_out:
        _check(w_scale is not None, "MX-fp8 activations need fp8 weights")
        plan = (nt_hint, split_hint) if nt_hint else _w8a8_mid_plan(M, w.shape[0], K, glu)
        _check(plan is not None and plan[0] & W8A8_FLAG and ((plan[0] >> 8) & 15) in MID_TILE_BN,
               "MX-fp8 activations need a W8A8 gemm_mid plan")
        nt, sp = plan
        return linear_w8a8(x, w, w_scale, bias, act, glu, out, (nt >> 8) & 15, (nt >> 12) & 15, sp,
                           partial_ok=partial_ok, ilv=bool(nt & W8A8_ILV), mx_out=mx_out)
    _bf16_rows(x, "x")
    fp8 = w_scale is not None
    if fp8:
        _check(w.dtype == torch.uint8 and w.is_contiguous() and w.is_cuda, "fp8 weight stored as uint8 [N, K]")
        _check(w_scale.dtype == torch.float32 and w_scale.numel() == w.shape[0], "w_scale [N] fp32")
        tuned = lib().gemm_tuned_get(M, w.shape[0], K, bool(glu), 1) if not nt_hint else None
        if tuned is not None and tuned[0] & W8A8_FLAG:  # the autotuner picked W8A8 for this M
            nt_hint, split_hint = tuned
        if nt_hint & W8A8_FLAG:
            return linear_w8a8(x, w, w_scale, bias, act, glu, out, (nt_hint >> 8) & 15, (nt_hint >> 12) & 15,
                               split_hint, partial_ok=partial_ok, ilv=bool(nt_hint & W8A8_ILV))
        if M > _FP8_PREFILL_M and not nt_hint and tuned is None:  # compute-bound: per-token fp8 activations
            return linear_w8a8(x, w, w_scale, bias, act, glu, out, partial_ok=partial_ok)  # on the MX-fp8 MFMA
    else:
        _bf16_rows(w, "w")
        _check(w.is_contiguous(), "w contiguous")
    N = w.shape[0]
    _check(w.shape[1] == K, f"weight K={w.shape[1]} != x K={K}")
    _check(K % 16 == 0, "K must be a multiple of 16")
    if glu:
        _check(N % 32 == 0, "glu needs N % 32 == 0")
    if bias is not None:
        _check(bias.dtype == torch.bfloat16 and bias.is_contiguous() and bias.numel() == N, "bias [N] bf16")
    nout = N // 2 if glu else N
    ws = _GEMM_WS.get(64 << 20, x.device)
    partial_ok = partial_ok and not glu and act in ("none", None) and out is None
    y = out if out is not None else (None if partial_ok else torch.empty(M, nout, dtype=x.dtype, device=x.device))
    if partial_ok and lib().gemm_partial_slabs(M, N, K, fp8, False, 0, int(nt_hint), int(split_hint),
                                               ws.numel() * 4) == 0:
        y = torch.empty(M, nout, dtype=x.dtype, device=x.device)  # this call finishes its output itself
    if y is not None:
        _bf16_rows(y, "out", nout)
    S = lib().gemm(x.data_ptr(), x.stride(0), w.data_ptr(), K, fp8, _ptr(w_scale), _ptr(bias), _ptr(y),
                   y.stride(0) if y is not None else nout, M, N, K, _ACT[act], bool(glu), ws.data_ptr(),
                   ws.numel() * 4, int(nt_hint), int(split_hint), bool(y is None), _stream())
    if y is None:
        if S <= 1:
            raise RuntimeError("internal: partial GEMM did not produce partial slabs")
        return PartialSum(ws, S, M, N, bias, x.device)
    return y


def linear_qkv(x, w, bias, positions, cos, sin, k_cache, v_cache, slots, nh, nkv, D, rot, style, do_rope=True,
               nt_hint=0, split_hint=0):
    """QKV projection whose GEMM epilogue applies RoPE and writes k / v into the paged cache (one launch
    instead of GEMM + rope_cache; same values). Returns the bf16 [T, N] qkv tensor, or None when this
    weight / cache / plan cannot take the fused epilogue (packed or fp8 weights, fp8 KV rows, streaming or
    big-tile plans, neox RoPE on tiles that are not head-aligned): the caller then runs linear + rope_cache."""
    if w.dim() != 2 or w.dtype != torch.bfloat16 or (k_cache is not None and k_cache.dtype != torch.bfloat16):
        return None
    M, K = x.shape
    _bf16_rows(x, "x")
    _bf16_rows(w, "w")
    _check(w.is_contiguous() and w.shape[1] == K, "w [N, K] contiguous")
    N = w.shape[0]
    _check(N == (nh + 2 * nkv) * D and D % 8 == 0, "qkv width")
    if bias is not None:
        _check(bias.dtype == torch.bfloat16 and bias.is_contiguous() and bias.numel() == N, "bias [N] bf16")
    _check(positions.dtype == torch.int64 and positions.numel() == M and positions.is_contiguous(), "positions")
    do_rope = bool(do_rope and rot > 0)
    if do_rope:
        _check(cos.dtype == torch.float32 and cos.is_contiguous() and cos.shape[1] == rot // 2, "cos table")
        _check(sin.shape == cos.shape and sin.is_contiguous(), "sin table")
    bs = 1
    if k_cache is not None:
        _kv_cache_check(k_cache, v_cache, nkv, D)
        _check(slots is not None and slots.dtype == torch.int64 and slots.numel() == M and slots.is_contiguous(),
               "slots")
        bs = k_cache.shape[2]
    ws = _GEMM_WS.get(64 << 20, x.device)
    y = torch.empty(M, N, dtype=x.dtype, device=x.device)
    rc = lib().gemm_qkv(x.data_ptr(), x.stride(0), w.data_ptr(), K, _ptr(bias), y.data_ptr(), y.stride(0), M, N, K,
                        ws.data_ptr(), ws.numel() * 4, int(nt_hint), int(split_hint), positions.data_ptr(),
                        _ptr(cos) if do_rope else 0, _ptr(sin) if do_rope else 0, _ptr(k_cache), _ptr(v_cache),
                        _ptr(slots) if k_cache is not None else 0, nh, nkv, D, rot, bs, 1 if style == "gptj" else 0,
                        do_rope, _stream())
    return y if rc == 0 else None


def add_norm_partial(p: PartialSum, weight, bias, eps, rms, residual, out=None, fp8_out=False):
    T, H = p.M, p.N
    _check(residual is not None and residual.is_contiguous() and residual.shape == (T, H), "residual [T, H]")
    _check(weight.numel() == H and weight.dtype == torch.bfloat16 and weight.is_contiguous(), "norm weight")
    y = out if out is not None else torch.empty(T, H, dtype=torch.bfloat16, device=residual.device)
    q8, s8 = _fp8_twin(y) if fp8_out else (None, None)
    lib().add_norm_partial(p.buf.data_ptr(), p.S, T * H, _ptr(p.bias), residual.data_ptr(), residual.data_ptr(),
                           weight.data_ptr(), _ptr(bias), y.data_ptr(), y.stride(0), T, H, float(eps), bool(rms),
                           _stream(), _ptr(q8), _ptr(s8))
    return y, residual


def w8a8_planned(M: int, N: int, K: int, glu: bool) -> bool:
    """Whether an fp8-weight linear of this shape runs W8A8 (per-token fp8 activations) at M rows: the tuned
    table's plan, else the static rule (W8A8 above _FP8_PREFILL_M rows)."""
    tuned = lib().gemm_tuned_get(M, N, K, bool(glu), 1)
    if tuned is not None:
        return bool(tuned[0] & W8A8_FLAG)
    return M > _FP8_PREFILL_M


def quant_fp8_rows(w):
    _bf16_rows(w, "w")
    _check(w.is_contiguous(), "w contiguous")
    N, K = w.shape
    q = torch.empty(N, K, dtype=torch.uint8, device=w.device)
    s = torch.empty(N, dtype=torch.float32, device=w.device)
    lib().quant_fp8_rows(w.data_ptr(), q.data_ptr(), s.data_ptr(), N, K, _stream())
    return q, s


# ---------------------------------------------------------------------------------- sampler
CAND_K = 64  # rows with 1 <= top_k <= CAND_K (or greedy) can be sampled from gathered candidates
CAND_KC = 128  # candidate slots per rank and row (>= CAND_K: ties at the K-th value ride along)
CAND_MAX_SHARD = 16384  # widest vocab shard the candidate kernel takes


def cand_topk(local, lo, V, temperature, top_k, K=CAND_K, KC=CAND_KC, out=None, shards=1):
    """Per-rank candidates of a vocab-parallel logit shard: [B, 2*KC] fp32 (KC scaled values, then KC
    global token ids as int32 bits). ``shards`` > 1: the row is cut into that many column shards sampled by
    one launch (grid.y), packed shard-major [B, shards * 2*KC] - the layout of gathered per-rank packs, so a
    single GPU samples its full vocabulary through the same two short kernels instead of one long
    row-per-workgroup pass."""
    _bf16_rows(local, "local logits")
    B, width = local.shape
    vl = -(-width // shards)
    _check(shards >= 1 and vl <= CAND_MAX_SHARD, "vocab shard too wide for the candidate sampler")
    for t, dt, nm in ((temperature, torch.float32, "temperature"), (top_k, torch.int32, "top_k")):
        _check(t.dtype == dt and t.numel() >= B and t.is_contiguous() and t.is_cuda, f"{nm} must be {dt}")
    pack = out if out is not None else torch.empty(B, shards * 2 * KC, dtype=torch.float32, device=local.device)
    _check(pack.shape == (B, shards * 2 * KC) and pack.is_contiguous() and pack.dtype == torch.float32,
           "candidate pack")
    # columns past `width` in the last shard are masked by the kernel's lo + j < V bound only if V <= width
    _check(V <= width or shards == 1, "sharded candidates need the vocabulary inside the logits row")
    lib().cand_topk(local.data_ptr(), local.stride(0), B, vl, int(lo), int(V), temperature.data_ptr(),
                    top_k.data_ptr(), int(K), int(KC), pack.data_ptr(), pack.stride(0), _stream(), int(shards))
    return pack


def sample_cand(pack, KC, temperature, top_k, top_p, seeds, out=None, out2=None):
    """Sample from gathered candidates ``pack`` [B, groups * 2*KC] (rank-major)."""
    _check(pack.is_cuda and pack.dtype == torch.float32 and pack.dim() == 2 and pack.stride(1) == 1, "pack")
    B = pack.shape[0]
    _check(pack.shape[1] % (2 * KC) == 0, "pack width must be a multiple of 2*KC")
    groups = pack.shape[1] // (2 * KC)
    for t, dt, nm in ((temperature, torch.float32, "temperature"), (top_k, torch.int32, "top_k"),
                      (top_p, torch.float32, "top_p"), (seeds, torch.int64, "seeds")):
        _check(t.dtype == dt and t.numel() >= B and t.is_contiguous() and t.is_cuda, f"{nm} must be {dt}")
    y = out if out is not None else torch.empty(B, dtype=torch.int64, device=pack.device)
    lib().sample_cand(pack.data_ptr(), pack.stride(0), B, groups, int(KC), temperature.data_ptr(), top_k.data_ptr(),
                      top_p.data_ptr(), seeds.data_ptr(), y.data_ptr(), _ptr(out2), _stream())
    return y


def sample(logits, temperature, top_k, top_p, seeds, vocab: Optional[int] = None, out=None, out2=None):
    _check(logits.is_cuda and logits.dim() == 2 and logits.stride(1) == 1, "logits [B, V]")
    _check(logits.dtype in (torch.bfloat16, torch.float32), "logits bf16/fp32")
    B = logits.shape[0]
    V = vocab or logits.shape[1]
    _check(V <= logits.shape[1], "vocab > logits width")
    for t, dt, nm in ((temperature, torch.float32, "temperature"), (top_k, torch.int32, "top_k"),
                      (top_p, torch.float32, "top_p"), (seeds, torch.int64, "seeds")):
        if t is not None:
            _check(t.dtype == dt and t.numel() >= B and t.is_contiguous() and t.is_cuda, f"{nm} must be {dt}")
    y = out if out is not None else torch.empty(B, dtype=torch.int64, device=logits.device)
    lib().sample(logits.data_ptr(), logits.stride(0), logits.dtype == torch.float32, B, V, _ptr(temperature),
                 _ptr(top_k), _ptr(top_p), _ptr(seeds), y.data_ptr(), _ptr(out2), _stream())
    return y


# ------------------------------------------------- fp32 residual stream / latent attention / mixture of experts
# Kernels that run in either storage type (csrc/anytype.h): bf16 in serving precision, fp32 as a true 32-bit model.
_DT = {torch.bfloat16: 0, torch.float32: 1}


def _dt(t: torch.Tensor, name: str) -> int:
    _check(t.is_cuda and t.device.index == torch.cuda.current_device(), f"{name} must be on the current GPU")
    _check(t.dtype in _DT, f"{name} must be bfloat16 or float32, got {t.dtype}")
    return _DT[t.dtype]


def _rows(t: torch.Tensor, name: str, cols: Optional[int] = None, dtype=None):
    _check(t.dim() == 2 and t.stride(1) == 1, f"{name} must be 2-D with contiguous rows")
    if cols is not None:
        _check(t.shape[1] == cols, f"{name} has {t.shape[1]} columns, expected {cols}")
    if dtype is not None:
        _check(t.dtype == dtype, f"{name} must be {dtype}, got {t.dtype}")
    _check(t.is_cuda and t.device.index == torch.cuda.current_device(), f"{name} must be on the current GPU")


def embed_scaled(ids, table, scale):
    T = ids.numel()
    V, H = table.shape
    _check(ids.dtype == torch.int64 and ids.is_contiguous() and ids.is_cuda, "ids must be contiguous int64 cuda")
    _check(table.is_contiguous(), "embedding table contiguous")
    x = torch.empty(T, H, dtype=torch.float32, device=table.device)
    lib().embed_scaled(ids.data_ptr(), table.data_ptr(), x.data_ptr(), T, H, V, float(scale), _dt(table, "table"),
                       _stream())
    return x


class MoEPending:
    """Expert outputs of a mixture-of-experts layer before they are weighted and summed (``moe_experts(...,
    combine=False)``): fp32 rows ``y`` [pairs, N] in expert order, ``place`` [T * top] the row of each (token, slot)
    pair, ``wts`` [T, top], ``shared`` [T, N] or None. resid_add_norm takes it as its fp32 addend and combines while
    it adds to the stream."""

    __slots__ = ("y", "place", "wts", "shared", "top", "ident", "shared_w")

    def __init__(self, y, place, wts, shared, top=None, ident=None, shared_w=None):
        self.shared_w = shared_w  # fp32 [T]: factor of the shared rows (None: 1)
        self.ident = ident  # [T, N]: the output of the identity experts (pairs whose place is -1)
        self.y, self.place, self.wts, self.shared = y, place, wts, shared
        self.top = top if top is not None else wts.shape[1]  # wts None: the outputs are summed unweighted


def resid_add_norm(x, a, b, w, woff, eps, out_dtype, want_y=True):
    T, H = x.shape
    _rows(x, "x", dtype=torch.float32)
    _check(x.is_contiguous(), "x contiguous")
    if a is not None:
        _rows(a, "a", H, out_dtype)
        _check(a.shape[0] == T, "a rows")
    pend = b if isinstance(b, MoEPending) else None
    if pend is not None:
        _check(pend.wts is not None and pend.ident is None and pend.shared_w is None, "resid_add_norm combines weighted expert outputs")
        top = pend.wts.shape[1]
        _check(pend.y.shape == (T * top, H) and pend.y.is_contiguous() and pend.place.numel() == T * top
               and pend.wts.shape[0] == T, "pending expert outputs do not fit the stream")
        if pend.shared is not None:
            _rows(pend.shared, "shared", H, out_dtype)
        b = None
    elif b is not None:
        _rows(b, "b", H, torch.float32)
        _check(b.shape[0] == T, "b rows")
    y = None
    if want_y:
        _check(w.dtype == out_dtype and w.is_contiguous() and w.numel() == H, "norm weight")
        y = torch.empty(T, H, dtype=out_dtype, device=x.device)
    _check(out_dtype in _DT, "out dtype bf16 / fp32")
    sh = pend.shared if pend is not None else None
    lib().resid_add_norm(x.data_ptr(), _ptr(a), a.stride(0) if a is not None else 0, _ptr(b),
                         b.stride(0) if b is not None else 0, _ptr(pend.y) if pend else 0,
                         _ptr(pend.place) if pend else 0, _ptr(pend.wts) if pend else 0,
                         pend.wts.shape[1] if pend else 0, _ptr(sh), sh.stride(0) if sh is not None else 0,
                         _ptr(w) if want_y else 0, float(woff), float(eps), _ptr(y), H, T, H, _DT[out_dtype], _stream())
    return y


def gemm_any(A, B, C, M, N, K, batch, sAb, sAm, sBb, sBn, sBk, sCb, sCm, bias=None):
    """C[b][m][n] = sum_k A[b][m][k] B[b][n][k] over element strides; the caller has checked that every index stays
    inside its tensor. bf16 operands with k contiguous run on the matrix cores (csrc/gemm_tile.hip), everything else
    (fp32 storage, k-major B) on the vector ALUs (csrc/gemm_any.hip)."""
    if A.dtype == torch.bfloat16 and B.dtype == torch.bfloat16 and sBk == 1:
        lib().gemm_tile(A.data_ptr(), B.data_ptr(), C.data_ptr(), int(M), int(N), int(K), int(batch), int(sAb),
                        int(sAm), int(sBb), int(sBn), int(sCb), int(sCm), _dt(C, "C"), _ptr(bias), _stream())
        return C
    lib().gemm_any(A.data_ptr(), B.data_ptr(), C.data_ptr(), int(M), int(N), int(K), int(batch), int(sAb), int(sAm),
                   int(sBb), int(sBn), int(sBk), int(sCb), int(sCm), _dt(A, "A"), _dt(B, "B"), _dt(C, "C"), _ptr(bias),
                   _stream())
    return C


def _mfma_ok(x, w, out_dtype) -> bool:
    """Can the bf16 MFMA GEMM (csrc/gemm.hip) take this product? bf16 everywhere, K % 16, N % 8, 16-B aligned rows."""
    return (x.dtype == torch.bfloat16 and w.dtype == torch.bfloat16 and out_dtype == torch.bfloat16
            and w.is_contiguous() and x.shape[1] % 16 == 0 and w.shape[0] % 8 == 0 and x.stride(1) == 1
            and x.data_ptr() % 16 == 0 and (x.stride(0) * 2) % 16 == 0 and w.data_ptr() % 16 == 0)


def prompt_plan(M: int, N: int, K: int):
    """(nt_hint, split) of a prompt's product that is too narrow to fill the chip with 256 x 256 tiles: 128 x 256 tiles, K split
    until there are about as many workgroups as compute units. (0, 0): the GEMM's own plan."""
    if M < 2048 or -(-M // 256) * -(-N // 256) >= 192 or N < 128 or lib().gemm_tuned_get(M, N, K, False, 0) is not None:
        return 0, 0
    split = 1
    while split < 4 and -(-M // 128) * -(-N // 256) * split * 2 <= 288 and K // (2 * split) >= 512:
        split *= 2
    return (12 | 16 | (512 if K % 64 == 0 else 0)) << 8, split


def linear_f(x, w, out_dtype, bias=None, act="none"):
    """act(x [M, K] . w [N, K]^T + bias) -> [M, N] in ``out_dtype`` with fp32 accumulation: the MFMA GEMM where it applies
    (bias and activation in its epilogue), else the tile GEMM or the strided VALU GEMM (fp32 storage, fp32 output, odd
    shapes) and the activation in a launch of its own."""
    M, K = x.shape
    N = w.shape[0]
    _rows(x, "x")
    _rows(w, "w", K)
    _check(w.is_contiguous(), "w contiguous")
    if bias is not None:
        _check(bias.dtype == w.dtype and bias.is_contiguous() and bias.numel() == N and bias.is_cuda, "bias [N] in w's type")
    if M == 0:
        return torch.empty(0, N, dtype=out_dtype, device=x.device)
    if _mfma_ok(x, w, out_dtype):
        nt, split = prompt_plan(M, N, K)
        return linear(x, w, bias, act, nt_hint=nt, split_hint=split)
    y = torch.empty(M, N, dtype=out_dtype, device=x.device)
    gemm_any(x, w, y, M, N, K, 1, 0, x.stride(0), 0, K, 1, 0, N, bias)
    return y if act in ("none", None) else act_fn(y, act)


def head_absorb(q, uk_t, out_dtype=torch.float32, extra=0):
    H, R, dim = uk_t.shape
    T = q.shape[0]
    _rows(q, "q")
    _check(extra >= 0 and q.shape[1] >= H * (dim + extra), "q too narrow")
    _check(uk_t.is_contiguous() and uk_t.dtype == q.dtype and uk_t.is_cuda, "uk_t [H, R, dim] in q's storage type")
    Rt = R + extra
    qa = torch.empty(T, H, Rt, dtype=out_dtype, device=q.device)
    if T:
        # batch = head: A(t, d) = q[t, h * (dim + extra) + d]; B(r, d) = uk_t[h, r, d]; C(t, r) = qa[t, h, r]
        gemm_any(q, uk_t, qa, T, R, dim, H, dim + extra, q.stride(0), R * dim, dim, 1, Rt, H * Rt)
    return qa


def head_expand(o, uv, out_dtype):
    T, H, Rt = o.shape
    R = uv.shape[1]
    _check(o.is_contiguous() and o.dtype in _DT and o.is_cuda and R <= Rt, "o [T, H, >= R] contiguous")
    _rows(uv, "uv", R)
    _check(uv.is_contiguous() and uv.shape[0] % H == 0, "uv [H * vdim, R]")
    vd = uv.shape[0] // H
    y = torch.empty(T, H * vd, dtype=out_dtype, device=o.device)
    if T:
        # batch = head: A(t, r) = o[t, h, r], r < R; B(v, r) = uv[h * vd + v, r]; C(t, v) = y[t, h * vd + v]
        gemm_any(o, uv, y, T, vd, R, H, Rt, H * Rt, vd * R, R, 1, vd, H * vd)
    return y


def latent_norm_cache(src, off, R, w, eps, cache, slots, rot=0, cs=None, qa=None, off_q=0, qdim=0,
                      q_src=None):
    T = src.shape[0]
    _rows(src, "src")
    rot = int(rot)
    _check(0 <= off and off + R + rot <= src.shape[1], "latent columns outside src")
    _check(cache.dtype == src.dtype and cache.is_contiguous() and cache.dim() == 3 and cache.shape[2] == R + rot,
           "latent cache [blocks, block_size, R + rot] in the model's storage type")
    _check(w.dtype == src.dtype and w.is_contiguous() and w.numel() == R, "latent norm weight")
    _check(slots.dtype == torch.int64 and slots.is_contiguous() and slots.numel() == T and slots.is_cuda, "slots")
    H = dq = rdims = 0
    if rot:
        _f32c(cs, "angles")
        _check(cs.dim() == 3 and cs.shape[0] == T and cs.shape[2] == 2 and 2 * cs.shape[1] <= rot,
               "angles [T, rotated dims / 2, 2], rotated dims <= rot")
        rdims = 2 * cs.shape[1]
        _check(qa.is_contiguous() and qa.is_cuda and qa.dim() == 3 and qa.shape[0] == T and qa.shape[2] == R + rot,
               "qa [T, H, R + rot] contiguous")
        H, dq = qa.shape[1], _dt(qa, "qa")
        qs = src if q_src is None else q_src
        _rows(qs, "q_src", dtype=src.dtype)
        _check(qs.shape[0] == T and off_q >= 0 and off_q + H * (qdim + rot) <= qs.shape[1], "query columns outside their rows")
    lib().latent_norm_cache(src.data_ptr(), src.stride(0), int(off), w.data_ptr(), float(eps), cache.data_ptr(),
                            slots.data_ptr(), T, R, rot, rdims, _ptr(cs) if rot else 0, _ptr(qa) if rot else 0,
                            qs.data_ptr() + int(off_q) * qs.element_size() if rot else 0, qs.stride(0) if rot else 0, H,
                            int(qdim), _dt(src, "src"), dq, _stream())


def rms_cols(src, off, n, w, eps, out_dtype):
    T = src.shape[0]
    _rows(src, "src", dtype=out_dtype)
    _check(0 <= off and off + n <= src.shape[1], "columns outside src")
    _check(w.dtype == src.dtype and w.is_contiguous() and w.numel() == n and w.is_cuda, "norm weight [n] in src's type")
    out = torch.empty(T, n, dtype=out_dtype, device=src.device)
    lib().rms_cols(src.data_ptr() + int(off) * src.element_size(), src.stride(0), w.data_ptr(), float(eps), out.data_ptr(), T,
                   int(n), _dt(src, "src"), _stream())
    return out


def rope_angles(positions, freqs):
    T = positions.numel()
    _check(positions.dtype == torch.int64 and positions.is_contiguous() and positions.is_cuda, "positions: int64 cuda")
    _f32c(freqs, "freqs")
    cs = torch.empty(T, freqs.numel(), 2, dtype=torch.float32, device=positions.device)
    lib().rope_angles(positions.data_ptr(), freqs.data_ptr(), cs.data_ptr(), T, freqs.numel(), _stream())
    return cs


LATENT_MFMA_RANKS = (64, 128, 256)  # latent ranks the MFMA extend kernel is built for (csrc/attention_extend.hip)
_LATENT_MFMA = os.environ.get("LLMSS_LATENT_MFMA", "1") != "0"  # 0: every rank on the generic kernel (A/B runs)


def latent_qa_dtype(cache) -> torch.dtype:
    """Storage type latent_attn wants its absorbed queries in: bf16 where the MFMA kernel runs, else fp32."""
    if cache.is_cuda and cache.dtype == torch.bfloat16 and cache.shape[2] in LATENT_MFMA_RANKS and _LATENT_MFMA:
        return torch.bfloat16
    return torch.float32


def latent_key_split(B: int, window: int, max_ctx: int):
    """(nsplit, keys per split) for a decode step of B single-token rows whose visible range is at most
    min(window, max_ctx) keys: about 512 workgroups, whole 64-key tiles per split (more splits write and read more partial
    rows than their shorter key walks save)."""
    keys = min(window, max_ctx) if window > 0 else max_ctx
    tiles = -(-keys // 64) + (1 if window > 0 else 0)  # a window may straddle one more tile
    nsplit = max(1, min(tiles, 512 // max(1, B)))
    per = -(-tiles // nsplit)
    return -(-tiles // per), per * 64


def latent_attn(qa, cache, block_tables, cu_q, ctx_lens, window, scale, max_qlen=0, max_ctx=0, out=None):
    """``qa`` [T, H, R]. bf16 queries over a bf16 cache of rank 64 / 128 / 256 run the MFMA extend kernel as
    multi-query attention whose one key/value head is the latent row (keys = values = cache, bf16 output); anything
    else runs the generic kernel (fp32 queries, fp32 output)."""
    T, H, R = qa.shape
    _check(qa.is_contiguous() and qa.is_cuda, "qa [T, H, R] contiguous")
    _check(cache.is_contiguous() and cache.dim() == 3 and cache.shape[2] == R, "latent cache [blocks, block_size, R]")
    B = cu_q.numel() - 1
    for t, nm in ((cu_q, "cu_q"), (ctx_lens, "ctx_lens"), (block_tables, "block_tables")):
        _check(t.dtype == torch.int32 and t.is_contiguous() and t.is_cuda, f"{nm} must be contiguous int32 cuda")
    _check(ctx_lens.numel() >= B and block_tables.dim() == 2 and block_tables.shape[0] >= B, "batch sizes")
    if qa.dtype == torch.bfloat16:
        _check(latent_qa_dtype(cache) == torch.bfloat16 and max_qlen > 0, "bf16 queries: MFMA ranks and max_qlen only")
        kv = cache.view(cache.shape[0], 1, cache.shape[1], R)  # [blocks, one kv head, block_size, R]
        split = latent_key_split(T, window, max_ctx) if max_qlen == 1 and T == B and max_ctx > 0 else None
        o = attn_extend(qa.view(T, H * R), kv, kv, block_tables, cu_q, ctx_lens[:B], max_qlen, H, 1, R, scale,
                        window=window, key_split=split, out=None if out is None else out.view(T, H * R))
        return o.view(T, H, R)
    _check(qa.dtype == torch.float32, "qa fp32")
    _check(R <= 1024, "latent rank above 1024")
    if out is None:
        out = torch.empty(T, H, R, dtype=torch.float32, device=qa.device)
    _check(out.dtype == torch.float32 and out.is_contiguous() and tuple(out.shape) == (T, H, R), "out fp32 [T, H, R]")
    lib().latent_attn(qa.data_ptr(), H * R, cache.data_ptr(), block_tables.data_ptr(), block_tables.shape[1],
                      cu_q.data_ptr(), ctx_lens.data_ptr(), out.data_ptr(), H * R, T, B, H, R, cache.shape[1],
                      int(window), float(scale), _dt(cache, "cache"), _stream())
    return out


def glu_clamp(gu, F, limit, alpha):
    T = gu.shape[0]
    _rows(gu, "gu")
    _check(gu.shape[1] >= 2 * F, "gate | up too narrow")
    out = torch.empty(T, F, dtype=gu.dtype, device=gu.device)
    lib().glu_clamp(gu.data_ptr(), gu.stride(0), out.data_ptr(), F, T, F, float(limit), float(alpha), _dt(gu, "gu"),
                    _stream())
    return out


_SCORE = {"sigmoid": 0, "softmax": 1, "chosen": 2}


def _route_args(E, top, corr, bias, score):
    _check(1 <= top <= E and E <= 4096, "1 <= top <= experts <= 4096")
    _check(score in _SCORE and not (score == "chosen" and corr is not None), "score: sigmoid, softmax or chosen (no correction)")
    for t, nm in ((corr, "correction"), (bias, "router bias")):
        if t is not None:
            _check(t.dtype == torch.float32 and t.is_contiguous() and t.numel() == E and t.is_cuda, f"{nm} fp32 [E]")


def moe_route(z, corr, top, normalize=True, score="sigmoid", bias=None, gate=False):
    T, E = z.shape[0], z.shape[1] - int(bool(gate))
    _rows(z, "z", dtype=torch.float32)
    _check(z.is_contiguous(), "router logits contiguous")
    _route_args(E, top, corr, bias, score)
    idx = torch.empty(T, top, dtype=torch.int32, device=z.device)
    wts = torch.empty(T, top, dtype=torch.float32, device=z.device)
    sg = torch.empty(T, dtype=torch.float32, device=z.device) if gate else None
    lib().moe_route(z.data_ptr(), _ptr(corr), idx.data_ptr(), wts.data_ptr(), T, E, top, int(bool(normalize)),
                    _SCORE[score], _ptr(bias), _ptr(sg), _stream())
    return (idx, wts, sg) if gate else (idx, wts)


ROUTER_MFMA_MIN_ROWS = 256  # from here on a workgroup per token reads the router's weights too often
ROUTER_FUSED_MAX_ROWS = 1024  # steps of at most this many tokens compute logits and routing in one launch


def moe_router(h, router, corr, top, normalize=True, score="sigmoid", bias=None, gate=False):
    """(idx [T, top] int32, wts [T, top] fp32(, gate fp32 [T])) from the layer input: fp32 router logits, then moe_route. Few
    rows (a decode step): one fused launch, a workgroup per token; a prompt of bf16 rows and up to 128 outputs: one launch on
    the matrix cores, 16 tokens per workgroup; else the matrix-core GEMM with fp32 output, then moe_route."""
    T, K = h.shape
    E = router.shape[0] - int(bool(gate))
    _rows(h, "h")
    mfma = (h.dtype == torch.bfloat16 and T > ROUTER_MFMA_MIN_ROWS and lib().moe_router_mfma_ok(E, int(bool(gate)), K) and h.data_ptr() % 16 == 0
            and h.stride(0) % 8 == 0 and router.data_ptr() % 16 == 0)
    if T > ROUTER_FUSED_MAX_ROWS and not mfma:
        return moe_route(linear_f(h, router, torch.float32), corr, top, normalize, score, bias, gate)
    _check(router.dtype == h.dtype and router.is_contiguous() and router.shape[1] == K and router.is_cuda,
           "router [E (+ 1), K] in h's storage type")
    _route_args(E, top, corr, bias, score)
    idx = torch.empty(T, top, dtype=torch.int32, device=h.device)
    wts = torch.empty(T, top, dtype=torch.float32, device=h.device)
    sg = torch.empty(T, dtype=torch.float32, device=h.device) if gate else None
    if mfma:
        lib().moe_router_mfma(h.data_ptr(), h.stride(0), router.data_ptr(), _ptr(corr), idx.data_ptr(), wts.data_ptr(), T, E, K,
                              top, int(bool(normalize)), _SCORE[score], _ptr(bias), _ptr(sg), _stream())
        return (idx, wts, sg) if gate else (idx, wts)
    lib().moe_router(h.data_ptr(), h.stride(0), router.data_ptr(), _ptr(corr), idx.data_ptr(), wts.data_ptr(), T, E, K,
                     top, _dt(h, "h"), int(bool(normalize)), _SCORE[score], _ptr(bias), _ptr(sg), _stream())
    return (idx, wts, sg) if gate else (idx, wts)


_MOE_PP = os.environ.get("LLMSS_MOE_PP", "1") != "0"  # 0: grouped products on the tile kernel at every size (A/B runs)


def moe_experts(h, idx, wts, gate, up, down, limit, alpha, shared=None, combine=True, act="glu_clamp",
                weight_input=False, identity=False, shared_w=None, interleaved=False):
    """``identity``: indices from E on are identity experts. ``combine=False``: leave the weighting and summing to the next residual add (returns a :class:`MoEPending`).
    ``weight_input``: the weights scale the two input products in the gate / up epilogue (the experts have no
    biases), and the outputs are summed plainly (``MoEPending.wts`` is None)."""
    T, K = h.shape
    E, F, _ = up.shape
    if interleaved:
        _check(gate is None and act == "silu" and h.dtype == torch.bfloat16 and F % 32 == 0 and not weight_input,
               "interleaved gate / up rows: bf16, silu, groups of 16 rows")
        F //= 2
    N = down.shape[1]
    top = idx.shape[1]
    dt = _dt(h, "h")
    _rows(h, "h")
    _check(interleaved or (gate is None) == (act == "gelu"), "experts without a gate: act gelu")
    UF = 2 * F if interleaved else F
    for t, nm, shp in ((up if gate is None else gate, "gate", (E, UF, K)), (up, "up", (E, UF, K)), (down, "down", (E, N, F))):
        _check(t.dtype == h.dtype and t.is_contiguous() and tuple(t.shape) == shp and t.is_cuda, f"{nm} {shp}")
    _check(idx.dtype == torch.int32 and idx.is_contiguous() and idx.shape == (T, top) and idx.is_cuda, "idx")
    _check(wts.dtype == torch.float32 and wts.is_contiguous() and wts.shape == (T, top) and wts.is_cuda, "wts")
    if shared is not None:
        _rows(shared, "shared", N, h.dtype)
        _check(shared.shape[0] == T, "shared rows")
    if shared_w is not None:
        _check(shared_w.dtype == torch.float32 and shared_w.is_contiguous() and shared_w.numel() == T and shared_w.is_cuda
               and shared is not None, "shared_w fp32 [T]")
    out = torch.empty(T, N, dtype=torch.float32, device=h.device) if combine or T == 0 else None
    if T == 0:
        return out
    P = T * top
    # rows per tile of the grouped GEMMs: 128 where the experts get enough rows to fill big tiles (bf16 only)
    rows = 128 if h.dtype == torch.bfloat16 and P >= 128 * E else 64
    # ungated experts with still more rows each: the dense GEMMs' 256x256 ping-pong kernel
    # (gated ones with their gate and up rows interleaved, the activation in the epilogue)
    pp = (gate is None and h.dtype == torch.bfloat16 and P >= 384 * E and min(F, N) >= 256 and F % 8 == 0 and K % 8 == 0
          and h.stride(0) % 8 == 0 and not weight_input and h.data_ptr() % 16 == 0 and _MOE_PP)
    if pp:
        rows = 256
    maxt = -(-P // rows) + min(E, P)
    _check(maxt <= 65535, "too many (token, expert) pairs in one step")
    dev = h.device
    meta = torch.empty(1 + (E + 1) + 2 * maxt, dtype=torch.int32, device=dev)
    order = torch.empty(P, dtype=torch.int32, device=dev)
    place = torch.empty(P, dtype=torch.int32, device=dev)
    act_ = torch.empty(P, F, dtype=h.dtype, device=dev)
    y = torch.empty(P, N, dtype=torch.float32, device=dev)
    _check(act in ("glu_clamp", "silu", "gelu"), "expert activation: glu_clamp, silu or gelu (no gate)")
    _check(not identity or (K == N and not weight_input), "identity experts give the input row itself")
    pw, silu = (wts.data_ptr() if weight_input else 0), int(act == "silu")
    L = lib()
    st = _stream()
    L.moe_group(idx.data_ptr(), P, E, maxt, meta.data_ptr(), order.data_ptr(), place.data_ptr(), rows, st)
    if pp:
        L.moe_pp(3 if interleaved else 1, h.data_ptr(), h.stride(0), up.data_ptr(), meta.data_ptr(), order.data_ptr(),
                 act_.data_ptr(), E, maxt, top, UF, K, 0 if interleaved else _ACT["gelu"], st)
        L.moe_pp(2, act_.data_ptr(), F, down.data_ptr(), meta.data_ptr(), order.data_ptr(), y.data_ptr(), E, maxt, 1, N, F,
                 0, st)
    elif h.dtype == torch.bfloat16:  # matrix cores (csrc/gemm_tile.hip)
        L.moe_gate_up_tile(h.data_ptr(), h.stride(0), up.data_ptr() if interleaved else _ptr(gate), up.data_ptr(),
                           meta.data_ptr(), order.data_ptr(), act_.data_ptr(), E, maxt, top, F, K, float(limit), float(alpha),
                           rows, pw, silu, int(interleaved), st)
        L.moe_down_tile(act_.data_ptr(), down.data_ptr(), meta.data_ptr(), y.data_ptr(), E, maxt, N, F, rows, st)
    else:
        L.moe_gate_up(h.data_ptr(), h.stride(0), _ptr(gate), up.data_ptr(), meta.data_ptr(), order.data_ptr(),
                      act_.data_ptr(), E, maxt, top, F, K, float(limit), float(alpha), dt, pw, silu, st)
        L.moe_down(act_.data_ptr(), down.data_ptr(), meta.data_ptr(), y.data_ptr(), E, maxt, N, F, dt, st)
    if not combine:
        return MoEPending(y, place, None if weight_input else wts, shared, top, h if identity else None, shared_w)
    L.moe_combine(y.data_ptr(), place.data_ptr(), 0 if weight_input else wts.data_ptr(), _ptr(shared),
                  shared.stride(0) if shared is not None else 0, out.data_ptr(), T, N, top, dt,
                  h.data_ptr() if identity else 0, h.stride(0), _ptr(shared_w), st)
    return out


# ----------------------------------- residual streams / convolution tails / matrix-state recurrences / sink attention
def _i32(t, name, n=None):
    _check(t.dtype == torch.int32 and t.is_contiguous() and t.is_cuda, f"{name} must be contiguous int32 cuda")
    if n is not None:
        _check(t.numel() >= n, f"{name} too short")


def _f32c(t, name):
    _check(t.dtype == torch.float32 and t.is_contiguous() and t.is_cuda, f"{name} must be contiguous fp32 cuda")


def embed_streams(ids, positions, table, pos_table, streams):
    T = ids.numel()
    V, W = table.shape
    for t, nm in ((ids, "ids"), (positions, "positions")):
        _check(t.dtype == torch.int64 and t.is_contiguous() and t.is_cuda and t.numel() == T, f"{nm}: int64 [T] cuda")
    _check(table.is_contiguous(), "embedding table contiguous")
    if pos_table is not None:
        _check(pos_table.is_contiguous() and pos_table.dtype == table.dtype and pos_table.shape[1] == W,
               "position table [positions, W] in the table's storage type")
    x = torch.empty(streams, T, W, dtype=torch.float32, device=table.device)
    lib().embed_streams(ids.data_ptr(), positions.data_ptr(), table.data_ptr(), _ptr(pos_table), x.data_ptr(),
                        int(streams), T, W, V, pos_table.shape[0] if pos_table is not None else 1, _dt(table, "table"),
                        _stream())
    return x


def stream_add_norm(x, y, mix, outw, c, inw, w, eps, rms, out_dtype):
    S, T, W = x.shape
    _check(x.dtype == torch.float32 and x.is_contiguous() and x.is_cuda, "x fp32 [S, T, W] contiguous")
    dt = None
    if y is not None:
        _rows(y, "y", W)
        _check(y.shape[0] == T, "y rows")
        _f32c(mix, "mix")
        _f32c(outw, "outw")
        _check(mix.numel() == S * S and outw.numel() == S, "mix [S, S], outw [S]")
        dt = y.dtype
    h = None
    if w is not None:
        _check(w.is_contiguous() and w.numel() == W and w.is_cuda, "norm weight [W]")
        _check(dt is None or w.dtype == dt, "norm weight in y's storage type")
        dt = w.dtype
        if inw is not None:
            _f32c(inw, "inw")
            _check(inw.numel() == S, "inw [S]")
        _check(out_dtype in (dt, torch.float32), "h in the storage type or fp32")
        h = torch.empty(T, W, dtype=out_dtype, device=x.device)
    if dt is None or T == 0:
        return h
    _check(dt in _DT, "storage type bf16 / fp32")
    lib().stream_add_norm(x.data_ptr(), _ptr(y), y.stride(0) if y is not None else 0, _ptr(mix), _ptr(outw), float(c),
                          _ptr(inw) if w is not None else 0, _ptr(w), float(eps), int(bool(rms)), _ptr(h), W, S, T, W,
                          _DT[dt], int(h is not None and h.dtype == torch.float32), _stream())
    return h


def causal_conv(x, w, state, cu, ctx_lens, state_slots, residual, silu, out_dtype, bias=None, single=False):
    """``single``: every sequence of the step has one row - the tails are renewed in the same launch."""
    T, C = x.shape
    _rows(x, "x")
    taps = w.shape[1]
    _check(w.shape[0] == C and w.is_contiguous() and w.is_cuda, "conv weight [C, taps]")
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(state_slots, "state_slots", B)
    if taps > 1:
        _f32c(state, "state")
        _check(state.dim() == 3 and tuple(state.shape[1:]) == (taps - 1, C), "state [slots, taps - 1, C]")
    if bias is not None:
        _check(bias.dtype == w.dtype and bias.is_contiguous() and bias.numel() == C and bias.is_cuda, "conv bias [C]")
    _check(not single or T == B, "single: one row per sequence")
    out = torch.empty(T, C, dtype=out_dtype, device=x.device)
    lib().causal_conv(x.data_ptr(), x.stride(0), w.data_ptr(), _ptr(state) if taps > 1 else 0, cu.data_ptr(),
                      ctx_lens.data_ptr(), state_slots.data_ptr(), out.data_ptr(), C, T, B, C, taps,
                      int(bool(residual)), int(bool(silu)), _dt(x, "x"), _dt(w, "w"), _DT[out_dtype], _ptr(bias),
                      int(bool(single)), _stream())
    return out


def gated_group_norm(o, gate, w, eps, act, c, out=None, out_dtype=None, groups=0, gate_first=False):
    T, N = o.shape
    _rows(o, "o", dtype=torch.float32)
    if groups:
        _check(N % groups == 0 and w.numel() == N and w.is_contiguous(), "a weight per column, groups dividing the row")
        n = N // groups
    else:
        n = w.numel()
        _check(N % n == 0 and w.is_contiguous(), "the group size (len(w)) must divide the row")
    _rows(gate, "gate", N)
    if out is None:
        out = torch.empty(T, N, dtype=out_dtype, device=o.device)
    _rows(out, "out", N)
    _check(gate.dtype == w.dtype == out.dtype and gate.shape[0] == T and out.shape[0] == T, "gate / w / out types, rows")
    lib().gated_group_norm(o.data_ptr(), o.stride(0), gate.data_ptr(), gate.stride(0), w.data_ptr(), float(eps),
                           {"sigmoid": 0, "silu": 1}[act], float(c), out.data_ptr(), out.stride(0), T, N // n, n,
                           _dt(w, "w"), int(bool(groups)), int(bool(gate_first)), 0, 0, 1.0, _stream())
    return out


def glu_act(gu, F, act):
    T = gu.shape[0]
    _rows(gu, "gu")
    _check(gu.shape[1] >= 2 * F, "gate | up too narrow")
    out = torch.empty(T, F, dtype=gu.dtype, device=gu.device)
    lib().glu_act(gu.data_ptr(), gu.stride(0), out.data_ptr(), F, T, F, {"gelu_tanh": 0, "silu": 1}[act],
                  _dt(gu, "gu"), _stream())
    return out


def _rec_common(q, k, v, state, cu, ctx_lens, state_slots, heads, kv_heads, dim, vdim):
    T = q.shape[0]
    for t, nm, cols in ((q, "q", kv_heads * dim), (k, "k", kv_heads * dim), (v, "v", heads * vdim)):
        _rows(t, nm, cols)
        _check(t.shape[0] == T and t.dtype == q.dtype, f"{nm} rows / type")
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(state_slots, "state_slots", B)
    _f32c(state, "state")
    _check(state.dim() == 4 and tuple(state.shape[1:]) == (heads, dim, vdim), "state [slots, heads, dim, vdim]")
    return T, B, torch.empty(T, heads * vdim, dtype=torch.float32, device=q.device)


def decay_recurrence(q, k, v, decay, state, cu, ctx_lens, state_slots, heads, dim, vdim, silu_in=True):
    T, B, out = _rec_common(q, k, v, state, cu, ctx_lens, state_slots, heads, heads, dim, vdim)
    _f32c(decay, "decay")
    _check(decay.numel() == heads, "decay [heads]")
    if T and silu_in and T > B:
        # portions: every workgroup of a head stages the head's whole q and k, so the activation is applied once
        # beforehand (fp32 rows) instead of in each of them
        nqk, nv = heads * dim, heads * vdim
        act = torch.empty(T, 2 * nqk + nv, dtype=torch.float32, device=q.device)
        for src, off, n in ((q, 0, nqk), (k, nqk, nqk), (v, 2 * nqk, nv)):
            lib().silu_f32(src.data_ptr(), src.stride(0), act.data_ptr() + 4 * off, act.stride(0), T, n, _dt(src, "q"),
                           _stream())
        q, k, v, silu_in = act[:, :nqk], act[:, nqk:2 * nqk], act[:, 2 * nqk:], False
    if T:
        lib().recurrence(0, q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), k.stride(0), v.stride(0), 0, 0, 0, 0,
                         decay.data_ptr(), 0, state.data_ptr(), cu.data_ptr(), ctx_lens.data_ptr(),
                         state_slots.data_ptr(), out.data_ptr(), heads * vdim, B, heads, heads, dim, vdim,
                         int(bool(silu_in)), 0, _dt(q, "q"), 0, 0, 0, 0, _stream())
    return out


def _delta_args(q, a, b_, A_log, dt_bias, heads):
    T = q.shape[0]
    _f32c(A_log, "A_log")
    _f32c(dt_bias, "dt_bias")
    _check(A_log.numel() == heads and dt_bias.numel() == heads, "A_log, dt_bias [heads]")
    _rows(a, "a", heads)
    _rows(b_, "b", heads)
    # a and b are columns of one projection: addressed from a's base with b's offset in elements
    _check(a.dtype == b_.dtype and a.stride(0) == b_.stride(0) and a.shape[0] == T and b_.shape[0] == T
           and a.untyped_storage().data_ptr() == b_.untyped_storage().data_ptr(), "a and b: columns of one tensor")


def delta_recurrence(q, k, v, a, b_, A_log, dt_bias, state, cu, ctx_lens, state_slots, heads, kv_heads, dim, vdim, first=0):
    """``first``: the first sequence the walk takes (the rows of the sequences before it are left alone)."""
    T, B, out = _rec_common(q, k, v, state, cu, ctx_lens, state_slots, heads, kv_heads, dim, vdim)
    _delta_args(q, a, b_, A_log, dt_bias, heads)
    off_b = (b_.data_ptr() - a.data_ptr()) // a.element_size()
    ready = 0
    if T > B:  # portions: the per-token decay and write strength once per (token, head), not per workgroup
        gates = torch.empty(T, 2 * heads, dtype=torch.float32, device=q.device)
        lib().delta_gates(a.data_ptr(), b_.data_ptr(), a.stride(0), A_log.data_ptr(), dt_bias.data_ptr(),
                          gates.data_ptr(), T, heads, _dt(a, "a"), _stream())
        a, off_b, ready = gates, heads, 1
    if T:
        lib().recurrence(1, q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), k.stride(0), v.stride(0),
                         a.data_ptr(), a.stride(0), 0, int(off_b), A_log.data_ptr(), dt_bias.data_ptr(),
                         state.data_ptr(), cu.data_ptr() + 4 * first, ctx_lens.data_ptr() + 4 * first,
                         state_slots.data_ptr() + 4 * first, out.data_ptr(), heads * vdim, B - first, heads, kv_heads, dim,
                         vdim, 0, ready, _dt(q, "q"), _dt(a, "a"), 0, 0, 0, _stream())
    return out


_DELTA_MFMA = os.environ.get("LLMSS_DELTA_MFMA", "1") != "0"  # 0: portions token by token (A/B runs)


def delta_mix(q, k, v, a, b_, A_log, dt_bias, state, cu, ctx_lens, state_slots, heads, kv_heads, dim, vdim, gate, w, eps,
              scale, out, max_qlen=0, num_decode=0):
    """The ``num_decode`` leading single-row sequences (all of them when ``max_qlen`` is 1) take one fused launch; portions of
    bf16 rows the chunked form on the matrix cores, everything else the token-by-token walk, then the per-head norm and
    gate."""
    N = heads * vdim
    _rows(gate, "gate", N)
    _rows(out, "out", N)
    _check(w.is_contiguous() and w.numel() == vdim and gate.dtype == w.dtype == out.dtype and gate.shape[0] == q.shape[0]
           and out.shape[0] == q.shape[0], "gate / norm weight / out in one storage type")
    T, B = q.shape[0], cu.numel() - 1
    if T == 0:
        return out
    L, st, dt, es = lib(), _stream(), _dt(out, "out"), out.element_size()
    nd = B if max_qlen == 1 else int(num_decode)
    _check(0 <= nd <= B and (nd < B or T == B), "num_decode outside the step")
    same = q.dtype == k.dtype == v.dtype == a.dtype == out.dtype
    if not (same and L.delta_step_ok(dim, vdim) and state.data_ptr() % 16 == 0):
        nd = 0
    qkv = (q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), k.stride(0), v.stride(0))
    ab = (a.data_ptr(), b_.data_ptr(), a.stride(0), A_log.data_ptr(), dt_bias.data_ptr(), state.data_ptr())
    o = None
    if nd < B and not (same and q.dtype == torch.bfloat16 and max_qlen > 0 and _DELTA_MFMA and L.delta_chunk_ok(dim, vdim)
                       and not any(p % 16 for p in qkv[:2]) and not any(x % 8 for x in qkv[3:5])):
        o = delta_recurrence(q, k, v, a, b_, A_log, dt_bias, state, cu, ctx_lens, state_slots, heads, kv_heads, dim, vdim, nd)
    else:
        _, _, o = _rec_common(q, k, v, state, cu, ctx_lens, state_slots, heads, kv_heads, dim, vdim)
        _delta_args(q, a, b_, A_log, dt_bias, heads)
        if nd < B:
            work = torch.empty(4, T, heads, 64, dtype=torch.bfloat16, device=q.device)
            aux = torch.empty(T, heads, 4, dtype=torch.float32, device=q.device)
            L.delta_chunk(*qkv, *ab, cu.data_ptr() + 4 * nd, ctx_lens.data_ptr() + 4 * nd, state_slots.data_ptr() + 4 * nd,
                          o.data_ptr(), work.data_ptr(), aux.data_ptr(), T, B - nd, int(max_qlen), heads, kv_heads, dim,
                          vdim, st)
    if nd:
        L.delta_step(*qkv, *ab, cu.data_ptr(), ctx_lens.data_ptr(), state_slots.data_ptr(), gate.data_ptr(), gate.stride(0),
                     w.data_ptr(), float(eps), float(scale), out.data_ptr(), out.stride(0), nd, heads, kv_heads, dim, vdim,
                     dt, st)
    if nd < B:  # the portions' rows: nd .. T - 1 (single-row sequences come first)
        L.gated_group_norm(o.data_ptr() + 4 * nd * N, N, gate.data_ptr() + es * nd * gate.stride(0), gate.stride(0),
                           w.data_ptr(), float(eps), 1, float(scale), out.data_ptr() + es * nd * out.stride(0),
                           out.stride(0), T - nd, heads, vdim, dt, 0, 0, 0, 0, 1.0, st)
    return out


def rope_bias_cache(proj, off_q, off_k, off_v, bias, positions, table, rot, k_cache, v_cache, slots, heads, kv_heads,
                    dim, vdim):
    T = proj.shape[0]
    _rows(proj, "proj")
    nq, nk, nv = heads * dim, kv_heads * dim, kv_heads * vdim
    _check(min(off_q, off_k, off_v) >= 0 and max(off_q + nq, off_k + nk, off_v + nv) <= proj.shape[1],
           "q / k / v columns outside the projection")
    if bias is not None:
        _check(bias.dtype == proj.dtype and bias.is_contiguous() and bias.numel() == nq + nk + nv, "bias q | k | v")
    for c, n, nm in ((k_cache, nk, "k cache"), (v_cache, nv, "v cache")):
        _check(c.dtype == proj.dtype and c.is_contiguous() and c.dim() == 3 and c.shape[2] == n,
               f"{nm} [blocks, block_size, {n}] in the model's storage type")
    for t, nm in ((positions, "positions"), (slots, "slots")):
        _check(t.dtype == torch.int64 and t.is_contiguous() and t.is_cuda and t.numel() == T, f"{nm}: int64 [T] cuda")
    npos = 1
    if rot:
        _f32c(table, "angle table")
        _check(table.dim() == 3 and table.shape[1] == rot // 2 and table.shape[2] == 2, "angle table [npos, rot / 2, 2]")
        npos = table.shape[0]
    q = torch.empty(T, nq, dtype=torch.float32, device=proj.device)
    lib().rope_bias_cache(proj.data_ptr(), proj.stride(0), int(off_q), int(off_k), int(off_v), _ptr(bias),
                          positions.data_ptr(), _ptr(table) if rot else 0, npos, int(rot), q.data_ptr(),
                          k_cache.data_ptr(), v_cache.data_ptr(), slots.data_ptr(), T, heads, kv_heads, dim, vdim,
                          _dt(proj, "proj"), _stream())
    return q


_SINK_MFMA = os.environ.get("LLMSS_SINK_MFMA", "1") != "0"  # 0: every shape on the vector kernel (A/B runs)


def sink_attn(q, k_cache, v_cache, block_tables, cu, ctx_lens, heads, kv_heads, dim, vdim, scale, softcap,
              all_groups, max_qlen=0, num_decode=0, sink=True, chunk=0, vshare=1, precise=False):
    """``max_qlen`` (the longest portion of the step, known on the host) > 0: a bf16 cache of a shape the matrix-core
    kernel is built for runs on it, the ``num_decode`` leading single-row sequences in one launch and the portions
    in another; everything else runs the vector kernel. ``precise``: the matrix-core kernel takes queries and softmax
    weights as two bf16 numbers each (value and remainder), for designs that define scores and weights in 32-bit."""
    T = q.shape[0]
    _rows(q, "q", heads * dim, torch.float32)
    _check(q.is_contiguous(), "q contiguous")
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(block_tables, "block_tables")
    _check(block_tables.dim() == 2 and block_tables.shape[0] >= B, "block tables [B, blocks]")
    _check(vshare >= 1 and kv_heads % vshare == 0 and chunk >= 0, "vshare must divide the key heads")
    vh = kv_heads // vshare
    _check(k_cache.is_contiguous() and v_cache.is_contiguous() and k_cache.dtype == v_cache.dtype
           and k_cache.dim() == 3 and k_cache.shape[2] == kv_heads * dim and v_cache.shape[2] == vh * vdim
           and k_cache.shape[:2] == v_cache.shape[:2], "k / v cache [blocks, block_size, kv_heads * dim | vdim]")
    R = vh * vdim if all_groups else vdim
    out = torch.empty(T, heads, R, dtype=torch.float32, device=q.device)
    nd = int(num_decode)
    _check(0 <= nd <= B, "num_decode outside the step")
    mfma = (k_cache.dtype == torch.bfloat16 and max_qlen > 0 and lib().sink_attn_mfma_ok(dim, vdim, int(bool(precise)))
            and k_cache.data_ptr() % 16 == 0 and v_cache.data_ptr() % 16 == 0 and _SINK_MFMA)
    common = (heads, kv_heads, dim, vdim, k_cache.shape[1], float(scale), float(softcap or 0.0), int(bool(all_groups)),
              int(bool(sink)), int(chunk), int(vshare))
    if mfma:
        # the leading single-row sequences get a grid of their own (one row block each): in the portions' grid every
        # one of them would launch a whole prompt's worth of workgroups that exit at once, and those are not free
        maxb = block_tables.shape[1]
        for first, n, ql in ((0, nd, 1), (nd, B - nd, int(max_qlen))):
            if n > 0:
                lib().sink_attn_mfma(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(),
                                     block_tables.data_ptr() + 4 * first * maxb, maxb, cu.data_ptr() + 4 * first,
                                     ctx_lens.data_ptr() + 4 * first, out.data_ptr(), n, ql, *common,
                                     int(bool(precise)), 0, 0, 0, 1, 0, 0, 0, 0, 0, 0, _stream())
    else:
        lib().sink_attn(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), block_tables.data_ptr(),
                        block_tables.shape[1], cu.data_ptr(), ctx_lens.data_ptr(), out.data_ptr(), T, B, *common, 0, 0, 0,
                        _dt(k_cache, "k cache"), _stream())
    return out


def sink_attn_mix(q, k_cache, v_cache, block_tables, cu, ctx_lens, talk, c, heads, kv_heads, dim, vdim, scale, softcap,
                  out, max_qlen=0, num_decode=0, max_ctx=0):
    """Sink attention, head mixing and the branch scale, written to ``out`` [T, heads * vdim]: sink_attn (weighted
    sums of every head over all value groups when ``talk`` is given) followed by talk_mix. (A two-pass form for steps
    of single rows - scores of every head first, then mixed weights against each head's own group, so that keys and
    values are each read once - was measured at twice the time of the matrix-core kernel at 64 rows x 1024 keys:
    too few workgroups without a split over keys. It is not kept.)"""
    O = sink_attn(q, k_cache, v_cache, block_tables, cu, ctx_lens, heads, kv_heads, dim, vdim, scale, softcap,
                  talk is not None, max_qlen=max_qlen, num_decode=num_decode)
    return talk_mix(O, talk, c, heads, kv_heads, vdim, out=out)


def talk_mix(O, talk, c, heads, kv_heads, vdim, out=None, out_dtype=None):
    T = O.shape[0]
    R = kv_heads * vdim if talk is not None else vdim
    _check(O.dtype == torch.float32 and O.is_contiguous() and tuple(O.shape[1:]) == (heads, R), "O fp32 [T, heads, R]")
    if talk is not None:
        _f32c(talk, "talk")
        _check(talk.numel() == heads * heads, "talk [heads, heads]")
    if out is None:
        out = torch.empty(T, heads * vdim, dtype=out_dtype, device=O.device)
    _rows(out, "out", heads * vdim)
    lib().talk_mix(O.data_ptr(), _ptr(talk), float(c), out.data_ptr(), out.stride(0), T, heads, kv_heads, vdim,
                   _dt(out, "out"), _stream())
    return out


# ---------------------- blocks normed on the sublayer's output / depth average / bigram embedding / differential attention
def embed_bigram(ids, positions, table, scale, bigram, mul_prev, mul_cur, prev, cu, ctx_lens, state_slots, hist):
    T = ids.numel()
    V, W = table.shape
    for t, nm in ((ids, "ids"), (positions, "positions")):
        _check(t.dtype == torch.int64 and t.is_contiguous() and t.is_cuda and t.numel() == T, f"{nm}: int64 [T] cuda")
    _check(table.is_contiguous() and bigram.is_contiguous() and bigram.dtype == table.dtype and bigram.dim() == 2
           and bigram.shape[1] == W and bigram.shape[0] >= 2, "bigram table [buckets + 1, W] in the table's type")
    _check(prev.dtype == torch.int64 and prev.is_contiguous() and prev.is_cuda, "prev: int64 [slots] cuda")
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(state_slots, "state_slots", B)
    _check(hist.dtype == torch.float32 and hist.is_contiguous() and hist.dim() == 3 and hist.shape[0] >= 2
           and tuple(hist.shape[1:]) == (T, W) and hist.is_cuda, "hist fp32 [>= 2, T, W]")
    lib().embed_bigram(ids.data_ptr(), positions.data_ptr(), table.data_ptr(), float(scale), bigram.data_ptr(),
                       bigram.shape[0] - 1, int(mul_prev), int(mul_cur), prev.data_ptr(), cu.data_ptr(),
                       ctx_lens.data_ptr(), state_slots.data_ptr(), B, hist[0].data_ptr(), hist[1].data_ptr(), T, W, V,
                       _dt(table, "table"), _stream())


def resid_norm_add(hist, n, y, w, eps, dwa=None):
    S, T, W = hist.shape
    _check(hist.dtype == torch.float32 and hist.is_contiguous() and hist.is_cuda, "hist fp32 [slots, T, W]")
    _check(0 <= n < S - (1 if dwa is not None else 0), "hist slot outside the buffer")
    _rows(y, "y", W)
    _check(y.shape[0] == T and w.dtype == y.dtype and w.is_contiguous() and w.numel() == W, "y rows / norm weight")
    if dwa is not None:
        _f32c(dwa, "dwa")
        _check(dwa.numel() == n + 1, "dwa [n + 1]")
    lib().resid_norm_add(hist.data_ptr(), T * W, int(n), y.data_ptr(), y.stride(0), w.data_ptr(), float(eps),
                         _ptr(dwa), T, W, _dt(y, "y"), _stream())
    return hist[n + 1] if dwa is not None else hist[n]


def gate_mul(y, src, col):
    T, N = y.shape
    _rows(y, "y")
    _rows(src, "src")
    _check(src.dtype == y.dtype and src.shape[0] == T and 0 <= col and col + N <= src.shape[1], "gate columns")
    lib().gate_mul(y.data_ptr(), y.stride(0), src.data_ptr() + col * src.element_size(), src.stride(0), T, N,
                   _dt(y, "y"), _stream())
    return y


def act_fn(x, act, params=()):
    T, F = x.shape
    _rows(x, "x")
    out = torch.empty(T, F, dtype=x.dtype, device=x.device)
    a, b = (float(params[0]), float(params[1])) if act == "xielu" else (0.0, 0.0)
    lib().act_fn(x.data_ptr(), x.stride(0), out.data_ptr(), F, T, F, {"gelu_tanh": 0, "silu": 1, "xielu": 2, "gelu": 3, "relu2": 4}[act], a, b,
                 _dt(x, "x"), _stream())
    return out


def qk_norm_cache(proj, off_q, off_k, off_v, qw, kw, eps, k_cache, v_cache, slots, heads, kv_heads, maps, dim, vdim):
    T = proj.shape[0]
    _rows(proj, "proj")
    nq, nk, nv = heads * maps * dim, kv_heads * maps * dim, kv_heads * vdim
    _check(min(off_q, off_k, off_v) >= 0 and max(off_q + nq, off_k + nk, off_v + nv) <= proj.shape[1],
           "q / k / v columns outside the projection")
    for w_, nm in ((qw, "q norm"), (kw, "k norm")):
        if w_ is not None:
            _check(w_.dtype == proj.dtype and w_.is_contiguous() and w_.numel() == dim and w_.is_cuda, f"{nm} [dim]")
    for c, n, nm in ((k_cache, nk, "k cache"), (v_cache, nv, "v cache")):
        _check(c.dtype == proj.dtype and c.is_contiguous() and c.dim() == 3 and c.shape[2] == n,
               f"{nm} [blocks, block_size, {n}] in the model's storage type")
    _check(slots.dtype == torch.int64 and slots.is_contiguous() and slots.is_cuda and slots.numel() == T, "slots")
    q = torch.empty(T, nq, dtype=torch.float32, device=proj.device)
    lib().qk_norm_cache(proj.data_ptr(), proj.stride(0), int(off_q), int(off_k), int(off_v), _ptr(qw), _ptr(kw),
                        float(eps), q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), slots.data_ptr(), T, heads,
                        kv_heads, maps, dim, vdim, _dt(proj, "proj"), _stream())
    return q


def diff_combine(O, lam, eps, mult, heads, kv_heads, vdim, out_dtype):
    T = O.shape[0]
    _check(O.dtype == torch.float32 and O.is_contiguous() and tuple(O.shape[1:]) == (2 * heads, vdim) and O.is_cuda,
           "O fp32 [T, 2 * heads, vdim]")
    _check(out_dtype in _DT, "out dtype bf16 / fp32")
    y = torch.empty(T, heads * vdim, dtype=out_dtype, device=O.device)
    lib().diff_combine(O.data_ptr(), float(lam), float(eps), float(mult), y.data_ptr(), y.stride(0), T, heads,
                       kv_heads, vdim, _DT[out_dtype], _stream())
    return y


# ------------------- blocks normed on both sides / token input / windowed sigmoid attention with pooled blocks / SSD
def sandwich_add_norm(x, y, r, rb, wpost, eps, add, wnext, out_dtype, groups=1):
    """``y``: rows in the storage type, a :class:`MoEPending` (combined while it is read) or a ``PairPending`` (the results
    of two mixers, normed and joined while they are read)."""
    T, W = x.shape
    _rows(x, "x", dtype=torch.float32)
    _check(x.is_contiguous(), "x contiguous")
    _check(out_dtype in _DT, "storage type bf16 / fp32")
    pend = y if isinstance(y, MoEPending) else None
    pair = y if isinstance(y, PairPending) else None
    sh = None
    if pair is not None:
        for t_, nm in ((pair.yl, "left"), (pair.yr, "right")):
            _rows(t_, nm, W, out_dtype)
            _check(t_.shape[0] == T, "pair rows")
        for t_ in (pair.wl, pair.wr) if pair.scales is None else ():
            _f32c(t_, "pair weights")
            _check(t_.numel() == W, "pair weights [W]")
        y = pair.yl
    _check(groups >= 1 and W % groups == 0, "the norm's parts must divide the row")
    if pend is not None:
        _check(pend.y.shape == (T * pend.top, W) and pend.y.is_contiguous() and pend.place.numel() == T * pend.top,
               "pending expert outputs do not fit the stream")
        if pend.ident is not None:
            _rows(pend.ident, "ident", W, out_dtype)
            _check(pend.ident.shape[0] == T, "ident rows")
        if pend.wts is not None:
            _check(tuple(pend.wts.shape) == (T, pend.top) and pend.wts.is_contiguous(), "pending weights [T, top]")
        sh = pend.shared
        if sh is not None:
            _rows(sh, "shared", W, out_dtype)
    elif y is not None:
        _rows(y, "y", W, out_dtype)
        _check(y.shape[0] == T, "y rows")
    if y is not None:
        _f32c(wpost, "wpost")
        _check(wpost.numel() == W, "wpost [W]")
        if r is not None:
            _rows(r, "r", W, out_dtype)
            _f32c(rb, "rb")
            _check(r.shape[0] == T and rb.numel() == W, "gate logits [T, W], bias [W]")
    if add is not None:
        _f32c(add, "add")
        _check(tuple(add.shape) in ((T, W), (W,)), "add fp32 [T, W] or [W]")
    h = None
    if wnext is not None:
        _f32c(wnext, "wnext")
        _check(wnext.numel() == W, "wnext [W]")
        h = torch.empty(T, W, dtype=out_dtype, device=x.device)
    dense = y if pend is None else None
    lib().sandwich_add_norm(x.data_ptr(), _ptr(dense), dense.stride(0) if dense is not None else 0,
                            _ptr(pend.y) if pend else 0, _ptr(pend.place) if pend else 0,
                            _ptr(pend.wts) if pend else 0, pend.top if pend else 0, _ptr(sh),
                            sh.stride(0) if sh is not None else 0, _ptr(r) if y is not None else 0,
                            r.stride(0) if (r is not None and y is not None) else 0, _ptr(rb), _ptr(wpost), _ptr(add),
                            _ptr(wnext), _ptr(h), W, float(eps), int(groups),
                            _ptr(pend.ident) if pend else 0, pend.ident.stride(0) if pend and pend.ident is not None else 0,
                            _ptr(pair.yr) if pair else 0, pair.yr.stride(0) if pair else 0, _ptr(pair.wl) if pair else 0,
                            _ptr(pair.wr) if pair else 0, *(pair.scales if pair and pair.scales else (0.0, 0.0)),
                            W if add is not None and add.dim() == 2 else 0,
                            _ptr(pend.shared_w) if pend else 0, T, W, _DT[out_dtype], _stream())
    return h


def token_side_add(x, ids, table, col0, gate_w, proj_w, norm_w, eps, add, wnext, out_dtype):
    T, W = x.shape
    _rows(x, "x", dtype=torch.float32)
    _check(x.is_contiguous(), "x contiguous")
    d = gate_w.shape[0]
    _check(ids.dtype == torch.int64 and ids.is_contiguous() and ids.is_cuda and ids.numel() == T, "ids: int64 [T] cuda")
    _rows(table, "token table", dtype=out_dtype)
    _check(0 <= col0 and col0 + d <= table.shape[1], "the layer's columns lie outside the token table")
    _check(gate_w.dtype == out_dtype and gate_w.is_contiguous() and tuple(gate_w.shape) == (d, W) and gate_w.is_cuda,
           "gate [d, W] in the storage type")
    _check(proj_w.dtype == out_dtype and proj_w.is_contiguous() and tuple(proj_w.shape) == (W, d) and proj_w.is_cuda,
           "proj [W, d] in the storage type")
    _f32c(norm_w, "norm_w")
    _check(norm_w.numel() == W, "norm_w [W]")
    if add is not None:
        _f32c(add, "add")
        _check(tuple(add.shape) == (T, W), "add fp32 [T, W]")
    h = None
    if wnext is not None:
        _f32c(wnext, "wnext")
        _check(wnext.numel() == W, "wnext [W]")
        h = torch.empty(T, W, dtype=out_dtype, device=x.device)
    lib().token_side_add(x.data_ptr(), ids.data_ptr(), table.data_ptr(), table.stride(0), table.shape[0], int(col0), d,
                         gate_w.data_ptr(), proj_w.data_ptr(), norm_w.data_ptr(), _ptr(add), _ptr(wnext), _ptr(h), W,
                         float(eps), T, W, _DT[out_dtype], _stream())
    return h


def rope_pairs_cache(proj, off_q, off_k, off_v, cs, k_cache, v_cache, slots, heads, kv_heads, dim, vdim):
    T = proj.shape[0]
    _rows(proj, "proj")
    nq, nk, nv = heads * dim, kv_heads * dim, kv_heads * vdim
    _check(min(off_q, off_k, off_v) >= 0 and max(off_q + nq, off_k + nk, off_v + nv) <= proj.shape[1],
           "q / k / v columns outside the projection")
    for c, n, nm in ((k_cache, nk, "k cache"), (v_cache, nv, "v cache")):
        _check(c.dtype == proj.dtype and c.is_contiguous() and c.dim() == 3 and c.shape[2] == n,
               f"{nm} [blocks, block_size, {n}] in the model's storage type")
    _check(slots.dtype == torch.int64 and slots.is_contiguous() and slots.is_cuda and slots.numel() == T, "slots")
    rdims = 0
    if cs is not None:
        _f32c(cs, "angles")
        _check(cs.dim() == 3 and cs.shape[0] == T and cs.shape[2] == 2 and 2 * cs.shape[1] <= dim,
               "angles [T, rotated dims / 2, 2], rotated dims <= dim")
        rdims = 2 * cs.shape[1]
    q = torch.empty(T, nq, dtype=torch.float32, device=proj.device)
    lib().rope_pairs_cache(proj.data_ptr(), proj.stride(0), int(off_q), int(off_k), int(off_v), _ptr(cs), rdims,
                           q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), slots.data_ptr(), T, heads, kv_heads,
                           dim, vdim, _dt(proj, "proj"), _stream())
    return q


def _pool_caches(k_cache, v_cache, kp_cache, vp_cache, pool):
    _check(k_cache.is_contiguous() and v_cache.is_contiguous() and k_cache.dtype == v_cache.dtype and k_cache.dim() == 3
           and v_cache.dim() == 3 and k_cache.shape[:2] == v_cache.shape[:2] and k_cache.is_cuda,
           "k / v cache [blocks, block_size, n]")
    if not pool:
        return 0
    bs = k_cache.shape[1]
    per = -(-bs // pool)
    for c, full, nm in ((kp_cache, k_cache, "pooled keys"), (vp_cache, v_cache, "pooled values")):
        _check(c.is_cuda and c.is_contiguous() and c.dtype == full.dtype
               and tuple(c.shape) == (full.shape[0], per, full.shape[2]),
               f"{nm} [blocks, ceil(block_size / pool), n] in the pages' storage type")
    return per


def pool_update(k_cache, v_cache, kp_cache, vp_cache, block_tables, cu, ctx_lens, pool, max_qlen=0):
    """``max_qlen``: the step's longest portion (known on the host; bounds the blocks a portion can complete)."""
    per = _pool_caches(k_cache, v_cache, kp_cache, vp_cache, pool)
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(block_tables, "block_tables")
    _check(block_tables.dim() == 2 and block_tables.shape[0] >= B and pool >= 1 and max_qlen >= 1, "block tables, pool")
    lib().pool_update(k_cache.data_ptr(), v_cache.data_ptr(), kp_cache.data_ptr(), vp_cache.data_ptr(),
                      block_tables.data_ptr(), block_tables.shape[1], cu.data_ptr(), ctx_lens.data_ptr(), B,
                      int(max_qlen), k_cache.shape[2], v_cache.shape[2], k_cache.shape[1], int(pool), per,
                      _dt(k_cache, "k cache"), _stream())


_POOL_MFMA = os.environ.get("LLMSS_POOL_MFMA", "1") != "0"  # 0: every shape on the vector kernel (A/B runs)


def pool_key_split(B: int, kv_heads: int, window: int, pool: int, max_ctx: int) -> int:
    """Workgroups that share a single row's visible keys (at most min(window, max_ctx) positions and max_ctx / pool
    pooled blocks): about 1024 workgroups in flight, whole 64-key tiles per split, at most 16 splits."""
    keys = min(window, max_ctx) + (max_ctx // pool if pool else 0) if window > 0 else max_ctx
    tiles = -(-max(keys, 1) // 64)
    return max(1, min(tiles, 16, 1024 // max(1, B * kv_heads)))


def pool_window_attn(q, k_cache, v_cache, kp_cache, vp_cache, block_tables, cu, ctx_lens, pb, heads, kv_heads, dim,
                     vdim, scale, window, pool, out_dtype, max_qlen=0, num_decode=0, max_ctx=0):
    """``max_qlen`` (the longest portion of the step, known on the host) > 0: bf16 pages of a shape the matrix-core
    kernel is built for run on it, the ``num_decode`` leading single-row sequences in one launch - their keys split
    over workgroups when ``max_ctx`` (an upper bound of every context length) is given - and the portions in
    another; everything else runs the vector kernel."""
    T = q.shape[0]
    _rows(q, "q", heads * dim, torch.float32)
    _check(q.is_contiguous(), "q contiguous")
    per = _pool_caches(k_cache, v_cache, kp_cache, vp_cache, pool)
    _check(k_cache.shape[2] == kv_heads * dim and v_cache.shape[2] == kv_heads * vdim, "cache rows: kv_heads * dim | vdim")
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(block_tables, "block_tables")
    _check(block_tables.dim() == 2 and block_tables.shape[0] >= B, "block tables [B, blocks]")
    _f32c(pb, "pb")
    _check(pb.numel() == heads and out_dtype in _DT, "pb [heads]; out bf16 / fp32")
    out = torch.empty(T, heads * vdim, dtype=out_dtype, device=q.device)
    nd = int(num_decode)
    _check(0 <= nd <= B, "num_decode outside the step")
    al = lambda t: t is None or t.data_ptr() % 16 == 0
    if (k_cache.dtype == torch.bfloat16 and max_qlen > 0 and _POOL_MFMA and lib().pool_attn_mfma_ok(dim, vdim)
            and al(k_cache) and al(v_cache) and (not pool or (al(kp_cache) and al(vp_cache)))):
        maxb = block_tables.shape[1]
        for first, n, ql in ((0, nd, 1), (nd, B - nd, int(max_qlen))):
            if n <= 0:
                continue
            row0 = 0 if first == 0 else nd  # single-row sequences come first: sequence b's row is row b
            rows = n if ql == 1 else T - row0
            nsplit = pool_key_split(n, kv_heads, int(window), int(pool), int(max_ctx)) if ql == 1 and max_ctx > 0 else 1
            part = torch.empty(nsplit, rows, heads * vdim, dtype=torch.float32, device=q.device) if nsplit > 1 else None
            lib().pool_window_attn_mfma(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(),
                                        _ptr(kp_cache) if pool else 0, _ptr(vp_cache) if pool else 0,
                                        block_tables.data_ptr() + 4 * first * maxb, maxb, cu.data_ptr() + 4 * first,
                                        ctx_lens.data_ptr() + 4 * first, pb.data_ptr(), out.data_ptr(),
                                        int(out_dtype == torch.float32), _ptr(part), nsplit, row0, rows, n, ql, heads,
                                        kv_heads, dim, vdim, k_cache.shape[1], float(scale), int(window), int(pool),
                                        per, _stream())
        return out
    lib().pool_window_attn(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), _ptr(kp_cache) if pool else 0,
                           _ptr(vp_cache) if pool else 0, block_tables.data_ptr(), block_tables.shape[1], cu.data_ptr(),
                           ctx_lens.data_ptr(), pb.data_ptr(), out.data_ptr(), int(out_dtype == torch.float32), T, B,
                           heads, kv_heads, dim, vdim, k_cache.shape[1], float(scale), int(window), int(pool), per,
                           _dt(k_cache, "k cache"), _stream())
    return out


def ssd_recurrence(x, Bm, Cm, dt, A_log, dt_bias, D, state, cu, ctx_lens, state_slots, heads, groups, N, vdim):
    """The state-space scan on the matrix-state recurrence kernel: keys = B, queries = C (one per group), values = x."""
    T, B, out = _rec_common(Cm, Bm, x, state, cu, ctx_lens, state_slots, heads, groups, N, vdim)
    for t, nm in ((A_log, "A_log"), (dt_bias, "dt_bias"), (D, "D")):
        _f32c(t, nm)
        _check(t.numel() == heads, f"{nm} [heads]")
    _rows(dt, "dt", heads)
    _check(dt.shape[0] == T, "dt rows")
    if T:
        lib().recurrence(2, Cm.data_ptr(), Bm.data_ptr(), x.data_ptr(), Cm.stride(0), Bm.stride(0), x.stride(0),
                         dt.data_ptr(), dt.stride(0), 0, 0, A_log.data_ptr(), dt_bias.data_ptr(), state.data_ptr(),
                         cu.data_ptr(), ctx_lens.data_ptr(), state_slots.data_ptr(), out.data_ptr(), heads * vdim, B,
                         heads, groups, N, vdim, 0, 0, _dt(x, "x"), _dt(dt, "dt"), D.data_ptr(), 0, 0,
                         _stream())
    return out


def selective_scan(x, dt, dt_bias, Bm, Cm, A, D, z, state, cu, ctx_lens, state_slots, out_dtype):
    T, inner = x.shape
    N = A.shape[1]
    _rows(x, "x", dtype=out_dtype)
    _rows(z, "z", inner, out_dtype)
    _rows(dt, "dt", inner, torch.float32)
    _rows(Bm, "B", N, out_dtype)
    _rows(Cm, "C", N, out_dtype)
    _check(z.shape[0] == T and dt.shape[0] == T and Bm.shape[0] == T and Cm.shape[0] == T and Bm.stride(0) == Cm.stride(0),
           "rows of z / dt / B / C, one row stride for B and C")
    for t, nm, shp in ((A, "A", (inner, N)), (D, "D", (inner,)), (dt_bias, "dt_bias", (inner,))):
        _f32c(t, nm)
        _check(tuple(t.shape) == shp, f"{nm} {shp}")
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(state_slots, "state_slots", B)
    _f32c(state, "state")
    _check(state.dim() == 3 and tuple(state.shape[1:]) == (inner, N), "state [slots, inner, N]")
    out = torch.empty(T, inner, dtype=out_dtype, device=x.device)
    if T:
        lib().selective_scan(x.data_ptr(), x.stride(0), dt.data_ptr(), dt.stride(0), dt_bias.data_ptr(), Bm.data_ptr(),
                             Cm.data_ptr(), Bm.stride(0), A.data_ptr(), D.data_ptr(), z.data_ptr(), z.stride(0),
                             state.data_ptr(), cu.data_ptr(), ctx_lens.data_ptr(), state_slots.data_ptr(), out.data_ptr(),
                             inner, B, inner, N, int(T == B), _dt(x, "x"), _stream())
    return out


# ---------- heads on their way into the cache / softmax over a window with kept positions / exponential-gate recurrence
def head_prep_cache(proj, off_q, off_k, off_v, conv, tail, qw, kw, v_norm, eps, cs, vcs, k_cache, v_cache, slots, heads,
                    kv_heads, dim, vdim, cu, ctx_lens, state_slots, single=False, q_dtype=torch.float32):
    """``single``: every sequence of the step has one row - its workgroup then renews the convolution's tail as well."""
    T = proj.shape[0]
    _rows(proj, "proj")
    nq, nk, nv = heads * dim, kv_heads * dim, kv_heads * vdim
    _check(min(off_q, off_k, off_v) >= 0 and max(off_q + nq, off_k + nk, off_v + nv) <= proj.shape[1],
           "q / k / v columns outside the projection")
    for c, n, nm in ((k_cache, nk, "k cache"), (v_cache, nv, "v cache")):
        _check(c.dtype == proj.dtype and c.is_contiguous() and c.dim() == 3 and c.shape[2] == n and c.is_cuda,
               f"{nm} [blocks, block_size, {n}] in the model's storage type")
    _check(slots.dtype == torch.int64 and slots.is_contiguous() and slots.is_cuda and slots.numel() == T, "slots")
    for w_, nm in ((qw, "q norm"), (kw, "k norm")):
        if w_ is not None:
            _f32c(w_, nm)
            _check(w_.numel() == dim, f"{nm} [dim]")
    half = 0
    if cs is not None:
        _f32c(cs, "angles")
        _check(cs.dim() == 3 and cs.shape[0] == T and cs.shape[2] == 2 and 2 * cs.shape[1] <= dim,
               "angles [T, rotated dims / 2, 2], rotated dims <= dim")
        half = cs.shape[1]
    if vcs is not None:
        _f32c(vcs, "value angles")
        _check(tuple(vcs.shape) == (T, vdim // 2, 2) and vdim % 2 == 0, "value angles [T, vdim / 2, 2]")
    B = cu.numel() - 1
    taps = 0
    if conv is not None:
        taps = conv.shape[0]
        _check(conv.dtype == proj.dtype and conv.is_contiguous() and conv.is_cuda
               and tuple(conv.shape) == (taps, nq + nk + nv), "conv weight [taps, q | k | v columns]")
        _i32(cu, "cu")
        _i32(ctx_lens, "ctx_lens", B)
        _i32(state_slots, "state_slots", B)
        if taps > 1:
            _f32c(tail, "tail")
            _check(tail.dim() == 3 and tuple(tail.shape[1:]) == (taps - 1, nq + nk + nv), "tail [slots, taps - 1, columns]")
        _check(not single or T == B, "single: one row per sequence")
    _check(q_dtype == torch.float32 or q_dtype == proj.dtype, "queries in fp32 or the storage type")
    q = torch.empty(T, nq, dtype=q_dtype, device=proj.device)
    lib().head_prep(proj.data_ptr(), proj.stride(0), int(off_q), int(off_k), int(off_v), _ptr(conv), taps,
                    _ptr(tail) if taps > 1 else 0, int(bool(single)), cu.data_ptr(), ctx_lens.data_ptr(),
                    _ptr(state_slots) if conv is not None else 0, B, _ptr(qw), _ptr(kw), int(bool(v_norm)), float(eps),
                    _ptr(cs), half, _ptr(vcs), q.data_ptr(), int(q_dtype == torch.bfloat16), k_cache.data_ptr(),
                    v_cache.data_ptr(), slots.data_ptr(), T, heads, kv_heads, dim, vdim, _dt(proj, "proj"), _stream())
    return q


def window_q_dtype(k_cache, dim, vdim) -> torch.dtype:
    """Storage type window_attn wants its queries in: bf16 where the matrix-core kernel runs, else fp32."""
    ok = k_cache.dtype == torch.bfloat16 and _SINK_MFMA and lib().sink_attn_mfma_ok(dim, vdim, 1) and \
        k_cache.data_ptr() % 16 == 0
    return torch.bfloat16 if ok else torch.float32


def window_attn(q, k_cache, v_cache, block_tables, cu, ctx_lens, heads, kv_heads, dim, vdim, scale, softcap, window,
                keep_first, sinks, vcs, out_dtype, max_qlen=0, num_decode=0, max_ctx=0):
    """The sink attention kernels (csrc/attention_sink.hip) over a window with kept first positions. ``max_qlen`` (the longest
    portion, known on the host) > 0: bf16 pages of a shape the matrix-core kernel takes run on it, the ``num_decode``
    leading single-row sequences in one launch - their keys split over workgroups when ``max_ctx`` (an upper bound of every
    context length) is given - and the portions in another; everything else runs the vector kernel."""
    T = q.shape[0]
    _rows(q, "q", heads * dim)
    _check(q.is_contiguous() and q.dtype in _DT, "q contiguous, fp32 or bf16")
    B = cu.numel() - 1
    _i32(cu, "cu")
    _i32(ctx_lens, "ctx_lens", B)
    _i32(block_tables, "block_tables")
    _check(block_tables.dim() == 2 and block_tables.shape[0] >= B, "block tables [B, blocks]")
    _check(k_cache.is_contiguous() and v_cache.is_contiguous() and k_cache.dtype == v_cache.dtype and k_cache.is_cuda
           and k_cache.dim() == 3 and k_cache.shape[2] == kv_heads * dim and v_cache.shape[2] == kv_heads * vdim
           and k_cache.shape[:2] == v_cache.shape[:2], "k / v cache [blocks, block_size, kv_heads * dim | vdim]")
    _check(window >= 0 and keep_first >= 0 and out_dtype in _DT, "window, kept positions, out type")
    if sinks is not None:
        _f32c(sinks, "sinks")
        _check(sinks.numel() == heads, "sinks [heads]")
    if vcs is not None:
        _f32c(vcs, "value angles")
        _check(tuple(vcs.shape) == (T, vdim // 2, 2) and vdim % 2 == 0, "value angles [T, vdim / 2, 2]")
    y = torch.empty(T, heads * vdim, dtype=out_dtype, device=q.device)
    if T == 0:
        return y
    nd = int(num_decode)
    _check(0 <= nd <= B, "num_decode outside the step")
    sink, od = int(sinks is not None), _DT[out_dtype]
    maxb, bs = block_tables.shape[1], k_cache.shape[1]
    shape = (heads, kv_heads, dim, vdim, bs, float(scale), float(softcap or 0.0), 0, sink, 0, 1)
    L, st = lib(), _stream()
    if not (k_cache.dtype == torch.bfloat16 and max_qlen > 0 and L.sink_attn_mfma_ok(dim, vdim, 1) and _SINK_MFMA
            and k_cache.data_ptr() % 16 == 0 and v_cache.data_ptr() % 16 == 0):
        _check(q.dtype == torch.float32, "bf16 queries: matrix-core shapes and max_qlen only")
        O = torch.empty(T, heads, vdim, dtype=torch.float32, device=q.device)
        L.sink_attn(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), block_tables.data_ptr(), maxb, cu.data_ptr(),
                    ctx_lens.data_ptr(), O.data_ptr(), T, B, *shape, _ptr(sinks), int(window), int(keep_first),
                    _dt(k_cache, "k cache"), st)
        L.attn_finish(O.data_ptr(), 0, 1, 0, T, sink, _ptr(sinks), _ptr(vcs), y.data_ptr(), heads, vdim, od, st)
        return y
    for first, n, ql in ((0, nd, 1), (nd, B - nd, int(max_qlen))):
        if n <= 0:
            continue
        row0 = first  # single-row sequences come first: sequence b's row is row b
        rows = n if ql == 1 else T - row0
        nsplit = pool_key_split(n, kv_heads, int(window) + int(keep_first) if window else 0, 0, int(max_ctx)) \
            if ql == 1 and max_ctx > 0 else 1
        # straight into the result rows where no join and no turn-back over separate value tiles is left to do
        direct = nsplit == 1 and out_dtype == torch.bfloat16 and (vcs is None or vdim in (64, 128, 256)) and vdim % 4 == 0
        O = y if direct else torch.empty(nsplit, rows, heads, vdim, dtype=torch.float32, device=q.device)
        ml = torch.empty(nsplit, rows, heads, 2, dtype=torch.float32, device=q.device) if nsplit > 1 else None
        # (a finished fp32 block is addressed by the step's rows too: shift its base to row 0)
        out_ptr = y.data_ptr() if direct else O.data_ptr() - 4 * row0 * heads * vdim
        L.sink_attn_mfma(q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), block_tables.data_ptr() + 4 * first * maxb,
                         maxb, cu.data_ptr() + 4 * first, ctx_lens.data_ptr() + 4 * first, out_ptr, n, ql, *shape,
                         2 if q.dtype == torch.bfloat16 else 1,
                         _ptr(sinks), int(window), int(keep_first), nsplit, O.data_ptr() if nsplit > 1 else 0, _ptr(ml),
                         row0, rows, _ptr(vcs), int(direct), st)
        if not direct:
            L.attn_finish(O.data_ptr(), _ptr(ml), nsplit, row0, rows, sink, _ptr(sinks), _ptr(vcs), y.data_ptr(), heads,
                          vdim, od, st)
    return y


_MLSTM_MFMA = os.environ.get("LLMSS_MLSTM_MFMA", "1") != "0"  # 0: portions token by token (A/B runs)


def mlstm_mix(q, k, v, zi, zf, bi, bf, cap, S, n, m, cu, ctx_lens, state_slots, heads, dim, vdim, gate, w, eps, out_dtype,
              max_qlen=0, num_decode=0):
    """The ``num_decode`` leading single-row sequences (all of them when ``max_qlen`` is 1) take one fused launch; portions
    the gates' scan, then bf16 rows the chunked form on the matrix cores and everything else the token-by-token recurrence
    with the normaliser as one more column, then the per-head norm and gate."""
    T, B, num = _rec_common(q, k, v, S, cu, ctx_lens, state_slots, heads, heads, dim, vdim)
    for t, nm, shp in ((n, "n", (heads, dim)), (m, "m", (heads,))):
        _f32c(t, nm)
        _check(tuple(t.shape[1:]) == shp and t.shape[0] == S.shape[0], f"{nm} [slots, ...]")
    for t, nm in ((zi, "zi"), (zf, "zf")):
        _rows(t, nm, heads)
        _check(t.shape[0] == T and t.dtype == q.dtype and t.stride(0) == zi.stride(0), "gate columns of one projection")
    for t, nm in ((bi, "bi"), (bf, "bf")):
        _f32c(t, nm)
        _check(t.numel() == heads, f"{nm} [heads]")
    N = heads * vdim
    _rows(gate, "gate", N)
    _check(w.is_contiguous() and w.numel() == N and gate.dtype == w.dtype == out_dtype and gate.shape[0] == T,
           "gate / norm weight / out in one storage type")
    y = torch.empty(T, N, dtype=out_dtype, device=q.device)
    if T == 0:
        return y
    L, st, dt, es = lib(), _stream(), _dt(q, "q"), y.element_size()
    nd = B if max_qlen == 1 else int(num_decode)
    _check(0 <= nd <= B and (nd < B or T == B), "num_decode outside the step")
    if not (L.mlstm_step_ok(dim, vdim) and S.data_ptr() % 16 == 0):
        nd = 0
    zs = (zi.data_ptr(), zf.data_ptr(), zi.stride(0), bi.data_ptr(), bf.data_ptr(), float(cap))
    if nd:
        L.mlstm_step(q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), k.stride(0), v.stride(0), *zs, S.data_ptr(),
                     n.data_ptr(), m.data_ptr(), cu.data_ptr(), ctx_lens.data_ptr(), state_slots.data_ptr(),
                     gate.data_ptr(), gate.stride(0), w.data_ptr(), float(eps), float(dim) ** -0.5, y.data_ptr(), N, nd,
                     heads, dim, vdim, dt, st)
    if nd == B:
        return y
    # the portions: rows nd .. T - 1 (single-row sequences come first)
    seqs = (cu.data_ptr() + 4 * nd, ctx_lens.data_ptr() + 4 * nd, state_slots.data_ptr() + 4 * nd)
    gates = torch.empty(T, heads, 4, dtype=torch.float32, device=q.device)
    ab = torch.empty(T, 2 * heads, dtype=torch.float32, device=q.device)
    den = torch.empty(T, heads, dtype=torch.float32, device=q.device)
    L.mlstm_gates(*zs, m.data_ptr(), *seqs, gates.data_ptr(), ab.data_ptr(), B - nd, heads, dt, st)
    qkv = (q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), k.stride(0), v.stride(0))
    if (q.dtype == torch.bfloat16 and _MLSTM_MFMA and L.mlstm_chunk_ok(dim, vdim)
            and not any(p % 16 for p in qkv[:3]) and not any(x % 8 for x in qkv[3:])):
        L.mlstm_chunk(*qkv, gates.data_ptr(), S.data_ptr(), n.data_ptr(), *seqs, num.data_ptr(), den.data_ptr(), B - nd,
                      heads, dim, vdim, st)
    else:
        L.recurrence(2, *qkv, ab.data_ptr(), 2 * heads, 0, heads, 0, 0, S.data_ptr(), *seqs, num.data_ptr(), N, B - nd,
                     heads, heads, dim, vdim, 0, 1, dt, 1, 0, n.data_ptr(), den.data_ptr(), st)
    L.gated_group_norm(num.data_ptr() + 4 * nd * N, N, gate.data_ptr() + es * nd * gate.stride(0), gate.stride(0),
                       w.data_ptr(), float(eps), 0, 1.0, y.data_ptr() + es * nd * N, N, T - nd, heads, vdim, _dt(w, "w"), 1,
                       0, den.data_ptr() + 4 * nd * heads, gates.data_ptr() + 16 * nd * heads, float(dim) ** -0.5, st)
    return y
