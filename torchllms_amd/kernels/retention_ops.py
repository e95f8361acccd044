"""Retention: linear attention whose state fades by a constant per head, over rotated queries and keys, with the norm
of every head's result and its gate."""

from __future__ import annotations

from typing import Optional

import torch

from .base import KernelError, _gpu, _ptr, _stream, check, core, dtype_code
from .sequence_ops import ScanSegments, _step_rows, state_region

#: the most channels of a key that the kernels take (values: any number)
RETENTION_MAX_KEY_DIM = 256
#: tokens of a segment when a prompt's segments run side by side, the longest row of a step from which on they do, and
#: the most channels of keys and of values for which they do
RETENTION_SEGMENT = 64
RETENTION_SEGMENTS_FROM = 32
RETENTION_SEGMENT_CHANNELS = 128


def retention_segments_supported(dtype: torch.dtype, head_dim: int, v_head_dim: int, rotary_dim: int) -> bool:
    """Whether ``retention`` takes segments for these sizes (bfloat16 models: in 32-bit every row is walked in one piece,
    so that no bit depends on how a prompt was cut into steps)."""
    return (dtype == torch.bfloat16 and head_dim % 4 == 0 and v_head_dim % 4 == 0 and rotary_dim % 8 == 0
            and max(head_dim, v_head_dim) <= RETENTION_SEGMENT_CHANNELS)


def retention(
    proj: torch.Tensor,
    q_offset: int,
    k_offset: int,
    v_offset: int,
    gate_offset: int,
    cos_sin: Optional[torch.Tensor],
    rotary_dim: int,
    decay: torch.Tensor,
    eps: float,
    state: torch.Tensor,
    state_offset: int,
    qo_indptr: torch.Tensor,
    slot_ids: torch.Tensor,
    n_heads: int,
    head_dim: int,
    v_head_dim: int,
    segments: Optional[ScanSegments] = None,
    single_rows: int = 0,
) -> torch.Tensor:
    """Retention over each request's tokens, in 32-bit.  Of ``proj`` [n, ..] the columns of q and k (H heads of dk each),
    v and the gate (H heads of dv) are read from their offsets.  q and k are rotated on the way (the first ``rotary_dim``
    channels of a head, channel i with channel i + rotary_dim / 2, by the step's table ``cos_sin`` float32
    [n, rotary_dim / 2, 2]) and k is multiplied by dk^-1/2.  Per head ``S <- decay[h] S + k v^T; o = S^T q``; then o over
    its root mean square, times silu of the gate.  ``S`` lives at ``state_offset`` of the request's state row,
    H * dv * dk floats.  Returns [n, H * dv].

    With ``segments`` (of at most ``RETENTION_SEGMENT`` tokens, bfloat16; see ``retention_segments_supported``) the first
    ``single_rows`` rows of the step, one token each, are walked, and of the others the segments run side by side on the
    matrix cores (32-bit ones): what a segment leaves by itself, the states that enter the segments, the results."""
    _gpu(proj, cos_sin, decay)
    H, dk, dv = n_heads, head_dim, v_head_dim
    n = proj.shape[0]
    if proj.dim() != 2 or proj.stride(1) != 1:
        raise KernelError("retention: proj must be a matrix with contiguous rows")
    for off, size, what in ((q_offset, H * dk, "q"), (k_offset, H * dk, "k"), (v_offset, H * dv, "v"), (gate_offset, H * dv, "gate")):
        if off < 0 or off + size > proj.shape[1]:
            raise KernelError(f"retention: the columns of {what} do not lie in the rows of proj")
    if rotary_dim < 0 or rotary_dim % 2 or rotary_dim > dk:
        raise KernelError(f"retention: {rotary_dim} rotated channels of a head of {dk}")
    if rotary_dim > 0 and (cos_sin is None or cos_sin.dtype != torch.float32 or tuple(cos_sin.shape) != (n, rotary_dim // 2, 2)
                           or not cos_sin.is_contiguous()):
        raise KernelError(f"retention: cos_sin must be contiguous float32 [{n}, {rotary_dim // 2}, 2]")
    if tuple(decay.shape) != (H,) or decay.dtype != torch.float32 or not decay.is_contiguous():
        raise KernelError(f"retention: decay must be a float32 vector of {H} entries")
    n_seqs = _step_rows(None, qo_indptr, slot_ids, n, state)
    region, stride = state_region(state, state_offset, H * dv * dk)
    out = torch.empty((n, H * dv), dtype=proj.dtype, device=proj.device)
    if segments is not None:
        if not retention_segments_supported(proj.dtype, dk, dv, rotary_dim) or segments.length > RETENTION_SEGMENT:
            raise KernelError(f"retention: segments are not for {proj.dtype} with {dk} and {dv} channels, {rotary_dim} rotated, or too long")
        n_rows = n_seqs - single_rows
        if not 0 <= single_rows <= n_seqs or segments.row_seg.numel() != n_rows + 1:
            raise KernelError("retention: the segments are not those of this step's rows")
        if single_rows:
            check(
                core().tl_retention(
                    proj.data_ptr(), proj.stride(0), q_offset, k_offset, v_offset, gate_offset, _ptr(cos_sin), rotary_dim, decay.data_ptr(),
                    region, stride, qo_indptr.data_ptr(), slot_ids.data_ptr(), out.data_ptr(), None, single_rows, single_rows, H, dk, dv,
                    float(eps), dtype_code(proj.dtype), _stream(),
                )
            )
        ws = torch.empty((segments.n, H * dv * dk), dtype=torch.float32, device=proj.device)
        slots = slot_ids[single_rows:]
        check(
            core().tl_retention_chunks(
                proj.data_ptr(), proj.stride(0), q_offset, k_offset, v_offset, gate_offset, _ptr(cos_sin), rotary_dim, decay.data_ptr(), region,
                stride, slots.data_ptr(), out.data_ptr(), n_rows, H, dk, dv, float(eps), segments.segs.data_ptr(), segments.row_seg.data_ptr(),
                segments.n, ws.data_ptr(), dtype_code(proj.dtype), _stream(),
            )
        )
        return out
    o_raw = None
    if dv > core().tl_retention_block_columns():
        o_raw = torch.empty((n, H * dv), dtype=torch.float32, device=proj.device)
    check(
        core().tl_retention(
            proj.data_ptr(), proj.stride(0), q_offset, k_offset, v_offset, gate_offset, _ptr(cos_sin), rotary_dim, decay.data_ptr(), region,
            stride, qo_indptr.data_ptr(), slot_ids.data_ptr(), out.data_ptr(), _ptr(o_raw), n, n_seqs, H, dk, dv, float(eps),
            dtype_code(proj.dtype), _stream(),
        )
    )
    return out
