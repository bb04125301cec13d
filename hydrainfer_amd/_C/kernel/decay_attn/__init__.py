"""Linear attention with a fixed decay per head (csrc/decay_attn.hip, libhydra_mix.so):
    S <- decay_h S + k v^T,   o = S^T q,
a float32 state [dim, vdim] per head and sequence in the sequence's state slot.  Portions of prompts run 32 tokens at a time
on the matrix cores with float operands; a batch of single tokens streams every state once, rotates q and k on their way
in and may finish with the head's norm and gate.  A portion that starts at position 0 starts from zeros without reading
its slot."""
import ctypes
from typing import List, Optional

import torch
from torch import Tensor

from hydrainfer_amd import _lib
from hydrainfer_amd._C.kernel.rotary import LAYOUTS, RotaryPart, rotary_parts
from hydrainfer_amd._C.kernel.seq_mix import ACT, _batch, _code, _f32, _piece, _ptr, _rows, gated_group_norm
from hydrainfer_amd._C.kernel.stream_ops import SequenceState

CHUNK = 32                    # HXM_DECAY_CHUNK


def decay_powers(decay: List[float], device) -> Tensor:
    """float32 [heads, CHUNK + 1]: decay_h ** n, each rounded once (decay ** 0 is 1, also of a decay of 0)."""
    return torch.tensor([[float(d) ** n for n in range(CHUNK + 1)] for d in decay], dtype=torch.float64).to(device=device, dtype=torch.float32)


def decay_attention(q: Tensor, k: Tensor, v: Tensor, powers: Tensor, seq: SequenceState, offset: int, q_cu: Tensor, positions: Tensor,
                    heads: int, dim: int, vdim: int, act: Optional[str] = None, k_scale: float = 1.0, max_q_len: int = 0,
                    inv_freq: Optional[Tensor] = None, layout: str = "halves") -> Tensor:
    """q, k: [n_tokens, heads * dim], v: [n_tokens, heads * vdim] (views of a projection's columns will do; q and k of one
    dtype), each through `act` first; with inv_freq (float64 [rot_dims / 2]) the first rot_dims channels of every head of q
    and k turn by the position; then k is multiplied by k_scale.  powers: decay_powers(...).  The slot's piece is heads * dim
    * vdim floats.  max_q_len 1: every sequence brings one token.  Returns o: float32 [n_tokens, heads * vdim]."""
    return _run(q, k, v, powers, seq, offset, q_cu, positions, heads, dim, vdim, act, k_scale, max_q_len, inv_freq, layout)


def decay_attention_gated(q: Tensor, k: Tensor, v: Tensor, gate: Tensor, powers: Tensor, seq: SequenceState, offset: int, q_cu: Tensor,
                          positions: Tensor, heads: int, dim: int, vdim: int, eps: float, gate_act: str = "silu",
                          act: Optional[str] = None, k_scale: float = 1.0, max_q_len: int = 0, inv_freq: Optional[Tensor] = None,
                          layout: str = "halves") -> Tensor:
    """decay_attention with every head's result divided by its root mean square (eps inside the root, no weight) and
    multiplied by gate_act(gate); [n_tokens, heads * vdim] of gate's dtype.  Single tokens: one launch."""
    if max_q_len == 1:
        return _run(q, k, v, powers, seq, offset, q_cu, positions, heads, dim, vdim, act, k_scale, 1, inv_freq, layout, gate, gate_act, eps)
    o = _run(q, k, v, powers, seq, offset, q_cu, positions, heads, dim, vdim, act, k_scale, max_q_len, inv_freq, layout)
    return gated_group_norm(o, gate.dtype, group=vdim, eps=eps, gate=gate, gate_act=gate_act)


def _run(q, k, v, powers, seq, offset, q_cu, positions, heads, dim, vdim, act, k_scale, max_q_len, inv_freq, layout, gate=None,
         gate_act="silu", eps=0.0):
    _lib.require_gpu(q, k, v, powers, inv_freq, gate)
    single = max_q_len == 1
    if inv_freq is not None and not single:
        # portions: q and k turned by a row kernel, left as float (they enter the recurrence)
        if act not in (None, "none"):
            raise _lib.HydraHipError("decay_attention: an activation and a rotation together are for single tokens only")
        q, k = rotary_parts([RotaryPart(q, heads, dim, inv_freq, layout=layout, f32=True),
                             RotaryPart(k, heads, dim, inv_freq, layout=layout, f32=True, scale=k_scale)], positions)
        k_scale, inv_freq = 1.0, None
    _rows(q, heads * dim, "decay_attention: q")
    T = q.shape[0]
    _rows(k, heads * dim, "decay_attention: k", T, q.dtype); _rows(v, heads * vdim, "decay_attention: v", T)
    _f32(powers, heads * (CHUNK + 1), "decay_attention: powers")
    n_seq = _batch(seq, q_cu, positions, T, "decay_attention")
    if single and T > n_seq:
        raise _lib.HydraHipError("decay_attention: max_q_len 1 with more tokens than sequences")
    base, stride = _piece(seq, offset, heads * dim * vdim, "decay_attention")
    if gate is not None:
        _rows(gate, heads * vdim, "decay_attention: gate", T)
    out = torch.empty((T, heads * vdim), dtype=torch.float32 if gate is None else gate.dtype, device=q.device)
    a = _lib.hxm_decay_attn_args()
    a.out, a.q, a.k, a.v = out.data_ptr(), q.data_ptr(), k.data_ptr(), v.data_ptr()
    a.out_stride, a.q_stride, a.k_stride, a.v_stride = out.stride(0), q.stride(0), k.stride(0), v.stride(0)
    a.qk_dtype, a.v_dtype, a.act, a.k_scale, a.decay_pow = _code(q.dtype), _code(v.dtype), ACT[act], float(k_scale), powers.data_ptr()
    a.state, a.slot_stride, a.slots, a.q_cu, a.positions = base, stride, seq.slots.data_ptr(), q_cu.data_ptr(), positions.data_ptr()
    a.n_tokens, a.n_seq, a.heads, a.dim, a.vdim, a.single = T, n_seq, int(heads), int(dim), int(vdim), int(single)
    a.inv_freq, a.rot_dims, a.layout = None, 0, LAYOUTS[layout]
    if inv_freq is not None:
        if inv_freq.dtype != torch.float64 or not inv_freq.is_contiguous() or not 1 <= inv_freq.numel() <= dim // 2:
            raise _lib.HydraHipError("decay_attention: inv_freq must be contiguous float64 [rot_dims / 2], rot_dims at most dim")
        a.inv_freq, a.rot_dims = inv_freq.data_ptr(), 2 * inv_freq.numel()
    a.finish, a.gate, a.gate_stride = int(gate is not None), _ptr(gate), gate.stride(0) if gate is not None else 0
    a.gate_act, a.eps, a.dtype = ACT[gate_act], float(eps), _code(out.dtype)
    _lib.mix_check(_lib.mix_lib().hxm_decay_attention(ctypes.byref(a), _lib.current_stream()), "decay_attention")
    return out
