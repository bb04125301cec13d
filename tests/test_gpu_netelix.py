"""GPU: the Netelix path (kernels of libhydra_mix.so, the model, the engine's scheduler / cache / state-slot managers)
against the float64 restatement in tests/netelix_oracle.py.  Small made-up configurations and random weights; float32 runs
are held to a tight tolerance (a window that is one token off, a lost state or a stale page moves the logits by percents),
bfloat16 runs to a loose one."""
import json
import math
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import netelix_oracle as oracle  # noqa: E402

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
TOL32, TOL16 = 2e-4, 6e-2
F = torch.float64


@pytest.fixture(autouse=True)
def _leave_the_device_rng_alone():
    state = torch.cuda.get_rng_state(DEV) if torch.cuda.is_available() else None
    yield
    if state is not None:
        torch.cuda.set_rng_state(state, DEV)


def _shape(kind: str):
    from hydrainfer_amd.layer.rotary_spec import RotarySpec as R
    from hydrainfer_amd.model.netelix import MixerSpec as M, NetelixLayer as L, NetelixShape
    att = lambda H, G, D, V, scale, window, mix, rot: M("attention", H, D, V, kv_heads=G, scale=scale, window=window, v_mix=mix, rot=rot)
    ret = lambda H, D, V, decay, rot: M("retention", H, D, V, decay=decay, rot=rot)
    lit = lambda H, D, V, decay: M("lightning", H, D, V, decay=decay)
    if kind == "hybrid":      # attention first; blended values in the second and the last attention; sizes of the matrix-core forms
        return NetelixShape(101, 96, [
            L(att(4, 4, 24, 16, 0.3, 33, False, R(8, 900.0)), 72),
            L(att(6, 3, 16, 40, 0.5, 24, True, R(16, 5000.0)), None),
            L(ret(3, 16, 24, [0.9, 0.99, 0.5], R(8, 1000.0)), None),
            L(lit(2, 40, 8, [0.97, 0.75]), 56),
            L(att(3, 3, 32, 40, 0.4, 17, True, R(12, 300.0)), 40)], norm_eps=1e-5)
    if kind == "odd":         # nothing a multiple of four: every kernel's element-by-element path; no rotation, window of one
        return NetelixShape(45, 38, [
            L(ret(3, 7, 5, [0.95, 0.3, 1.0], R(6, 77.0)), 26),
            L(att(3, 1, 6, 9, 0.6, 5, True, R(2, 50.0)), None),
            L(lit(1, 9, 11, [0.98]), 11),
            L(att(2, 1, 10, 9, 0.7, 1, True, R(10, 200.0)), 30),
            L(ret(2, 10, 3, [0.0, 0.9], None), None),
            L(att(5, 1, 7, 9, 0.5, None, True, None), None)], norm_eps=1e-4)
    if kind == "wide":        # states of the widest layout, several value blocks, heads of one
        return NetelixShape(61, 64, [
            L(lit(2, 130, 72, [0.995, 0.9]), None),
            L(ret(1, 64, 96, [0.99], R(64, 1e6)), 48),
            L(att(8, 2, 32, 32, 0.3, 40, True, R(32, 10000.0)), 96),
            L(lit(4, 128, 32, [0.5, 0.9, 0.99, 0.999]), None)], norm_eps=1e-6)
    if kind == "recurrent":   # no attention mixer: the cache pool has a plane nobody uses
        return NetelixShape(33, 48, [L(ret(6, 16, 8, [0.6 + 0.06 * i for i in range(6)], R(16, 100.0)), None),
                                     L(lit(3, 16, 16, [0.9, 0.8, 0.7]), 32)], norm_eps=1e-5)
    if kind == "attention":   # no recurrence: no state slots
        return NetelixShape(37, 40, [L(att(4, 2, 16, 16, 0.5, 9, False, R(8, 100.0)), 24),
                                     L(att(2, 2, 16, 8, 0.5, 21, True, R(16, 100.0)), None)], norm_eps=1e-5)
    raise KeyError(kind)


def _weights(shape, seed=0):
    from hydrainfer_amd.model.netelix import tensor_shapes
    g = torch.Generator().manual_seed(seed)
    W = {}
    for k, s in tensor_shapes(shape).items():
        tail = k.rsplit(".", 1)[-1]
        if tail in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.3 * torch.randn(s, generator=g)
        elif tail in ("ls1", "ls2"):
            t = 0.6 + 0.3 * torch.randn(s, generator=g)
        elif tail == "vmix":
            t = 0.2 + 0.6 * torch.rand(s, generator=g)
        elif k == "embed":
            t = torch.randn(s, generator=g)
        else:
            t = 1.5 * torch.randn(s, generator=g) / math.sqrt(s[-1])
        W[k] = t.to(torch.bfloat16).float()       # representable in a bfloat16 checkpoint: both dtypes see the same weights
    return W


def _model(shape, W, dtype):
    from hydrainfer_amd.model.llava import TextLanguageModel
    from hydrainfer_amd.model.netelix import NetelixForCausalLM
    return TextLanguageModel(NetelixForCausalLM.from_state_dict(shape, W, dtype, DEV))


def _replayer(lm, dtype, max_tokens, max_live=4):
    from hydrainfer_amd.engine.trace import TraceReplayer
    return TraceReplayer(lm, dtype, DEV, max_tokens, max_live_requests=max_live)


def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _run(rp, requests, schedule):
    """schedule: steps of [(request, n_tokens)]; every position's logits are wanted.  Returns {request: [n, vocab]}."""
    at = {r: 0 for r in requests}
    got = {r: [] for r in requests}
    with torch.inference_mode():
        for step in schedule:
            entries, end = [], []
            for r, n in step:
                toks = requests[r][at[r]:at[r] + n]
                entries.append({"id": r, "tokens": toks, "want": list(range(len(toks)))})
                at[r] += n
                if at[r] == len(requests[r]):
                    end.append(r)
            lg = rp.step(entries, end).float().cpu()
            o = 0
            for e in entries:
                got[e["id"]].append(lg[o:o + len(e["tokens"])])
                o += len(e["tokens"])
    return {r: torch.cat(v) for r, v in got.items()}


def _close(got, ref, tol, what=""):
    d = got.double().cpu() - ref
    assert torch.isfinite(d).all(), f"{what}: not finite"
    if tol < 1e-2:
        err = d.abs().max().item() / max(1.0, ref.abs().max().item())
    else:
        err = d.pow(2).mean().sqrt().item() / max(1e-6, ref.pow(2).mean().sqrt().item())
    assert err <= tol, f"{what}: relative error {err:.3e} > {tol}"


def _dev(t, dtype=torch.float32):
    return t.to(device=DEV, dtype=dtype).contiguous()


def _i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def _batch(state, parts):
    """parts: [(slot, first position, n tokens)] -> (SequenceState, q_cu, positions)."""
    from hydrainfer_amd._C.kernel.stream_ops import SequenceState
    q_cu, pos, tok_seq = [0], [], []
    for s, (slot, p0, n) in enumerate(parts):
        q_cu.append(q_cu[-1] + n)
        pos += list(range(p0, p0 + n))
        tok_seq += [s] * n
    return SequenceState(state, _i32([p[0] for p in parts]), _i32(tok_seq)), _i32(q_cu), _i32(pos)


def _through_portions(fn, inputs, plan, floats):
    """Two sequences "a" and "b" in portions through state slots 0 and 2 (plan: per step how many tokens of each), stale slots
    poisoned; then b's inputs whole through slot 0, which held a.  fn(rows {name: [n, ...]}, seq, q_cu, positions, longest
    portion).  Returns {"a", "b", "c"} and the state after each."""
    state = torch.full((3, 1, floats), 7.0, dtype=torch.float32, device=DEV)
    out, at, last = {"a": [], "b": [], "c": []}, {"a": 0, "b": 0}, {}
    for step in plan:
        parts = [(r, s, at[r], n) for r, s, n in zip("ab", (0, 2), step) if n]
        seq, q_cu, pos = _batch(state, [(s, p0, n) for _, s, p0, n in parts])
        rows = {k: torch.cat([inputs[r][k][p0:p0 + n] for r, _, p0, n in parts]) for k in inputs["a"]}
        y, o = fn(rows, seq, q_cu, pos, max(n for *_, n in parts)), 0
        for r, _, _, n in parts:
            out[r].append(y[o:o + n]); o += n
            at[r] += n
    assert all(at[r] == next(iter(inputs[r].values())).shape[0] for r in "ab")
    last["a"], last["b"] = state[0].cpu().clone(), state[2].cpu().clone()
    seq, q_cu, pos = _batch(state, [(0, 0, at["b"])])
    out["c"].append(fn(inputs["b"], seq, q_cu, pos, at["b"]))
    assert torch.all(state[1] == 7.0)                     # a slot nobody holds
    return {r: torch.cat(v).cpu() for r, v in out.items()}, last


# ------------------------------------------------------------------------------------------------ mechanisms alone
# steps: portions of one and two tokens, at, below and over a chunk of 32, one sequence joining late and sitting steps out
PLAN = [(5, 0), (1, 2), (2, 0), (1, 1), (0, 1), (31, 2), (32, 33), (2, 34), (1, 0), (75, 1), (1, 1), (1, 1)]
N_A, N_B = (sum(p[i] for p in PLAN) for i in (0, 1))


@pytest.mark.parametrize("H,D,V,decay,rot,act,layout,odd", [
    (2, 16, 16, [0.9, 0.99], None, None, "halves", 0), (3, 7, 5, [0.5, 1.0, 0.0], 6, None, "halves", 1), (2, 32, 48, [0.97, 0.001], 32, None, "halves", 0),
    (2, 40, 33, [0.98, 0.9], 8, None, "interleaved", 3), (1, 64, 96, [0.999], 64, None, "halves", 0), (2, 128, 128, [0.97, 0.65], None, "silu", "halves", 0),
    (2, 130, 72, [0.99, 0.95], None, "silu", "halves", 2), (1, 256, 20, [0.9], 16, None, "halves", 0), (4, 9, 300, [0.7, 0.8, 0.9, 1.0], None, "silu", "halves", 0),
    (1, 12, 1100, [0.9], 12, None, "interleaved", 0), (1, 1, 1, [0.9], None, "silu", "halves", 0)])
def test_decayed_sum_through_portions_and_slots(H, D, V, decay, rot, act, layout, odd):
    from hydrainfer_amd._C.kernel.decay_attn import decay_attention, decay_attention_gated, decay_powers
    g = torch.Generator().manual_seed(D + V)
    k_scale, base, eps = 0.3, 50.0, 1e-4
    powers = decay_powers(decay, DEV)
    freq = None if rot is None else torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F, device=DEV)
    at = [0, H * D, 2 * H * D, 2 * H * D + H * V, 2 * H * D + 2 * H * V]
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2 if act else 2e-5)):
        x = {r: torch.randn(n, at[-1] + odd, generator=g).to(dtype) for r, n in (("a", N_A), ("b", N_B))}
        ref, gated, states = {}, {}, {}
        for r in x:
            q, k, v, gt = (x[r][:, at[i] + odd:at[i + 1] + odd].to(F) for i in range(4))
            if act:
                q, k, v = oracle.silu(q), oracle.silu(k), oracle.silu(v)
            n = q.shape[0]
            q, k = q.reshape(n, H, D), k.reshape(n, H, D)
            if rot:
                q, k = (oracle.turned(z, torch.arange(n), rot, base, layout == "interleaved") for z in (q, k))
            o, S = oracle.decayed_sum(q, k * k_scale, v.reshape(n, H, V), decay)
            ref[r], states[r] = o.reshape(n, H * V), S.reshape(-1)
            gated[r] = oracle.over_rms(o, eps).reshape(n, H * V) * oracle.silu(gt)
        cols = lambda rows: [_dev(rows["x"], dtype)[:, at[i] + odd:at[i + 1] + odd] for i in range(4)]        # views of one projection
        args = lambda seq, q_cu, pos: (powers, seq, 4, q_cu, pos, H, D, V)                                    # the piece starts at 4
        kw = dict(act=act, k_scale=k_scale, inv_freq=freq, layout=layout)

        def plain(rows, seq, q_cu, pos, longest):
            q, k, v, _ = cols(rows)
            return decay_attention(q, k, v, *args(seq, q_cu, pos), max_q_len=longest, **kw)

        def finished(rows, seq, q_cu, pos, longest):
            q, k, v, gt = cols(rows)
            return decay_attention_gated(q, k, v, gt, *args(seq, q_cu, pos), eps=eps, gate_act="silu", max_q_len=longest, **kw)
        inputs = {r: {"x": x[r]} for r in x}
        got, last = _through_portions(plain, inputs, PLAN, 4 + H * D * V)
        for r, b in (("a", "a"), ("b", "b"), ("c", "b")):
            assert got[r].dtype == torch.float32
            _close(got[r], ref[b], tol, f"{dtype}: {r}")
        for r in "ab":
            _close(last[r][0, 4:], states[r], tol, f"{dtype}: the state of {r}")
            assert torch.all(last[r][0, :4] == 7.0)
        got, _ = _through_portions(finished, inputs, PLAN, 4 + H * D * V)
        for r, b in (("a", "a"), ("b", "b"), ("c", "b")):
            assert got[r].dtype == dtype
            _close(got[r], gated[b], 2e-2 if dtype == torch.bfloat16 else 5e-4, f"{dtype}: normed and gated, {r}")


@pytest.mark.parametrize("D,V", [(16, 16), (64, 40), (130, 33)])
def test_decayed_sum_asks_for_tokens_far_back(D, V):
    """Keys that carry next to nothing but for one, hundreds of tokens (many chunks) back: only a state carried through every
    chunk and portion in between returns its value, weakened by exactly decay ^ distance."""
    from hydrainfer_amd._C.kernel.decay_attn import decay_attention, decay_powers
    g = torch.Generator().manual_seed(V)
    n, mark, decay = 600, 37, [0.998]
    spike = torch.randn(D, generator=g)
    spike /= spike.norm()
    q, k, v = torch.randn(n, D, generator=g), 1e-3 * torch.randn(n, D, generator=g), torch.randn(n, V, generator=g)
    k[mark] = 30.0 * spike
    for i in (mark, mark + 1, 63, 64, 65, 96, 500, n - 2, n - 1):
        q[i] = spike
    ref, _ = oracle.decayed_sum(q.to(F)[:, None], k.to(F)[:, None], v.to(F)[:, None], decay)
    ref = ref[:, 0]
    want = 30.0 * decay[0] ** (n - 1 - mark) * v[mark].to(F)
    assert (ref[n - 1] - want).abs().max() < 0.1 * want.abs().max()
    powers = decay_powers(decay, DEV)
    for cuts in ([n], [100, 1, 2, 33, 64, 400], [40] + [2] * 30 + [470] + [1] * 30):
        state, at, out = torch.full((2, 1, D * V), 3.0, device=DEV), 0, []
        for c in cuts:
            seq, q_cu, pos = _batch(state, [(1, at, c)])
            out.append(decay_attention(_dev(q[at:at + c]), _dev(k[at:at + c]), _dev(v[at:at + c]), powers, seq, 0, q_cu, pos, 1, D, V, max_q_len=c))
            at += c
        assert at == n
        _close(torch.cat(out), ref, 1e-5, f"portions {cuts[:6]}")


@pytest.mark.parametrize("H,G,D,V,rd,layout,mag,pad", [(6, 2, 80, 56, 48, "interleaved", 1.0, 0), (6, 3, 16, 40, 16, "interleaved", 1.2, 0),
                                                       (3, 1, 6, 9, 2, "interleaved", 1.0, 0), (5, 2, 128, 128, 64, "halves", 1.0, 0),
                                                       (2, 2, 96, 24, 0, "halves", 1.0, 0), (2, 1, 10, 6, 4, "halves", 1.0, 1),
                                                       (2, 2, 256, 256, 256, "interleaved", 1.0, 0), (40, 4, 40, 8, 24, "interleaved", 1.0, 8),
                                                       (3, 3, 7, 5, 6, "halves", 0.9, 0)])
def test_head_norms_rotation_blended_values_and_cache_rows(H, G, D, V, rd, layout, mag, pad):
    """What a token's q | k | v row needs before attention, in one launch; sizes that take the eight-channel, the two-channel
    and the one-channel form."""
    from hydrainfer_amd._C.kernel.rotary import RotaryPart, rotary_parts
    g = torch.Generator().manual_seed(D + V)
    T, bs, base, eps, lam = 37, 16, 1000.0, 1e-3, 0.3
    nb = 4
    pos = torch.randint(0, 100000, (T,), generator=g)
    pos[0], pos[1] = 0, 99999
    slots = torch.randperm(nb * bs, generator=g)[:T]
    hs = max(D, V) + pad
    qw, kw = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.3 * torch.randn(D, generator=g)
    freq = None if rd == 0 else torch.tensor([base ** (-2.0 * i / rd) for i in range(rd // 2)], dtype=F, device=DEV)
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        x = (0.1 + torch.rand(T, 1, generator=g)) * torch.randn(T, pad + (H + G) * D + G * V, generator=g)
        first = torch.randn(T, pad + 3 + G * V, generator=g)
        x, first = x.to(dtype), first.to(dtype)
        q, k, v = x[:, pad:pad + H * D], x[:, pad + H * D:pad + (H + G) * D], x[:, pad + (H + G) * D:]
        turn = lambda z: oracle.turned(z, pos, rd, base, layout == "interleaved")
        scale_turned = lambda z: torch.cat([z[..., :rd] * mag, z[..., rd:]], dim=-1)
        qr = scale_turned(turn(oracle.head_norm(q.to(F).reshape(T, H, D), qw.to(F), eps)))
        kr = scale_turned(turn(oracle.head_norm(k.to(F).reshape(T, G, D), kw.to(F), eps)))
        vr = oracle.mixed_values(v.to(F), first[:, pad + 3:].to(F), lam).reshape(T, G, V)
        xd, fd = _dev(x, dtype), _dev(first, dtype)
        pool = torch.randn(2, nb, bs, G + 1, hs, generator=g).to(device=DEV, dtype=dtype)
        before = pool.clone()
        kc, vc = pool[0], pool[1]
        qd, kd, vd = xd[:, pad:pad + H * D], xd[:, pad + H * D:pad + (H + G) * D], xd[:, pad + (H + G) * D:]
        both = dict(inv_freq=freq, layout=layout, mag=mag, norm_eps=eps)
        outs = rotary_parts([RotaryPart(qd, H, D, norm_w=_dev(qw), **both),
                             RotaryPart(kd, G, D, norm_w=_dev(kw), cache=kc, cache_head_stride=hs, **both),
                             RotaryPart(vd, G, V, cache=vc, cache_head_stride=hs, mix=fd[:, pad + 3:], mix_w=lam)], _i32(pos.tolist()), _i32(slots.tolist()))
        assert outs[1] is None and outs[2] is None and outs[0].dtype == dtype
        _close(outs[0], qr.reshape(T, H * D), tol, f"{dtype} queries")
        flat, old = pool.view(2, nb * bs, G + 1, hs), before.view(2, nb * bs, G + 1, hs)
        sl = slots.to(DEV)
        _close(flat[0, sl, :G, :D], kr, tol, f"{dtype} cached keys")
        _close(flat[1, sl, :G, :V], vr, tol, f"{dtype} cached values")
        untouched = torch.ones(nb * bs, dtype=torch.bool); untouched[slots] = False
        assert torch.equal(flat[:, untouched.to(DEV)], old[:, untouched.to(DEV)]) and torch.equal(flat[:, :, G], old[:, :, G])
        assert torch.equal(flat[0, :, :G, D:], old[0, :, :G, D:]) and torch.equal(flat[1, :, :G, V:], old[1, :, :G, V:])
        # float results of either dtype, scaled (what enters a recurrence)
        o = rotary_parts([RotaryPart(qd, H, D, freq, layout=layout, mag=mag, f32=True),
                          RotaryPart(kd, G, D, freq, layout=layout, mag=mag, f32=True, scale=0.25)], _i32(pos.tolist()))
        assert o[0].dtype == o[1].dtype == torch.float32
        _close(o[0], scale_turned(turn(q.to(F).reshape(T, H, D))).reshape(T, H * D), 2e-6, f"{dtype} float queries")
        _close(o[1], 0.25 * scale_turned(turn(k.to(F).reshape(T, G, D))).reshape(T, G * D), 2e-6, f"{dtype} float keys")


@pytest.mark.parametrize("H,G,D,V,window,dtype", [(6, 2, 80, 56, 67, torch.bfloat16), (6, 2, 80, 56, 50, torch.float32), (3, 1, 6, 9, 5, torch.float32),
                                                  (8, 2, 32, 32, 40, torch.bfloat16), (6, 3, 16, 40, 24, torch.bfloat16), (2, 2, 128, 64, 300, torch.bfloat16),
                                                  (2, 1, 10, 9, 1, torch.float32), (5, 5, 24, 24, 33, torch.bfloat16)])
def test_window_attention_one_key_standing_out(H, G, D, V, window, dtype):
    """Keys and values of different sizes.  One key is made to stand out (some queries ask for exactly it): a query whose
    window still holds it returns its value, the next one must not see it — in rows of a prompt's portion and in rows decoded
    alone, at page borders, with other sequences' rows in the pool."""
    from hydrainfer_amd._C.kernel.biased_attn import biased_attention
    g = torch.Generator().manual_seed(D + window)
    bs, scale, n, mark = 16, 0.4, window + 70, 37
    k, v, q = 0.3 * torch.randn(n, G, D, generator=g), torch.randn(n, G, V, generator=g), 0.3 * torch.randn(n, H, D, generator=g)
    spike = torch.randn(D, generator=g)
    spike = spike / spike.norm() * 6.0
    k[mark] = spike
    for i in (mark, mark + 1, mark + window - 1, mark + window, n - 1):
        q[i] = spike * 3.0
    k, v, q = (t.to(dtype).to(F) for t in (k, v, q))
    ref = oracle.attend(q, k, v, scale, window)
    n_blocks = (n + bs - 1) // bs
    hs = max(D, V)
    pool = torch.randn(2, 2 * n_blocks + 3, bs, G, hs, generator=g).to(device=DEV, dtype=dtype)
    kc, vc = pool[0], pool[1]
    table = torch.randperm(2 * n_blocks + 3, generator=g)[:n_blocks]
    rows = (table[:, None] * bs + torch.arange(bs)[None, :]).reshape(-1)[:n].to(DEV)
    kc.view(-1, G, hs)[rows, :, :D] = k.to(device=DEV, dtype=dtype)
    vc.view(-1, G, hs)[rows, :, :V] = v.to(device=DEV, dtype=dtype)
    tol = 3e-2 if dtype == torch.bfloat16 else 1e-5
    for form in (("auto", "tile", "rows") if dtype == torch.bfloat16 else ("rows",)):
        for lo, hi in ((0, n), (0, 50), (50, n - 20)) + tuple((t, t + 1) for t in range(n - 20, n)) + ((mark + window - 1, mark + window), (mark + window, mark + window + 1)):
            T = hi - lo
            out = biased_attention(_dev(q[lo:hi], dtype), kc, vc, V, _i32([0] * T), _i32(list(range(lo, hi))), _i32([0, T]),
                                   _i32(table.tolist()), _i32([0, n_blocks]), scale, None, "window", window, max_q_len=T, kv_heads=G,
                                   max_kv_len=hi, form=form)
            _close(out, ref[lo:hi], tol, f"{form} rows {lo}..{hi}")
    inside, outside = ref[mark + window - 1, 0], ref[mark + window, 0]
    assert (inside - v[mark, 0]).abs().mean() < 0.1 * (outside - v[mark, 0]).abs().mean()


@pytest.mark.parametrize("W_", [96, 38, 2048])
def test_embedding_rows_and_output_norms(W_):
    from hydrainfer_amd._C.kernel.depth_ops import depth_norm
    g = torch.Generator().manual_seed(W_)
    T, vocab, eps = 21, 53, 1e-3
    table, w, ids = torch.randn(vocab, W_, generator=g), torch.randn(W_, generator=g), torch.randint(0, vocab, (T,), generator=g)
    for dtype, tol in ((torch.float32, 2e-6), (torch.bfloat16, 2e-2)):
        tb = table.to(dtype)
        ref = oracle.over_rms(tb.to(F)[ids], eps) * w.to(F)
        for it in (torch.int32, torch.int64):
            x, h = torch.empty(T, W_, device=DEV), torch.empty(T, W_, dtype=dtype, device=DEV)
            out = depth_norm(None, dtype, eps, y=_dev(tb, dtype), y_ids=ids.to(it).to(DEV), post_w=_dev(w), post_norm="rms", x_out=x, cast_out=h)
            assert out is h
            _close(x, ref, 2e-6, "embedding, normed")
            _close(h, ref, tol, "its operand copy")
        y = torch.randn(T, W_, generator=g).to(dtype)
        x0 = torch.randn(T, W_, generator=g)
        ref = x0.to(F) + oracle.over_rms(y.to(F), eps) * w.to(F)
        x = _dev(x0)
        depth_norm(x, dtype, eps, y=_dev(y, dtype), post_w=_dev(w), post_norm="rms", x_out=x, cast_out=h)
        _close(x, ref, 2e-6, "a normed result joins the residual")
        _close(h, ref, tol, "its operand copy")
    bad = torch.tensor([0, vocab, -1], device=DEV)                   # ids outside the table count as zeros
    x = torch.empty(3, W_, device=DEV)
    depth_norm(None, torch.float32, eps, y=_dev(table), y_ids=bad, post_w=_dev(w), post_norm="rms", x_out=x)
    assert torch.all(x[1:] == 0) and x[0].abs().max() > 0


def test_gated_feed_forward_and_joint_norm():
    from hydrainfer_amd._C.kernel.seq_mix import clamped_glu, gated_group_norm
    g = torch.Generator().manual_seed(3)
    for ff in (40, 26):
        gu = 3 * torch.randn(9, 2 * ff, generator=g)
        _close(clamped_glu(_dev(gu)[:, :ff], _dev(gu)[:, ff:], 0.0, 1.0, 0.0), oracle.silu(gu[:, :ff].to(F)) * gu[:, ff:].to(F), 1e-6, "silu gate")
    for n in (48, 33, 4096, 1100):
        o, gate, w = 4 * torch.randn(5, n, generator=g), torch.randn(5, n, generator=g), torch.randn(n, generator=g)
        ref = oracle.over_rms(o.to(F), 1e-3) * w.to(F) * oracle.sigmoid(gate.to(F))
        _close(gated_group_norm(_dev(o), torch.float32, group=n, eps=1e-3, w=_dev(w), gate=_dev(gate), gate_act="sigmoid"), ref, 1e-5, f"joint norm {n}")


# ------------------------------------------------------------------------------------------------ the model in the engine
@pytest.mark.parametrize("kind", ["hybrid", "odd", "wide", "recurrent", "attention"])
def test_whole_prompts_match_the_oracle_layer_by_layer(kind):
    shape = _shape(kind)
    W = _weights(shape, seed=11)
    toks = _tokens(75, shape.vocab_size, 4)
    passed = []
    ref = oracle.forward(shape.to_config(), W, toks, passed)
    for dtype, tol in ((torch.float32, TOL32), (torch.bfloat16, 0.1 if kind == "odd" else TOL16)):
        lm = _model(shape, W, dtype)
        rp = _replayer(lm, dtype, 128)
        lm.language_model.layer_trace = []
        got = _run(rp, {"a": toks}, [[("a", 75)]])["a"]
        trace, lm.language_model.layer_trace = lm.language_model.layer_trace, None
        assert len(trace) == len(passed) == len(shape.layers)
        for r, (a, b) in enumerate(zip(trace, passed)):
            _close(a.cpu(), b, tol, f"{kind} {dtype}: the residual after layer {r}")
        _close(got, ref, tol, f"{kind} {dtype}: logits")


def test_specs_the_engine_reads():
    h, r, a = (_model(_shape(k), _weights(_shape(k)), torch.float32).language_model for k in ("hybrid", "recurrent", "attention"))
    assert h.cache_spec() == {"n_layers": 3, "n_tokens": 2, "n_heads": 4, "head_size": 40} and h.shape.cache_plane == {0: 0, 1: 1, 4: 2}
    assert h.shape.state_piece == {2: 0, 3: 3 * 16 * 24} and h.state_spec() == {"rows": 1, "width": 3 * 16 * 24 + 2 * 40 * 8}
    assert r.cache_spec()["n_layers"] == 1 and r.shape.cache_plane == {} and a.state_spec() is None
    assert h.first_mixed == 1 and h.lw[1].v_mix is None and h.lw[4].v_mix is not None and a.lw[1].v_mix is None


@pytest.mark.parametrize("kind", ["hybrid", "odd", "wide", "attention"])
def test_decoding_token_by_token_and_portions_of_every_size_equal_the_whole_prompt(kind):
    shape = _shape(kind)
    W = _weights(shape, seed=13)
    n = 90
    toks = _tokens(n, shape.vocab_size, 6)
    ref = oracle.forward(shape.to_config(), W, toks)
    lm = _model(shape, W, torch.float32)
    rp = _replayer(lm, torch.float32, 96)
    # from the very first token on, one token a step: the first tokens of a sequence, every window and page edge
    got = _run(rp, {"a": toks}, [[("a", 1)] for _ in range(n)])["a"]
    _close(got, ref, TOL32, "decoded from the first token")
    # portions down to two tokens, cut inside pages, windows and chunks; then single tokens
    cuts = [2, 3, 2, 9, 16, 1, 15, 2, 7]
    cuts += [1] * (n - sum(cuts))
    got = _run(rp, {"b": toks}, [[("b", c)] for c in cuts])["b"]
    _close(got, ref, TOL32, "portions")
    got = _run(rp, {"c": toks}, [[("c", 33)], [("c", 31)], [("c", 26)]])["c"]
    _close(got, ref, TOL32, "three portions")


def test_mixed_batches_reused_pages_and_slots():
    """Five unequal requests through a pool for two and a half of them and three state slots: portions beside single
    tokens in one batch, requests that sit steps out, pages and slots handed on to later requests."""
    shape = _shape("hybrid")
    W = _weights(shape, seed=14)
    lens = {"a": 70, "b": 23, "c": 41, "d": 1, "e": 64}
    reqs = {r: _tokens(n, shape.vocab_size, 20 + i) for i, (r, n) in enumerate(lens.items())}
    ref = {r: oracle.forward(shape.to_config(), W, t) for r, t in reqs.items()}
    schedule = [[("a", 30), ("b", 2)], [("b", 1), ("a", 1)], [("a", 17), ("b", 20), ("c", 3)], [("c", 1)],
                [("a", 22), ("c", 30)],                                  # a ends: its pages and slot go back
                [("d", 1), ("c", 2)],                                    # d takes a's slot, ends at once
                [("e", 2), ("c", 1)], [("e", 31), ("c", 1)], [("c", 1), ("e", 1)], [("e", 30), ("c", 2)]]
    for dtype, tol in ((torch.float32, TOL32), (torch.bfloat16, TOL16)):
        lm = _model(shape, W, dtype)
        rp = _replayer(lm, dtype, 80 + 32 + 48, max_live=3)
        kv, sm = rp.node.kv_cache_block_manager, rp.node.batch_scheduler.context.state_manager
        free0 = len(kv.shared_cache.to_be_evicted)       # blocks no request holds
        assert free0 == kv.n_blocks
        got = _run(rp, reqs, schedule)
        for r in reqs:
            _close(got[r], ref[r], tol, f"request {r} in mixed batches ({dtype})")
        assert len(kv.shared_cache.to_be_evicted) == free0 and sm.get_num_available_slots() == 3
        assert sm.n_allocated_total == 5
        # and again on the used pool: every page and slot now has had an owner before
        got = _run(rp, {"a": reqs["a"], "e": reqs["e"]}, [[("a", 35), ("e", 64)], [("a", 35)]])
        _close(got["a"], ref["a"], tol, "second use of the pool")
        _close(got["e"], ref["e"], tol, "second use of the pool")


def test_long_decoding_past_several_windows():
    shape = _shape("hybrid")
    W = _weights(shape, seed=15)
    toks = _tokens(10 + 150, shape.vocab_size, 8)
    ref = oracle.forward(shape.to_config(), W, toks)
    for dtype, tol in ((torch.float32, TOL32), (torch.bfloat16, TOL16)):
        lm = _model(shape, W, dtype)
        got = _run(_replayer(lm, dtype, 160), {"a": toks}, [[("a", 10)]] + [[("a", 1)] for _ in range(150)])["a"]
        _close(got, ref, tol, f"150 decoded tokens ({dtype})")


def test_long_prompts_in_portions_with_slow_decays():
    """Several hundred tokens, decays next to one: what the first chunk left still counts in the last token."""
    shape = _shape("wide")
    for l in shape.layers:
        if l.mixer.recurrent:
            l.mixer.decay = [1.0 - 0.002 / (i + 1) for i in range(l.mixer.heads)]
    W = _weights(shape, seed=17)
    n = 420
    toks = _tokens(n, shape.vocab_size, 9)
    ref = oracle.forward(shape.to_config(), W, toks)
    other = oracle.forward(shape.to_config(), W, [(toks[0] + 1) % shape.vocab_size] + toks[1:])
    assert (other[-1] - ref[-1]).abs().max() > 20 * TOL32 * ref.abs().max()           # (the first token shows in the last logits)
    lm = _model(shape, W, torch.float32)
    rp = _replayer(lm, torch.float32, 448)
    for cuts in ([n], [130, 2, 63, 1, 100, 64, 40] + [1] * 20):
        assert sum(cuts) == n
        _close(_run(rp, {"a": toks}, [[("a", c)] for c in cuts])["a"], ref, TOL32, f"portions {cuts[:7]}")


def test_checkpoint_without_the_first_blend_and_values_blended_for_real():
    shape = _shape("hybrid")
    W = _weights(shape, seed=21)
    toks = _tokens(40, shape.vocab_size, 3)
    ref = oracle.forward(shape.to_config(), W, toks)
    W1 = {k: v for k, v in W.items() if k != "l1.mix.vmix"}              # the first blended layer's number is not used
    _close(_run(_replayer(_model(shape, W1, torch.float32), torch.float32, 48), {"a": toks}, [[("a", 40)]])["a"], ref, TOL32, "without it")
    W2 = dict(W, **{"l4.mix.vmix": torch.tensor(0.0)})
    off = oracle.forward(shape.to_config(), W2, toks)
    assert (off - ref).abs().max() > 50 * TOL32
    _close(_run(_replayer(_model(shape, W2, torch.float32), torch.float32, 48), {"a": toks}, [[("a", 40)]])["a"], off, TOL32, "weight zero")
    with pytest.raises(RuntimeError):
        _model(shape, {k: v for k, v in W.items() if k != "l4.mix.vmix"}, torch.float32)


def test_greedy_generation_through_the_offline_engine():
    """The framework's own entry point: requests in, the scheduler batches prompts (chunked under a small token budget)
    and decode steps, greedy tokens out.  Compared with the oracle wherever its top-1 margin is not a near-tie."""
    from hydrainfer_amd.engine.offline import OfflineInferenceEngine, OfflineRequest
    shape = _shape("hybrid")
    W = _weights(shape, seed=16)
    lm = _model(shape, W, torch.float32)
    eng = OfflineInferenceEngine(lm, None, torch.float32, device=DEV, max_running_requests=3, token_budgets=24,
                                 max_context=96, warm_up=False)
    prompts = [_tokens(n, shape.vocab_size, 30 + i) for i, n in enumerate((37, 5, 18, 50, 1))]
    n_new = 12
    outs = eng.generate([OfflineRequest(token_ids=p, max_tokens=n_new) for p in prompts])
    for p, o in zip(prompts, outs):
        want, margins = oracle.greedy(shape.to_config(), W, p, n_new)
        assert len(o.output_token_ids) == n_new
        for i, (a, b, m) in enumerate(zip(o.output_token_ids, want, margins)):
            if m < 1e-3:
                break            # a near-tie: either token is right, what follows depends on it
            assert a == b, f"prompt of {len(p)}: token {i} is {a}, the oracle says {b} (margin {m:.3g})"
    kv, sm = eng.node.kv_cache_block_manager, eng.node.batch_scheduler.context.state_manager
    assert sm.get_num_available_slots() == 3 and sm.n_allocated_total == 5
    assert len(kv.shared_cache.to_be_evicted) == kv.n_blocks


def test_registry_and_trace_run_command_line(tmp_path):
    """A checkpoint directory through the registry, and bin/trace_run as a user starts it: steps on standard input,
    `done <step>` lines and .f32 files out."""
    import subprocess
    import numpy as np
    import safetensors.torch
    from hydrainfer_amd.model.registry import architecture_of, load_model
    shape = _shape("odd")
    W = _weights(shape, seed=18)
    model_dir, out_dir = tmp_path / "model", tmp_path / "out"
    model_dir.mkdir()
    (model_dir / "config.json").write_text(json.dumps(shape.to_config()))
    safetensors.torch.save_file({k: v.to(torch.bfloat16) for k, v in W.items()}, str(model_dir / "model.safetensors"))
    assert architecture_of(str(model_dir)) == "Netelix"
    lm, vision = load_model(str(model_dir), torch.float32, DEV)
    assert vision is None and lm.language_model.shape.to_config() == shape.to_config()
    a, b = _tokens(21, shape.vocab_size, 40), _tokens(9, shape.vocab_size, 41)
    ra, rb = oracle.forward(shape.to_config(), W, a), oracle.forward(shape.to_config(), W, b)
    _close(_run(_replayer(lm, torch.float32, 32), {"a": a}, [[("a", 21)]])["a"], ra, TOL32, "loaded checkpoint")
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:8], "want": []}, {"id": "a", "tokens": a[17:18], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[18:], "want": [2]}, {"id": "b", "tokens": b[8:], "want": [0]}], "end": ["a", "b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(model_dir), "--dtype", "float32", "--out", str(out_dir),
                        "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True,
                       timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    read = lambda n: torch.from_numpy(np.fromfile(str(out_dir / f"{n}.f32"), dtype="<f4")).view(-1, shape.vocab_size)
    _close(read(0), ra[[0, 16]], TOL32, "step 0")
    _close(read(1), ra[[17]], TOL32, "step 1")
    _close(read(2), torch.cat([ra[[20]], rb[[8]]]), TOL32, "step 2")


def test_chat_endpoint_serves_a_checkpoint_directory(tmp_path):
    """`python -m hydrainfer_amd.entrypoint --checkpoint DIR` in parts: registry -> node -> front end -> HTTP endpoint.  The
    streams carry the tokens the offline engine generates for the same token ids."""
    import asyncio
    from types import SimpleNamespace
    import safetensors.torch
    from hydrainfer_amd.engine.offline import OfflineInferenceEngine, OfflineRequest
    from hydrainfer_amd.entrypoint.__main__ import build_checkpoint_server
    from hydrainfer_amd.entrypoint.api_protocol import parse_chat_completion_request as parse
    from tests.test_api_server import _client_stream, _payload
    shape = _shape("hybrid")
    W = _weights(shape, seed=19)
    (tmp_path / "config.json").write_text(json.dumps(shape.to_config()))
    safetensors.torch.save_file({k: v.to(torch.bfloat16) for k, v in W.items()}, str(tmp_path / "model.safetensors"))
    args = SimpleNamespace(checkpoint=str(tmp_path), max_running=4, max_tokens=128, tokenizer=None, host="127.0.0.1", port=0, dtype="fp32")
    server, front = build_checkpoint_server(args, torch.float32, torch.device(DEV))
    jobs = [("what a fine day it is today", 6), ("one two three four five six seven eight nine ten eleven twelve", 9), ("hello", 4)]

    async def go():
        await server.start()
        front.start()
        try:
            return await asyncio.gather(*[_client_stream(f"http://127.0.0.1:{server.port}/v1", _payload(t, None, n)) for t, n in jobs])
        finally:
            front.stop()
            await server.close()
    got = asyncio.run(go())
    assert front.error is None and front.n_admitted == len(jobs)
    eng = OfflineInferenceEngine.from_checkpoint(str(tmp_path), torch.float32, DEV, max_running_requests=4, max_context=128, warm_up=False)
    for (text, n_events, done), (prompt, n) in zip(got, jobs):
        assert done and n_events == n + 1 and len(text.split()) == n
        ids = server._token_request(parse(_payload(prompt, None, n))).token_ids
        want = eng.generate([OfflineRequest(token_ids=ids, max_tokens=n)])[0].output_token_ids
        assert text == "".join(server.tokenizer.decode(t) for t in want)
