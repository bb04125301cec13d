"""Netelix — a decoder-only hybrid of two linear attentions with fixed decays and windowed attention, normed behind its
sublayers only:

  * x = rms_norm(embed[token]) * w; a layer is x <- x + ls1 * norm_1(mixer(x)), then (if it has a feed-forward)
    x <- x + ls2 * norm_2(ff(x)): the sublayers read the residual itself, what they return is RMS-normed, weighted and
    scaled channel by channel;
  * mixer `retention`: q, k with rotary positions (channels i, i + dims / 2), k times dim^-1/2; per head
    S <- decay_h S + k v^T, o = S^T q; every head's o over its root mean square, times silu(W_g x), then W_o;
  * mixer `lightning`: q, k, v through silu, the same recurrence without positions; the concatenated heads RMS-normed
    together with a weight, times sigmoid(W_g x), then W_o;
  * mixer `attention`: grouped-query attention, an RMS norm with a weight on every head of q and k, then rotary positions
    (channels 2 i, 2 i + 1), a sliding window; in every layer marked for it but the first such, the values are blended with
    that first layer's values of the same token (one learned number per layer), and so cached;
  * feed-forward: W_down (silu(W_gate x) * W_up x);
  * logits = head . norm(x).

Every size and constant comes from config.json (`NetelixShape.from_config`), every tensor from model.safetensors under the
names of `tensor_shapes`.  The residual, norms, angles, turned queries and keys of the recurrences, decays, states, scores
and softmax weights are float32; the matrix products run in the model's dtype (bfloat16 with float accumulation, or
float32).

The compute path: library GEMMs (torch.matmul) for the projections and the kernels of libhydra_mix.so (_C.kernel.decay_attn,
.rotary, .biased_attn, .depth_ops, .seq_mix).  The model plugs into the engine through the interface LlamaForCausalLM has;
`cache_spec` asks the block manager for a key and a value plane per attention mixer, `state_spec` asks the state-slot
manager for one flat row per sequence in which every recurrent mixer owns its matrix states."""
import json
import math
import os
from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch
from torch import Tensor

from hydrainfer_amd._C.kernel.biased_attn import biased_attention
from hydrainfer_amd._C.kernel.decay_attn import decay_attention, decay_attention_gated, decay_powers
from hydrainfer_amd._C.kernel.depth_ops import depth_norm
from hydrainfer_amd._C.kernel.rotary import RotaryPart, rotary_parts
from hydrainfer_amd._C.kernel.seq_mix import clamped_glu, gated_group_norm
from hydrainfer_amd._C.kernel.stream_ops import SequenceState
from hydrainfer_amd.layer.rotary_spec import RotarySpec

ARCHITECTURE = "Netelix"


@dataclass
class MixerSpec:
    type: str                         # "retention" | "lightning" | "attention"
    heads: int
    dim: int                          # q / k size per head
    vdim: int                         # v size per head
    decay: List[float] = field(default_factory=list)      # retention, lightning: one per head
    kv_heads: int = 0                 # attention
    scale: float = 1.0                # attention
    window: Optional[int] = None      # attention: position i sees j with 0 <= i - j < window; None: every j <= i
    v_mix: bool = False               # attention: values are blended with those of the first such layer
    rot: Optional[RotarySpec] = None  # retention, attention

    @property
    def recurrent(self) -> bool:
        return self.type != "attention"


@dataclass
class NetelixLayer:
    mixer: MixerSpec
    ff: Optional[int] = None          # inner size of the feed-forward; None: the layer has none


def _round4(n: int) -> int:
    return (n + 3) // 4 * 4


@dataclass
class NetelixShape:
    vocab_size: int
    hidden_size: int
    layers: List[NetelixLayer]
    norm_eps: float = 1e-6
    cache_plane: Dict[int, int] = field(default_factory=dict)          # layer with attention -> its cache plane
    state_piece: Dict[int, int] = field(default_factory=dict)          # layer with a recurrence -> first float in a slot
    state_floats: int = 0
    max_position_embeddings: int = 1 << 24      # positions are computed, not looked up: no table bounds them

    def __post_init__(self):
        self.cache_plane, self.state_piece, at = {}, {}, 0
        mixed = None
        for i, l in enumerate(self.layers):
            m = l.mixer
            if m.rot and (m.rot.dims % 2 or m.rot.dims > m.dim):
                raise ValueError(f"layer {i}: rot.dims must be even and at most dim")
            if m.type in ("retention", "lightning"):
                if len(m.decay) != m.heads:
                    raise ValueError(f"layer {i}: {len(m.decay)} decays for {m.heads} heads")
                if m.dim > 256:
                    raise ValueError(f"layer {i}: a matrix state has at most 256 key channels")
                if m.rot and m.rot.factor:
                    raise ValueError(f"layer {i}: retention turns by plain frequencies")
                self.state_piece[i] = at
                at += _round4(m.heads * m.dim * m.vdim)
            elif m.type == "attention":
                if m.heads % m.kv_heads:
                    raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
                if m.v_mix:
                    mixed = mixed or (m.kv_heads, m.vdim)
                    if mixed != (m.kv_heads, m.vdim):
                        raise ValueError(f"layer {i}: blended values must have the first blended layer's kv_heads and vdim")
                self.cache_plane[i] = len(self.cache_plane)
            else:
                raise ValueError(f"layer {i}: unknown mixer type {m.type!r}")
        self.state_floats = at

    # what the engine's cache pool and parameter builders ask of a model's shape
    def _attn(self):
        return [l.mixer for l in self.layers if l.mixer.type == "attention"]

    @property
    def num_hidden_layers(self) -> int:          # cache planes: one (keys, values) per attention mixer
        return max(1, len(self.cache_plane))

    @property
    def num_attention_heads(self) -> int:
        return max([m.heads for m in self._attn()] or [1])

    @property
    def num_key_value_heads(self) -> int:
        return max([m.kv_heads for m in self._attn()] or [1])

    @property
    def head_dim(self) -> int:
        return max([max(m.dim, m.vdim) for m in self._attn()] or [1])

    @classmethod
    def from_config(cls, cfg: dict) -> "NetelixShape":
        if cfg.get("architecture") != ARCHITECTURE:
            raise ValueError(f"not a {ARCHITECTURE} configuration: {cfg.get('architecture')!r}")
        layers = []
        for i, l in enumerate(cfg["layers"]):
            m, kind = l["mixer"], l["type"]
            heads, dim = int(m["heads"]), int(m["dim"])
            vdim = int(m.get("vdim") or dim)
            if kind in ("retention", "lightning"):
                mixer = MixerSpec(kind, heads, dim, vdim, decay=[float(d) for d in m["decay"]],
                                  rot=RotarySpec.from_config(m.get("rot")) if kind == "retention" else None)
            elif kind == "attention":
                mask = m.get("mask") or {}
                mixer = MixerSpec(kind, heads, dim, vdim, kv_heads=int(m.get("kv_heads") or heads), scale=float(m["scale"]),
                                  window=int(mask["size"]) if mask.get("size") else None, v_mix=bool(m.get("v_mix")),
                                  rot=RotarySpec.from_config(m.get("rot")))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            mlp = l.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layers.append(NetelixLayer(mixer, None if mlp is None else int(mlp["ff"])))
        return cls(vocab_size=int(cfg["vocab"]), hidden_size=int(cfg["width"]), layers=layers,
                   norm_eps=float((cfg.get("norm") or {}).get("eps", 1e-6)))

    def to_config(self) -> dict:
        out = []
        for l in self.layers:
            m = l.mixer
            mixer = {"dim": m.dim, "heads": m.heads, "vdim": m.vdim}
            if m.recurrent:
                mixer["decay"] = list(m.decay)
            else:
                mixer.update({"kv_heads": m.kv_heads, "scale": m.scale})
                if m.window:
                    mixer["mask"] = {"size": m.window}
                if m.v_mix:
                    mixer["v_mix"] = True
            if m.rot:
                mixer["rot"] = m.rot.to_config()
            out.append({"type": m.type, "mixer": mixer, "mlp": None if l.ff is None else {"kind": "dense", "ff": l.ff}})
        return {"architecture": ARCHITECTURE, "vocab": self.vocab_size, "width": self.hidden_size,
                "norm": {"eps": self.norm_eps}, "layers": out}


def tensor_shapes(shape: NetelixShape) -> Dict[str, tuple]:
    """Name -> shape of every tensor of a checkpoint of this shape (linear weights are [out, in])."""
    W = shape.hidden_size
    out = {"embed": (shape.vocab_size, W), "embed.norm": (W,), "final.norm": (W,), "head": (shape.vocab_size, W)}
    for i, l in enumerate(shape.layers):
        m, p = l.mixer, f"l{i}."
        x = p + "mix."
        kv = m.heads if m.recurrent else m.kv_heads
        out.update({p + "norm1": (W,), p + "ls1": (W,), x + "q": (m.heads * m.dim, W), x + "k": (kv * m.dim, W),
                    x + "v": (kv * m.vdim, W), x + "o": (W, m.heads * m.vdim)})
        if m.recurrent:
            out[x + "g"] = (m.heads * m.vdim, W)
            if m.type == "lightning":
                out[x + "norm"] = (m.heads * m.vdim,)
        else:
            out.update({x + "q.norm": (m.dim,), x + "k.norm": (m.dim,)})
            if m.v_mix:
                out[x + "vmix"] = ()
        if l.ff is not None:
            out.update({p + "norm2": (W,), p + "ls2": (W,), p + "mlp.gate": (l.ff, W), p + "mlp.up": (l.ff, W), p + "mlp.down": (W, l.ff)})
    return out


class _LayerWeights:
    pass


class NetelixForCausalLM:
    supports_graph_decode = False      # the engine's captured decode step is built around the Llama launch sequence

    def __init__(self, shape: NetelixShape, dtype: torch.dtype, device, state: Dict[str, Tensor]):
        if dtype not in (torch.float32, torch.bfloat16):
            raise ValueError("Netelix runs in bfloat16 or float32")
        self.shape, self.dtype, self.device = shape, dtype, torch.device(device)
        self.layer_trace: Optional[List[Tensor]] = None    # tests: when a list, the residual after every layer
        dev = self.device
        f32 = lambda t: t.to(device=dev, dtype=torch.float32).contiguous()
        act = lambda t: t.to(device=dev, dtype=dtype).contiguous()
        # a sublayer's norm weight and its channel scale are one vector (the product of two bfloat16 numbers is exact in float)
        scaled = lambda w, s: (f32(w) * f32(s)).contiguous()
        self.embed_table, self.head = act(state["embed"]), act(state["head"])
        self.embed_norm, self.final_norm = f32(state["embed.norm"]), f32(state["final.norm"])
        self.first_mixed: Optional[int] = next((i for i, l in enumerate(shape.layers) if l.mixer.v_mix), None)
        self.lw: List[_LayerWeights] = []
        for i, l in enumerate(shape.layers):
            m, p = l.mixer, f"l{i}."
            x = p + "mix."
            w = _LayerWeights()
            w.post1 = scaled(state[p + "norm1"], state[p + "ls1"])
            w.w_in = act(torch.cat([state[x + s] for s in ("qkvg" if m.recurrent else "qkv")], dim=0))
            w.o = act(state[x + "o"])
            w.freq, w.mag = None, 1.0
            if m.rot and m.rot.dims >= 2:
                freq, w.mag = m.rot.frequencies()
                w.freq = torch.tensor(freq, dtype=torch.float64, device=dev)
            if m.recurrent:
                w.powers = decay_powers(m.decay, dev)
                w.o_norm = f32(state[x + "norm"]) if m.type == "lightning" else None
            else:
                w.q_norm, w.k_norm = f32(state[x + "q.norm"]), f32(state[x + "k.norm"])
                w.v_mix = float(state[x + "vmix"]) if m.v_mix and i != self.first_mixed else None
            if l.ff is not None:
                w.post2 = scaled(state[p + "norm2"], state[p + "ls2"])
                w.gate_up = act(torch.cat([state[p + "mlp.gate"], state[p + "mlp.up"]], dim=0))
                w.down = act(state[p + "mlp.down"])
            self.lw.append(w)

    # ------------------------------------------------------------------ construction
    @classmethod
    def from_state_dict(cls, shape: NetelixShape, sd: Dict[str, Tensor], dtype, device) -> "NetelixForCausalLM":
        want = tensor_shapes(shape)
        # the first blended layer's number is not used: a checkpoint may leave it out
        first = next((f"l{i}.mix.vmix" for i, l in enumerate(shape.layers) if l.mixer.v_mix), None)
        missing = [k for k in want if k not in sd and k != first]
        if missing:
            raise RuntimeError(f"{len(missing)} tensors missing from the checkpoint, e.g. {missing[:3]}")
        for k, shp in want.items():
            if k in sd and tuple(sd[k].shape) != shp and not (shp == () and sd[k].numel() == 1):
                raise RuntimeError(f"tensor {k}: shape {tuple(sd[k].shape)} in the checkpoint, {shp} by config.json")
        return cls(shape, dtype, device, {k: sd[k] for k in want if k in sd})

    @staticmethod
    def random_state_dict(shape: NetelixShape, seed: int = 0) -> Dict[str, Tensor]:
        """Random bfloat16 weights of a size that keeps activations O(1): linears N(0, 1/fan_in), norm weights near one,
        channel scales around a half."""
        g = torch.Generator().manual_seed(seed)
        sd = {}
        for k, shp in tensor_shapes(shape).items():
            tail = k.rsplit(".", 1)[-1]
            if tail in ("norm", "norm1", "norm2"):
                t = 1.0 + 0.1 * torch.randn(shp, generator=g)
            elif tail in ("ls1", "ls2"):
                t = 0.5 + 0.1 * torch.randn(shp, generator=g)
            elif tail == "vmix":
                t = torch.rand(shp, generator=g)
            elif k == "embed":
                t = torch.randn(shp, generator=g)
            else:
                t = torch.randn(shp, generator=g) / math.sqrt(shp[-1])
            sd[k] = t.to(torch.bfloat16)      # checkpoints hold bfloat16
        return sd

    @classmethod
    def random_init(cls, shape: NetelixShape, dtype, device, seed: int = 0) -> "NetelixForCausalLM":
        return cls(shape, dtype, device, cls.random_state_dict(shape, seed))

    # ------------------------------------------------------------------ what the engine asks
    def cache_spec(self) -> dict:
        """Planes and row size of the paged cache: a key and a value plane per attention mixer."""
        sh = self.shape
        return {"n_layers": sh.num_hidden_layers, "n_tokens": 2, "n_heads": sh.num_key_value_heads, "head_size": sh.head_dim}

    def state_spec(self) -> Optional[dict]:
        """What a sequence carries from step to step beside the cache: one flat row, a piece of it for every recurrent
        mixer's matrix states."""
        return {"rows": 1, "width": self.shape.state_floats} if self.shape.state_floats else None

    def prepare_decode(self, max_rows: int = 64, keep_row_major: bool = True) -> None:
        """Nothing to prepare: decode steps run on the same weights as portions of prompts."""

    def weight_bytes(self, tokens: int = 1) -> int:
        e = torch.empty((), dtype=self.dtype).element_size()
        n = self.head.numel()
        for l, w in zip(self.shape.layers, self.lw):
            n += w.w_in.numel() + w.o.numel()
            if l.ff is not None:
                n += w.gate_up.numel() + w.down.numel()
        return n * e

    def embed(self, input_ids: Tensor) -> Tensor:
        return input_ids

    # ------------------------------------------------------------------ mixers
    def _recurrent(self, i: int, h: Tensor, pos: Tensor, params, seq: SequenceState) -> Tensor:
        m, w, sh = self.shape.layers[i].mixer, self.lw[i], self.shape
        H, D, V = m.heads, m.dim, m.vdim
        ap = params.attention_params[0]
        proj = torch.matmul(h, w.w_in.t())                                    # [T, q | k | v | gate]
        q, k, v, gate = proj.split([H * D, H * D, H * V, H * V], dim=1)
        where = (w.powers, seq, sh.state_piece[i], ap.q_cu_seq_lens, pos, H, D, V)
        if m.type == "retention":
            y = decay_attention_gated(q, k, v, gate, *where, eps=sh.norm_eps, gate_act="silu", k_scale=D ** -0.5,
                                      max_q_len=ap.q_max_seq_len, inv_freq=w.freq, layout="halves")
        else:
            o = decay_attention(q, k, v, *where, act="silu", max_q_len=ap.q_max_seq_len)
            y = gated_group_norm(o, self.dtype, group=H * V, eps=sh.norm_eps, w=w.o_norm, gate=gate, gate_act="sigmoid")
        return torch.matmul(y, w.o.t())

    def _attention(self, i: int, h: Tensor, pos: Tensor, params, seq: SequenceState, first_values: Dict[str, Tensor]) -> Tensor:
        m, w, sh = self.shape.layers[i].mixer, self.lw[i], self.shape
        T, H, G, D, V = h.shape[0], m.heads, m.kv_heads, m.dim, m.vdim
        ap = params.attention_params[sh.cache_plane[i]]
        kc, vc = ap.kv_cache.get_kv_cache()
        hs = kc.stride(2)                                                     # columns from one head of a cache row to the next
        proj = torch.matmul(h, w.w_in.t())                                    # [T, q | k | v]
        q, k, v = proj.split([H * D, G * D, G * V], dim=1)
        if m.v_mix:
            first_values.setdefault("v", v)
        blend = {} if w.v_mix is None else {"mix": first_values["v"], "mix_w": w.v_mix}
        turn = dict(inv_freq=w.freq, layout="interleaved", mag=w.mag, norm_eps=sh.norm_eps)
        q = rotary_parts([RotaryPart(q, H, D, norm_w=w.q_norm, **turn),
                          RotaryPart(k, G, D, norm_w=w.k_norm, cache=kc, cache_head_stride=hs, **turn),
                          RotaryPart(v, G, V, cache=vc, cache_head_stride=hs, **blend)], pos, ap.new_cache_slots)[0]
        o = biased_attention(q.view(T, H, D), kc, vc, V, seq.tok_seq, pos, ap.q_cu_seq_lens, ap.block_tables, ap.cu_blocks_lens,
                             m.scale, None, "window" if m.window else "causal", m.window or 0, max_q_len=ap.q_max_seq_len,
                             kv_heads=G, max_kv_len=ap.kv_max_seq_len)
        return torch.matmul(o.view(T, H * V), w.o.t())

    def _feed_forward(self, i: int, h: Tensor) -> Tensor:
        ff, w = self.shape.layers[i].ff, self.lw[i]
        gu = torch.matmul(h, w.gate_up.t())
        return torch.matmul(clamped_glu(gu[:, :ff], gu[:, ff:], 0.0, 1.0, 0.0), w.down.t())        # silu(gate) * up

    # ------------------------------------------------------------------ forward
    def forward_hidden(self, input_ids: Tensor, position_ids: Tensor, model_params) -> Tensor:
        """The normed output [n_selected, width] of model_params.selected_token_ids (all rows if None).  Every token's keys
        and values go to the cache and every sequence's state slot is brought up to date."""
        sh, dt = self.shape, self.dtype
        if input_ids.dtype not in (torch.int32, torch.int64):
            raise ValueError("Netelix takes token ids (its embedding is normed in float)")
        if position_ids.dtype != torch.int32:
            position_ids = position_ids.to(torch.int32)
        input_ids, pos = input_ids.contiguous(), position_ids.contiguous()
        seq = model_params.sequence_state
        if seq is None:
            if self.state_spec() is not None:
                raise ValueError("Netelix needs LanguageModelParameters.sequence_state (the batch's sequences and their state slots)")
            q_cu = model_params.attention_params[0].q_cu_seq_lens
            tok_seq = torch.repeat_interleave(torch.arange(q_cu.numel() - 1, device=q_cu.device), q_cu.diff().long(),
                                              output_size=input_ids.shape[0]).to(torch.int32)
            seq = SequenceState(None, None, tok_seq)
        T, W, L, eps = input_ids.shape[0], sh.hidden_size, len(sh.layers), sh.norm_eps
        x = torch.empty((T, W), dtype=torch.float32, device=self.device)      # the residual
        # the residual as the sublayers' operand: itself, or its copy in the activations' type
        h = x if dt == torch.float32 else torch.empty((T, W), dtype=dt, device=self.device)
        cast = None if dt == torch.float32 else h
        depth_norm(None, dt, eps, y=self.embed_table, y_ids=input_ids, post_w=self.embed_norm, post_norm="rms", x_out=x, cast_out=cast)
        sel = model_params.selected_token_ids
        rows = sel.to(torch.int32).contiguous() if sel is not None and self.layer_trace is None else None
        out, first_values = None, {}
        for i, (l, w) in enumerate(zip(sh.layers, self.lw)):
            y = self._recurrent(i, h, pos, model_params, seq) if l.mixer.recurrent else \
                self._attention(i, h, pos, model_params, seq, first_values)
            post = w.post1
            if l.ff is not None:
                depth_norm(x, dt, eps, y=y, post_w=post, post_norm="rms", x_out=x, cast_out=cast)
                y, post = self._feed_forward(i, h), w.post2
            if i < L - 1:
                depth_norm(x, dt, eps, y=y, post_w=post, post_norm="rms", x_out=x, cast_out=cast)
            else:      # the last result joins the residual of the selected rows, which is normed for the head
                out = depth_norm(x, dt, eps, y=y, post_w=post, post_norm="rms", x_out=None if rows is not None else x,
                                 next_w=self.final_norm, rows=rows, rms=True)
            if self.layer_trace is not None:
                self.layer_trace.append(x.clone())
        if out is None:
            out = depth_norm(x, dt, eps, next_w=self.final_norm, rows=rows, rms=True)
        if rows is None and sel is not None:
            out = out.index_select(0, sel.to(torch.int64))
        return out

    def forward_logits(self, input_ids: Tensor, position_ids: Tensor, model_params) -> Tensor:
        """float32 logits [n_selected, vocab]."""
        x = self.forward_hidden(input_ids, position_ids, model_params)
        return torch.matmul(x, self.head.t()).float()

    def forward(self, input_ids: Tensor, position_ids: Tensor, model_params) -> Tensor:
        """Greedy token ids of the selected rows, like the framework's other models."""
        return torch.argmax(self.forward_logits(input_ids, position_ids, model_params), dim=-1)

    __call__ = forward


def read_shape(model_path: str) -> NetelixShape:
    with open(os.path.join(model_path, "config.json")) as f:
        return NetelixShape.from_config(json.load(f))
