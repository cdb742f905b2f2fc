"""Ragged decoder for designs whose ``config.json`` lists every layer (own mixer and feed-forward sizes
per layer), served from the paged cache like the other families.

Where ``hf_decoder.py`` describes a whole model with one set of sizes, here a ``LayeredSpec`` holds one
``LayerSpec`` per layer: head counts, key and value sizes, window and feed-forward width may differ
from layer to layer, and the KV cache takes its geometry per layer from ``kv_shapes``. The residual
stream is 32-bit. Mechanisms are ops with parameters (ops/mix_attention.py, ops/residual_norm.py), and
an architecture is one entry of ``ARCHITECTURES``: a function from its config to the spec plus a function
from its checkpoint tensors to the packed layout:
  * q | k | v | output gate -> ONE projection weight [nq dk + nkv (dk + dv) + nq dv, width];
  * gate | up -> one [2 ff, width] weight, ff zero-padded to a multiple of 16 (exact: the padding
    contributes silu(0) * 0);
  * per-head attention numbers as fp32 (ops/mix_attention.MixParams).

Tobinex: x = embed * scale; per layer x <- norm1(alpha x + attention(x)), x <- norm2(alpha x + ff(x)), RMS
norms with weights stored around zero, q / k norms over the whole projection, no rotation, distance
bias, window with kept first tokens, softmax sink, talking heads, output gate, SwiGLU, tied LM head.
"""
import json
import os
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from ....ops.activation import gated_act
from ....ops.linear import fused_addnorm_linear, fused_gatesum_linear, fused_swiglu_linear, linear
from ....ops.mix_attention import MixParams, cache_row, mix_attention, mix_attention_parts
from ....ops.residual_norm import embed_scale, qkv_norm_append, residual_rms_norm

FF_MULTIPLE = 16


@dataclass
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None   # None: every key up to the query
    keep_first: int = 0            # keys always visible in front of the window


@dataclass
class LayerSpec:
    mixer: AttentionSpec
    ff: int = 0                    # 0: no feed-forward
    act: str = "silu"


@dataclass
class LayeredSpec:
    architecture: str
    vocab_size: int
    width: int
    eps: float
    alpha: float                   # residual factor of the norm-after-sum layers
    embed_scale: float = 1.0
    norm_offset: float = 1.0       # 1: norm weights stored around zero; 0: plain
    layers: List[LayerSpec] = field(default_factory=list)

    @classmethod
    def from_dict(cls, d):
        layers = [LayerSpec(**{**x, "mixer": AttentionSpec(**x["mixer"])}) for x in d["layers"]]
        return cls(**{**d, "layers": layers})


# ------------------------------------------------------------------------------------- Tobinex
def _tobinex_spec(c):
    layers = []
    for i, L in enumerate(c["layers"]):
        if L["type"] != "attention":
            raise NotImplementedError(f"layer {i}: mixer type {L['type']!r}")
        m, f = L["mixer"], L.get("mlp")
        if m["heads"] % m["kv_heads"]:
            raise ValueError(f"layer {i}: {m['heads']} heads do not divide by {m['kv_heads']} kv heads")
        if f is not None and f["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward kind {f['kind']!r}")
        mask = m.get("mask") or {}
        layers.append(LayerSpec(AttentionSpec(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]),
                                              float(m["scale"]), mask.get("size"), int(mask.get("keep_first") or 0)),
                                ff=int(f["ff"]) if f is not None else 0))
    return LayeredSpec(c["architecture"], int(c["vocab"]), int(c["width"]), float(c["norm"]["eps"]),
                       float(c["postln_alpha"]), float(c["embedding"]["scale"]), 1.0, layers)


def _tobinex_weights(spec, sd):
    def get(name, *shape):
        if name not in sd:
            raise KeyError(f"missing checkpoint tensor {name}")
        if tuple(sd[name].shape) != shape:
            raise ValueError(f"{name}: shape {tuple(sd[name].shape)}, the configuration says {shape}")
        return sd[name]
    H = spec.width
    W = {"embed": get("embed", spec.vocab_size, H), "final": get("final.norm", H), "layers": []}
    for i, L in enumerate(spec.layers):
        a, p = L.mixer, f"l{i}.mix."
        nq, nkv, dk, dv = a.heads, a.kv_heads, a.dim, a.vdim
        d = {"norm1": get(f"l{i}.norm1", H),
             "qkvg": torch.cat([get(p + "q", nq * dk, H), get(p + "k", nkv * dk, H), get(p + "v", nkv * dv, H),
                                get(p + "g", nq * dv, H)]),
             "q_norm": get(p + "q.norm", nq * dk), "k_norm": get(p + "k.norm", nkv * dk), "o": get(p + "o", H, nq * dv),
             "r1": get(p + "r1", nq).float(), "r2": get(p + "r2", nq).float(), "sink": get(p + "sink", nq).float(),
             "talk": get(p + "talk", nq, nq).float()}
        if L.ff:
            p, pad = f"l{i}.mlp.", -L.ff % FF_MULTIPLE
            rows = (lambda w: torch.nn.functional.pad(w, (0, 0, 0, pad)))
            d["norm2"] = get(f"l{i}.norm2", H)
            d["gu"] = torch.cat([rows(get(p + "gate", L.ff, H)), rows(get(p + "up", L.ff, H))])
            d["down"] = torch.nn.functional.pad(get(p + "down", H, L.ff), (0, pad))
        W["layers"].append(d)
    return W


# architecture name in config.json -> (config dict -> LayeredSpec, (spec, state dict) -> packed weights)
ARCHITECTURES = {"Tobinex": (_tobinex_spec, _tobinex_weights)}


def is_layered_config(cfg):
    return cfg.get("architecture") in ARCHITECTURES


# ------------------------------------------------------------------------------------- decoder
class RaggedLayeredDecoder:
    """Engine-facing model (InferenceEngineV2 protocol: num_layers / kv_shapes / dtype / device /
    vocab_size / forward(batch, kv_cache) -> fp32 logits of ``batch.last_idx``)."""

    FP32_KEYS = ("r1", "r2", "sink", "talk")   # never rounded to the compute dtype
    QUANT_KEYS = ("qkvg", "o", "gu", "down")

    def __init__(self, spec: LayeredSpec, weights, dtype=torch.bfloat16, device=None, weight_quant=None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"{spec.architecture}: dtype {dtype} (bfloat16 or float32)")
        self.spec = spec
        self._dtype, self._device = dtype, torch.device(device) if device is not None else torch.device("cpu")

        def mv(k, t):
            return t.to(device=self._device, dtype=torch.float32 if k in self.FP32_KEYS else dtype).contiguous()
        self.w = {k: mv(k, v) for k, v in weights.items() if k != "layers"}
        self.w["layers"] = [{k: mv(k, v) for k, v in L.items()} for L in weights["layers"]]
        self.weight_quant = weight_quant
        if weight_quant:
            from ....ops.fp_quantizer import quantized_weight
            for L in self.w["layers"]:
                for k in self.QUANT_KEYS:
                    if k in L:
                        L[k] = quantized_weight(L[k], weight_quant)
        self._finish()

    def _finish(self):
        s = self.spec
        self.tp, self.tp_rank = 1, 0
        self.num_layers, self.vocab_size = len(s.layers), s.vocab_size
        self.kv_shapes = []
        for L in s.layers:  # one row length for k and v of a layer: the matrix-core kernels take one
            a = L.mixer
            dk, dv = cache_row(a.dim, self._dtype), cache_row(a.vdim, self._dtype)
            if dk != a.dim or dv != a.vdim or self._dtype == torch.bfloat16:
                dk = dv = max(dk, dv)
            self.kv_shapes.append((a.kv_heads, dk, dv))
        self._mix = [MixParams(L["r1"], L["r2"], L["sink"], L["talk"]) for L in self.w["layers"]]
        self.model = self

    @classmethod
    def restore(cls, spec, w, dtype, device, weight_quant=None):
        """From weights already in their served form (serialization.py)."""
        m = cls.__new__(cls)
        m.spec, m.w, m._dtype, m._device, m.weight_quant = spec, w, dtype, device, weight_quant
        m._finish()
        return m

    @property
    def device(self):
        return self._device

    @property
    def dtype(self):
        return self._dtype

    def state_dict(self):
        sd = {k: v for k, v in self.w.items() if torch.is_tensor(v)}
        for i, L in enumerate(self.w["layers"]):
            sd.update({f"layers.{i}.{k}": v for k, v in L.items() if torch.is_tensor(v)})
        return sd

    # decode (<= 2 tokens): the norm after the residual sum runs as the prologue of the next projection, the
    # gated sum of the attention's KV splits as the output projection's, SwiGLU as the down projection's
    FUSE_MAX_T = 2  # at 4 rows every workgroup rebuilding them costs more than the launches saved

    def _fusable(self, T):
        return (T <= self.FUSE_MAX_T and self._device.type == "cuda" and self._dtype == torch.bfloat16
                and os.environ.get("SXE_DECODE_FUSE", "1") == "1")

    def _attn(self, proj, L, li, batch, kv_cache):
        """``proj`` [T, q | k | v | gate] -> the mixer's output [T, width]."""
        a = self.spec.layers[li].mixer
        nq, nkv, dk, dv = a.heads, a.kv_heads, a.dim, a.vdim
        kc, vc = kv_cache.layer_kv(li)
        q = qkv_norm_append(proj, L["q_norm"], L["k_norm"], kc, vc, batch.slots, nq, nkv, dk, dv, self.spec.eps)
        gate = proj[:, nq * dk + nkv * (dk + dv):]
        args = (q, kc, vc, batch, dk, dv, a.scale, self._mix[li], a.window, a.keep_first, gate)
        parts = mix_attention_parts(*args) if self._fusable(proj.shape[0]) else None
        if parts is None:
            return linear(mix_attention(*args), L["o"])
        o, part = parts
        y = fused_gatesum_linear(part, gate, L["o"]) if part is not None else None
        if y is not None:
            return y
        if part is not None:
            o = (part.sum(0) * torch.sigmoid(gate.float())).to(proj.dtype)
        return linear(o, L["o"])

    def _norm_linear(self, pending, x, xb, weight):
        """The projection of the layer input: ``linear(xb, weight)`` when no norm is pending, else the
        pending ``(y, norm weight)`` -- x <- norm(alpha x + y) -- and the projection, in one launch where the
        fused kernel covers it. Returns (projection, x, xb); x may come back as the fused kernel's state."""
        if pending is None:
            return linear(xb, weight), x, xb
        s = self.spec
        if self._fusable(pending[0].shape[0]):
            r = fused_addnorm_linear(pending[0], x, pending[1], s.alpha, s.eps, s.norm_offset, weight)
            if r is not None:
                return r[0], r[1], None
        x, xb = residual_rms_norm(self._stream(x), pending[0], pending[1], s.alpha, s.eps, s.norm_offset)
        return linear(xb, weight), x, xb

    def _stream(self, x):
        """The fp32 residual stream itself (a fused state holds the sum in front of its norm)."""
        if isinstance(x, tuple):
            return residual_rms_norm(x[0], None, x[2], 1.0, self.spec.eps, self.spec.norm_offset)[0]
        return x

    @torch.no_grad()
    def forward(self, batch, kv_cache):
        s, W = self.spec, self.w
        x, xb = embed_scale(W["embed"], batch.input_ids, s.embed_scale)
        pending = None  # the last sublayer's (output, norm weight), not yet added to x
        for li, L in enumerate(W["layers"]):
            proj, x, xb = self._norm_linear(pending, x, xb, L["qkvg"])
            pending = (self._attn(proj, L, li, batch, kv_cache), L["norm1"])
            if "gu" in L:
                gu, x, xb = self._norm_linear(pending, x, xb, L["gu"])
                y = fused_swiglu_linear(gu, L["down"]) if self._fusable(gu.shape[0]) and s.layers[li].act == "silu" else None
                if y is None:
                    y = linear(gated_act(gu, s.layers[li].act), L["down"])
                pending = (y, L["norm2"])
        if pending is not None:
            x, _ = residual_rms_norm(self._stream(x), pending[0], pending[1], s.alpha, s.eps, s.norm_offset)
        _, h = residual_rms_norm(x, None, W["final"], 1.0, s.eps, s.norm_offset, index=batch.last_idx, need_x=False)
        return linear(h, W["embed"]).float()


def load_layered_decoder(path, dtype=torch.bfloat16, device=None, weight_quant=None, tp_size=1):
    """A checkpoint directory (config.json + *.safetensors) -> RaggedLayeredDecoder."""
    from .hf_decoder import _load_state_dict
    if tp_size > 1:
        raise NotImplementedError("layered decoders run on one GPU: talking heads couple all heads of a token, "
                                  "so heads cannot be split over tensor-parallel ranks")
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    make_spec, make_weights = ARCHITECTURES[cfg["architecture"]]
    spec = make_spec(cfg)
    return RaggedLayeredDecoder(spec, make_weights(spec, _load_state_dict(path)), dtype=dtype, device=device,
                                weight_quant=weight_quant)

