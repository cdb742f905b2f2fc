"""Ragged decoder for designs whose ``config.json`` lists every layer (own mixer and feed-forward sizes
per layer), served from the paged cache like the other families.

Where ``hf_decoder.py`` describes a whole model with one set of sizes, here a ``LayeredSpec`` holds one
``LayerSpec`` per layer: mixer kind, head counts, key and value sizes, window and feed-forward may differ
from layer to layer, and the cache takes its geometry per layer from ``kv_shapes`` (paged rows) and
``state_shapes`` (recurrent state of a sequence). The residual stream is 32-bit. Mechanisms are ops with
parameters (ops/mix_attention.py, ops/latent_attention.py, ops/linear_attention.py, ops/moe.py,
ops/residual_norm.py), and an architecture is one entry of ``ARCHITECTURES``: a function from its config to
the spec plus a function from its checkpoint tensors to the packed layout:
  * projections of one input -> ONE weight (q | k | v | output gate; query latent | latent | key part);
  * gate | up -> one [2 ff, width] weight, ff zero-padded to a multiple of 16 (exact: the padding
    contributes silu(0) * 0); experts stacked [E, ff, width] / [E, width, ff];
  * per-head attention numbers as fp32.

Two residual forms (``LayeredSpec.residual``):
  * "after": x <- norm(alpha x + sublayer(x));
  * "sandwich": x <- x + norm_b(sublayer(norm_a(x))).
``loop`` runs a range of layers several times with the same weights; every pass is a layer run of its own
with its own cache or state, so ``num_layers`` counts runs.

Tobinex: x = embed * scale; "after" with RMS norms stored around zero; q / k norms over the whole
projection, no rotation, distance bias, window with kept first tokens, softmax sink, talking heads, output
gate, SwiGLU, tied LM head.
Bipotar: normed embedding; "sandwich" with plain RMS norms; linear attention with a decayed state or windowed
latent attention; SwiGLU or routed experts with squared relu; a loop that adds the embedding output ahead of
every pass but the first; separate scaled LM head.
"""
import json
import os
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from ....ops.activation import gated_act
from ....ops.latent_attention import latent_append, latent_attention, latent_row, rotation_table
from ....ops.linear import (fused_addnorm_linear, fused_gatenorm_linear, fused_gatesum_linear, fused_sandwich_linear,
                            fused_swiglu_linear, linear)
from ....ops.linear_attention import decay_attention, decay_table
from ....ops.mix_attention import MixParams, cache_row, mix_attention, mix_attention_parts
from ....ops.moe import expert_mlp, fused_sandwich_route, route_topk
from ....ops.residual_norm import (embed_norm, embed_scale, gated_rms_norm, qkv_norm_append, residual_rms_norm,
                                   sandwich_norm)

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
class LatentSpec:
    """Keys and values from a cached latent (ops/latent_attention.py)."""
    heads: int
    dim: int                       # unrotated query / key size of a head
    rot_dim: int                   # rotated query size of a head; one rotated key part for all heads
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    window: Optional[int] = None


@dataclass
class LinearSpec:
    """Linear attention with a decayed state (ops/linear_attention.py)."""
    heads: int
    dim: int
    vdim: int
    decay: List[float] = field(default_factory=list)


MIXERS = {c.__name__: c for c in (AttentionSpec, LatentSpec, LinearSpec)}


@dataclass
class MoESpec:
    experts: int
    top: int
    ff: int
    act: str = "relu2"


@dataclass
class LayerSpec:
    mixer: object                  # one of MIXERS
    ff: int = 0                    # 0: no dense feed-forward
    act: str = "silu"
    moe: Optional[MoESpec] = None


@dataclass
class LoopSpec:
    start: int
    stop: int
    times: int


@dataclass
class LayeredSpec:
    architecture: str
    vocab_size: int
    width: int
    eps: float
    alpha: float = 1.0             # residual factor of the norm-after-sum layers
    embed_scale: float = 1.0
    norm_offset: float = 1.0       # 1: norm weights stored around zero; 0: plain
    layers: List[LayerSpec] = field(default_factory=list)
    residual: str = "after"        # "after" | "sandwich"
    loop: Optional[LoopSpec] = None
    logit_scale: float = 1.0

    def runs(self):
        """[(layer index, whether the embedding output is added to x ahead of it)] in the order they run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, False) for i in range(n)]
        a, b = self.loop.start, self.loop.stop
        out = [(i, False) for i in range(a)]
        for t in range(self.loop.times):
            out += [(i, t > 0 and i == a) for i in range(a, b)]
        return out + [(i, False) for i in range(b, n)]

    def to_dict(self):
        from dataclasses import asdict
        d = asdict(self)
        for x, L in zip(d["layers"], self.layers):
            x["mixer_kind"] = type(L.mixer).__name__
        return d

    @classmethod
    def from_dict(cls, d):
        layers = []
        for x in d["layers"]:
            x = dict(x)
            kind, moe = MIXERS[x.pop("mixer_kind", "AttentionSpec")], x.get("moe")
            layers.append(LayerSpec(**{**x, "mixer": kind(**x["mixer"]), "moe": MoESpec(**moe) if moe else None}))
        return cls(**{**d, "layers": layers, "loop": LoopSpec(**d["loop"]) if d.get("loop") else None})


def checkpoint_tensor(sd, name, *shape):
    if name not in sd:
        raise KeyError(f"missing checkpoint tensor {name}")
    if tuple(sd[name].shape) != shape:
        raise ValueError(f"{name}: shape {tuple(sd[name].shape)}, the configuration says {shape}")
    return sd[name]


def pack_dense_ff(get, p, ff, width):
    """SwiGLU weights: gate | up in one, ff zero-padded."""
    pad = -ff % FF_MULTIPLE
    rows = (lambda w: torch.nn.functional.pad(w, (0, 0, 0, pad)))
    return {"gu": torch.cat([rows(get(p + "gate", ff, width)), rows(get(p + "up", ff, width))]),
            "down": torch.nn.functional.pad(get(p + "down", width, ff), (0, pad))}


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
        return checkpoint_tensor(sd, name, *shape)
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
            d["norm2"] = get(f"l{i}.norm2", H)
            d.update(pack_dense_ff(get, f"l{i}.mlp.", L.ff, H))
        W["layers"].append(d)
    return W


# ------------------------------------------------------------------------------------- Bipotar
def _bipotar_mixer(i, kind, m):
    if kind == "lightning":
        decay = m["decay"] if isinstance(m["decay"], list) else [m["decay"]] * m["heads"]
        if len(decay) != m["heads"]:
            raise ValueError(f"layer {i}: {len(decay)} decays for {m['heads']} heads")
        return LinearSpec(int(m["heads"]), int(m["dim"]), int(m["vdim"]), [float(d) for d in decay])
    if kind == "latent_attention":
        if m["rot"]["dims"] != m["rot_dim"] or m["rot_dim"] % 2:
            raise ValueError(f"layer {i}: rotation over {m['rot']['dims']} of {m['rot_dim']} rotated dimensions")
        size = (m.get("mask") or {}).get("size")
        return LatentSpec(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["q_rank"]),
                          int(m["kv_rank"]), float(m["scale"]), float(m["rot"]["base"]), None if size is None else int(size))
    raise NotImplementedError(f"layer {i}: mixer type {kind!r}")


def _bipotar_spec(c):
    layers = []
    for i, L in enumerate(c["layers"]):
        f = L.get("mlp") or {"kind": "dense", "ff": 0}
        layer = LayerSpec(_bipotar_mixer(i, L["type"], L["mixer"]))
        if f["kind"] == "dense":
            layer.ff = int(f["ff"])
        elif f["kind"] == "moe":
            layer.moe = MoESpec(int(f["router"]["experts"]), int(f["router"]["top"]), int(f["expert"]["ff"]))
            if not 0 < layer.moe.top <= layer.moe.experts:
                raise ValueError(f"layer {i}: {layer.moe.top} of {layer.moe.experts} experts")
        else:
            raise NotImplementedError(f"layer {i}: feed-forward kind {f['kind']!r}")
        layers.append(layer)
    loop = c.get("loop")
    if loop is not None:
        loop = LoopSpec(int(loop["start"]), int(loop["stop"]), int(loop["times"]))
        if not 0 <= loop.start <= loop.stop <= len(layers):
            raise ValueError(f"loop over layers {loop.start} .. {loop.stop - 1} of {len(layers)}")
    return LayeredSpec(c["architecture"], int(c["vocab"]), int(c["width"]), float(c["norm"]["eps"]), norm_offset=0.0,
                       layers=layers, residual="sandwich", loop=loop, logit_scale=float(c.get("logit_scale", 1.0)))


def _bipotar_weights(spec, sd):
    def get(name, *shape):
        return checkpoint_tensor(sd, name, *shape)
    D, V = spec.width, spec.vocab_size
    W = {"embed": get("embed", V, D), "embed_norm": get("embed.norm", D), "final": get("final.norm", D),
         "head": get("head", V, D), "layers": []}
    for i, L in enumerate(spec.layers):
        a, p = L.mixer, f"l{i}.mix."
        d = {"norm1": get(f"l{i}.norm1", D), "norm1b": get(f"l{i}.norm1b", D)}
        if isinstance(a, LinearSpec):
            kd, vd = a.heads * a.dim, a.heads * a.vdim
            d["qkvg"] = torch.cat([get(p + "q", kd, D), get(p + "k", kd, D), get(p + "v", vd, D), get(p + "g", vd, D)])
            d["o_norm"], d["o"], d["decay"] = get(p + "norm", vd), get(p + "o", D, vd), decay_table(a.decay)
        else:
            H, R = a.heads, a.kv_rank
            uk, uv = get(p + "uk", H * a.dim, R), get(p + "uv", H * a.vdim, R)
            d["dqkv"] = torch.cat([get(p + "dq", a.q_rank, D), get(p + "dkv", R + a.rot_dim, D)])
            d["q_norm"], d["kv_norm"] = get(p + "dq.norm", a.q_rank), get(p + "dkv.norm", R)
            d["uq"], d["o"] = get(p + "uq", H * (a.dim + a.rot_dim), a.q_rank), get(p + "o", D, H * a.vdim)
            d["uk"], d["uv"] = uk.view(H, a.dim, R).transpose(1, 2), uv.view(H, a.vdim, R)
            d["ukv"] = torch.cat([uk, uv])
        if L.ff or L.moe:
            p = f"l{i}.mlp."
            d["norm2"], d["norm2b"] = get(f"l{i}.norm2", D), get(f"l{i}.norm2b", D)
            if L.ff:
                d.update(pack_dense_ff(get, p, L.ff, D))
            else:
                E, F = L.moe.experts, L.moe.ff
                d["router"] = get(p + "router", E, D)
                d["e_up"] = torch.stack([get(f"{p}e{e}.up", F, D) for e in range(E)])
                d["e_down"] = torch.stack([get(f"{p}e{e}.down", D, F) for e in range(E)])
        W["layers"].append(d)
    return W


# architecture name in config.json -> (config dict -> LayeredSpec, (spec, state dict) -> packed weights)
ARCHITECTURES = {"Tobinex": (_tobinex_spec, _tobinex_weights), "Bipotar": (_bipotar_spec, _bipotar_weights)}


# csrc/kernels sources a checkout with nothing built compiles to serve an architecture
SERVING_UNITS = {"Tobinex": ("act", "mix_attn", "residual_norm", "skinny_gemm"),
                 "Bipotar": ("act", "experts", "grouped_gemm", "latent_attn", "linear_attn", "residual_norm", "skinny_gemm")}


def ensure_library(path):
    """The HIP library that serving the checkpoint in ``path`` needs, compiled if nothing is built."""
    from ....ops import native
    with open(os.path.join(path, "config.json")) as f:
        arch = json.load(f).get("architecture")
    if arch in SERVING_UNITS:
        native.ensure_serving_library(arch.lower(), SERVING_UNITS[arch])
    else:
        native.ensure_serving_library()


def is_layered_config(cfg):
    return cfg.get("architecture") in ARCHITECTURES


# ------------------------------------------------------------------------------------- decoder
class RaggedLayeredDecoder:
    """Engine-facing model (InferenceEngineV2 protocol: num_layers / kv_shapes / dtype / device /
    vocab_size / forward(batch, kv_cache) -> fp32 logits of ``batch.last_idx``)."""

    FP32_KEYS = ("r1", "r2", "sink", "talk", "decay")   # never rounded to the compute dtype
    QUANT_KEYS = ("qkvg", "dqkv", "uq", "o", "gu", "down")
    device_routing = True   # expert counts never go through the host: decode steps can be captured

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
        self.runs = s.runs()
        self.num_layers, self.vocab_size = len(self.runs), s.vocab_size
        self.kv_shapes = [self._kv_shape(s.layers[i].mixer) for i, _ in self.runs]
        self.state_shapes = [self._state_shape(s.layers[i].mixer) for i, _ in self.runs]
        self._mix = [MixParams(L["r1"], L["r2"], L["sink"], L["talk"]) if "r1" in L else None for L in self.w["layers"]]
        self.model = self

    def _kv_shape(self, a):
        """(kv heads, k row, v row) of a layer's paged cache."""
        if isinstance(a, LinearSpec):
            return (0, 0, 0)
        if isinstance(a, LatentSpec):
            return (1, sum(latent_row(a.kv_rank, a.rot_dim, self._dtype)), 0)
        # one row length for k and v of a layer: the matrix-core kernels take one
        dk, dv = cache_row(a.dim, self._dtype), cache_row(a.vdim, self._dtype)
        if dk != a.dim or dv != a.vdim or self._dtype == torch.bfloat16:
            dk = dv = max(dk, dv)
        return (a.kv_heads, dk, dv)

    @staticmethod
    def _state_shape(a):
        return (a.heads, a.dim, a.vdim) if isinstance(a, LinearSpec) else None

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
        if self.spec.residual == "sandwich":
            return self._forward_sandwich(batch, kv_cache)
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

    # ------------------------------------------------------------------------- norm on both sides
    # The sum and the norms between two sublayers stay pending until the next sublayer's first product asks for
    # its input: at decode that product builds it in its own launch.
    def _normed(self, st, pre, index=None, last=False):
        """The next sublayer's input rms(x) * pre, the pending sum taken into x first."""
        if st.pending is not None:
            y, post, slots, add = st.pending
            st.x, st.h = sandwich_norm(st.x, y, post, pre, self.spec.eps, slots, add, index, need_x=not last)
            st.pending = None
        return st.h

    def _project(self, st, pre, weight):
        if st.pending is not None and self._fusable(st.x.shape[0]):
            y, post, slots, add = st.pending
            r = fused_sandwich_linear(st.x, y, post, pre, self.spec.eps, slots, add, weight)
            if r is not None:
                st.x, st.pending = r[1], None
                return r[0]
        return linear(self._normed(st, pre), weight)

    def _linear_mixer(self, st, L, a, run, batch, kv_cache):
        """Decayed linear attention."""
        proj = self._project(st, L["norm1"], L["qkvg"])
        o = decay_attention(proj, kv_cache.layer_state(run), L["decay"], batch, a.heads, a.dim, a.vdim)
        gate = proj[:, a.heads * (2 * a.dim + a.vdim):]
        y = fused_gatenorm_linear(o, L["o_norm"], gate, self.spec.eps, L["o"]) if self._fusable(o.shape[0]) else None
        return linear(gated_rms_norm(o, L["o_norm"], gate, self.spec.eps), L["o"]) if y is None else y

    def _latent_mixer(self, st, L, a, run, batch, kv_cache):
        proj = self._project(st, L["norm1"], L["dqkv"])
        cache = kv_cache.layer_kv(run)[0]
        rot = self._rotation(batch, a)
        cq = latent_append(proj, L["q_norm"], L["kv_norm"], cache, batch.slots, rot, a.q_rank, a.kv_rank, a.rot_dim, self.spec.eps)
        o = latent_attention(linear(cq, L["uq"]), L["uk"], L["uv"], L["ukv"], cache, batch, rot, a.heads, a.dim, a.rot_dim,
                             a.vdim, a.kv_rank, a.scale, a.window)
        return linear(o, L["o"])

    def _rotation(self, batch, a):
        """The step's rotation table, shared by the layers with the same rotation."""
        key = (a.rot_dim, a.rot_base)
        if key not in self._rot:
            self._rot[key] = rotation_table(batch.positions, *key)
        return self._rot[key]

    def _feed_forward(self, st, L, spec):
        """-> (output rows, slots): slots None for one row a token (ops/residual_norm.sandwich_norm)."""
        if spec.moe is None:
            gu = self._project(st, L["norm2"], L["gu"])
            y = fused_swiglu_linear(gu, L["down"]) if self._fusable(gu.shape[0]) and spec.act == "silu" else None
            return (linear(gated_act(gu, spec.act), L["down"]) if y is None else y), None
        r = None
        if st.pending is not None and self._fusable(st.x.shape[0]):
            y, post, slots, add = st.pending
            r = fused_sandwich_route(st.x, y, post, L["norm2"], self.spec.eps, slots, add, L["router"], spec.moe.top)
        if r is not None:
            (st.x, h, routing), st.pending = r, None
        else:
            h = self._normed(st, L["norm2"])
            routing = route_topk(h, L["router"], spec.moe.top)
        return expert_mlp(h, routing, L["e_up"], L["e_down"], spec.moe.act)

    def _forward_sandwich(self, batch, kv_cache):
        s, W = self.spec, self.w
        self._rot = {}
        x0, h = embed_norm(W["embed"], batch.input_ids, W["embed_norm"], s.eps, W["layers"][self.runs[0][0]]["norm1"])
        st = _Stream(x0, h)
        for r, (i, again) in enumerate(self.runs):
            L, spec = W["layers"][i], s.layers[i]
            if again:
                st.pending = st.pending[:3] + (x0,)
            mixer = self._linear_mixer if isinstance(spec.mixer, LinearSpec) else self._latent_mixer
            st.pending = (mixer(st, L, spec.mixer, r, batch, kv_cache), L["norm1b"], None, None)
            if "norm2" in L:
                y, slots = self._feed_forward(st, L, spec)
                st.pending = (y, L["norm2b"], slots, None)
        h = self._normed(st, W["final"], batch.last_idx, last=True)
        return linear(h, W["head"]).float() * s.logit_scale


@dataclass
class _Stream:
    """The 32-bit residual stream between sublayers: x, and either the normed input ``h`` of the next sublayer or
    the last one's ``pending`` (output, its norm weight, slots, rows to add) that x does not hold yet."""
    x: torch.Tensor
    h: Optional[torch.Tensor] = None
    pending: Optional[tuple] = None


def load_layered_decoder(path, dtype=torch.bfloat16, device=None, weight_quant=None, tp_size=1):
    """A checkpoint directory (config.json + *.safetensors) -> RaggedLayeredDecoder."""
    from .hf_decoder import _load_state_dict
    if tp_size > 1:
        raise NotImplementedError("layered decoders run on one GPU: talking heads and norms over all heads couple the heads "
                                  "of a token, so heads cannot be split over tensor-parallel ranks")
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    make_spec, make_weights = ARCHITECTURES[cfg["architecture"]]
    spec = make_spec(cfg)
    return RaggedLayeredDecoder(spec, make_weights(spec, _load_state_dict(path)), dtype=dtype, device=device,
                                weight_quant=weight_quant)

