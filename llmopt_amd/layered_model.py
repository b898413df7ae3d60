"""Layered decoders over bfloat16 weights: an ordered list of layers, each a mixer (attention over chunks
with a softmax sink, Mamba-2, or window attention and the gated delta rule side by side) and an optional
feed-forward (dense or routed experts), on a float32 residual stream.  The Barovik and Koketar designs are
such decoders.

What a design fixes beyond its layers is a `Design`: norms in front of the sublayers or on their outputs, how
their weights are stored, the feed-forward's activation, a head of its own or the embedding's.

`LayeredConfig` is the parsed config.json, `LayeredModel` holds the device weights and the state pool and
runs steps.  A step is a dispatch list over the entry points of csrc/ops_dense.cpp, the same list for one
token and for many: the entries choose matrix-vector or matrix-core kernels by the token count.  The
one-token list, with the logits and their argmax behind it, is frozen into a retained plan (one HIP graph)
whose step words carry position and slot, so that it serves every sequence.
"""
from __future__ import annotations

import os
import struct
from dataclasses import dataclass
from typing import Optional, Sequence as Tokens

import numpy as np

from .decode_step import u32s
from .native import Buffer, DispatchList, Prebaked, Runtime
from .safetensors_file import SafetensorsFile, from_bfloat16, to_bfloat16
from .sequence_state import RecurrentShape, RingShape, Sequence, StatePool

SILU, GELU_TANH, CLAMPED = 0, 1, 2  # gate activations of the feed-forward entries
_ALIGNED = 8  # parts of a joint projection start at multiples of this


@dataclass(frozen=True)
class Design:
    name: str
    norm_after: bool = False      # norms on the sublayers' outputs, else on their inputs
    norm_offset: float = 0.0      # added to every stored weight of the stream's norms
    dense_activation: int = GELU_TANH
    tied_head: bool = False       # logits through the embedding table


DESIGNS = {design.name: design for design in (
    Design("Barovik"),
    Design("Koketar", norm_after=True, norm_offset=1.0, dense_activation=CLAMPED, tied_head=True))}


@dataclass(frozen=True)
class AttentionMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float  # 0: none
    chunk: int      # 0: none
    v_mix: bool

    @property
    def columns(self) -> int:
        return self.heads * self.dim + self.kv_heads * (self.dim + self.vdim)


@dataclass(frozen=True)
class Mamba2Mixer:
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_groups: int

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    @property
    def columns(self) -> int:
        return self.inner + self.channels + self.heads


@dataclass(frozen=True)
class Rotation:
    dims: int      # rotated components of a head, the first ones; 0: none
    base: float
    factor: float  # every frequency is divided by it

    @property
    def frequencies(self) -> np.ndarray:
        return self.base ** (-2.0 * np.arange(self.dims // 2, dtype=np.float64) / max(1, self.dims)) / self.factor


@dataclass(frozen=True)
class WindowMixer:
    """Attention with a norm per head on queries and keys, rotation, and a sliding window."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float  # 0: none
    window: int     # 0: none
    rotation: Rotation

    @property
    def columns(self) -> int:
        return self.heads * self.dim + self.kv_heads * (self.dim + self.vdim)

    @property
    def out(self) -> int:
        return self.heads * self.vdim


@dataclass(frozen=True)
class DeltaMixer:
    """The gated delta rule with a decay per head and key channel."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim

    @property
    def out(self) -> int:
        return self.heads * self.vdim


@dataclass(frozen=True)
class ParallelMixer:
    """Two mixers on one input; their outputs are scaled and added."""
    left: WindowMixer
    right: DeltaMixer
    left_scale: float
    right_scale: float

    @property
    def out(self) -> int:
        return self.left.out + self.right.out


@dataclass(frozen=True)
class JointColumns:
    """Where the parts of a parallel layer's one input projection lie: the window attention's q | k | v, the delta
    rule's q | k | v, the inputs of its low-rank products, and (float32, behind `split`) its write strengths."""
    conv: int
    decay: int
    gate: int
    split: int
    total: int

    @staticmethod
    def of(mixer: ParallelMixer, decay_rank: int, gate_rank: int) -> "JointColumns":
        up = lambda n: (n + _ALIGNED - 1) // _ALIGNED * _ALIGNED
        conv = up(mixer.left.columns)
        decay = up(conv + mixer.right.channels)
        gate = up(decay + decay_rank)
        split = up(gate + gate_rank)
        return JointColumns(conv, decay, gate, split, split + mixer.right.heads)


@dataclass(frozen=True)
class DenseFfn:
    ff: int
    activation: int = GELU_TANH
    limit: float = 0.0  # CLAMPED


@dataclass(frozen=True)
class RoutedFfn:
    experts: int
    top: int
    ff: int
    shared_ff: int  # 0: no shared expert


@dataclass(frozen=True)
class Layer:
    mixer: object
    ffn: object  # None: no feed-forward


@dataclass(frozen=True)
class LayeredConfig:
    vocabulary: int
    width: int
    epsilon: float
    embedding_scale: float
    layers: tuple[Layer, ...]
    design: Design = DESIGNS["Barovik"]
    residual_scale: float = 1.0
    logit_softcap: float = 0.0  # 0: none

    @staticmethod
    def parse(config: dict) -> "LayeredConfig":
        design = DESIGNS[config.get("architecture", "Barovik")]
        layers = []
        for entry in config["layers"]:
            m, kind = entry["mixer"], entry["type"]
            if kind == "attention":
                mask = m.get("mask")
                mixer = AttentionMixer(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]),
                                       float(m.get("softcap") or 0.0), int(mask["size"]) if mask else 0,
                                       bool(m.get("v_mix")))
                if mixer.heads % mixer.kv_heads:
                    raise ValueError("heads must be a multiple of kv_heads")
            elif kind == "mamba2":
                mixer = Mamba2Mixer(m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"])
                if mixer.heads % mixer.groups or mixer.inner % mixer.norm_groups:
                    raise ValueError("heads must be a multiple of groups, heads * vdim of norm_groups")
            elif kind == "parallel":
                mixer = _parallel_mixer(m)
            else:
                raise ValueError(f"unknown mixer type {kind}")
            f = entry.get("mlp")
            if f is None:
                ffn = None
            elif f["kind"] == "dense":
                ffn = DenseFfn(f["ff"], design.dense_activation, float(f.get("limit") or 0.0))
                if ffn.activation == CLAMPED and ffn.limit <= 0.0:
                    raise ValueError("a clamped feed-forward needs a positive limit")
            elif f["kind"] == "moe":
                shared = f.get("shared")
                ffn = RoutedFfn(f["router"]["experts"], f["router"]["top"], f["expert"]["ff"],
                                shared["ff"] if shared else 0)
            else:
                raise ValueError(f"unknown feed-forward kind {f['kind']}")
            if design.norm_after and not (isinstance(mixer, ParallelMixer) and isinstance(ffn, (DenseFfn, type(None)))):
                raise ValueError("norms on outputs go with parallel mixers and dense feed-forwards")
            if not design.norm_after and isinstance(mixer, ParallelMixer):
                raise ValueError("parallel mixers go with norms on outputs")
            layers.append(Layer(mixer, ffn))
        mixing = {(l.mixer.kv_heads, l.mixer.vdim) for l in layers
                  if isinstance(l.mixer, AttentionMixer) and l.mixer.v_mix}
        if len(mixing) > 1:
            raise ValueError("layers that mix values need values of one shape")
        return LayeredConfig(config["vocab"], config["width"], float(config["norm"]["eps"]),
                             float(config.get("embedding", {}).get("scale", 1.0)), tuple(layers), design,
                             float(config.get("residual_mult", 1.0)), float(config.get("logit_softcap") or 0.0))

    def tensor_shapes(self) -> dict[str, tuple[int, ...]]:
        """Every tensor of the weight file.  (A sink may be absent: the softmax then has none.)  None: a size that only
        the file knows (the ranks of low-rank products)."""
        w = self.width
        shapes: dict[str, tuple[int, ...]] = {"embed": (self.vocabulary, w)}
        for index, layer in enumerate(self.layers):
            p, m, f = f"l{index}.", layer.mixer, layer.ffn
            shapes[p + "norm1"] = (w,)
            if isinstance(m, AttentionMixer):
                shapes.update({p + "mix.q": (m.heads * m.dim, w), p + "mix.k": (m.kv_heads * m.dim, w),
                               p + "mix.v": (m.kv_heads * m.vdim, w), p + "mix.sink": (m.heads,),
                               p + "mix.o": (w, m.heads * m.vdim)})
                if m.v_mix:
                    shapes[p + "mix.vmix"] = ()
            elif isinstance(m, ParallelMixer):
                left, right, q = m.left, m.right, p + "mix.left."
                shapes.update({q + "q": (left.heads * left.dim, w), q + "k": (left.kv_heads * left.dim, w),
                               q + "v": (left.kv_heads * left.vdim, w), q + "q.norm": (left.dim,),
                               q + "k.norm": (left.dim,), q + "o": (w, left.out)})
                q, keys, values = p + "mix.right.", right.kv_heads * right.dim, right.heads * right.vdim
                for name, rows in (("q", keys), ("k", keys), ("v", values)):
                    shapes.update({q + name: (rows, w), q + name + ".conv": (rows, right.taps)})
                decays = right.heads * right.dim
                shapes.update({q + "b": (right.heads, w), q + "A_log": (right.heads,), q + "norm": (right.vdim,),
                               q + "a1": (None, w), q + "a2": (decays, None), q + "dt_bias": (decays,),
                               q + "g1": (None, w), q + "g2": (values, None), q + "o": (w, values)})
            else:
                shapes.update({p + "mix.in": (m.columns, w), p + "mix.conv": (m.channels, m.taps),
                               p + "mix.conv.b": (m.channels,), p + "mix.dt_bias": (m.heads,),
                               p + "mix.A_log": (m.heads,), p + "mix.D": (m.heads,), p + "mix.norm": (m.inner,),
                               p + "mix.o": (w, m.inner)})
            if f is None:
                continue
            shapes[p + "norm2"] = (w,)
            if isinstance(f, DenseFfn):
                shapes.update(self._gated(p + "mlp.", f.ff))
                continue
            shapes[p + "mlp.router"] = (f.experts, w)
            for e in range(f.experts):
                shapes.update(self._gated(f"{p}mlp.e{e}.", f.ff))
            if f.shared_ff:
                shapes.update(self._gated(p + "mlp.shared.", f.shared_ff))
                shapes[p + "mlp.shared.sg"] = (1, w)
        shapes["final.norm"] = (w,)
        if not self.design.tied_head:
            shapes["head"] = (self.vocabulary, w)
        return shapes

    def _gated(self, prefix: str, ff: int) -> dict:
        return {prefix + "gate": (ff, self.width), prefix + "up": (ff, self.width), prefix + "down": (self.width, ff)}

    def random_tensors(self, rng, rank: int = 12) -> dict[str, np.ndarray]:
        """Seeded weights of this shape (bfloat16 patterns): projections that keep the scale of their input.
        rank: that of low-rank products."""
        out = {}
        for name, shape in self.tensor_shapes().items():
            shape = tuple(rank if size is None else size for size in shape)
            kind = name.rsplit(".", 1)[-1]
            if "norm" in kind:
                value = rng.uniform(0.5, 1.5, shape) - (0.0 if name.startswith("l") and ".mix." in name
                                                        else self.design.norm_offset)
            elif kind in ("A_log", "dt_bias", "D", "b", "sink") and len(shape) < 2:
                value = rng.uniform(-1.0, 1.0, shape)
            elif kind == "vmix":
                value = rng.uniform(0.2, 0.8, shape)
            elif kind == "conv":
                value = rng.standard_normal(shape) / np.sqrt(shape[-1])
            else:
                value = rng.standard_normal(shape, dtype=np.float32) * (0.5 if name == "embed" else shape[-1] ** -0.5)
            out[name] = to_bfloat16(value)
        return out


def _parallel_mixer(m: dict) -> ParallelMixer:
    left, right = m["left"], m["right"]
    mask, rot = left.get("mask"), left.get("rot")
    scaling = (rot or {}).get("scaling")
    rotation = Rotation(rot["dims"], float(rot["base"]), float(scaling["factor"]) if scaling else 1.0) if rot else \
        Rotation(0, 1.0, 1.0)
    window = WindowMixer(left["heads"], left["kv_heads"], left["dim"], left["vdim"], float(left["scale"]),
                         float(left.get("softcap") or 0.0), int(mask["size"]) if mask else 0, rotation)
    delta = DeltaMixer(right["heads"], right["kv_heads"], right["dim"], right["vdim"], right["conv"])
    for part in (window, delta):
        if part.heads % part.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
    if rotation.dims % 2 or rotation.dims > window.dim:
        raise ValueError("a head rotates an even number of its components")
    return ParallelMixer(window, delta, float(m["left_scale"]), float(m["right_scale"]))


def _state_shapes(mixer, max_context: int) -> tuple:
    """What a layer carries from token to token."""
    if isinstance(mixer, AttentionMixer):
        return (RingShape.of(mixer.kv_heads, mixer.dim, mixer.vdim, mixer.chunk, max_context),)
    if isinstance(mixer, Mamba2Mixer):
        return (RecurrentShape(mixer.heads, mixer.vdim, mixer.state, mixer.channels, mixer.taps),)
    left, right = mixer.left, mixer.right
    return (RingShape.of(left.kv_heads, left.dim, left.vdim, left.window, max_context),
            RecurrentShape(right.heads, right.vdim, right.dim, right.channels, right.taps))


class _Tensors:
    """Checked access to a weight source: a safetensors file or a mapping of bfloat16 patterns."""

    def __init__(self, config: LayeredConfig, source):
        self._shapes, self._source = config.tensor_shapes(), source

    def __contains__(self, name):
        return name in self._source

    def __getitem__(self, name) -> np.ndarray:
        shape = self._shapes[name]
        if isinstance(self._source, SafetensorsFile):
            if None in shape:
                own = self._source.numpy(name).shape
                shape = tuple(o if s is None else s for s, o in zip(shape, own)) if len(own) == len(shape) else shape
            return self._source.bfloat16(name, shape)
        array = np.asarray(self._source[name])
        if array.dtype != np.uint16 or array.ndim != len(shape) or \
                any(s is not None and s != n for s, n in zip(shape, array.shape)):
            raise ValueError(f"tensor {name} must be bfloat16 patterns of shape {list(shape)}")
        return array


class LayeredModel:
    """Device weights, state pool and steps of one layered decoder.

    activations: "bfloat16" or "float32" (weights are bfloat16 in both).  slots: sequences that can be
    live at once; max_context: the longest of them."""

    def __init__(self, runtime: Runtime, config: LayeredConfig, tensors, activations: str = "bfloat16",
                 slots: int = 8, max_context: int = 32768):
        if activations not in ("bfloat16", "float32"):
            raise ValueError(f"unknown activation type {activations}")
        self.runtime, self.config = runtime, config
        self.suffix, self.element = ("_bf16", 2) if activations == "bfloat16" else ("_f32", 4)
        self.vocabulary = config.vocabulary
        self._shapes = [_state_shapes(layer.mixer, max_context) for layer in config.layers]
        self.state = StatePool(runtime, self._shapes, slots, max_context, self.element)
        self._upload(_Tensors(config, tensors))
        self._work: Optional[_Work] = None
        self._lists: dict[int, DispatchList] = {}
        self._decode: Optional[_DecodePlan] = None

    @staticmethod
    def load(runtime: Runtime, directory: str, config: dict, **options) -> "LayeredModel":
        path = os.path.join(directory, "model.safetensors")
        return LayeredModel(runtime, LayeredConfig.parse(config), SafetensorsFile(path), **options)

    # ---- weights ----
    def _upload(self, t: _Tensors) -> None:
        put = self.runtime.buffer_of_bytes
        stack = lambda names: put(np.concatenate([t[name] for name in names]))
        self.embed, self.final_norm = put(t["embed"]), put(t["final.norm"])
        self.head = self.embed if self.config.design.tied_head else put(t["head"])
        self.layers = []
        mixing_seen = False
        for index, layer in enumerate(self.config.layers):
            p, m, f = f"l{index}.", layer.mixer, layer.ffn
            d = {"norm1": put(t[p + "norm1"])}
            if isinstance(m, ParallelMixer):
                d.update(self._upload_parallel(t, p + "mix.", m))
            else:
                d["o"] = put(t[p + "mix.o"])
            if isinstance(m, AttentionMixer):
                d["qkv"] = stack([p + "mix.q", p + "mix.k", p + "mix.v"])
                d["sink"] = put(t[p + "mix.sink"]) if p + "mix.sink" in t else None
                # values: as they are, the first to be mixed in, or mixed with those
                d["mix"] = (0, 0.0)
                if m.v_mix:
                    d["mix"] = (2, float(from_bfloat16(t[p + "mix.vmix"]))) if mixing_seen else (1, 0.0)
                    mixing_seen = True
            elif isinstance(m, Mamba2Mixer):
                for key in ("in", "conv", "conv.b", "dt_bias", "A_log", "D", "norm"):
                    d[key] = put(t[p + "mix." + key])
            if f is not None:
                d["norm2"] = put(t[p + "norm2"])
                p += "mlp."
                if isinstance(f, DenseFfn):
                    d["ffn"] = [put(t[p + key]) for key in ("gate", "up", "down")]
                else:
                    d["router"] = stack([p + "router"] + ([p + "shared.sg"] if f.shared_ff else []))
                    d["ffn"] = [stack([f"{p}e{e}.{key}" for e in range(f.experts)]) for key in ("gate", "up", "down")]
                    d["shared"] = [put(t[p + "shared." + key]) for key in ("gate", "up", "down")] if f.shared_ff \
                        else d["ffn"]
            self.layers.append(d)

    def _upload_parallel(self, t: _Tensors, p: str, m: ParallelMixer) -> dict:
        """One input projection for both mixers and one output projection over their rows side by side."""
        put, width, q = self.runtime.buffer_of_bytes, self.config.width, p + "right."
        decay_in, decay, gate_in, gate = t[q + "a1"], t[q + "a2"], t[q + "g1"], t[q + "g2"]
        if decay_in.shape[0] != decay.shape[1] or gate_in.shape[0] != gate.shape[1]:
            raise ValueError(f"the low-rank products of {q} do not fit together")
        columns = JointColumns.of(m, decay_in.shape[0], gate_in.shape[0])
        joint = np.zeros((columns.total, width), dtype=np.uint16)
        for start, names in ((0, [p + "left.q", p + "left.k", p + "left.v"]), (columns.conv, [q + "q", q + "k", q + "v"]),
                             (columns.decay, [q + "a1"]), (columns.gate, [q + "g1"]), (columns.split, [q + "b"])):
            part = np.concatenate([t[name] for name in names])
            joint[start:start + len(part)] = part
        frequencies = m.left.rotation.frequencies
        return {"columns": columns, "ranks": (decay_in.shape[0], gate_in.shape[0]), "joint": put(joint),
                "o": put(np.concatenate([t[p + "left.o"], t[q + "o"]], axis=1)),
                "q_norm": put(t[p + "left.q.norm"]), "k_norm": put(t[p + "left.k.norm"]),
                "frequencies": put(frequencies if len(frequencies) else np.zeros(1)),
                "conv": put(np.concatenate([t[q + name + ".conv"] for name in "qkv"])),
                "decay": put(decay), "gate": put(gate), "dt_bias": put(t[q + "dt_bias"]), "A_log": put(t[q + "A_log"]),
                "norm": put(t[q + "norm"])}

    # ---- the step's dispatch list ----
    def _pending(self, work: "_Work", stream: "_Stream") -> tuple[list, bytes]:
        """Operands and parameters of a pending output; the new stream is in the other buffer afterwards."""
        c = self.config
        buffers = [work.streams[stream.at], work.output, stream.pending or self.final_norm, work.streams[1 - stream.at]]
        parameters = u32s(int(stream.pending is not None)) + struct.pack("<fff", c.epsilon, c.design.norm_offset,
                                                                         c.residual_scale)
        return buffers, parameters

    def _parallel_dispatches(self, index: int, m: int, work: "_Work", stream: "_Stream") -> list[tuple]:
        """A layer whose sublayers read the stream itself and whose outputs stay pending."""
        c, layer, d, s = self.config, self.config.layers[index], self.layers[index], self.suffix
        mixer, columns, slots = layer.mixer, d["columns"], self.state.slots
        left, right, eps = mixer.left, mixer.right, struct.pack("<f", c.epsilon)
        (ring, _), ((keys, values), (conv_ring, state)) = self._shapes[index], self.state.regions[index]
        grid = ((m, 1, 1), (256, 1, 1))
        buffers, pending = self._pending(work, stream)
        out = [("llmopt_joint_input" + s, buffers + [d["joint"], work.step, d["conv"], conv_ring, work.projected, work.extra],
                u32s(m, c.width, columns.total, columns.split, columns.conv, right.channels, right.taps, slots) + pending,
                *grid)]
        stream.joined()
        out.append(("llmopt_rotary_attention" + s,
                    [work.projected, d["q_norm"], d["k_norm"], d["frequencies"], work.step, keys, values, work.mixed],
                    u32s(m, left.heads, left.kv_heads, left.dim, left.vdim, columns.split, mixer.out, ring.capacity,
                         ring.span, 1, slots, left.rotation.dims) + struct.pack("<ff", left.scale, left.softcap) + eps +
                    struct.pack("<f", mixer.left_scale), *grid))
        out.append(("llmopt_gated_delta" + s,
                    [work.projected, work.extra, d["decay"], d["dt_bias"], d["A_log"], d["gate"], d["norm"], d["conv"],
                     conv_ring, state, work.step, work.mixed],
                    u32s(m, right.heads, right.kv_heads, right.dim, right.vdim, right.taps, slots, columns.split, columns.conv,
                         columns.decay, columns.gate, columns.split, *d["ranks"], mixer.out, left.out) + eps +
                    struct.pack("<f", mixer.right_scale), *grid))
        out.append(("llmopt_linear_store" + s, [work.mixed, d["o"], work.output], u32s(m, c.width, mixer.out), *grid))
        stream.pending = d["norm1"]
        if layer.ffn is not None:
            buffers, pending = self._pending(work, stream)
            out.append(("llmopt_pending_gated_ffn" + s, buffers + [*d["ffn"], work.output],
                        u32s(m, c.width, layer.ffn.ff, layer.ffn.activation) + struct.pack("<f", layer.ffn.limit) + pending,
                        *grid))
            stream.joined()
            stream.pending = d["norm2"]
        return out

    def _layer_dispatches(self, index: int, m: int, work: "_Work", stream: "_Stream") -> list[tuple]:
        if isinstance(self.config.layers[index].mixer, ParallelMixer):
            return self._parallel_dispatches(index, m, work, stream)
        c, layer, d, (shape,) = self.config, self.config.layers[index], self.layers[index], self._shapes[index]
        mixer, ffn, s = layer.mixer, layer.ffn, self.suffix
        ((first, second),) = self.state.regions[index]
        eps = struct.pack("<f", c.epsilon)
        grid = ((m, 1, 1), (256, 1, 1))
        out = []
        if isinstance(mixer, AttentionMixer):
            sizes = (mixer.heads, mixer.kv_heads, mixer.dim, mixer.vdim)
            ring = (shape.capacity, shape.span, self.state.slots)
            mode, mix = d["mix"]
            out.append(("llmopt_rms_qkv_chunk" + s,
                        [work.stream, d["norm1"], d["qkv"], work.step, work.projected, work.first_values, first, second],
                        u32s(m, c.width, *sizes) + eps + struct.pack("<If", mode, mix) + u32s(*ring), *grid))
            out.append(("llmopt_chunk_attention" + s,
                        [work.projected, d["sink"] or d["norm1"], work.step, first, second, work.mixed],
                        u32s(m, *sizes, *ring, int(d["sink"] is not None)) +
                        struct.pack("<ff", mixer.scale, mixer.softcap), *grid))
            out.append(("llmopt_linear_add" + s, [work.mixed, d["o"], work.stream],
                        u32s(m, c.width, mixer.heads * mixer.vdim), *grid))
        else:
            sizes = (mixer.heads, mixer.vdim, mixer.groups, mixer.state, mixer.taps, self.state.slots)
            out.append(("llmopt_rms_ssm_input" + s,
                        [work.stream, d["norm1"], d["in"], work.step, d["conv"], d["conv.b"], d["dt_bias"], first,
                         work.projected, work.dt], u32s(m, c.width, *sizes) + eps, *grid))
            out.append(("llmopt_ssm_mix" + s,
                        [work.step, work.projected, work.dt, d["conv"], d["conv.b"], d["dt_bias"], d["A_log"], d["D"],
                         first, second, work.mixed], u32s(m, *sizes), *grid))
            out.append(("llmopt_gated_norm_linear_add" + s,
                        [work.mixed, work.projected, d["norm"], d["o"], work.stream],
                        u32s(m, mixer.inner, mixer.inner + mixer.channels, mixer.norm_groups, c.width) + eps, *grid))
        if isinstance(ffn, DenseFfn):
            out.append(("llmopt_rms_gated_ffn_add" + s, [work.stream, d["norm2"], *d["ffn"]],
                        u32s(m, c.width, ffn.ff) + eps + u32s(ffn.activation), *grid))
        elif isinstance(ffn, RoutedFfn):
            out.append(("llmopt_rms_routed_ffn_add" + s,
                        [work.stream, d["norm2"], d["router"], *d["ffn"], *d["shared"]],
                        u32s(m, c.width, ffn.experts, ffn.top, ffn.ff, ffn.shared_ff) + eps + u32s(SILU), *grid))
        return out

    def _embedding(self, m: int, work: "_Work") -> tuple:
        c = self.config
        return ("llmopt_embedding_scaled_bf16", [work.tokens, self.embed, work.stream],
                u32s(m, c.vocabulary, c.width) + struct.pack("<f", c.embedding_scale), (m, 1, 1), (256, 1, 1))

    def _logits(self, rows: int, m: int, work: "_Work", stream: "_Stream", index: Buffer, out: Buffer) -> tuple:
        c = self.config
        if c.design.norm_after:
            buffers, pending = self._pending(work, stream)
            return ("llmopt_pending_logits" + self.suffix, buffers + [index, self.final_norm, self.head, out],
                    u32s(rows, c.width, c.vocabulary, m) + pending + struct.pack("<f", c.logit_softcap),
                    (rows, 1, 1), (256, 1, 1))
        return ("llmopt_rms_logits" + self.suffix, [work.stream, index, self.final_norm, self.head, out],
                u32s(rows, c.width, c.vocabulary) + struct.pack("<f", c.epsilon) + u32s(m), (rows, 1, 1), (256, 1, 1))

    def dispatches(self, m: int, work: "_Work") -> tuple[list[tuple], "_Stream"]:
        """The step's list, and where it leaves the stream."""
        out, stream = [self._embedding(m, work)], _Stream()
        for index in range(len(self.layers)):
            out += self._layer_dispatches(index, m, work, stream)
        return out, stream

    def _observe(self, m: int, work: "_Work", stream: "_Stream", out: Buffer, batch) -> None:
        """The stream behind the layers so far, a pending output included, into `out`."""
        if stream.pending is None:
            batch.copy(work.streams[stream.at].view(0, m * self.config.width * 4), out)
            return
        buffers, pending = self._pending(work, stream)
        batch.dispatch_all(DispatchList([("llmopt_norm_add_f32", buffers[:3] + [out], u32s(m, self.config.width) + pending,
                                          (m, 1, 1), (256, 1, 1))]))

    # ---- steps ----
    def open(self) -> Sequence:
        return self.state.open()

    def close(self, sequence: Sequence) -> None:
        self.state.close(sequence)

    def step(self, sequence: Sequence, tokens: Tokens[int], want: Tokens[int] = (),
             streams: Optional[list] = None) -> np.ndarray:
        """Runs the next tokens of a sequence; returns the float32 logits [len(want), vocabulary] at the
        places `want` among them.  streams: a list that receives the residual stream after every layer."""
        tokens = np.asarray(tokens, dtype=np.int64).reshape(-1)
        m = len(tokens)
        if m == 0:
            raise ValueError("a step has at least one token")
        if m and (tokens.min() < 0 or tokens.max() >= self.vocabulary):
            raise ValueError("a token is outside the vocabulary")
        want = np.asarray(want, dtype=np.uint32).reshape(-1)
        if len(want) and int(want.max()) >= m:
            raise ValueError("a wanted place is outside the step")
        self.state.reserve(sequence, m)
        if m == 1 and streams is None:
            plan = self.decode_plan()
            plan.execute(int(tokens[0]), sequence)
            rows = plan.logits.numpy(np.float32, (1, self.vocabulary)) if len(want) else \
                np.zeros((1, self.vocabulary), dtype=np.float32)
            return rows[want.astype(np.int64)]
        if self._work is None or self._work.m < m:
            self._lists.clear()
            self._work = _Work(self, m)
        work = self._work
        work.tokens.write(tokens)
        work.step.write(np.array([sequence.position, sequence.slot], dtype=np.uint32))
        batch = self.runtime.begin_batch()
        observed = []
        if streams is None:
            if m not in self._lists:
                if len(self._lists) >= 64:
                    self._lists.clear()
                dispatches, stream = self.dispatches(m, work)
                self._lists[m] = DispatchList(dispatches), stream
            batch.dispatch_all(self._lists[m][0])
            stream = self._lists[m][1]
        else:
            stream = _Stream()
            batch.dispatch_all(DispatchList([self._embedding(m, work)]))
            for index in range(len(self.layers)):
                batch.dispatch_all(DispatchList(self._layer_dispatches(index, m, work, stream)))
                observed.append(self.runtime.create_buffer(m * self.config.width * 4))
                self._observe(m, work, stream, observed[-1], batch)
        logits = None
        if len(want):
            index = self.runtime.buffer_of_bytes(want)
            logits = self.runtime.create_buffer(len(want) * self.vocabulary * 4)
            batch.dispatch_all(DispatchList([self._logits(len(want), m, work, stream, index, logits)]))
        batch.commit()
        sequence.position += m
        if streams is not None:
            streams += [b.numpy(np.float32, (m, self.config.width)) for b in observed]
        if logits is None:
            return np.zeros((0, self.vocabulary), dtype=np.float32)
        return logits.numpy(np.float32, (len(want), self.vocabulary))

    def decode_plan(self) -> "_DecodePlan":
        if self._decode is None:
            self._decode = _DecodePlan(self)
        return self._decode

    def decode(self, sequence: Sequence, token: int) -> int:
        """One token through the retained plan; returns the argmax of its logits."""
        self.state.reserve(sequence, 1)
        return self.decode_plan().execute(token, sequence)

    def logits_row(self) -> np.ndarray:
        """The logits the last one-token step left."""
        return self.decode_plan().logits.numpy(np.float32, (self.vocabulary,))


@dataclass
class _Stream:
    """Where a list being built has the residual stream: in which buffer, and the norm of an output that has not
    joined it yet."""
    at: int = 0
    pending: Optional[Buffer] = None

    def joined(self) -> None:
        if self.pending is not None:
            self.at, self.pending = 1 - self.at, None


class _Work:
    """Activations of a step of up to m tokens, shared by all layers."""

    def __init__(self, model: LayeredModel, m: int):
        c, create = model.config, model.runtime.create_buffer
        self.m = m
        projected = mixed = heads = values = extra = 1
        for layer in c.layers:
            mixer = layer.mixer
            if isinstance(mixer, AttentionMixer):
                projected, mixed = max(projected, mixer.columns), max(mixed, mixer.heads * mixer.vdim)
                values = max(values, mixer.kv_heads * mixer.vdim)
            elif isinstance(mixer, ParallelMixer):
                mixed, extra = max(mixed, mixer.out), max(extra, mixer.right.heads)
            else:
                projected, mixed, heads = max(projected, mixer.columns), max(mixed, mixer.inner), max(heads, mixer.heads)
        for d in model.layers:
            if "columns" in d:
                projected = max(projected, d["columns"].total)
        element = 4 if m == 1 else model.element  # one token: recurrent mixers keep their rows in float32
        self.tokens = create(m * 8)
        self.step = create(8)
        # a pending output joins the stream from one buffer to the other
        self.streams = [create(m * c.width * 4) for _ in range(2 if c.design.norm_after else 1)]
        self.stream = self.streams[0]
        self.output = create(m * c.width * 4) if c.design.norm_after else None
        self.extra = create(m * extra * 4)
        self.projected = create(m * projected * element)
        self.mixed = create(m * mixed * element)
        self.dt = create(m * heads * 4)
        self.first_values = create(m * values * 4)


class _DecodePlan:
    """One token, its logits and their argmax as one HIP graph for every position and slot."""

    def __init__(self, model: LayeredModel):
        work = _Work(model, 1)
        self.work = work
        self.logits = model.runtime.create_buffer(model.vocabulary * 4)
        self.token = model.runtime.create_buffer(4)
        self.dispatches, stream = model.dispatches(1, work)
        self.dispatches.append(model._logits(1, 1, work, stream, work.step, self.logits))
        self.dispatches.append(("llmopt_argmax_f32", [self.logits, self.token], u32s(1, model.vocabulary),
                                (256, 1, 1), (256, 1, 1)))
        self.plan = Prebaked(model.runtime, self.dispatches, work.tokens, self.token)
        self.plan.bind_step(work.step, model.state.max_context - 1, model.state.slots)

    def execute(self, token: int, sequence: Sequence) -> int:
        out = self.plan.execute(token, sequence.position, sequence.slot)
        sequence.position += 1
        return out
