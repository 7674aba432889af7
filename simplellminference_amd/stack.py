"""Block-stack models (include/sli.h ``sli_stack_config``): decoders of parallel blocks with attention and retention
mixers, or of sequential sublayers with latent attention and mixtures of experts, behind the same engine handle, decode
loop and greedy sampling as ``LlamaModel``.

``StackModel`` takes any ``StackSpec``; ``Rugudra`` and ``Bokulix`` read one design's ``config.json`` into it."""
from __future__ import annotations

import ctypes
import os
import re
from dataclasses import dataclass, field

import numpy as np

from . import _lib
from ._lib import DT_F16, DT_F32, BlockDesc, StackConfig as _CStackConfig, call
from .checkpoint import SafeTensors
from .model import LlamaModel

# storage per --dtype: bfloat16 checkpoints are served with fp16 weights and cache (every bfloat16 value of magnitude
# 2^-14 .. 65504 is an fp16 value), float32 in fp32 throughout
MIXERS = ("attention", "retention", "latent")  # sli_mixer_kind
ARRANGEMENTS = ("parallel", "sequential")  # sli_stack_arrangement

DTYPES = {"bfloat16": DT_F16, "bf16": DT_F16, "float16": DT_F16, "f16": DT_F16, "fp16": DT_F16,
          "float32": DT_F32, "f32": DT_F32, "fp32": DT_F32}


@dataclass(frozen=True)
class BlockSpec:
    mixer: str  # of MIXERS
    heads: int
    dim: int
    vdim: int
    kv_heads: int = 0
    scale: float = 1.0
    decay: tuple[float, ...] = ()
    rot_dims: int = 0
    rot_base: float = 10000.0
    ff: int = 0  # rows of the feed-forward (of each expert)
    ff_limit: float = 0.0
    kv_rank: int = 0  # latent attention
    window: int = 0  # latent attention: positions a query sees, itself included (0: all)
    experts: int = 0  # 0: a dense feed-forward
    top: int = 0


@dataclass(frozen=True)
class StackSpec:
    vocab_size: int
    width: int
    blocks: tuple[BlockSpec, ...]
    loop: tuple[int, int, int] = (0, 0, 1)  # blocks start .. stop - 1 run `times` times
    taps: int = 1
    eps: float = 1e-6
    emb_scale: float = 1.0
    residual_mult: float = 1.0
    max_length: int = 1024
    extra: dict = field(default_factory=dict, compare=False)
    arrangement: str = "parallel"
    positions: int = 0  # rows of the learned position table (0: none)
    runs: tuple[int, ...] = ()  # block of every run (empty: by `loop`)
    layer_names: tuple[int, ...] = ()  # block i's tensors are l<layer_names[i]>.* in the file (empty: l<i>.*)

    @property
    def order(self) -> list[int]:
        """Block index of every run of a forward pass."""
        if self.runs:
            return list(self.runs)
        a, b, n = self.loop
        return list(range(a)) + list(range(a, b)) * n + list(range(b, len(self.blocks)))

    def tensor_names(self, names) -> list[tuple[str, str]]:
        """(name in the file, name in the model) of the tensors to place. Left out: what a block without a feed-forward
        may still name of its second sublayer."""
        block_of = {n: i for i, n in enumerate(self.layer_names or range(len(self.blocks)))}
        out = []
        for name in names:
            m = re.fullmatch(r"l(\d+)\.(.+)", name)
            i = block_of.get(int(m[1])) if m else None
            if i is None:
                out.append((name, name if not m else f"l{len(self.blocks)}.{m[2]}"))  # (no block's: refused by the model)
            elif self.blocks[i].ff or m[2] not in ("norm2", "canon2", "rg2", "rg2.b"):
                out.append((name, f"l{i}.{m[2]}"))
        return out


class StackModel(LlamaModel):
    """The engine handle of a block-stack model: ``predict``, ``predict_batch``, ``predict_prefill``, ``step``,
    ``logits``, ``state`` … as on ``LlamaModel``; ``feed`` runs the next tokens of any sequences as one batch."""

    def __init__(self, spec: StackSpec, model_path: str = "", dtype: str = "bfloat16", batch: int = 1, device: int = 0,
                 seed: int | None = None, tokenizer_path: str = ""):
        self.spec = self.config = spec
        self.model_path, self.tokenizer_path = model_path, tokenizer_path
        if dtype not in DTYPES:
            raise ValueError(f"unknown dtype {dtype!r}")
        self.w_dtype = self.kv_dtype = DTYPES[dtype]
        self.tp_rank, self.tp_size = 0, 1
        self.device, self.seed, self.batch = device, seed, batch
        self._h = None
        self.encode_layer = None

    def init(self) -> "StackModel":
        if self.tokenizer_path:
            from .encode import SPELayer
            self.encode_layer = SPELayer(self.tokenizer_path)
        s = self.spec
        blocks = (BlockDesc * len(s.blocks))()
        decay: list[float] = []
        for d, b in zip(blocks, s.blocks):
            if b.mixer not in MIXERS:
                raise ValueError(f"unknown mixer {b.mixer!r}")
            d.mixer = MIXERS.index(b.mixer)
            d.heads, d.kv_heads, d.dim, d.vdim = b.heads, b.kv_heads, b.dim, b.vdim
            d.scale, d.rot_dims, d.rot_base = b.scale, b.rot_dims, b.rot_base
            d.ff, d.ff_limit = b.ff, b.ff_limit
            d.kv_rank, d.window, d.experts, d.top = b.kv_rank, b.window, b.experts, b.top
            if d.mixer == 1:
                if len(b.decay) != b.heads:
                    raise ValueError("retention: one decay per head")
                decay += list(b.decay)
        dec = np.ascontiguousarray(decay or [0.0], np.float32)
        if s.arrangement not in ARRANGEMENTS:
            raise ValueError(f"unknown arrangement {s.arrangement!r}")
        runs = np.ascontiguousarray(s.runs, np.int32)
        c = _CStackConfig(s.vocab_size, s.width, len(s.blocks), *s.loop, s.taps, s.eps, s.emb_scale, s.residual_mult,
                          blocks, dec.ctypes.data_as(_lib.P_f), self.w_dtype, s.max_length, self.batch, self.device,
                          ARRANGEMENTS.index(s.arrangement), s.positions,
                          runs.ctypes.data_as(_lib.P_i32) if runs.size else None, runs.size)
        h = ctypes.c_void_p()
        call("sli_stack_create", ctypes.byref(c), ctypes.byref(h))
        self._h = h
        return self._load_weights()

    def _load_weights(self) -> "StackModel":
        if self.model_path:
            st = SafeTensors(os.path.join(self.model_path, "model.safetensors"))
            for name, placed in self.spec.tensor_names(st.names()):
                self.set_tensor(placed, st.get(name))
        elif self.seed is not None:
            call("sli_model_init_synthetic", self._h, self.seed)
        return self

    def set_tensor(self, name: str, value: np.ndarray):
        t = np.ascontiguousarray(value, np.float32)
        call("sli_stack_set_tensor", self._h, name.encode(), t.ctypes.data_as(ctypes.c_void_p), t.size)

    @property
    def local_vocab(self) -> int:
        return self.spec.vocab_size

    @property
    def runs(self) -> int:
        return int(_lib.load().sli_stack_runs(self._h))

    def feed(self, slots, starts, tokens, want=None, want_hidden: bool = False):
        """One batch: sequence slot slots[i] goes on with tokens[i] from position starts[i] (0: a new sequence).
        want[i]: ascending places among tokens[i] whose logits are returned, as rows of one [wanted, vocab] array in
        entry order. want_hidden: also the residual after every block run, [runs, tokens, width]."""
        n = len(slots)
        lens = np.array([len(t) for t in tokens], np.int32)
        toks = np.ascontiguousarray(np.concatenate([np.asarray(t, np.int32) for t in tokens]), np.int32)
        want = want or [[] for _ in range(n)]
        wn = np.array([len(w) for w in want], np.int32)
        wl = np.ascontiguousarray([p for w in want for p in w] or [0], np.int32)
        sl, sp = np.ascontiguousarray(slots, np.int32), np.ascontiguousarray(starts, np.int32)
        out = np.empty((int(wn.sum()), self.local_vocab), np.float32)
        hid = np.empty((self.runs, toks.size, self.spec.width), np.float32) if want_hidden else None
        ptr = [a.ctypes.data_as(ctypes.c_void_p) for a in (sl, sp, lens, toks, wn, wl, out)]
        call("sli_model_feed", self._h, n, *ptr, hid.ctypes.data_as(ctypes.c_void_p) if want_hidden else None)
        return (out, hid) if want_hidden else out

    def predict_prefill(self, prompt_ids, max_length: int, want_logits: bool = False):
        if self.batch != 1:
            raise ValueError("predict_prefill: batch 1 (predict_batch_prefill for a batch)")
        return super().predict_prefill(prompt_ids, max_length, want_logits)

    def predict_batch_prefill(self, prompts, max_length: int) -> np.ndarray:
        """Greedy tokens [batch, max_length] (the token fed at each position) of `batch` prompts: the prompts in packed
        passes, then decode steps until the shortest sequence has max_length tokens."""
        if len(prompts) != self.batch:
            raise ValueError(f"need {self.batch} prompts")
        lens = np.array([len(p) for p in prompts], np.int32)
        if lens.max() > max_length or max_length > self.spec.max_length:
            raise ValueError("max_length must be in [longest prompt, max_length of the model]")
        ld = int(lens.max())
        P = np.zeros((self.batch, ld), np.int32)
        for b, p in enumerate(prompts):
            P[b, :len(p)] = p
        call("sli_model_prefill_batch", self._h, P.ctypes.data_as(ctypes.c_void_p), lens.ctypes.data_as(ctypes.c_void_p), ld)
        for _ in range(max_length - int(lens.min())):
            self.step()
        return np.stack([self.history(b, max_length) for b in range(self.batch)])


def rugudra_spec(cfg: dict, max_length: int) -> StackSpec:
    """A ``config.json`` of architecture "Rugudra" as a StackSpec."""
    blocks = []
    for e in cfg["layers"]:
        m, f = e["mixer"], e.get("mlp")
        if f is not None and f["kind"] != "dense":
            raise ValueError(f"unknown feed-forward kind {f['kind']!r}")
        ff = {"ff": f["ff"], "ff_limit": f["limit"]} if f is not None else {}
        if e["type"] == "attention":
            blocks.append(BlockSpec("attention", m["heads"], m["dim"], m["vdim"], kv_heads=m["kv_heads"],
                                    scale=m["scale"], **ff))
        elif e["type"] == "retention":
            blocks.append(BlockSpec("retention", m["heads"], m["dim"], m["vdim"], decay=tuple(m["decay"]),
                                    rot_dims=m["rot"]["dims"], rot_base=m["rot"]["base"], **ff))
        else:
            raise ValueError(f"unknown layer type {e['type']!r}")
    lp = cfg.get("loop")
    return StackSpec(cfg["vocab"], cfg["width"], tuple(blocks), (lp["start"], lp["stop"], lp["times"]) if lp else (0, 0, 1),
                     cfg["canon"]["taps"], cfg["norm"]["eps"], cfg["embedding"]["scale"], cfg["residual_mult"], max_length)


class Rugudra(StackModel):
    """Parallel blocks with an input convolution before each sublayer, retention and sink attention with a logarithmic
    distance bias, a clamped gated feed-forward, and a looped range of layers."""

    @classmethod
    def from_config(cls, cfg: dict, max_length: int, **kw) -> "Rugudra":
        return cls(rugudra_spec(cfg, max_length), **kw)


def bokulix_spec(cfg: dict, max_length: int) -> StackSpec:
    """A ``config.json`` of architecture "Bokulix" as a StackSpec. A layer with ``weights_of`` is another run of that
    layer's block."""
    blocks, names, runs, block_of = [], [], [], {}
    for i, e in enumerate(cfg["layers"]):
        if e.get("weights_of") is not None:
            continue
        if e["type"] != "latent_attention":
            raise ValueError(f"unknown layer type {e['type']!r}")
        m, f = e["mixer"], e.get("mlp")
        if f is not None and f["kind"] != "moe":
            raise ValueError(f"unknown feed-forward kind {f['kind']!r}")
        ff = {"ff": f["expert"]["ff"], "experts": f["router"]["experts"], "top": f["router"]["top"]} if f is not None else {}
        block_of[i] = len(blocks)
        names.append(i)
        blocks.append(BlockSpec("latent", m["heads"], m["dim"], m["vdim"], scale=m["scale"], kv_rank=m["kv_rank"],
                                window=(m.get("mask") or {}).get("size", 0), **ff))
    for i, e in enumerate(cfg["layers"]):
        seen = {i}
        while cfg["layers"][i].get("weights_of") is not None:
            i = cfg["layers"][i]["weights_of"]
            if i in seen or not 0 <= i < len(cfg["layers"]):
                raise ValueError("weights_of names no layer with weights")
            seen.add(i)
        runs.append(block_of[i])
    n = cfg["max_positions"]
    return StackSpec(cfg["vocab"], cfg["width"], tuple(blocks), taps=cfg["canon"]["taps"], eps=cfg["norm"]["eps"],
                     max_length=min(max_length, n), arrangement="sequential", positions=n, runs=tuple(runs),
                     layer_names=tuple(names))


class Bokulix(StackModel):
    """Sequential sublayers, each gated and normed on its output: windowed latent attention behind an input convolution,
    and a mixture of experts; learned positions, layers that share their weights."""

    @classmethod
    def from_config(cls, cfg: dict, max_length: int, **kw) -> "Bokulix":
        return cls(bokulix_spec(cfg, max_length), **kw)
