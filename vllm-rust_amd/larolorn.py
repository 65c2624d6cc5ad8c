"""Host-side driver of the Larolorn decoder family (libvmx `vmx_larolorn_*`).

A Larolorn model is a stack of layers listed in its config.json whose sublayers read the residual stream as it is and whose results
are RMS-normed before they are added, `x <- x + m N1(mixer(x)); x <- x + m N2(ff(x))`.  Mixers: "latent_attention" (compressed keys /
values in a paged cache, one rotated key part for all heads, a sliding window, a sigmoid per head on the output) and "parallel"
(grouped-query attention inside chunks of positions with a learned sink, beside a matrix memory with one constant decay per head in a
state slot per sequence; half the sum of the two normed branches).  Feed-forward: "dense" (a clamped sigmoid-gated product) or none.
A layer may run with another layer's weights (`weights_of`), with a cache and a state of its own.  This file reads the configuration,
hands the checkpoint's tensors to the library under their file names and wraps the one forward entry point.  All arithmetic happens
in the library.
"""
from __future__ import annotations

import ctypes as C
import dataclasses
import json
import math
import re
from pathlib import Path

import numpy as np
import torch

from ._lib import LarolornConfig, LarolornLayerConfig, check, lib
from .rotation import RotationSpec

VMX_F32, VMX_BF16 = 0, 1
MIXERS = {"latent_attention": 0, "parallel": 9}
MLPS = {None: 0, "dense": 8}


@dataclasses.dataclass
class LarolornLayerSpec:
    mixer: str = "latent_attention"
    # latent attention (dim: unrotated query / key coordinates) / the left attention of "parallel"
    heads: int = 4
    dim: int = 32
    vdim: int = 32
    scale: float = 0.125
    mask: int = 0                # latent attention: window, parallel: chunk (0: every earlier key)
    rot: RotationSpec = dataclasses.field(default_factory=RotationSpec)
    rot_dim: int = 16            # latent attention: rotated coordinates
    kv_rank: int = 64
    kv_heads: int = 4            # parallel
    # the right side of "parallel"
    r_heads: int = 0
    r_dim: int = 0
    r_vdim: int = 0
    decay: tuple = ()            # one constant per head
    mlp: str | None = "dense"
    ff: int = 64
    limit: float = 7.0
    weights_of: int | None = None    # the layer whose weights it runs with (None: its own)

    @staticmethod
    def from_config(entry: dict) -> "LarolornLayerSpec":
        kind, m = entry["type"], entry["mixer"]
        if kind not in MIXERS:
            raise ValueError(f"Larolorn: unknown layer type `{kind}`")
        a = m if kind == "latent_attention" else m["left"]
        s = LarolornLayerSpec(mixer=kind, heads=int(a["heads"]), dim=int(a["dim"]), vdim=int(a.get("vdim", a["dim"])), mlp=None)
        s.mask = int((a.get("mask") or {}).get("size") or 0)
        s.rot = RotationSpec.from_config(a.get("rot"))
        if kind == "latent_attention":
            s.rot_dim, s.kv_rank = int(a["rot_dim"]), int(a["kv_rank"])
            s.scale = float(a.get("scale", 1.0 / math.sqrt(s.dim + s.rot_dim)))
        else:
            r = m["right"]
            s.kv_heads = int(a.get("kv_heads", s.heads))
            s.scale = float(a.get("scale", 1.0 / math.sqrt(s.dim)))
            s.r_heads, s.r_dim, s.r_vdim = int(r["heads"]), int(r["dim"]), int(r.get("vdim", r["dim"]))
            s.decay = tuple(float(d) for d in r["decay"])
            if len(s.decay) != s.r_heads:
                raise ValueError(f"Larolorn: {len(s.decay)} decays for {s.r_heads} heads")
        ff = entry.get("mlp")
        if ff is not None:
            if ff["kind"] != "dense":
                raise ValueError(f"Larolorn: unknown feed-forward kind `{ff['kind']}`")
            s.mlp, s.ff, s.limit = "dense", int(ff["ff"]), float(ff["limit"])
        s.weights_of = None if entry.get("weights_of") is None else int(entry["weights_of"])
        return s

    def to_config(self) -> dict:
        a = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.mask:
            a["mask"] = {"size": self.mask}
        if self.rot.dims:
            a["rot"] = self.rot.to_config()
        if self.mixer == "latent_attention":
            m = dict(a, rot_dim=self.rot_dim, kv_rank=self.kv_rank)
        else:
            m = {"left": dict(a, kv_heads=self.kv_heads),
                 "right": {"heads": self.r_heads, "dim": self.r_dim, "vdim": self.r_vdim, "decay": list(self.decay)}}
        e = {"type": self.mixer, "mixer": m, "mlp": {"kind": "dense", "ff": self.ff, "limit": self.limit} if self.mlp else None}
        if self.weights_of is not None:
            e["weights_of"] = self.weights_of
        return e


@dataclasses.dataclass
class LarolornSpec:
    vocab: int
    width: int
    layers: list
    norm_eps: float = 1e-6
    residual_mult: float = 1.0
    logit_scale: float = 1.0

    @staticmethod
    def from_config(cfg: dict) -> "LarolornSpec":
        return LarolornSpec(vocab=int(cfg["vocab"]), width=int(cfg["width"]), layers=[LarolornLayerSpec.from_config(e) for e in cfg["layers"]],
                            norm_eps=float(cfg["norm"]["eps"]), residual_mult=float(cfg.get("residual_mult", 1.0)),
                            logit_scale=float(cfg.get("logit_scale", 1.0)))

    def to_config(self) -> dict:
        return {"architecture": "Larolorn", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "residual_mult": self.residual_mult, "logit_scale": self.logit_scale, "layers": [l.to_config() for l in self.layers]}

    def weights_layer(self, i: int) -> int:
        """The layer whose tensors layer i runs with (itself, or the end of its chain of references)."""
        seen = [i]
        while self.layers[i].weights_of is not None:
            i = self.layers[i].weights_of
            if not 0 <= i < len(self.layers) or i in seen:
                raise ValueError(f"Larolorn: layer {seen[0]} refers to weights that no layer has")
            seen.append(i)
        return i

    def tensor_shapes(self) -> dict:
        """Name -> shape of every checkpoint tensor, in file order."""
        W, out = self.width, {}
        out["embed"] = (self.vocab, W)
        for i, l in enumerate(self.layers):
            if l.weights_of is not None:
                continue
            p = f"l{i}."
            out[p + "norm1"] = (W,)
            if l.mlp:
                out[p + "norm2"] = (W,)
            H, D, V = l.heads, l.dim, l.vdim
            if l.mixer == "latent_attention":
                R, RD = l.kv_rank, l.rot_dim
                out[p + "mix.q"], out[p + "mix.dkv"], out[p + "mix.dkv.norm"] = (H * (D + RD), W), (R + RD, W), (R,)
                out[p + "mix.uk"], out[p + "mix.uv"], out[p + "mix.g"], out[p + "mix.o"] = (H * D, R), (H * V, R), (H, W), (W, H * V)
            else:
                G, RH, RD, RV = l.kv_heads, l.r_heads, l.r_dim, l.r_vdim
                q = p + "mix.left."
                for nm, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
                    out[q + nm], out[q + nm + ".b"] = (rows, W), (rows,)
                out[q + "q.norm"], out[q + "k.norm"], out[q + "sink"] = (H * D,), (G * D,), (H,)
                out[q + "o"], out[q + "o.b"] = (W, H * V), (W,)
                q = p + "mix.right."
                out[q + "q"], out[q + "k"], out[q + "v"], out[q + "g"] = (RH * RD, W), (RH * RD, W), (RH * RV, W), (RH * RV, W)
                out[q + "o"], out[q + "norm"] = (W, RH * RV), (RH * RV,)
                out[p + "mix.left.out"], out[p + "mix.right.out"] = (W,), (W,)
            if l.mlp:
                out[p + "mlp.gate"], out[p + "mlp.up"], out[p + "mlp.down"] = (l.ff, W), (l.ff, W), (W, l.ff)
        out["final.norm"] = (W,)
        out["head"] = (self.vocab, W)
        return out


def synthetic_weights(spec: LarolornSpec, seed: int = 0, device="cpu") -> dict:
    """Seeded random-init checkpoint (bf16 tensors on `device`): matrices ~ 1 / sqrt(in), gains around 1, biases and sinks of order 1."""
    g = torch.Generator(device=device).manual_seed(seed)

    def randn(shape):
        return torch.randn(shape, generator=g, device=device)
    ck = {}
    for name, shape in spec.tensor_shapes().items():
        if re.search(r"(norm[12]?|\.out)$", name):
            t = 1.0 + 0.1 * randn(shape)
        elif name.endswith(".b"):
            t = 0.5 * randn(shape)
        elif name == "embed" or name.endswith(".sink"):
            t = randn(shape)
        else:
            t = randn(shape) / math.sqrt(shape[-1])
        ck[name] = t.to(torch.bfloat16)
    return ck


class LarolornForCausalLM:
    """The executor handle: weights, paged caches, memory state slots and workspaces live in the library."""

    architecture = "Larolorn"

    def __init__(self, spec: LarolornSpec, dtype: str = "bfloat16", block_size: int = 16, num_blocks: int = 256, max_tokens: int = 2048,
                 max_seqs: int = 64, device: int = 0):
        if dtype not in ("bfloat16", "float32"):
            raise ValueError(f"Larolorn runs in bfloat16 or float32, not `{dtype}`")
        self.spec, self.dtype = spec, dtype
        self.block_size, self.num_blocks, self.max_tokens, self.max_seqs = block_size, num_blocks, max_tokens, max_seqs
        self.vocab_size = spec.vocab
        self.state_slots = max_seqs          # the engine hands one to every live sequence
        self.device = torch.device("cuda", device)
        cfg = LarolornConfig(spec.vocab, spec.width, len(spec.layers), spec.norm_eps, spec.residual_mult, spec.logit_scale,
                             VMX_F32 if dtype == "float32" else VMX_BF16, block_size, num_blocks, max_tokens, max_seqs, self.state_slots)
        layers = (LarolornLayerConfig * len(spec.layers))()
        keep = []                            # host arrays the library reads during create
        for i, l in enumerate(spec.layers):
            decay = (C.c_float * max(len(l.decay), 1))(*l.decay)
            keep.append(decay)
            src = spec.weights_layer(i)
            layers[i] = LarolornLayerConfig(MIXERS[l.mixer], l.heads, l.dim, l.vdim, l.scale, l.mask, l.rot.to_struct(), l.rot_dim, l.kv_rank, l.kv_heads,
                                            l.r_heads, l.r_dim, l.r_vdim, C.cast(decay, C.POINTER(C.c_float)) if l.decay else None, MLPS[l.mlp], l.ff,
                                            l.limit, -1 if src == i else src)
        self._h = C.c_void_p()
        check(lib.vmx_larolorn_create(C.byref(cfg), layers, C.byref(self._h)))

    @classmethod
    def from_pretrained(cls, model_dir, dtype: str = "bfloat16", **kw) -> "LarolornForCausalLM":
        cfg = json.loads((Path(model_dir) / "config.json").read_text())
        model = cls(LarolornSpec.from_config(cfg), dtype=dtype, **kw)
        model.load_checkpoint(model_dir)
        return model

    def close(self):
        if self._h:
            lib.vmx_larolorn_destroy(self._h)
            self._h = C.c_void_p()

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass

    @staticmethod
    def _stream():
        return torch.cuda.current_stream().cuda_stream

    def load_tensor(self, name: str, t) -> None:
        """t: bf16 torch tensor (host or device) or a numpy uint16 array of bf16 bit patterns."""
        if isinstance(t, np.ndarray):
            assert t.dtype == np.uint16, f"{name}: bf16 bit patterns expected"
            t = np.ascontiguousarray(t)
            check(lib.vmx_larolorn_load_tensor(self._h, name.encode(), t.ctypes.data, t.nbytes, self._stream()))
            return
        assert t.dtype == torch.bfloat16, f"{name}: bf16 expected, got {t.dtype}"
        t = t.contiguous()
        check(lib.vmx_larolorn_load_tensor(self._h, name.encode(), t.data_ptr(), t.numel() * 2, self._stream()))

    def load_state(self, tensors: dict) -> None:
        for name, t in tensors.items():
            self.load_tensor(name, t)
        self.check_loaded()

    def check_loaded(self) -> None:
        if lib.vmx_larolorn_missing_tensors(self._h) != 0:
            raise ValueError(lib.vmx_last_error().decode("utf-8", "replace"))

    def load_checkpoint(self, model_dir) -> None:
        """Every tensor of the directory's *.safetensors files under its own name (the library's safetensors reader)."""
        from .checkpoint import CheckpointDir
        ck = CheckpointDir(model_dir)
        try:
            for name in ck.where:
                f = ck._file(ck.where[name])
                dtype = f.info(lib.vmx_safetensors_find(f._h, name.encode()))[1]
                if dtype != "BF16":
                    raise ValueError(f"{model_dir}: tensor `{name}` is {dtype}; Larolorn checkpoints hold bf16")
                m = re.fullmatch(r"l(\d+)\.norm2", name)
                if m and int(m.group(1)) < len(self.spec.layers) and self.spec.layers[int(m.group(1))].mlp is None:
                    continue                 # norm of a feed-forward this layer does not have
                self.load_tensor(name, ck.get(name))
        finally:
            ck.close()
        self.check_loaded()

    def forward(self, tokens, prev_tokens, positions, slots, seq_ids, block_tables, logit_rows=None, want_logits: bool = True,
                want_greedy: bool = False, layer_trace: bool = False, seq_starts=None, state_slots=None):
        """One packed step; every argument an int32 CUDA tensor ([T] each, block_tables [S, max_blocks], seq_starts [S + 1],
        state_slots [S], logit_rows [n]); prev_tokens is not used by this design.
        Returns (logits f32 [n, vocab] or None, greedy ids int32 [n] or None, trace f32 [layers, T, width] or None)."""
        if seq_starts is None or state_slots is None:
            raise ValueError("Larolorn carries recurrent state: the step needs seq_starts and state_slots")
        T = tokens.numel()
        S = seq_starts.numel() - 1           # the sequences of THIS step; the block table may hold more rows
        if S < 1 or state_slots.numel() != S or block_tables.shape[0] < S:
            raise ValueError(f"Larolorn: {S} sequences by seq_starts, {state_slots.numel()} state slots, {block_tables.shape[0]} block-table rows")
        if not all(a.numel() == T for a in (positions, slots, seq_ids)):
            raise ValueError("Larolorn: tokens, positions, slots and seq_ids must have one entry per token")
        n = 0 if logit_rows is None else logit_rows.numel()
        logits = torch.empty((n, self.spec.vocab), dtype=torch.float32, device=self.device) if n else None
        ids = torch.empty(n, dtype=torch.int32, device=self.device) if (n and want_greedy) else None
        trace = torch.empty((len(self.spec.layers), T, self.spec.width), dtype=torch.float32, device=self.device) if layer_trace else None
        check(lib.vmx_larolorn_forward(self._h, tokens.data_ptr(), positions.data_ptr(), slots.data_ptr(), seq_ids.data_ptr(), T,
                                       block_tables.data_ptr(), S, block_tables.shape[1], seq_starts.data_ptr(),
                                       state_slots.data_ptr(), None if not n else logit_rows.data_ptr(), n,
                                       None if logits is None else logits.data_ptr(), None if ids is None else ids.data_ptr(),
                                       None if trace is None else trace.data_ptr(), self._stream()))
        return (logits if want_logits else None), ids, trace
