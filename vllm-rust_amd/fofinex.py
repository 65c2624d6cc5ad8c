"""Host-side driver of the Fofinex decoder family (libvmx `vmx_fofinex_*`).

A Fofinex model is a stack of layers listed in its config.json whose sublayers sit between two layer norms, `x <- x + N1b(mixer(
N1(x))); x <- x + N2b(ff(N2(x)))`; the embedding is normed once more and doubles as the output matrix.  Mixers: "latent_attention"
(low-rank queries, compressed keys / values in a paged cache, one rotated key part for all heads with stretched rotation
frequencies; a layer may attend over an earlier layer's cache) and "mlstm" (a matrix memory with exponential input gate, forget
gate, normaliser and running maximum in a state slot per sequence).  Feed-forwards: "dense" (biased, tanh-GELU gate) and "moe"
(experts chosen by corrected sigmoid scores inside the best groups, squared ReLU, a gated shared expert).  This file reads the
configuration, hands the checkpoint's tensors to the library under their file names and wraps the one forward entry point.  All
arithmetic happens in the library.
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

from ._lib import FofinexConfig, FofinexLayerConfig, check, lib
from .rotation import RotationSpec

VMX_F32, VMX_BF16 = 0, 1
MIXERS = {"latent_attention": 0, "mlstm": 8}
MLPS = {None: 0, "dense": 6, "moe": 7}


@dataclasses.dataclass
class FofinexLayerSpec:
    mixer: str = "latent_attention"
    heads: int = 4
    dim: int = 32                # latent attention: unrotated query / key coordinates; mlstm: key size
    vdim: int = 32
    # latent attention
    rot_dim: int = 16
    kv_rank: int = 64
    q_rank: int = 48
    scale: float = 0.125
    rot: RotationSpec = dataclasses.field(default_factory=RotationSpec)
    kv_from: int | None = None   # the earlier layer whose latents it attends over (None: its own)
    # mlstm
    gate_cap: float = 15.0
    mlp: str | None = "dense"
    ff: int = 64                 # dense
    experts: int = 4             # moe
    top: int = 1
    groups: int = 1
    keep_groups: int = 1
    expert_ff: int = 32
    shared_ff: int = 0           # 0: no shared expert
    router_scale: float = 1.0

    @staticmethod
    def from_config(entry: dict) -> "FofinexLayerSpec":
        kind, m = entry["type"], entry["mixer"]
        if kind not in MIXERS:
            raise ValueError(f"Fofinex: unknown layer type `{kind}`")
        s = FofinexLayerSpec(mixer=kind, heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m.get("vdim", m["dim"])), mlp=None)
        if kind == "latent_attention":
            s.rot_dim, s.kv_rank, s.q_rank = int(m["rot_dim"]), int(m["kv_rank"]), int(m["q_rank"])
            s.scale = float(m.get("scale", 1.0 / math.sqrt(s.dim + s.rot_dim)))
            s.rot = RotationSpec.from_config(m.get("rot"))
            s.kv_from = None if m.get("kv_from") is None else int(m["kv_from"])
        else:
            s.gate_cap = float(m["gate_cap"])
        ff = entry.get("mlp")
        if ff is None:
            return s
        s.mlp = ff["kind"]
        if s.mlp == "dense":
            s.ff = int(ff["ff"])
        elif s.mlp == "moe":
            r = ff["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            s.experts, s.top, s.groups, s.keep_groups = int(r["experts"]), int(r["top"]), int(g["count"]), int(g["keep"])
            s.router_scale = float(r.get("scale", 1.0))
            s.expert_ff = int(ff["expert"]["ff"])
            s.shared_ff = int((ff.get("shared") or {}).get("ff") or 0)
        else:
            raise ValueError(f"Fofinex: unknown feed-forward kind `{s.mlp}`")
        return s

    def to_config(self) -> dict:
        m = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim}
        if self.mixer == "latent_attention":
            m.update(rot_dim=self.rot_dim, kv_rank=self.kv_rank, q_rank=self.q_rank, scale=self.scale)
            if self.rot.dims:
                m["rot"] = self.rot.to_config()
            if self.kv_from is not None:
                m["kv_from"] = self.kv_from
        else:
            m["gate_cap"] = self.gate_cap
        ff = None
        if self.mlp == "dense":
            ff = {"kind": "dense", "ff": self.ff}
        elif self.mlp == "moe":
            ff = {"kind": "moe", "expert": {"ff": self.expert_ff},
                  "router": {"experts": self.experts, "top": self.top, "groups": {"count": self.groups, "keep": self.keep_groups}, "scale": self.router_scale}}
            if self.shared_ff:
                ff["shared"] = {"ff": self.shared_ff}
        return {"type": self.mixer, "mixer": m, "mlp": ff}


@dataclasses.dataclass
class FofinexSpec:
    vocab: int
    width: int
    layers: list
    norm_eps: float = 1e-6

    @staticmethod
    def from_config(cfg: dict) -> "FofinexSpec":
        return FofinexSpec(vocab=int(cfg["vocab"]), width=int(cfg["width"]), layers=[FofinexLayerSpec.from_config(e) for e in cfg["layers"]],
                           norm_eps=float(cfg["norm"]["eps"]))

    def to_config(self) -> dict:
        return {"architecture": "Fofinex", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "layers": [l.to_config() for l in self.layers]}

    def tensor_shapes(self) -> dict:
        """Name -> shape of every checkpoint tensor, in file order."""
        W, out = self.width, {}
        out["embed"], out["embed.norm"] = (self.vocab, W), (W,)
        for i, l in enumerate(self.layers):
            p = f"l{i}."
            for nm in ("norm1", "norm2", "norm1b", "norm2b") if l.mlp else ("norm1", "norm1b"):
                out[p + nm] = (W,)
            H, D, V = l.heads, l.dim, l.vdim
            if l.mixer == "latent_attention":
                R, RD, Q = l.kv_rank, l.rot_dim, l.q_rank
                out[p + "mix.dq"], out[p + "mix.dq.norm"], out[p + "mix.uq"] = (Q, W), (Q,), (H * (D + RD), Q)
                if l.kv_from is None:
                    out[p + "mix.dkv"], out[p + "mix.dkv.norm"] = (R + RD, W), (R,)
                out[p + "mix.uk"], out[p + "mix.uv"], out[p + "mix.o"] = (H * D, R), (H * V, R), (W, H * V)
            else:
                out[p + "mix.q"], out[p + "mix.k"], out[p + "mix.v"] = (H * D, W), (H * D, W), (H * V, W)
                out[p + "mix.g"], out[p + "mix.o"], out[p + "mix.norm"] = (H * V, W), (W, H * V), (H * V,)
                out[p + "mix.i"], out[p + "mix.i.b"], out[p + "mix.f"], out[p + "mix.f.b"] = (H, W), (H,), (H, W), (H,)
            if l.mlp == "dense":
                out[p + "mlp.gate"], out[p + "mlp.gate.b"] = (l.ff, W), (l.ff,)
                out[p + "mlp.up"], out[p + "mlp.up.b"] = (l.ff, W), (l.ff,)
                out[p + "mlp.down"], out[p + "mlp.down.b"] = (W, l.ff), (W,)
            elif l.mlp == "moe":
                for e in range(l.experts):
                    out[p + f"mlp.e{e}.up"], out[p + f"mlp.e{e}.down"] = (l.expert_ff, W), (W, l.expert_ff)
                out[p + "mlp.router"], out[p + "mlp.correction"] = (l.experts, W), (l.experts,)
                if l.shared_ff:
                    out[p + "mlp.shared.up"], out[p + "mlp.shared.down"], out[p + "mlp.shared.sg"] = (l.shared_ff, W), (W, l.shared_ff), (1, W)
        out["final.norm"] = (W,)
        return out


def synthetic_weights(spec: FofinexSpec, seed: int = 0, device="cpu") -> dict:
    """Seeded random-init checkpoint (bf16 tensors on `device`): matrices ~ 1 / sqrt(in), gains around 1, biases of order 1,
    forget gates that keep the memories' time scales between a few and a few hundred tokens, corrections of both signs."""
    g = torch.Generator(device=device).manual_seed(seed)

    def randn(shape):
        return torch.randn(shape, generator=g, device=device)
    ck = {}
    for name, shape in spec.tensor_shapes().items():
        if re.search(r"norm[12]?b?$", name):
            t = 1.0 + 0.1 * randn(shape)
        elif name.endswith("mix.f.b"):
            t = 3.0 + 1.5 * randn(shape)
        elif name.endswith(".b"):
            t = 0.5 * randn(shape)
        elif name.endswith("correction"):
            t = 0.3 * randn(shape) - 0.3
        elif name == "embed":
            t = randn(shape)
        else:
            t = randn(shape) / math.sqrt(shape[-1])
        ck[name] = t.to(torch.bfloat16)
    return ck


class FofinexForCausalLM:
    """The executor handle: weights, paged latent caches, memory state slots and workspaces live in the library."""

    architecture = "Fofinex"

    def __init__(self, spec: FofinexSpec, dtype: str = "bfloat16", block_size: int = 16, num_blocks: int = 256, max_tokens: int = 2048,
                 max_seqs: int = 64, device: int = 0):
        if dtype not in ("bfloat16", "float32"):
            raise ValueError(f"Fofinex runs in bfloat16 or float32, not `{dtype}`")
        self.spec, self.dtype = spec, dtype
        self.block_size, self.num_blocks, self.max_tokens, self.max_seqs = block_size, num_blocks, max_tokens, max_seqs
        self.vocab_size = spec.vocab
        self.state_slots = max_seqs          # the engine hands one to every live sequence
        self.device = torch.device("cuda", device)
        cfg = FofinexConfig(spec.vocab, spec.width, len(spec.layers), spec.norm_eps, VMX_F32 if dtype == "float32" else VMX_BF16, block_size, num_blocks,
                            max_tokens, max_seqs, self.state_slots)
        layers = (FofinexLayerConfig * len(spec.layers))()
        for i, l in enumerate(spec.layers):
            layers[i] = FofinexLayerConfig(MIXERS[l.mixer], l.heads, l.dim, l.vdim, l.rot_dim, l.kv_rank, l.q_rank, l.scale, l.rot.to_struct(),
                                           -1 if l.kv_from is None else l.kv_from, l.gate_cap, MLPS[l.mlp], l.ff, l.experts, l.top, l.groups,
                                           l.keep_groups, l.expert_ff, l.shared_ff, l.router_scale)
        self._h = C.c_void_p()
        check(lib.vmx_fofinex_create(C.byref(cfg), layers, C.byref(self._h)))

    @classmethod
    def from_pretrained(cls, model_dir, dtype: str = "bfloat16", **kw) -> "FofinexForCausalLM":
        cfg = json.loads((Path(model_dir) / "config.json").read_text())
        model = cls(FofinexSpec.from_config(cfg), dtype=dtype, **kw)
        model.load_checkpoint(model_dir)
        return model

    def close(self):
        if self._h:
            lib.vmx_fofinex_destroy(self._h)
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
            check(lib.vmx_fofinex_load_tensor(self._h, name.encode(), t.ctypes.data, t.nbytes, self._stream()))
            return
        assert t.dtype == torch.bfloat16, f"{name}: bf16 expected, got {t.dtype}"
        t = t.contiguous()
        check(lib.vmx_fofinex_load_tensor(self._h, name.encode(), t.data_ptr(), t.numel() * 2, self._stream()))

    def load_state(self, tensors: dict) -> None:
        for name, t in tensors.items():
            self.load_tensor(name, t)
        self.check_loaded()

    def check_loaded(self) -> None:
        if lib.vmx_fofinex_missing_tensors(self._h) != 0:
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
                    raise ValueError(f"{model_dir}: tensor `{name}` is {dtype}; Fofinex checkpoints hold bf16")
                m = re.fullmatch(r"l(\d+)\.norm2b?", name)
                if m and int(m.group(1)) < len(self.spec.layers) and self.spec.layers[int(m.group(1))].mlp is None:
                    continue                 # norms of a feed-forward this layer does not have
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
            raise ValueError("Fofinex carries recurrent state: the step needs seq_starts and state_slots")
        T = tokens.numel()
        S = seq_starts.numel() - 1           # the sequences of THIS step; the block table may hold more rows
        if S < 1 or state_slots.numel() != S or block_tables.shape[0] < S:
            raise ValueError(f"Fofinex: {S} sequences by seq_starts, {state_slots.numel()} state slots, {block_tables.shape[0]} block-table rows")
        if not all(a.numel() == T for a in (positions, slots, seq_ids)):
            raise ValueError("Fofinex: tokens, positions, slots and seq_ids must have one entry per token")
        n = 0 if logit_rows is None else logit_rows.numel()
        logits = torch.empty((n, self.spec.vocab), dtype=torch.float32, device=self.device) if n else None
        ids = torch.empty(n, dtype=torch.int32, device=self.device) if (n and want_greedy) else None
        trace = torch.empty((len(self.spec.layers), T, self.spec.width), dtype=torch.float32, device=self.device) if layer_trace else None
        check(lib.vmx_fofinex_forward(self._h, tokens.data_ptr(), positions.data_ptr(), slots.data_ptr(), seq_ids.data_ptr(), T,
                                      block_tables.data_ptr(), S, block_tables.shape[1], seq_starts.data_ptr(),
                                      state_slots.data_ptr(), None if not n else logit_rows.data_ptr(), n,
                                      None if logits is None else logits.data_ptr(), None if ids is None else ids.data_ptr(),
                                      None if trace is None else trace.data_ptr(), self._stream()))
        return (logits if want_logits else None), ids, trace
