"""Models whose weights are stored padded with zeros, so that every product meets the tile
kernels' alignment whatever the sizes: the width, feature counts and head sizes are rounded up
at load time, which leaves every product unchanged; norms divide by the true sizes.

What such models share: checkpoint reading, the padded layouts, and the stream step around
every sublayer. A subclass gives ``_layer`` (one layer's tensors), ``init_random`` and the
layers' forward pass.
"""
from __future__ import annotations

import math
import os

import torch

from operator_amd import ops
from operator_amd.ops import decoder as dec
from operator_amd.parallel.comm import Group

from .base import DecoderModel, ForwardBatch


class PaddedModel(DecoderModel):
    LAYOUT_FUNCS = ("load_checkpoint", "_build", "_gate_up", "_down", "_put", "_padded")

    def __init__(self, cfg, device: str | torch.device = "cuda", tp: Group | None = None,
                 dtype: torch.dtype = torch.bfloat16, weight_dtype: str = "bfloat16"):
        self.tp = tp or Group.single()
        if self.tp.world != 1:
            raise ValueError(f"{cfg.arch} models run on one GPU (tensor parallel degree 1)")
        if weight_dtype != "bfloat16":
            raise ValueError(f"{cfg.arch} weights are stored in the compute dtype, not {weight_dtype!r}")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"{cfg.arch} computes in bfloat16 or float32, not {dtype}")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.ld = max(128, dec.pad_to(cfg.hidden, 64))
        self.gu_block = ops.GU_BLOCK
        self.layers: list = []
        self.embed = self.final_norm = self.lm_head = None

    def prefill_plan(self) -> tuple[int, int]:
        return dec.GD_VARIANT, dec.GD_BLOCK_Q

    # ------------------------------------------------------------------ weights
    def _padded(self, w: torch.Tensor, n: int) -> torch.Tensor:
        """fp32 vector ``w`` followed by zeros up to ``n``."""
        t = torch.zeros(n, device=self.device)
        t[:w.numel()] = w.float()
        return t

    def _put(self, rows: int, cols: int, parts, dtype=None) -> torch.Tensor:
        """Zero [rows, cols] with each (row, col, tensor) of ``parts`` placed in it."""
        t = torch.zeros(rows, cols, dtype=dtype or self.dtype, device=self.device)
        for r, c, p in parts:
            t[r:r + p.shape[0], c:c + p.shape[1]] = p
        return t

    def _gate_up(self, gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
        n = max(128, dec.pad_to(gate.shape[0], 64))
        return ops.interleave_gate_up(self._put(n, self.ld, [(0, 0, gate)]), self._put(n, self.ld, [(0, 0, up)]))

    def _down(self, w: torch.Tensor) -> torch.Tensor:
        return self._put(self.ld, max(128, dec.pad_to(w.shape[1], 64)), [(0, 0, w)])

    def _layer(self, i: int, get, has):
        raise NotImplementedError

    def _build(self, get, has) -> "PaddedModel":
        """Packed, padded weights from ``get(name, shape)`` (checkpoint tensor names)."""
        c, V = self.cfg, self.cfg.vocab_size
        self.embed = self._put(V, self.ld, [(0, 0, get("embed", (V, c.hidden)))])
        self.layers = [self._layer(i, get, has) for i in range(c.layers)]
        self.final_norm = self._padded(get("final.norm", (c.hidden,)).float(), self.ld)
        self.lm_head = self._put(dec.pad_to(V, 64), self.ld, [(0, 0, get("head", (V, c.hidden)))])
        if self.device.type == "cuda":
            torch.cuda.synchronize(self.device)
        return self

    def load_checkpoint(self, path: str) -> "PaddedModel":
        """Weights of a checkpoint directory (safetensors), checked against ``cfg``'s shapes."""
        from safetensors import safe_open

        names: dict = {}
        for f in sorted(f for f in os.listdir(path) if f.endswith(".safetensors")):
            sf = safe_open(os.path.join(path, f), framework="pt", device="cpu")
            names.update({k: sf for k in sf.keys()})
        if not names:
            raise FileNotFoundError(f"no *.safetensors in {path}")

        def get(name, shape):
            t = names[name].get_tensor(name)
            if t.numel() != math.prod(shape) or (t.dim() > 1 and tuple(t.shape) != tuple(shape)):
                raise ValueError(f"{path}: {name} is {tuple(t.shape)}, {tuple(shape)} expected")
            return t.reshape(shape).to(self.device, self.dtype)

        return self._build(get, lambda name: name in names)

    # ------------------------------------------------------------------ forward
    def _step(self, x, y: dec.SublayerOut, hc: dec.Stream, after: tuple | None, fb: ForwardBatch,
              post_w: torch.Tensor | None = None) -> torch.Tensor:
        """Finish a sublayer; ``after`` = (stream coefficients, norm weight) of the next one, None
        at the end of the model (only the rows whose logits are wanted, streams left as they are).
        ``post_w``: weight of the norm of the sublayer's output."""
        c = self.cfg
        if after is not None:
            return dec.stream_step(x, y, hc, after[0], after[1], c.hidden, c.rms_eps, self.dtype, post_w=post_w)
        if fb.residual_sink is None:
            return dec.stream_step(x, y, hc, None, self.final_norm, c.hidden, c.rms_eps, self.dtype,
                                   rows=fb.logits_index, write_x=False, post_w=post_w)
        h = dec.stream_step(x, y, hc, None, self.final_norm, c.hidden, c.rms_eps, self.dtype, post_w=post_w)
        return h if fb.logits_index is None else h.index_select(0, fb.logits_index)
