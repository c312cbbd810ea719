"""Token embedding and output head.

Embedding gather into the float32 residual stream (models/src/llama.rs:470, 481).  The head is a bias-free product
with the embedding matrix when tied, else with its own [vocab, width] matrix (models/src/llama.rs:476-477,
482-486); logits leave in float32 straight from the float32 accumulators.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..kernels import ops
from .base import Part, WeightSpec
from .linear import linear


class TokenEmbedding(Part):
    def __init__(self, vocab_size: int, width: int, name: str = "weight", scale: float = 1.0,
                 sinusoid_base: Optional[float] = None):
        # ``scale`` multiplies the rows on their way into the stream; a head tied to the table reads it without
        # ``sinusoid_base`` b: a vector of the token's position p is added to its row, sin(p b^(-2i / width)) in column
        # 2i and the cosine of the same in column 2i + 1
        self.sinusoid_base = None if sinusoid_base is None else float(sinusoid_base)
        self.reads_positions = self.sinusoid_base is not None
        self.freq: Optional[torch.Tensor] = None
        self.vocab_size, self.width, self.name, self.scale = int(vocab_size), int(width), str(name), float(scale)
        self.weight: Optional[torch.Tensor] = None

    def graph_safe(self) -> bool:
        return True

    def weight_specs(self) -> Dict[str, WeightSpec]:
        return {self.name: WeightSpec((self.vocab_size, self.width), "embedding")}

    def load(self, get, device, act_dtype) -> None:
        self.weight = get(self.name).to(device).contiguous()
        if self.reads_positions:
            i = torch.arange((self.width + 1) // 2, dtype=torch.float64)
            self.freq = torch.pow(torch.tensor(self.sinusoid_base, dtype=torch.float64), -2.0 * i / self.width).to(device)

    def device_bytes(self) -> int:
        return 0  # a step reads only the rows of its tokens

    def forward(self, tokens: torch.Tensor, norm=None, out=None, positions=None):
        """The float32 residual rows of ``tokens`` (into ``out`` where given); with ``norm`` (the norm that reads them
        first) a pair (rows, that norm begun or None).  ``positions`` [T] is given where ``reads_positions`` says so."""
        if self.reads_positions:
            rows = ops.embed_sinusoid(tokens, self.weight, positions, self.freq, self.scale, out)
            return rows if norm is None else (rows, None)
        if norm is None:
            return ops.embed(tokens, self.weight, out, self.scale)
        # (a norm that cannot begin scaled rows is not asked to)
        got = norm.embed(self.weight, tokens) if self.scale == 1.0 else \
            norm.embed_scaled(self.weight, tokens, self.scale)
        return got if got is not None else (ops.embed(tokens, self.weight, scale=self.scale), None)


class OutputHead(Part):
    def __init__(self, width: int, vocab_size: int, tied_to: Optional[TokenEmbedding] = None, name: str = "weight"):
        self.width, self.vocab_size, self.tied_to, self.name = int(width), int(vocab_size), tied_to, str(name)
        self.weight: Optional[torch.Tensor] = None
        self.tiled = None

    def graph_safe(self) -> bool:
        return True

    def weight_specs(self) -> Dict[str, WeightSpec]:
        return {} if self.tied_to is not None else {self.name: WeightSpec((self.vocab_size, self.width))}

    def load(self, get, device, act_dtype) -> None:
        self.weight = self.tied_to.weight if self.tied_to is not None else get(self.name).to(device).contiguous()
        # a second copy in the order the streaming kernel's waves read it, for steps of few rows (the row-major one
        # serves the embedding's gather and the products of many rows)
        self.tiled = None
        if act_dtype is torch.bfloat16 and self.weight.dtype is torch.bfloat16 and self.weight.is_cuda:
            from ..kernels import gemm_bf16
            plan = gemm_bf16.tiled_plan(self.vocab_size, self.width, swiglu=False)
            if plan is not None:
                self.tiled = gemm_bf16.tile_weight(self.weight, *plan)

    def device_bytes(self) -> int:
        return self.weight.numel() * self.weight.element_size()

    def forward(self, x) -> torch.Tensor:
        return linear(x, self.weight, torch.float32, tiled=self.tiled)
