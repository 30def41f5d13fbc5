"""What layered model families share: a stack of layers whose mixers own their share of the paged cache and
of the state slots, an fp32 residual stream, weights from safetensors.

A layer has ``mixer`` (``mixers.py``, ``latent.py``, ``mlstm.py``, ``masked.py``: ``bind``, ``unbind``, ``kv_elements_per_token``,
``state_bytes_per_slot``); a family implements ``load_tensors`` and ``forward_layers``.
"""
from __future__ import annotations

import torch
from torch import nn

from .loader import TensorFolder


def load_rows(param: torch.Tensor, first: int, parts) -> None:
    """Copies tensors into consecutive rows of a fused weight, from row ``first`` on."""
    for t in parts:
        param[first: first + t.shape[0]].copy_(t)
        first += t.shape[0]


class LayeredModel(nn.Module):

    def __init__(self, cfg, tied: bool = False):
        super().__init__()
        # 32-bit accumulation in the library's matrix products, and full fp32 ones
        torch.backends.cuda.matmul.allow_bf16_reduced_precision_reduction = False
        torch.backends.cuda.matmul.allow_tf32 = False
        self.cfg = cfg
        self.embed = nn.Parameter(torch.empty(cfg.vocab_size, cfg.hidden_size))
        self.head = self.embed if tied else nn.Parameter(torch.empty(cfg.vocab_size, cfg.hidden_size))
        self.layers: list = []

    def random_weights(self, device, seed: int) -> None:
        gen = torch.Generator(device=device).manual_seed(seed)
        with torch.no_grad():
            for p in self.parameters():
                if p.dim() >= 2:
                    p.normal_(0.0, 0.02 if p.shape[-2] > 8 else 0.5, generator=gen)

    @torch.no_grad()
    def load_weights(self, folder: str) -> None:
        tensors = TensorFolder(folder)
        self.embed.copy_(tensors.take("embed", self.embed.shape))
        if self.head is not self.embed:
            self.head.copy_(tensors.take("head", self.head.shape))
        self.load_tensors(tensors.take)
        if tensors.unused():
            raise ValueError(f"tensors without a place in the model: {', '.join(tensors.unused()[:5])}")

    def load_tensors(self, take) -> None:
        raise NotImplementedError

    # ---- cache and state ---------------------------------------------------------------------------
    def kv_bytes_per_token(self) -> int:
        return self.embed.element_size() * sum(l.mixer.kv_elements_per_token() for l in self.layers)

    def state_bytes_per_slot(self) -> int:
        return sum(l.mixer.state_bytes_per_slot(self.embed.element_size()) for l in self.layers)

    def bind_cache(self, num_blocks: int, block: int, slots: int) -> None:
        for l in self.layers:
            l.mixer.bind(num_blocks, block, slots, self.embed.dtype, self.embed.device)

    def unbind_cache(self) -> None:
        for l in self.layers:
            l.mixer.unbind()

    # ---- forward -------------------------------------------------------------------------------------
    def forward_layers(self, input_ids, positions, hidden, residual, first: int, last: int):
        """Layers ``[first, last)``: ``hidden`` is the normed input of the next layer (whatever form the family
        gives it), ``residual`` the fp32 stream, updated in place.  After the last layer ``hidden`` is the final
        norm -- of the rows in the Context's ``logit_rows`` only, when they are given.  (Positions follow from
        the row groups.)"""
        raise NotImplementedError

    def finish(self, hidden, residual) -> torch.Tensor:
        return hidden

    def forward(self, input_ids, positions) -> torch.Tensor:
        return self.forward_layers(input_ids, positions, None, None, 0, len(self.layers))[0]
