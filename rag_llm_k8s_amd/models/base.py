"""What the serving engine asks of a decoder model beyond forward(): work lists, workspaces, state slots."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch

from ..ops.backend import AttnMeta


@dataclass
class StepInput:
    ids: torch.Tensor  # int32 [T]
    positions: torch.Tensor  # int32 [T]
    slots: torch.Tensor  # int32 [T]
    meta: AttnMeta
    logits_idx: Optional[torch.Tensor] = None  # int32 [n] rows that need logits (None = all)
    # asynchronous decode: carry[i] >= 0 -> ids[i] = carry_src[carry[i]] (previous step's sampled token,
    # resolved on the device by the embedding kernel)
    carry: Optional[torch.Tensor] = None
    carry_src: Optional[torch.Tensor] = None


class DecoderModel:
    """Defaults: one attention geometry (Hq, Hkv, D) for every layer, no recurrent state."""

    recurrent = False  # True: every live sequence owns a state slot (allocate_state)

    def prefill_work(self, q_lens, device):
        """(tiles, qtiles) device work lists of a prefill step."""
        from ..ops.native import build_prefill_tiles

        return build_prefill_tiles(q_lens, self.Hq, self.Hkv).to(device), {}

    def decode_work(self, max_kv_len, batch):
        """(part_tiles, max_parts, ws_o, ws_ml) of a decode step of `batch` rows (split-K attention)."""
        from ..ops.native import decode_partitions

        pt, mp = decode_partitions(max_kv_len, batch, self.Hkv)
        if mp == 1:
            return pt, mp, None, None
        f32 = dict(dtype=torch.float32, device=self.device)
        return (pt, mp, torch.empty((batch, self.Hq, mp, self.D), **f32),
                torch.empty((batch, self.Hq, mp, 2), **f32))

    def key_rows(self, q_lens, kv_lens, device):
        """Packed key rows of a prefill step by window (models that expand cached latents)."""
        return {}

    def state_bytes_per_slot(self):
        return 0

    def allocate_state(self, num_slots):
        return None
