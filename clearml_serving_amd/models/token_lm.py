"""Base of the language models that run on flat token batches
(engines/llm/token_batch.py): weights by checkpoint name, and what the engine
asks of such a model."""

from typing import Any, Dict, Iterator, List, Optional, Tuple

import torch
import torch.nn as nn

from .mixers import GroupedAttention, LatentAttention, RgLru, _fill

# checkpoint name -> (padded operand, true shape, shape to fill it in)
Held = Dict[str, Tuple[torch.Tensor, tuple, Optional[tuple]]]


def held(dst: torch.Tensor, *shape: int, fill_as: Optional[tuple] = None):
    return dst, shape, fill_as


class TokenBatchLayer(nn.Module):
    """``mix``: the mixer; ``mlp``: the feed-forward or None."""

    def held(self) -> Held:
        """the layer's own tensors (norms)"""
        raise NotImplementedError

    def parts(self) -> Iterator[Tuple[str, nn.Module]]:
        """(prefix, module) of what a checkpoint holds for the sublayers"""
        yield "mix.", self.mix
        if self.mlp is not None:
            yield "mlp.", self.mlp


class TokenBatchForCausalLM(nn.Module):
    # one forward for prompt portions and single tokens together
    token_batch = True
    supports_float32 = True
    tp_size = 1
    layers: nn.ModuleList  # of TokenBatchLayer

    def held(self) -> Held:
        """tensors outside the layers"""
        raise NotImplementedError

    def ignored(self) -> List[str]:
        """names that a checkpoint may hold and nothing uses"""
        return []

    def random_tensor(self, name: str, shape: tuple,
                      gen: torch.Generator) -> torch.Tensor:
        raise NotImplementedError

    # ---- weights ---------------------------------------------------- #
    def _all_held(self) -> Held:
        out = dict(self.held())
        for i, layer in enumerate(self.layers):
            out.update({"l{}.{}".format(i, k): v
                        for k, v in layer.held().items()})
        return out

    def checkpoint_shapes(self) -> Dict[str, tuple]:
        out = {k: shape for k, (_, shape, _) in self._all_held().items()}
        for i, layer in enumerate(self.layers):
            for q, mod in layer.parts():
                for k, s in mod.shapes().items():
                    out["l{}.{}{}".format(i, q, k)] = tuple(s)
        return out

    def _fit(self, state: Dict[str, torch.Tensor]) -> None:
        """sizes that are not in the configuration"""
        for i, layer in enumerate(self.layers):
            for q, mod in layer.parts():
                if hasattr(mod, "fit"):
                    try:
                        mod.fit(lambda name, q="l{}.{}".format(i, q):
                                state[q + name])
                    except KeyError:
                        pass  # reported as missing below

    def load_checkpoint(self, state: Dict[str, torch.Tensor]) -> None:
        self._fit(state)
        want = self.checkpoint_shapes()
        missing = sorted(set(want) - set(state))
        extra = sorted(set(state) - set(want) - set(self.ignored()))
        if missing or extra:
            raise ValueError("checkpoint does not fit the configuration: "
                             "missing {}, unexpected {}".format(
                                 missing[:8], extra[:8]))
        for k, s in want.items():
            if tuple(state[k].shape) != tuple(s):
                raise ValueError("checkpoint tensor '{}' is {}, expected {}"
                                 .format(k, tuple(state[k].shape), s))
        for k, (dst, _, fill_as) in self._all_held().items():
            src = state[k]
            _fill(dst.data, src if fill_as is None else src.reshape(fill_as))
        for i, layer in enumerate(self.layers):
            for q, mod in layer.parts():
                mod.pack(lambda name, q="l{}.{}".format(i, q):
                         state[q + name])

    def init_random(self, seed: int = 1234) -> None:
        """seeded weights, scaled like a fresh model's"""
        gen = torch.Generator().manual_seed(seed)
        self.load_checkpoint({
            name: self.random_tensor(name, shape, gen).to(torch.bfloat16)
            for name, shape in self.checkpoint_shapes().items()})

    def finalize(self) -> None:
        """call once weights, device and type are settled"""
        for layer in self.layers:
            for _, mod in layer.parts():
                if hasattr(mod, "finalize"):
                    mod.finalize()

    # ---- what the engine needs to know ------------------------------ #
    def cache_layout(self) -> List[tuple]:
        """per layer run, in order: ("paged", elements per token[, tokens per
        pooled row]), ("state",
        shape of a slot's float state[, channels and taps of a ring of past
        inputs]), ("both", layout, layout) or ("shared", run)"""
        raise NotImplementedError

    def batch_params(self, dtype: torch.dtype) -> Dict[str, Any]:
        """how a TokenBatch for this model is to be cut"""
        attn = [a for m in self.layers for a in m.mix.modules()
                if isinstance(a, (LatentAttention, GroupedAttention))]
        rec = [m.mix for m in self.layers if isinstance(m.mix, RgLru)]
        # the recurrence holds two tiles of one block's channels in LDS
        wide = max([m.bp for m in rec], default=32)
        tile = 64 if 128 * (wide + 8) * dtype.itemsize <= 160 * 1024 else 16
        # few queries per sequence: absorbed attention; prompts: rebuilt keys
        expand = (dtype == torch.bfloat16
                  and all(m.can_expand() for m in attn))
        return {"tile": tile, "absorb_max": 8 if expand else None,
                "windows": sorted({m.view for m in attn}, key=str)}
