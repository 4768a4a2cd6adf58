"""Lurepel: a decoder whose layers mix tokens by grouped softmax attention within chunks of positions: the values are the
keys as projected, queries and keys are turned in neighbouring pairs (slow pairs slowed down by wavelength) and brought to
unit root mean square without a weight, every softmax sum holds one more term of score 0, every head's output is multiplied by
one sigmoid gate; dense feed-forwards with a tanh-form GELU gate, or routed experts chosen by corrected softmax scores, some of
which hand their input through, or none; RMSNorms on the embedding's output, on what every sublayer gives (the residual itself
is never normed within a layer) and ahead of the head.

Tensor names and shapes (D width, V vocab, per layer N):
  embed [V, D]; embed.norm [D]; final.norm [D]; head [V, D]
  lN.norm1 [D], and lN.norm2 where the layer has a feed-forward
  attention:  lN.mix.q [heads * dim, D], .k [kv_heads * dim, D], .g [heads, D], .o [D, heads * dim]
  dense:      lN.mlp.gate / .up [ff, D], .down [D, ff]
  experts:    lN.mlp.router [experts + identity, D], .correction [experts + identity], lN.mlp.eK.gate / .up [ff, D], .down [D, ff]
"""

from __future__ import annotations

from ..config.lurepel import LurepelConfig
from ..parts.embedding import NormedEmbedding
from ..registry import register_architecture
from .decoder import build_decoder


def build_lurepel(config: LurepelConfig):
    return build_decoder(
        config, position_encoding="none", layer_prefix="l{}.", final_norm_name="final.norm", head_name="head",
        make_embedding=lambda c: NormedEmbedding(c.vocab, c.hidden, "embed", c.rms_eps, "embed.norm"))


register_architecture("Lurepel", LurepelConfig, build_lurepel)
