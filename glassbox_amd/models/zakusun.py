"""The Zakusun decoder assembled from parts.

Every sublayer reads the grouped RMS norm of the residual plus a convolution of it over time (``ConvNormBlock`` of
``ConvolvedNorm``s); the mixer is attention through a latent, which is all that a position leaves in the cache
(``LatentCacheAttention``, with a sink a head and a gate a channel); the feed-forward is ``RoutedExperts`` chosen by the
logits, weighted by the softmax over the chosen ones, with clamped gated units.  Behind every layer stands a weighted sum of
the embedding's output and of all layers' results so far (``DepthAverage``).  The embedding adds a sinusoid of the position
(``SinusoidEmbedding``), and its table is the head, whose logits are scaled.  Tensor names: ``embed``, ``l<i>.norm1``,
``l<i>.canon1``, ``l<i>.mix.*``, ``l<i>.norm2``, ``l<i>.canon2``, ``l<i>.mlp.*``, ``l<i>.dwa``, ``final.norm``.
"""
from __future__ import annotations

from ..config import register_architecture
from ..config.zakusun import ZakusunConfig
from ..parts.attention import LatentCacheAttention
from ..parts.block import ConvNormBlock
from ..parts.conv import ConvolvedNorm
from ..parts.depth import DepthAverage
from ..parts.embedding import LMHead, SinusoidEmbedding
from ..parts.model import DecoderModel, LayerCall
from ..parts.moe import RoutedExperts
from ..parts.norm import GroupRMSNorm

#: where a part's tensor stands in the checkpoint, behind the layer's number
_NAMES = {"in1.norm.weight": "norm1", "in1.conv": "canon1", "in2.norm.weight": "norm2", "in2.conv": "canon2"}


def build_zakusun(cfg: ZakusunConfig) -> DecoderModel:
    d, eps = cfg.width, cfg.norm_eps

    def entry(place: int) -> ConvolvedNorm:
        return ConvolvedNorm(GroupRMSNorm(d, cfg.norm_groups, eps), cfg.canon_taps, place)

    blocks = []
    for layer in cfg.layers:
        m, mlp = layer["mixer"], layer["mlp"]
        mixer = LatentCacheAttention(d, m["heads"], m["dim"], m["vdim"], m["kv_rank"], m["scale"], eps, sink=True)
        ffn = None
        if mlp is not None:
            ffn = RoutedExperts(d, mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"], correction=False,
                                scoring="chosen", bias=True, unit="clamped", limit=mlp["expert"]["limit"])
        blocks.append(ConvNormBlock(entry(0), mixer, entry(1) if ffn is not None else None, ffn))

    def source(name: str) -> str:
        kind, _, rest = name.partition(".")
        if kind.startswith("blk"):
            return f"l{kind[3:]}.{_NAMES.get(rest, rest)}"
        if kind.startswith("depth"):
            return f"l{kind[5:]}.dwa"
        return name[:-len(".weight")] if name.endswith(".weight") else name

    embedding = SinusoidEmbedding(cfg.vocab, d)
    return DecoderModel(cfg, embedding, blocks, [LayerCall(block=i, cache=i) for i in range(len(blocks))],
                        GroupRMSNorm(d, cfg.norm_groups, eps),
                        LMHead(cfg.vocab, d, tied_to=embedding, scale=cfg.logit_scale, any_size=True),
                        names=("embed", "blk{}", "final.norm", "head"), sources=source,
                        depth=[DepthAverage(i + 2) for i in range(len(blocks))],
                        arg_keys={"width": "width", "groups": "norm.groups", "taps": "canon.taps", "vocab": "vocab",
                                  "kv_rank": "layers[].mixer.kv_rank", "n_experts": "layers[].mlp.router.experts",
                                  "top": "layers[].mlp.router.top"})


register_architecture("Zakusun", ZakusunConfig, build_zakusun)
