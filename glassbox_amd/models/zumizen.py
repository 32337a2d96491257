"""The Zumizen decoder assembled from parts.

Every layer norms what its sublayers give back and nothing they read: x += n1(mixer(x)), then x += n2(experts(x))
(``OutputNormBlock`` with ``RMSNorm``s).  The mixer *parallel* is two mixers over the same rows (``SideBySide``): attention with biases
(``GatedAttention`` without a gate: head norms, no rotation but a distance bias, runs of ``mask.size`` positions, a sink of score 0)
and the gated delta rule with one decay a head (``GatedDeltaRule``), each times a constant; *channel_delta* is the gated delta
rule with a decay a key channel and a sigmoid gate through a narrow middle.  The feed-forward is ``RoutedExperts`` by sigmoid scores
that are the weights as they stand and multiply what an expert reads.  The embedding is scaled and adds a row chosen by
the token and the one before it (``PairHashEmbedding``); the logits are bounded.  Tensor names: ``embed``, ``bigram``,
``l<i>.norm1``, ``l<i>.mix.*`` (``l<i>.mix.left.*``, ``l<i>.mix.right.*``), ``l<i>.norm2``, ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from ..config import register_architecture
from ..config.zumizen import ZumizenConfig
from ..parts.attention import GatedAttention
from ..parts.block import OutputNormBlock
from ..parts.conv import TimeConv
from ..parts.delta_rule import GatedDeltaRule
from ..parts.embedding import Embedding, LMHead, PairHashEmbedding
from ..parts.model import DecoderModel, LayerCall
from ..parts.moe import RoutedExperts
from ..parts.norm import RMSNorm
from ..parts.side_by_side import SideBySide


def _delta(cfg: ZumizenConfig, m, **options) -> GatedDeltaRule:
    return GatedDeltaRule(cfg.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], cfg.norm_eps, **options)


def _mixer(cfg: ZumizenConfig, layer):
    m = layer["mixer"]
    if layer["type"] == "channel_delta":
        return _delta(cfg, m, decay="channel", gate="low", gate_act="sigmoid", decay_rank=m.get("decay_rank"),
                      gate_rank=m.get("gate_rank"))
    a = m["left"]
    left = GatedAttention(cfg.width, a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["scale"], cfg.norm_eps, bias=True, qk_norm="head",
                          chunk=(a.get("mask") or {"size": 0})["size"], sink="zero", gate=None, slope=True, out_bias=True,
                          result_scale=m["left_scale"])
    return SideBySide(left, _delta(cfg, m["right"], decay="head", gate="full", gate_act="silu", result_scale=m["right_scale"]))


def _experts(cfg: ZumizenConfig, mlp) -> RoutedExperts:
    r = mlp["router"]
    return RoutedExperts(cfg.width, r["experts"], r["top"], mlp["expert"]["ff"], correction=False, scoring="sigmoid", renorm=False,
                         weigh_in=True)


def _source(name: str) -> str:
    """The checkpoint names a norm or a table by its place alone."""
    if name.endswith(".weight"):
        name = name[:-len(".weight")]
    return {"embed.pairs": "bigram"}.get(name, name)


def build_zumizen(cfg: ZumizenConfig) -> DecoderModel:
    d, eps = cfg.width, cfg.norm_eps
    norm = lambda: RMSNorm(d, eps, adds=True)
    blocks = []
    for layer in cfg.layers:
        ffn = _experts(cfg, layer["mlp"]) if layer["mlp"] is not None else None
        blocks.append(OutputNormBlock(TimeConv(d, 0), _mixer(cfg, layer), norm(), ffn, norm() if ffn is not None else None,
                                      names=("in", "mix", "norm1", "mlp", "norm2")))
    schedule = [LayerCall(block=i, cache=i) for i in range(len(blocks))]
    if cfg.bigram is not None:
        embedding = PairHashEmbedding(cfg.vocab, d, *cfg.bigram, scale=cfg.embedding_scale)
    else:
        embedding = Embedding(cfg.vocab, d, scale=cfg.embedding_scale)
    return DecoderModel(cfg, embedding, blocks, schedule, norm(), LMHead(cfg.vocab, d, any_size=True, softcap=cfg.logit_softcap),
                        names=("embed", "l{}", "final.norm", "head"), sources=_source,
                        arg_keys={"width": "width", "dim": "layers[].mixer.dim", "vdim": "layers[].mixer.vdim",
                                  "taps": "layers[].mixer.conv", "n_experts": "layers[].mlp.router.experts",
                                  "top": "layers[].mlp.router.top", "vocab": "vocab"})


register_architecture("Zumizen", ZumizenConfig, build_zumizen)
