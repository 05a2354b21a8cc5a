"""Vefulix: several residual streams (hyper-connections) through layers that each name their mixer, assembled from parts.

Per sublayer the streams are read under learned shares, normed (layer norm with bias), and all written from the old ones and
the sublayer's output (`HyperConnectedBlock`). Mixers: a matrix memory with exponential gates (`MatrixMemory`), a gated delta
rule with one decay per head (`GatedDelta`), attention over a cached latent with queries from a latent of their own and a sink
per head, without positions (`LatentAttention`). Feed-forwards: routed experts beside a shared one (`RoutedExperts`, `SwiGLU`).
The embedding's rows pass a norm and are every stream; behind the layers the streams' sum passes the final norm, and the head
bends its logits under a cap.

Checkpoint names: `embed`, `embed.norm`, `l<i>.norm1|norm2`, `l<i>.hc1|hc2.in|out|mix`, `l<i>.mix.<tensor>`,
`l<i>.mlp.router`, `l<i>.mlp.e<j>|shared.gate|up|down`, `final.norm`, `head`; `.b` behind a norm, the router and the matrix
memory's gates for biases (`l<i>.mix.b` itself is the delta rule's write strength).
"""
from __future__ import annotations

from ..config.model_config import VefulixConfig
from ..parts.base import LayerCall, make_part
from ..parts.embedding import LMHead, TokenEmbedding
from ..registry import register_architecture
from .model import DecoderModel, WeightSource


@register_architecture("Vefulix")
def build_vefulix(cfg: VefulixConfig) -> DecoderModel:
    h, eps = cfg.hidden_size, cfg.norm_eps
    layers, order, sources = [], [], {}

    def norm(mine, stored):
        sources[mine + ".weight"], sources[mine + ".bias"] = [WeightSource(stored)], [WeightSource(stored + ".b")]
        return make_part("norm", "layer", size=h, eps=eps)

    def packed(mine, blocks):
        """`blocks`: (checkpoint tensor, rows) one after the other in one engine parameter."""
        at, out = 0, []
        for name, rows in blocks:
            out.append(WeightSource(name, at, rows))
            at += rows
        sources[mine] = out

    for i, layer in enumerate(cfg.layers):
        m, ck, me = layer.mixer, f"l{i}.mix.", f"layers.{i}.mixer."
        H, dn, nv = m["heads"], m["dim"], m["vdim"]
        if layer.kind == "mlstm":
            mixer = make_part("mixer", "mlstm", hidden_size=h, num_heads=H, key_dim=dn, value_dim=nv, gate_cap=m["gate_cap"], norm_eps=eps)
            packed(me + "in_proj.weight", [(ck + "q", H * dn), (ck + "k", H * dn), (ck + "v", H * nv), (ck + "g", H * nv), (ck + "i", H), (ck + "f", H)])
            same = (("i_bias", "i.b"), ("f_bias", "f.b"), ("norm_weight", "norm"))
        elif layer.kind == "delta":
            G = m["kv_heads"]
            mixer = make_part("mixer", "gated_delta", hidden_size=h, num_heads=H, key_heads=G, key_dim=dn, value_dim=nv, taps=m["conv"],
                              decay_rank=None, gate_rank=None, norm_eps=eps, gate_activation="silu")
            packed(me + "in_proj.weight", [(ck + "q", G * dn), (ck + "k", G * dn), (ck + "v", H * nv), (ck + "g", H * nv), (ck + "b", H), (ck + "a", H)])
            packed(me + "conv_weight", [(ck + "q.conv", G * dn), (ck + "k.conv", G * dn), (ck + "v.conv", H * nv)])
            same = (("A_log", "A_log"), ("dt_bias", "dt_bias"), ("norm_weight", "norm"))
        else:
            R, Rq = m["kv_rank"], m["q_rank"]
            mixer = make_part("mixer", "latent_attention", hidden_size=h, num_heads=H, nope_dim=dn, rot_dim=0, value_dim=nv, rank=R,
                              scale=m["scale"], norm_eps=eps, position=None, query_rank=Rq, sinks=True)
            packed(me + "in_proj.weight", [(ck + "dq", Rq), (ck + "dkv", R)])
            same = (("query_norm_weight", "dq.norm"), ("latent_norm_weight", "dkv.norm"), ("uq.weight", "uq"), ("uk", "uk"), ("uv", "uv"), ("sinks", "sink"))
        for mine, stored in same + (("o.weight", "o"),):
            sources[me + mine] = [WeightSource(ck + stored)]
        f, ffn = layer.mlp, None
        if f is not None:
            ck, me = f"l{i}.mlp.", f"layers.{i}.feed_forward."
            E, F, shared = f["experts"], f["ff"], None
            if f["shared_ff"] is not None:
                I = f["shared_ff"]
                shared = make_part("feed_forward", "swiglu", hidden_size=h, intermediate_size=I)
                packed(me + "shared.gate_up.weight", [(ck + "shared.gate", I), (ck + "shared.up", I)])
                sources[me + "shared.down.weight"] = [WeightSource(ck + "shared.down")]
            ffn = make_part("feed_forward", "moe", hidden_size=h, intermediate_size=F, num_experts=E, top=f["top"], shared=shared,
                            scoring="chosen", router_bias=True)
            sources[me + "router"], sources[me + "router_bias"] = [WeightSource(ck + "router")], [WeightSource(ck + "router.b")]
            packed(me + "gate_up", [(f"{ck}e{e}.{x}", F) for e in range(E) for x in ("gate", "up")])
            packed(me + "down", [(f"{ck}e{e}.down", h) for e in range(E)])
        for q in (1, 2) if f is not None else (1,):
            for mine, stored in (("read", "in"), ("out", "out"), ("mix", "mix")):
                sources[f"layers.{i}.{mine}{q}"] = [WeightSource(f"l{i}.hc{q}.{stored}")]
        layers.append(make_part("block", "hyper_connected", streams=cfg.streams, norm1=norm(f"layers.{i}.norm1", f"l{i}.norm1"), mixer=mixer,
                                norm2=norm(f"layers.{i}.norm2", f"l{i}.norm2") if f is not None else None, feed_forward=ffn))
        order.append(LayerCall(i))
    embedding = TokenEmbedding(cfg.vocab_size, h, norm=norm("embedding.norm", "embed.norm"))
    head = LMHead(cfg.vocab_size, h, softcap=cfg.logit_softcap)
    sources["embedding.weight"] = [WeightSource("embed")]
    sources["head.weight"] = [WeightSource("head")]
    return DecoderModel(cfg, embedding, layers, order, norm("final_norm", "final.norm"), head, sources)
