"""Venezen: a pre-norm decoder some of whose layers run several times with the same weights, assembled from parts.

Per layer x += mixer(norm1(x)), x += feed_forward(norm2(x)), layer norms without biases (`PreNormBlock`). The layers inside the
config's loop stand in the run order once per pass, each entry with pages of its own; the entry that begins a pass behind the
first takes the embedding's output into the stream again (`LayerCall.add_start`). Mixers: attention over a latent that all heads
share with one rotated key part (`LatentAttention`); attention whose values are its keys, without positions but for a bias that
falls with the distance, under a window, with a sink that scores 0 (`Attention`). Feed-forwards: dense with biases (`SwiGLU`), or
routed experts under a clamped gate, some of which hand their input on, beside a shared one (`RoutedExperts`, `ClampedGLU`). The
embedding's rows are multiplied by a constant; the head is the embedding table itself.

Checkpoint names: `embed`, `l<i>.norm1|norm2`, `l<i>.mix.<tensor>`, `l<i>.mlp.gate|up|down` (`.b` behind them for biases),
`l<i>.mlp.router|correction`, `l<i>.mlp.e<j>|shared.gate|up|down`, `final.norm`.
"""
from __future__ import annotations

from ..config.model_config import VenezenConfig
from ..parts.base import LayerCall, make_part
from ..parts.embedding import LMHead, TokenEmbedding
from ..registry import register_architecture
from .model import DecoderModel, WeightSource
from .sigosun import _kernel_head_size

GATE_ALPHA = 1.702             # the clamped gate's factor inside its sigmoid


def slopes(heads: int) -> list:
    """What a head's scores lose per token of distance: a geometric series from 2^(-8 / heads) down to 2^-8."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


@register_architecture("Venezen")
def build_venezen(cfg: VenezenConfig) -> DecoderModel:
    h, eps = cfg.hidden_size, cfg.norm_eps
    layers, sources = [], {}
    rotations: dict = {}                      # layers with equal rotations share one table

    def norm(mine, stored):
        sources[mine + ".weight"] = [WeightSource(stored)]
        return make_part("norm", "layer", size=h, eps=eps, bias=False)

    def packed(mine, blocks):
        """`blocks`: (checkpoint tensor, rows) one after the other in one engine parameter."""
        at, out = 0, []
        for name, rows in blocks:
            out.append(WeightSource(name, at, rows))
            at += rows
        sources[mine] = out

    for i, layer in enumerate(cfg.layers):
        m, ck, me = layer.mixer, f"l{i}.mix.", f"layers.{i}.mixer."
        H, dn = m["heads"], m["dim"]
        if layer.kind == "latent_attention":
            dr, R = m["rot_dim"], m["kv_rank"]
            position = None
            if dr:
                key = (dr, m["rot_base"])
                if key not in rotations:
                    rotations[key] = make_part("position_encoding", "rotary", head_dim=dr, theta=m["rot_base"], exact_angles=True)
                position = rotations[key]
            mixer = make_part("mixer", "latent_attention", hidden_size=h, num_heads=H, nope_dim=dn, rot_dim=dr, value_dim=m["vdim"], rank=R,
                              scale=m["scale"], norm_eps=eps, position=position)
            packed(me + "in_proj.weight", [(ck + "q", H * (dn + dr)), (ck + "dkv", R + dr)])
            same = (("latent_norm_weight", "dkv.norm"), ("uk", "uk"), ("uv", "uv"))
        else:
            G = m["kv_heads"]
            mixer = make_part("mixer", "attention", hidden_size=h, num_heads=H, num_kv_heads=G, head_dim=dn, scale=m["scale"],
                              window=m["window"], values_are_keys=True, slopes=slopes(H), sink_score=0.0, kernel_dim=_kernel_head_size(dn, dn))
            packed(me + "qkv.weight", [(ck + "q", H * dn), (ck + "k", G * dn)])
            same = ()
        for mine, stored in same + (("o.weight", "o"),):
            sources[me + mine] = [WeightSource(ck + stored)]
        f, ffn = layer.mlp, None
        ck, me = f"l{i}.mlp.", f"layers.{i}.feed_forward."
        if f is not None and f["kind"] == "dense":
            F = f["ff"]
            ffn = make_part("feed_forward", "swiglu", hidden_size=h, intermediate_size=F, bias=True)
            packed(me + "gate_up.weight", [(ck + "gate", F), (ck + "up", F)])
            packed(me + "gate_up_bias", [(ck + "gate.b", F), (ck + "up.b", F)])
            sources[me + "down.weight"], sources[me + "down_bias"] = [WeightSource(ck + "down")], [WeightSource(ck + "down.b")]
        elif f is not None:
            E, F, shared = f["experts"], f["ff"], None
            if f["shared_ff"] is not None:
                I = f["shared_ff"]
                shared = make_part("feed_forward", "clamped_glu", hidden_size=h, intermediate_size=I, limit=f["shared_limit"], alpha=GATE_ALPHA)
                packed(me + "shared.gate_up.weight", [(ck + "shared.gate", I), (ck + "shared.up", I)])
                sources[me + "shared.down.weight"] = [WeightSource(ck + "shared.down")]
            ffn = make_part("feed_forward", "moe", hidden_size=h, intermediate_size=F, num_experts=E, top=f["top"], shared=shared,
                            scoring="softmax", correction=True, normalise=True, route_scale=f["scale"], identity=f["identity"],
                            clamp=(f["limit"], GATE_ALPHA))
            sources[me + "router"], sources[me + "correction"] = [WeightSource(ck + "router")], [WeightSource(ck + "correction")]
            packed(me + "gate_up", [(f"{ck}e{e}.{x}", F) for e in range(E) for x in ("gate", "up")])
            packed(me + "down", [(f"{ck}e{e}.down", h) for e in range(E)])
        layers.append(make_part("block", "pre_norm", norm1=norm(f"layers.{i}.norm1", f"l{i}.norm1"), mixer=mixer,
                                norm2=norm(f"layers.{i}.norm2", f"l{i}.norm2") if ffn is not None else None, feed_forward=ffn))
    order = [LayerCall(i, add_start=again) for i, again in cfg.run_order()]
    embedding = TokenEmbedding(cfg.vocab_size, h, scale=cfg.embedding_scale)
    sources["embedding.weight"] = [WeightSource("embed")]
    return DecoderModel(cfg, embedding, layers, order, norm("final_norm", "final.norm"), LMHead(cfg.vocab_size, h, tied_to=embedding), sources)
