"""Small Kelasun configurations for the tests: they differ from layer to layer and from one another in every size and option: the order of
the two kinds of layer, one head and several, one key/value head and as many as heads, values larger and smaller than keys, sizes that
are multiples of 16 and sizes that are not of 8, stretched and plain frequencies, a rotated part that turns whole, in part and not at all,
temperatures that change within a page, far apart and not at all, one to all experts a token, a shared expert of the experts' size, of
another and none, layers without a feed-forward."""
import plain_kelasun as P

KEL = {
    # both kinds in turn; a temperature that steps every 16 and every 5 positions
    "A": (P.make_config(vocab=97, width=64, alpha=1.5, logit_scale=0.5, layers=[
        P.biased_layer(mlp=P.experts_mlp()),
        P.latent_layer(mlp=P.experts_mlp(ff=16, experts=6, top=3, shared=None)),
        P.biased_layer(heads=6, kv_heads=3, dim=8, vdim=24, q_temp=(0.7, 5), mlp=None),
        P.latent_layer(heads=2, dim=8, rot_dim=16, vdim=24, kv_rank=32, q_rank=16, base=1000.0, scaling=(8.0, 256, 4.0, 0.5), mlp=P.experts_mlp(ff=40, experts=5, top=1, shared=40)),
    ]), 11),
    # sizes the matrix-core kernels take (multiples of 16); the latent layer first; the scale of the scores and of the logits away from
    # the customary ones
    "B": (P.make_config(vocab=211, width=96, eps=1e-6, alpha=2.5, logit_scale=1.7, layers=[
        P.latent_layer(heads=4, dim=32, rot_dim=32, vdim=48, kv_rank=64, q_rank=48, base=500000.0, scaling=(2.0, 128, 32.0, 1.0), scale=0.3, mlp=P.experts_mlp(ff=32, experts=16, top=4, shared=48)),
        P.biased_layer(heads=4, kv_heads=1, dim=32, vdim=64, q_temp=(0.2, 64), scale=0.4, mlp=P.experts_mlp(ff=64, experts=4, top=2, shared=64)),
        P.biased_layer(heads=3, kv_heads=3, dim=16, vdim=16, q_temp=None, mlp=P.experts_mlp(ff=16, experts=3, top=3, shared=16)),
    ]), 12),
    # one head, one expert, one dimension of everything that may be one; no rotation at all
    "C": (P.make_config(vocab=33, width=32, eps=1e-3, alpha=1.0, logit_scale=1.0, layers=[
        P.biased_layer(heads=1, kv_heads=1, dim=8, vdim=8, q_temp=(1.0, 1), mlp=P.experts_mlp(ff=8, experts=1, top=1, shared=None)),
        P.latent_layer(heads=1, dim=8, rot_dim=0, vdim=8, kv_rank=8, q_rank=1, scaling=None, mlp=P.experts_mlp(ff=8, experts=2, top=1, shared=24)),
    ]), 13),
    # sizes that are no multiple of 8: heads of 12 + 6 and of 20, values of 10 and 7, latents of 20 and 9, experts of 13; a width that is no
    # multiple of 8; frequencies that are not stretched; a ramp as narrow as it gets
    "D": (P.make_config(vocab=131, width=36, alpha=0.8, logit_scale=0.25, layers=[
        P.latent_layer(heads=3, dim=12, rot_dim=6, vdim=10, kv_rank=20, q_rank=9, base=20.0, scaling=None, mlp=P.experts_mlp(ff=13, experts=9, top=2, shared=11)),
        P.biased_layer(heads=5, kv_heads=5, dim=20, vdim=7, q_temp=(0.5, 23), mlp=None),
        P.latent_layer(heads=1, dim=4, rot_dim=10, vdim=12, kv_rank=12, q_rank=30, base=30.0, scaling=(3.0, 64, 2.0, 2.0), mlp=P.experts_mlp(ff=7, experts=4, top=4, shared=5)),
        P.biased_layer(heads=2, kv_heads=1, dim=12, vdim=36, q_temp=(0.4, 100), mlp=P.experts_mlp(ff=20, experts=7, top=5, shared=None)),
    ]), 14),
}
# only a piece of the rotated part turns
KEL["D"][0]["layers"][2]["mixer"]["rot"]["dims"] = 8
