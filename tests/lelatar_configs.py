"""Small Lelatar configurations for the tests: they differ from each other in every size and option."""
import plain_lelatar as P

LEL = {
    # both kinds of layer, a loop in the middle over two layers, layers with and without a feed-forward
    "A": (P.make_config(vocab=97, width=64, layers=[
        P.parallel_layer(),
        P.mamba_layer(),
        P.parallel_layer(left=P.left_sizes(heads=2, kv_heads=1, dim=24, vdim=24, rot_dims=24, base=100.0, scale=0.3),
                         right=P.right_sizes(heads=6, kv_heads=3, dim=8, vdim=20, conv=2), ff=None),
        P.mamba_layer(heads=6, vdim=8, state=16, groups=3, norm_groups=1, conv=4, ff=40),
    ], loop=(1, 3, 2)), 11),
    # no loop, no second token table; sizes that are no multiple of 8 or 16; one head, one group; a convolution of one tap and one of six
    "B": (P.make_config(vocab=61, width=40, eps=1e-6, loop=None, side=None, layers=[
        P.mamba_layer(heads=1, vdim=12, state=5, groups=1, norm_groups=1, conv=1, ff=20),
        P.parallel_layer(left=P.left_sizes(heads=3, kv_heads=3, dim=12, vdim=20, rot_dims=6), right=P.right_sizes(heads=1, kv_heads=1, dim=20, vdim=12, conv=6), ff=9),
        P.mamba_layer(heads=10, vdim=6, state=70, groups=5, norm_groups=4, conv=6),
        P.parallel_layer(left=P.left_sizes(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=None), right=P.right_sizes(heads=3, kv_heads=3, dim=10, vdim=7, conv=1), ff=24),
    ]), 21),
    # the whole model is the loop, three passes; a head of more than 64 keys and more than 64 values
    "C": (P.make_config(vocab=33, width=32, side=5, loop=(0, 2, 3), layers=[
        P.mamba_layer(heads=2, vdim=72, state=24, groups=2, norm_groups=8, conv=3),
        P.parallel_layer(left=P.left_sizes(heads=2, kv_heads=2, dim=32, vdim=16, rot_dims=2, base=3.0), right=P.right_sizes(heads=2, kv_heads=1, dim=72, vdim=16, conv=3), ff=16),
    ]), 13),
    # a width that is no multiple of 8, one pass of a loop over the last layer, only recurrent layers
    "D": (P.make_config(vocab=50, width=36, side=12, loop=(2, 3, 1), layers=[
        P.mamba_layer(heads=4, vdim=8, state=8, groups=1, norm_groups=2, conv=2, ff=14), P.mamba_layer(heads=3, vdim=12, state=9, groups=3, norm_groups=3, conv=5),
        P.mamba_layer(heads=2, vdim=20, state=16, groups=2, norm_groups=1, conv=4),
    ]), 14),
}
