"""Small Vabirax configurations for the tests: sizes that are no multiples of anything the kernels tile by, layers that differ
from each other, and the limits of the kernels' register and LDS variants."""


def cases(fh):
    """{name: config}"""
    lay, conf = fh.synth.vabirax_layer, fh.synth.vabirax_config
    #            heads dim rot vdim q_rank kv_rank ff window
    return {
        # every layer another shape, one without a feed-forward, the loop in the middle
        "uneven": conf(90, 203, [lay(5, 20, 6, 44, 50, 70, 130, 9), lay(3, 48, 24, 24, 33, 40, None, 64, base=777.0),
                                 lay(2, 7, 10, 65, 21, 130, 77, 30), lay(4, 33, 2, 12, 70, 17, 51, 33, scale=0.9)], loop=(1, 3, 2), embedding_scale=1.7, eps=3e-3),
        # more heads than one workgroup of the decode attention takes, window one past a tile; no loop
        "many_heads": conf(128, 257, [lay(21, 32, 32, 32, 64, 64, 96, 65)] * 2),
        # the sizes the published latent-attention models use per head; a loop over one layer
        "wide_head": conf(160, 120, [lay(2, 128, 64, 128, 192, 512, 100, 100), lay(3, 64, 32, 64, 48, 256, 60, 128)], loop=(0, 1, 3), embedding_scale=0.5),
        # ranks past the first LDS layout of the decode attention, the largest head
        "large_rank": conf(70, 97, [lay(3, 96, 32, 96, 40, 700, 64, 70), lay(2, 190, 56, 256, 30, 1000, None, 40)]),
        # values that are 1, a loop that runs once
        "ones": conf(33, 11, [lay(1, 1, 2, 1, 4, 5, 1, 1), lay(1, 3, 2, 2, 3, 4, 6, 2)], loop=(1, 2, 1)),
        # no mask: every earlier position is visible
        "no_window": conf(64, 150, [lay(4, 16, 16, 16, 32, 96, 64, None)] * 2, loop=(0, 2, 2)),
        # part of the rotated dimensions turns
        "part_rotation": conf(72, 90, [lay(2, 24, 20, 16, 24, 32, 40, 17, rot_dims=12)]),
    }
