"""Small Kakirax configurations for the tests: sizes that are no multiples of anything the kernels tile by, layers that differ
from each other, shared weights, and the limits of the kernels' register and LDS variants."""


def cases(fh):
    """{name: (config, rank of the decays' maps)}"""
    att, gla, conf = fh.synth.kakirax_attention, fh.synth.kakirax_gla, fh.synth.kakirax_config
    # att: heads kv_heads dim vdim ff; gla: heads dim vdim ff
    return {
        # every layer another shape, with and without a feed-forward; one layer of each kind runs twice
        "uneven": (conf(90, 203, [gla(5, 20, 44, None), att(6, 2, 20, 44, 130, base=777.0, rot_dims=12, scaling=(5.0, 1.5, 6.0, 40)), gla(3, 48, 24, 77, tau=3.0),
                                  att(3, 3, 34, 12, None, scale=0.4), 0, gla(2, 7, 65, 51, tau=40.0), 1], embedding_scale=9.5, eps=3e-3, cap=7.0), 11),
        # more query heads per key / value head than one workgroup of the decode attention takes; many linear heads
        "many_heads": (conf(128, 257, [att(40, 2, 32, 32, 96), gla(21, 32, 32, 96), att(17, 1, 64, 64, None)], embedding_scale=11.0), 16),
        # the largest heads; the largest rank of the decays' map
        "wide": (conf(160, 120, [gla(2, 256, 256, 100), att(2, 1, 256, 256, 100, scaling=(8.0, 1.0, 4.0, 64)), gla(1, 130, 200, None), att(3, 1, 130, 230, None)],
                      embedding_scale=12.5, cap=50.0), 128),
        # the variants between
        "middle": (conf(192, 90, [gla(3, 64, 96, None), gla(2, 100, 128, 70), att(4, 2, 90, 40, None), att(2, 2, 128, 100, 40), att(4, 4, 64, 32, None), gla(2, 33, 70, None)],
                        embedding_scale=13.0), 33),
        # values that are 1 (or 2, where a pair has to be); eps keeps the norm of a lone value from being its mere sign
        "ones": (conf(33, 11, [gla(1, 1, 1, 1, tau=1.0), att(1, 1, 2, 1, 1), 0, att(2, 1, 3, 2, None, rot_dims=2)], embedding_scale=1.0, eps=0.5, cap=1.0), 1),
        # one kind of layer only; a layer that runs three times in a row
        "attention_only": (conf(64, 150, [att(4, 2, 16, 16, 64), 0, 0], embedding_scale=8.0), 16),
        "linear_only": (conf(70, 61, [gla(3, 16, 32, 40), gla(2, 24, 16, None), 1], embedding_scale=8.0), 4),
    }
