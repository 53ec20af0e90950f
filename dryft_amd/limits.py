"""Sizes the kernels take, in one place for the configuration classes and the parts that check them."""

MAX_HEAD_DIM = 256             # the widest attention head any kernel takes
MATRIX_CORE_HEAD_STEP = 16     # bfloat16 attention runs on the matrix cores for head sizes in these steps and on
                               # the plain kernel (float arithmetic, any size) for the rest
MAX_LATENT_WIDTH = 960         # the widest cached row (latent and rotated key part) the kernels that attend to latents take
MAX_LINEAR_STATE = 256         # the most key channels and value columns a head of linear attention keeps
MAX_NORM_GROUPS = 256          # the most parts a norm of a stream is taken in
MAX_STREAMS = 8                # the most copies of a residual stream (the stream kernel keeps them in registers, per column)
MAX_EXPERTS = 512              # the most experts a router chooses among
