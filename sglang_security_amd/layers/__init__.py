"""Building blocks of checkpoint-loaded decoders: each takes its sizes and constants as parameters, keeps its weights in
the layout its kernels stream, and works on the rows of one step (engine.StepBatch)."""
