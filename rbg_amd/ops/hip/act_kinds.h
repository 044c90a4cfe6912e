// Gated activations by number, for kernels and bindings.
#pragma once

enum GluAct { GLU_GELU = 0, GLU_SILU = 1, GLU_CLAMPED = 2 };
