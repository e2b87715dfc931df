// Scalar functions of the element-wise work, in f32 on the hardware's exp2 and reciprocal (about one unit in the last place
// each; the divide and expf of the math library cost ten times the instructions and the recurrence is bound by them).
#pragma once

#include "mesh_common.hpp"

namespace mesh {

// exp(-v), finite for every v: beyond 2^126 the sigmoid below is zero to f32 anyway
__device__ __forceinline__ float act_exp_neg(float v) { return __builtin_amdgcn_exp2f(fminf(v * -1.44269504088896341f, 126.f)); }
__device__ __forceinline__ float act_sigmoid(float v) { return __builtin_amdgcn_rcpf(1.0f + act_exp_neg(v)); }
__device__ __forceinline__ float act_silu(float v) { return v * act_sigmoid(v); }
__device__ __forceinline__ float act_gelu_tanh(float v) { return 0.5f * v * (1.0f + tanhf(0.7978845608028654f * (v + 0.044715f * v * v * v))); }

// the gates of a minimal gated recurrence from their pre-activations: the state becomes keep * state + in, keep = 1 - z and
// in = z * candidate; keep is formed without subtracting, so nothing cancels where z is nearly 1
struct MinGruGate { float keep, in; };
__device__ __forceinline__ MinGruGate min_gru_gate(float pz, float u) {
    const float e = act_exp_neg(pz), z = __builtin_amdgcn_rcpf(1.0f + e);
    return {e * z, z * (u >= 0.f ? u + 0.5f : act_sigmoid(u))};
}

}  // namespace mesh
