// Shared device helpers for the gfx950 kernels: element types, conversions, reductions.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace egpt {

constexpr int kWave = 64;  // CDNA wavefront width

// bfloat16 as raw bits; arithmetic is always done in float.
struct bf16_t {
    uint16_t bits;
};

__device__ __forceinline__ float to_float(float v) { return v; }
__device__ __forceinline__ float to_float(bf16_t v) { return __uint_as_float(static_cast<uint32_t>(v.bits) << 16); }

// round to nearest even; NaN stays NaN
__device__ __forceinline__ uint16_t f32_to_bf16_bits(float f) {
    uint32_t u = __float_as_uint(f);
    if ((u & 0x7fffffffu) > 0x7f800000u) return static_cast<uint16_t>((u >> 16) | 0x0040u);
    u += 0x7fffu + ((u >> 16) & 1u);
    return static_cast<uint16_t>(u >> 16);
}

template <typename T>
__device__ __forceinline__ T from_float(float v);
template <>
__device__ __forceinline__ float from_float<float>(float v) { return v; }
template <>
__device__ __forceinline__ bf16_t from_float<bf16_t>(float v) { return bf16_t{f32_to_bf16_bits(v)}; }

// The QKV epilogue's arithmetic, spelled out operation by operation: several kernels do it (one by one, four
// pairs at a time, inside the decode attention) and must leave the same bits, which they would not if the
// compiler were free to contract each one's multiplications and additions in its own way.
__device__ __forceinline__ float scale_then_bias(float x, float scale, float bias) { return __fmaf_rn(x, scale, bias); }
__device__ __forceinline__ float inv_rms(float ss, float inv_hidden, float eps) {
    return 1.0f / sqrtf(__fmaf_rn(ss, inv_hidden, eps));
}
__device__ __forceinline__ void rotate_pair(float a, float b, float c, float s, float& ra, float& rb) {
    ra = __fmaf_rn(a, c, -__fmul_rn(b, s));
    rb = __fmaf_rn(a, s, __fmul_rn(b, c));
}

// The activation of a gated feed-forward's gate: 0 silu, z / (1 + exp(-z)); 1 the tanh form of gelu,
// z / 2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), which is z / (1 + exp(-2 sqrt(2 / pi) (z + 0.044715 z^3))).
constexpr int kGateSilu = 0, kGateGeluTanh = 1;
constexpr int kUngatedRelu2 = 2;         // no gate: the square of relu (where a product can begin with either)
__device__ __forceinline__ float gate_exponent(float z, int act) {
    return act == kGateSilu ? z : 1.5957691216057308f * fmaf(0.044715f * z * z, z, z);
}
__device__ __forceinline__ float gate_activation(float z, int act) { return z / (1.0f + expf(-gate_exponent(z, act))); }

// The residual stream of steps of few tokens in 64-bit fixed point (units of 2^-32).  Several workgroups that split
// a product's k range add their partial results straight into it with integer atomics: integer addition does not
// care for the order, so the sum is the same bits whatever the scheduling, and the kernels that read the stream
// read one small tensor instead of every workgroup's partial sums.  A float32 value times 2^32 is an integer for
// every magnitude of 2^-8 and above and is rounded to one below (an absolute error of at most 2^-33, whatever the
// other values of the stream are); the stream holds magnitudes below 2^31.  What does not fit is not hidden as
// a small number: a magnitude of 2^31 or more, an infinity or a NaN enters as the largest magnitude of its sign
// (NaN: the negative one), which the norm behind it turns into a row of zeros and one entry of +-sqrt(width) - a
// step of more than 16 rows, and the float32 path, keep such values in float32 and show them as they are.
typedef long long fixed_t;
constexpr float kFixedOne = 4294967296.0f;
constexpr float kFixedLimit = 2147483648.0f;          // 2^31
__device__ __forceinline__ fixed_t to_fixed(float v) {
    if (!(fabsf(v) < kFixedLimit)) return v > 0.f ? 0x7fffffffffffffffLL : -0x7fffffffffffffffLL - 1;
    return __float2ll_rn(v * kFixedOne);
}
__device__ __forceinline__ float fixed_to_float(fixed_t v) { return __ll2float_rn(v) * (1.0f / kFixedOne); }
__device__ __forceinline__ void fixed_add(fixed_t* p, float v) {
    atomicAdd(reinterpret_cast<unsigned long long*>(p), static_cast<unsigned long long>(to_fixed(v)));
}
// what a residual stream of either kind is read and written as
__device__ __forceinline__ float residual_load(const float* p) { return *p; }
__device__ __forceinline__ float residual_load(const fixed_t* p) { return fixed_to_float(*p); }
__device__ __forceinline__ void residual_store(float* p, float v) { *p = v; }
__device__ __forceinline__ void residual_store(fixed_t* p, float v) { *p = to_fixed(v); }

// The output of a product arrives either as one tensor of the activation type, or as float32 partial
// sums [n_splits][rows][cols] of a split-k product, which are added here in split order.
template <typename T>
struct ProductView {
    const T* whole;          // used when n_splits == 0
    const float* partial;    // used when n_splits > 0
    int n_splits;
    size_t split_stride;     // rows * cols
    __device__ __forceinline__ bool present() const { return whole != nullptr || partial != nullptr; }
    __device__ __forceinline__ float at(size_t idx) const {
        if (n_splits == 0) return to_float(whole[idx]);
        if (n_splits == 1) return partial[idx];          // a product written out in float32: one load, not a round of sixteen
        // up to sixteen loads in flight at a time (a chain of dependent kernels pays for round trips, not
        // bytes); the order of the additions is fixed
        float v = 0.f;
        for (int s0 = 0; s0 < n_splits; s0 += 16) {
            float t[16];
#pragma unroll
            for (int i = 0; i < 16; ++i) t[i] = s0 + i < n_splits ? partial[(s0 + i) * split_stride + idx] : 0.f;
#pragma unroll
            for (int i = 0; i < 16; ++i) v += t[i];
        }
        return v;
    }
};

// A product whose x operand was (h * norm weight) still lacks each row's factor 1 / sqrt(sum_s ss[s][row] / hidden + eps):
// the sums of squares arrive beside it (null: the product is complete).
struct RowFactor {
    const float* ss;
    int splits, n_rows, hidden;
    float eps;
    __device__ __forceinline__ float of(int row) const {
        if (ss == nullptr) return 1.0f;
        float total = 0.f;
        for (int s = 0; s < splits; ++s) total += ss[static_cast<size_t>(s) * n_rows + row];
        return inv_rms(total, 1.0f / static_cast<float>(hidden), eps);
    }
};

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = kWave / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, kWave);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int o = kWave / 2; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, kWave));
    return v;
}

// Sum over a block of up to 1024 threads; every thread gets the result.  `scratch` holds >= 16 floats.
__device__ __forceinline__ float block_sum(float v, float* scratch) {
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int n_waves = (blockDim.x + kWave - 1) / kWave;
    v = wave_sum(v);
    __syncthreads();  // scratch may still be read from an earlier call
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < n_waves; ++w) total += scratch[w];
    return total;
}
__device__ __forceinline__ float block_max(float v, float* scratch) {
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int n_waves = (blockDim.x + kWave - 1) / kWave;
    v = wave_max(v);
    __syncthreads();
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float m = scratch[0];
    for (int w = 1; w < n_waves; ++w) m = fmaxf(m, scratch[w]);
    return m;
}

}  // namespace egpt

// Error codes returned by every entry point (0 = launched).
#define EGPT_OK 0
#define EGPT_BAD_ARGUMENT 1
#define EGPT_UNSUPPORTED_SIZE 2
#define EGPT_LAUNCH_FAILED 3
#define EGPT_STATIC_SCRATCH_TOO_SMALL 4
#define EGPT_STATIC_SCRATCH_UNRESOLVED 5

#define EGPT_CHECK_LAUNCH()                                   \
    do {                                                      \
        hipError_t e_ = hipGetLastError();                    \
        if (e_ != hipSuccess) return EGPT_LAUNCH_FAILED;      \
    } while (0)
