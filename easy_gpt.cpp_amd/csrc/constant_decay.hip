// Linear attention whose state decays by one constant per head and step, from the input product to the gated heads:
//   S_t = d_h S_(t-1) + (c k_t) v_t^T,   o_t = S_t^T q_t,   out_t = o_t / rms(o_t) * weight * act(gate_t),
// with queries and keys rotated by their position on the way in, c a constant factor on the keys, the norm per head (the
// weight may be absent) and the gate from further columns of the product.  Everything between the product and `out` is
// float32, the matrix products too (v_mfma_f32_16x16x4_f32: float32 operands and accumulation).
//
// A constant decay lets a portion of a prompt be computed in chunks of C tokens instead of token by token.  With i, j the
// places in a chunk of n tokens and S the state before it:
//   o_i = sum_(j <= i) d^(i - j) (q_i . c k_j) v_j + d^(i + 1) S^T q_i
//   S'  = d^n S + sum_j d^(n - 1 - j) (c k_j) v_j^T
// Three kernels: every chunk's own sum of the second line (all chunks at once), a walk over the chunks that turns the sums
// into the states before each chunk (elementwise, all elements at once), and the outputs (all chunks at once).  The powers
// of d come from a table that the caller computed in float64, so no power is ever divided by another.
// Steps of few tokens per request walk them one by one in a kernel that keeps a head's state in registers.
#include "api.h"
#include "common.h"

namespace egpt {

typedef __attribute__((ext_vector_type(4))) float d_f32x4;

constexpr int kDecayPowers = 65;           // d^0 .. d^64 per head

template <typename T>
struct DecayArgs {
    ProductView<T> proj;
    const float* flat;                     // proj as one float32 tensor whose heads start on 16 bytes, or null
    int head_fours;                        // with flat: queries and keys may be rotated four places at a time too
    int proj_width, q_off, k_off, v_off, g_off;
    float k_scale;
    const float* cos_sin;                  // [tokens][rot_dims / 2][2]
    int rot_dims, interleaved;
    float mag;
    const float* powers;                   // [heads][kDecayPowers]
    float* states;                         // [slots][heads][dk][dv]
    const int32_t* slots;
    const unsigned char* fresh;            // may be null
    const int32_t* q_start;
    const int32_t* q_len;
    int n_seqs;
    float* chunk_states;                   // [chunks][heads][dk][dv]
    const T* norm_w;                       // [dv] or null
    float eps;
    int gate_act;                          // 0 silu, 1 sigmoid
    T* out;                                // [tokens][heads * dv]
    int heads, dk, dv;
};

// the wait between matrix instructions in a loop of unknown length and the first read of their results
__device__ __forceinline__ void products_ready() {
    __builtin_amdgcn_sched_barrier(0);
    asm volatile("s_nop 15");
    __builtin_amdgcn_sched_barrier(0);
}

// the places (a, b) of a head that slot s of its pairs holds: two that turn together, or two neighbours that pass (b may be dk)
__device__ __forceinline__ bool pair_places(int s, int rot_dims, int interleaved, int& a, int& b) {
    const int half = rot_dims / 2;
    if (s < half) {
        a = interleaved ? 2 * s : s;
        b = interleaved ? 2 * s + 1 : s + half;
        return true;
    }
    a = rot_dims + 2 * (s - half);
    b = a + 1;
    return false;
}
__device__ __forceinline__ int pair_slots(int dk, int rot_dims) { return rot_dims / 2 + (dk - rot_dims + 1) / 2; }

__device__ __forceinline__ float gate_value(float z, int act) {
    const float sig = 1.0f / (1.0f + expf(-z));
    return act == 0 ? z * sig : sig;
}
template <typename T>
__device__ __forceinline__ float gate_of(const DecayArgs<T>& a, size_t t, int column) {
    return gate_value(a.proj.at(t * a.proj_width + a.g_off + column), a.gate_act);
}

// which request and which of its chunks a workgroup has; false: none
template <typename T>
__device__ __forceinline__ bool find_chunk(const DecayArgs<T>& a, int index, int chunk, int& b, int& c) {
    b = 0, c = index;
    for (; b < a.n_seqs; ++b) {
        const int n = (a.q_len[b] + chunk - 1) / chunk;
        if (c < n) return true;
        c -= n;
    }
    return false;
}

// Rotated heads of a chunk's tokens into LDS [chunk][row], columns dk .. padded and rows behind the chunk's tokens zero.
template <typename T, int C, int THREADS, typename F>
__device__ __forceinline__ void stage_heads(const DecayArgs<T>& a, int offset, int h, int t0, int n, int padded, int row, float* dst,
                                            F factor) {
    const int pads = padded - a.dk;
    for (int idx = threadIdx.x; idx < C * pads; idx += THREADS) dst[(idx / pads) * row + a.dk + idx % pads] = 0.f;
    if (a.head_fours) {                                   // halves that turn together, four places of each at a time
        const int half = a.rot_dims / 2, turns = half / 4, items = turns + (a.dk - a.rot_dims) / 4;
#pragma unroll 4
        for (int idx = threadIdx.x; idx < C * items; idx += THREADS) {
            const int tt = idx / items, s = idx % items;
            const bool turned = s < turns;
            const int pa = turned ? 4 * s : a.rot_dims + 4 * (s - turns);
            float4 x = float4{0.f, 0.f, 0.f, 0.f}, y = x;
            if (tt < n) {
                const size_t t = static_cast<size_t>(t0 + tt), at = t * a.proj_width + offset + h * a.dk;
                const float f = factor(tt);
                x = *reinterpret_cast<const float4*>(a.flat + at + pa);
                if (turned) {
                    y = *reinterpret_cast<const float4*>(a.flat + at + pa + half);
                    const float4 c0 = *reinterpret_cast<const float4*>(a.cos_sin + t * a.rot_dims + 8 * s);
                    const float4 c1 = *reinterpret_cast<const float4*>(a.cos_sin + t * a.rot_dims + 8 * s + 4);
                    rotate_pair(x.x, y.x, c0.x * a.mag, c0.y * a.mag, x.x, y.x);
                    rotate_pair(x.y, y.y, c0.z * a.mag, c0.w * a.mag, x.y, y.y);
                    rotate_pair(x.z, y.z, c1.x * a.mag, c1.y * a.mag, x.z, y.z);
                    rotate_pair(x.w, y.w, c1.z * a.mag, c1.w * a.mag, x.w, y.w);
                    y.x *= f, y.y *= f, y.z *= f, y.w *= f;
                }
                x.x *= f, x.y *= f, x.z *= f, x.w *= f;
            }
            *reinterpret_cast<float4*>(dst + tt * row + pa) = x;
            if (turned) *reinterpret_cast<float4*>(dst + tt * row + pa + half) = y;
        }
        return;
    }
    const int slots = pair_slots(a.dk, a.rot_dims);
#pragma unroll 4
    for (int idx = threadIdx.x; idx < C * slots; idx += THREADS) {
        const int tt = idx / slots, s = idx % slots;
        int pa, pb;
        const bool turned = pair_places(s, a.rot_dims, a.interleaved, pa, pb);
        float x = 0.f, y = 0.f;
        if (tt < n) {
            const size_t t = static_cast<size_t>(t0 + tt), at = t * a.proj_width + offset + h * a.dk;
            x = a.proj.at(at + pa);
            if (pb < a.dk) y = a.proj.at(at + pb);
            if (turned) {
                const float2 cs = *reinterpret_cast<const float2*>(a.cos_sin + t * a.rot_dims + 2 * s);
                rotate_pair(x, y, cs.x * a.mag, cs.y * a.mag, x, y);
            }
            const float f = factor(tt);
            x *= f, y *= f;
        }
        dst[tt * row + pa] = x;
        if (pb < a.dk) dst[tt * row + pb] = y;
    }
}

template <typename T, int C, int WIDTH, int THREADS>
__device__ __forceinline__ void stage_values(const DecayArgs<T>& a, int h, int t0, int n, int row, float* dst) {
    if (a.flat != nullptr) {                              // four features at a time (dv is a multiple of four)
#pragma unroll 8
        for (int idx = threadIdx.x; idx < C * (WIDTH / 4); idx += THREADS) {
            const int tt = idx / (WIDTH / 4), f = idx % (WIDTH / 4) * 4;
            float4 v = float4{0.f, 0.f, 0.f, 0.f};
            if (tt < n && f < a.dv)
                v = *reinterpret_cast<const float4*>(a.flat + static_cast<size_t>(t0 + tt) * a.proj_width + a.v_off + h * a.dv + f);
            *reinterpret_cast<float4*>(dst + tt * row + f) = v;
        }
        return;
    }
#pragma unroll 4
    for (int idx = threadIdx.x; idx < C * WIDTH; idx += THREADS) {
        const int tt = idx / WIDTH, f = idx % WIDTH;
        dst[tt * row + f] = (tt < n && f < a.dv) ? a.proj.at(static_cast<size_t>(t0 + tt) * a.proj_width + a.v_off + h * a.dv + f) : 0.f;
    }
}

// DT neighbouring floats (DT a power of two; 16-byte pieces where DT allows)
template <int DT>
__device__ __forceinline__ void load_run(const float* p, float* v) {
    if constexpr (DT == 1) v[0] = p[0];
    else if constexpr (DT == 2) {
        const float2 x = *reinterpret_cast<const float2*>(p);
        v[0] = x.x, v[1] = x.y;
    } else {
#pragma unroll
        for (int i = 0; i < DT; i += 4) {
            const float4 x = *reinterpret_cast<const float4*>(p + i);
            v[i] = x.x, v[i + 1] = x.y, v[i + 2] = x.z, v[i + 3] = x.w;
        }
    }
}

// The matrix tiles below: 16 rows x 16 columns, a lane (lj = lane % 16, lg = lane / 16) holds operand values of row (or
// column) lj at the four summation places 4 lg .. 4 lg + 3 of a group of 16, and of a result the rows 4 lg .. 4 lg + 3 of
// column lj.  Value features are dealt to columns so that column lj of the DT tiles holds the neighbours lj * DT .. lj * DT +
// DT - 1: a lane's features are one run in memory.
//
// A chunk's own sum: chunk_states[chunk][h] = sum_j d^(n - 1 - j) (c k_j) v_j^T, one workgroup per (chunk, head), C = 16 RT.
template <typename T, int DT, int RT>
__global__ __launch_bounds__(64 * RT) void chunk_sums_kernel(DecayArgs<T> a) {
    constexpr int C = 16 * RT, THREADS = 64 * RT, VROW = 16 * DT + 4;
    extern __shared__ __attribute__((aligned(16))) float decay_smem[];
    int b, c;
    if (!find_chunk(a, blockIdx.x, C, b, c)) return;
    const int h = blockIdx.y, n = min(C, a.q_len[b] - c * C), t0 = a.q_start[b] + c * C;
    const int dkp = (a.dk + 15) / 16 * 16, krow = dkp + 4;
    float* k_s = decay_smem;
    float* v_s = k_s + C * krow;
    const float* pw = a.powers + h * kDecayPowers;
    stage_heads<T, C, THREADS>(a, a.k_off, h, t0, n, dkp, krow, k_s, [&](int tt) { return a.k_scale * pw[n - 1 - tt]; });
    stage_values<T, C, 16 * DT, THREADS>(a, h, t0, n, VROW, v_s);
    __syncthreads();
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, lj = lane % 16, lg = lane / 16;
    float* dst = a.chunk_states + (static_cast<size_t>(blockIdx.x) * a.heads + h) * a.dk * a.dv;
    for (int r = wave; r < dkp / 16; r += RT) {
        d_f32x4 acc[DT];
#pragma unroll
        for (int d = 0; d < DT; ++d) acc[d] = d_f32x4{0.f, 0.f, 0.f, 0.f};
        for (int j0 = 0; j0 < n; j0 += 16) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float kv = k_s[(j0 + lg * 4 + i) * krow + r * 16 + lj];
                float vv[DT];
                load_run<DT>(v_s + (j0 + lg * 4 + i) * VROW + lj * DT, vv);
#pragma unroll
                for (int d = 0; d < DT; ++d) acc[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(kv, vv[d], acc[d], 0, 0, 0);
            }
        }
        products_ready();
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int row = r * 16 + lg * 4 + v;
            if (row >= a.dk) continue;
            float* at = dst + static_cast<size_t>(row) * a.dv + lj * DT;
            if constexpr (DT % 4 == 0) {
                if (a.dv == 16 * DT) {
#pragma unroll
                    for (int d = 0; d < DT; d += 4)
                        *reinterpret_cast<float4*>(at + d) = float4{acc[d][v], acc[d + 1][v], acc[d + 2][v], acc[d + 3][v]};
                    continue;
                }
            }
#pragma unroll
            for (int d = 0; d < DT; ++d)
                if (lj * DT + d < a.dv) at[d] = acc[d][v];
        }
    }
}

// The states before every chunk, in place of the chunks' sums, and the state behind the step into the request's record.
// A thread owns VEC neighbouring elements of one (request, head)'s matrix and walks the chunks, eight loads in flight.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void chunk_states_kernel(DecayArgs<T> a, int chunk) {
    const int b = blockIdx.x, h = blockIdx.y;
    const size_t per_head = static_cast<size_t>(a.dk) * a.dv;
    const size_t e = (static_cast<size_t>(blockIdx.z) * 256 + threadIdx.x) * VEC;
    const int total = a.q_len[b];
    if (e >= per_head || total <= 0) return;
    size_t first = 0;
    for (int i = 0; i < b; ++i) first += (a.q_len[i] + chunk - 1) / chunk;
    const int n_chunks = (total + chunk - 1) / chunk;
    float* record = a.states + (static_cast<size_t>(a.slots[b]) * a.heads + h) * per_head + e;
    const float* pw = a.powers + h * kDecayPowers;
    const float whole = pw[chunk], rest = pw[total - (n_chunks - 1) * chunk];
    float s[VEC];
    const bool anew = a.fresh != nullptr && a.fresh[b] != 0;
#pragma unroll
    for (int i = 0; i < VEC; ++i) s[i] = 0.f;
    if (!anew) load_run<VEC>(record, s);
    const size_t stride = static_cast<size_t>(a.heads) * per_head;
    float* at = a.chunk_states + (first * a.heads + h) * per_head + e;
    constexpr int U = 8;
    for (int c0 = 0; c0 < n_chunks; c0 += U) {
        float u[U][VEC];
#pragma unroll
        for (int i = 0; i < U; ++i)
            if (c0 + i < n_chunks) load_run<VEC>(at + (c0 + i) * stride, u[i]);
#pragma unroll
        for (int i = 0; i < U; ++i) {
            if (c0 + i >= n_chunks) break;
            float* dst = at + (c0 + i) * stride;
            const float d = c0 + i + 1 < n_chunks ? whole : rest;
            if constexpr (VEC == 4) *reinterpret_cast<float4*>(dst) = float4{s[0], s[1], s[2], s[3]};
            else *dst = s[0];
#pragma unroll
            for (int k = 0; k < VEC; ++k) s[k] = fmaf(d, s[k], u[i][k]);
        }
    }
    if constexpr (VEC == 4) *reinterpret_cast<float4*>(record) = float4{s[0], s[1], s[2], s[3]};
    else *record = s[0];
}

// A chunk's outputs: one workgroup per (chunk, head), a wavefront per 16 of its tokens.
template <typename T, int DT, int RT>
__global__ __launch_bounds__(64 * RT) void chunk_outputs_kernel(DecayArgs<T> a) {
    constexpr int C = 16 * RT, THREADS = 64 * RT, VROW = 16 * DT + 4;
    extern __shared__ __attribute__((aligned(16))) float decay_smem[];
    __shared__ float pw_s[kDecayPowers];
    int b, c;
    if (!find_chunk(a, blockIdx.x, C, b, c)) return;
    const int h = blockIdx.y, n = min(C, a.q_len[b] - c * C), t0 = a.q_start[b] + c * C;
    const int dkp = (a.dk + 15) / 16 * 16, krow = dkp + 4;
    float* q_s = decay_smem;
    float* k_s = q_s + C * krow;
    float* v_s = k_s + C * krow;
    if (threadIdx.x < kDecayPowers) pw_s[threadIdx.x] = a.powers[h * kDecayPowers + threadIdx.x];
    if (THREADS < kDecayPowers && threadIdx.x == 0) pw_s[kDecayPowers - 1] = a.powers[h * kDecayPowers + kDecayPowers - 1];
    stage_heads<T, C, THREADS>(a, a.q_off, h, t0, n, dkp, krow, q_s, [](int) { return 1.0f; });
    stage_heads<T, C, THREADS>(a, a.k_off, h, t0, n, dkp, krow, k_s, [&](int) { return a.k_scale; });
    stage_values<T, C, 16 * DT, THREADS>(a, h, t0, n, VROW, v_s);
    __syncthreads();
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, lj = lane % 16, lg = lane / 16;
    if (wave * 16 >= n) return;
    const int row = wave * 16 + lj;                       // the token of the chunk whose operand values this lane holds
    const float* q_row = q_s + row * krow + lg * 4;
    const int pieces = dkp / 16;
    d_f32x4 o[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d) o[d] = d_f32x4{0.f, 0.f, 0.f, 0.f};
    const bool whole_runs = a.dv == 16 * DT;              // every lane's run of features lies inside the head
    // the gates of this lane's results (in flight from here on)
    constexpr bool KEEP_GATES = DT <= 8;
    float gates[4][KEEP_GATES ? DT : 1];
    const bool gates_here = KEEP_GATES && a.flat != nullptr && whole_runs;
    if constexpr (KEEP_GATES) if (gates_here) {
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int tt = min(wave * 16 + lg * 4 + v, n - 1);
            load_run<DT>(a.flat + static_cast<size_t>(t0 + tt) * a.proj_width + a.g_off + h * a.dv + lj * DT, gates[v]);
        }
    }
    // the state before the chunk (a new request's first chunk has none), its rows read a piece ahead
    if (c > 0 || !(a.fresh != nullptr && a.fresh[b] != 0)) {
        const float* state = a.chunk_states + (static_cast<size_t>(blockIdx.x) * a.heads + h) * a.dk * a.dv;
        const float through = pw_s[row + 1];
        auto state_piece = [&](int kk, float (&sv)[4][DT]) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int key = kk * 16 + lg * 4 + i;
                const float* src = state + static_cast<size_t>(key) * a.dv + lj * DT;
                if (whole_runs && a.dk % 16 == 0) {
                    load_run<DT>(src, sv[i]);
                } else {
#pragma unroll
                    for (int d = 0; d < DT; ++d) sv[i][d] = key < a.dk && lj * DT + d < a.dv ? src[d] : 0.f;
                }
            }
        };
        auto state_product = [&](int kk, const float (&sv)[4][DT]) {
            const float4 q4 = *reinterpret_cast<const float4*>(q_row + kk * 16);
            const float qv[4] = {q4.x * through, q4.y * through, q4.z * through, q4.w * through};
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int d = 0; d < DT; ++d) o[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[i], sv[i][d], o[d], 0, 0, 0);
        };
        float sa[4][DT], sb[4][DT];                       // (two sets in turn)
        state_piece(0, sa);
        for (int kk = 0; kk < pieces; kk += 2) {
            if (kk + 1 < pieces) state_piece(kk + 1, sb);
            state_product(kk, sa);
            if (kk + 1 < pieces) {
                if (kk + 2 < pieces) state_piece(kk + 2, sa);
                state_product(kk + 1, sb);
            }
        }
    }
    // the chunk's own tokens up to each row's: scores transposed, so that a lane holds four keys of its row, which are the
    // second product's operand as they lie in registers
    for (int kt = 0; kt <= wave; ++kt) {
        d_f32x4 acc = d_f32x4{0.f, 0.f, 0.f, 0.f};
        const float* k_row = k_s + (kt * 16 + lj) * krow + lg * 4;
        for (int kk = 0; kk < pieces; ++kk) {
            const float4 k4 = *reinterpret_cast<const float4*>(k_row + kk * 16);
            const float4 q4 = *reinterpret_cast<const float4*>(q_row + kk * 16);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.x, q4.x, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.y, q4.y, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.z, q4.z, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.w, q4.w, acc, 0, 0, 0);
        }
        products_ready();
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int key = kt * 16 + lg * 4 + i;
            const float p = key <= row ? acc[i] * pw_s[max(row - key, 0)] : 0.f;
            float vv[DT];
            load_run<DT>(v_s + key * VROW + lj * DT, vv);
#pragma unroll
            for (int d = 0; d < DT; ++d) o[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(p, vv[d], o[d], 0, 0, 0);
        }
    }
    products_ready();
#pragma unroll
    for (int v = 0; v < 4; ++v) {
        const int tt = wave * 16 + lg * 4 + v;
        float ss = 0.f;
#pragma unroll
        for (int d = 0; d < DT; ++d) ss = fmaf(o[d][v], o[d][v], ss);      // (features beyond dv are zeros)
#pragma unroll
        for (int off = 8; off > 0; off >>= 1) ss += __shfl_xor(ss, off, kWave);
        if (tt >= n) continue;
        const float inv = inv_rms(ss, 1.0f / static_cast<float>(a.dv), a.eps);
        const size_t t = static_cast<size_t>(t0 + tt);
        T* dst = a.out + t * a.heads * a.dv + static_cast<size_t>(h) * a.dv;
        float y[DT];
#pragma unroll
        for (int d = 0; d < DT; ++d) {
            const int f = lj * DT + d;
            y[d] = 0.f;
            if (f >= a.dv) continue;
            y[d] = o[d][v] * inv;
            if (a.norm_w != nullptr) y[d] *= to_float(a.norm_w[f]);
            y[d] *= gates_here ? gate_value(gates[v][KEEP_GATES ? d : 0], a.gate_act) : gate_of(a, t, h * a.dv + f);
        }
        if constexpr (sizeof(T) == 2 && DT % 8 == 0) {
            if (whole_runs) {
#pragma unroll
                for (int d = 0; d < DT; d += 8) {
                    uint32_t w[4];
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        w[i] = f32_to_bf16_bits(y[d + 2 * i]) | (static_cast<uint32_t>(f32_to_bf16_bits(y[d + 2 * i + 1])) << 16);
                    *reinterpret_cast<uint4*>(dst + lj * DT + d) = uint4{w[0], w[1], w[2], w[3]};
                }
                continue;
            }
        }
#pragma unroll
        for (int d = 0; d < DT; ++d)
            if (lj * DT + d < a.dv) dst[lj * DT + d] = from_float<T>(y[d]);
    }
}

// Token by token: one workgroup per (request, head) with the head's state in registers.  Threads are columns (VEC
// neighbours each) x row groups; a thread keeps rows group, group + groups, ... (NV of them) of its columns.
template <typename T, int NV, int VEC>
__global__ __launch_bounds__(1024) void decay_steps_kernel(DecayArgs<T> a) {
    extern __shared__ __attribute__((aligned(16))) float decay_smem[];
    __shared__ float scratch[16];
    const int b = blockIdx.x, h = blockIdx.y;
    const int n = a.q_len[b];
    if (n <= 0) return;
    const int dk = a.dk, dv = a.dv, t0 = a.q_start[b];
    const int columns = (dv + VEC - 1) / VEC, groups = blockDim.x / columns;
    const int col = threadIdx.x % columns, group = threadIdx.x / columns;
    const bool active = group < groups;
    float* q_s = decay_smem;
    float* k_s = q_s + dk;
    float* v_s = k_s + dk + ((2 * dk) & 3 ? 4 - ((2 * dk) & 3) : 0);      // (on 16 bytes)
    float* g_s = v_s + (dv + 3) / 4 * 4;
    float* part_s = g_s + dv;
    float* record = a.states + (static_cast<size_t>(a.slots[b]) * a.heads + h) * dk * dv;
    const bool anew = a.fresh != nullptr && a.fresh[b] != 0;
    float s[NV][VEC];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int r = group + i * groups;
#pragma unroll
        for (int e = 0; e < VEC; ++e) s[i][e] = 0.f;
        if (active && !anew && r < dk) load_run<VEC>(record + static_cast<size_t>(r) * dv + col * VEC, s[i]);
    }
    const float decay = a.powers[h * kDecayPowers + 1];
    const int slots = pair_slots(dk, a.rot_dims);
    for (int i0 = 0; i0 < n; ++i0) {
        const size_t t = static_cast<size_t>(t0 + i0), row = t * a.proj_width;
        __syncthreads();                              // the token before is written out
        for (int idx = threadIdx.x; idx < 2 * slots + 2 * dv; idx += blockDim.x) {
            if (idx >= 2 * slots) {
                const int f = idx - 2 * slots;
                if (f < dv) v_s[f] = a.proj.at(row + a.v_off + h * dv + f);
                else g_s[f - dv] = gate_of(a, t, h * dv + (f - dv));
                continue;
            }
            const bool key = idx >= slots;
            int pa, pb;
            const int sl = key ? idx - slots : idx;
            const bool turned = pair_places(sl, a.rot_dims, a.interleaved, pa, pb);
            const size_t at = row + (key ? a.k_off : a.q_off) + h * dk;
            float x = a.proj.at(at + pa), y = pb < dk ? a.proj.at(at + pb) : 0.f;
            if (turned) {
                const float2 cs = *reinterpret_cast<const float2*>(a.cos_sin + t * a.rot_dims + 2 * sl);
                rotate_pair(x, y, cs.x * a.mag, cs.y * a.mag, x, y);
            }
            float* dst = key ? k_s : q_s;
            const float f = key ? a.k_scale : 1.0f;
            dst[pa] = x * f;
            if (pb < dk) dst[pb] = y * f;
        }
        __syncthreads();
        if (active) {
            float vv[VEC], o[VEC];
            load_run<VEC>(v_s + col * VEC, vv);
#pragma unroll
            for (int e = 0; e < VEC; ++e) o[e] = 0.f;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int r = group + i * groups;
                const float kr = r < dk ? k_s[r] : 0.f, qr = r < dk ? q_s[r] : 0.f;
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    s[i][e] = fmaf(decay, s[i][e], kr * vv[e]);
                    o[e] = fmaf(s[i][e], qr, o[e]);
                }
            }
#pragma unroll
            for (int e = 0; e < VEC; ++e) part_s[group * columns * VEC + col * VEC + e] = o[e];
        }
        __syncthreads();
        float o = 0.f;
        if (threadIdx.x < dv)
            for (int g = 0; g < groups; ++g) o += part_s[g * columns * VEC + threadIdx.x];
        const float inv = inv_rms(block_sum(o * o, scratch), 1.0f / static_cast<float>(dv), a.eps);
        if (threadIdx.x < dv) {
            float y = o * inv;
            if (a.norm_w != nullptr) y *= to_float(a.norm_w[threadIdx.x]);
            a.out[(t * a.heads + h) * dv + threadIdx.x] = from_float<T>(y * g_s[threadIdx.x]);
        }
    }
    if (active) {
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int r = group + i * groups;
            if (r >= dk) continue;
            float* dst = record + static_cast<size_t>(r) * dv + col * VEC;
            if constexpr (VEC == 4) *reinterpret_cast<float4*>(dst) = float4{s[i][0], s[i][1], s[i][2], s[i][3]};
            else *dst = s[i][0];
        }
    }
}

constexpr int kDecayWidest = 256;          // the widest key and value of these kernels

static size_t chunk_lds(int dk, int dt, int chunk, int heads_staged) {
    const int krow = (dk + 15) / 16 * 16 + 4;
    return (static_cast<size_t>(heads_staged) * chunk * krow + static_cast<size_t>(chunk) * (16 * dt + 4)) * sizeof(float);
}
static int value_tiles(int dv) {
    int dt = 1;
    while (16 * dt < dv) dt *= 2;
    return dt;
}
// 64 tokens to a chunk while two workgroups of the outputs kernel share a CU's LDS, else 32
static int decay_chunk(int dk, int dv) { return chunk_lds(dk, value_tiles(dv), 64, 2) <= 80 * 1024 ? 64 : 32; }

template <typename K>
static int allow_lds(K kernel, size_t lds) {
    if (lds > 160 * 1024 - 1024) return EGPT_UNSUPPORTED_SIZE;
    if (lds > 48 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                                               static_cast<int>(lds)) != hipSuccess)
        return EGPT_LAUNCH_FAILED;
    return EGPT_OK;
}

template <typename T, int DT, int RT>
static int launch_chunks(const DecayArgs<T>& a, int n_chunks, hipStream_t s) {
    constexpr int C = 16 * RT;
    const size_t lds1 = chunk_lds(a.dk, DT, C, 1), lds2 = chunk_lds(a.dk, DT, C, 2);
    if (int e = allow_lds(chunk_sums_kernel<T, DT, RT>, lds1)) return e;
    if (int e = allow_lds(chunk_outputs_kernel<T, DT, RT>, lds2)) return e;
    const dim3 grid(n_chunks, a.heads);
    chunk_sums_kernel<T, DT, RT><<<grid, 64 * RT, lds1, s>>>(a);
    const size_t per_head = static_cast<size_t>(a.dk) * a.dv;
    if (per_head % 4 == 0)
        chunk_states_kernel<T, 4><<<dim3(a.n_seqs, a.heads, static_cast<unsigned>((per_head / 4 + 255) / 256)), 256, 0, s>>>(a, C);
    else
        chunk_states_kernel<T, 1><<<dim3(a.n_seqs, a.heads, static_cast<unsigned>((per_head + 255) / 256)), 256, 0, s>>>(a, C);
    chunk_outputs_kernel<T, DT, RT><<<grid, 64 * RT, lds2, s>>>(a);
    return EGPT_OK;
}

template <typename T, int RT>
static int launch_chunks_for(const DecayArgs<T>& a, int n_chunks, hipStream_t s) {
    switch (value_tiles(a.dv)) {
        case 1: return launch_chunks<T, 1, RT>(a, n_chunks, s);
        case 2: return launch_chunks<T, 2, RT>(a, n_chunks, s);
        case 4: return launch_chunks<T, 4, RT>(a, n_chunks, s);
        case 8: return launch_chunks<T, 8, RT>(a, n_chunks, s);
        case 16: return launch_chunks<T, 16, RT>(a, n_chunks, s);
        default: return EGPT_UNSUPPORTED_SIZE;
    }
}

template <typename T, int VEC>
static int launch_steps(const DecayArgs<T>& a, hipStream_t s) {
    const int columns = (a.dv + VEC - 1) / VEC;
    // the narrowest workgroup whose threads keep at most 32 values of the state each and that reads a token's values and
    // gates in one round, else the widest
    const int items = 2 * (a.rot_dims / 2 + (a.dk - a.rot_dims + 1) / 2) + 2 * a.dv;
    int threads = 256, rows = 0;
    for (;; threads *= 2) {
        rows = (a.dk + threads / columns - 1) / (threads / columns);
        if ((rows * VEC <= 32 && items <= threads) || threads == 1024) break;
    }
    const int groups = threads / columns;
    const size_t lds = (static_cast<size_t>(2 * a.dk + 4) + (a.dv + 3) / 4 * 4 + a.dv + static_cast<size_t>(groups) * columns * VEC) * sizeof(float);
    if (lds > 48 * 1024) return EGPT_UNSUPPORTED_SIZE;
    const dim3 grid(a.n_seqs, a.heads);
#define EGPT_STEPS(NV)                                                          \
    if (rows <= NV) {                                                           \
        decay_steps_kernel<T, NV, VEC><<<grid, threads, lds, s>>>(a);           \
        return EGPT_OK;                                                         \
    }
    EGPT_STEPS(1) EGPT_STEPS(2) EGPT_STEPS(4) EGPT_STEPS(8) EGPT_STEPS(16)
    if constexpr (VEC == 1) {
        EGPT_STEPS(32) EGPT_STEPS(64)
    }
#undef EGPT_STEPS
    return EGPT_UNSUPPORTED_SIZE;
}

template <typename T>
static int launch_decay(DecayArgs<T>& a, const void* proj, int n_splits, int n_tokens, int n_chunks, hipStream_t s) {
    a.proj.whole = n_splits == 0 ? static_cast<const T*>(proj) : nullptr;
    a.proj.partial = n_splits > 0 ? static_cast<const float*>(proj) : nullptr;
    a.proj.n_splits = n_splits;
    a.proj.split_stride = static_cast<size_t>(n_tokens) * a.proj_width;
    a.flat = n_splits == 1 ? static_cast<const float*>(proj) : (n_splits == 0 && sizeof(T) == 4 ? static_cast<const float*>(proj) : nullptr);
    const bool fours = a.proj_width % 4 == 0 && a.dv % 4 == 0 && a.v_off % 4 == 0 && a.g_off % 4 == 0 &&
                       reinterpret_cast<uintptr_t>(proj) % 16 == 0;
    if (!fours) a.flat = nullptr;
    a.head_fours = a.flat != nullptr && !a.interleaved && a.rot_dims % 8 == 0 && a.dk % 4 == 0 && a.q_off % 4 == 0 && a.k_off % 4 == 0;
    if (n_chunks > 0) return decay_chunk(a.dk, a.dv) == 64 ? launch_chunks_for<T, 4>(a, n_chunks, s) : launch_chunks_for<T, 2>(a, n_chunks, s);
    if (a.dv % 4 == 0) return launch_steps<T, 4>(a, s);
    return launch_steps<T, 1>(a, s);
}

}  // namespace egpt

using namespace egpt;

extern "C" int egpt_decay_chunk(int dk, int dv) {
    return dk > 0 && dv > 0 && dk <= kDecayWidest && dv <= kDecayWidest ? decay_chunk(dk, dv) : 0;
}

extern "C" int egpt_constant_decay(const void* proj, int n_splits, int proj_width, int q_off, int k_off, int v_off, int g_off,
                                   float k_scale, const float* cos_sin, int rot_dims, int interleaved, float mag,
                                   const float* powers, float* states, const int32_t* slots, const unsigned char* fresh,
                                   const int32_t* q_start, const int32_t* q_len, int n_seqs, int n_tokens, float* chunk_states,
                                   int n_chunks, const void* norm_w, float eps, int gate_act, void* out, int heads, int dk, int dv,
                                   int dtype, void* stream) {
    if (!proj || !powers || !states || !slots || !q_start || !q_len || !out || n_splits < 0 || n_seqs <= 0 || n_tokens < 0 ||
        n_chunks < 0 || (n_chunks > 0 && !chunk_states) || heads <= 0 || dk <= 0 || dv <= 0 || q_off < 0 || k_off < 0 || v_off < 0 ||
        g_off < 0 || (dtype != 0 && dtype != 1) || (gate_act != 0 && gate_act != 1))
        return EGPT_BAD_ARGUMENT;
    if (q_off + heads * dk > proj_width || k_off + heads * dk > proj_width || v_off + heads * dv > proj_width ||
        g_off + heads * dv > proj_width)
        return EGPT_BAD_ARGUMENT;
    if (rot_dims < 0 || rot_dims % 2 || rot_dims > dk || (rot_dims > 0 && !cos_sin)) return EGPT_BAD_ARGUMENT;
    if (dk > kDecayWidest || dv > kDecayWidest || heads > 65535) return EGPT_UNSUPPORTED_SIZE;
    if (n_tokens == 0) return EGPT_OK;
    hipStream_t s = static_cast<hipStream_t>(stream);
    int code;
#define EGPT_DECAY(T_)                                                                                                              \
    do {                                                                                                                            \
        DecayArgs<T_> a;                                                                                                            \
        a.proj_width = proj_width; a.q_off = q_off; a.k_off = k_off; a.v_off = v_off; a.g_off = g_off; a.k_scale = k_scale;         \
        a.cos_sin = cos_sin; a.rot_dims = rot_dims; a.interleaved = interleaved; a.mag = mag; a.powers = powers; a.states = states; \
        a.slots = slots; a.fresh = fresh; a.q_start = q_start; a.q_len = q_len; a.n_seqs = n_seqs; a.chunk_states = chunk_states;   \
        a.norm_w = static_cast<const T_*>(norm_w); a.eps = eps; a.gate_act = gate_act; a.out = static_cast<T_*>(out);               \
        a.heads = heads; a.dk = dk; a.dv = dv;                                                                                      \
        code = launch_decay<T_>(a, proj, n_splits, n_tokens, n_chunks, s);                                                          \
    } while (0)
    if (dtype == 0) EGPT_DECAY(float);
    else EGPT_DECAY(bf16_t);
#undef EGPT_DECAY
    if (code != EGPT_OK) return code;
    EGPT_CHECK_LAUNCH();
    return EGPT_OK;
}
