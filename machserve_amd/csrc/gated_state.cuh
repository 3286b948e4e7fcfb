// Linear attention whose memory is a matrix per head, S [d (key channel), dv (value channel)], under gates that depend on
// the token: gated linear attention (a decay per key channel) and the gated delta rule (a decay per head, and a write that
// first takes away what the state already holds for the key).
//
//   gated linear:  S <- diag(alpha) S + k v^T,                                          o = S^T q
//   delta rule:    S <- g S;  u = beta (v - S^T k);  S <- S + k u^T,                    o = S^T q
//
// Behind both, in the kernel that makes o: a head's o is divided by its root mean square over dv, times one weight for all
// heads, times silu of a gate, rounded to the element type for the output projection.
//
// A step's rows are the tokens of several requests, each request's rows contiguous and in order (seq_q_start, seq_q_len); a
// request's state lives in slot seq_slot[s] of [slots, H, d, dvp] 32-bit floats (dvp: dv filled up to a multiple of 4 with
// zeros) and is read at the start of the request's rows and written back after its last.
//   single rows (decoding)      a block a request and head; the state is read, changed and written once (here)
//   gated linear, many rows     a thread a value channel with its column of S in registers, token after token; long portions
//                               in segments side by side (gated_linear.hip)
//   delta rule, many rows       chunks of 64 tokens as small matrix products (gated_delta.hip)
// Decays, their logarithms, step sizes, unit norms, states and every sum and product here are 32-bit in every build; what a
// token gets depends on the cut of its prompt by rounding only, and on nothing else the step holds.
#pragma once
#include "recurrence.cuh"

namespace ms {

// Rows given as partial sums [n, T, ld]: a projection's output whose parts the reader adds up.
struct Sums {
    const float* p;
    int n;
    size_t stride;
    int ld;
};
__device__ __forceinline__ float sum_at(const Sums& a, int t, int c) {
    const float* src = a.p + (size_t)t * a.ld + c;
    float v = 0.f;
#pragma unroll 8
    for (int i = 0; i < a.n; ++i) v += src[i * a.stride];
    return v;
}

constexpr int MAX_DIM = 256;  // of keys and of values

// ---- what both rules' kernels read --------------------------------------------------------------------------
struct StateArgs {
    Sums q, k, v;            // columns q_col + head * d, k_col + head * d, v_col + h * dv; q and k: of head h / (H / G)
    int q_col, k_col, v_col;
    float q_scale;
    const float* decay;      // gated linear: alpha [T, H * d]; delta rule: lg [T, H]
    const float* beta;       // [T, H] (delta rule)
    Sums gate;               // columns g_col + h * dv
    int g_col;
    const float* norm;       // [dv]
    float eps;
    float* state;            // [slots, H, d, dvp]
    const int* seq_q_start;
    const int* seq_q_len;
    const int* seq_slot;
    int S;
    elem_t* out;             // [T, ld_out], zeros behind H * dv
    int ld_out;
    int T, H, G, d, dv, dvp;
};

__device__ __forceinline__ void zero_tail(const StateArgs& a, int t) {
    for (int c = a.H * a.dv + threadIdx.x; c < a.ld_out; c += blockDim.x) a.out[(size_t)t * a.ld_out + c] = from_f32<elem_t>(0.f);
}

// ---- single rows --------------------------------------------------------------------------------------------
// Request s has the one row s.  A thread holds 4 neighbouring value channels of every RG-th key channel; all of the state is
// asked for at once.  Both products with the old state (S^T k and S^T q) are summed in one pass: with the state's new
// value S' = g S + k u^T,  o = S'^T q = g S^T q + (q . k) u.
template <int CG, int DP, bool DELTA>
__global__ __launch_bounds__(256) void state_step_kernel(StateArgs a) {
    constexpr int RG = 256 / CG, RPT = DP / RG, W = 4 * CG;
    __shared__ float qs[DP], ks[DP], ws[DP], us[W];
    __shared__ float red[DELTA ? 2 : 1][RG][W];
    __shared__ float scratch[4];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, cg = tid % CG, rg = tid / CG;
    const int kh = h / (a.H / a.G);
    float* st = a.state + (((size_t)a.seq_slot[t] * a.H + h) * a.d) * a.dvp + cg * 4;
    const bool col_in = cg * 4 < a.dvp;
    f32x4 S[RPT];
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
        const int i = j * RG + rg;
        S[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
        if (col_in && i < a.d) S[j] = *reinterpret_cast<const f32x4*>(st + (size_t)i * a.dvp);
    }
    // this thread's numbers of q, k, v and the gate (it drops what lies beyond a head): every load on one straight path
    const bool live = tid < a.dv, in = tid < a.d;
    const int ci = min(tid, a.d - 1), cv = min(tid, a.dv - 1);
    const float alpha = DELTA ? 0.f : a.decay[((size_t)t * a.H + h) * a.d + ci];
    float vc = 0.f, zc = 0.f, qv = 0.f, kv = 0.f;
    const float* gp = a.gate.p + (size_t)t * a.gate.ld + a.g_col + h * a.dv + cv;
    if constexpr (DELTA) {
        qv = a.q.p[(size_t)t * a.q.ld + a.q_col + kh * a.d + ci];
        kv = a.k.p[(size_t)t * a.k.ld + a.k_col + kh * a.d + ci];
        vc = a.v.p[(size_t)t * a.v.ld + a.v_col + h * a.dv + cv];
#pragma unroll 4
        for (int p = 0; p < a.gate.n; ++p) zc += gp[p * a.gate.stride];
    } else {  // columns of the same rows
        const float* rp = a.q.p + (size_t)t * a.q.ld;
#pragma unroll 4
        for (int p = 0; p < a.q.n; ++p) {
            const float* r = rp + p * a.q.stride;
            qv += r[a.q_col + kh * a.d + ci];
            kv += r[a.k_col + kh * a.d + ci];
            vc += r[a.v_col + h * a.dv + cv];
            zc += gp[p * a.gate.stride];
        }
    }
    qv = in ? qv * a.q_scale : 0.f;
    kv = in ? kv : 0.f;
    if (!live) vc = 0.f;
    if (tid < DP) {
        qs[tid] = qv;
        ks[tid] = kv;
        if (!DELTA) ws[tid] = in ? alpha : 0.f;
    }
    float qk = qv * kv;
    const float g = DELTA ? expf(a.decay[(size_t)t * a.H + h]) : 1.f, beta = DELTA ? a.beta[(size_t)t * a.H + h] : 1.f;
    if (!DELTA && tid < W) us[tid] = vc;
    if (DELTA) qk = block_sum<256>(qk, scratch);  // (a barrier: the rows are in LDS)
    else __syncthreads();
    {
        f32x4 pk = (f32x4){0.f, 0.f, 0.f, 0.f}, pq = pk;
        const f32x4 u4 = DELTA ? pk : *reinterpret_cast<const f32x4*>(&us[cg * 4]);
#pragma unroll
        for (int j = 0; j < RPT; ++j) {
            const int i = j * RG + rg;
            const float kv = ks[i], qv = qs[i];
            if (DELTA) pk += S[j] * kv;
            else S[j] = S[j] * ws[i] + u4 * kv;
            pq += S[j] * qv;
        }
        *reinterpret_cast<f32x4*>(&red[0][rg][cg * 4]) = pq;
        if constexpr (DELTA) *reinterpret_cast<f32x4*>(&red[1][rg][cg * 4]) = pk;
    }
    __syncthreads();
    float o = 0.f;
    if (tid < W) {
        float sk = 0.f;
#pragma unroll
        for (int r = 0; r < RG; ++r) {
            o += red[0][r][tid];
            if constexpr (DELTA) sk += red[1][r][tid];
        }
        if constexpr (DELTA) {
            const float u = beta * (vc - g * sk);
            us[tid] = u;
            o = g * o + qk * u;
        }
    }
    const float ss = block_sum<256>(live ? o * o : 0.f, scratch);
    if constexpr (DELTA) {  // (block_sum's barriers: the writes are in LDS)
        const f32x4 u4 = *reinterpret_cast<const f32x4*>(&us[cg * 4]);
#pragma unroll
        for (int j = 0; j < RPT; ++j) S[j] = S[j] * g + u4 * ks[j * RG + rg];
    }
#pragma unroll
    for (int j = 0; j < RPT; ++j) {
        const int i = j * RG + rg;
        if (col_in && i < a.d) *reinterpret_cast<f32x4*>(st + (size_t)i * a.dvp) = S[j];
    }
    if (live) a.out[(size_t)t * a.ld_out + h * a.dv + tid] = from_f32<elem_t>(o / sqrtf(ss / (float)a.dv + a.eps) * a.norm[tid] * silu_f(zc));
    if (h == 0) zero_tail(a, t);
}

inline int check_state(const StateArgs& a, const char* what) {
    MS_REQUIRE(a.T > 0 && a.S > 0 && a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.H <= 65535, "%s: T=%d S=%d, %d heads over %d", what, a.T, a.S, a.H, a.G);
    MS_REQUIRE(a.d > 0 && a.d <= MAX_DIM && a.dv > 0 && a.dv <= MAX_DIM, "%s: heads of %d and %d, at most %d", what, a.d, a.dv, MAX_DIM);
    MS_REQUIRE(a.dvp >= a.dv && a.dvp % 4 == 0 && a.dvp < a.dv + 4 && a.ld_out >= a.H * a.dv, "%s: values of %d in %d, rows of %d", what, a.dv, a.dvp, a.ld_out);
    MS_REQUIRE(a.q_col >= 0 && a.q_col + a.G * a.d <= a.q.ld && a.k_col >= 0 && a.k_col + a.G * a.d <= a.k.ld && a.v_col >= 0 &&
                   a.v_col + a.H * a.dv <= a.v.ld && a.g_col >= 0 && a.g_col + a.H * a.dv <= a.gate.ld,
               "%s: columns beyond the rows", what);
    MS_REQUIRE(a.q.p && a.k.p && a.v.p && a.gate.p && a.decay && a.norm && a.state && a.seq_q_start && a.seq_q_len && a.seq_slot && a.out,
               "%s: a buffer is missing", what);
    MS_REQUIRE((reinterpret_cast<uintptr_t>(a.state)) % 16 == 0, "%s: the state must be 16-byte aligned", what);
    return 0;
}

template <bool DELTA>
inline int launch_step(const StateArgs& a, hipStream_t stream) {
    MS_REQUIRE(a.S == a.T, "single rows: %d rows of %d requests", a.T, a.S);
    const dim3 grid(a.T, a.H);
#define MS_STEP(CG, DP) hipLaunchKernelGGL((state_step_kernel<CG, DP, DELTA>), grid, dim3(256), 0, stream, a)
#define MS_STEP_D(CG)                    \
    do {                                 \
        if (a.d <= 32) MS_STEP(CG, 32);  \
        else if (a.d <= 64) MS_STEP(CG, 64); \
        else if (a.d <= 128) MS_STEP(CG, 128); \
        else MS_STEP(CG, 256);           \
    } while (0)
    if (a.dv <= 32) MS_STEP_D(8);
    else if (a.dv <= 64) MS_STEP_D(16);
    else if (a.dv <= 128) MS_STEP_D(32);
    else MS_STEP_D(64);
#undef MS_STEP_D
#undef MS_STEP
    return check_launch("gated state, single rows");
}

}  // namespace ms
