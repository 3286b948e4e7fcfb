// Gated linear attention (see gated_state.cuh): the decays, the walk over many rows, and its entry points.
#include "gated_state.cuh"

namespace ms {

// ---- gated linear attention's decays ------------------------------------------------------------------------
// alpha[t, c] = sigmoid(z)^(1 / tau) with z = b[c] + sum_r wt[r, c] low[t, r], low = R columns of `in` from col on; `wt` is the
// projection transposed, [R, C].  A block takes ROWS rows and 256 channels: a weight is read once for all of its rows.
// (the two-byte builds take the hardware's 32-bit exponential and logarithm: off by units of the last place of a decay)
__device__ __forceinline__ float key_decay_of(float z, float inv_tau) {
#ifdef MS_ELEM_HALF
    const float sp = z < -20.f ? -z : __logf(1.0f + __expf(-z));
    return __expf(-inv_tau * sp);
#else
    return expf(-inv_tau * softplus_f(-z));
#endif
}

template <int ROWS>
__global__ __launch_bounds__(256) void key_decay_kernel(Sums in, int col, const float* __restrict__ wt, const float* __restrict__ b,
                                                        float inv_tau, float* __restrict__ alpha, int T, int C, int R) {
    extern __shared__ float low[];  // [ROWS][R]
    const int t0 = blockIdx.x * ROWS, c = blockIdx.y * 256 + threadIdx.x;
    const int nr = min(ROWS, T - t0);
    for (int i = threadIdx.x; i < nr * R; i += 256) low[i] = sum_at(in, t0 + i / R, col + i % R);
    __syncthreads();
    if (c >= C) return;
    float acc[ROWS];
    const float bias = b[c];
#pragma unroll
    for (int k = 0; k < ROWS; ++k) acc[k] = bias;
#pragma unroll 8
    for (int r = 0; r < R; ++r) {
        const float w = wt[(size_t)r * C + c];
#pragma unroll
        for (int k = 0; k < ROWS; ++k) acc[k] += w * low[(k < nr ? k : 0) * R + r];
    }
#pragma unroll
    for (int k = 0; k < ROWS; ++k)
        if (k < nr) alpha[(size_t)(t0 + k) * C + c] = key_decay_of(acc[k], inv_tau);
}

// ---- gated linear attention over many rows ---------------------------------------------------------------------
// A thread is a value channel and holds its column of S in registers (DP of them; the rows beyond d stay zero).  Tokens come
// WALK_BATCH at a time through LDS; the next batch's numbers are asked for before the current batch is walked.  seg_len 0: a
// block walks all of a request's rows.  Else a request's rows are cut into segments (numbered by piece_of): LOCAL walks
// each from zero and leaves what it adds (carry [numbers, H, d, dvp]) and the product of its decays (cdec [numbers, H, d]),
// the carry kernel replaces what it adds by the state that comes into it, and the second walk makes the outputs.
constexpr int WALK_BATCH = 8;
struct WalkArgs {
    StateArgs a;
    int seg_len;
    float* carry;
    float* cdec;
};

template <int DP, int NT, bool LOCAL>
__global__ __launch_bounds__(NT) void state_walk_kernel(WalkArgs w) {
    constexpr int TB = WALK_BATCH, NW = NT / 64, KPT = TB * DP / NT;
    const StateArgs& a = w.a;
    __shared__ __align__(16) float qs[LOCAL ? 1 : TB][DP], ks[TB][DP], ws[TB][DP];
    __shared__ float vs[TB][NT], os[LOCAL ? 1 : TB][NT], part[TB][NW];
    const int h = blockIdx.y, j = threadIdx.x, d = a.d;
    Piece pc{(int)blockIdx.x, 0};
    if (w.seg_len) pc = piece_of(blockIdx.x, w.seg_len, a.seq_q_start, a.S);
    const int left = a.seq_q_len[pc.s] - pc.first;
    if (left <= 0) return;  // the same for the whole block
    const int n = w.seg_len ? min(left, w.seg_len) : left;
    const bool last = n == left;
    if (LOCAL && last) return;  // nobody needs what the last segment passes on
    const int q0 = a.seq_q_start[pc.s] + pc.first, kh = h / (a.H / a.G);
    const bool live = j < a.dv;
    const size_t head = (size_t)d * a.dvp;
    float* st = a.state + ((size_t)a.seq_slot[pc.s] * a.H + h) * head + j;
    float* pass = w.seg_len ? w.carry + ((size_t)blockIdx.x * a.H + h) * head + j : nullptr;
    float S[DP];
    {
        const float* from = w.seg_len ? pass : st;
#pragma unroll
        for (int i = 0; i < DP; ++i) S[i] = (!LOCAL && live && i < d) ? from[(size_t)i * a.dvp] : 0.f;
    }
    float pq[LOCAL ? 1 : KPT], pk[KPT], pw[KPT], pv[TB], pg[LOCAL ? 1 : TB];
    const float nw = live ? a.norm[j] : 0.f;
    auto fetch = [&](int j0) {  // tokens j0 .. j0 + TB - 1 (the last one again beyond the end)
        // all of one partial sum's loads go out on one straight path, then the next sum's
#pragma unroll
        for (int u = 0; u < KPT; ++u) {
            const int idx = j + u * NT, b = idx / DP, c = idx % DP;
            const int t = q0 + min(j0 + b, n - 1);
            pw[u] = a.decay[((size_t)t * a.H + h) * d + min(c, d - 1)];
        }
        for (int part_sum = 0; part_sum < a.k.n; ++part_sum) {
            const size_t off = part_sum * a.k.stride;  // (q, k, v and gate are columns of the same rows)
#pragma unroll
            for (int u = 0; u < KPT; ++u) {
                const int idx = j + u * NT, b = idx / DP, c = idx % DP;
                const size_t row = off + (size_t)(q0 + min(j0 + b, n - 1)) * a.k.ld + kh * d + min(c, d - 1);
                const float kv = a.k.p[row + a.k_col];
                pk[u] = part_sum ? pk[u] + kv : kv;
                if (!LOCAL) {
                    const float qv = a.k.p[row + a.q_col];
                    pq[u] = part_sum ? pq[u] + qv : qv;
                }
            }
#pragma unroll
            for (int b = 0; b < TB; ++b) {
                const size_t row = off + (size_t)(q0 + min(j0 + b, n - 1)) * a.k.ld + h * a.dv + (live ? j : 0);
                const float vv = a.k.p[row + a.v_col];
                pv[b] = part_sum ? pv[b] + vv : vv;
                if (!LOCAL) {
                    const float gv = a.k.p[row + a.g_col];
                    pg[b] = part_sum ? pg[b] + gv : gv;
                }
            }
        }
    };
    float prod[LOCAL ? (DP + NT - 1) / NT : 1];  // LOCAL: the product of the decays of key channels j, j + NT, ...
#pragma unroll
    for (int u = 0; u < (LOCAL ? (DP + NT - 1) / NT : 1); ++u) prod[u] = 1.f;
    fetch(0);
    for (int j0 = 0; j0 < n; j0 += TB) {
        const int nb = min(TB, n - j0);
        __syncthreads();  // the batch before has been walked by everyone
#pragma unroll
        for (int u = 0; u < KPT; ++u) {
            const int idx = j + u * NT, b = idx / DP, c = idx % DP;
            const bool in = c < d;
            ks[b][c] = in ? pk[u] : 0.f;
            ws[b][c] = in ? pw[u] : 0.f;
            if (!LOCAL) qs[b][c] = in ? pq[u] * a.q_scale : 0.f;
        }
        float gv[LOCAL ? 1 : TB];
#pragma unroll
        for (int b = 0; b < TB; ++b) {
            vs[b][j] = live ? pv[b] : 0.f;
            if (!LOCAL) gv[b] = pg[b];
        }
        __syncthreads();
        if (j0 + TB < n) fetch(j0 + TB);
        if constexpr (LOCAL) {
#pragma unroll
            for (int u = 0; u < (DP + NT - 1) / NT; ++u) {
                const int c = j + u * NT;
                if (c < DP)
                    for (int b = 0; b < nb; ++b) prod[u] *= ws[b][c];
            }
        }
        // the batch's outputs wait in LDS, each in its thread's own place: their norms are worked out together behind the walk
#pragma unroll 1
        for (int b = 0; b < nb; ++b) {
            const float vj = vs[b][j];
            float o0 = 0.f, o1 = 0.f, o2 = 0.f, o3 = 0.f;  // four chains of sums side by side
#pragma unroll
            for (int i = 0; i < DP; i += 4) {
                const float4 k4 = *reinterpret_cast<const float4*>(&ks[b][i]);
                const float4 w4 = *reinterpret_cast<const float4*>(&ws[b][i]);
                S[i] = fmaf(w4.x, S[i], k4.x * vj);
                S[i + 1] = fmaf(w4.y, S[i + 1], k4.y * vj);
                S[i + 2] = fmaf(w4.z, S[i + 2], k4.z * vj);
                S[i + 3] = fmaf(w4.w, S[i + 3], k4.w * vj);
                if (!LOCAL) {
                    const float4 q4 = *reinterpret_cast<const float4*>(&qs[b][i]);
                    o0 = fmaf(q4.x, S[i], o0);
                    o1 = fmaf(q4.y, S[i + 1], o1);
                    o2 = fmaf(q4.z, S[i + 2], o2);
                    o3 = fmaf(q4.w, S[i + 3], o3);
                }
            }
            if (!LOCAL) os[b][j] = (o0 + o1) + (o2 + o3);
        }
        if constexpr (!LOCAL) {
            float ob[TB], ss[TB];
#pragma unroll
            for (int b = 0; b < TB; ++b) {
                ob[b] = (live && b < nb) ? os[b][j] : 0.f;
                ss[b] = wave_sum(ob[b] * ob[b]);
            }
            if constexpr (NW > 1) {  // the head's other waves
                if ((j & 63) == 0) {
#pragma unroll
                    for (int b = 0; b < TB; ++b) part[b][j >> 6] = ss[b];
                }
                __syncthreads();
#pragma unroll
                for (int b = 0; b < TB; ++b) {
                    ss[b] = part[b][0];
#pragma unroll
                    for (int q = 1; q < NW; ++q) ss[b] += part[b][q];
                }
            }
#pragma unroll
            for (int b = 0; b < TB; ++b) {
                const int t = q0 + j0 + b;
                if (b >= nb) continue;
                if (live) a.out[(size_t)t * a.ld_out + h * a.dv + j] = from_f32<elem_t>(ob[b] / sqrtf(ss[b] / (float)a.dv + a.eps) * nw * silu_f(gv[b]));
                if (h == 0) zero_tail(a, t);
            }
        }
    }
    if (LOCAL) {
#pragma unroll
        for (int u = 0; u < (LOCAL ? (DP + NT - 1) / NT : 1); ++u)
            if (j + u * NT < d) w.cdec[((size_t)blockIdx.x * a.H + h) * d + j + u * NT] = prod[u];
    }
    if (j >= a.dvp) return;  // the columns that fill dv up hold zeros
    if (LOCAL) {
#pragma unroll
        for (int i = 0; i < DP; ++i)
            if (i < d) pass[(size_t)i * a.dvp] = S[i];
    } else if (last) {
#pragma unroll
        for (int i = 0; i < DP; ++i)
            if (i < d) st[(size_t)i * a.dvp] = S[i];
    }
}

// Between the two walks: S_in(next) = diag(product of the segment's decays) S_in + what the segment adds, from the slot's state.
__global__ __launch_bounds__(256) void state_carry_kernel(WalkArgs w) {
    const StateArgs& a = w.a;
    const int s = blockIdx.x, h = blockIdx.y, idx = blockIdx.z * 256 + threadIdx.x, head = a.d * a.dvp;
    if (idx >= head) return;
    const int i = idx / a.dvp, base = piece_base(s, w.seg_len, a.seq_q_start);
    const int nseg = (a.seq_q_len[s] + w.seg_len - 1) / w.seg_len;
    float Sin = a.state[((size_t)a.seq_slot[s] * a.H + h) * head + idx];
    for (int seg = 0; seg < nseg; ++seg) {
        const size_t at = (size_t)(base + seg) * a.H + h;
        float* p = w.carry + at * head + idx;
        const bool more = seg + 1 < nseg;
        const float dec = more ? w.cdec[at * a.d + i] : 0.f, add = more ? *p : 0.f;
        *p = Sin;
        Sin = dec * Sin + add;
    }
}

}  // namespace ms

using namespace ms;

extern "C" int ms_gated_state_max_dim() { return MAX_DIM; }
extern "C" int ms_gated_state_max_rank() { return 1536; }  // eight rows of it lie in LDS

extern "C" int ms_key_decay(const float* in, int n_partials, int ld, int col, const float* wt, const float* b, float tau, float* alpha, int T,
                            int C, int R, hipStream_t stream) {
    MS_REQUIRE(T > 0 && C > 0 && R > 0 && n_partials > 0 && col >= 0 && col + R <= ld, "key decay: T=%d C=%d, %d columns at %d of %d", T, C, R, col, ld);
    MS_REQUIRE(R <= ms_gated_state_max_rank(), "key decay: a bottleneck of %d, at most %d", R, ms_gated_state_max_rank());
    MS_REQUIRE(tau > 0.f && in && wt && b && alpha, "key decay: tau %g, or a buffer is missing", (double)tau);
    const Sums rows{in, n_partials, (size_t)T * ld, ld};
    if (T >= 128)
        hipLaunchKernelGGL(key_decay_kernel<8>, dim3(ceil_div(T, 8), ceil_div(C, 256)), dim3(256), (size_t)8 * R * sizeof(float), stream, rows, col,
                           wt, b, 1.0f / tau, alpha, T, C, R);
    else
        hipLaunchKernelGGL(key_decay_kernel<1>, dim3(T, ceil_div(C, 256)), dim3(256), (size_t)R * sizeof(float), stream, rows, col, wt, b, 1.0f / tau,
                           alpha, T, C, R);
    return check_launch("key decay");
}

// Gated linear attention.  rows: float [n_partials, T, ld] with q [H, d], k [H, d], v [H, dv] and gate [H, dv] at their columns;
// alpha float [T, H * d].  single: every request has one row.  seg_len > 0: segments side by side with carry float
// [T / seg_len + S, H, d, dvp] and cdec float [T / seg_len + S, H, d] as workspace.
extern "C" int ms_gated_linear(const float* rows, int n_partials, int ld, int q_col, int k_col, int v_col, int g_col, float q_scale,
                               const float* alpha, const float* norm, float eps, float* state, const int* seq_q_start, const int* seq_q_len,
                               const int* seq_slot, int S, void* out, int ld_out, int T, int H, int d, int dv, int dvp, int single,
                               int seg_len, float* carry, float* cdec, hipStream_t stream) {
    const Sums in{rows, n_partials, (size_t)T * ld, ld};
    const StateArgs a{in, in, in, q_col, k_col, v_col, q_scale, alpha, nullptr, in, g_col, norm, eps, state, seq_q_start, seq_q_len, seq_slot, S,
                      (elem_t*)out, ld_out, T, H, H, d, dv, dvp};
    MS_REQUIRE(n_partials > 0, "gated linear: no rows");
    if (int rc = check_state(a, "gated linear")) return rc;
    if (single) return launch_step<false>(a, stream);
    MS_REQUIRE(seg_len == 0 || (seg_len > 0 && carry && cdec), "gated linear: segments of %d need their workspace", seg_len);
    const WalkArgs w{a, seg_len, carry, cdec};
#define MS_WALK(DP, NT, LOCAL, X) hipLaunchKernelGGL((state_walk_kernel<DP, NT, LOCAL>), dim3(X, H), dim3(NT), 0, stream, w)
#define MS_WALK_N(DP, LOCAL, X)                   \
    do {                                          \
        if (dv <= 64) MS_WALK(DP, 64, LOCAL, X);  \
        else if (dv <= 128) MS_WALK(DP, 128, LOCAL, X); \
        else MS_WALK(DP, 256, LOCAL, X);          \
    } while (0)
#define MS_WALK_D(LOCAL, X)                       \
    do {                                          \
        if (d <= 32) MS_WALK_N(32, LOCAL, X);     \
        else if (d <= 64) MS_WALK_N(64, LOCAL, X); \
        else if (d <= 128) MS_WALK_N(128, LOCAL, X); \
        else MS_WALK_N(256, LOCAL, X);            \
    } while (0)
    if (seg_len == 0) {
        MS_WALK_D(false, S);
        return check_launch("gated linear");
    }
    const int numbers = T / seg_len + S;
    MS_WALK_D(true, numbers);
    if (int rc = check_launch("gated linear, segments from zero")) return rc;
    hipLaunchKernelGGL(state_carry_kernel, dim3(S, H, ceil_div(d * dvp, 256)), dim3(256), 0, stream, w);
    if (int rc = check_launch("gated linear, states between segments")) return rc;
    MS_WALK_D(false, numbers);
#undef MS_WALK_D
#undef MS_WALK_N
#undef MS_WALK
    return check_launch("gated linear, segments");
}
