// The gated delta rule (see gated_state.cuh): its rows, the chunks over many rows, and its entry points.
#include "gated_state.cuh"

namespace ms {

constexpr int MAX_TAPS = 16;

// ---- the delta rule's rows: convolution, unit norms, step sizes and decays -----------------------------------
// in: q [G, d], k [G, d], v [H, dv], gate [H, dv], then at b_col and a_col one number a head each.  On every channel of q, k
// and v a causal convolution over time (w [C, taps], last tap the current row; earlier inputs from state [slots, taps - 1, C],
// oldest first) and SiLU; q and k of a head divided by sqrt(sum of squares + 1e-6), q times q_scale; beta = sigmoid(b);
// lg = -exp(a_log) softplus(a + dt_bias), the logarithm of the head's decay.
struct DeltaRowsArgs {
    Sums in;
    const float* w;
    float* state;
    const float* a_log;    // [H]
    const float* dt_bias;  // [H]
    const int* seq_q_start;
    const int* seq_q_len;
    const int* seq_slot;
    int S;
    float* q;     // [T, G * d]
    float* k;     // [T, G * d]
    float* v;     // [T, H * dv]
    float* beta;  // [T, H]
    float* lg;    // [T, H]
    int T, H, G, d, dv, taps, b_col, a_col;
    float q_scale;
};
constexpr float UNIT_EPS = 1e-6f;

// A wave takes one head of q, k or v (or the step sizes and decays) over ROWS rows; a lane EPL of its channels, whose last
// inputs it keeps, so that every input is read once (and again at the start of a block's rows).  A request with a single
// row gets its state brought up to date here: nobody else reads it.
template <int TAPS, int EPL, int ROWS>
__global__ __launch_bounds__(256) void delta_rows_kernel(DeltaRowsArgs a) {
    const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int t0 = blockIdx.x * ROWS;
    if (unit > 2 * a.G + a.H) return;
    if (unit == 2 * a.G + a.H) {
        for (int r = 0; r < ROWS && t0 + r < a.T; ++r)
            for (int h = lane; h < a.H; h += 64) {
                const int t = t0 + r;
                a.beta[(size_t)t * a.H + h] = sigmoid_f(sum_at(a.in, t, a.b_col + h));
                a.lg[(size_t)t * a.H + h] = -expf(a.a_log[h]) * softplus_f(sum_at(a.in, t, a.a_col + h) + a.dt_bias[h]);
            }
        return;
    }
    const bool is_v = unit >= 2 * a.G;
    const int dim = is_v ? a.dv : a.d;
    const int c0 = is_v ? 2 * a.G * a.d + (unit - 2 * a.G) * a.dv : unit * a.d;  // first channel, also the column of `in`
    const int C = 2 * a.G * a.d + a.H * a.dv, keep = a.taps - 1;
    float wv[EPL][TAPS], win[EPL][TAPS] = {};  // index b: the input b rows back; win[.][0] is not kept
    int ch[EPL];
    bool on[EPL];
#pragma unroll
    for (int e = 0; e < EPL; ++e) {
        on[e] = lane + e * 64 < dim;
        ch[e] = c0 + (on[e] ? lane + e * 64 : 0);
#pragma unroll
        for (int b = 0; b < TAPS; ++b) {
            const float w = a.w[(size_t)ch[e] * a.taps + max(keep - b, 0)];
            wv[e][b] = b <= keep ? w : 0.f;
        }
    }
    int s = seq_of_row(t0, a.seq_q_start, a.S);
    int q0 = a.seq_q_start[s], len = a.seq_q_len[s];
    auto load_window = [&](int t) {  // the inputs before row t
        const float* st = a.state + (size_t)a.seq_slot[s] * keep * C;
        if (keep == 0) return;
        // a place reads the step's rows or the state (the same for the whole wave): the address is chosen, not the load
        for (int p = 0; p < a.in.n; ++p)
#pragma unroll
            for (int b = 1; b < TAPS; ++b) {
                const int back = min(b, keep), idx = t - back - q0;  // counted from the request's first row
                const bool fresh = idx >= 0;
                const float* src = fresh ? a.in.p + p * a.in.stride + (size_t)(t - back) * a.in.ld : st + (size_t)(keep + idx) * C;
                const bool counts = b <= keep && (fresh || p == 0);
#pragma unroll
                for (int e = 0; e < EPL; ++e) {
                    const float v = src[ch[e]];
                    win[e][b] = (p ? win[e][b] : 0.f) + (counts ? v : 0.f);
                }
            }
    };
    float x[ROWS][EPL];  // the rows' own inputs, all of one partial sum's loads on one straight path
#pragma unroll
    for (int r = 0; r < ROWS; ++r)
#pragma unroll
        for (int e = 0; e < EPL; ++e) x[r][e] = 0.f;
    for (int p = 0; p < a.in.n; ++p)
#pragma unroll
        for (int r = 0; r < ROWS; ++r)
#pragma unroll
            for (int e = 0; e < EPL; ++e) x[r][e] += a.in.p[p * a.in.stride + (size_t)min(t0 + r, a.T - 1) * a.in.ld + ch[e]];
    load_window(t0);
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
        const int t = t0 + r;
        if (t >= a.T) return;
        if (t >= q0 + len) {  // the next request's first row
            do {
                ++s;
                q0 = a.seq_q_start[s];
                len = a.seq_q_len[s];
            } while (len == 0 && s + 1 < a.S);
            load_window(t);
        }
        float y[EPL], ss = 0.f;
#pragma unroll
        for (int e = 0; e < EPL; ++e) {
            const float cur = x[r][e];
            float acc = wv[e][0] * cur;
#pragma unroll
            for (int b = 1; b < TAPS; ++b) acc += wv[e][b] * win[e][b];
#pragma unroll
            for (int b = TAPS - 1; b > 1; --b) win[e][b] = win[e][b - 1];
            if constexpr (TAPS > 1) win[e][1] = cur;
            y[e] = on[e] ? silu_f(acc) : 0.f;
            ss += y[e] * y[e];
        }
        if (len == 1 && keep > 0) {
            float* st = a.state + (size_t)a.seq_slot[s] * keep * C;
#pragma unroll
            for (int e = 0; e < EPL; ++e)
                if (on[e]) {
#pragma unroll
                    for (int b = 1; b < TAPS; ++b)
                        if (b <= keep) st[(size_t)(keep - b) * C + ch[e]] = win[e][b];
                }
        }
        if (!is_v) {
            ss = wave_sum(ss);
            const float f = (unit < a.G ? a.q_scale : 1.0f) / sqrtf(ss + UNIT_EPS);
            float* dst = (unit < a.G ? a.q + (size_t)t * a.G * a.d + unit * a.d : a.k + (size_t)t * a.G * a.d + (unit - a.G) * a.d);
#pragma unroll
            for (int e = 0; e < EPL; ++e)
                if (on[e]) dst[lane + e * 64] = y[e] * f;
        } else {
            float* dst = a.v + (size_t)t * a.H * a.dv + (unit - 2 * a.G) * a.dv;
#pragma unroll
            for (int e = 0; e < EPL; ++e)
                if (on[e]) dst[lane + e * 64] = y[e];
        }
    }
}

// The convolution's state after the step, for requests of several rows: their last taps - 1 inputs, old ones where the
// step brought fewer.  Comes after the kernel above.
__global__ __launch_bounds__(256) void delta_conv_state_kernel(Sums in, float* __restrict__ state, const int* __restrict__ seq_q_start,
                                                               const int* __restrict__ seq_q_len, const int* __restrict__ seq_slot, int C, int taps) {
    const int s = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    const int n = seq_q_len[s], q0 = seq_q_start[s], keep = taps - 1;
    if (c >= C || n <= 1) return;
    float* st = state + (size_t)seq_slot[s] * keep * C + c;
    float v[MAX_TAPS];
    for (int i = 0; i < keep; ++i) {
        const int idx = n - keep + i;  // among the step's rows; negative: an older input
        v[i] = idx >= 0 ? sum_at(in, q0 + idx, c) : st[(size_t)(keep + idx) * C];
    }
    for (int i = 0; i < keep; ++i) st[(size_t)i * C] = v[i];
}

// ---- the delta rule over many rows: chunks of 64 tokens -----------------------------------------------------------
// For the tokens i, j = 0 .. n - 1 of a chunk, L_i = sum of lg up to i (so exp(L_i - L_j) is the decay from j to i), and the
// state S before the chunk, unrolling the rule gives
//     (I + A) U = diag(beta) V - diag(beta e^L) K S,     A_ij = beta_i exp(L_i - L_j) (k_i . k_j)  for j < i, else 0
//     o_i = e^(L_i) S^T q_i + sum_{j <= i} exp(L_i - L_j) (q_i . k_j) u_j
//     S after = e^(L_n) S + sum_j exp(L_n - L_j) k_j u_j^T.
// delta_solve (all chunks side by side): W = (I + A)^-1 diag(beta e^L) K and U0 = (I + A)^-1 diag(beta) V by forward
// substitution in blocks of 16 tokens; delta_pass (a request's chunks in order): U = U0 - W S, the state before every chunk and
// the state after the last; delta_out (all chunks side by side): o, its norm and gate.  All products run on the matrix
// cores' 32-bit form.  The order of sums within a chunk does not depend on where the portion was cut other than through
// the chunk's own start.
constexpr int CH = 64;        // tokens of a chunk: one a lane where their decays are summed
constexpr int SL = 64;        // channels of q and k that a block holds in LDS at a time
constexpr int LDP = SL + 4;   // their row stride

// What the kernels hand on lies per (chunk's number, head) in whole tiles of 16, zeros beyond the chunk's tokens and the head's
// channels, with the index that an operand's four steps run over innermost: every load of an operand is 16 bytes, without
// conditions.
struct DeltaChunkArgs {
    StateArgs a;   // q and k already unit vectors and scaled: one partial sum, columns from 0
    float* W;      // [numbers, H, CH, dk16]
    float* Kt;     // [numbers, H, dk16, CH]: exp(L_n - L_j) k_j
    float* U0;     // [numbers, H, dv16, CH]
    float* U;      // [numbers, H, dv16, CH]
    float* Sb;     // [numbers, H, dv16, dk16]: the state before each chunk
    float* total;  // [numbers, H]: exp(L_n)
    int dk16, dv16;
};

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// lane i: the sum of v over lanes 0 .. i
__device__ __forceinline__ float lane_sums(float v, int lane) {
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
        const float up = __shfl_up(v, o, WAVE);
        if (lane >= o) v += up;
    }
    return v;
}

// lane i: the sum of lg of the chunk's tokens up to i (tokens beyond n add nothing)
__device__ __forceinline__ float decay_sums(const float* __restrict__ lg, int t0, int n, int H, int h, int lane) {
    return lane_sums(lane < n ? lg[(size_t)(t0 + lane) * H + h] : 0.f, lane);
}

// CH rows of channels c0 .. c0 + SL of `src` (row stride ld), zeros beyond n rows and d channels: asked for here, a number of
// every fourth row a thread ...
struct Slice {
    float v[CH * SL / 256];
};
__device__ __forceinline__ void ask_slice(Slice& t, const float* __restrict__ src, size_t ld, int c0, int n, int d) {
    const int c = min(c0 + (int)(threadIdx.x % SL), d - 1), r0 = threadIdx.x / SL;
#pragma unroll
    for (int u = 0; u < CH * SL / 256; ++u) t.v[u] = src[(size_t)min(r0 + u * (256 / SL), n - 1) * ld + c];
}
// ... and put into LDS here
__device__ __forceinline__ void put_slice(float* dst, const Slice& t, int c0, int n, int d) {
    const int c = threadIdx.x % SL, r0 = threadIdx.x / SL;
#pragma unroll
    for (int u = 0; u < CH * SL / 256; ++u) {
        const int r = r0 + u * (256 / SL);
        dst[r * LDP + c] = (r < n && c0 + c < d) ? t.v[u] : 0.f;
    }
}

// The lower triangle's ten tiles of 16 x 16 over four waves: tile number -> row and column tile.
__device__ __forceinline__ void lower_tile(int t, int& rt, int& ct) {
    rt = t >= 6 ? 3 : t >= 3 ? 2 : t >= 1 ? 1 : 0;
    ct = t - (rt * (rt + 1)) / 2;
}

__global__ __launch_bounds__(256) void delta_solve_kernel(DeltaChunkArgs p) {
    const StateArgs& a = p.a;
    __shared__ __align__(16) float Ks[CH * LDP], As[CH * LDP];
    __shared__ float Ls[CH], bs[CH];
    const Piece pc = piece_of(blockIdx.x, CH, a.seq_q_start, a.S);
    const int left = a.seq_q_len[pc.s] - pc.first;
    if (left <= 0) return;  // the same for the whole block
    const int n = min(left, CH), t0 = a.seq_q_start[pc.s] + pc.first, h = blockIdx.y, kh = h / (a.H / a.G);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, grp = lane >> 4;
    const size_t ldk = (size_t)a.G * a.d;
    const float* kp = a.k.p + (size_t)t0 * ldk + (size_t)kh * a.d;
    const size_t at = (size_t)blockIdx.x * a.H + h;
    if (wave == 0) {
        Ls[lane] = decay_sums(a.decay, t0, n, a.H, h, lane);
        bs[lane] = lane < n ? a.beta[(size_t)(t0 + lane) * a.H + h] : 0.f;
    }
    const int used = (n + 15) / 16, tiles = used * (used + 1) / 2;  // row tiles with tokens, and their lower triangle
    // Right sides, two tiles of 16 columns a wave at a time: K's (filled up to dk16 with zeros), then V's.  The first two are
    // asked for here, ahead of all else.
    const size_t ldv = (size_t)a.H * a.dv;
    const int cts = (p.dk16 + p.dv16) / 16;
    int ct0 = wave, c[2];
    bool is_k[2], in[2];
    f32x4 X[2][4];
    auto ask = [&]() {
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            const int ct = min(ct0 + u * 4, cts - 1);
            is_k[u] = ct * 16 < p.dk16;
            c[u] = ct * 16 - (is_k[u] ? 0 : p.dk16) + r16;
            in[u] = c[u] < (is_k[u] ? a.d : a.dv);
            const float* src = is_k[u] ? kp + (in[u] ? c[u] : 0) : a.v.p + (size_t)t0 * ldv + (size_t)h * a.dv + (in[u] ? c[u] : 0);
            const size_t ld = is_k[u] ? ldk : ldv;
#pragma unroll
            for (int b = 0; b < 4; ++b)
#pragma unroll
                for (int i = 0; i < 4; ++i) X[u][b][i] = src[(size_t)min(b * 16 + grp * 4 + i, n - 1) * ld];
        }
    };
    ask();
    f32x4 acc[3];
#pragma unroll
    for (int u = 0; u < 3; ++u) acc[u] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int c0 = 0; c0 < a.d; c0 += SL) {
        Slice ks;
        ask_slice(ks, kp, ldk, c0, n, a.d);
        if (c0) __syncthreads();
        put_slice(Ks, ks, c0, n, a.d);
        __syncthreads();
        const float e = expf(Ls[CH - 1] - Ls[lane]);  // (the sums stay as they are beyond the chunk's end)
        for (int c = wave; c < min(SL, p.dk16 - c0); c += 4) p.Kt[(at * p.dk16 + c0 + c) * CH + lane] = e * Ks[lane * LDP + c];
#pragma unroll
        for (int u = 0; u < 3; ++u) {
            const int tile = wave + u * 4;
            if (tile >= tiles) continue;
            int rt, ct;
            lower_tile(tile, rt, ct);
#pragma unroll
            for (int kk = 0; kk < SL / 16; ++kk) {
                const f32x4 x = *reinterpret_cast<const f32x4*>(&Ks[(rt * 16 + r16) * LDP + kk * 16 + grp * 4]);
                const f32x4 y = *reinterpret_cast<const f32x4*>(&Ks[(ct * 16 + r16) * LDP + kk * 16 + grp * 4]);
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[u] = mfma_f32(x[i], y[i], acc[u]);
            }
        }
    }
    if (tid == 0) p.total[at] = expf(Ls[CH - 1]);
#pragma unroll
    for (int u = 0; u < 3; ++u) {
        const int tile = wave + u * 4;
        if (tile >= tiles) continue;
        int rt, ct;
        lower_tile(tile, rt, ct);
        const int j = ct * 16 + r16;
#pragma unroll
        for (int ii = 0; ii < 4; ++ii) {
            const int i = rt * 16 + grp * 4 + ii;
            As[i * LDP + j] = j < i ? bs[i] * expf(Ls[i] - Ls[j]) * acc[u][ii] : 0.f;
        }
    }
    __syncthreads();
    // the diagonal's blocks are replaced by the inverses of I + A there: a wave a block, a lane a column
    if (wave < used && lane < 16) {
        float* D = As + wave * 16 * LDP + wave * 16;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float v = i == lane ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; ++j) v = fmaf(-D[i * LDP + j], x[j], v);
            x[i] = v;
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) D[i * LDP + lane] = x[i];
    }
    __syncthreads();
    // A block of 16 solved rows is an accumulator, which serves the blocks below as an operand as it is (see delta_pass_kernel).
    for (; ct0 < cts; ct0 += 8) {
        if (ct0 != wave) ask();
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int b = 0; b < 4; ++b)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int r = b * 16 + grp * 4 + i;
                    X[u][b][i] = in[u] ? X[u][b][i] * (bs[r] * (is_k[u] ? expf(Ls[r]) : 1.f)) : 0.f;  // (beta is zero beyond the chunk's end)
                }
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            if (b >= used) continue;
#pragma unroll
            for (int e = 0; e < b; ++e) {
                const f32x4 m = *reinterpret_cast<const f32x4*>(&As[(b * 16 + r16) * LDP + e * 16 + grp * 4]);
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int u = 0; u < 2; ++u) X[u][b] = mfma_f32(-m[i], X[u][e][i], X[u][b]);
            }
            const f32x4 m = *reinterpret_cast<const f32x4*>(&As[(b * 16 + r16) * LDP + b * 16 + grp * 4]);
            f32x4 Y[2] = {(f32x4){0.f, 0.f, 0.f, 0.f}, (f32x4){0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int u = 0; u < 2; ++u) Y[u] = mfma_f32(m[i], X[u][b][i], Y[u]);
#pragma unroll
            for (int u = 0; u < 2; ++u) X[u][b] = Y[u];
        }
        // tokens beyond the chunk's end and columns beyond the head came out as zeros
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            if (ct0 + u * 4 >= cts) continue;
            if (is_k[u]) {
                float* dst = p.W + at * CH * p.dk16 + c[u];
#pragma unroll
                for (int b = 0; b < 4; ++b)
#pragma unroll
                    for (int i = 0; i < 4; ++i) dst[(size_t)(b * 16 + grp * 4 + i) * p.dk16] = X[u][b][i];
            } else {
                float* dst = p.U0 + (at * p.dv16 + c[u]) * CH + grp * 4;
#pragma unroll
                for (int b = 0; b < 4; ++b) *reinterpret_cast<f32x4*>(dst + b * 16) = X[u][b];
            }
        }
    }
}

// A block walks a request's chunks for one head and 16 value channels.  Wave w holds the state's rows of the 16-wide tiles
// w * KT .. w * KT + KT - 1 as accumulators, which serve as operands as they are: lane (grp, r16) holds rows grp * 4 + i of
// column r16, and supplies them as the four steps i of a product over those rows.
// FULL: every wave's tiles lie within the head.  Operands are asked for a chunk ahead, into one of two sets of registers in
// turn, and no load or store of the loop stands behind a condition.
template <int KT>
struct PassOperands {
    f32x4 W[4][KT], K[KT][4], U[4];
    float g;
};

template <int KT, bool FULL>
__global__ __launch_bounds__(256) void delta_pass_kernel(DeltaChunkArgs p) {
    const StateArgs& a = p.a;
    __shared__ f32x4 part[2][4][4][64];
    // heads first: the blocks of one head, which read the same W and k, lie on one XCD where the heads are a multiple of 8
    const int s = blockIdx.z, h = blockIdx.x, n0 = blockIdx.y * 16;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, grp = lane >> 4;
    const int len = a.seq_q_len[s];
    if (len <= 0) return;
    const int col = n0 + r16;
    const bool col_in = col < a.dv;
    float* st = a.state + ((size_t)a.seq_slot[s] * a.H + h) * a.d * a.dvp;
    f32x4 S[KT];
    int k0[KT], kk[KT];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
        k0[kt] = (wave * KT + kt) * 16;
        kk[kt] = FULL ? k0[kt] : min(k0[kt], p.dk16 - 16);  // a tile beyond the head reads its last one; its state stays zero
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int k = k0[kt] + grp * 4 + i;
            S[kt][i] = (k < a.d && col_in) ? st[(size_t)k * a.dvp + col] : 0.f;
        }
    }
    const int nch = (len + CH - 1) / CH;
    const size_t at0 = (size_t)piece_base(s, CH, a.seq_q_start) * a.H + h, step = a.H;
    PassOperands<KT> A, B;
    auto fetch = [&](PassOperands<KT>& o, int ch) {
        const size_t at = at0 + ch * step;
        o.g = p.total[at];
        const float* wp = p.W + (at * CH + r16) * p.dk16 + grp * 4;
        const float* kp = p.Kt + (at * p.dk16 + r16) * CH + grp * 4;
        const float* up = p.U0 + (at * p.dv16 + col) * CH + grp * 4;
#pragma unroll
        for (int rt = 0; rt < 4; ++rt)
#pragma unroll
            for (int kt = 0; kt < KT; ++kt) o.W[rt][kt] = *reinterpret_cast<const f32x4*>(wp + (size_t)rt * 16 * p.dk16 + kk[kt]);
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
            o.U[rt] = *reinterpret_cast<const f32x4*>(up + rt * 16);
#pragma unroll
            for (int kt = 0; kt < KT; ++kt) o.K[kt][rt] = *reinterpret_cast<const f32x4*>(kp + (size_t)kk[kt] * CH + rt * 16);
        }
    };
    auto chunk = [&](PassOperands<KT>& cur, PassOperands<KT>& next, int ch, int buf) {
        const size_t at = at0 + ch * step;
        fetch(next, min(ch + 1, nch - 1));
        __builtin_amdgcn_sched_barrier(0);  // the loads go out ahead of the products, not among them
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
            f32x4 ws = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kt = 0; kt < KT; ++kt)
#pragma unroll
                for (int i = 0; i < 4; ++i) ws = mfma_f32(cur.W[rt][kt][i], S[kt][i], ws);
            part[buf][wave][rt][lane] = ws;
        }
        // the state before the chunk, for the kernel that makes the outputs
#pragma unroll
        for (int kt = 0; kt < KT; ++kt)
            if (FULL || k0[kt] < p.dk16) *reinterpret_cast<f32x4*>(p.Sb + (at * p.dv16 + col) * p.dk16 + k0[kt] + grp * 4) = S[kt];
        __syncthreads();  // the waves' shares of W S are in LDS (the other half was read before they were written)
        f32x4 own = cur.U[0];
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
            f32x4 ws = part[buf][0][rt][lane];
#pragma unroll
            for (int w = 1; w < 4; ++w) ws += part[buf][w][rt][lane];
            cur.U[rt] -= ws;
            own = rt == wave ? cur.U[rt] : own;
        }
        *reinterpret_cast<f32x4*>(p.U + (at * p.dv16 + col) * CH + wave * 16 + grp * 4) = own;  // a wave leaves a quarter
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {
            S[kt] *= cur.g;
            if (!FULL && k0[kt] >= p.dk16)
#pragma unroll
                for (int rt = 0; rt < 4; ++rt) cur.K[kt][rt] = (f32x4){0.f, 0.f, 0.f, 0.f};
        }
#pragma unroll
        for (int rt = 0; rt < 4; ++rt)
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int kt = 0; kt < KT; ++kt) S[kt] = mfma_f32(cur.K[kt][rt][i], cur.U[rt][i], S[kt]);
    };
    fetch(A, 0);
    for (int ch = 0; ch < nch; ch += 2) {
        chunk(A, B, ch, 0);
        if (ch + 1 >= nch) break;
        chunk(B, A, ch + 1, 1);
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int k = k0[kt] + grp * 4 + i;
            if (k < a.d && col_in) st[(size_t)k * a.dvp + col] = S[kt][i];
        }
}

// Wave w makes the value channels of the 16-wide tiles w, w + 4, ... (CT of them) for all of a chunk's tokens.
template <int CT>
__global__ __launch_bounds__(256) void delta_out_kernel(DeltaChunkArgs p) {
    const StateArgs& a = p.a;
    __shared__ __align__(16) float Qs[CH * LDP], Ks[CH * LDP];
    __shared__ float Ls[CH], rows[4][CH];
    const Piece pc = piece_of(blockIdx.x, CH, a.seq_q_start, a.S);
    const int left = a.seq_q_len[pc.s] - pc.first;
    if (left <= 0) return;  // the same for the whole block
    const int n = min(left, CH), t0 = a.seq_q_start[pc.s] + pc.first, h = blockIdx.y, kh = h / (a.H / a.G);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, grp = lane >> 4;
    const int used = (n + 15) / 16, tiles = used * (used + 1) / 2;
    const size_t ldk = (size_t)a.G * a.d;
    const float* qp = a.q.p + (size_t)t0 * ldk + (size_t)kh * a.d;
    const float* kp = a.k.p + (size_t)t0 * ldk + (size_t)kh * a.d;
    const size_t at = (size_t)blockIdx.x * a.H + h;
    if (wave == 0) Ls[lane] = decay_sums(a.decay, t0, n, a.H, h, lane);
    f32x4 O[4][CT], P[3];
#pragma unroll
    for (int u = 0; u < 3; ++u) P[u] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
        for (int c = 0; c < CT; ++c) O[rt][c] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int c0 = 0; c0 < a.d; c0 += SL) {
        Slice qs, ks;
        ask_slice(qs, qp, ldk, c0, n, a.d);
        ask_slice(ks, kp, ldk, c0, n, a.d);
        f32x4 B[SL / 16][CT];  // the state's rows c0 .. c0 + SL of this wave's columns (rows beyond it meet zeros of q)
#pragma unroll
        for (int kk = 0; kk < SL / 16; ++kk)
#pragma unroll
            for (int c = 0; c < CT; ++c)
                B[kk][c] = *reinterpret_cast<const f32x4*>(p.Sb + (at * p.dv16 + min((wave + 4 * c) * 16, p.dv16 - 16) + r16) * p.dk16 +
                                                           min(c0 + kk * 16, p.dk16 - 16) + grp * 4);
        if (c0) __syncthreads();
        put_slice(Qs, qs, c0, n, a.d);
        put_slice(Ks, ks, c0, n, a.d);
        __syncthreads();
#pragma unroll
        for (int u = 0; u < 3; ++u) {
            const int tile = wave + u * 4;
            if (tile >= tiles) continue;
            int rt, ct;
            lower_tile(tile, rt, ct);
#pragma unroll
            for (int kk = 0; kk < SL / 16; ++kk) {
                const f32x4 x = *reinterpret_cast<const f32x4*>(&Qs[(rt * 16 + r16) * LDP + kk * 16 + grp * 4]);
                const f32x4 y = *reinterpret_cast<const f32x4*>(&Ks[(ct * 16 + r16) * LDP + kk * 16 + grp * 4]);
#pragma unroll
                for (int i = 0; i < 4; ++i) P[u] = mfma_f32(x[i], y[i], P[u]);
            }
        }
#pragma unroll
        for (int rt = 0; rt < 4; ++rt) {
            if (rt >= used) continue;
#pragma unroll
            for (int kk = 0; kk < SL / 16; ++kk) {
                const f32x4 x = *reinterpret_cast<const f32x4*>(&Qs[(rt * 16 + r16) * LDP + kk * 16 + grp * 4]);
#pragma unroll
                for (int c = 0; c < CT; ++c)
#pragma unroll
                    for (int i = 0; i < 4; ++i) O[rt][c] = mfma_f32(x[i], B[kk][c][i], O[rt][c]);
            }
        }
    }
    __syncthreads();  // everyone has read the keys: the scores take their place
    float* Ps = Ks;
#pragma unroll
    for (int u = 0; u < 3; ++u) {
        const int tile = wave + u * 4;
        if (tile >= tiles) continue;
        int rt, ct;
        lower_tile(tile, rt, ct);
        const int j = ct * 16 + r16;
#pragma unroll
        for (int ii = 0; ii < 4; ++ii) {
            const int i = rt * 16 + grp * 4 + ii;
            Ps[i * LDP + j] = j <= i ? expf(Ls[i] - Ls[j]) * P[u][ii] : 0.f;
        }
    }
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
        for (int ii = 0; ii < 4; ++ii) {
            const float f = expf(Ls[rt * 16 + grp * 4 + ii]);
#pragma unroll
            for (int c = 0; c < CT; ++c) O[rt][c][ii] *= f;
        }
    f32x4 Uf[4][CT];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
#pragma unroll
        for (int c = 0; c < CT; ++c)
            Uf[jt][c] = *reinterpret_cast<const f32x4*>(p.U + (at * p.dv16 + min((wave + 4 * c) * 16, p.dv16 - 16) + r16) * CH + jt * 16 + grp * 4);
    __syncthreads();
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) {
        if (rt >= used) continue;
#pragma unroll
        for (int jt = 0; jt <= rt; ++jt) {
            const f32x4 x = *reinterpret_cast<const f32x4*>(&Ps[(rt * 16 + r16) * LDP + jt * 16 + grp * 4]);
#pragma unroll
            for (int c = 0; c < CT; ++c)
#pragma unroll
                for (int i = 0; i < 4; ++i) O[rt][c] = mfma_f32(x[i], Uf[jt][c][i], O[rt][c]);
        }
    }
    float nw[CT];
#pragma unroll
    for (int c = 0; c < CT; ++c) nw[c] = a.norm[min((wave + 4 * c) * 16 + r16, a.dv - 1)];
    // the gates of this lane's places, every load on one straight path
    f32x4 Z[4][CT];
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
        for (int c = 0; c < CT; ++c) Z[rt][c] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int q = 0; q < a.gate.n; ++q) {
        const float* gp = a.gate.p + q * a.gate.stride + (size_t)t0 * a.gate.ld + a.g_col + h * a.dv;
#pragma unroll
        for (int rt = 0; rt < 4; ++rt)
#pragma unroll
            for (int c = 0; c < CT; ++c)
#pragma unroll
                for (int ii = 0; ii < 4; ++ii)
                    Z[rt][c][ii] += gp[(size_t)min(rt * 16 + grp * 4 + ii, n - 1) * a.gate.ld + min((wave + 4 * c) * 16 + r16, a.dv - 1)];
    }
    // the heads' norms: a row's squares over this wave's columns, then over the waves
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
        for (int ii = 0; ii < 4; ++ii) {
            float ss = 0.f;
#pragma unroll
            for (int c = 0; c < CT; ++c) ss += (wave + 4 * c) * 16 + r16 < a.dv ? O[rt][c][ii] * O[rt][c][ii] : 0.f;
#pragma unroll
            for (int o = 1; o < 16; o <<= 1) ss += __shfl_xor(ss, o, WAVE);
            if (r16 == 0) rows[wave][rt * 16 + grp * 4 + ii] = ss;
        }
    __syncthreads();
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
        for (int ii = 0; ii < 4; ++ii) {
            const int i = rt * 16 + grp * 4 + ii, t = t0 + i;
            if (i >= n) continue;
            const float ss = (rows[0][i] + rows[1][i]) + (rows[2][i] + rows[3][i]);
            const float inv = 1.0f / sqrtf(ss / (float)a.dv + a.eps);
#pragma unroll
            for (int c = 0; c < CT; ++c) {
                const int col = (wave + 4 * c) * 16 + r16;
                if (col < a.dv)
                    a.out[(size_t)t * a.ld_out + h * a.dv + col] =
                        from_f32<elem_t>(O[rt][c][ii] * inv * nw[c] * silu_f(Z[rt][c][ii]));
            }
        }
    if (h == 0)
        for (int i = 0; i < n; ++i) zero_tail(a, t0 + i);
}

}  // namespace ms

using namespace ms;

extern "C" int ms_gated_state_max_taps() { return MAX_TAPS; }
// floats of the workspace of the delta rule's chunks
extern "C" long ms_delta_work(int T, int S, int H, int d, int dv) {
    const long dk16 = ceil_div(d, 16) * 16, dv16 = ceil_div(dv, 16) * 16;
    return (long)(T / CH + S) * H * (2 * CH * (dk16 + dv16) + dk16 * dv16 + 1);
}

// in: float [n_partials, T, ld].  many: requests of several rows may be among the step's (their states are then brought up
// to date by a second launch).
extern "C" int ms_delta_rows(const float* in, int n_partials, int ld, const float* w, float* state, const float* a_log, const float* dt_bias,
                             const int* seq_q_start, const int* seq_q_len, const int* seq_slot, int S, float* q, float* k, float* v,
                             float* beta, float* lg, int T, int H, int G, int d, int dv, int taps, int b_col, int a_col, float q_scale,
                             int many, hipStream_t stream) {
    MS_REQUIRE(T > 0 && S > 0 && n_partials > 0 && H > 0 && G > 0 && H % G == 0, "delta rows: T=%d S=%d, %d heads over %d", T, S, H, G);
    MS_REQUIRE(d > 0 && d <= MAX_DIM && dv > 0 && dv <= MAX_DIM, "delta rows: heads of %d and %d, at most %d", d, dv, MAX_DIM);
    MS_REQUIRE(taps >= 1 && taps <= MAX_TAPS && (taps == 1 || state), "delta rows: %d taps (1 to %d) and their state", taps, MAX_TAPS);
    const int C = 2 * G * d + H * dv;
    MS_REQUIRE(ld >= C && b_col >= 0 && a_col >= 0 && b_col + H <= ld && a_col + H <= ld, "delta rows: rows of %d numbers", ld);
    MS_REQUIRE(in && w && a_log && dt_bias && seq_q_start && seq_q_len && seq_slot && q && k && v && beta && lg, "delta rows: a buffer is missing");
    const DeltaRowsArgs a{Sums{in, n_partials, (size_t)T * ld, ld}, w, state, a_log, dt_bias, seq_q_start, seq_q_len, seq_slot, S,
                          q, k, v, beta, lg, T, H, G, d, dv, taps, b_col, a_col, q_scale};
    const int units = 2 * G + H + 1, wide = d > dv ? d : dv;
#define MS_ROWS(TP, E, R) hipLaunchKernelGGL((delta_rows_kernel<TP, E, R>), dim3(ceil_div(T, R), ceil_div(units, 4)), dim3(256), 0, stream, a)
#define MS_ROWS_E(TP, R)                     \
    do {                                     \
        if (wide <= 64) MS_ROWS(TP, 1, R);   \
        else if (wide <= 128) MS_ROWS(TP, 2, R); \
        else MS_ROWS(TP, 4, R);              \
    } while (0)
    const bool tall = T >= 256;
    if (taps <= 4) {
        if (tall) MS_ROWS_E(4, 8);
        else MS_ROWS_E(4, 1);
    } else {
        if (tall) MS_ROWS_E(MAX_TAPS, 8);
        else MS_ROWS_E(MAX_TAPS, 1);
    }
#undef MS_ROWS_E
#undef MS_ROWS
    if (int rc = check_launch("delta rows")) return rc;
    if (taps == 1 || !many) return 0;
    hipLaunchKernelGGL(delta_conv_state_kernel, dim3(S, ceil_div(C, 256)), dim3(256), 0, stream, a.in, state, seq_q_start, seq_q_len, seq_slot, C, taps);
    return check_launch("delta rows, convolution state");
}

// The gated delta rule.  q, k float [T, G * d] (unit vectors, q scaled), v float [T, H * dv], lg and beta float [T, H] as
// ms_delta_rows leaves them; gate: columns g_col on of float [n_partials, T, ld].  single: every request has one row; else
// work float [(T / 64 + S) H (2 * 64 dk16 + 2 * 64 dv16 + dk16 dv16 + 1)] (ms_delta_work) is the workspace.
extern "C" int ms_gated_delta(const float* q, const float* k, const float* v, const float* lg, const float* beta, const float* gate,
                              int n_partials, int ld, int g_col, const float* norm, float eps, float* state, const int* seq_q_start,
                              const int* seq_q_len, const int* seq_slot, int S, void* out, int ld_out, int T, int H, int G, int d, int dv,
                              int dvp, int single, float* work, hipStream_t stream) {
    const Sums qs{q, 1, 0, G * d}, ks{k, 1, 0, G * d}, vs{v, 1, 0, H * dv}, gs{gate, n_partials, (size_t)T * ld, ld};
    const StateArgs a{qs, ks, vs, 0, 0, 0, 1.0f, lg, beta, gs, g_col, norm, eps, state, seq_q_start, seq_q_len, seq_slot, S,
                      (elem_t*)out, ld_out, T, H, G, d, dv, dvp};
    MS_REQUIRE(n_partials > 0 && beta, "gated delta: no rows");
    if (int rc = check_state(a, "gated delta")) return rc;
    if (single) return launch_step<true>(a, stream);
    MS_REQUIRE(work && S <= 65535, "gated delta: chunks of %d need their workspace", CH);
    MS_REQUIRE((reinterpret_cast<uintptr_t>(work)) % 16 == 0, "gated delta: the workspace must be 16-byte aligned");
    const int numbers = T / CH + S, dk16 = ceil_div(d, 16) * 16, dv16 = ceil_div(dv, 16) * 16;
    const size_t nh = (size_t)numbers * H, kf = nh * CH * dk16, vf = nh * CH * dv16;
    const DeltaChunkArgs p{a, work, work + kf, work + 2 * kf, work + 2 * kf + vf, work + 2 * kf + 2 * vf, work + 2 * kf + 2 * vf + nh * dk16 * dv16,
                           dk16, dv16};
    hipLaunchKernelGGL(delta_solve_kernel, dim3(numbers, H), dim3(256), 0, stream, p);
    if (int rc = check_launch("gated delta, chunks solved")) return rc;
    const dim3 grid(H, ceil_div(dv, 16), S);
#define MS_PASS(KT)                                                                                                         \
    do {                                                                                                                    \
        if (dk16 == 64 * KT) hipLaunchKernelGGL((delta_pass_kernel<KT, true>), grid, dim3(256), 0, stream, p);              \
        else hipLaunchKernelGGL((delta_pass_kernel<KT, false>), grid, dim3(256), 0, stream, p);                             \
    } while (0)
    if (d <= 64) MS_PASS(1);
    else if (d <= 128) MS_PASS(2);
    else MS_PASS(4);
#undef MS_PASS
    if (int rc = check_launch("gated delta, states between chunks")) return rc;
    if (dv <= 64) hipLaunchKernelGGL(delta_out_kernel<1>, dim3(numbers, H), dim3(256), 0, stream, p);
    else if (dv <= 128) hipLaunchKernelGGL(delta_out_kernel<2>, dim3(numbers, H), dim3(256), 0, stream, p);
    else hipLaunchKernelGGL(delta_out_kernel<4>, dim3(numbers, H), dim3(256), 0, stream, p);
    return check_launch("gated delta, outputs");
}
