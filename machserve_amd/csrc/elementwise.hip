// Memory-bound kernels around the matrix products: embedding gather, RMS norm (optionally
// of gathered rows), and rotation of q and k fused with the write of k and v into pages.
//
// Role in the reference: embed_batched, rms_norm, rope_batched, kv_store_paged
// (crates/mach-model/src/kernels.rs:578-585, 63-80, 589-660, 1148-1168).
// Norm statistics, rotation angles and the rotation itself are 32-bit in both builds.
#include "common.cuh"

namespace ms {

// x[t, :] = float(table[tokens[t], :]) * scale
__global__ __launch_bounds__(256) void embed_kernel(const int* __restrict__ tokens, const elem_t* __restrict__ table,
                                                    float* __restrict__ x, int d, float scale) {
    arguments_now(tokens, table, x, d, scale);
    const int t = blockIdx.x;
    const elem_t* src = table + (size_t)tokens[t] * d;
    float* dst = x + (size_t)t * d;
    for (int c = threadIdx.x; c < d; c += 256) dst[c] = to_f32(src[c]) * scale;
}

// tokens[rows[i]] = sampled[src[i]] for the i with 0 <= rows[i] < n_tokens and 0 <= src[i] < n_sampled: the input of
// those rows of a step that the step before it sampled, taken on the device (the host has not seen them yet)
__global__ __launch_bounds__(256) void feed_tokens_kernel(int* __restrict__ tokens, const int* __restrict__ sampled,
                                                          const int* __restrict__ rows, const int* __restrict__ src, int n,
                                                          int n_tokens, int n_sampled) {
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int r = rows[i], s = src[i];
    if (r >= 0 && r < n_tokens && s >= 0 && s < n_sampled) tokens[r] = sampled[s];
}

// r = rows ? rows[i] : i;  v = x[r, :] + sum_p partials[p, r, :] (in order);  if partials are given
// and no rows are gathered, x[r, :] = v is written back (the residual stream takes the pending
// sums);  out[i, :] = v * rsqrt(mean(v^2) + eps) * w.
template <typename OutT>
__global__ __launch_bounds__(256) void rmsnorm_kernel(float* __restrict__ x, const float* __restrict__ partials,
                                                      int n_partials, size_t partial_stride,
                                                      const int* __restrict__ rows, const float* __restrict__ w,
                                                      OutT* __restrict__ out, int d, float eps) {
    __shared__ float scratch[4];
    extern __shared__ float vals[];  // d floats: the summed row
    const int i = blockIdx.x;
    const size_t r = rows ? rows[i] : i;
    float* src = x + r * d;
    float ss = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {
        const float wc = w[c];  // requested with the row, not after the reduction
        float v = src[c];
        for (int p = 0; p < n_partials; ++p) v += partials[p * partial_stride + r * d + c];
        if (n_partials > 0 && !rows) src[c] = v;
        vals[c] = v * wc;
        ss += v * v;
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    OutT* dst = out + (size_t)i * d;
    for (int c = threadIdx.x; c < d; c += 256) dst[c] = from_f32<OutT>(vals[c] * inv);
}

// Layer norm with the same handling of rows and pending sums: v as above,
// out[i, :] = (v - mean(v)) * rsqrt(mean((v - mean(v))^2) + eps) * w + b (b may be null).  The variance is the mean of
// the squared deviations, taken in a second pass over the row in LDS.
template <typename OutT>
__global__ __launch_bounds__(256) void layernorm_kernel(float* __restrict__ x, const float* __restrict__ partials,
                                                        int n_partials, size_t partial_stride,
                                                        const int* __restrict__ rows, const float* __restrict__ w,
                                                        const float* __restrict__ b, OutT* __restrict__ out, int d, float eps) {
    __shared__ float scratch[4];
    extern __shared__ float vals[];  // d floats: the summed row
    const int i = blockIdx.x;
    const size_t r = rows ? rows[i] : i;
    float* src = x + r * d;
    float sum = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {
        float v = src[c];
        for (int p = 0; p < n_partials; ++p) v += partials[p * partial_stride + r * d + c];
        if (n_partials > 0 && !rows) src[c] = v;
        vals[c] = v;
        sum += v;
    }
    const float mean = block_sum<256>(sum, scratch) / (float)d;
    float ss = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {
        const float dv = vals[c] - mean;
        ss += dv * dv;
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    OutT* dst = out + (size_t)i * d;
    for (int c = threadIdx.x; c < d; c += 256) dst[c] = from_f32<OutT>((vals[c] - mean) * inv * w[c] + (b ? b[c] : 0.f));
}

// The same for widths that are a multiple of four and at most 1024 * G.  A thread owns G groups of
// four consecutive columns (group t, t + 256, ...) and asks for all of the row it needs - stream,
// weights and the NP pending sums - before it uses the first value, so the kernel pays one memory
// round trip instead of one per column and pending sum.  The sums are added in the same order.
// With more than eight pending sums (MORE, NP = 8) the rest, up to eight again, follows in a second
// round of loads.
// With CENTER the row's mean is taken off before the squares are summed and `bias` (may be null) is added at the end:
// a layer norm, (v - mean) * rsqrt(mean((v - mean)^2) + eps) * w + bias; the stream takes the sums as they are.
template <typename OutT, int G, int NP, bool MORE = false, bool CENTER = false>
__global__ __launch_bounds__(256) void rmsnorm_wide_kernel(float* __restrict__ x, const float* __restrict__ partials,
                                                           size_t partial_stride, const int* __restrict__ rows,
                                                           const float* __restrict__ w, OutT* __restrict__ out, int d,
                                                           float eps, int n_more, const float* __restrict__ bias) {
    arguments_now(x, partials, partial_stride, rows, w, out, d, eps, n_more, bias);
    __shared__ float scratch[4];
    const int i = blockIdx.x, ng = d / 4;
    const size_t r = rows ? rows[i] : i;
    f32x4* src = reinterpret_cast<f32x4*>(x + r * d);
    const f32x4* w4 = reinterpret_cast<const f32x4*>(w);
    f32x4 v[G], wv[G], bv[G], pend[NP > 0 ? NP : 1][G];
    int at[G];
#pragma unroll
    for (int g = 0; g < G; ++g) {
        const int c4 = threadIdx.x + g * 256;
        at[g] = c4 < ng ? c4 : 0;  // a group beyond the row reads group 0 and is dropped
        v[g] = src[at[g]];
        wv[g] = w4[at[g]];
        bv[g] = (f32x4){0.f, 0.f, 0.f, 0.f};
        if constexpr (CENTER) {
            if (bias) bv[g] = reinterpret_cast<const f32x4*>(bias)[at[g]];
        }
    }
#pragma unroll
    for (int p = 0; p < NP; ++p)
#pragma unroll
        for (int g = 0; g < G; ++g) pend[p][g] = reinterpret_cast<const f32x4*>(partials + p * partial_stride + r * d)[at[g]];
    if constexpr (MORE) {
        static_assert(NP == 8, "a second round follows a full first one");
#pragma unroll
        for (int g = 0; g < G; ++g)
#pragma unroll
            for (int p = 0; p < NP; ++p) v[g] += pend[p][g];
        // sums beyond the last one read the last one again and count for nothing
#pragma unroll
        for (int p = 0; p < NP; ++p)
#pragma unroll
            for (int g = 0; g < G; ++g)
                pend[p][g] = reinterpret_cast<const f32x4*>(partials + (size_t)(NP + min(p, n_more - 1)) * partial_stride + r * d)[at[g]];
#pragma unroll
        for (int g = 0; g < G; ++g)
#pragma unroll
            for (int p = 0; p < NP; ++p) {
                const float keep = p < n_more ? 1.f : 0.f;
                v[g] += pend[p][g] * keep;
            }
    }
    float ss = 0.f, sum = 0.f;
#pragma unroll
    for (int g = 0; g < G; ++g) {
        if constexpr (!MORE) {
#pragma unroll
            for (int p = 0; p < NP; ++p) v[g] += pend[p][g];
        }
        if (threadIdx.x + g * 256 < ng) {
            if ((NP > 0 || MORE) && !rows) src[at[g]] = v[g];
            if constexpr (CENTER) sum += v[g].x + v[g].y + v[g].z + v[g].w;
            else ss += v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w;
        }
    }
    if constexpr (CENTER) {
        const float mean = block_sum<256>(sum, scratch) / (float)d;
#pragma unroll
        for (int g = 0; g < G; ++g) {
            v[g] -= mean;
            if (threadIdx.x + g * 256 < ng) ss += v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w;
        }
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    OutT* dst = out + (size_t)i * d;
#pragma unroll
    for (int g = 0; g < G; ++g) {
        if (threadIdx.x + g * 256 >= ng) continue;
        const f32x4 o = v[g] * wv[g] * inv + bv[g];
        typedef OutT out4_t __attribute__((ext_vector_type(4)));  // the group's four values in one store
        const out4_t o4 = {from_f32<OutT>(o.x), from_f32<OutT>(o.y), from_f32<OutT>(o.z), from_f32<OutT>(o.w)};
        *reinterpret_cast<out4_t*>(dst + (size_t)at[g] * 4) = o4;
    }
}

// x[t, :] += sum_p partials[p, t, :] (in order): pending sums folded in without a norm
__global__ __launch_bounds__(256) void add_partials_kernel(float* __restrict__ x, const float* __restrict__ partials,
                                                           int n_partials, size_t partial_stride, size_t n) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    float v = x[i];
    for (int p = 0; p < n_partials; ++p) v += partials[p * partial_stride + i];
    x[i] = v;
}

// x[t, :] += y / sqrt(mean(y^2) + eps) * w with y = sum_p partials[p, t, :] (in order): a branch's output, given as
// the partial sums of its last product, normalised and added to the stream in one pass.
// With `bias` (or null) y also holds a bias of the product, added after the sums.  PAIR: two branches side by side,
// y = fa sum_p partials[p, t, :] + fb sum_p pb[p, t, :] (no bias).
template <bool PAIR>
__global__ __launch_bounds__(256) void norm_add_kernel(float* __restrict__ x, const float* __restrict__ partials, int n_partials,
                                                       size_t partial_stride, const float* __restrict__ w, int d, float eps,
                                                       const float* __restrict__ bias, float fa, const float* __restrict__ pb, int nb,
                                                       float fb) {
    __shared__ float scratch[4];
    extern __shared__ float vals[];  // d floats: the summed row
    const size_t r = blockIdx.x;
    float ss = 0.f;
    // four columns at c: up to eight sums asked for at once, added in order
    auto sum4 = [&](const float* __restrict__ from, int n, int c) {
        const float* src = from + r * d + c;
        f32x4 v = (f32x4){0.f, 0.f, 0.f, 0.f};
        int p = 0;
        for (; p + 8 <= n; p += 8) {
            f32x4 q[8];
#pragma unroll
            for (int k = 0; k < 8; ++k) q[k] = *reinterpret_cast<const f32x4*>(src + (size_t)(p + k) * partial_stride);
#pragma unroll
            for (int k = 0; k < 8; ++k) v += q[k];
        }
        for (; p < n; ++p) v += *reinterpret_cast<const f32x4*>(src + (size_t)p * partial_stride);
        return v;
    };
    if (d % 4 == 0 && partial_stride % 4 == 0) {
        // few trips to memory a row
        for (int c = threadIdx.x * 4; c < d; c += 1024) {
            f32x4 v = sum4(partials, n_partials, c);
            if constexpr (PAIR) v = v * fa + sum4(pb, nb, c) * fb;
            else if (bias) v += *reinterpret_cast<const f32x4*>(bias + c);
            *reinterpret_cast<f32x4*>(vals + c) = v;
            ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        }
    } else {
        for (int c = threadIdx.x; c < d; c += 256) {
            float v = 0.f;
            for (int p = 0; p < n_partials; ++p) v += partials[(size_t)p * partial_stride + r * d + c];
            if constexpr (PAIR) {
                float b = 0.f;
                for (int p = 0; p < nb; ++p) b += pb[(size_t)p * partial_stride + r * d + c];
                v = v * fa + b * fb;
            } else if (bias) {
                v += bias[c];
            }
            vals[c] = v;
            ss += v * v;
        }
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    float* dst = x + r * d;
    for (int c = threadIdx.x; c < d; c += 256) dst[c] += vals[c] * inv * w[c];
}

// A branch's norm behind it and the next branch's norm ahead of it, in one pass over the row:
// x[t, :] += y / rms(y) * w  with y as norm_add_kernel has it,  then  out[t, :] = x / rms(x) * w2 in the element type.
// For widths that are a multiple of four and at most 1024 * G, and up to NP sums a branch: a thread owns G groups of four
// columns and asks for everything the row needs before it uses the first value (sums beyond the last one read the last one
// again and count for nothing).
template <int G, int NP, bool PAIR>
__global__ __launch_bounds__(256) void norm_add_norm_kernel(float* __restrict__ x, const float* __restrict__ pa, int na, float fa,
                                                            const float* __restrict__ pb, int nb, float fb, size_t partial_stride,
                                                            const float* __restrict__ w, float eps, const float* __restrict__ w2, float eps2,
                                                            elem_t* __restrict__ out, int d) {
    arguments_now(x, pa, na, fa, pb, nb, fb, partial_stride, w, eps, w2, eps2, out, d);
    __shared__ float scratch[4];
    const size_t r = blockIdx.x;
    const int ng = d / 4;
    f32x4* row = reinterpret_cast<f32x4*>(x + r * d);
    const f32x4* sa = reinterpret_cast<const f32x4*>(pa + r * d);
    const f32x4* sb = PAIR ? reinterpret_cast<const f32x4*>(pb + r * d) : nullptr;
    const size_t stride4 = partial_stride / 4;
    f32x4 v[G], wv[G], w2v[G], qa[NP][G], qb[PAIR ? NP : 1][G];
#pragma unroll
    for (int g = 0; g < G; ++g) {
        const int c4 = threadIdx.x + g * 256, at = c4 < ng ? c4 : 0;  // a group beyond the row reads group 0 and is dropped
        v[g] = row[at];
        wv[g] = reinterpret_cast<const f32x4*>(w)[at];
        w2v[g] = reinterpret_cast<const f32x4*>(w2)[at];
#pragma unroll
        for (int p = 0; p < NP; ++p) {
            qa[p][g] = sa[(size_t)min(p, na - 1) * stride4 + at];
            if constexpr (PAIR) qb[p][g] = sb[(size_t)min(p, nb - 1) * stride4 + at];
        }
    }
    float ss = 0.f;
    f32x4 y[G];
#pragma unroll
    for (int g = 0; g < G; ++g) {
        f32x4 a = qa[0][g];
#pragma unroll
        for (int p = 1; p < NP; ++p) a += qa[p][g] * (p < na ? 1.f : 0.f);
        y[g] = a * fa;
        if constexpr (PAIR) {
            f32x4 b = qb[0][g];
#pragma unroll
            for (int p = 1; p < NP; ++p) b += qb[p][g] * (p < nb ? 1.f : 0.f);
            y[g] += b * fb;
        }
        if (threadIdx.x + g * 256 < ng) ss += y[g].x * y[g].x + y[g].y * y[g].y + y[g].z * y[g].z + y[g].w * y[g].w;
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    float s2 = 0.f;
#pragma unroll
    for (int g = 0; g < G; ++g) {
        v[g] += y[g] * inv * wv[g];
        if (threadIdx.x + g * 256 < ng) s2 += v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w;
    }
    s2 = block_sum<256>(s2, scratch);
    const float inv2 = 1.0f / sqrtf(s2 / (float)d + eps2);
#pragma unroll
    for (int g = 0; g < G; ++g) {
        const int c4 = threadIdx.x + g * 256;
        if (c4 >= ng) continue;
        row[c4] = v[g];
        const f32x4 o = v[g] * w2v[g] * inv2;
        typedef elem_t out4_t __attribute__((ext_vector_type(4)));
        *reinterpret_cast<out4_t*>(out + r * d + (size_t)c4 * 4) = (out4_t){from_f32<elem_t>(o.x), from_f32<elem_t>(o.y), from_f32<elem_t>(o.z), from_f32<elem_t>(o.w)};
    }
}

// x[t, :] += first[t, :] (null: nothing) + row: what comes ahead of a pass over looped layers
__global__ __launch_bounds__(256) void open_pass_kernel(float* __restrict__ x, const float* __restrict__ first, const float* __restrict__ row,
                                                        int d, size_t n) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    float v = x[i];
    if (first) v += first[i];
    x[i] = v + row[i % d];
}

// x[t, :] = v / sqrt(mean(v^2) + eps) * w with v = alpha * x[t, :] + sum_p partials[p, t, :] (in order) + bias: the norm that
// comes after a residual sum.  The row also goes out in the element type (`out`, null where that is float: x itself is the
// row then), which is what the next branch reads.  This form takes any width and any number of sums.
__global__ __launch_bounds__(256) void sum_norm_kernel(float* __restrict__ x, const float* __restrict__ partials, int n_partials,
                                                       size_t partial_stride, const float* __restrict__ bias, float alpha,
                                                       const float* __restrict__ w, elem_t* __restrict__ out, int d, float eps) {
    __shared__ float scratch[4];
    extern __shared__ float vals[];  // d floats: the summed row
    const size_t r = blockIdx.x;
    float* row = x + r * d;
    float ss = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {
        float y = 0.f;
#pragma unroll 8
        for (int p = 0; p < n_partials; ++p) y += partials[(size_t)p * partial_stride + r * d + c];
        const float v = alpha * row[c] + (y + (bias ? bias[c] : 0.f));
        vals[c] = v;
        ss += v * v;
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    for (int c = threadIdx.x; c < d; c += 256) {  // a thread meets its own columns again
        const float v = vals[c] * inv * w[c];
        row[c] = v;
        if (out) out[r * d + c] = from_f32<elem_t>(v);
    }
}

// The same for widths that are a multiple of four and at most 1024 * G, and up to NP sums: a thread owns G groups of four
// columns and asks for everything the row needs before it uses the first value (sums beyond the last one read the last one
// again and count for nothing).
template <int G, int NP>
__global__ __launch_bounds__(256) void sum_norm_wide_kernel(float* __restrict__ x, const float* __restrict__ partials, int n_partials,
                                                            size_t partial_stride, const float* __restrict__ bias, float alpha,
                                                            const float* __restrict__ w, elem_t* __restrict__ out, int d, float eps) {
    arguments_now(x, partials, n_partials, partial_stride, bias, alpha, w, out, d, eps);
    __shared__ float scratch[4];
    const size_t r = blockIdx.x;
    const int ng = d / 4;
    f32x4* row = reinterpret_cast<f32x4*>(x + r * d);
    const f32x4* src = reinterpret_cast<const f32x4*>(partials + r * d);
    const size_t stride4 = partial_stride / 4;
    f32x4 v[G], wv[G], bv[G], q[NP][G];
#pragma unroll
    for (int g = 0; g < G; ++g) {
        const int c4 = threadIdx.x + g * 256, at = c4 < ng ? c4 : 0;  // a group beyond the row reads group 0 and is dropped
        v[g] = row[at];
        wv[g] = reinterpret_cast<const f32x4*>(w)[at];
        bv[g] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int p = 0; p < NP; ++p) q[p][g] = src[(size_t)min(p, n_partials - 1) * stride4 + at];
    }
    if (bias)
#pragma unroll
        for (int g = 0; g < G; ++g) {
            const int c4 = threadIdx.x + g * 256;
            bv[g] = reinterpret_cast<const f32x4*>(bias)[c4 < ng ? c4 : 0];
        }
    float ss = 0.f;
#pragma unroll
    for (int g = 0; g < G; ++g) {
        f32x4 y = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int p = 0; p < NP; ++p) y += q[p][g] * (p < n_partials ? 1.f : 0.f);
        v[g] = v[g] * alpha + (y + bv[g]);
        if (threadIdx.x + g * 256 < ng) ss += v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w;
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
#pragma unroll
    for (int g = 0; g < G; ++g) {
        const int c4 = threadIdx.x + g * 256;
        if (c4 >= ng) continue;
        const f32x4 o = v[g] * inv * wv[g];
        row[c4] = o;
        typedef elem_t out4_t __attribute__((ext_vector_type(4)));
        if (out) *reinterpret_cast<out4_t*>(out + r * d + (size_t)c4 * 4) = (out4_t){from_f32<elem_t>(o.x), from_f32<elem_t>(o.y), from_f32<elem_t>(o.z), from_f32<elem_t>(o.w)};
    }
}

// Two branches side by side, each given as the partial sums of its last product: every branch's sum is normalised with
// a weight of its own, half their sum is normalised again, and that is added to the stream:
// y = (rms(a) * wa + rms(b) * wb) / 2;  x[t, :] += rms(y) * w.
__global__ __launch_bounds__(256) void pair_norm_add_kernel(float* __restrict__ x, const float* __restrict__ pa, int na,
                                                            const float* __restrict__ wa, const float* __restrict__ pb, int nb,
                                                            const float* __restrict__ wb, size_t partial_stride,
                                                            const float* __restrict__ w, int d, float eps) {
    __shared__ float scratch[4];
    extern __shared__ float vals[];  // 2 d floats: the two summed rows
    float* va = vals;
    float* vb = vals + d;
    const size_t r = blockIdx.x;
    float sa = 0.f, sb = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {
        float a = 0.f, b = 0.f;
        for (int p = 0; p < na; ++p) a += pa[(size_t)p * partial_stride + r * d + c];
        for (int p = 0; p < nb; ++p) b += pb[(size_t)p * partial_stride + r * d + c];
        va[c] = a;
        vb[c] = b;
        sa += a * a;
        sb += b * b;
    }
    sa = block_sum<256>(sa, scratch);
    sb = block_sum<256>(sb, scratch);
    const float ia = 1.0f / sqrtf(sa / (float)d + eps), ib = 1.0f / sqrtf(sb / (float)d + eps);
    float ss = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {  // a thread meets its own columns again: no barrier in between
        const float y = 0.5f * (va[c] * ia * wa[c] + vb[c] * ib * wb[c]);
        va[c] = y;
        ss += y * y;
    }
    ss = block_sum<256>(ss, scratch);
    const float inv = 1.0f / sqrtf(ss / (float)d + eps);
    float* dst = x + r * d;
    for (int c = threadIdx.x; c < d; c += 256) dst[c] += va[c] * inv * w[c];
}

// out[t, c] = act(in[t, c]) * in[t, n + c]: the gated product of a feed-forward whose gate and up projections were one
// product with biases, left as 32-bit sums
__global__ __launch_bounds__(256) void gate_mul_kernel(const float* __restrict__ in, elem_t* __restrict__ out, int n, int act) {
    const size_t t = blockIdx.x;
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) out[t * n + c] = from_f32<elem_t>(gate_activation(in[t * 2 * n + c], act) * in[t * 2 * n + n + c]);
}

// out[t, :] = the stream's row in the element type: the input of a branch that reads the stream as it is.
__global__ __launch_bounds__(256) void round_rows_kernel(const float* __restrict__ x, elem_t* __restrict__ out, size_t n) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i < n) out[i] = from_f32<elem_t>(x[i]);
}

// x[t, :] = float(table[tokens[t], :]) + float(pairs[row(t), :]) with row(t) = (previous * mul_prev + tokens[t] * mul_cur) mod
// buckets, and row `buckets` for a request's first token.  The previous token is the row before in the step, or, for the
// first row of a request's portion, what the request's slot of `prev [slots]` holds.
__global__ __launch_bounds__(256) void embed_pair_kernel(const int* __restrict__ tokens, const elem_t* __restrict__ table,
                                                         const elem_t* __restrict__ pairs, const int* __restrict__ prev,
                                                         const int* __restrict__ seq_q_start, const int* __restrict__ seq_pos0,
                                                         const int* __restrict__ seq_slot, int S, float* __restrict__ x, int d,
                                                         long mul_prev, long mul_cur, long buckets) {
    const int t = blockIdx.x;
    int lo = 0, hi = S - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (seq_q_start[mid] <= t) lo = mid;
        else hi = mid - 1;
    }
    const int j = t - seq_q_start[lo];
    const int tok = tokens[t];
    long row = buckets;
    if (seq_pos0[lo] + j > 0) {
        const int before = j > 0 ? tokens[t - 1] : prev[seq_slot[lo]];
        row = ((long)before * mul_prev + (long)tok * mul_cur) % buckets;
    }
    const elem_t* a = table + (size_t)tok * d;
    const elem_t* b = pairs + (size_t)row * d;
    float* dst = x + (size_t)t * d;
    for (int c = threadIdx.x; c < d; c += 256) dst[c] = to_f32(a[c]) + to_f32(b[c]);
}

// prev[slot of request s] = the last token of its rows in this step
__global__ __launch_bounds__(256) void last_token_kernel(const int* __restrict__ tokens, const int* __restrict__ seq_q_start,
                                                         const int* __restrict__ seq_q_len, const int* __restrict__ seq_slot, int S,
                                                         int* __restrict__ prev) {
    const int s = blockIdx.x * 256 + threadIdx.x;
    if (s < S && seq_q_len[s] > 0) prev[seq_slot[s]] = tokens[seq_q_start[s] + seq_q_len[s] - 1];
}

// v = logits * scale;  logits = cap > 0 ? cap * tanh(v / cap) : v
__global__ __launch_bounds__(256) void softcap_kernel(float* __restrict__ logits, size_t n, float scale, float cap) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const float v = logits[i] * scale;
    logits[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
}

struct RopeArgs {
    const float* qkv;       // [n_partials, T, stride] partial sums of: q heads, then (if written) k heads, v heads
    const float* bias;      // [stride] or null, added to the sum
    int n_partials;
    size_t partial_stride;
    const int* positions;   // [T]
    const float* inv_freq;  // [hd / 2] or null: no rotation
    const int* slot_map;    // [T] page * ps + offset of the row's key, or null: nothing is written
    elem_t* q_out;          // [T, H * hd]
    elem_t* kpool;          // [pages, KV, ps, hd]
    elem_t* vpool;          // [pages, KV, hd, ps]
    int stride, H, KV, hd, ps;
};

__global__ __launch_bounds__(256) void rope_kv_write_kernel(RopeArgs a) {
    __shared__ float cs[128], sn[128];
    extern __shared__ float row[];  // stride floats: this row's sums with the bias added
    const int t = blockIdx.x, half = a.hd / 2;
    const int width = a.H * a.hd + (a.slot_map ? 2 * a.KV * a.hd : 0);
    for (int c = threadIdx.x; c < width; c += 256) {
        float v = a.bias ? a.bias[c] : 0.f;
        for (int p = 0; p < a.n_partials; ++p) v += a.qkv[p * a.partial_stride + (size_t)t * a.stride + c];
        row[c] = v;
    }
    if (threadIdx.x < half) {
        float c = 1.f, s = 0.f;
        if (a.inv_freq) {
            const float ang = (float)a.positions[t] * a.inv_freq[threadIdx.x];
            sincosf(ang, &s, &c);
        }
        cs[threadIdx.x] = c;
        sn[threadIdx.x] = s;
    }
    __syncthreads();
    // q: pairs (j, j + half) of every head
    for (int p = threadIdx.x; p < a.H * half; p += 256) {
        const int h = p / half, j = p % half;
        const float x0 = row[h * a.hd + j], x1 = row[h * a.hd + j + half];
        elem_t* o = a.q_out + ((size_t)t * a.H + h) * a.hd;
        o[j] = from_f32<elem_t>(x0 * cs[j] - x1 * sn[j]);
        o[j + half] = from_f32<elem_t>(x0 * sn[j] + x1 * cs[j]);
    }
    if (!a.slot_map) return;
    const int slot = a.slot_map[t];
    if (slot < 0) return;
    const int page = slot / a.ps, off = slot % a.ps;
    const float* krow = row + a.H * a.hd;
    const float* vrow = krow + a.KV * a.hd;
    for (int p = threadIdx.x; p < a.KV * half; p += 256) {
        const int h = p / half, j = p % half;
        const float x0 = krow[h * a.hd + j], x1 = krow[h * a.hd + j + half];
        elem_t* o = a.kpool + (((size_t)page * a.KV + h) * a.ps + off) * a.hd;
        o[j] = from_f32<elem_t>(x0 * cs[j] - x1 * sn[j]);
        o[j + half] = from_f32<elem_t>(x0 * sn[j] + x1 * cs[j]);
    }
    for (int p = threadIdx.x; p < a.KV * a.hd; p += 256) {
        const int h = p / a.hd, dd = p % a.hd;
        a.vpool[(((size_t)page * a.KV + h) * a.hd + dd) * a.ps + off] = from_f32<elem_t>(vrow[p]);
    }
}

// cs[t, j] = (cos, sin) of positions[t] * inv_freq[j]: the angles of a step's rows, once for every layer that rotates
// by these frequencies, for the product that rotates in its own epilogue (it cannot share a row's sines among its
// lanes as the kernels here do).  The same expression as above: the same values.
__global__ __launch_bounds__(256) void rope_table_kernel(const int* __restrict__ positions, const float* __restrict__ inv_freq,
                                                         float* __restrict__ cs, int n, int half) {
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int t = i / half, j = i - t * half;
    float c, s;
    sincosf((float)positions[t] * inv_freq[j], &s, &c);
    cs[2 * (size_t)i] = c;
    cs[2 * (size_t)i + 1] = s;
}

// The same in quads: head sizes that are multiples of 8, rows whose stride is a multiple of 4 and
// 16-byte aligned buffers.  A thread takes four neighbouring pairs (j .. j + 3, j + half .. + 3) of one
// head: two 16-byte loads per partial sum, all asked for before the first is used, and two 8-byte
// (bfloat16) or 16-byte stores.  Nothing is staged in LDS but the row's cosines and sines.
template <int NP>
__global__ __launch_bounds__(256) void rope_kv_write_quads_kernel(RopeArgs a) {
    __shared__ float cs[128], sn[128];
    const int t = blockIdx.x, half = a.hd / 2, hq = half / 4;
    if (threadIdx.x < half) {
        float c = 1.f, s = 0.f;
        if (a.inv_freq) {
            const float ang = (float)a.positions[t] * a.inv_freq[threadIdx.x];
            sincosf(ang, &s, &c);
        }
        cs[threadIdx.x] = c;
        sn[threadIdx.x] = s;
    }
    const bool writes = a.slot_map != nullptr;
    const int slot = writes ? a.slot_map[t] : -1;
    const int page = slot >= 0 ? slot / a.ps : 0, off = slot >= 0 ? slot % a.ps : 0;
    const float* rowp = a.qkv + (size_t)t * a.stride;
    auto summed = [&](int c) {  // bias + the partial sums of columns c .. c + 3, in order
        f32x4 v[NP];
#pragma unroll
        for (int p = 0; p < NP; ++p) v[p] = *reinterpret_cast<const f32x4*>(rowp + p * a.partial_stride + c);
        f32x4 r = a.bias ? *reinterpret_cast<const f32x4*>(a.bias + c) : (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int p = 0; p < NP; ++p) r += v[p];
        return r;
    };
    auto store_quad = [](elem_t* o, const f32x4& v) {
#ifdef MS_ELEM_HALF
        half4_t b = {(elem_t)v[0], (elem_t)v[1], (elem_t)v[2], (elem_t)v[3]};
        *reinterpret_cast<half4_t*>(o) = b;
#else
        *reinterpret_cast<f32x4*>(o) = v;
#endif
    };
    // q heads, then k heads: pairs (j, j + half)
    const int rot_heads = a.H + (writes ? a.KV : 0);
    const int n_rot = rot_heads * hq;
    // v heads: quads of the head's elements
    const int n_v = writes ? a.KV * (a.hd / 4) : 0;
    __syncthreads();
    for (int it = threadIdx.x; it < n_rot + n_v; it += 256) {
        if (it < n_rot) {
            const int h = it / hq, j = (it % hq) * 4;
            const f32x4 x0 = summed(h * a.hd + j), x1 = summed(h * a.hd + half + j);
            f32x4 lo, hi;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                lo[e] = x0[e] * cs[j + e] - x1[e] * sn[j + e];
                hi[e] = x0[e] * sn[j + e] + x1[e] * cs[j + e];
            }
            elem_t* o;
            if (h < a.H) o = a.q_out + ((size_t)t * a.H + h) * a.hd;
            else if (slot >= 0) o = a.kpool + (((size_t)page * a.KV + (h - a.H)) * a.ps + off) * a.hd;
            else continue;
            store_quad(o + j, lo);
            store_quad(o + half + j, hi);
        } else if (slot >= 0) {
            const int q = it - n_rot, h = q / (a.hd / 4), dd = (q % (a.hd / 4)) * 4;
            const f32x4 v = summed((a.H + a.KV + h) * a.hd + dd);
            elem_t* o = a.vpool + (((size_t)page * a.KV + h) * a.hd + dd) * a.ps + off;
#pragma unroll
            for (int e = 0; e < 4; ++e) o[(size_t)e * a.ps] = from_f32<elem_t>(v[e]);
        }
    }
}

}  // namespace ms

using namespace ms;

// The widest row that the norm and the rotation kernels hold in a block's LDS (floats); a model asks for these
// when it is put together, so that a wider one is refused then, with the size's name, not at its first step.
constexpr int MAX_ROW_FLOATS = 15000;
extern "C" int ms_max_norm_width() { return MAX_ROW_FLOATS; }
extern "C" int ms_max_rope_row() { return MAX_ROW_FLOATS; }

// cs [T, half, 2] (float) = cosine and sine of positions[t] * inv_freq[j].
extern "C" int ms_rope_table(const int* positions, const float* inv_freq, float* cs, int T, int half, hipStream_t stream) {
    MS_REQUIRE(T > 0 && half > 0 && positions && inv_freq && cs, "rope table: T=%d, %d frequencies", T, half);
    MS_REQUIRE((long)T * half < 2147483647L, "rope table: %d rows of %d frequencies", T, half);
    const int n = T * half;
    hipLaunchKernelGGL(rope_table_kernel, dim3((unsigned)ceil_div(n, 256)), dim3(256), 0, stream, positions, inv_freq, cs, n, half);
    return check_launch("rope_table");
}

extern "C" int ms_embed(const int* tokens, const void* table, float* x, int T, int d, float scale, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0, "embed: empty problem T=%d d=%d", T, d);
    hipLaunchKernelGGL(embed_kernel, dim3(T), dim3(256), 0, stream, tokens, (const elem_t*)table, x, d, scale);
    return check_launch("embed");
}

extern "C" int ms_feed_tokens(int* tokens, const int* sampled, const int* rows, const int* src, int n, int n_tokens, int n_sampled,
                              hipStream_t stream) {
    MS_REQUIRE(n > 0 && n_tokens > 0 && n_sampled > 0, "feed_tokens: empty problem n=%d tokens=%d sampled=%d", n, n_tokens, n_sampled);
    MS_REQUIRE(tokens && sampled && rows && src, "feed_tokens: a buffer is missing");
    hipLaunchKernelGGL(feed_tokens_kernel, dim3(ceil_div(n, 256)), dim3(256), 0, stream, tokens, sampled, rows, src, n, n_tokens, n_sampled);
    return check_launch("feed_tokens");
}

// rows may be null (identity).  out is float when out_f32 != 0, else the element type.
// partials [n_partials, T, d] are pending sums of the stream x [T, d] (n_partials may be 0); see the
// kernel for what is written back.
// The launch of the kernel above for the widths and numbers of pending sums it is built for; false: not taken.
template <bool CENTER>
static bool launch_wide_norm(float* x, const float* partials, int n_partials, size_t ps, const int* rows, const float* w,
                             const float* bias, void* out, bool f32_out, int n, int d, float eps, hipStream_t stream) {
    const int groups = d % 4 == 0 ? (d <= 1024 ? 1 : (d <= 2048 ? 2 : (d <= 4096 ? 4 : 0))) : 0;
    const bool aligned = (reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(w) | reinterpret_cast<uintptr_t>(partials) |
                          reinterpret_cast<uintptr_t>(bias)) % 16 == 0;
    if (!(groups && aligned && n_partials <= 16)) return false;
#define MS_NORM(OUT_, G_, NP_)                                                                                                      \
    hipLaunchKernelGGL((rmsnorm_wide_kernel<OUT_, G_, NP_, false, CENTER>), dim3(n), dim3(256), 0, stream, x, partials, ps, rows, w, \
                       (OUT_*)out, d, eps, 0, bias)
#define MS_NORM_MORE(OUT_, G_)                                                                                                    \
    hipLaunchKernelGGL((rmsnorm_wide_kernel<OUT_, G_, 8, true, CENTER>), dim3(n), dim3(256), 0, stream, x, partials, ps, rows, w, \
                       (OUT_*)out, d, eps, n_partials - 8, bias)
#define MS_NORM_NP(OUT_, G_)                                    \
    switch (n_partials) {                                       \
        case 0: MS_NORM(OUT_, G_, 0); break;                    \
        case 1: MS_NORM(OUT_, G_, 1); break;                    \
        case 2: MS_NORM(OUT_, G_, 2); break;                    \
        case 3: MS_NORM(OUT_, G_, 3); break;                    \
        case 4: MS_NORM(OUT_, G_, 4); break;                    \
        case 5: MS_NORM(OUT_, G_, 5); break;                    \
        case 6: MS_NORM(OUT_, G_, 6); break;                    \
        case 7: MS_NORM(OUT_, G_, 7); break;                    \
        case 8: MS_NORM(OUT_, G_, 8); break;                    \
        default: MS_NORM_MORE(OUT_, G_); break;                 \
    }
#define MS_NORM_G(OUT_)                                         \
    if (groups == 1) { MS_NORM_NP(OUT_, 1) }                    \
    else if (groups == 2) { MS_NORM_NP(OUT_, 2) }               \
    else { MS_NORM_NP(OUT_, 4) }
    if (f32_out) { MS_NORM_G(float) } else { MS_NORM_G(elem_t) }
#undef MS_NORM_G
#undef MS_NORM_NP
#undef MS_NORM_MORE
#undef MS_NORM
    return true;
}

extern "C" int ms_rmsnorm(float* x, const float* partials, int n_partials, int T, const int* rows, const float* w,
                          void* out, int out_f32, int n, int d, float eps, hipStream_t stream) {
    MS_REQUIRE(n > 0 && d > 0, "rmsnorm: empty problem n=%d d=%d", n, d);
    MS_REQUIRE(d <= MAX_ROW_FLOATS, "rmsnorm: width %d exceeds the row buffer of %d", d, MAX_ROW_FLOATS);
    MS_REQUIRE(n_partials == 0 || partials, "rmsnorm: %d partial sums without a buffer", n_partials);
    const size_t ps = (size_t)T * d, smem = (size_t)d * sizeof(float);
    const bool f32_out = out_f32 || !kHalf;
    if (launch_wide_norm<false>(x, partials, n_partials, ps, rows, w, nullptr, out, f32_out, n, d, eps, stream)) return check_launch("rmsnorm");
    if (f32_out)
        hipLaunchKernelGGL(rmsnorm_kernel<float>, dim3(n), dim3(256), smem, stream, x, partials, n_partials, ps, rows, w,
                           (float*)out, d, eps);
    else
        hipLaunchKernelGGL(rmsnorm_kernel<elem_t>, dim3(n), dim3(256), smem, stream, x, partials, n_partials, ps, rows, w,
                           (elem_t*)out, d, eps);
    return check_launch("rmsnorm");
}

extern "C" int ms_layernorm(float* x, const float* partials, int n_partials, int T, const int* rows, const float* w, const float* b,
                            void* out, int out_f32, int n, int d, float eps, hipStream_t stream) {
    MS_REQUIRE(n > 0 && d > 0, "layernorm: empty problem n=%d d=%d", n, d);
    MS_REQUIRE(d <= MAX_ROW_FLOATS, "layernorm: width %d exceeds the row buffer of %d", d, MAX_ROW_FLOATS);
    MS_REQUIRE(n_partials == 0 || partials, "layernorm: %d partial sums without a buffer", n_partials);
    const size_t ps = (size_t)T * d, smem = (size_t)d * sizeof(float);
    if (launch_wide_norm<true>(x, partials, n_partials, ps, rows, w, b, out, out_f32 || !kHalf, n, d, eps, stream)) return check_launch("layernorm");
    if (out_f32 || !kHalf)
        hipLaunchKernelGGL(layernorm_kernel<float>, dim3(n), dim3(256), smem, stream, x, partials, n_partials, ps, rows, w, b,
                           (float*)out, d, eps);
    else
        hipLaunchKernelGGL(layernorm_kernel<elem_t>, dim3(n), dim3(256), smem, stream, x, partials, n_partials, ps, rows, w, b,
                           (elem_t*)out, d, eps);
    return check_launch("layernorm");
}

extern "C" int ms_norm_add(float* x, const float* partials, int n_partials, const float* w, int T, int d, float eps, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && n_partials > 0, "norm_add: empty problem T=%d d=%d with %d sums", T, d, n_partials);
    MS_REQUIRE(d <= MAX_ROW_FLOATS, "norm_add: width %d exceeds the row buffer of %d", d, MAX_ROW_FLOATS);
    MS_REQUIRE(x && partials && w, "norm_add: a buffer is missing");
    hipLaunchKernelGGL(norm_add_kernel<false>, dim3(T), dim3(256), (size_t)d * sizeof(float), stream, x, partials, n_partials, (size_t)T * d, w,
                       d, eps, (const float*)nullptr, 1.f, (const float*)nullptr, 0, 0.f);
    return check_launch("norm_add");
}

extern "C" int ms_norm_add_bias(float* x, const float* partials, int n_partials, const float* bias, const float* w, int T, int d,
                                float eps, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && n_partials > 0, "norm_add: empty problem T=%d d=%d with %d sums", T, d, n_partials);
    MS_REQUIRE(d <= MAX_ROW_FLOATS, "norm_add: width %d exceeds the row buffer of %d", d, MAX_ROW_FLOATS);
    MS_REQUIRE(x && partials && w, "norm_add: a buffer is missing");
    hipLaunchKernelGGL(norm_add_kernel<false>, dim3(T), dim3(256), (size_t)d * sizeof(float), stream, x, partials, n_partials, (size_t)T * d, w,
                       d, eps, bias, 1.f, (const float*)nullptr, 0, 0.f);
    return check_launch("norm_add");
}

// x += rmsnorm(fa sum(pa) + fb sum(pb)) * w
extern "C" int ms_norm_add_weighted(float* x, const float* pa, int na, float fa, const float* pb, int nb, float fb, const float* w, int T, int d,
                                    float eps, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && na > 0 && nb > 0, "norm_add_weighted: empty problem T=%d d=%d with %d and %d sums", T, d, na, nb);
    MS_REQUIRE(d <= MAX_ROW_FLOATS, "norm_add_weighted: width %d exceeds the row buffer of %d", d, MAX_ROW_FLOATS);
    MS_REQUIRE(x && pa && pb && w, "norm_add_weighted: a buffer is missing");
    hipLaunchKernelGGL(norm_add_kernel<true>, dim3(T), dim3(256), (size_t)d * sizeof(float), stream, x, pa, na, (size_t)T * d, w, d, eps,
                       (const float*)nullptr, fa, pb, nb, fb);
    return check_launch("norm_add_weighted");
}

// Whether ms_norm_add_norm takes rows of d numbers with na and nb sums (nb 0: one branch).
extern "C" int ms_norm_add_norm_takes(int d, int na, int nb) {
    const int g = d % 4 == 0 ? (d <= 1024 ? 1 : (d <= 2048 ? 2 : (d <= 4096 ? 4 : 0))) : 0, most = na > nb ? na : nb;
    return g > 0 && na >= 1 && most * g * (nb ? 2 : 1) <= 16 && most <= 8;
}

// x += rmsnorm(fa sum(pa) + fb sum(pb)) * w (pb null: the first branch alone), out = rmsnorm(x) * w2 in the element type
extern "C" int ms_norm_add_norm(float* x, const float* pa, int na, float fa, const float* pb, int nb, float fb, const float* w, float eps,
                                const float* w2, float eps2, void* out, int T, int d, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && ms_norm_add_norm_takes(d, na, pb ? nb : 0), "norm_add_norm: T=%d d=%d with %d and %d sums", T, d, na, nb);
    MS_REQUIRE(x && pa && w && w2 && out && (pb == nullptr) == (nb == 0), "norm_add_norm: a buffer is missing");
    MS_REQUIRE((reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(pa) | reinterpret_cast<uintptr_t>(pb) | reinterpret_cast<uintptr_t>(w) |
                reinterpret_cast<uintptr_t>(w2) | reinterpret_cast<uintptr_t>(out)) % 16 == 0, "norm_add_norm: buffers must be 16-byte aligned");
    const size_t ps = (size_t)T * d;
    const int groups = d <= 1024 ? 1 : (d <= 2048 ? 2 : 4), most = na > nb ? na : nb;
#define MS_NAN(G_, NP_, PAIR_)                                                                                                            \
    hipLaunchKernelGGL((norm_add_norm_kernel<G_, NP_, PAIR_>), dim3(T), dim3(256), 0, stream, x, pa, na, fa, pb, nb, fb, ps, w, eps, w2, eps2, \
                       (elem_t*)out, d)
    if (pb == nullptr) {
        if (groups == 1) { if (most == 1) MS_NAN(1, 1, false); else if (most == 2) MS_NAN(1, 2, false); else if (most <= 4) MS_NAN(1, 4, false); else MS_NAN(1, 8, false); }
        else if (groups == 2) { if (most == 1) MS_NAN(2, 1, false); else if (most == 2) MS_NAN(2, 2, false); else if (most <= 4) MS_NAN(2, 4, false); else MS_NAN(2, 8, false); }
        else { if (most == 1) MS_NAN(4, 1, false); else if (most == 2) MS_NAN(4, 2, false); else MS_NAN(4, 4, false); }
    } else {
        if (groups == 1) { if (most == 1) MS_NAN(1, 1, true); else if (most == 2) MS_NAN(1, 2, true); else if (most <= 4) MS_NAN(1, 4, true); else MS_NAN(1, 8, true); }
        else if (groups == 2) { if (most == 1) MS_NAN(2, 1, true); else if (most == 2) MS_NAN(2, 2, true); else MS_NAN(2, 4, true); }
        else { if (most == 1) MS_NAN(4, 1, true); else MS_NAN(4, 2, true); }
    }
#undef MS_NAN
    return check_launch("norm_add_norm");
}

extern "C" int ms_open_pass(float* x, const float* first, const float* row, int T, int d, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && x && row, "open_pass: empty problem T=%d d=%d", T, d);
    const size_t n = (size_t)T * d;
    hipLaunchKernelGGL(open_pass_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, x, first, row, d, n);
    return check_launch("open_pass");
}

// x [T, d] <- rmsnorm(alpha x + sum of partials [n_partials, T, d] + bias) * w; out [T, d] in the element type, or null.
extern "C" int ms_sum_norm(float* x, const float* partials, int n_partials, const float* bias, float alpha, const float* w, void* out,
                           int T, int d, float eps, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && n_partials > 0, "sum_norm: empty problem T=%d d=%d with %d sums", T, d, n_partials);
    MS_REQUIRE(d <= MAX_ROW_FLOATS, "sum_norm: width %d exceeds the row buffer of %d", d, MAX_ROW_FLOATS);
    MS_REQUIRE(x && partials && w, "sum_norm: a buffer is missing");
    const size_t ps = (size_t)T * d;
    const int groups = d % 4 == 0 ? (d <= 1024 ? 1 : (d <= 2048 ? 2 : (d <= 4096 ? 4 : 0))) : 0;
    const bool aligned = (reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(w) | reinterpret_cast<uintptr_t>(partials) |
                          reinterpret_cast<uintptr_t>(bias) | reinterpret_cast<uintptr_t>(out)) % 16 == 0;
    if (groups && aligned && n_partials <= (groups == 4 ? 8 : 16)) {
#define MS_SUM_NORM(G_, NP_)                                                                                                           \
    hipLaunchKernelGGL((sum_norm_wide_kernel<G_, NP_>), dim3(T), dim3(256), 0, stream, x, partials, n_partials, ps, bias, alpha, w, \
                       (elem_t*)out, d, eps)
#define MS_SUM_NORM_NP(G_, MOST_)                        \
    if (n_partials == 1) MS_SUM_NORM(G_, 1);             \
    else if (n_partials == 2) MS_SUM_NORM(G_, 2);        \
    else if (n_partials <= 4) MS_SUM_NORM(G_, 4);        \
    else if (n_partials <= 8) MS_SUM_NORM(G_, 8);        \
    else MS_SUM_NORM(G_, MOST_)
        if (groups == 1) { MS_SUM_NORM_NP(1, 16); }
        else if (groups == 2) { MS_SUM_NORM_NP(2, 16); }
        else { MS_SUM_NORM_NP(4, 8); }
#undef MS_SUM_NORM_NP
#undef MS_SUM_NORM
    } else {
        hipLaunchKernelGGL(sum_norm_kernel, dim3(T), dim3(256), (size_t)d * sizeof(float), stream, x, partials, n_partials, ps, bias, alpha, w,
                           (elem_t*)out, d, eps);
    }
    return check_launch("sum_norm");
}

extern "C" int ms_pair_norm_add(float* x, const float* pa, int na, const float* wa, const float* pb, int nb, const float* wb,
                                const float* w, int T, int d, float eps, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && na > 0 && nb > 0, "pair_norm_add: empty problem T=%d d=%d with %d and %d sums", T, d, na, nb);
    MS_REQUIRE(2 * d <= MAX_ROW_FLOATS, "pair_norm_add: width %d exceeds half the row buffer of %d", d, MAX_ROW_FLOATS);
    MS_REQUIRE(x && pa && pb && wa && wb && w, "pair_norm_add: a buffer is missing");
    hipLaunchKernelGGL(pair_norm_add_kernel, dim3(T), dim3(256), (size_t)2 * d * sizeof(float), stream, x, pa, na, wa, pb, nb, wb,
                       (size_t)T * d, w, d, eps);
    return check_launch("pair_norm_add");
}

extern "C" int ms_gate_mul(const float* in, void* out, int T, int n, int act, hipStream_t stream) {
    MS_REQUIRE(T > 0 && n > 0 && in && out, "gate_mul: empty problem T=%d n=%d", T, n);
    MS_REQUIRE(act >= 0 && act < ACT_COUNT, "gate_mul: activation %d", act);
    hipLaunchKernelGGL(gate_mul_kernel, dim3(T, ceil_div(n, 256)), dim3(256), 0, stream, in, (elem_t*)out, n, act);
    return check_launch("gate_mul");
}

extern "C" int ms_round_rows(const float* x, void* out, long n, hipStream_t stream) {
    MS_REQUIRE(n > 0 && x && out, "round_rows: empty problem");
    hipLaunchKernelGGL(round_rows_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, x, (elem_t*)out, (size_t)n);
    return check_launch("round_rows");
}

extern "C" int ms_embed_pair(const int* tokens, const void* table, const void* pairs, int* prev, const int* seq_q_start,
                             const int* seq_q_len, const int* seq_pos0, const int* seq_slot, int S, float* x, int T, int d,
                             long mul_prev, long mul_cur, long buckets, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && S > 0, "embed_pair: empty problem T=%d d=%d S=%d", T, d, S);
    MS_REQUIRE(buckets > 0 && mul_prev >= 0 && mul_cur >= 0 && mul_prev < (1L << 31) && mul_cur < (1L << 31),
               "embed_pair: %ld buckets, multipliers %ld and %ld", buckets, mul_prev, mul_cur);
    hipLaunchKernelGGL(embed_pair_kernel, dim3(T), dim3(256), 0, stream, tokens, (const elem_t*)table, (const elem_t*)pairs,
                       (const int*)prev, seq_q_start, seq_pos0, seq_slot, S, x, d, mul_prev, mul_cur, buckets);
    int rc = check_launch("embed_pair");
    if (rc) return rc;
    hipLaunchKernelGGL(last_token_kernel, dim3((unsigned)ceil_div(S, 256)), dim3(256), 0, stream, tokens, seq_q_start, seq_q_len,
                       seq_slot, S, prev);
    return check_launch("last_token");
}

extern "C" int ms_softcap(float* logits, long n, float scale, float cap, hipStream_t stream) {
    MS_REQUIRE(n > 0 && logits, "softcap: empty problem");
    hipLaunchKernelGGL(softcap_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, logits, (size_t)n, scale, cap);
    return check_launch("softcap");
}

extern "C" int ms_add_partials(float* x, const float* partials, int n_partials, int T, int d, hipStream_t stream) {
    MS_REQUIRE(T > 0 && d > 0 && n_partials > 0, "add_partials: empty problem");
    const size_t n = (size_t)T * d;
    hipLaunchKernelGGL(add_partials_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, x, partials,
                       n_partials, n, n);
    return check_launch("add_partials");
}

// Sum the partial sums of the q/k/v projection, add the bias, rotate q (and k) by the rows'
// positions and write k, v into their pages.  inv_freq null: no
// rotation.  slot_map null: the rows hold q only and nothing is written (a layer that reads
// another layer's cache).
extern "C" int ms_rope_kv_write(const float* qkv, int n_partials, const float* bias, int stride, const int* positions,
                                const float* inv_freq,
                                const int* slot_map, void* q_out, void* kpool, void* vpool, int T, int H, int KV,
                                int hd, int ps, hipStream_t stream) {
    MS_REQUIRE(T > 0, "rope: no rows");
    MS_REQUIRE(hd % 2 == 0 && hd >= 2 && hd <= 256, "rope: head size %d must be even and at most 256", hd);
    MS_REQUIRE(stride >= H * hd + (slot_map ? 2 * KV * hd : 0), "rope: row stride %d too small for %d+2*%d heads of %d",
               stride, H, KV, hd);
    MS_REQUIRE(!slot_map || (kpool && vpool && ps > 0), "rope: cache write without pools");
    MS_REQUIRE(n_partials >= 1, "rope: %d partial sums", n_partials);
    MS_REQUIRE(stride <= MAX_ROW_FLOATS, "rope: a row of %d values exceeds the row buffer of %d", stride, MAX_ROW_FLOATS);
    RopeArgs a{qkv, bias, n_partials, (size_t)T * stride, positions, inv_freq, slot_map, (elem_t*)q_out, (elem_t*)kpool,
               (elem_t*)vpool, stride, H, KV, hd, ps};
    const bool aligned = ((reinterpret_cast<uintptr_t>(qkv) | reinterpret_cast<uintptr_t>(bias) | reinterpret_cast<uintptr_t>(q_out) |
                           reinterpret_cast<uintptr_t>(kpool)) & 15) == 0;
    // (up to eight partial sums: a portion of 65 to 128 rows cuts the projection's K seven times)
    if (hd % 8 == 0 && stride % 4 == 0 && a.partial_stride % 4 == 0 && aligned && n_partials <= 8) {
        switch (n_partials) {
            case 1: hipLaunchKernelGGL(rope_kv_write_quads_kernel<1>, dim3(T), dim3(256), 0, stream, a); break;
            case 2: hipLaunchKernelGGL(rope_kv_write_quads_kernel<2>, dim3(T), dim3(256), 0, stream, a); break;
            case 3: hipLaunchKernelGGL(rope_kv_write_quads_kernel<3>, dim3(T), dim3(256), 0, stream, a); break;
            case 4: hipLaunchKernelGGL(rope_kv_write_quads_kernel<4>, dim3(T), dim3(256), 0, stream, a); break;
            case 5: hipLaunchKernelGGL(rope_kv_write_quads_kernel<5>, dim3(T), dim3(256), 0, stream, a); break;
            case 6: hipLaunchKernelGGL(rope_kv_write_quads_kernel<6>, dim3(T), dim3(256), 0, stream, a); break;
            case 7: hipLaunchKernelGGL(rope_kv_write_quads_kernel<7>, dim3(T), dim3(256), 0, stream, a); break;
            default: hipLaunchKernelGGL(rope_kv_write_quads_kernel<8>, dim3(T), dim3(256), 0, stream, a); break;
        }
        return check_launch("rope_kv_write");
    }
    hipLaunchKernelGGL(rope_kv_write_kernel, dim3(T), dim3(256), (size_t)stride * sizeof(float), stream, a);
    return check_launch("rope_kv_write");
}
