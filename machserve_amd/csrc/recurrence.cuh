// What the kernels of recurrences share: the request a row belongs to, and the functions of their gates (32-bit in every build).
#pragma once
#include "common.cuh"

namespace ms {

// The request that row t belongs to: the last s with seq_q_start[s] <= t (starts ascend with s).
__device__ __forceinline__ int seq_of_row(int t, const int* __restrict__ seq_q_start, int S) {
    int lo = 0, hi = S - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (seq_q_start[mid] <= t) lo = mid;
        else hi = mid - 1;
    }
    return lo;
}

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

// Requests' rows cut into pieces of L rows, all pieces of a step numbered in one list: request s has the numbers from
// seq_q_start[s] / L + s on (ceil(rows / L) of them: its range never reaches the next request's), so T rows of S requests
// have at most T / L + S numbers, and some numbers stand for no piece.
struct Piece {
    int s, first;  // the request, and the piece's first row counted from the request's first row of the step
};
__device__ __forceinline__ int piece_base(int s, int L, const int* __restrict__ seq_q_start) { return seq_q_start[s] / L + s; }
__device__ __forceinline__ Piece piece_of(int number, int L, const int* __restrict__ seq_q_start, int S) {
    int lo = 0, hi = S - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) >> 1;
        if (piece_base(mid, L, seq_q_start) <= number) lo = mid;
        else hi = mid - 1;
    }
    return Piece{lo, (number - piece_base(lo, L, seq_q_start)) * L};
}

}  // namespace ms
