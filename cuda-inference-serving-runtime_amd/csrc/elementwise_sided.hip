// Row-wise kernels of models whose embedding adds a vector of the position and whose layers read a table by the token:
//   x[r] = table[token_r] * scale + the sinusoids of position r, and the norm that reads x first
//   act[r, c] = gelu_tanh(z[r, c]) * side[token_r, first + c]
// The residual stream, angles and norms are float; `T` is the storage type of activations (float or bf16).
#include "common.h"

// ------------------------------------------------------------------ embedding with sinusoidal positions
// One block a row.  Columns 2 i and 2 i + 1 of a position's vector are sine and cosine of 2 pi position turns[i]; the
// turns are double, so that the angle of a far position keeps the bits that a float angle would have lost.  With
// norm_w the norm that reads the rows first is made on the way: normed = rmsnorm(x) * norm_w.
template <typename TE, typename TH>
__global__ void __launch_bounds__(256)
embedding_sinusoid_kernel(const int* __restrict__ tokens, const int* __restrict__ positions, const TE* __restrict__ table,
                          const double* __restrict__ turns, float* __restrict__ out, const float* __restrict__ norm_w, float eps,
                          TH* __restrict__ normed, int dim, int vocab, float scale) {
    __shared__ float red[4];
    const int row = blockIdx.x;
    int tok = tokens[row];
    tok = tok < 0 ? 0 : tok >= vocab ? vocab - 1 : tok;
    const double at = (double)positions[row];
    const TE* e = table + (size_t)tok * dim;
    float* o = out + (size_t)row * dim;
    float ss = 0.f;
    for (int d = 2 * threadIdx.x; d < dim; d += 512) {
        double t = at * turns[d / 2];
        t -= floor(t);
        float s, c;
        sincosf((float)(t * 6.283185307179586), &s, &c);
        const float v0 = load_f32(e + d) * scale + s;
        o[d] = v0;
        ss += v0 * v0;
        if (d + 1 < dim) {
            const float v1 = load_f32(e + d + 1) * scale + c;
            o[d + 1] = v1;
            ss += v1 * v1;
        }
    }
    if (!norm_w) return;
    const float rs = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)dim + eps);
    for (int d = 2 * threadIdx.x; d < dim; d += 512)          // (a thread reads back what it wrote itself)
        for (int j = 0; j < 2 && d + j < dim; ++j) store_f32(normed + (size_t)row * dim + d + j, o[d + j] * rs * norm_w[d + j]);
}

extern "C" int cisr_embedding_sinusoid(const int* tokens, const int* positions, const void* table, const double* turns, float* out,
                                       const float* norm_w, float eps, void* normed, int rows, int dim, int vocab, float scale,
                                       int table_dtype, int normed_dtype, hipStream_t stream) {
    if (rows <= 0) return 0;
    if (dim <= 0 || vocab <= 0 || !turns || (norm_w && !normed)) return (int)hipErrorInvalidValue;
#define EMB(TE, TH) embedding_sinusoid_kernel<TE, TH><<<rows, 256, 0, stream>>>(tokens, positions, (const TE*)table, turns, out, norm_w, eps, (TH*)normed, dim, vocab, scale)
    if (table_dtype == DT_F32) { if (normed_dtype == DT_F32) EMB(float, float); else EMB(float, bf16_t); }
    else { if (normed_dtype == DT_F32) EMB(bf16_t, float); else EMB(bf16_t, bf16_t); }
#undef EMB
    return CISR_LAUNCH_CHECK();
}

// ------------------------------------------------------------------ a table row of the token, gated
// act[r, c] = gelu_tanh(z[r * ldz + c]) * side[token_r * ld_side + first + c] for c < width, zero for width <= c < padded.
template <typename T>
__global__ void __launch_bounds__(256)
side_gate_kernel(const float* __restrict__ z, int ldz, const int* __restrict__ tokens, const T* __restrict__ side, int ld_side, int first,
                 T* __restrict__ act, int width, int padded, int vocab, size_t n) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const size_t row = i / padded;
    const int c = (int)(i % padded);
    float v = 0.f;
    if (c < width) {
        int tok = tokens[row];
        tok = tok < 0 ? 0 : tok >= vocab ? vocab - 1 : tok;
        v = unary_activation(z[row * ldz + c], ACT_GELU_TANH) * load_f32(side + (size_t)tok * ld_side + first + c);
    }
    store_f32(act + i, v);
}

extern "C" int cisr_side_gate(const float* z, int ldz, const int* tokens, const void* side, int ld_side, int first, void* act, int rows,
                              int width, int padded, int vocab, int dtype, hipStream_t stream) {
    const size_t n = (size_t)rows * padded;
    if (n == 0) return 0;
    if (width <= 0 || padded < width || first < 0 || first + width > ld_side || ldz < width || vocab <= 0) return (int)hipErrorInvalidValue;
    const unsigned blocks = (unsigned)((n + 255) / 256);
    if (dtype == DT_F32) side_gate_kernel<float><<<blocks, 256, 0, stream>>>(z, ldz, tokens, (const float*)side, ld_side, first, (float*)act, width, padded, vocab, n);
    else side_gate_kernel<bf16_t><<<blocks, 256, 0, stream>>>(z, ldz, tokens, (const bf16_t*)side, ld_side, first, (bf16_t*)act, width, padded, vocab, n);
    return CISR_LAUNCH_CHECK();
}
