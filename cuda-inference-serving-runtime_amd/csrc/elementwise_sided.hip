// Row-wise kernels of models whose embedding adds a vector of the position and whose layers read a table by the token:
//   x[r] = table[token_r] * scale + the sinusoids of position r, and the norm that reads x first
//   act[r, c] = gelu_tanh(z[r, c]) * side[token_r, first + c]
// The residual stream, angles and norms are float; `T` is the storage type of activations (float or bf16).
#include "common.h"

// ------------------------------------------------------------------ embedding with sinusoidal positions
// One block a row.  Columns 2 i and 2 i + 1 of a position's vector are sine and cosine of 2 pi position turns[i]; the
// turns are double, so that the angle of a far position keeps the bits that a float angle would have lost.  With
// norm_w the norm that reads the rows first is made on the way: normed = rmsnorm(x) * norm_w.
// P > 0: a thread's column pairs wait in registers (rows of up to 512 P columns), all their loads on their way together;
// P 0: any width, the row is read back.
template <typename TE, typename TH, int P>
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
    auto vector_of = [&](double turn, float& s, float& c) {
        double t = at * turn;
        t -= rint(t);
        sincospif((float)(2.0 * t), &s, &c);
    };
    float ss = 0.f;
    if constexpr (P > 0) {
        double turn[P];
        float v[P][2], w[P][2];
#pragma unroll
        for (int i = 0; i < P; ++i) {
            const int d = 2 * (threadIdx.x + 256 * i);
            turn[i] = d < dim ? turns[d / 2] : 0.0;
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const int dd = min(d + j, dim - 1);
                v[i][j] = load_f32(e + dd);
                w[i][j] = norm_w ? norm_w[dd] : 1.f;
            }
        }
#pragma unroll
        for (int i = 0; i < P; ++i) {
            const int d = 2 * (threadIdx.x + 256 * i);
            float add[2];
            vector_of(turn[i], add[0], add[1]);
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                v[i][j] = v[i][j] * scale + add[j];
                if (d + j < dim) { o[d + j] = v[i][j]; ss += v[i][j] * v[i][j]; }
            }
        }
        if (!norm_w) return;
        const float rs = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)dim + eps);
#pragma unroll
        for (int i = 0; i < P; ++i) {
            const int d = 2 * (threadIdx.x + 256 * i);
#pragma unroll
            for (int j = 0; j < 2; ++j) if (d + j < dim) store_f32(normed + (size_t)row * dim + d + j, v[i][j] * rs * w[i][j]);
        }
    } else {
        for (int d = 2 * threadIdx.x; d < dim; d += 512) {
            float add[2];
            vector_of(turns[d / 2], add[0], add[1]);
            for (int j = 0; j < 2 && d + j < dim; ++j) {
                const float v = load_f32(e + d + j) * scale + add[j];
                o[d + j] = v;
                ss += v * v;
            }
        }
        if (!norm_w) return;
        const float rs = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)dim + eps);
        for (int d = 2 * threadIdx.x; d < dim; d += 512)          // (a thread reads back what it wrote itself)
            for (int j = 0; j < 2 && d + j < dim; ++j) store_f32(normed + (size_t)row * dim + d + j, o[d + j] * rs * norm_w[d + j]);
    }
}

extern "C" int cisr_embedding_sinusoid(const int* tokens, const int* positions, const void* table, const double* turns, float* out,
                                       const float* norm_w, float eps, void* normed, int rows, int dim, int vocab, float scale,
                                       int table_dtype, int normed_dtype, hipStream_t stream) {
    if (rows <= 0) return 0;
    if (dim <= 0 || vocab <= 0 || !turns || (norm_w && !normed)) return (int)hipErrorInvalidValue;
#define EMB_P(TE, TH, P) embedding_sinusoid_kernel<TE, TH, P><<<rows, 256, 0, stream>>>(tokens, positions, (const TE*)table, turns, out, norm_w, eps, (TH*)normed, dim, vocab, scale)
#define EMB(TE, TH) do { if (dim <= 512) EMB_P(TE, TH, 1); else if (dim <= 1024) EMB_P(TE, TH, 2); else if (dim <= 2048) EMB_P(TE, TH, 4); \
                         else if (dim <= 4096) EMB_P(TE, TH, 8); else EMB_P(TE, TH, 0); } while (0)
    if (table_dtype == DT_F32) { if (normed_dtype == DT_F32) EMB(float, float); else EMB(float, bf16_t); }
    else { if (normed_dtype == DT_F32) EMB(bf16_t, float); else EMB(bf16_t, bf16_t); }
#undef EMB
#undef EMB_P
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

// Steps of few rows: the gate's product as well, z = h[r] . w[c] with bf16 operands.  grid (padded / 16, rows): a block of
// four waves makes 16 columns of one row, a wave 4 of them, all loads of a row of w in flight together; hidden % 8 == 0 and
// at most 64 x 8 x SIDE_CHUNKS.
#define SIDE_CHUNKS 16
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4_side;
__global__ void __launch_bounds__(256)
side_rows_kernel(const bf16_t* __restrict__ h, int ldh, const bf16_t* __restrict__ w, const int* __restrict__ tokens,
                 const bf16_t* __restrict__ side, int ld_side, int first, bf16_t* __restrict__ act, int hidden, int width, int padded, int vocab) {
    const int row = blockIdx.y, wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
    const int c0 = (blockIdx.x * 4 + wave) * 4;
    if (c0 >= padded) return;
    const bf16_t* hr = h + (size_t)row * ldh;
    int tok = tokens[row];
    tok = tok < 0 ? 0 : tok >= vocab ? vocab - 1 : tok;
    const bool mine = lane < 4 && c0 + lane < width;
    const float e = mine ? bf16_to_f32(side[(size_t)tok * ld_side + first + c0 + lane]) : 0.f;
    const u32x4_side zero = {0u, 0u, 0u, 0u};
    float sum[4] = {0.f, 0.f, 0.f, 0.f};
    const int chunks = (hidden + 511) / 512;
#pragma unroll
    for (int c = 0; c < SIDE_CHUNKS; ++c) {
        if (c >= chunks) continue;
        const int k = (c * 64 + lane) * 8;
        const u32x4_side a = k < hidden ? *(const u32x4_side*)(hr + k) : zero;
        u32x4_side b[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) b[j] = k < hidden ? *(const u32x4_side*)(w + (size_t)min(c0 + j, padded - 1) * hidden + k) : zero;
        const uint32_t aw[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const uint32_t bw[4] = {b[j].x, b[j].y, b[j].z, b[j].w};
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                sum[j] = fmaf(__uint_as_float(aw[x] << 16), __uint_as_float(bw[x] << 16), sum[j]);
                sum[j] = fmaf(__uint_as_float(aw[x] & 0xffff0000u), __uint_as_float(bw[x] & 0xffff0000u), sum[j]);
            }
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) sum[j] = wave_sum(sum[j]);
    if (lane < 4 && c0 + lane < padded)
        act[(size_t)row * padded + c0 + lane] = f32_to_bf16(mine ? unary_activation(lane == 0 ? sum[0] : lane == 1 ? sum[1] : lane == 2 ? sum[2] : sum[3], ACT_GELU_TANH) * e : 0.f);
}

extern "C" int cisr_side_rows(const void* h, int ldh, const void* w, const int* tokens, const void* side, int ld_side, int first, void* act,
                              int rows, int hidden, int width, int padded, int vocab, hipStream_t stream) {
    if (rows <= 0) return 0;
    if (hidden <= 0 || hidden % 8 || ldh % 8 || hidden > 512 * SIDE_CHUNKS || width <= 0 || padded < width || first < 0 || first + width > ld_side ||
        vocab <= 0 || rows > 65535 || ((uintptr_t)h) % 16 || ((uintptr_t)w) % 16)
        return (int)hipErrorInvalidValue;
    side_rows_kernel<<<dim3((padded + 15) / 16, rows), 256, 0, stream>>>((const bf16_t*)h, ldh, (const bf16_t*)w, tokens, (const bf16_t*)side, ld_side, first,
                                                                       (bf16_t*)act, hidden, width, padded, vocab);
    return CISR_LAUNCH_CHECK();
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
