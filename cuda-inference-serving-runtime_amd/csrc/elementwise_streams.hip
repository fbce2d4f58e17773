// Row-wise kernels of models whose residual is several streams (hyper-connections).  A row of x holds its `S` streams one
// after the other, x[t, s * H + d], float.  Around a sublayer,
//
//   u = sum_s in[s] x_s,  h = rmsnorm(u) * w          what the sublayer reads
//   x_t <- sum_s mix[s, t] x_s + out[t] y             the right side as it was (row s of mix: where x_s goes)
//
// and the two meet in one kernel: the write of a sublayer's result y and the read (and norm) of the sublayer that comes
// next, so a row of streams makes one trip to memory a sublayer.  y is finished float rows or the partial sums of a cut
// product, added in slice order on the way.  The embedding fills the streams and makes the first read the same way.
// With it: logits <- cap tanh(logits / cap).
#include "common.h"

#define MAX_STREAMS 8

struct StreamArgs {
    float* x; int H;
    const float* y; int slices; long long slice_stride;       // slices 0: y is finished rows
    const float* mix; const float* out;                       // null: x is only read
    const float* in; const float* w; float eps;               // w null: no read
    void* h;                                                  // [n_rows, H]
    const int* rows;                                          // rows of x to read (read only), or null
    const int* ids; const void* table; int vocab;             // embedding: the streams' first contents
};

enum { STREAMS_READ = 0, STREAMS_STEP = 1, STREAMS_EMBED = 2 };

// One block a row, NT threads, R words of four floats a thread (H <= 4 NT R), everything in registers.
template <int S, int MODE, typename T, typename TE, int NT, int R>
__global__ void __launch_bounds__(NT) streams_kernel(StreamArgs p) {
    __shared__ float red[NT / WAVE];
    const int row = blockIdx.x, tid = threadIdx.x, n4 = p.H / 4;
    const int src = MODE == STREAMS_READ && p.rows ? p.rows[row] : row;
    float4* xr = (float4*)(p.x + (size_t)src * S * p.H);
    float4 v[R][S], u[R];
    if (MODE == STREAMS_EMBED) {
        int id = p.ids[row];
        if (id < 0 || id >= p.vocab) id = 0;                  // padding rows; real ids are checked on the host
        const TE* e = (const TE*)p.table + (size_t)id * p.H;
#pragma unroll
        for (int i = 0; i < R; ++i) {
            const int c = min(tid + NT * i, n4 - 1);
            const float4 a = make_float4(load_f32(e + 4 * c), load_f32(e + 4 * c + 1), load_f32(e + 4 * c + 2), load_f32(e + 4 * c + 3));
#pragma unroll
            for (int s = 0; s < S; ++s) {
                v[i][s] = a;
                if (tid + NT * i < n4) xr[(size_t)s * n4 + c] = a;
            }
        }
    } else {
#pragma unroll
        for (int i = 0; i < R; ++i)
#pragma unroll
            for (int s = 0; s < S; ++s) v[i][s] = xr[(size_t)s * n4 + min(tid + NT * i, n4 - 1)];
    }
    if (MODE == STREAMS_STEP) {
        float4 y[R];
#pragma unroll
        for (int i = 0; i < R; ++i) y[i] = ((const float4*)(p.y + (size_t)row * p.H))[min(tid + NT * i, n4 - 1)];
        for (int k = 1; k < p.slices; ++k)
#pragma unroll
            for (int i = 0; i < R; ++i) {
                const float4 a = ((const float4*)(p.y + k * p.slice_stride + (size_t)row * p.H))[min(tid + NT * i, n4 - 1)];
                y[i].x += a.x; y[i].y += a.y; y[i].z += a.z; y[i].w += a.w;
            }
#pragma unroll
        for (int i = 0; i < R; ++i) {
            float4 nv[S];
#pragma unroll
            for (int t = 0; t < S; ++t) {
                float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
                for (int s = 0; s < S; ++s) {
                    const float m = p.mix[s * S + t];
                    a.x += m * v[i][s].x; a.y += m * v[i][s].y; a.z += m * v[i][s].z; a.w += m * v[i][s].w;
                }
                const float o = p.out[t];
                a.x += o * y[i].x; a.y += o * y[i].y; a.z += o * y[i].z; a.w += o * y[i].w;
                nv[t] = a;
                if (tid + NT * i < n4) xr[(size_t)t * n4 + tid + NT * i] = a;
            }
#pragma unroll
            for (int t = 0; t < S; ++t) v[i][t] = nv[t];
        }
    }
    if (!p.w) return;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < R; ++i) {
        float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int s = 0; s < S; ++s) {
            const float m = p.in[s];
            a.x += m * v[i][s].x; a.y += m * v[i][s].y; a.z += m * v[i][s].z; a.w += m * v[i][s].w;
        }
        u[i] = a;
        if (tid + NT * i < n4) ss += a.x * a.x + a.y * a.y + a.z * a.z + a.w * a.w;
    }
    const float scale = 1.0f / sqrtf((NT == WAVE ? wave_sum(ss) : block_sum<NT>(ss, red)) / (float)p.H + p.eps);
#pragma unroll
    for (int i = 0; i < R; ++i) {
        const int c = tid + NT * i;
        if (c >= n4) continue;
        const float4 g = ((const float4*)p.w)[c];
        const float a = u[i].x * scale * g.x, b = u[i].y * scale * g.y, cc = u[i].z * scale * g.z, d = u[i].w * scale * g.w;
        if (sizeof(T) == 4) ((float4*)((float*)p.h + (size_t)row * p.H))[c] = make_float4(a, b, cc, d);
        else ((uint2*)((bf16_t*)p.h + (size_t)row * p.H))[c] = make_uint2(pack_bf16x2(a, b), pack_bf16x2(cc, d));
    }
}

// Any width (at most 16,384) and alignment: element by element, the row that is normed waits in LDS for its scale.
template <int S, int MODE, typename T, typename TE>
__global__ void __launch_bounds__(256) streams_plain_kernel(StreamArgs p) {
    __shared__ float red[4];
    extern __shared__ float kept[];
    const int row = blockIdx.x;
    const int src = MODE == STREAMS_READ && p.rows ? p.rows[row] : row;
    float* xr = p.x + (size_t)src * S * p.H;
    const TE* e = nullptr;
    if (MODE == STREAMS_EMBED) {
        int id = p.ids[row];
        if (id < 0 || id >= p.vocab) id = 0;
        e = (const TE*)p.table + (size_t)id * p.H;
    }
    float ss = 0.f;
    for (int d = threadIdx.x; d < p.H; d += 256) {
        float v[S];
#pragma unroll
        for (int s = 0; s < S; ++s) {
            v[s] = MODE == STREAMS_EMBED ? load_f32(e + d) : xr[(size_t)s * p.H + d];
            if (MODE == STREAMS_EMBED) xr[(size_t)s * p.H + d] = v[s];
        }
        if (MODE == STREAMS_STEP) {
            float y = p.y[(size_t)row * p.H + d];
            for (int k = 1; k < p.slices; ++k) y += p.y[k * p.slice_stride + (size_t)row * p.H + d];
            float nv[S];
#pragma unroll
            for (int t = 0; t < S; ++t) {
                float a = 0.f;
#pragma unroll
                for (int s = 0; s < S; ++s) a += p.mix[s * S + t] * v[s];
                nv[t] = a + p.out[t] * y;
                xr[(size_t)t * p.H + d] = nv[t];
            }
#pragma unroll
            for (int t = 0; t < S; ++t) v[t] = nv[t];
        }
        if (!p.w) continue;
        float u = 0.f;
#pragma unroll
        for (int s = 0; s < S; ++s) u += p.in[s] * v[s];
        kept[d] = u;
        ss += u * u;
    }
    if (!p.w) return;
    const float scale = 1.0f / sqrtf(block_sum<256>(ss, red) / (float)p.H + p.eps);
    T* h = (T*)p.h + (size_t)row * p.H;
    for (int d = threadIdx.x; d < p.H; d += 256) store_f32(h + d, kept[d] * scale * p.w[d]);     // (a thread reads back what it wrote)
}

template <int S, int MODE, typename T, typename TE>
static int launch_streams_of(const StreamArgs& p, int n_rows, hipStream_t stream) {
    const bool vec = p.H % 4 == 0 && p.H <= 8192 && (uintptr_t)p.x % 16 == 0 && (uintptr_t)p.y % 16 == 0 && (uintptr_t)p.w % 16 == 0 &&
                     (uintptr_t)p.h % 16 == 0 && (uintptr_t)p.table % 16 == 0 && p.slice_stride % 4 == 0;
    const int n4 = p.H / 4;
#define STREAMS(NT, R) streams_kernel<S, MODE, T, TE, NT, R><<<n_rows, NT, 0, stream>>>(p)
    if (!vec) streams_plain_kernel<S, MODE, T, TE><<<n_rows, 256, (size_t)p.H * sizeof(float), stream>>>(p);
    else if (n4 <= 64) STREAMS(64, 1);
    else if (n4 <= 128) STREAMS(128, 1);
    else if (n4 <= 256) STREAMS(256, 1);
    else if (n4 <= 512) STREAMS(512, 1);
    else if (n4 <= 1024) STREAMS(1024, 1);
    else STREAMS(1024, 2);
#undef STREAMS
    return CISR_LAUNCH_CHECK();
}

template <int MODE, typename T, typename TE>
static int launch_streams(const StreamArgs& p, int streams, int n_rows, hipStream_t stream) {
    if (p.H <= 0 || p.H > 16384 || streams < 1 || streams > MAX_STREAMS) return (int)hipErrorInvalidValue;
    switch (streams) {
        case 1: return launch_streams_of<1, MODE, T, TE>(p, n_rows, stream);
        case 2: return launch_streams_of<2, MODE, T, TE>(p, n_rows, stream);
        case 3: return launch_streams_of<3, MODE, T, TE>(p, n_rows, stream);
        case 4: return launch_streams_of<4, MODE, T, TE>(p, n_rows, stream);
        case 5: return launch_streams_of<5, MODE, T, TE>(p, n_rows, stream);
        case 6: return launch_streams_of<6, MODE, T, TE>(p, n_rows, stream);
        case 7: return launch_streams_of<7, MODE, T, TE>(p, n_rows, stream);
        default: return launch_streams_of<8, MODE, T, TE>(p, n_rows, stream);
    }
}

// h[r] = rmsnorm(sum_s in[s] x[rows ? rows[r] : r, s]) * w
extern "C" int cisr_streams_read(const float* x, const float* in, const float* w, float eps, void* h, const int* rows, int n_rows,
                                 int H, int streams, int out_dtype, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (!in || !w || !h) return (int)hipErrorInvalidValue;
    StreamArgs p = {};
    p.x = (float*)x; p.H = H; p.in = in; p.w = w; p.eps = eps; p.h = h; p.rows = rows;
    if (out_dtype == DT_F32) return launch_streams<STREAMS_READ, float, float>(p, streams, n_rows, stream);
    return launch_streams<STREAMS_READ, bf16_t, float>(p, streams, n_rows, stream);
}

// x_t <- sum_s mix[s, t] x_s + out[t] y in place (y: finished rows [n_rows, H], or with slices > 0 that many partial sums,
// [slices, n_rows, H]); with w also the read of what comes next, h = rmsnorm(sum_s in[s] x_s) * w of the new streams.
extern "C" int cisr_streams_step(float* x, const float* y, int slices, const float* mix, const float* out, const float* in,
                                 const float* w, float eps, void* h, int n_rows, int H, int streams, int out_dtype,
                                 hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (!y || !mix || !out || slices < 0 || (w && (!in || !h))) return (int)hipErrorInvalidValue;
    StreamArgs p = {};
    p.x = x; p.H = H; p.y = y; p.slices = slices; p.slice_stride = (long long)n_rows * H; p.mix = mix; p.out = out;
    p.in = in; p.w = w; p.eps = eps; p.h = h;
    if (out_dtype == DT_F32) return launch_streams<STREAMS_STEP, float, float>(p, streams, n_rows, stream);
    return launch_streams<STREAMS_STEP, bf16_t, float>(p, streams, n_rows, stream);
}

// x_s = table[ids[r]] for every stream; with w also the first read.  h has the table's type.
extern "C" int cisr_streams_embed(const int* ids, const void* table, float* x, const float* in, const float* w, float eps, void* h,
                                  int n_rows, int H, int streams, int vocab, int dtype, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (!ids || !table || vocab <= 0 || (w && (!in || !h))) return (int)hipErrorInvalidValue;
    StreamArgs p = {};
    p.x = x; p.H = H; p.in = in; p.w = w; p.eps = eps; p.h = h; p.ids = ids; p.table = table; p.vocab = vocab;
    if (dtype == DT_F32) return launch_streams<STREAMS_EMBED, float, float>(p, streams, n_rows, stream);
    return launch_streams<STREAMS_EMBED, bf16_t, bf16_t>(p, streams, n_rows, stream);
}

// ------------------------------------------------------------------------------------------------ capped logits
__global__ void __launch_bounds__(256) softcap_kernel(float* __restrict__ x, size_t n, float cap, float inv) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i + 4 <= n) {
        float4 v = *(float4*)(x + i);
        v.x = cap * tanhf(v.x * inv); v.y = cap * tanhf(v.y * inv); v.z = cap * tanhf(v.z * inv); v.w = cap * tanhf(v.w * inv);
        *(float4*)(x + i) = v;
    } else {
        for (size_t j = i; j < n; ++j) x[j] = cap * tanhf(x[j] * inv);
    }
}

extern "C" int cisr_softcap(float* x, long long n, float cap, hipStream_t stream) {
    if (n <= 0) return 0;
    if (!(cap > 0.f) || (uintptr_t)x % 16) return (int)hipErrorInvalidValue;
    softcap_kernel<<<(unsigned)((n + 1023) / 1024), 256, 0, stream>>>(x, (size_t)n, cap, 1.0f / cap);
    return CISR_LAUNCH_CHECK();
}
