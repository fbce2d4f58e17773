// Linear attention with a decay a head that no input changes, S <- lambda S + k v^T, o = S^T q, with q, k and v the silu of
// the stored rows (float): single rows by a kernel that takes a head's whole state in 16-byte accesses, prompt portions
// chunk by chunk on the matrix cores (float operands, v_mfma_f32_16x16x4_f32).  With a chunk's rows counted from 0, n of
// them, and S0 the state at its start:
//
//   end:      E = sum_i lambda^(n - 1 - i) k_i v_i^T                              (all chunks side by side)
//   carry:    S0 of the next chunk = lambda^n S0 + E                             (an element a thread, chunk after chunk)
//   results:  o_i = lambda^(i + 1) S0^T q_i + sum_(j <= i) lambda^(i - j) (q_i . k_j) v_j     (all chunks side by side)
//
// A chunk's slot in the buffer of states is seg_start / 64 + segment + its number, so the number of slots is a function of
// the numbers of rows and segments only (a segment without rows owns a slot without a chunk).  Powers of lambda are made in
// double and rounded once.
#include "common.h"

#define LCHUNK 64

typedef __attribute__((ext_vector_type(4))) float f32x4_t;

struct LightningArgs {
    const float* q; int ldq;          // q[t * ldq + head * R + r]
    const float* k; int ldk;
    const float* v; int ldv;          // v[t * ldv + head * C + c]
    const float* decay;               // [heads]
    float* out; int ldo;              // out[t * ldo + head * C + c]
    float* state; long long slot_stride;   // state + slot * slot_stride + (head * R + r) * C + c
    const int* seg_start; const int* state_slots;
    int R, C, heads, segments;
    float* carry;                     // [slots][heads][R][C]
};

// an element at a 32-bit byte offset from a base that is uniform over the wave (no 64-bit arithmetic a load)
__device__ __forceinline__ float element_at(const float* base, uint32_t element) { return *(const float*)((const char*)base + (uint32_t)(element * 4u)); }

__device__ __forceinline__ float silu_of(float z) { return z / (1.0f + expf(-z)); }

__device__ __forceinline__ double power_of(double x, int n) {
    double y = 1.0;
    for (; n > 0; n >>= 1, x *= x) if (n & 1) y *= x;
    return y;
}

// The segment whose chunk slots hold `slot`.
__device__ __forceinline__ int lightning_segment(const int* seg_start, int segments, int slot) {
    int lo = 0, hi = segments - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) / 2;
        if (seg_start[mid] / LCHUNK + mid <= slot) lo = mid; else hi = mid - 1;
    }
    return lo;
}

struct LightningChunk { int seg, t0, n; };      // n rows from t0; n <= 0: no chunk
__device__ __forceinline__ LightningChunk lightning_chunk(const LightningArgs& p, int slot) {
    LightningChunk c;
    c.seg = lightning_segment(p.seg_start, p.segments, slot);
    const int s0 = p.seg_start[c.seg];
    c.t0 = s0 + (slot - s0 / LCHUNK - c.seg) * LCHUNK;
    c.n = c.t0 < s0 ? 0 : min(LCHUNK, p.seg_start[c.seg + 1] - c.t0);
    return c;
}

// ------------------------------------------------------------------------------------------ the chunks' own end states
// A block a (chunk, head, 128 columns): the keys, silu'd and decayed to the chunk's end, wait in LDS; a wave owns 16-column
// tiles and all rows of the state, four row tiles at a time; its values come straight from memory.
#define LCOLS 128
__global__ void __launch_bounds__(256, 4) lightning_end_kernel(LightningArgs p) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float pw[LCHUNK];
    const LightningChunk ch = lightning_chunk(p, blockIdx.x);
    if (ch.n <= 0) return;
    const int head = blockIdx.y, tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid / WAVE), lane = tid % WAVE, r = lane % 16, g = lane / 16;
    const int R = p.R, C = p.C, n = ch.n, Rp = (R + 63) / 64 * 64, RS = Rp + 16;
    const float* vh = p.v + (size_t)ch.t0 * p.ldv + (size_t)head * C;
    // a wave's first tile's values are asked for before the keys' way into LDS, every following tile's during the one before
    float b[LCHUNK / 4];
    auto ask = [&](int ct) {
        const int cc = min((int)blockIdx.z * LCOLS + ct * 16 + r, C - 1);
#pragma unroll
        for (int s = 0; s < LCHUNK / 4; ++s) b[s] = element_at(vh, (uint32_t)(min(4 * s + g, n - 1) * p.ldv + cc));
    };
    ask(wave);
    if (tid < n) pw[tid] = (float)power_of((double)p.decay[head], n - 1 - tid);
    __syncthreads();
    const float* kh = p.k + (size_t)ch.t0 * p.ldk + (size_t)head * R;
    for (int c = lane; c < Rp; c += 64)
#pragma unroll 8
        for (int i = wave; i < LCHUNK; i += 4) {
            const float x = element_at(kh, (uint32_t)(min(i, n - 1) * p.ldk + min(c, R - 1)));
            lds[i * RS + c] = i < n && c < R ? silu_of(x) * pw[i] : 0.f;
        }
    __syncthreads();
    float* end = p.carry + ((size_t)blockIdx.x * p.heads + head) * R * C;
#pragma unroll 1
    for (int ct = wave; ct < LCOLS / 16; ct += 4) {
        const int c = blockIdx.z * LCOLS + ct * 16 + r;
        if (blockIdx.z * LCOLS + ct * 16 >= C) break;                // (uniform over the wave)
        float val[LCHUNK / 4];
#pragma unroll
        for (int s = 0; s < LCHUNK / 4; ++s) val[s] = silu_of(b[s]);   // (rows behind the last are the last: their keys are zero)
        ask(ct + 4);
#pragma unroll 1
        for (int rt0 = 0; rt0 < Rp / 16; rt0 += 4) {
            f32x4_t acc[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < LCHUNK / 4; ++s) {
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(lds[(4 * s + g) * RS + (rt0 + j) * 16 + r], val[s], acc[j], 0, 0, 0);
            }
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int row = (rt0 + j) * 16 + 4 * g + e;
                    if (row < R && c < C) *(float*)((char*)end + (uint32_t)(row * C + c) * 4u) = acc[j][e];
                }
        }
    }
}

// ------------------------------------------------------------------------------------------ the states at the chunks' starts
// A thread an element of a segment's state: carry[chunk] (its own end) becomes the state at its start; the segment's state
// moves on.  Eight chunks' loads are on their way together.
__global__ void __launch_bounds__(256) lightning_carry_kernel(LightningArgs p) {
    const int seg = blockIdx.y;
    const size_t idx = (size_t)blockIdx.x * 256 + threadIdx.x, all = (size_t)p.heads * p.R * p.C;
    const int s0 = p.seg_start[seg], len = p.seg_start[seg + 1] - s0;
    if (len <= 0 || idx >= all) return;
    const int chunks = (len + LCHUNK - 1) / LCHUNK;
    float* carry = p.carry + (size_t)(s0 / LCHUNK + seg) * all + idx;
    float* state = p.state + (long long)p.state_slots[seg] * p.slot_stride + idx;
    const double lambda = (double)p.decay[idx / ((size_t)p.R * p.C)];
    const float whole = (float)power_of(lambda, LCHUNK), last = (float)power_of(lambda, len - (chunks - 1) * LCHUNK);
    float S = *state;
    for (int c0 = 0; c0 < chunks; c0 += 8) {
        float own[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) own[j] = carry[(size_t)min(c0 + j, chunks - 1) * all];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            if (c0 + j >= chunks) continue;
            carry[(size_t)(c0 + j) * all] = S;
            S = (c0 + j == chunks - 1 ? last : whole) * S + own[j];
        }
    }
    *state = S;
}

// ------------------------------------------------------------------------------------------ the chunks' results
// A block a (chunk, head, 128 columns).  Queries and keys wait in LDS; the wave w makes the 16 rows w of the decayed scores
// P, which then take the keys' place; a wave owns 16-column tiles of the results and all four row tiles, with the state and
// the values straight from memory (each read once a block).
__global__ void __launch_bounds__(256, 3) lightning_out_kernel(LightningArgs p) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float pw[LCHUNK + 1];
    const LightningChunk ch = lightning_chunk(p, blockIdx.x);
    if (ch.n <= 0) return;
    const int head = blockIdx.y, tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid / WAVE), lane = tid % WAVE, r = lane % 16, g = lane / 16;
    const int R = p.R, C = p.C, n = ch.n, Rp = (R + 63) / 64 * 64, RS = Rp + 4, PS = LCHUNK + 4;
    float* sq = lds;
    const float* vh = p.v + (size_t)ch.t0 * p.ldv + (size_t)head * C;
    const float* start = p.carry + ((size_t)blockIdx.x * p.heads + head) * R * C;
    float b[LCHUNK / 4], s0[16];         // a tile's values, and sixteen rows of the state: a wave's first are asked for here
    auto ask_values = [&](int ct) {
        const int cc = min((int)blockIdx.z * LCOLS + ct * 16 + r, C - 1);
#pragma unroll
        for (int s = 0; s < LCHUNK / 4; ++s) b[s] = element_at(vh, (uint32_t)(min(4 * s + g, n - 1) * p.ldv + cc));
    };
    auto ask_state = [&](int ct, int k0) {
        const int cc = min((int)blockIdx.z * LCOLS + ct * 16 + r, C - 1);
#pragma unroll
        for (int s = 0; s < 16; ++s) s0[s] = element_at(start, (uint32_t)(min(k0 + 4 * s + g, R - 1) * C + cc));
    };
    ask_state(wave, 0);
    ask_values(wave);
    float* sk = lds + LCHUNK * RS;       // and P, [LCHUNK][PS], once the scores are made (RS >= PS)
    if (tid <= LCHUNK) pw[tid] = (float)power_of((double)p.decay[head], tid);
    const float* qh = p.q + (size_t)ch.t0 * p.ldq + (size_t)head * R;
    const float* kh = p.k + (size_t)ch.t0 * p.ldk + (size_t)head * R;
    for (int c = lane; c < Rp; c += 64)
#pragma unroll 8
        for (int i = wave; i < LCHUNK; i += 4) {
            const int row = min(i, n - 1);
            const float x = element_at(qh, (uint32_t)(row * p.ldq + min(c, R - 1))), y = element_at(kh, (uint32_t)(row * p.ldk + min(c, R - 1)));
            const bool in = i < n && c < R;
            sq[i * RS + c] = in ? silu_of(x) : 0.f;
            sk[i * RS + c] = in ? silu_of(y) : 0.f;
        }
    __syncthreads();
    f32x4_t sc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) sc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k0 = 0; k0 < Rp; k0 += 4) {
        const float a = sq[(wave * 16 + r) * RS + k0 + g];
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (j <= wave) sc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, sk[(j * 16 + r) * RS + k0 + g], sc[j], 0, 0, 0);
    }
    __syncthreads();                     // (every wave has read its keys)
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int row = wave * 16 + 4 * g + e, col = j * 16 + r;
            sk[row * PS + col] = col <= row ? sc[j][e] * pw[max(row - col, 0)] : 0.f;
        }
    __syncthreads();
    const int row_tiles = (n + 15) / 16;
#pragma unroll 1
    for (int ct = wave; ct < LCOLS / 16; ct += 4) {
        const int c = blockIdx.z * LCOLS + ct * 16 + r;
        if (blockIdx.z * LCOLS + ct * 16 >= C) break;                // (uniform over the wave)
        f32x4_t acc[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
        for (int k0 = 0; k0 < Rp; k0 += 64) {                        // sixteen steps' loads of the state together
            if (k0 > 0) ask_state(ct, k0);
#pragma unroll
            for (int s = 0; s < 16; ++s) {
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(sq[(j * 16 + r) * RS + k0 + 4 * s + g], s0[s], acc[j], 0, 0, 0);
            }
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[j][e] *= pw[j * 16 + 4 * g + e + 1];
        ask_state(ct + 4, 0);
#pragma unroll
        for (int s = 0; s < LCHUNK / 4; ++s) {
            const float value = silu_of(b[s]);
#pragma unroll
            for (int j = s / 4; j < 4; ++j)                           // (row tiles before this key's see none of it)
                acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(sk[(j * 16 + r) * PS + 4 * s + g], value, acc[j], 0, 0, 0);
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j == 0) ask_values(ct + 4);
            if (j >= row_tiles) continue;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int row = j * 16 + 4 * g + e;
                if (row < n && c < C) p.out[(size_t)(ch.t0 + row) * p.ldo + (size_t)head * C + c] = acc[j][e];
            }
        }
    }
}

// ------------------------------------------------------------------------------------------ single rows
// A block a (segment, head), every segment one row (segments without a row are skipped): a thread takes four neighbouring
// columns of every (256 / (C / 4))-th row of the state, eight rows' loads on their way together; the columns' sums meet in
// LDS.  C a multiple of 4 and at most 1,024, the state's rows 16-byte aligned.
__global__ void __launch_bounds__(256) lightning_step_kernel(LightningArgs p) {
    __shared__ float sq[256], sk[256];
    __shared__ __attribute__((aligned(16))) f32x4_t part[256];
    const int seg = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, R = p.R, C4 = p.C / 4;
    const int t = p.seg_start[seg];
    if (p.seg_start[seg + 1] <= t) return;
    const int groups = 256 / C4, c4 = tid % C4, rg = tid / C4;
    const bool live = rg < groups;
    f32x4_t* S = (f32x4_t*)(p.state + (long long)p.state_slots[seg] * p.slot_stride + (size_t)head * R * p.C) + c4;
    f32x4_t now[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int row = rg + j * groups;
        now[j] = live && row < R ? S[(size_t)row * C4] : (f32x4_t){0.f, 0.f, 0.f, 0.f};
    }
    f32x4_t v = *(const f32x4_t*)(p.v + (size_t)t * p.ldv + (size_t)head * p.C + 4 * c4);
    if (tid < R) {
        sq[tid] = silu_of(p.q[(size_t)t * p.ldq + (size_t)head * R + tid]);
        sk[tid] = silu_of(p.k[(size_t)t * p.ldk + (size_t)head * R + tid]);
    }
    const float lambda = p.decay[head];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = silu_of(v[e]);
    __syncthreads();
    f32x4_t sum = {0.f, 0.f, 0.f, 0.f};
    for (int j0 = 0; j0 * groups < R; j0 += 8) {
        if (j0 > 0) {
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int row = rg + (j0 + j) * groups;
                now[j] = live && row < R ? S[(size_t)row * C4] : (f32x4_t){0.f, 0.f, 0.f, 0.f};
            }
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int row = rg + (j0 + j) * groups;
            if (!live || row >= R) continue;
            const float k = sk[row], q = sq[row];
#pragma unroll
            for (int e = 0; e < 4; ++e) { now[j][e] = lambda * now[j][e] + k * v[e]; sum[e] += now[j][e] * q; }
            S[(size_t)row * C4] = now[j];
        }
    }
    part[tid] = sum;
    __syncthreads();
    if (tid < C4) {
        for (int i = 1; i < groups; ++i) sum += part[i * C4 + tid];
        *(f32x4_t*)(p.out + (size_t)t * p.ldo + (size_t)head * p.C + 4 * tid) = sum;
    }
}

static int lightning_bad(const LightningArgs& p) {
    return p.R <= 0 || p.R > 256 || p.C <= 0 || p.heads <= 0 || p.heads > 65535 || p.segments > 65535;
}

extern "C" int cisr_lightning_step(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* decay, float* out,
                                   int ldo, float* state, long long slot_stride, const int* seg_start, const int* state_slots, int segments,
                                   int heads, int R, int C, hipStream_t stream) {
    if (segments <= 0) return 0;
    const LightningArgs p{q, ldq, k, ldk, v, ldv, decay, out, ldo, state, slot_stride, seg_start, state_slots, R, C, heads, segments, nullptr};
    if (lightning_bad(p) || C % 4 || C > 1024 || ldv % 4 || ldo % 4 || slot_stride % 4 || ((uintptr_t)v) % 16 || ((uintptr_t)out) % 16 || ((uintptr_t)state) % 16)
        return (int)hipErrorInvalidValue;
    lightning_step_kernel<<<dim3(segments, heads), 256, 0, stream>>>(p);
    return CISR_LAUNCH_CHECK();
}

// `slots`: of the buffer of states, at least rows / 64 + segments.
extern "C" int cisr_lightning_chunks(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* decay, float* out,
                                     int ldo, float* state, long long slot_stride, const int* seg_start, const int* state_slots, int segments,
                                     int heads, int R, int C, int slots, float* carry, hipStream_t stream) {
    if (segments <= 0 || slots <= 0) return 0;
    const LightningArgs p{q, ldq, k, ldk, v, ldv, decay, out, ldo, state, slot_stride, seg_start, state_slots, R, C, heads, segments, carry};
    if ((long long)LCHUNK * ldq >= (1 << 29) || (long long)LCHUNK * ldk >= (1 << 29) || (long long)LCHUNK * ldv >= (1 << 29) || (long long)R * C >= (1 << 29))
        return (int)hipErrorInvalidValue;                       // (offsets inside a chunk's rows fit 32 bits)
    if (lightning_bad(p) || !carry || (C + LCOLS - 1) / LCOLS > 65535) return (int)hipErrorInvalidValue;
    const dim3 grid(slots, heads, (C + LCOLS - 1) / LCOLS);
    const size_t end_lds = (size_t)LCHUNK * ((R + 63) / 64 * 64 + 16) * sizeof(float);
    const size_t out_lds = (size_t)2 * LCHUNK * ((R + 63) / 64 * 64 + 4) * sizeof(float);
    hipError_t e = hipSuccess;
    if (end_lds > 65536 - 1024) e = hipFuncSetAttribute((const void*)lightning_end_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)end_lds);
    if (e == hipSuccess && out_lds > 65536 - 1024) e = hipFuncSetAttribute((const void*)lightning_out_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)out_lds);
    if (e != hipSuccess) return (int)e;
    lightning_end_kernel<<<grid, 256, end_lds, stream>>>(p);
    int err = CISR_LAUNCH_CHECK();
    if (err) return err;
    lightning_carry_kernel<<<dim3((unsigned)(((size_t)heads * R * C + 255) / 256), segments), 256, 0, stream>>>(p);
    err = CISR_LAUNCH_CHECK();
    if (err) return err;
    lightning_out_kernel<<<grid, 256, out_lds, stream>>>(p);
    return CISR_LAUNCH_CHECK();
}
