// The gated delta rule with a decay a key channel over prompt portions, chunk by chunk on the matrix cores (float operands,
// v_mfma_f32_16x16x4_f32).  A segment's rows in chunks of 16; with D(t, i) the product of a chunk's decays g_(i+1) .. g_t,
// channel by channel, D(t) that of g_0 .. g_t, and S0 the state at the chunk's start:
//
//   A[t, i] = beta_t sum_r k_t k_i D(t, i), i < t          P[t, i] = sum_r q_t k_i D(t, i), i <= t
//   M = (I + A)^-1 diag(beta)
//   U = M (V - Kg S0),   Kg_t = D(t) k_t                      (the rows' writes u_t)
//   o_t = (D(t) q_t)^T S0 + sum_i P[t, i] u_i
//   S  <- D(15) S0 + sum_i (D(15, i) k_i) u_i^T
//
// Every product of decays is made by multiplying decays along the rows: no quotients and no differences of logarithms, so a
// channel whose decays vanish within a chunk costs neither range nor precision.  A first kernel makes, chunk by chunk and
// all side by side, what does not need the state: M V, M Kg, D q, P, D(15, i) k and D(15); a second walks a segment's chunks
// in order, a block a (head, 16 columns of S): its waves own the rows of S in turn, two products with S0, one meeting through
// LDS, one product into S.  Rows behind a segment's end count as k = q = v = 0 with decays of one.
#include "common.h"

#define CHUNK 16

typedef __attribute__((ext_vector_type(4))) float f32x4_t;

struct ChunkArgs {
    const float* q; int ldq;          // q[t * ldq + (head / share) * R + r]
    const float* k; int ldk;
    const float* v; int ldv;          // v[t * ldv + head * C + c]
    const float* g; int ldg;          // g[t * ldg + head * R + r]
    const float* b; int ldb;          // b[t * ldb + head], beta = sigmoid(b)
    float* out; int ldo;
    float* state; long long slot_stride;
    const int* seg_start; const int* state_slots;
    int R, C, share, heads, segments;
    float q_scale;
    int Rp, Cp;                       // R and C rounded up to 16
    int slot0, slots;                 // this launch's chunk slots (a chunk's slot: seg_start / 16 + segment + its number)
    float* work;                      // [slots][heads][chunk_floats]
};

// Floats of a (chunk, head): M Kg and D q as [16][Rp], D(15, i) k as [Rp][16], M V as [Cp][16], P as [16][16], D(15) [Rp].
__host__ __device__ __forceinline__ int chunk_floats(int Rp, int Cp) { return 3 * CHUNK * Rp + CHUNK * Cp + CHUNK * CHUNK + Rp; }

// The segment whose chunk slots hold `slot` (segments without rows own a slot without a chunk).
__device__ __forceinline__ int segment_of_slot(const int* seg_start, int segments, int slot) {
    int lo = 0, hi = segments - 1;
    while (lo < hi) {
        const int mid = (lo + hi + 1) / 2;
        if (seg_start[mid] / CHUNK + mid <= slot) lo = mid; else hi = mid - 1;
    }
    return lo;
}

template <int CTRL>
__device__ __forceinline__ float lanes_moved(float x) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xF, 0xF, false));
}

// the sum over the 16 lanes of an aligned row, in each of them
__device__ __forceinline__ float row_sum(float x) {
    x += lanes_moved<0xB1>(x);                   // quad_perm [1, 0, 3, 2]
    x += lanes_moved<0x4E>(x);                   // quad_perm [2, 3, 0, 1]
    x += lanes_moved<0x141>(x);                  // row_half_mirror
    x += lanes_moved<0x140>(x);                  // row_mirror
    return x;
}

__global__ void __launch_bounds__(256, 4) channel_chunk_kernel(ChunkArgs p) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float sA[CHUNK][CHUNK + 1], sBeta[CHUNK];
    __shared__ __attribute__((aligned(16))) float sM[CHUNK][CHUNK];
    const int slot = p.slot0 + blockIdx.y, head = blockIdx.x, tid = threadIdx.x;
    const int seg = segment_of_slot(p.seg_start, p.segments, slot);
    const int t0 = p.seg_start[seg] + (slot - p.seg_start[seg] / CHUNK - seg) * CHUNK, t1 = p.seg_start[seg + 1];
    if (t0 >= t1 || t0 < p.seg_start[seg]) return;
    const int n = min(CHUNK, t1 - t0), R = p.R, C = p.C, Rp = p.Rp, RS = Rp + 4;
    float* sk = lds;
    float* sq = sk + CHUNK * RS;
    float* sg = sq + CHUNK * RS;
    const float* kh = p.k + (size_t)t0 * p.ldk + (size_t)(head / p.share) * R;
    const float* qh = p.q + (size_t)t0 * p.ldq + (size_t)(head / p.share) * R;
    const float* gh = p.g + (size_t)t0 * p.ldg + (size_t)head * R;
    for (int idx = tid; idx < CHUNK * Rp; idx += 256) {
        const int i = idx / Rp, r = idx % Rp, tt = min(i, n - 1), rr = min(r, R - 1);
        const bool in = r < R && i < n;
        const float k = kh[tt * p.ldk + rr], q = qh[tt * p.ldq + rr], g = gh[tt * p.ldg + rr];
        sk[i * RS + r] = in ? k : 0.f;
        sq[i * RS + r] = in ? q * p.q_scale : 0.f;
        sg[i * RS + r] = in ? g : 1.f;
    }
    if (tid < CHUNK) sBeta[tid] = tid < n ? 1.0f / (1.0f + expf(-p.b[(size_t)(t0 + tid) * p.ldb + head])) : 0.f;
    __syncthreads();
    float* work = p.work + ((size_t)blockIdx.y * p.heads + head) * chunk_floats(Rp, p.Cp);
    float* wP = work + 3 * CHUNK * Rp + CHUNK * p.Cp;
    // column i of A and P: sixteen neighbouring threads, each with every sixteenth run of four channels, carry k_i down the
    // rows behind i (times their decays) and meet
    {
        const int i = tid / 16, part = tid % 16;
        f32x4_t x[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) x[j] = 64 * j + 4 * part < Rp ? *(const f32x4_t*)(sk + i * RS + 64 * j + 4 * part) : (f32x4_t){0.f, 0.f, 0.f, 0.f};
        for (int t = 0; t < CHUNK; ++t) {
            float a = 0.f, b = 0.f;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int r = 64 * j + 4 * part;
                if (64 * j >= Rp) break;                           // (uniform)
                if (r >= Rp || t < i) continue;
                const f32x4_t k = *(const f32x4_t*)(sk + t * RS + r), q = *(const f32x4_t*)(sq + t * RS + r);
                if (t > i) x[j] *= *(const f32x4_t*)(sg + t * RS + r);
                a += (x[j][0] * k[0] + x[j][1] * k[1]) + (x[j][2] * k[2] + x[j][3] * k[3]);
                b += (x[j][0] * q[0] + x[j][1] * q[1]) + (x[j][2] * q[2] + x[j][3] * q[3]);
            }
            a = row_sum(a);
            b = row_sum(b);
            if (part == t) {
                sA[t][i] = sBeta[t] * a;                           // (only i < t is read)
                wP[t * CHUNK + i] = b;                             // (0 for i > t)
            }
        }
    }
    __syncthreads();
    // column j of the inverse of the unit triangle I + A by forward substitution, times beta_j
    if (tid < CHUNK) {
        float x[CHUNK];
#pragma unroll
        for (int t = 0; t < CHUNK; ++t) {
            float s = t == tid ? 1.f : 0.f;
#pragma unroll
            for (int i = 0; i < t; ++i) s -= sA[t][i] * x[i];
            x[t] = s;
            __builtin_amdgcn_sched_barrier(0);                     // (the rows' operands are not asked for all at once: registers)
        }
#pragma unroll
        for (int t = 0; t < CHUNK; ++t) sM[t][tid] = x[t] * sBeta[tid];
    }
    __syncthreads();
    // a thread a channel (M Kg and the other operands over the state's rows) or a column of v (M V)
    for (int idx = tid; idx < Rp + p.Cp; idx += 256) {
        const bool key = idx < Rp;
        const int c = key ? idx : idx - Rp;
        float x[CHUNK];
        if (key) {
            float* wq = work + CHUNK * Rp + c;
            float* wk = work + 2 * CHUNK * Rp + (size_t)c * CHUNK;
            float d = 1.f, kd[CHUNK];
#pragma unroll
            for (int i = 0; i < CHUNK; ++i) {
                d *= sg[i * RS + c];
                x[i] = sk[i * RS + c] * d;
                wq[(size_t)i * Rp] = sq[i * RS + c] * d;
            }
            work[3 * CHUNK * Rp + CHUNK * p.Cp + CHUNK * CHUNK + c] = d;
            d = 1.f;
#pragma unroll
            for (int i = CHUNK - 1; i >= 0; --i) {
                kd[i] = sk[i * RS + c] * d;
                d *= sg[i * RS + c];
            }
#pragma unroll
            for (int i = 0; i < CHUNK; i += 4) *(f32x4_t*)(wk + i) = (f32x4_t){kd[i], kd[i + 1], kd[i + 2], kd[i + 3]};
        } else {
#pragma unroll
            for (int i = 0; i < CHUNK; ++i) x[i] = i < n && c < C ? p.v[(size_t)(t0 + min(i, n - 1)) * p.ldv + (size_t)head * C + min(c, C - 1)] : 0.f;
        }
        float y[CHUNK];
#pragma unroll
        for (int t = 0; t < CHUNK; ++t) {
            float s = 0.f;
#pragma unroll
            for (int i = 0; i <= t; ++i) s += sM[t][i] * x[i];
            y[t] = s;
            __builtin_amdgcn_sched_barrier(0);
        }
        if (key) {
#pragma unroll
            for (int t = 0; t < CHUNK; ++t) work[(size_t)t * Rp + c] = y[t];
        } else {
            float* wv = work + 3 * CHUNK * Rp + (size_t)c * CHUNK;
#pragma unroll
            for (int t = 0; t < CHUNK; t += 4) *(f32x4_t*)(wv + t) = (f32x4_t){y[t], y[t + 1], y[t + 2], y[t + 3]};
        }
    }
}

// A block a (head, segment, 16 columns), five waves.  The state's rows in tiles of 16: wave w < 4 owns the tiles w NT ..
// w NT + NT - 1, in the matrix instruction's result layout (lane l: rows 4 (l / 16) + i of the tile, column l % 16), which
// serves as its right operand as it is when the left operand's inner index runs alike: every operand is a 16-byte load.
// A chunk is M Kg S0 (each wave its rows' share), the meeting of the four shares through LDS, (D q) S0 while they travel,
// and the new S; the fifth wave adds the shares of (D q) S0 and P U, one chunk behind, and writes the results.
// AHEAD chunks' operands are in flight (an even number).  The loads of a chunk are kept together in program order: they
// return in order, so a chunk's wait then leaves those of the chunks behind it in flight.
template <int NT, int AHEAD>
__global__ void __launch_bounds__(320) __attribute__((amdgpu_waves_per_eu(2, 2))) channel_walk_kernel(ChunkArgs p) {
    __shared__ f32x4_t share_w[2][4][WAVE], share_o[2][4][WAVE];         // [chunk parity][wave][lane]
    const int head = blockIdx.x, seg = blockIdx.z, wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
    const int t0 = p.seg_start[seg], t1 = p.seg_start[seg + 1];
    if (t1 <= t0) return;
    const int base = t0 / CHUNK + seg, chunks = (t1 - t0 + CHUNK - 1) / CHUNK;
    const int first = max(base, p.slot0), last = min(base + chunks, p.slot0 + p.slots);
    if (first >= last) return;
    const int m = lane % 16, kg = lane / 16, R = p.R, C = p.C, Rp = p.Rp;
    const int c = blockIdx.y * 16 + m;
    const size_t per = (size_t)chunk_floats(Rp, p.Cp);
    auto operands = [&](int slot) { return (const char*)(p.work + ((size_t)(min(slot, last - 1) - p.slot0) * p.heads + head) * per); };
    // byte offsets of this lane's words from a chunk's operands (a uniform address): 32 bits
    const unsigned at_u = (3u * CHUNK * Rp + c * CHUNK + 4 * kg) * 4u;
    auto writes = [&](f32x4_t u, int par) {          // the rows' writes: M V - M Kg S0
        return u - ((share_w[par][0][lane] + share_w[par][1][lane]) + (share_w[par][2][lane] + share_w[par][3][lane]));
    };
    if (wave == 4) {
        const unsigned at_p = (3u * CHUNK * Rp + CHUNK * p.Cp + m * CHUNK + 4 * kg) * 4u;
        struct Result { f32x4_t u, pr; } ring[AHEAD];
        auto fetch = [&](Result& r, int slot) {
            const char* w = operands(slot);
            r.u = *(const f32x4_t*)(w + at_u);
            r.pr = *(const f32x4_t*)(w + at_p);
        };
#pragma unroll
        for (int d = 0; d < AHEAD; ++d) fetch(ring[d], first + d);
        f32x4_t u = {0.f, 0.f, 0.f, 0.f}, pr = u;
        auto finish = [&](int slot, int par) {       // o of the chunk before, whose shares are there now
            f32x4_t y = (share_o[par][0][lane] + share_o[par][1][lane]) + (share_o[par][2][lane] + share_o[par][3][lane]);
#pragma unroll
            for (int i = 0; i < 4; ++i) y = __builtin_amdgcn_mfma_f32_16x16x4f32(pr[i], u[i], y, 0, 0, 0);
            const int row = t0 + (slot - base) * CHUNK + 4 * kg;
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (row + i < t1 && c < C) p.out[(size_t)(row + i) * p.ldo + (size_t)head * C + c] = y[i];
        };
        for (int turn = first; turn < last; turn += AHEAD)
#pragma unroll
            for (int d = 0; d < AHEAD; ++d) {
                if (turn + d < last) {
                    __syncthreads();
                    if (turn + d > first) finish(turn + d - 1, (d + 1) & 1);
                    u = writes(ring[d].u, d & 1);
                    pr = ring[d].pr;
                }
                fetch(ring[d], turn + d + AHEAD);
            }
        __syncthreads();
        finish(last - 1, (last - 1 - first) & 1);
        return;
    }
    float* state = p.state + (long long)p.state_slots[seg] * p.slot_stride + (size_t)head * R * C;
    f32x4_t S[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = (wave * NT + j) * 16 + 4 * kg + i;
            S[j][i] = r < R && c < C ? state[(size_t)r * C + c] : 0.f;
        }
    struct Operands { f32x4_t kg[NT], qg[NT], kd[NT], g[NT], u; } ring[AHEAD];
    unsigned at_k[NT], at_d[NT], at_g[NT];
    float mine[NT];
    const unsigned q_words = CHUNK * Rp * 4u;
#pragma unroll
    for (int j = 0; j < NT; ++j) {
        const unsigned r = min((wave * NT + j) * 16, Rp - 16);          // (a wave without this tile reads another: its S stays zero)
        mine[j] = (wave * NT + j) * 16 < Rp ? 1.f : 0.f;
        at_k[j] = (m * Rp + r + 4 * kg) * 4u;
        at_d[j] = (2u * CHUNK * Rp + (r + m) * CHUNK + 4 * kg) * 4u;
        at_g[j] = (3u * CHUNK * Rp + CHUNK * p.Cp + CHUNK * CHUNK + r + 4 * kg) * 4u;
    }
    auto fetch = [&](Operands& o, int slot) {
        const char* w = operands(slot);
#pragma unroll
        for (int j = 0; j < NT; ++j) o.kg[j] = *(const f32x4_t*)(w + at_k[j]);
#pragma unroll
        for (int j = 0; j < NT; ++j) o.qg[j] = *(const f32x4_t*)(w + q_words + at_k[j]);
        o.u = *(const f32x4_t*)(w + at_u);
#pragma unroll
        for (int j = 0; j < NT; ++j) {
            o.g[j] = *(const f32x4_t*)(w + at_g[j]);
            o.kd[j] = *(const f32x4_t*)(w + at_d[j]);
        }
    };
    auto walk = [&](Operands& now, int par) {
        f32x4_t w = {0.f, 0.f, 0.f, 0.f}, o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) w = __builtin_amdgcn_mfma_f32_16x16x4f32(now.kg[j][i], S[j][i], w, 0, 0, 0);
        share_w[par][wave][lane] = w;
        __syncthreads();           // (the other parity's shares were read before the barrier before this one's writes)
        const f32x4_t u = writes(now.u, par);
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
            for (int i = 0; i < 4; ++i) o = __builtin_amdgcn_mfma_f32_16x16x4f32(now.qg[j][i], S[j][i], o, 0, 0, 0);
        share_o[par][wave][lane] = o;
#pragma unroll
        for (int j = 0; j < NT; ++j) S[j] *= now.g[j];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int j = 0; j < NT; ++j) S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(now.kd[j][i] * mine[j], u[i], S[j], 0, 0, 0);
    };
#pragma unroll
    for (int d = 0; d < AHEAD; ++d) {
        fetch(ring[d], first + d);
        __builtin_amdgcn_sched_barrier(0);
    }
    // (a turn past the last chunk loads a chunk again and does nothing: no way out of the unrolled loop, so that the waits of
    // every turn stay exact)
    for (int turn = first; turn < last; turn += AHEAD)
#pragma unroll
        for (int d = 0; d < AHEAD; ++d) {
            if (turn + d < last) walk(ring[d], d & 1);          // (uniform over the block)
            __builtin_amdgcn_sched_barrier(0);
            fetch(ring[d], turn + d + AHEAD);
            __builtin_amdgcn_sched_barrier(0);
        }
    __syncthreads();               // (the last chunk's shares of (D q) S0 are there)
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = (wave * NT + j) * 16 + 4 * kg + i;
            if (r < R && c < C) state[(size_t)r * C + c] = S[j][i];
        }
}

// Chunk slots of a step, and floats of `work` a slot takes.
extern "C" int cisr_channel_chunk_slots(int rows, int segments) { return rows / CHUNK + segments; }
extern "C" long long cisr_channel_chunk_floats(int heads, int R, int C) {
    return (long long)heads * chunk_floats((R + 15) / 16 * 16, (C + 15) / 16 * 16);
}

// The step's rows in launches of `slab` chunk slots each (two kernels a slab); work: slab * cisr_channel_chunk_floats floats.
extern "C" int cisr_channel_chunks(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* g, int ldg,
                                   const float* b, int ldb, float* out, int ldo, float* state, long long slot_stride,
                                   const int* seg_start, const int* state_slots, int rows, int segments, int heads, int R, int C,
                                   int share, float q_scale, float* work, int slab, hipStream_t stream) {
    if (rows <= 0 || segments <= 0 || heads <= 0) return 0;
    if (R <= 0 || R > 256 || C <= 0 || share <= 0 || heads % share || segments > 65535 || (C + 15) / 16 > 65535 || slab <= 0 || slab > 65535 ||
        (uintptr_t)work % 16)
        return (int)hipErrorInvalidValue;
    ChunkArgs p{q, ldq, k, ldk, v, ldv, g, ldg, b, ldb, out, ldo, state, slot_stride, seg_start, state_slots, R, C, share, heads, segments,
                q_scale, (R + 15) / 16 * 16, (C + 15) / 16 * 16, 0, 0, work};
    const int total = rows / CHUNK + segments, nt = (p.Rp / 16 + 3) / 4;
    const size_t lds = (size_t)3 * CHUNK * (p.Rp + 4) * sizeof(float);
    for (p.slot0 = 0; p.slot0 < total; p.slot0 += slab) {
        p.slots = min(slab, total - p.slot0);
        channel_chunk_kernel<<<dim3(heads, p.slots), 256, lds, stream>>>(p);
        int err = CISR_LAUNCH_CHECK();
        if (err) return err;
        const dim3 grid(heads, p.Cp / 16, segments);
        if (nt == 1) channel_walk_kernel<1, 4><<<grid, 320, 0, stream>>>(p);
        else if (nt == 2) channel_walk_kernel<2, 4><<<grid, 320, 0, stream>>>(p);
        else if (nt == 3) channel_walk_kernel<3, 2><<<grid, 320, 0, stream>>>(p);
        else channel_walk_kernel<4, 2><<<grid, 320, 0, stream>>>(p);
        err = CISR_LAUNCH_CHECK();
        if (err) return err;
    }
    return 0;
}
